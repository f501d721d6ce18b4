// Fused activation kernels: SwiGLU (silu(gate)*up) and tanh-GELU.
// Pure HBM-streaming ops; bf16×8 vector loads/stores, fp32 math.
#include "common.h"
#include <algorithm>

// x: [rows, 2F] laid out (gate ‖ up); out: [rows, F].
// 2-D grid (rows × column-chunks): a batch-256 decode row is 43 iterations
// for one 256-thread workgroup — 256 WGs can't fill 256 CUs with latency
// hidden (profiles: 83 us/call at B=256); chunking columns restores
// parallelism.
template <int BLOCK>
__global__ void silu_mul_kernel(bf16_t* __restrict__ out,
                                const bf16_t* __restrict__ x, long rows,
                                int f) {
  const long row = blockIdx.x;
  const uint4* gv = reinterpret_cast<const uint4*>(x + row * 2L * f);
  const uint4* uv = reinterpret_cast<const uint4*>(x + row * 2L * f + f);
  uint4* ov = reinterpret_cast<uint4*>(out + row * (long)f);
  const int nvec = f / 8;
  for (int i = blockIdx.y * BLOCK + threadIdx.x; i < nvec;
       i += gridDim.y * BLOCK) {
    uint4 g = gv[i], u = uv[i];
    float2 gf[4] = {unpack_bf16x2(g.x), unpack_bf16x2(g.y),
                    unpack_bf16x2(g.z), unpack_bf16x2(g.w)};
    float2 uf[4] = {unpack_bf16x2(u.x), unpack_bf16x2(u.y),
                    unpack_bf16x2(u.z), unpack_bf16x2(u.w)};
    unsigned int o[4];
    #pragma unroll
    for (int j = 0; j < 4; ++j) {
      float a = gf[j].x, b = gf[j].y;
      float sa = a / (1.f + __expf(-a));
      float sb = b / (1.f + __expf(-b));
      o[j] = pack_bf16x2(sa * uf[j].x, sb * uf[j].y);
    }
    ov[i] = make_uint4(o[0], o[1], o[2], o[3]);
  }
}

DEV_INLINE float gelu_tanh_f(float v) {
  const float c = 0.7978845608028654f;  // sqrt(2/pi)
  float inner = c * (v + 0.044715f * v * v * v);
  return 0.5f * v * (1.f + tanhf(inner));
}

template <int BLOCK>
__global__ void gelu_kernel(bf16_t* __restrict__ out,
                            const bf16_t* __restrict__ x, long n8) {
  const uint4* xv = reinterpret_cast<const uint4*>(x);
  uint4* ov = reinterpret_cast<uint4*>(out);
  for (long i = blockIdx.x * BLOCK + threadIdx.x; i < n8;
       i += (long)gridDim.x * BLOCK) {
    uint4 u = xv[i];
    float2 f[4] = {unpack_bf16x2(u.x), unpack_bf16x2(u.y),
                   unpack_bf16x2(u.z), unpack_bf16x2(u.w)};
    unsigned int o[4];
    #pragma unroll
    for (int j = 0; j < 4; ++j)
      o[j] = pack_bf16x2(gelu_tanh_f(f[j].x), gelu_tanh_f(f[j].y));
    ov[i] = make_uint4(o[0], o[1], o[2], o[3]);
  }
}

void launch_silu_mul(bf16_t* out, const bf16_t* x, long rows, int f,
                     hipStream_t stream) {
  constexpr int BLOCK = 256;
  // >=2048 workgroups to fill 8 XCDs (guide: a launch needs >>256 WGs)
  int chunks = 1;
  while (rows * chunks < 2048 && chunks * BLOCK * 8 < f) chunks *= 2;
  silu_mul_kernel<BLOCK><<<dim3(rows, chunks), dim3(BLOCK), 0, stream>>>(
      out, x, rows, f);
}

// Any width, float or bf16: the 32-bit path, and widths the vector kernel
// does not take.
template <class T, int BLOCK>
__global__ void silu_mul_any_kernel(T* __restrict__ out,
                                    const T* __restrict__ x, int f) {
  const long row = blockIdx.x;
  for (int i = blockIdx.y * BLOCK + threadIdx.x; i < f;
       i += gridDim.y * BLOCK) {
    const float g = (float)x[row * 2L * f + i];
    const float u = (float)x[row * 2L * f + f + i];
    out[row * (long)f + i] = (T)(g / (1.f + expf(-g)) * u);
  }
}

void launch_silu_mul_any(float* out, const float* x, long rows, int f,
                         hipStream_t stream) {
  silu_mul_any_kernel<float, 256><<<dim3(rows, 4), dim3(256), 0, stream>>>(
      out, x, f);
}

void launch_silu_mul_any(bf16_t* out, const bf16_t* x, long rows, int f,
                         hipStream_t stream) {
  silu_mul_any_kernel<bf16_t, 256><<<dim3(rows, 4), dim3(256), 0, stream>>>(
      out, x, f);
}

void launch_gelu(bf16_t* out, const bf16_t* x, long n, hipStream_t stream) {
  constexpr int BLOCK = 256;
  long n8 = n / 8;
  int grid = (int)std::min((n8 + BLOCK - 1) / BLOCK, (long)4096);
  gelu_kernel<BLOCK><<<dim3(grid), dim3(BLOCK), 0, stream>>>(out, x, n8);
}
