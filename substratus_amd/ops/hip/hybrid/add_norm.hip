// Row operations of layers that add to a 32-bit residual without norms of
// their own:
//
//   add_norm    x += rows + weighed picked rows + scale * table[token] + vec,
//               whatever of it is given, and y = norm(x): with b layer norm
//               (x - mean) / sqrt(var + eps) * w + b, else RMS norm
//   joint_gate  out = rms(o) over the whole row * w * sigmoid(gate)
//   glu         hidden values of a gated feed-forward from [gate | up]
//   softcap     x = cap * tanh(x / cap)
#include "add_norm.h"

namespace {

constexpr int RCAP = 8;       // vectors per thread; the launcher checks the row

template <class T, int VEC, int BLOCK>
__global__ __launch_bounds__(BLOCK)
void add_norm_kernel(AddNorm<T> a) {
  __shared__ float scratch[2][BLOCK / WAVE];
  const long row = blockIdx.x;
  const int nvec = a.width / VEC;
  float* xr = a.x + row * a.width;
  const T* emb = nullptr;
  if (a.table != nullptr)
    emb = a.table + (long)min(max(a.tokens[row], 0), a.vocab - 1) * a.width;
  float xk[RCAP][VEC];
  #pragma unroll
  for (int kk = 0; kk < RCAP; ++kk) {
    const int i = threadIdx.x + kk * BLOCK;
    if (i >= nvec) break;
    if (a.fresh) {
      #pragma unroll
      for (int j = 0; j < VEC; ++j) xk[kk][j] = 0.f;
    } else {
      ldv<VEC>(xr + i * VEC, xk[kk]);
    }
    float f[VEC];
    if (a.rows != nullptr) {
      ldv<VEC>(a.rows + row * a.width + i * VEC, f);
      #pragma unroll
      for (int j = 0; j < VEC; ++j) xk[kk][j] += f[j];
    }
    if (emb != nullptr) {
      ldv<VEC>(emb + i * VEC, f);
      #pragma unroll
      for (int j = 0; j < VEC; ++j) xk[kk][j] += f[j] * a.scale;
    }
    if (a.vec != nullptr) {
      ldv<VEC>(a.vec + i * VEC, f);
      #pragma unroll
      for (int j = 0; j < VEC; ++j) xk[kk][j] += f[j];
    }
  }
  if (a.pool != nullptr) {
    constexpr int P = 4;                         // rows on their way at once
    for (int p = 0; p < a.picks; p += P) {
      const T* src[P];
      float w[P];
      #pragma unroll
      for (int q = 0; q < P; ++q) {
        const long i = row * a.picks + min(p + q, a.picks - 1);
        src[q] = a.pool + (long)a.at[i] * a.width;
        w[q] = p + q < a.picks ? a.wt[i] : 0.f;
      }
      #pragma unroll
      for (int kk = 0; kk < RCAP; ++kk) {
        const int i = threadIdx.x + kk * BLOCK;
        if (i >= nvec) break;
        float f[P][VEC];
        #pragma unroll
        for (int q = 0; q < P; ++q) ldv<VEC>(src[q] + i * VEC, f[q]);
        #pragma unroll
        for (int q = 0; q < P; ++q)
          #pragma unroll
          for (int j = 0; j < VEC; ++j) xk[kk][j] += w[q] * f[q][j];
      }
    }
  }
  const float inv_n = 1.f / (float)a.width;
  float mean = 0.f;
  if (a.b != nullptr) {
    #pragma unroll
    for (int kk = 0; kk < RCAP; ++kk) {
      if (threadIdx.x + kk * BLOCK >= nvec) break;
      #pragma unroll
      for (int j = 0; j < VEC; ++j) mean += xk[kk][j];
    }
    mean = block_sum<BLOCK / WAVE>(mean, scratch[0]) * inv_n;
  }
  float ss = 0.f;
  #pragma unroll
  for (int kk = 0; kk < RCAP; ++kk) {
    const int i = threadIdx.x + kk * BLOCK;
    if (i >= nvec) break;
    stv<VEC>(xr + i * VEC, xk[kk]);
    #pragma unroll
    for (int j = 0; j < VEC; ++j) {
      xk[kk][j] -= mean;
      ss += xk[kk][j] * xk[kk][j];
    }
  }
  ss = block_sum<BLOCK / WAVE>(ss, scratch[1]);
  const float inv = 1.f / sqrtf(ss * inv_n + a.eps);
  T* yr = a.y + row * a.width;
  #pragma unroll
  for (int kk = 0; kk < RCAP; ++kk) {
    const int i = threadIdx.x + kk * BLOCK;
    if (i >= nvec) break;
    float w[VEC], o[VEC];
    ldv<VEC>(a.w + i * VEC, w);
    #pragma unroll
    for (int j = 0; j < VEC; ++j) o[j] = xk[kk][j] * inv * w[j];
    if (a.b != nullptr) {
      ldv<VEC>(a.b + i * VEC, w);
      #pragma unroll
      for (int j = 0; j < VEC; ++j) o[j] += w[j];
    }
    stv<VEC>(yr + i * VEC, o);
  }
}

constexpr int BLOCK = 256;

template <class T, int VEC>
__global__ __launch_bounds__(BLOCK)
void joint_gate_kernel(T* __restrict__ out, long out_ld,
                       const T* __restrict__ o, const float* __restrict__ w,
                       const T* __restrict__ gate, long g_ld, int n,
                       float eps) {
  __shared__ float scratch[BLOCK / WAVE];
  const long row = blockIdx.x;
  const T* r = o + row * n;
  float ss = 0.f;
  for (int i = threadIdx.x * VEC; i < n; i += BLOCK * VEC) {
    float f[VEC];
    ldv<VEC>(r + i, f);
    #pragma unroll
    for (int j = 0; j < VEC; ++j) ss += f[j] * f[j];
  }
  ss = block_sum<BLOCK / WAVE>(ss, scratch);
  const float inv = 1.f / sqrtf(ss / (float)n + eps);
  for (int i = threadIdx.x * VEC; i < n; i += BLOCK * VEC) {
    float f[VEC], g[VEC], v[VEC];
    ldv<VEC>(r + i, f);
    ldv<VEC>(gate + row * g_ld + i, g);
    ldv<VEC>(w + i, v);
    #pragma unroll
    for (int j = 0; j < VEC; ++j) f[j] *= inv * v[j] * sigmoid_f(g[j]);
    stv<VEC>(out + row * out_ld + i, f);
  }
}

template <class T, int VEC>
__global__ __launch_bounds__(BLOCK)
void glu_kernel(T* __restrict__ out, long out_ld, const T* __restrict__ x,
                long ld, int f, Glu kind, float limit) {
  const long row = blockIdx.x;
  const int i = (blockIdx.y * BLOCK + threadIdx.x) * VEC;
  if (i >= f) return;
  float g[VEC], u[VEC];
  ldv<VEC>(x + row * ld + i, g);
  ldv<VEC>(x + row * ld + f + i, u);
  #pragma unroll
  for (int j = 0; j < VEC; ++j) g[j] = glu_f(kind, g[j], u[j], limit);
  stv<VEC>(out + row * out_ld + i, g);
}

template <class T, int VEC>
__global__ __launch_bounds__(BLOCK)
void softcap_kernel(T* __restrict__ x, long n, float cap) {
  const long i = ((long)blockIdx.x * BLOCK + threadIdx.x) * VEC;
  if (i >= n) return;
  float f[VEC];
  ldv<VEC>(x + i, f);
  #pragma unroll
  for (int j = 0; j < VEC; ++j) f[j] = cap * tanhf(f[j] / cap);
  stv<VEC>(x + i, f);
}

template <class T>
bool fours(const T* p, long ld) {
  return ld % 4 == 0 && reinterpret_cast<uintptr_t>(p) % (4 * sizeof(T)) == 0;
}

}  // namespace

int add_norm_max_width(int width) {
  return 1024 * RCAP * (width % 4 == 0 ? 4 : 1);
}

template <class T>
void launch_add_norm(const AddNorm<T>& a, long n, hipStream_t stream) {
  auto go = [&](auto vec, auto block) {
    constexpr int V = decltype(vec)::value, B = decltype(block)::value;
    add_norm_kernel<T, V, B><<<dim3(n), dim3(B), 0, stream>>>(a);
  };
  using std::integral_constant;
  auto by_block = [&](auto vec) {
    const int nvec = a.width / decltype(vec)::value;
    if (nvec <= 128) go(vec, integral_constant<int, 64>{});
    else if (nvec <= 256 * RCAP) go(vec, integral_constant<int, 256>{});
    else go(vec, integral_constant<int, 1024>{});
  };
  if (a.width % 4 == 0) by_block(integral_constant<int, 4>{});
  else by_block(integral_constant<int, 1>{});
}

template <class T>
void launch_joint_gate(T* out, long out_ld, const T* o, const float* w,
                       const T* gate, long g_ld, long rows, int n, float eps,
                       hipStream_t stream) {
  if (n % 4 == 0 && fours(out, out_ld) && fours(gate, g_ld))
    joint_gate_kernel<T, 4><<<dim3(rows), BLOCK, 0, stream>>>(
        out, out_ld, o, w, gate, g_ld, n, eps);
  else
    joint_gate_kernel<T, 1><<<dim3(rows), BLOCK, 0, stream>>>(
        out, out_ld, o, w, gate, g_ld, n, eps);
}

template <class T>
void launch_glu(T* out, long out_ld, const T* x, long ld, long rows, int f,
                Glu kind, float limit, hipStream_t stream) {
  if (f % 4 == 0 && fours(out, out_ld) && fours(x, ld))
    glu_kernel<T, 4><<<dim3(rows, (f / 4 + BLOCK - 1) / BLOCK), BLOCK, 0,
                       stream>>>(out, out_ld, x, ld, f, kind, limit);
  else
    glu_kernel<T, 1><<<dim3(rows, (f + BLOCK - 1) / BLOCK), BLOCK, 0,
                       stream>>>(out, out_ld, x, ld, f, kind, limit);
}

template <class T>
void launch_softcap(T* x, long n, float cap, hipStream_t stream) {
  if (fours(x, n))
    softcap_kernel<T, 4><<<dim3((n / 4 + BLOCK - 1) / BLOCK), BLOCK, 0,
                           stream>>>(x, n, cap);
  else
    softcap_kernel<T, 1><<<dim3((n + BLOCK - 1) / BLOCK), BLOCK, 0, stream>>>(
        x, n, cap);
}

#define INSTANTIATE(T)                                                       \
  template void launch_add_norm<T>(const AddNorm<T>&, long, hipStream_t);    \
  template void launch_joint_gate<T>(T*, long, const T*, const float*,       \
      const T*, long, long, int, float, hipStream_t);                        \
  template void launch_glu<T>(T*, long, const T*, long, long, int, Glu,      \
                              float, hipStream_t);                           \
  template void launch_softcap<T>(T*, long, float, hipStream_t);
INSTANTIATE(float)
INSTANTIATE(bf16_t)
