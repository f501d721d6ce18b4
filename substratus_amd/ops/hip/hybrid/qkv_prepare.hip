// Everything between an attention layer's input projection and its scores,
// in one pass over the projected row of each token:
//   * RMS norm of the whole query projection (all heads at once), in place,
//   * RMS norm of the whole key projection, written to the paged K cache,
//   * values blended with an earlier layer's values of the same token,
//     v <- (1 - lam) v + lam v_first, written to the paged V cache.
// Norm and blend are optional (null weights / null v_first). Row layout:
// [q: nq | k: nk | v: nv | ...], rows `ld` elements apart, so the fused
// projection is consumed as it is. Caches: [blocks, kv_heads, block, d].
#include "typed.h"

#define PBLOCK 256

template <class T, int VEC>
__global__ __launch_bounds__(PBLOCK)
void qkv_prepare_kernel(T* __restrict__ buf, long ld, int nq, int nk, int nv,
                        const float* __restrict__ qw,
                        const float* __restrict__ kw, float eps,
                        const T* __restrict__ v_first, long vf_ld,
                        const float* __restrict__ lam,
                        T* __restrict__ kc, T* __restrict__ vc,
                        const int* __restrict__ slots, int kv_heads,
                        int block_size) {
  __shared__ float scratch[2][PBLOCK / WAVE];
  const long row = blockIdx.x;
  T* q = buf + row * ld;
  const T* k = q + nq;
  const T* v = k + nk;
  float sq = 0.f, sk = 0.f;
  if (qw != nullptr) {
    for (int i = threadIdx.x * VEC; i < nq + nk; i += PBLOCK * VEC) {
      float f[VEC];
      ldv<VEC>(q + i, f);
      float s = 0.f;
      #pragma unroll
      for (int j = 0; j < VEC; ++j) s += f[j] * f[j];
      if (i < nq) sq += s; else sk += s;
    }
    sq = block_sum<PBLOCK / WAVE>(sq, scratch[0]);
    sk = block_sum<PBLOCK / WAVE>(sk, scratch[1]);
    const float inv = 1.f / sqrtf(sq / (float)nq + eps);
    for (int i = threadIdx.x * VEC; i < nq; i += PBLOCK * VEC) {
      float f[VEC], w[VEC];
      ldv<VEC>(q + i, f);
      ldv<VEC>(qw + i, w);
      #pragma unroll
      for (int j = 0; j < VEC; ++j) f[j] *= inv * w[j];
      stv<VEC>(q + i, f);
    }
  }
  const int slot = slots[row];
  const long page = slot / block_size, at = slot % block_size;
  const int dim = nk / kv_heads, vdim = nv / kv_heads;
  const float kinv = qw != nullptr ? 1.f / sqrtf(sk / (float)nk + eps) : 1.f;
  for (int i = threadIdx.x * VEC; i < nk; i += PBLOCK * VEC) {
    float f[VEC];
    ldv<VEC>(k + i, f);
    if (qw != nullptr) {
      float w[VEC];
      ldv<VEC>(kw + i, w);
      #pragma unroll
      for (int j = 0; j < VEC; ++j) f[j] *= kinv * w[j];
    }
    const int h = i / dim;
    stv<VEC>(kc + ((page * kv_heads + h) * block_size + at) * dim + i % dim, f);
  }
  const float l = v_first != nullptr ? *lam : 0.f;
  for (int i = threadIdx.x * VEC; i < nv; i += PBLOCK * VEC) {
    float f[VEC];
    ldv<VEC>(v + i, f);
    if (v_first != nullptr) {
      float a[VEC];
      ldv<VEC>(v_first + row * vf_ld + i, a);
      #pragma unroll
      for (int j = 0; j < VEC; ++j) f[j] = (1.f - l) * f[j] + l * a[j];
    }
    const int h = i / vdim;
    stv<VEC>(vc + ((page * kv_heads + h) * block_size + at) * vdim + i % vdim,
             f);
  }
}

template <class T>
void launch_qkv_prepare(T* buf, long ld, int nq, int nk, int nv,
                        const float* qw, const float* kw, float eps,
                        const T* v_first, long vf_ld, const float* lam, T* kc,
                        T* vc, const int* slots, long rows, int kv_heads,
                        int block_size, hipStream_t stream) {
  const int dim = nk / kv_heads, vdim = nv / kv_heads;
  const bool vec = dim % 4 == 0 && vdim % 4 == 0 && nq % 4 == 0 &&
                   ld % 4 == 0 && vf_ld % 4 == 0;
  if (vec)
    qkv_prepare_kernel<T, 4><<<dim3(rows), dim3(PBLOCK), 0, stream>>>(
        buf, ld, nq, nk, nv, qw, kw, eps, v_first, vf_ld, lam, kc, vc, slots,
        kv_heads, block_size);
  else
    qkv_prepare_kernel<T, 1><<<dim3(rows), dim3(PBLOCK), 0, stream>>>(
        buf, ld, nq, nk, nv, qw, kw, eps, v_first, vf_ld, lam, kc, vc, slots,
        kv_heads, block_size);
}

template void launch_qkv_prepare<float>(float*, long, int, int, int,
    const float*, const float*, float, const float*, long, const float*,
    float*, float*, const int*, long, int, int, hipStream_t);
template void launch_qkv_prepare<bf16_t>(bf16_t*, long, int, int, int,
    const float*, const float*, float, const bf16_t*, long, const float*,
    bf16_t*, bf16_t*, const int*, long, int, int, hipStream_t);
