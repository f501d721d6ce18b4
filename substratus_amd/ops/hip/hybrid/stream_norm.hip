// Norms of a 32-bit residual stream, fused with what surrounds them.
//
//   stream_norm   x += mult * rms(delta) * (off + w_post)
//                 y  = rms(x) * (off + w_pre)
//   embed_norm    x  = scale * table[token] + pos[position]
//                 y  = rms(x) * (off + w_pre)
//
// Without w_pre, y is x. delta is a row per token, or the weighted sum of
// `picks` rows of a pool (what a mixture of experts adds), formed on the way.
//
// with rms(z) = z / sqrt(mean(z^2) + eps). A block that norms both before and
// after its sublayer needs exactly one of these between two matrix products:
// the row of delta and the row of x are read once and stay in registers for
// both reductions. `off` is 1 for weights stored around zero, else 0;
// out_scale multiplies y (a logit scale folds in here, in 32 bits).
#include "typed.h"

enum Source { EMBED, ROW, PICKED };

template <class T, int VEC, int BLOCK, Source SRC>
__global__ __launch_bounds__(BLOCK)
void stream_norm_kernel(T* __restrict__ y, float* __restrict__ x,
                        const T* __restrict__ delta,     // [rows, width]
                        const int* __restrict__ at,      // [rows, picks]
                        const float* __restrict__ wt,    // [rows, picks]
                        int picks,
                        const T* __restrict__ table,     // [vocab, width]
                        const int* __restrict__ tokens,  // [rows]
                        const T* __restrict__ pos, // [max_pos, width] or null
                        const int* __restrict__ positions,   // [rows]
                        int max_pos,
                        const float* __restrict__ w_post,
                        const float* __restrict__ w_pre, int width, int vocab,
                        float off, float eps, float out_scale,
                        float mult) {
  constexpr int RCAP = 8;   // vectors per thread; the launcher checks the row
  __shared__ float scratch[2][BLOCK / WAVE];
  const long row = blockIdx.x;
  const int nvec = width / VEC;
  float* xr = x + row * width;
  float xk[RCAP][VEC];
  const float inv_n = 1.f / (float)width;

  if constexpr (SRC == EMBED) {
    const int tok = min(max(tokens[row], 0), vocab - 1);
    const T* src = table + (long)tok * width;
    #pragma unroll
    for (int kk = 0; kk < RCAP; ++kk) {
      const int i = threadIdx.x + kk * BLOCK;
      if (i >= nvec) break;
      ldv<VEC>(src + i * VEC, xk[kk]);
      #pragma unroll
      for (int j = 0; j < VEC; ++j) xk[kk][j] *= mult;
      if (pos != nullptr) {
        const int p = min(max(positions[row], 0), max_pos - 1);
        float f[VEC];
        ldv<VEC>(pos + (long)p * width + i * VEC, f);
        #pragma unroll
        for (int j = 0; j < VEC; ++j) xk[kk][j] += f[j];
      }
    }
  } else {
    float dk[RCAP][VEC];
    if constexpr (SRC == PICKED) {
      constexpr int P = 4;                       // rows on their way at once
      #pragma unroll
      for (int kk = 0; kk < RCAP; ++kk)
        #pragma unroll
        for (int j = 0; j < VEC; ++j) dk[kk][j] = 0.f;
      for (int p = 0; p < picks; p += P) {
        const T* src[P];
        float w[P];
        #pragma unroll
        for (int q = 0; q < P; ++q) {
          const long i = row * picks + min(p + q, picks - 1);
          src[q] = delta + (long)at[i] * width;
          w[q] = p + q < picks ? wt[i] : 0.f;
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
            for (int j = 0; j < VEC; ++j) dk[kk][j] += w[q] * f[q][j];
        }
      }
    }
    float ss = 0.f;
    #pragma unroll
    for (int kk = 0; kk < RCAP; ++kk) {
      const int i = threadIdx.x + kk * BLOCK;
      if (i >= nvec) break;
      if constexpr (SRC == ROW)
        ldv<VEC>(delta + row * width + i * VEC, dk[kk]);
      ldv<VEC>(xr + i * VEC, xk[kk]);
      #pragma unroll
      for (int j = 0; j < VEC; ++j) ss += dk[kk][j] * dk[kk][j];
    }
    ss = block_sum<BLOCK / WAVE>(ss, scratch[0]);
    const float inv = mult / sqrtf(ss * inv_n + eps);
    #pragma unroll
    for (int kk = 0; kk < RCAP; ++kk) {
      const int i = threadIdx.x + kk * BLOCK;
      if (i >= nvec) break;
      float w[VEC];
      ldv<VEC>(w_post + i * VEC, w);
      #pragma unroll
      for (int j = 0; j < VEC; ++j)
        xk[kk][j] += dk[kk][j] * inv * (off + w[j]);
    }
  }

  T* yr = y + row * width;
  float ss = 0.f;
  #pragma unroll
  for (int kk = 0; kk < RCAP; ++kk) {
    const int i = threadIdx.x + kk * BLOCK;
    if (i >= nvec) break;
    stv<VEC>(xr + i * VEC, xk[kk]);
    if (w_pre == nullptr) stv<VEC>(yr + i * VEC, xk[kk]);
    #pragma unroll
    for (int j = 0; j < VEC; ++j) ss += xk[kk][j] * xk[kk][j];
  }
  if (w_pre == nullptr) return;
  ss = block_sum<BLOCK / WAVE>(ss, scratch[1]);
  const float inv = out_scale / sqrtf(ss * inv_n + eps);
  #pragma unroll
  for (int kk = 0; kk < RCAP; ++kk) {
    const int i = threadIdx.x + kk * BLOCK;
    if (i >= nvec) break;
    float w[VEC], o[VEC];
    ldv<VEC>(w_pre + i * VEC, w);
    #pragma unroll
    for (int j = 0; j < VEC; ++j) o[j] = xk[kk][j] * inv * (off + w[j]);
    stv<VEC>(yr + i * VEC, o);
  }
}

int stream_norm_max_width(int width) {
  return 1024 * 8 * (width % 4 == 0 ? 4 : 1);
}

template <class T, Source SRC>
static void launch(T* y, float* x, const T* delta, const int* at,
                   const float* wt, int picks, const T* table,
                   const int* tokens, const T* pos, const int* positions,
                   int max_pos, const float* w_post, const float* w_pre,
                   long rows, int width, int vocab, float off, float eps,
                   float out_scale, float mult, hipStream_t stream) {
  auto go = [&](auto vec, auto block) {
    constexpr int V = decltype(vec)::value, B = decltype(block)::value;
    stream_norm_kernel<T, V, B, SRC><<<dim3(rows), dim3(B), 0, stream>>>(
        y, x, delta, at, wt, picks, table, tokens, pos, positions, max_pos,
        w_post, w_pre, width, vocab, off, eps, out_scale, mult);
  };
  using std::integral_constant;
  auto by_block = [&](auto vec) {
    const int nvec = width / decltype(vec)::value;
    if (nvec <= 128) go(vec, integral_constant<int, 64>{});
    else if (nvec <= 256 * 8) go(vec, integral_constant<int, 256>{});
    else go(vec, integral_constant<int, 1024>{});
  };
  if (width % 4 == 0) by_block(integral_constant<int, 4>{});
  else by_block(integral_constant<int, 1>{});
}

// at, wt null: delta is [rows, width]
template <class T>
void launch_stream_norm(T* y, float* x, const T* delta, const int* at,
                        const float* wt, int picks, const float* w_post,
                        const float* w_pre, long rows, int width, float off,
                        float eps, float out_scale, float mult,
                        hipStream_t stream) {
  if (at == nullptr)
    launch<T, ROW>(y, x, delta, at, wt, picks, nullptr, nullptr, nullptr,
                   nullptr, 0, w_post, w_pre, rows, width, 0, off, eps,
                   out_scale, mult, stream);
  else
    launch<T, PICKED>(y, x, delta, at, wt, picks, nullptr, nullptr, nullptr,
                      nullptr, 0, w_post, w_pre, rows, width, 0, off, eps,
                      out_scale, mult, stream);
}

template <class T>
void launch_embed_norm(T* y, float* x, const T* table, const int* tokens,
                       float scale, const T* pos, const int* positions,
                       int max_pos, const float* w_pre, long rows, int width,
                       int vocab, float off, float eps, hipStream_t stream) {
  launch<T, EMBED>(y, x, nullptr, nullptr, nullptr, 0, table, tokens, pos,
                   positions, max_pos, nullptr, w_pre, rows, width, vocab, off,
                   eps, 1.f, scale, stream);
}

#define INSTANTIATE(T)                                                        \
  template void launch_stream_norm<T>(T*, float*, const T*, const int*,       \
      const float*, int, const float*, const float*, long, int, float, float, \
      float, float, hipStream_t);                                             \
  template void launch_embed_norm<T>(T*, float*, const T*, const int*, float, \
      const T*, const int*, int, const float*, long, int, int, float, float,  \
      hipStream_t);
INSTANTIATE(float)
INSTANTIATE(bf16_t)
