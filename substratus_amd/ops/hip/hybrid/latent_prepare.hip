// Everything between a latent-attention layer's input projection and its
// scores, in one pass over the projected row of each token:
//   * the rotated part of every query head, in place, or the RMS-normed
//     latent that queries are made of, in place,
//   * the RMS-normed latent and the rotated key part, to the paged cache
//     (layers that use another one's latents have neither).
// Row layout: [queries, head by head: dim | rot_dim][...][latent | key part],
// or [queries' latent][...][latent | key part].
//
// Element i of a rotated part turns with element i + half. Angles are formed
// as turns in 64 bits, whole turns dropped, so that positions far away are as
// exact as near ones.
#include "attention_ctx.h"

namespace {

constexpr int BLOCK = 256;

template <class T>
__global__ __launch_bounds__(BLOCK)
void latent_prepare_kernel(T* __restrict__ buf, long ld, int heads, int dim,
                           int rot_dim, int c_at, int rank,
                           const float* __restrict__ norm, float eps,
                           const double* __restrict__ turns, int half,
                           const int* __restrict__ positions,
                           T* __restrict__ cache, const int* __restrict__ slots,
                           const float* __restrict__ q_norm, int q_rank) {
  extern __shared__ float s_cs[];               // cos, sin of every pair
  __shared__ float scratch[2][BLOCK / WAVE];
  const long row = blockIdx.x;
  T* q = buf + row * ld;
  const double pos = positions[row];
  for (int i = threadIdx.x; i < half; i += BLOCK) {
    double t = pos * turns[i];
    t -= rint(t);
    float s, c;
    sincospif((float)(2.0 * t), &s, &c);
    s_cs[2 * i] = c;
    s_cs[2 * i + 1] = s;
  }
  __syncthreads();
  for (int i = threadIdx.x; i < heads * half; i += BLOCK) {
    const int h = i / half, j = i % half;
    T* p = q + (long)h * (dim + rot_dim) + dim + j;
    const float u = ld1(p), v = ld1(p + half);
    const float c = s_cs[2 * j], s = s_cs[2 * j + 1];
    st1(p, u * c - v * s);
    st1(p + half, v * c + u * s);
  }
  if (q_norm != nullptr) {
    float ss = 0.f;
    for (int i = threadIdx.x; i < q_rank; i += BLOCK) {
      const float f = ld1(q + i);
      ss += f * f;
    }
    ss = block_sum<BLOCK / WAVE>(ss, scratch[1]);
    const float inv = 1.f / sqrtf(ss / (float)q_rank + eps);
    for (int i = threadIdx.x; i < q_rank; i += BLOCK)
      st1(q + i, ld1(q + i) * inv * q_norm[i]);
  }
  if (c_at < 0) return;
  const T* lat = q + c_at;
  float ss = 0.f;
  for (int i = threadIdx.x; i < rank; i += BLOCK) {
    const float f = ld1(lat + i);
    ss += f * f;
  }
  ss = block_sum<BLOCK / WAVE>(ss, scratch[0]);
  const float inv = 1.f / sqrtf(ss / (float)rank + eps);
  T* out = cache + (long)slots[row] * (rank + rot_dim);
  for (int i = threadIdx.x; i < rank; i += BLOCK)
    st1(out + i, ld1(lat + i) * inv * norm[i]);
  for (int j = threadIdx.x; j < rot_dim; j += BLOCK) {
    const float x = ld1(lat + rank + j);
    float y = x;
    if (j < half)
      y = x * s_cs[2 * j] - ld1(lat + rank + j + half) * s_cs[2 * j + 1];
    else if (j < 2 * half)
      y = x * s_cs[2 * (j - half)] +
          ld1(lat + rank + j - half) * s_cs[2 * (j - half) + 1];
    st1(out + rank + j, y);
  }
}

// Rows of contexts out of the pages, from the first key that an entry's rows
// see on: latents to c, key parts to kr. Sizes are in pieces of type P.
template <class P>
__global__ __launch_bounds__(BLOCK)
void latent_gather_kernel(P* __restrict__ c, P* __restrict__ kr,
                          const P* __restrict__ cache, int rank, int rot,
                          const int* __restrict__ block_table, int max_blocks,
                          const int* __restrict__ ctx_start,
                          const int* __restrict__ positions,
                          const int* __restrict__ seq_start, int window,
                          int block_size) {
  const int e = blockIdx.y;
  const int at = ctx_start[e], n = ctx_start[e + 1] - at;
  const int from = flat_from(window, positions[seq_start[e]]);
  const int page = from / block_size + blockIdx.x;
  // keys of the page that are asked for
  const int k0 = max(from, page * block_size);
  const int k1 = min(from + n, (page + 1) * block_size);
  if (k1 <= k0) return;
  const int row = rank + rot;
  const P* src = cache + ((long)block_table[(long)e * max_blocks + page] *
                          block_size + k0 % block_size) * row;
  for (int i = threadIdx.x; i < (k1 - k0) * row; i += BLOCK) {
    const long r = at + (long)(k0 - from) + i / row;
    const int d = i % row;
    if (d < rank) c[r * rank + d] = src[i];
    else kr[r * rot + d - rank] = src[i];
  }
}

}  // namespace

void launch_latent_gather(void* c, void* kr, const void* cache, int itemsize,
                          int rank, int rot, const int* block_table,
                          int max_blocks, const int* ctx_start,
                          const int* positions, const int* seq_start,
                          int window, int max_len, int entries, int block_size,
                          hipStream_t stream) {
  // pages that hold an entry's keys, the first and the last maybe in part
  const int pages = window <= 0 ? max_blocks
      : min(max_blocks, (window + max_len) / block_size + 2);
  auto go = [&](auto piece) {
    using P = decltype(piece);
    const int per = sizeof(P) / itemsize;
    latent_gather_kernel<P><<<dim3(pages, entries), BLOCK, 0, stream>>>(
        (P*)c, (P*)kr, (const P*)cache, rank / per, rot / per, block_table,
        max_blocks, ctx_start, positions, seq_start, window, block_size);
  };
  const int bytes = 16 / itemsize;
  if (rank % bytes == 0 && rot % bytes == 0) go(uint4{});
  else if (itemsize == 4) go(unsigned{});
  else go((unsigned short)0);
}

template <class T>
void launch_latent_prepare(T* buf, long ld, int heads, int dim, int rot_dim,
                           int c_at, int rank, const float* norm, float eps,
                           const double* turns, int half, const int* positions,
                           T* cache, const int* slots, const float* q_norm,
                           int q_rank, long rows, hipStream_t stream) {
  latent_prepare_kernel<T><<<dim3(rows), dim3(BLOCK),
                             2 * half * sizeof(float), stream>>>(
      buf, ld, heads, dim, rot_dim, c_at, rank, norm, eps, turns, half,
      positions, cache, slots, q_norm, q_rank);
}

template void launch_latent_prepare<float>(float*, long, int, int, int, int,
    int, const float*, float, const double*, int, const int*, float*,
    const int*, const float*, int, long, hipStream_t);
template void launch_latent_prepare<bf16_t>(bf16_t*, long, int, int, int, int,
    int, const float*, float, const double*, int, const int*, bf16_t*,
    const int*, const float*, int, long, hipStream_t);
