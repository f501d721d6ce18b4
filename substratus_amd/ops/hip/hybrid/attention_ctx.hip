// Attention over a paged cache for any head sizes, in float or bf16, for
// single tokens and portions of prompts: one wave per (row, query head).
//
//   score(i, j) = f(scale * q_i . k_j) + bias[h][min(i - j, nbias - 1)]
//                 - r1[h] ln(1 + r2[h] (i - j))
//                 with f(s) = s, or cap * tanh(s / cap) when cap > 0
//   visible: j <= i, and i / chunk == j / chunk when chunk > 0,
//            and i - j < window or j < keep when window > 0
//   out_h = softmax(score) v * sigmoid(gate_h) * mult   (gate optional)
//
// With a sink, the softmax's denominator has e^(sink_h) besides the keys.
// Instead of a softmax, a key's weight may be sigmoid(score + wbias_h).
//
// Query head h reads key/value head h / (heads / kv_heads). 64 keys at a
// time: lane = key for the scores, lane = column for the values. This is the
// whole 32-bit path, and the bf16 path of head sizes that the tiled kernels
// (attention_ctx_decode.hip, attention_ctx_prefill.hip) do not take.
#include "attention_ctx.h"

// CMAX: value columns per lane
template <class T, int CMAX>
__global__ __launch_bounds__(WAVE)
void attn_ctx_any_kernel(AttnCtx<T> a) {
  extern __shared__ float s_q[];                 // [dim] + [WAVE] weights
  float* s_p = s_q + a.dim;
  const Entry e = entry_of(a.seq_start, blockIdx.z);
  if ((int)blockIdx.x >= e.n) return;
  const long row = e.row0 + blockIdx.x;
  const int h = blockIdx.y, lane = threadIdx.x;
  const int kvh = h / (a.heads / a.kv_heads);
  const int pos = a.positions[row];
  const int lo = first_seen(a, pos);
  const Pieces part(a.keep, lo, pos / WAVE + 1, WAVE);
  const int* bt = a.block_table + (long)blockIdx.z * a.max_blocks;

  const T* q = a.q + row * a.q_ld + (long)h * a.dim;
  for (int i = lane; i < a.dim; i += WAVE) s_q[i] = ld1(q + i) * a.scale;
  __syncthreads();

  float acc[CMAX];
  #pragma unroll
  for (int c = 0; c < CMAX; ++c) acc[c] = 0.f;
  float m = -INFINITY, l = 0.f;
  if (a.sink != nullptr) { m = a.sink[h]; l = 1.f; }
  const bool sig = a.wbias != nullptr;
  if (sig) l = 1.f;                             // nothing to divide by
  for (int i = 0; i < part.n; ++i) {
    const int k0 = part.at(i) * WAVE, key = k0 + lane;
    float s = -INFINITY;
    if (key <= pos && (key >= lo || key < a.keep)) {
      const long page = bt[key / a.block_size];
      const T* k = a.kc + ((page * a.kv_heads + kvh) * a.block_size +
                           key % a.block_size) * a.dim;
      s = 0.f;
      for (int i = 0; i < a.dim; ++i) s += s_q[i] * ld1(k + i);
      if (a.cap > 0.f) s = a.cap * tanhf(s / a.cap);
      if (a.bias != nullptr)
        s += a.bias[(long)h * a.nbias + min(pos - key, a.nbias - 1)];
      if (a.r1 != nullptr)
        s -= a.r1[h] * log1pf(a.r2[h] * (float)(pos - key));
    }
    float p, keep = 1.f;
    if (sig) {
      p = sigmoid_f(s + a.wbias[h]);             // 0 of -inf
    } else {
      const float mn = fmaxf(m, wave_max(s));    // finite: some key is visible
      p = expf(s - mn);
      keep = expf(m - mn);
      l = l * keep + wave_sum(p);
      m = mn;
    }
    s_p[lane] = p;
    __syncthreads();
    #pragma unroll
    for (int c = 0; c < CMAX; ++c) acc[c] *= keep;
    const int nk = min(WAVE, pos - k0 + 1);
    for (int j = 0; j < nk; ++j) {
      const int kj = k0 + j;
      const long page = bt[kj / a.block_size];
      const T* v = a.vc + ((page * a.kv_heads + kvh) * a.block_size +
                           kj % a.block_size) * a.v_ld;
      const float pj = s_p[j];
      #pragma unroll
      for (int c = 0; c < CMAX; ++c) {
        const int col = lane + c * WAVE;
        if (col < a.vdim) acc[c] += pj * ld1(v + col);
      }
    }
    __syncthreads();
  }
  float g = a.mult / l;
  if (a.gate != nullptr) g *= sigmoid_f(ld1(a.gate + row * a.g_ld + h));
  T* out = a.out + row * a.out_ld + (long)h * a.vdim;
  #pragma unroll
  for (int c = 0; c < CMAX; ++c) {
    const int col = lane + c * WAVE;
    if (col < a.vdim) st1(out + col, acc[c] * g);
  }
}

template <class T>
void launch_attn_ctx_any(const AttnCtx<T>& a, int entries, int max_len,
                         hipStream_t stream) {
  auto go = [&](auto cmax) {
    attn_ctx_any_kernel<T, decltype(cmax)::value>
        <<<dim3(max_len, a.heads, entries), dim3(WAVE),
           (a.dim + WAVE) * sizeof(float), stream>>>(a);
  };
  if (a.vdim <= 4 * WAVE) go(std::integral_constant<int, 4>{});
  else go(std::integral_constant<int, ATTN_ANY_VDIM / WAVE>{});
}

template void launch_attn_ctx_any<float>(const AttnCtx<float>&, int, int,
                                         hipStream_t);
template void launch_attn_ctx_any<bf16_t>(const AttnCtx<bf16_t>&, int, int,
                                          hipStream_t);
