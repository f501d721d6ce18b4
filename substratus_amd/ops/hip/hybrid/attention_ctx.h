// Arguments shared by the cache-reading attention kernels.
#pragma once

#include "typed.h"

#include <type_traits>

template <class T>
struct AttnCtx {
  T* out;                  // row r, head h at out + r * out_ld + h * vdim
  const T* q;              // row r, head h at q + r * q_ld + h * dim
  const T* gate;           // row r, head h at gate + r * g_ld + h, or null;
                           // gate_each (flat only): its column c at
                           // gate + r * g_ld + h * vdim + c
  const T* kc;             // [blocks, kv_heads, block_size, dim]
  const T* vc;             // [blocks, kv_heads, block_size, vdim], rows of
                           // v_ld elements (values may be part of the keys)
  const float* bias;       // [heads, nbias] by distance, or null
  const float* r1;         // [heads]: r1 ln(1 + r2 distance) is taken off the
  const float* r2;         //   score, or null
  const float* wbias;      // [heads]: weights are sigmoid(score + wbias), not
                           //   a softmax, or null
  const float* sink;       // [heads], or null
  const int* positions;    // [rows]
  const int* seq_start;    // [entries + 1] row offsets, or null: one row each
  const int* block_table;  // [entries, max_blocks]
  long q_ld, g_ld, v_ld, out_ld;
  int heads, kv_heads, dim, vdim, nbias, chunk, max_blocks, block_size;
  int window;              // > 0: keys that a row sees, its own included
  int keep;                // with a window: a sequence's first keys, too
  float scale;
  float cap;               // > 0: scores are cap * tanh(score / cap)
  float mult;              // of the result
  bool quads;              // out: four columns at a time may be stored
  bool gate_each;
  // flat: keys and values are not paged; key flat_from + j of entry e is row
  // ctx_start[e] + j of kc and vc, whose rows are v_ld apart and hold one
  // piece per head; the last `shared` elements of every head's key are kr's
  const int* ctx_start;    // [entries + 1]
  const T* kr;             // [all keys, shared]
  int shared;
};

constexpr float LOG2E = 1.44269504088896340736f;

// First key that a row at `pos` sees, apart from the kept ones.
template <class T>
DEV_INLINE int first_seen(const AttnCtx<T>& a, int pos) {
  if (a.chunk > 0) return pos / a.chunk * a.chunk;
  return a.window > 0 ? max(pos - a.window + 1, 0) : 0;
}

// First key that lies there when keys are not paged, for an entry whose rows
// begin at position pos0.
DEV_INLINE int flat_from(int window, int pos0) {
  return window > 0 ? max(pos0 - window + 1, 0) : 0;
}

// What a key at distance n adds to head h's score, times log2(e).
template <class T>
DEV_INLINE float distance_bias2(const AttnCtx<T>& a, int h, int n) {
  float b = 0.f;
  if (a.bias != nullptr)
    b = a.bias[(long)h * a.nbias + min(max(n, 0), a.nbias - 1)] * LOG2E;
  if (a.r1 != nullptr)
    b -= a.r1[h] * __builtin_amdgcn_logf(1.f + a.r2[h] * (float)max(n, 0));
  return b;
}

// Pieces of a context (pages, steps) that hold visible keys, in order: those
// of the kept keys, then those from key `lo` to the last piece.
struct Pieces {
  int kept, skip, n;
  DEV_INLINE Pieces(int keep, int lo, int pieces, int size) {
    kept = min((keep + size - 1) / size, pieces);
    skip = max(lo / size - kept, 0);
    n = pieces - skip;
  }
  DEV_INLINE int at(int i) const { return i < kept ? i : i + skip; }
};

// tanh(z) = 1 - 2 / (e^(2z) + 1), to 1e-7 absolute; `z2` is 2 z log2(e)
DEV_INLINE float tanh_exp2(float z2) {
  return 1.f - 2.f * __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(z2) + 1.f);
}

// sigmoid of a score times log2(e); -inf gives 0
DEV_INLINE float sigmoid_exp2(float s2) {
  return __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-s2));
}

constexpr int ATTN_ANY_VDIM = 1024;   // largest value size

template <class T>
void launch_attn_ctx_any(const AttnCtx<T>&, int entries, int max_len,
                         hipStream_t);

bool attn_ctx_decode_supported(int dim, int vdim, int block_size);
int attn_ctx_decode_splits(int entries, int heads, int kv_heads, int span);
void launch_attn_ctx_decode(const AttnCtx<bf16_t>&, int entries, int splits,
                            float* part_o, float* part_ml, hipStream_t);

bool attn_ctx_prefill_supported(int dim, int vdim, int block_size);
void launch_attn_ctx_prefill(const AttnCtx<bf16_t>&, int entries, int max_len,
                             hipStream_t);

// One head of shared keys whose first columns are the values.
bool attn_latent_supported(int dim, int vdim, int block_size);
int attn_latent_splits(int entries, int max_len, int heads, int span);
void launch_attn_latent(const AttnCtx<bf16_t>&, int entries, int max_len,
                        int span, int splits, float* part_o, float* part_ml,
                        hipStream_t);
void launch_attn_ctx_merge(const AttnCtx<bf16_t>&, long rows, int splits,
                           const float* part_o, const float* part_ml,
                           hipStream_t);
