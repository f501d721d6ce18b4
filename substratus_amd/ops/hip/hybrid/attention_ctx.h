// Arguments shared by the cache-reading attention kernels.
#pragma once

#include "typed.h"

#include <type_traits>

template <class T>
struct AttnCtx {
  T* out;                  // [rows, heads * vdim]
  const T* q;              // row r, head h at q + r * q_ld + h * dim
  const T* gate;           // row r, head h at gate + r * g_ld + h, or null;
                           // flat: column c at gate + r * g_ld + h * vdim + c
  const T* kc;             // [blocks, kv_heads, block_size, dim]
  const T* vc;             // [blocks, kv_heads, block_size, vdim], rows of
                           // v_ld elements (values may be part of the keys)
  const float* bias;       // [heads, nbias] by distance, or null
  const int* positions;    // [rows]
  const int* seq_start;    // [entries + 1] row offsets, or null: one row each
  const int* block_table;  // [entries, max_blocks]
  long q_ld, g_ld, v_ld;
  int heads, kv_heads, dim, vdim, nbias, chunk, max_blocks, block_size;
  float scale;
  // flat: keys and values are not paged; key j of entry e is row
  // ctx_start[e] + j of kc and vc, whose rows are v_ld apart and hold one
  // piece per head; the last `shared` elements of every head's key are kr's
  const int* ctx_start;    // [entries + 1]
  const T* kr;             // [all keys, shared]
  int shared;
};

constexpr float LOG2E = 1.44269504088896340736f;

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
