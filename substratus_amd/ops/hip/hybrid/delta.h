// The gated delta rule (delta.hip, delta_chunk.hip). Per head, with q and k
// unit vectors (q also times dim^-1/2) and a decay per key channel:
//   g = exp(-rate softplus(z + zb)),  S <- diag(g) S
//   u = sigmoid(beta) (v - S^T k),    S <- S + k u^T
//   out = rms(S^T q) norm sigmoid(gate) mult
// Query and key head of head h: h / (heads / kv_heads). S lives in 32 bits,
// [slots, heads, dim, vdim]. A slot is read only when the entry's first row
// is not at position 0; slot < 0 marks a padded row.
#pragma once

#include "typed.h"

#include <type_traits>

template <class T>
struct Delta {
  T* out;                  // row r, head h at out + r * out_ld + h * vdim
  const T* qkv;            // [rows, q | k | v]
  const float* z;          // [rows, heads * dim]
  const float* zb;         // [heads * dim]
  const float* rate;       // [heads]
  const T* beta;           // row r, head h at beta + r * b_ld + h
  const T* gate;           // row r, head h at gate + r * g_ld + h * vdim
  const float* norm;       // [vdim]
  float* state;
  const int* state_slots;  // [entries]
  const int* positions;    // [rows]
  const int* seq_start;    // [entries + 1], or null: one row each
  long ld, out_ld, b_ld, g_ld;
  int heads, kv_heads, dim, vdim;
  float eps, mult;
};

constexpr float UNIT_EPS = 1e-6f;    // under the root of a unit vector's length

template <class T>
void launch_delta_recurrent(const Delta<T>&, int entries, hipStream_t);

// Portions by chunks of tokens: heads h0 .. h0 + heads - 1, with a workspace
// of delta_chunk_bytes per head.
bool delta_chunk_supported(const Delta<bf16_t>&, int max_len);
long delta_chunk_bytes(int dim, long rows, int entries);
void launch_delta_chunk(const Delta<bf16_t>&, int entries, int max_len, int h0,
                        int heads, void* ws, hipStream_t);
