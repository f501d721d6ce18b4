// Arguments shared by the gated-linear-attention kernels.
//
// Per head, with a decay per key channel c:
//   ln a_t[c] = ln(sigmoid(z_t[c])) / tau,  z_t = A2 (A1 h_t) + b
//   S_t = diag(a_t) S_(t-1) + k_t v_t^T,    o_t = S_t^T q_t * qscale
//   out_t = rms(o_t) * w * silu(g_t)
// Without A2 (Gla::decay given) the decays are constants per head, q, k and v
// pass silu, qscale is 1 and out_t = o_t ("constant" below).
//
// S lives in 32 bits, [slots, heads, dim, vdim]. A slot is read only when the
// entry's first row is not at position 0, so it needs no clearing between
// requests; slot < 0 marks a padded row, which touches no state.
#pragma once

#include "typed.h"

template <class T>
struct Gla {
  T* out;                // [rows, heads * vdim]
  const T* x;            // projected rows, ld apart, parts at the offsets below
  long ld;
  int k_off, v_off, g_off, a_off;   // q at 0; A1 h at a_off, `rank` wide
  const float* a2;       // [heads * dim, rank]
  const float* a2b;      // [heads * dim]
  const float* norm;     // [vdim]
  const float* decay;    // [heads], or null
  float* state;
  const int* state_slots;  // [entries]
  const int* positions;    // [rows]
  const int* seq_start;    // [entries + 1], or null: one row each
  int heads, dim, vdim, rank;
  float qscale, inv_tau, eps;
};

// silu, rounded as activations are
template <class T>
DEV_INLINE float silu_as(float z) {
  z *= sigmoid_f(z);
  if constexpr (sizeof(T) == 2) z = bf2f(f2bf(z));
  return z;
}

template <class T>
void launch_gla_recurrent(const Gla<T>&, int entries, hipStream_t);

bool gla_chunk_supported(int dim, int vdim, int rank);
int gla_chunk_segments(int entries, int heads, int max_len);
void launch_gla_chunk(const Gla<bf16_t>&, int entries, int max_len, int nseg,
                      float* ws, float* ws_decay, hipStream_t);
