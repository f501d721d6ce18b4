// Short causal convolutions over time (short_conv.hip).
#pragma once

#include "typed.h"

#include <type_traits>

template <class T>
struct Conv {
  const T* x;              // row r at x + r * ld
  long ld;
  const float* in_bias;    // [channels], added to every input, or null
  const float* weight;     // [channels, taps], the last tap is the row's own
  T* state;                // [slots, taps - 1, channels]: inputs without bias
  const int* state_slots;  // [entries], -1: none
  const int* positions;    // [rows]
  const int* seq_start;    // [entries + 1], or null: one row each
  int channels, taps;
  // plain
  T* out;                  // [rows, channels]
  const float* bias;       // [channels], or null
  bool act;                // silu
  // queries and keys
  T* q;                    // [rows, (channels / dim - kv) * dim]
  T* kc;                   // [blocks, kv, block_size, dim]
  T* vc;
  const float* rope;       // [rows, half, 2]: cosine, sine
  const int* slots;        // [rows]
  int half, kv, dim, block_size;
  // queries, keys and values: vc [blocks, kv, block_size, vdim]
  int vdim;
  float temp;              // q times 1 + temp ln(floor((p + 1) / every) + 1)
  int every;
  float v_eps;             // values over their root mean square, < 0: not
};

template <class T>
void launch_short_conv(const Conv<T>&, int entries, int max_len, hipStream_t);
bool conv_qkv_takes(int vdim);
template <class T>
void launch_conv_qkv(const Conv<T>&, int entries, int max_len, hipStream_t);
template <class T>
void launch_conv_rope(const Conv<T>&, int entries, int max_len, hipStream_t);
void launch_rope_table(float* out, const int* positions, const double* turns,
                       long rows, int half, hipStream_t);
