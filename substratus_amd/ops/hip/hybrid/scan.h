// Selective scans (scan.hip). Per channel c with a state S[c, 0 .. n - 1]:
//   dt = softplus(z + zb)
//   S <- exp(dt a) S + dt u B,   out = (S . C + d u) silu(gate)
// S lives in 32 bits, [slots, channels, n]. A slot is read only when the
// entry's first row is not at position 0; slot < 0 marks a padded row.
#pragma once

#include "typed.h"

#include <type_traits>

template <class T>
struct Scan {
  T* out;                  // row r at out + r * out_ld
  const T* u;              // [rows, channels]
  const T* gate;           // row r at gate + r * g_ld
  const float* z;          // [rows, channels]
  const float* zb;         // [channels]
  const T* low;            // row r has B at low + r * low_ld, then C
  const float* a;          // [channels, n]
  const float* d;          // [channels]
  float* state;
  const int* state_slots;  // [entries]
  const int* positions;    // [rows]
  const int* seq_start;    // [entries + 1], or null: one row each
  long out_ld, g_ld, low_ld;
  int channels, n;
};

constexpr int SCAN_MAX_STATE = 512;

int scan_segments(int entries, int channels, int n, int max_len);
// ws [entries, nseg, channels, n] and ws_dt [entries, nseg, channels] for
// nseg > 1
template <class T>
void launch_scan(const Scan<T>&, int entries, int max_len, int nseg,
                 float* ws, float* ws_dt, hipStream_t);
