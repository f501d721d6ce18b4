// Products of rows with one weight matrix per group, y = act(x w[g]^T):
//   * tiles null: every group has all m rows (the heads of a projection);
//     group g's part of a row starts at x + g * x_gs and y + g * y_gs;
//   * tiles given: rows are packed by group (the tokens of every expert) and
//     cut into tiles on the device; tiles[0] is their number, then come a
//     group and a first row for each, start[g + 1] ends group g.
#pragma once

#include "typed.h"

#include <type_traits>

enum class Act {
  NONE,
  GELU,      // exact gelu
  GATE,      // times sigmoid(gate[row][g][n]), or sigmoid(gate[row][g])
  SIDE,      // gelu_tanh, times table[tokens[row]][n]
  GLU,       // columns are gate and up in turn; y has half as many
};

template <class T, class Y>
struct GroupGemm {
  Y* y;
  const T* x;
  const T* w;              // [groups, n, k]
  long y_ld, y_gs, x_ld, x_gs;
  int m, n, k, groups;
  int splits;              // > 1: shares of the inner dimension, share s to
                           //   y + s * m * n (unpacked rows, one group)
  int tail;                // elements of x after k, appended to y as they are
  Act act;
  const int* src;          // packed row -> row of x, or null
  const int* start;
  const int* tiles;
  int max_tiles;           // bound of tiles[0]
  const T* gate;           // row r, group g, column n at
  long gate_ld, gate_gs;   //   gate + r * gate_ld + g * gate_gs + n,
  bool gate_each;          //   or not each column: without n
  const int* tokens;
  const T* table;          // row t at table + t * t_ld
  long t_ld;
  int vocab;
  Glu glu;
  float limit;             // of Glu::CLAMPED
  bool quads;              // set by launch_group_gemm: four columns at a time
};

struct Tile {
  int g, r0, r1;           // rows [r0, r1), r1 <= r0: nothing to do
};

template <class T, class Y>
DEV_INLINE Tile tile_of(const GroupGemm<T, Y>& a, int i, int g, int bm) {
  if (a.tiles == nullptr) return {g, i * bm, min((i + 1) * bm, a.m)};
  if (i >= a.tiles[0]) return {0, 0, 0};
  const int grp = a.tiles[1 + 2 * i], r0 = a.tiles[2 + 2 * i];
  return {grp, r0, min(r0 + bm, a.start[grp + 1])};
}

// FAST: to about 1e-7 and 1e-6, for bf16 results; erf by formula 7.1.26 of
// Abramowitz and Stegun, Handbook of Mathematical Functions.
template <bool FAST>
DEV_INLINE float gelu_erf_f(float v) {
  const float z = v * 0.70710678118654752440f;
  if constexpr (!FAST) return 0.5f * v * (1.f + erff(z));
  const float x = fabsf(z);
  const float t = __builtin_amdgcn_rcpf(1.f + 0.3275911f * x);
  const float p = t * (0.254829592f + t * (-0.284496736f + t * (1.421413741f +
                  t * (-1.453152027f + t * 1.061405429f))));
  const float e = p * __expf(-x * x);            // 1 - erf(x)
  return 0.5f * v * (z < 0.f ? e : 2.f - e);
}

template <bool FAST>
DEV_INLINE float gelu_tanh_f(float v) {
  const float in = 0.79788456080286535588f * (v + 0.044715f * v * v * v);
  if constexpr (!FAST) return 0.5f * v * (1.f + tanhf(in));
  // (1 + tanh(x)) / 2 = 1 / (1 + exp(-2 x))
  return v * __builtin_amdgcn_rcpf(1.f + __expf(-2.f * in));
}

// N columns of a row from n on, all of them there.
template <Act ACT, bool FAST, int N, class T, class Y>
DEV_INLINE void group_act(const GroupGemm<T, Y>& a, int r, int g, int n,
                          float* v) {
  float f[N];
  if constexpr (ACT == Act::GATE) {
    const T* p = a.gate + (long)r * a.gate_ld + (long)g * a.gate_gs;
    if (a.gate_each) {
      ldv<N>(p + n, f);
    } else {
      f[0] = ld1(p);
      #pragma unroll
      for (int j = 1; j < N; ++j) f[j] = f[0];
    }
  }
  if constexpr (ACT == Act::SIDE) {
    const int t = min(max(a.tokens[r], 0), a.vocab - 1);
    ldv<N>(a.table + (long)t * a.t_ld + n, f);
  }
  #pragma unroll
  for (int j = 0; j < N; ++j) {
    if constexpr (ACT == Act::GELU) v[j] = gelu_erf_f<FAST>(v[j]);
    if constexpr (ACT == Act::GATE) v[j] *= sigmoid_f(f[j]);
    if constexpr (ACT == Act::SIDE) v[j] = gelu_tanh_f<FAST>(v[j]) * f[j];
  }
}

typedef __attribute__((ext_vector_type(4))) float float4v;

// Four consecutive columns of a row, as far as they are there.
template <Act ACT, class Y>
DEV_INLINE void store4(const GroupGemm<bf16_t, Y>& a, Tile t, int r, int n,
                       float4v acc) {
  if (r >= t.r1 || n >= a.n) return;
  if constexpr (ACT == Act::GLU) {
    Y* y = a.y + (long)r * a.y_ld + t.g * a.y_gs + n / 2;
    const float v0 = glu_f(a.glu, acc[0], acc[1], a.limit);
    const float v1 = glu_f(a.glu, acc[2], acc[3], a.limit);
    if (a.quads) {
      const float v[2] = {v0, v1};
      stv<2>(y, v);
    } else {
      st1(y, v0);
      if (n + 2 < a.n) st1(y + 1, v1);
    }
    return;
  }
  Y* y = a.y + (long)r * a.y_ld + t.g * a.y_gs + n;
  if (a.quads) {
    float v[4] = {acc[0], acc[1], acc[2], acc[3]};
    group_act<ACT, true, 4>(a, r, t.g, n, v);
    stv<4>(y, v);
    return;
  }
  #pragma unroll
  for (int c = 0; c < 4; ++c) {
    float v = acc[c];
    if (n + c >= a.n) return;
    group_act<ACT, true, 1>(a, r, t.g, n + c, &v);
    st1(y + c, v);
  }
}

// Calls f(integral_constant<Act>) with the product's.
template <class F>
void by_act(Act act, F f) {
  switch (act) {
    case Act::NONE: f(std::integral_constant<Act, Act::NONE>{}); break;
    case Act::GELU: f(std::integral_constant<Act, Act::GELU>{}); break;
    case Act::GATE: f(std::integral_constant<Act, Act::GATE>{}); break;
    case Act::SIDE: f(std::integral_constant<Act, Act::SIDE>{}); break;
    case Act::GLU: f(std::integral_constant<Act, Act::GLU>{}); break;
  }
}

// What the blocks of a tile's first columns do on the side.
template <class T, class Y>
DEV_INLINE void copy_tail(const GroupGemm<T, Y>& a, Tile t, int tid,
                          int threads) {
  for (int i = tid; i < (t.r1 - t.r0) * a.tail; i += threads) {
    const long r = t.r0 + i / a.tail;
    const int c = i % a.tail;
    st1(a.y + r * a.y_ld + t.g * a.y_gs + a.n + c,
        ld1(a.x + r * a.x_ld + t.g * a.x_gs + a.k + c));
  }
}

// Row tile that suits `rows` rows in `groups` groups, with inner sizes that
// are multiples of `ks` (packed rows are cut once for two products).
int group_gemm_tile(long rows, int groups, bool bf16, int ks);

// Whether packed rows may come in tiles of this size.
template <class T, class Y>
bool group_gemm_takes(const GroupGemm<T, Y>&, int tile);

// Shares of the inner dimension that let one small product fill the chip.
template <class T, class Y>
int group_gemm_splits(const GroupGemm<T, Y>&);

template <class T, class Y>
void launch_group_gemm(const GroupGemm<T, Y>&, int tile, hipStream_t);

// Tiles of 128 or 256 rows (group_gemm_tile.hip).
template <class Y>
void launch_group_gemm_tile(const GroupGemm<bf16_t, Y>&, int tile,
                            hipStream_t);
