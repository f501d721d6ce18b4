// Products of rows with one weight matrix per group, y = act(x w[g]^T):
//   * tiles null: every group has all m rows (the heads of a projection);
//     group g's part of a row starts at x + g * x_gs and y + g * y_gs;
//   * tiles given: rows are packed by group (the tokens of every expert) and
//     cut into tiles on the device; tiles[0] is their number, then come a
//     group and a first row for each, start[g + 1] ends group g.
#pragma once

#include "typed.h"

enum class Act {
  NONE,
  GELU,      // exact gelu
  GATE,      // times sigmoid(gate[row][g][n])
  SIDE,      // gelu_tanh, times table[tokens[row]][n]
};

template <class T, class Y>
struct GroupGemm {
  Y* y;
  const T* x;
  const T* w;              // [groups, n, k]
  long y_ld, y_gs, x_ld, x_gs;
  int m, n, k, groups;
  int tail;                // elements of x after k, appended to y as they are
  Act act;
  const int* src;          // packed row -> row of x, or null
  const int* start;
  const int* tiles;
  int max_tiles;           // bound of tiles[0]
  const T* gate;           // row r, group g, column n at
  long gate_ld, gate_gs;   //   gate + r * gate_ld + g * gate_gs + n
  const int* tokens;
  const T* table;          // row t at table + t * t_ld
  long t_ld;
  int vocab;
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

DEV_INLINE float gelu_erf_f(float v) {
  return 0.5f * v * (1.f + erff(v * 0.70710678118654752440f));
}

template <class T, class Y>
DEV_INLINE float group_act(const GroupGemm<T, Y>& a, int r, int g, int n,
                           float v) {
  if (a.act == Act::GELU) return gelu_erf_f(v);
  if (a.act == Act::GATE)
    return v * sigmoid_f(ld1(a.gate + (long)r * a.gate_ld +
                             (long)g * a.gate_gs + n));
  if (a.act == Act::SIDE) {
    const float in = 0.79788456080286535588f * (v + 0.044715f * v * v * v);
    const int t = min(max(a.tokens[r], 0), a.vocab - 1);
    return 0.5f * v * (1.f + tanhf(in)) * ld1(a.table + (long)t * a.t_ld + n);
  }
  return v;
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

template <class T, class Y>
void launch_group_gemm(const GroupGemm<T, Y>&, int tile, hipStream_t);

// Tiles of 128 or 256 rows (group_gemm_tile.hip).
template <class Y>
void launch_group_gemm_tile(const GroupGemm<bf16_t, Y>&, int tile,
                            hipStream_t);
