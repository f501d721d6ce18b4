// Grouped products (group_gemm.h) in bf16 with many rows per group: tiles of
// 256 x 256 or 128 x 128 on the matrix cores.
//
// Both operands go to LDS by direct loads, 64 of the inner dimension at a
// time, one step ahead (a counted wait leaves the next step's loads in
// flight over the barrier). Rows of x are gathered by the addresses of those
// loads, so packing tokens by expert moves no data. A row's 16-byte pieces
// are permuted by the row to keep fragment reads free of bank conflicts.
// Rows and columns past the end are computed from clamped addresses and not
// stored. Weights are the first operand: a lane ends up with four consecutive
// columns of one row. Neighbouring tiles run on one XCD and share its L2.
#include "group_gemm.h"

namespace {

typedef __attribute__((ext_vector_type(8))) short short8;
typedef __attribute__((ext_vector_type(4))) float float4v;

constexpr int BK = 64;
constexpr int XCDS = 8;

DEV_INLINE void load_to_lds(const void* g, void* lds) {
  __builtin_amdgcn_global_load_lds(
      (const __attribute__((address_space(1))) unsigned int*)g,
      (__attribute__((address_space(3))) unsigned int*)lds, 16, 0, 0);
}

template <class Y, int BM, int BN, int WM, int WN>
__global__ __launch_bounds__(WM * WN * WAVE)
void group_gemm_tile_kernel(GroupGemm<bf16_t, Y> a) {
  constexpr int NW = WM * WN;
  constexpr int FM = BM / WM / 16, FN = BN / WN / 16;
  constexpr int LX = BM * BK * 2 / 1024 / NW;    // loads per wave and step
  constexpr int LW = BN * BK * 2 / 1024 / NW;
  __shared__ uint4 s_t[2][(BM + BN) * BK / 8];   // x, then w

  const int nt = (a.n + BN - 1) / BN;
  const int blocks = nt * (a.tiles != nullptr ? a.tiles[0]
                                              : (a.m + BM - 1) / BM);
  if ((int)blockIdx.x >= blocks) return;
  int id;
  {
    const int b = blockIdx.x, q = blocks / XCDS, r = blocks % XCDS,
              xcd = b % XCDS;
    id = (xcd < r ? xcd * (q + 1) : r * (q + 1) + (xcd - r) * q) + b / XCDS;
  }
  const Tile t = tile_of(a, id / nt, blockIdx.y, BM);
  const int n0 = id % nt * BN;
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
  const int lo = lane & 15, grp = lane >> 4;
  const int wm = wave / WN, wn = wave % WN;

  // the places this lane loads from: 8 lanes per row of 64
  const bf16_t* xp[LX];
  const bf16_t* wp[LW];
  #pragma unroll
  for (int i = 0; i < LX; ++i) {
    const int row = (wave * LX + i) * 8 + lane / 8, c = lane % 8;
    const int r = min(t.r0 + row, t.r1 - 1);
    xp[i] = a.x + (long)(a.src != nullptr ? a.src[r] : r) * a.x_ld +
            t.g * a.x_gs + (c ^ (row & 7)) * 8;
  }
  #pragma unroll
  for (int i = 0; i < LW; ++i) {
    const int row = (wave * LW + i) * 8 + lane / 8, c = lane % 8;
    wp[i] = a.w + ((long)t.g * a.n + min(n0 + row, a.n - 1)) * a.k +
            (c ^ (row & 7)) * 8;
  }
  auto load = [&](int buf, int k) {
    #pragma unroll
    for (int i = 0; i < LX; ++i)
      load_to_lds(xp[i] + k, &s_t[buf][(wave * LX + i) * WAVE]);
    #pragma unroll
    for (int i = 0; i < LW; ++i)
      load_to_lds(wp[i] + k, &s_t[buf][BM * BK / 8 + (wave * LW + i) * WAVE]);
  };

  float4v acc[FM][FN];
  #pragma unroll
  for (int i = 0; i < FM; ++i)
    #pragma unroll
    for (int j = 0; j < FN; ++j) acc[i][j] = (float4v){0.f, 0.f, 0.f, 0.f};

  const int steps = a.k / BK;
  load(0, 0);
  for (int s = 0; s < steps; ++s) {
    const int buf = s & 1;
    // the barrier that ended the last step has released the other buffer
    if (s + 1 < steps) {
      load(buf ^ 1, (s + 1) * BK);
      asm volatile("s_waitcnt vmcnt(%0)" :: "i"(LX + LW) : "memory");
    } else {
      asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    }
    asm volatile("s_barrier" ::: "memory");
    const uint4* xt = s_t[buf];
    const uint4* wt = xt + BM * BK / 8;
    short8 wf[FN][2];
    #pragma unroll
    for (int j = 0; j < FN; ++j) {
      const int row = wn * (BN / WN) + j * 16 + lo;
      #pragma unroll
      for (int k = 0; k < 2; ++k)
        wf[j][k] = *reinterpret_cast<const short8*>(
            &wt[row * 8 + ((k * 4 + grp) ^ (row & 7))]);
    }
    #pragma unroll
    for (int i = 0; i < FM; ++i) {
      const int row = wm * (BM / WM) + i * 16 + lo;
      #pragma unroll
      for (int k = 0; k < 2; ++k) {
        const short8 xf = *reinterpret_cast<const short8*>(
            &xt[row * 8 + ((k * 4 + grp) ^ (row & 7))]);
        #pragma unroll
        for (int j = 0; j < FN; ++j)
          acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              wf[j][k], xf, acc[i][j], 0, 0, 0);
      }
    }
    asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
  }

  const bool quads = a.n % 4 == 0 && a.y_ld % 4 == 0 && a.y_gs % 4 == 0;
  #pragma unroll
  for (int i = 0; i < FM; ++i) {
    const int r = t.r0 + wm * (BM / WM) + i * 16 + lo;
    if (r >= t.r1) continue;
    Y* y = a.y + (long)r * a.y_ld + t.g * a.y_gs;
    #pragma unroll
    for (int j = 0; j < FN; ++j) {
      const int n = n0 + wn * (BN / WN) + j * 16 + grp * 4;
      if (n >= a.n) continue;
      float v[4];
      #pragma unroll
      for (int c = 0; c < 4; ++c)
        v[c] = n + c < a.n ? group_act(a, r, t.g, n + c, acc[i][j][c]) : 0.f;
      if (quads) {
        stv<4>(y + n, v);
      } else {
        #pragma unroll
        for (int c = 0; c < 4; ++c)
          if (n + c < a.n) st1(y + n + c, v[c]);
      }
    }
  }
}

}  // namespace

template <class Y>
void launch_group_gemm_tile(const GroupGemm<bf16_t, Y>& a, int tile,
                            hipStream_t stream) {
  const int mt = a.tiles != nullptr ? a.max_tiles : (a.m + tile - 1) / tile;
  const dim3 grid((a.n + tile - 1) / tile * mt,
                  a.tiles != nullptr ? 1 : a.groups);
  if (tile == 256)
    group_gemm_tile_kernel<Y, 256, 256, 2, 4>
        <<<grid, dim3(8 * WAVE), 0, stream>>>(a);
  else
    group_gemm_tile_kernel<Y, 128, 128, 2, 2>
        <<<grid, dim3(4 * WAVE), 0, stream>>>(a);
}

template void launch_group_gemm_tile<bf16_t>(const GroupGemm<bf16_t, bf16_t>&,
                                             int, hipStream_t);
template void launch_group_gemm_tile<float>(const GroupGemm<bf16_t, float>&,
                                            int, hipStream_t);
