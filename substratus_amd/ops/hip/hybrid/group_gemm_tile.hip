// Grouped products (group_gemm.h) in bf16 with many rows per group: tiles of
// 256 x 256 or 128 x 128 on the matrix cores.
//
// Both operands go to LDS by direct loads, 64 of the inner dimension at a
// time, ahead of their use (counted waits leave later loads in flight over
// the barriers). Rows of x are gathered by the addresses of those
// loads, so packing tokens by expert moves no data. A row's 16-byte pieces
// are permuted by the row to keep fragment reads free of bank conflicts.
// Rows and columns past the end are computed from clamped addresses and not
// stored. Weights are the first operand: a lane ends up with four consecutive
// columns of one row. Neighbouring tiles run on one XCD and share its L2.
#include "group_gemm.h"

namespace {

typedef __attribute__((ext_vector_type(8))) short short8;

constexpr int BK = 64;
constexpr int XCDS = 8;

DEV_INLINE void load_to_lds(const void* g, void* lds) {
  __builtin_amdgcn_global_load_lds(
      (const __attribute__((address_space(1))) unsigned int*)g,
      (__attribute__((address_space(3))) unsigned int*)lds, 16, 0, 0);
}

// The workgroup's tile and first column. Workgroups are handed out to XCDs in
// turn, so consecutive tiles are those whose numbers are XCDS apart.
template <class Y>
DEV_INLINE Tile my_tile(const GroupGemm<bf16_t, Y>& a, int bm, int bn,
                        int* n0) {
  const int nt = (a.n + bn - 1) / bn;
  const int blocks = nt * (a.tiles != nullptr ? a.tiles[0]
                                              : (a.m + bm - 1) / bm);
  const int b = blockIdx.x, q = blocks / XCDS, r = blocks % XCDS,
            xcd = b % XCDS;
  if (b >= blocks) return {0, 0, 0};
  const int id =
      (xcd < r ? xcd * (q + 1) : r * (q + 1) + (xcd - r) * q) + b / XCDS;
  *n0 = id % nt * bn;
  return tile_of(a, id / nt, blockIdx.y, bm);
}

// One step ahead, two barriers per step.
template <class Y, Act ACT, int BM, int BN, int WM, int WN>
__global__ __launch_bounds__(WM * WN * WAVE)
void group_gemm_tile_kernel(GroupGemm<bf16_t, Y> a) {
  constexpr int NW = WM * WN;
  constexpr int FM = BM / WM / 16, FN = BN / WN / 16;
  constexpr int LX = BM * BK * 2 / 1024 / NW;    // loads per wave and step
  constexpr int LW = BN * BK * 2 / 1024 / NW;
  __shared__ uint4 s_t[2][(BM + BN) * BK / 8];   // x, then w

  int n0;
  const Tile t = my_tile(a, BM, BN, &n0);
  if (t.r1 <= t.r0) return;
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

  #pragma unroll
  for (int i = 0; i < FM; ++i)
    #pragma unroll
    for (int j = 0; j < FN; ++j)
      store4<ACT>(a, t, t.r0 + wm * (BM / WM) + i * 16 + lo,
                  n0 + wn * (BN / WN) + j * 16 + grp * 4, acc[i][j]);
}

// Eight waves on 256 x 256, in two groups half a phase apart: while one group
// reads fragments from LDS and starts loads, the other one, on the same
// SIMDs, keeps the matrix cores busy.
//
// A wave's 128 x 64 outputs are four quadrants, one per phase: rows X0, X1 of
// its x tile times columns W0, W1 of its w tile. Each of the four regions of
// a step's operands is read from LDS in one phase by all waves, and the phase
// after that starts the loads of the same region two steps later:
//
//   phase            0        1        2        3
//   reads            X0       W1       X1       W0 of the next step
//   starts loading   W0       X0       W1       X1      (two steps ahead)
//   multiplies       X0 W0    X0 W1    X1 W0    X1 W1
//
// So every region is loaded in the same order, two direct loads per wave and
// phase, and what the next phase reads was started seven phases before it:
// a wait for all but the last 12 loads is right in every phase. Past the
// last step the same loads are done again, into regions nobody reads.
constexpr int PBM = 256, PBN = 256, PNW = 8;

template <class Y, Act ACT>
__global__ __launch_bounds__(PNW * WAVE, 2)
void group_gemm_pingpong_kernel(GroupGemm<bf16_t, Y> a) {
  constexpr int REGION = 128 * BK / 8;           // 16-byte pieces
  __shared__ uint4 s_t[2 * 4 * REGION];
  enum { W0, X0, W1, X1 };
  int n0;
  const Tile t = my_tile(a, PBM, PBN, &n0);
  if (t.r1 <= t.r0) return;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / WAVE);
  const int lane = threadIdx.x % WAVE;
  const int lo = lane & 15, grp = lane >> 4;
  const int wm = wave / 4, wn = wave % 4;

  // places this lane loads from: by region, two rows each, 8 lanes per row
  const bf16_t* from[4][2];
  #pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int row = (wave * 2 + i) * 8 + lane / 8;   // of a region's 128
    const int k = ((lane % 8) ^ (row & 7)) * 8;
    #pragma unroll
    for (int h = 0; h < 2; ++h) {
      const int r = min(t.r0 + row / 64 * 128 + h * 64 + row % 64, t.r1 - 1);
      from[h ? X1 : X0][i] =
          a.x + (long)(a.src != nullptr ? a.src[r] : r) * a.x_ld +
          t.g * a.x_gs + k;
      const int n = min(n0 + row / 32 * 64 + h * 32 + row % 32, a.n - 1);
      from[h ? W1 : W0][i] = a.w + ((long)t.g * a.n + n) * a.k + k;
    }
  }
  const int steps = a.k / BK;
  auto load = [&](int region, int step) {
    const int k = min(step, steps - 1) * BK;
    #pragma unroll
    for (int i = 0; i < 2; ++i)
      load_to_lds(from[region][i] + k,
                  &s_t[((step & 1) * 4 + region) * REGION +
                       (wave * 2 + i) * WAVE]);
  };
  auto piece = [&](int region, int step, int row, int k) {
    return *reinterpret_cast<const short8*>(
        &s_t[((step & 1) * 4 + region) * REGION + row * 8 +
             ((k * 4 + grp) ^ (row & 7))]);
  };

  float4v acc[8][4];
  #pragma unroll
  for (int i = 0; i < 8; ++i)
    #pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = (float4v){0.f, 0.f, 0.f, 0.f};
  short8 xf[4][2], wf[2][2][2];
  auto read_x = [&](int h, int step) {
    #pragma unroll
    for (int i = 0; i < 4; ++i)
      #pragma unroll
      for (int k = 0; k < 2; ++k)
        xf[i][k] = piece(h ? X1 : X0, step, wm * 64 + i * 16 + lo, k);
  };
  auto read_w = [&](auto h, int step) {
    constexpr int H = decltype(h)::value;
    #pragma unroll
    for (int j = 0; j < 2; ++j)
      #pragma unroll
      for (int k = 0; k < 2; ++k)
        wf[H][j][k] = piece(H ? W1 : W0, step, wn * 32 + j * 16 + lo, k);
  };
  auto reads_done = [&] {
    asm volatile("s_waitcnt vmcnt(12) lgkmcnt(0)\n\ts_barrier" ::: "memory");
    __builtin_amdgcn_sched_barrier(0);
  };
  auto multiply = [&](auto xh, auto wh) {
    constexpr int XH = decltype(xh)::value, WH = decltype(wh)::value;
    __builtin_amdgcn_s_setprio(1);
    #pragma unroll
    for (int k = 0; k < 2; ++k)
      #pragma unroll
      for (int i = 0; i < 4; ++i)
        #pragma unroll
        for (int j = 0; j < 2; ++j)
          acc[XH * 4 + i][WH * 2 + j] =
              __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                  wf[WH][j][k], xf[i][k], acc[XH * 4 + i][WH * 2 + j], 0, 0,
                  0);
    __builtin_amdgcn_s_setprio(0);
    __builtin_amdgcn_sched_barrier(0);
    asm volatile("s_barrier" ::: "memory");
    __builtin_amdgcn_sched_barrier(0);
  };
  using std::integral_constant;
  constexpr integral_constant<int, 0> h0{};
  constexpr integral_constant<int, 1> h1{};

  #pragma unroll
  for (int s = 0; s < 2; ++s) {
    load(W0, s); load(X0, s); load(W1, s); load(X1, s);
  }
  asm volatile("s_waitcnt vmcnt(12)\n\ts_barrier" ::: "memory");
  read_w(h0, 0);
  asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
  if (wm == 1) asm volatile("s_barrier" ::: "memory");   // half a phase later
  for (int s = 0; s < steps; ++s) {
    read_x(0, s); load(W0, s + 2); reads_done(); multiply(h0, h0);
    read_w(h1, s); load(X0, s + 2); reads_done(); multiply(h0, h1);
    read_x(1, s); load(W1, s + 2); reads_done(); multiply(h1, h0);
    read_w(h0, s + 1); load(X1, s + 2); reads_done(); multiply(h1, h1);
  }
  if (wm == 0) asm volatile("s_barrier" ::: "memory");
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");

  #pragma unroll
  for (int i = 0; i < 8; ++i)
    #pragma unroll
    for (int j = 0; j < 4; ++j)
      store4<ACT>(a, t, t.r0 + wm * 128 + i * 16 + lo,
                  n0 + wn * 64 + j * 16 + grp * 4, acc[i][j]);
}

}  // namespace

template <class Y>
void launch_group_gemm_tile(const GroupGemm<bf16_t, Y>& a, int tile,
                            hipStream_t stream) {
  const int mt = a.tiles != nullptr ? a.max_tiles : (a.m + tile - 1) / tile;
  const dim3 grid((a.n + tile - 1) / tile * mt,
                  a.tiles != nullptr ? 1 : a.groups);
  by_act(a.act, [&](auto act) {
    constexpr Act ACT = decltype(act)::value;
    if (tile == 256)
      group_gemm_pingpong_kernel<Y, ACT>
          <<<grid, dim3(PNW * WAVE), 0, stream>>>(a);
    else
      group_gemm_tile_kernel<Y, ACT, 128, 128, 2, 2>
          <<<grid, dim3(4 * WAVE), 0, stream>>>(a);
  });
}

template void launch_group_gemm_tile<bf16_t>(const GroupGemm<bf16_t, bf16_t>&,
                                             int, hipStream_t);
template void launch_group_gemm_tile<float>(const GroupGemm<bf16_t, float>&,
                                            int, hipStream_t);
