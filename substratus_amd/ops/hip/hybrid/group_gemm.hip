// Grouped products (group_gemm.h) of few rows per group, and of any size:
//
//   stream   bf16, few rows per group: bound by reading the weights once.
//            Every wave takes a share of the inner dimension of a tile of
//            rows and 64 columns (4 waves; 16 and 32 columns where there are
//            few tiles; where the inner dimension is short, a share of the
//            rows), with both operands going from memory
//            straight into the matrix cores' registers (a fragment is 16
//            consecutive bytes of a row, so nothing is gained by LDS); there
//            is no barrier until the partial tiles are added up.
//   any      float, and bf16 sizes whose rows are not 16-byte pieces.
//
// Weights are the first operand, so a lane ends up with four consecutive
// columns of one row and stores them together.
#include "group_gemm.h"

namespace {

typedef __attribute__((ext_vector_type(8))) short short8;

constexpr int KC = 32;         // inner step of one matrix instruction

// ONCE: nobody reads it again
template <bool ONCE>
DEV_INLINE short8 frag(const bf16_t* p, bool there) {
  if (!there) return (short8){0, 0, 0, 0, 0, 0, 0, 0};
  if constexpr (ONCE) return __builtin_bit_cast(short8, nt_load_u4(p));
  else return *reinterpret_cast<const short8*>(p);
}

// FM, FN: 16-wide pieces of a wave's rows and columns; KW waves share the
// inner dimension, RW the rows
template <class Y, Act ACT, int FM, int FN, int KW, int RW>
__global__ __launch_bounds__(KW * RW * WAVE)
void group_gemm_stream_kernel(GroupGemm<bf16_t, Y> a) {
  constexpr int BM = FM * 16 * RW, BN = FN * 16, PAD = 4;
  static_assert(KW == 1 || RW == 1);
  const Tile t = tile_of(a, blockIdx.y, a.splits > 1 ? 0 : blockIdx.z, BM);
  if (t.r1 <= t.r0) return;
  const int share = a.splits > 1 ? blockIdx.z : 0;
  a.y += (long)share * a.m * a.n;
  const int n0 = blockIdx.x * BN;
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
  const int lo = lane & 15, kq = (lane >> 4) * 8;
  const int r0 = t.r0 + (RW > 1 ? wave * FM * 16 : 0);

  const bf16_t* wp[FN];
  const bf16_t* xp[FM];
  #pragma unroll
  for (int f = 0; f < FN; ++f)      // past the last column: computed, dropped
    wp[f] = a.w + ((long)t.g * a.n + min(n0 + f * 16 + lo, a.n - 1)) * a.k +
            kq;
  #pragma unroll
  for (int f = 0; f < FM; ++f) {
    const int r = min(r0 + f * 16 + lo, t.r1 - 1);
    xp[f] = a.x + (long)(a.src != nullptr ? a.src[r] : r) * a.x_ld +
            t.g * a.x_gs + kq;
  }
  float4v acc[FN][FM];
  #pragma unroll
  for (int i = 0; i < FN; ++i)
    #pragma unroll
    for (int j = 0; j < FM; ++j) acc[i][j] = (float4v){0.f, 0.f, 0.f, 0.f};

  const int chunks = (a.k + KC - 1) / KC, shares = KW * a.splits,
            part = share * KW + (KW > 1 ? wave : 0);
  const int c0 = chunks * part / shares, c1 = chunks * (part + 1) / shares;
  // U chunks at a time: their loads are in flight together
  auto steps = [&](int c, auto u, bool whole) {
    constexpr int U = decltype(u)::value;
    short8 wf[U][FN], xf[U][FM];
    #pragma unroll
    for (int i = 0; i < U; ++i) {
      const int k = (c + i) * KC;
      const bool there = whole || k + kq < a.k;
      #pragma unroll
      for (int f = 0; f < FN; ++f) wf[i][f] = frag<false>(wp[f] + k, there);
      #pragma unroll
      for (int f = 0; f < FM; ++f) xf[i][f] = frag<false>(xp[f] + k, there);
    }
    __builtin_amdgcn_sched_barrier(0);
    #pragma unroll
    for (int u = 0; u < U; ++u)
      #pragma unroll
      for (int i = 0; i < FN; ++i)
        #pragma unroll
        for (int j = 0; j < FM; ++j)
          acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              wf[u][i], xf[u][j], acc[i][j], 0, 0, 0);
  };
  constexpr int U = FM == 4 ? 2 : 4;
  const int full = min(c1, a.k / KC);
  int c = c0;
  if constexpr (FM == 1 && FN == 2)
    for (; c + 2 * U <= full; c += 2 * U)
      steps(c, std::integral_constant<int, 2 * U>{}, true);
  for (; c + U <= full; c += U)
    steps(c, std::integral_constant<int, U>{}, true);
  for (; c < full; ++c) steps(c, std::integral_constant<int, 1>{}, true);
  if (c < c1) steps(c, std::integral_constant<int, 1>{}, false);

  const int c4 = (lane >> 4) * 4;
  if constexpr (KW == 1) {
    #pragma unroll
    for (int i = 0; i < FN; ++i)
      #pragma unroll
      for (int j = 0; j < FM; ++j)
        store4<ACT>(a, t, r0 + j * 16 + lo, n0 + i * 16 + c4, acc[i][j]);
  } else {
    __shared__ alignas(16) float s_p[KW][BM][BN + PAD];
    #pragma unroll
    for (int i = 0; i < FN; ++i)
      #pragma unroll
      for (int j = 0; j < FM; ++j)
        *reinterpret_cast<float4v*>(&s_p[wave][j * 16 + lo][i * 16 + c4]) =
            acc[i][j];
    __syncthreads();
    for (int i = threadIdx.x; i < BM * BN / 4; i += KW * WAVE) {
      const int r = i / (BN / 4), c = i % (BN / 4) * 4;
      float4v v = {0.f, 0.f, 0.f, 0.f};
      #pragma unroll
      for (int w = 0; w < KW; ++w)
        v += *reinterpret_cast<const float4v*>(&s_p[w][r][c]);
      store4<ACT>(a, t, t.r0 + r, n0 + c, v);
    }
  }
  if (a.tail && blockIdx.x == 0)
    copy_tail(a, t, threadIdx.x, KW * RW * WAVE);
}

// 32 x 32 outputs per workgroup, 2 x 2 per thread, operands through LDS.
constexpr int AT = 32, AK = 16;

template <class T, class Y, Act ACT>
__global__ __launch_bounds__(256)
void group_gemm_any_kernel(GroupGemm<T, Y> a) {
  __shared__ float s_x[AK][AT + 1], s_w[AK][AT + 1];
  const Tile t = tile_of(a, blockIdx.y, blockIdx.z, AT);
  if (t.r1 <= t.r0) return;
  const int n0 = blockIdx.x * AT;
  const int tx = threadIdx.x % 16, ty = threadIdx.x / 16;
  float acc[2][2] = {{0.f, 0.f}, {0.f, 0.f}};
  for (int k0 = 0; k0 < a.k; k0 += AK) {
    for (int i = threadIdx.x; i < AT * AK; i += 256) {
      const int r = t.r0 + i / AK, n = n0 + i / AK, k = k0 + i % AK;
      const bool in = k < a.k;
      s_x[i % AK][i / AK] = in && r < t.r1
          ? ld1(a.x + (long)(a.src != nullptr ? a.src[r] : r) * a.x_ld +
                t.g * a.x_gs + k) : 0.f;
      s_w[i % AK][i / AK] = in && n < a.n
          ? ld1(a.w + ((long)t.g * a.n + n) * a.k + k) : 0.f;
    }
    __syncthreads();
    #pragma unroll
    for (int k = 0; k < AK; ++k)
      #pragma unroll
      for (int i = 0; i < 2; ++i)
        #pragma unroll
        for (int j = 0; j < 2; ++j)
          acc[i][j] += s_x[k][ty + 16 * i] * s_w[k][tx + 16 * j];
    __syncthreads();
  }
  #pragma unroll
  for (int i = 0; i < 2; ++i)
    #pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int r = t.r0 + ty + 16 * i, n = n0 + tx + 16 * j;
      if constexpr (ACT == Act::GLU) {
        const float up = __shfl_xor(acc[i][j], 1, WAVE);
        if (r < t.r1 && n < a.n && tx % 2 == 0)
          st1(a.y + (long)r * a.y_ld + t.g * a.y_gs + n / 2,
              glu_f(a.glu, acc[i][j], up, a.limit));
      } else if (r < t.r1 && n < a.n) {
        group_act<ACT, false, 1>(a, r, t.g, n, &acc[i][j]);
        st1(a.y + (long)r * a.y_ld + t.g * a.y_gs + n, acc[i][j]);
      }
    }
  if (a.tail && blockIdx.x == 0) copy_tail(a, t, threadIdx.x, 256);
}

// rows of both operands are whole, aligned 16-byte pieces
template <class Y>
bool pieces(const GroupGemm<bf16_t, Y>& a) {
  auto ok = [](const void* p) {
    return reinterpret_cast<uintptr_t>(p) % 16 == 0;
  };
  return a.k % 8 == 0 && a.x_ld % 8 == 0 && a.x_gs % 8 == 0 && ok(a.x) &&
         ok(a.w);
}

}  // namespace

int group_gemm_tile(long rows, int groups, bool bf16, int ks) {
  if (!bf16 || ks % 8) return AT;
  const long per = rows / groups;
  if (ks % 64 == 0 && per >= 96) return per >= 768 ? 256 : 128;
  return per <= 6 ? 16 : per <= 20 ? 32 : 64;
}

template <class T, class Y>
bool group_gemm_takes(const GroupGemm<T, Y>& a, int tile) {
  if constexpr (std::is_same_v<T, bf16_t>) {
    if (pieces(a) && (tile == 16 || tile == 32 || tile == 64)) return true;
    if (pieces(a) && (tile == 128 || tile == 256))
      return a.k % 64 == 0 && a.tail == 0;
  }
  return tile == AT;
}

// everything a store touches comes in aligned groups of four columns
template <class T, class Y>
bool by_quads(const GroupGemm<T, Y>& a) {
  auto ok = [](const void* p, size_t item) {
    return reinterpret_cast<uintptr_t>(p) % (4 * item) == 0;
  };
  if (a.act == Act::GLU)      // pairs
    return a.n % 4 == 0 && a.y_ld % 2 == 0 && a.y_gs % 2 == 0 &&
           reinterpret_cast<uintptr_t>(a.y) % (2 * sizeof(Y)) == 0;
  return a.n % 4 == 0 && a.y_ld % 4 == 0 && a.y_gs % 4 == 0 &&
         ok(a.y, sizeof(Y)) &&
         (!a.gate_each || (a.gate_ld % 4 == 0 && a.gate_gs % 4 == 0 &&
                           ok(a.gate, sizeof(T)))) &&
         a.t_ld % 4 == 0 && ok(a.table, sizeof(T));
}

template <class T, class Y>
int group_gemm_splits(const GroupGemm<T, Y>& a) {
  if constexpr (std::is_same_v<T, bf16_t>) {
    if (!pieces(a) || a.tiles != nullptr || a.groups != 1) return 1;
    const long groups = (long)((a.n + 31) / 32) * ((a.m + 15) / 16);
    int s = 1;     // every wave keeps at least two chunks
    while (s < 16 && groups * s < 128 && a.k / KC >= s * 16) s *= 2;
    return s;
  }
  return 1;
}

template <class T, class Y>
void launch_group_gemm(const GroupGemm<T, Y>& given, int tile,
                       hipStream_t stream) {
  GroupGemm<T, Y> a = given;
  a.quads = by_quads(a);
  const bool packed = a.tiles != nullptr, split = a.splits > 1;
  const int gz = packed ? 1 : split ? a.splits : a.groups;
  if (split) tile = 16;
  if constexpr (std::is_same_v<T, bf16_t>) {
    if (!packed && tile > 64 &&
        (!group_gemm_takes(a, tile) ||
         (long)((a.n + tile - 1) / tile) * ((a.m + tile - 1) / tile) * gz <
             128))
      tile = 64;
    if (group_gemm_takes(a, tile) && pieces(a)) {
      if (tile > 64) {
        launch_group_gemm_tile(a, tile, stream);
        return;
      }
      const bool flat = !packed && a.k <= 512 && tile == 64;
      auto groups = [&](int bn) {
        return (long)((a.n + bn - 1) / bn) *
               (packed ? a.max_tiles : (a.m + tile - 1) / tile) * gz;
      };
      // smaller tiles of unpacked rows while the chip is not full
      while (!packed && !flat && !split && tile > 16 && groups(64) < 512) tile /= 2;
      auto go = [&](auto fm, auto fn, auto kw, auto rw) {
        constexpr int FM = decltype(fm)::value, FN = decltype(fn)::value,
                      KW = decltype(kw)::value, RW = decltype(rw)::value;
        const dim3 grid((a.n + FN * 16 - 1) / (FN * 16),
                        packed ? a.max_tiles : (a.m + tile - 1) / tile, gz);
        by_act(a.act, [&](auto act) {
          group_gemm_stream_kernel<Y, decltype(act)::value, FM, FN, KW, RW>
              <<<grid, dim3(KW * RW * WAVE), 0, stream>>>(a);
        });
      };
      constexpr std::integral_constant<int, 1> c1{};
      constexpr std::integral_constant<int, 2> c2{};
      constexpr std::integral_constant<int, 4> c4{};
      constexpr std::integral_constant<int, 16> c16{};
      if (split) go(c1, c2, c4, c1);
      else if (flat) go(c1, c4, c1, c4);
      else if (tile == 16 && groups(64) < 256 && a.k >= 1024)
        go(c1, c2, c16, c1);
      else if (tile == 16) go(c1, c4, c4, c1);
      else if (tile == 32) go(c2, c4, c4, c1);
      else go(c4, c4, c4, c1);
      return;
    }
  }
  const int mt = packed ? a.max_tiles : (a.m + AT - 1) / AT;
  by_act(a.act, [&](auto act) {
    group_gemm_any_kernel<T, Y, decltype(act)::value>
        <<<dim3((a.n + AT - 1) / AT, mt, gz), 256, 0, stream>>>(a);
  });
}

#define INSTANTIATE(T, Y)                                                    \
  template int group_gemm_splits<T, Y>(const GroupGemm<T, Y>&);              \
  template bool group_gemm_takes<T, Y>(const GroupGemm<T, Y>&, int);         \
  template void launch_group_gemm<T, Y>(const GroupGemm<T, Y>&, int,         \
                                        hipStream_t);
INSTANTIATE(float, float)
INSTANTIATE(bf16_t, bf16_t)
INSTANTIATE(bf16_t, float)
