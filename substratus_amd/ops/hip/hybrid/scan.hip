// Selective scans over single tokens and portions of prompts (formulas in
// scan.h). A thread holds NP numbers of one channel's state in registers,
// `lanes` neighbouring threads a whole channel. B and C, which all channels
// share, go through LDS a few tokens at a time; u, z and the gate are loaded
// TB tokens ahead of their use.
//
// Long portions are cut into segments that run side by side: a first pass
// leaves each segment's own state and its summed step sizes, from which a
// second kernel forms the segments' initial states (the decay over a segment
// is exp(a * sum of dt)); the last pass writes outputs.
#include "scan.h"

namespace {

constexpr int BLOCK = 256;
constexpr int TB = 4;              // tokens loaded at once
constexpr float LOG2E = 1.44269504088896340736f;
constexpr float LN2 = 0.69314718055994530942f;

DEV_INLINE float exp2_f(float x) { return __builtin_amdgcn_exp2f(x); }

template <int NP>
DEV_INLINE void ld_state(const float* p, int n, bool vec, float* s) {
  if (vec && n == NP) {
    #pragma unroll
    for (int i = 0; i < NP; i += 4) ldv<4>(p + i, s + i);
  } else {
    #pragma unroll
    for (int i = 0; i < NP; ++i) s[i] = i < n ? p[i] : 0.f;
  }
}

template <int NP>
DEV_INLINE void st_state(float* p, int n, bool vec, const float* s) {
  if (vec && n == NP) {
    #pragma unroll
    for (int i = 0; i < NP; i += 4) stv<4>(p + i, s + i);
  } else {
    #pragma unroll
    for (int i = 0; i < NP; ++i)
      if (i < n) p[i] = s[i];
  }
}

// OUT: write outputs and the final state; else leave the segment's own state
// and step sizes in the workspace. tt: tokens of B and C in LDS, a multiple
// of TB.
template <class T, int NP, bool OUT>
__global__ __launch_bounds__(BLOCK)
void scan_kernel(Scan<T> a, int lanes, int tt, int nseg, int seg_len,
                 float* __restrict__ ws, float* __restrict__ ws_dt) {
  extern __shared__ float4 s_mem[];
  float* s_bc = reinterpret_cast<float*>(s_mem);   // [tt][B | C], padded
  const int npad = lanes * NP;
  const int e = blockIdx.y / nseg, seg = blockIdx.y % nseg;
  const Entry en = entry_of(a.seq_start, e);
  const int t0 = seg * seg_len;
  if (t0 >= en.n || (!OUT && t0 + seg_len >= en.n)) return;
  const int len = min(seg_len, en.n - t0);
  const bool last = t0 + seg_len >= en.n;
  const int tid = threadIdx.x, part = tid % lanes;
  const int chan = blockIdx.x * (BLOCK / lanes) + tid / lanes;
  const bool there = chan < a.channels;
  const int c = min(chan, a.channels - 1);
  const int i0 = part * NP, ni = min(max(a.n - i0, 0), NP);
  const bool vec = a.n % 4 == 0 && NP % 4 == 0;
  const long row0 = en.row0 + t0;
  const int slot = a.state_slots[e];
  float* slot_state = slot < 0 ? nullptr
      : a.state + ((long)slot * a.channels + c) * a.n + i0;
  float* seg_state =
      ws + (((long)e * nseg + seg) * a.channels + c) * a.n + i0;

  float s[NP], a2[NP];
  ld_state<NP>(a.a + (long)c * a.n + i0, ni, vec, a2);
  #pragma unroll
  for (int i = 0; i < NP; ++i) { a2[i] *= LOG2E; s[i] = 0.f; }
  const float* init = !OUT ? nullptr
      : nseg > 1 ? seg_state
      : a.positions[en.row0] > 0 ? slot_state : nullptr;
  if (init != nullptr) ld_state<NP>(init, ni, vec, s);
  const float zb = a.zb[c], d = a.d[c];
  float total = 0.f;

  // the next TB tokens' values, on their way while these are computed
  T un[TB], gn[TB];
  float zn[TB];
  auto load = [&](int t) {
    #pragma unroll
    for (int j = 0; j < TB; ++j) {
      const long r = row0 + min(t + j, len - 1);
      un[j] = a.u[r * a.channels + c];
      zn[j] = a.z[r * a.channels + c];
      if (OUT) gn[j] = a.gate[r * a.g_ld + c];
    }
  };
  load(0);
  for (int b0 = 0; b0 < len; b0 += tt) {
    const int nt = min(tt, len - b0);
    __syncthreads();
    for (int i = tid; i < nt * 2 * npad; i += BLOCK) {
      const int t = i / (2 * npad), k = i % (2 * npad);
      const int at = k < npad ? k : k - npad;
      s_bc[i] = at < a.n
          ? ld1(a.low + (row0 + b0 + t) * a.low_ld + (k < npad ? at
                                                              : a.n + at))
          : 0.f;
    }
    __syncthreads();
    for (int t1 = 0; t1 < nt; t1 += TB) {
      float u[TB], z[TB], g[TB];
      #pragma unroll
      for (int j = 0; j < TB; ++j) {
        u[j] = ld1(&un[j]);
        z[j] = zn[j];
        if (OUT) g[j] = ld1(&gn[j]);
      }
      load(b0 + t1 + TB);
      #pragma unroll
      for (int j = 0; j < TB; ++j) {
        if (t1 + j >= nt) break;
        const float dt = std::is_same_v<T, float>
            ? softplus_f(z[j] + zb) : softplus2_f(z[j] + zb) * LN2;
        const float dtu = dt * u[j];
        const float* bc = s_bc + (t1 + j) * 2 * npad + i0;
        float y = 0.f;
        #pragma unroll
        for (int i = 0; i < NP; i += 4) {
          float b[4], cc[4];
          ldv<4>(bc + i, b);
          if (OUT) ldv<4>(bc + npad + i, cc);
          #pragma unroll
          for (int k = 0; k < 4; ++k) {
            s[i + k] = exp2_f(dt * a2[i + k]) * s[i + k] + dtu * b[k];
            if (OUT) y += s[i + k] * cc[k];
          }
        }
        if (!OUT) total += dt;
        if (OUT) {
          for (int off = 1; off < lanes; off <<= 1)
            y += __shfl_xor(y, off, WAVE);
          if (part == 0 && there)
            st1(a.out + (row0 + b0 + t1 + j) * a.out_ld + c,
                (y + d * u[j]) * (std::is_same_v<T, float>
                                      ? g[j] * sigmoid_f(g[j])
                                      : fast_silu_f(g[j])));
        }
      }
    }
  }
  if (!there) return;
  if (!OUT) {
    st_state<NP>(seg_state + (long)a.channels * a.n, ni, vec, s);
    if (part == 0) ws_dt[((long)e * nseg + seg) * a.channels + c] = total;
  } else if (last && slot_state != nullptr) {
    st_state<NP>(slot_state, ni, vec, s);
  }
}

// ws[e][k] (k >= 1) holds the own state of segment k - 1; afterwards ws[e][k]
// is the state at the start of segment k.
template <class T>
__global__ __launch_bounds__(BLOCK)
void scan_join_kernel(Scan<T> a, int nseg, int seg_len, float* __restrict__ ws,
                      const float* __restrict__ ws_dt) {
  const int e = blockIdx.y;
  const long size = (long)a.channels * a.n;
  const long i = (long)blockIdx.x * BLOCK + threadIdx.x;
  if (i >= size) return;
  const Entry en = entry_of(a.seq_start, e);
  const int slot = a.state_slots[e];
  const float a2 = a.a[i] * LOG2E;
  float s = slot >= 0 && a.positions[en.row0] > 0
      ? a.state[slot * size + i] : 0.f;
  for (int k = 0; k < nseg && k * seg_len < en.n; ++k) {
    const long at = (long)e * nseg + k;
    if (k > 0)
      s = s * exp2_f(ws_dt[(at - 1) * a.channels + i / a.n] * a2) +
          ws[at * size + i];
    ws[at * size + i] = s;
  }
}

int lanes_of(int n, int np) {
  int l = 1;
  while (l * np < n) l *= 2;
  return l;
}

long waves_of(int entries, int channels, int n, int np) {
  return (long)entries * channels * lanes_of(n, np) / WAVE;
}

// Numbers of a state per thread: fewer where waves are few.
int np_of(int entries, int channels, int n) {
  int np = n <= 4 ? 4 : n <= 8 ? 8 : 16;
  if (np == 16 && n <= 256 && waves_of(entries, channels, n, np) < 2048)
    np = 8;
  return np;                       // n <= 512: at most 32 lanes
}

}  // namespace

// Segments per portion: at least two waves per SIMD.
// (The first pass over segments costs as much as half of the scan.)
int scan_segments(int entries, int channels, int n, int max_len) {
  const long waves = waves_of(entries, channels, n,
                              np_of(entries, channels, n));
  int k = 1;
  while (waves * k < 2048 && max_len >= k * 2 * 64 && k < 128) k *= 2;
  return k;
}

template <class T>
void launch_scan(const Scan<T>& a, int entries, int max_len, int nseg,
                 float* ws, float* ws_dt, hipStream_t stream) {
  const int seg_len = (max_len + nseg - 1) / nseg;
  auto go = [&](auto np) {
    constexpr int NP = decltype(np)::value;
    const int lanes = lanes_of(a.n, NP), per = BLOCK / lanes;
    // B and C of tt tokens in at most 32 KiB
    int tt = 32;
    while (tt > TB && tt * 2 * lanes * NP > 8192) tt /= 2;
    const dim3 grid((a.channels + per - 1) / per, entries * nseg);
    const size_t lds = sizeof(float) * tt * 2 * lanes * NP;
    if (nseg > 1) {
      scan_kernel<T, NP, false><<<grid, BLOCK, lds, stream>>>(
          a, lanes, tt, nseg, seg_len, ws, ws_dt);
      scan_join_kernel<T>
          <<<dim3(((long)a.channels * a.n + BLOCK - 1) / BLOCK, entries),
             BLOCK, 0, stream>>>(a, nseg, seg_len, ws, ws_dt);
    }
    scan_kernel<T, NP, true><<<grid, BLOCK, lds, stream>>>(
        a, lanes, tt, nseg, seg_len, ws, ws_dt);
  };
  switch (np_of(entries, a.channels, a.n)) {
    case 4: go(std::integral_constant<int, 4>{}); break;
    case 8: go(std::integral_constant<int, 8>{}); break;
    default: go(std::integral_constant<int, 16>{});
  }
}

template void launch_scan<float>(const Scan<float>&, int, int, int, float*,
                                 float*, hipStream_t);
template void launch_scan<bf16_t>(const Scan<bf16_t>&, int, int, int, float*,
                                  float*, hipStream_t);
