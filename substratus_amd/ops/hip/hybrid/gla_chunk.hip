// Gated linear attention over prompt portions, 32 tokens at a time on the
// matrix cores (formulas in gla.h).
//
// With b_t the decays' logarithms summed over the chunk's tokens up to t
// (per key channel) and S the state at the chunk's start, a chunk is
//
//   q~_t = q_t e^(b_t)    k~_s = k_s e^(-b_s)    k^_s = k_s e^(b_end - b_s)
//   O    = tril(q~ k~^T) V + q~ S
//   S   <- diag(e^(b_end)) S + k^^T V
//
// One workgroup per (segment of a portion, head); wave w owns value columns
// 32w .. 32w+31 and keeps its columns of S in accumulators for the whole
// segment. All waves together make q~, k~ and k^ for a chunk in LDS.
//
// What enters the recurrence counts as 32-bit data, so every factor that is
// not a bf16 projection is split into bf16 high and low parts and products
// are summed as hi*hi + hi*lo + lo*hi (2^-16 relative). V is bf16 already.
//
// The order of a contraction index is free as long as both operands agree,
// so channels and tokens are laid out in LDS in the order in which 32x32
// accumulators hold their rows ({0-3, 8-11 | 4-7, 12-15} of every 16):
// S and the masked score block feed the next product without a lane exchange.
//
// e^(-b_s) overflows when a channel decays by more than about e^-88 within
// 32 tokens. A chunk in which some channel decays by more than e^-60 takes
// its score block by direct summation of q k e^(b_t - b_s) instead, in which
// no exponent is positive.
//
// Long portions are cut into segments that run side by side: a first pass
// leaves each segment's own state and total decay, a scan turns those into
// the segments' initial states, and the second pass writes outputs.
#include "chunk.h"
#include "gla.h"

#include <type_traits>

namespace {

constexpr int MAXW = 8;             // waves per workgroup
constexpr int MAXRANK = 64;

// place of element i (of 16) so that a lane half reads 8 in a row
DEV_INLINE int perm16(int i) {
  return (i & ~12) | (i & 4) << 1 | (i & 8) >> 1;
}

DEV_INLINE unsigned raw16(bf16_t x) {
  return *reinterpret_cast<unsigned short*>(&x);
}

template <int DT>
struct Lds {
  static constexpr int DP = DT * 32;
  alignas(16) short q[2][C][DP + 8];      // [hi|lo][token][channel, permuted]
  alignas(16) short k[2][C][DP + 8];
  alignas(16) short kt[2][DP][C + 8];     // [hi|lo][channel][token, permuted]
  alignas(16) float end[DP];              // e^(b_end)
  float total[DP];                        // b_end (base 2) over the segment
  alignas(16) float ssq[MAXW][C];
  float score[C][C + 1];                  // [key][query] of a direct chunk
  int direct[2];
};

// OUT: write outputs and the final state; else leave the segment's own state
// and decay in the workspace. CONST: constant decays (gla.h).
//
// Making q~, k~ and k^ is divided into tasks of 32 channels: one kind makes
// q~, the other k~ and k^. Both begin with the channel block's decays, a
// product of the rows' A1 h with A2 on the matrix cores whose accumulators
// hold a channel per lane and the tokens in registers. A wave takes its tasks
// with their rows loaded a chunk ahead.
template <int DT, bool OUT, bool CONST>
__global__ __launch_bounds__(MAXW * WAVE)
void gla_chunk_kernel(Gla<bf16_t> a, int nseg, int seg_len,
                      float* __restrict__ ws, float* __restrict__ ws_decay) {
  constexpr int DP = DT * 32;
  constexpr int TASKS = OUT ? 2 * DT : DT;
  __shared__ Lds<DT> s;
  const int e = blockIdx.x / nseg, seg = blockIdx.x % nseg, h = blockIdx.y;
  const Entry en = entry_of(a.seq_start, e);
  const int t0 = seg * seg_len;
  if (t0 >= en.n || (!OUT && t0 + seg_len >= en.n)) return;
  const int len = min(seg_len, en.n - t0);
  const bool last = t0 + seg_len >= en.n;
  const int nw = blockDim.x / WAVE, tid = threadIdx.x;
  const int wave = __builtin_amdgcn_readfirstlane(tid / WAVE);
  const int lane = tid % WAVE;
  const int lo5 = lane & 31, hi = lane >> 5;
  const int col = wave * 32 + lo5;
  const bool col_ok = col < a.vdim;
  const long row0 = en.row0 + t0;
  const int ld = (int)a.ld;
  const int slot = a.state_slots[e];
  const long hstate = (long)a.dim * a.vdim;
  float* slot_state = slot < 0 ? nullptr
      : a.state + ((long)slot * a.heads + h) * hstate;
  float* seg_state =
      ws + (((long)e * nseg + seg) * a.heads + h) * hstate;

  // accumulator row r of a 32-row tile
  auto crow = [&](int r) { return (r & 3) + 8 * (r >> 2) + 4 * hi; };

  float16v st[DT];
  const float* init = !OUT ? nullptr
      : nseg > 1 ? seg_state
      : a.positions[en.row0] > 0 ? slot_state : nullptr;
  #pragma unroll
  for (int i = 0; i < DT; ++i)
    #pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int d = 32 * i + crow(r);
      st[i][r] = init != nullptr && d < a.dim && col_ok
          ? init[d * a.vdim + col] : 0.f;
    }
  const float inv_vdim = 1.f / (float)a.vdim;
  const float nweight = OUT && !CONST && col_ok ? a.norm[col] : 0.f;
  // per token, base 2
  const float ldecay = CONST ? fmaxf(log2f(a.decay[h]), -1e4f) : 0.f;
  // a projected value as it enters the recurrence
  auto value = [&](unsigned raw) {
    const float f = __uint_as_float(raw << 16);
    if constexpr (CONST) return silu_as<bf16_t>(f);
    else return f;
  };
  if (tid < 2) s.direct[tid] = 0;
  for (int d = tid; d < DP; d += blockDim.x) s.total[d] = 0.f;
  __syncthreads();

  // The segment's rows as a bounded buffer: rows past its end read as zero
  // and are not written, so the last chunk needs no code of its own.
  const auto rows_in = __builtin_amdgcn_make_buffer_rsrc(
      const_cast<bf16_t*>(a.x) + row0 * ld, 0, len * ld * 2, BUFFER_FLAGS);
  const int out_ld = a.heads * a.vdim;
  const auto rows_out = __builtin_amdgcn_make_buffer_rsrc(
      a.out + row0 * out_ld, 0, OUT ? len * out_ld * 2 : 0, BUFFER_FLAGS);

  // Column `at` of the rows of tokens crow(r) of the chunk at c0. (One word
  // per value until use: packing them would wait for the loads.)
  auto load16 = [&](int c0, int at, unsigned* f) {
    const int off = ((c0 + 4 * hi) * ld + at) * 2;
    #pragma unroll
    for (int r = 0; r < 16; ++r)
      f[r] = __builtin_amdgcn_raw_buffer_load_b16(
          rows_in, off + ((r & 3) + 8 * (r >> 2)) * ld * 2, 0, 0);
  };
  // a task's rows: q (kind 0) or k (kind 1) of channel block `tile`
  auto load_task = [&](int c0, int task, unsigned* f) {
    const int tile = OUT ? task >> 1 : task, kind = OUT ? task & 1 : 1;
    load16(c0, (kind ? a.k_off : 0) + h * a.dim +
               min(32 * tile + lo5, a.dim - 1), f);
  };
  auto load_a1 = [&](int c0, int r0, unsigned* f) {
    if constexpr (CONST) return;
    const int off = ((c0 + lo5) * ld + a.a_off) * 2;
    #pragma unroll
    for (int j = 0; j < 8; ++j)
      f[j] = __builtin_amdgcn_raw_buffer_load_b16(
          rows_in, off + min(r0 + 8 * hi + j, a.rank - 1) * 2, 0, 0);
  };
  auto pack8 = [&](const unsigned* f) {
    unsigned w[4];
    #pragma unroll
    for (int j = 0; j < 4; ++j) w[j] = f[2 * j] | f[2 * j + 1] << 16;
    return *reinterpret_cast<const short8*>(w);
  };
  // rows of A2 for channel block `tile`, zero outside rank and head
  auto load_a2 = [&](int tile, int r0, short8* wh, short8* wl) {
    if constexpr (CONST) return;
    const int d = 32 * tile + lo5;
    const float* w2 = a.a2 + (long)(h * a.dim + min(d, a.dim - 1)) * a.rank;
    float w[8];
    #pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int r = r0 + 8 * hi + j;
      w[j] = w2[min(r, a.rank - 1)];
      if (r >= a.rank) w[j] = 0.f;
    }
    split_rows<0>(w, wh, wl);
  };
  // Summed logs (base 2) of the decays, b[r] for token crow(r); returns their end.
  // The first 16 inner columns come loaded.
  auto logs = [&](int c0, int tile, const unsigned* a1, short8 wh, short8 wl,
                  float* b) {
    const int d = 32 * tile + lo5;
    if constexpr (CONST) {
      const float by = d < a.dim ? ldecay : 0.f;
      #pragma unroll
      for (int r = 0; r < 16; ++r) b[r] = by * min(crow(r) + 1, len - c0);
      return by * min(C, len - c0);
    }
    float16v z = {};
    z = mma(pack8(a1), wh, z);
    z = mma(pack8(a1), wl, z);
    for (int r0 = 16; r0 < a.rank; r0 += 16) {
      unsigned more[8];
      load_a1(c0, r0, more);
      load_a2(tile, r0, &wh, &wl);
      z = mma(pack8(more), wh, z);
      z = mma(pack8(more), wl, z);
    }
    const float zb = a.a2b[h * a.dim + min(d, a.dim - 1)];
    const int lim = d < a.dim ? len - c0 - 4 * hi : 0;
    float gs[4], og[4];
    #pragma unroll
    for (int g = 0; g < 4; ++g) {
      #pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int r = 4 * g + j;
        const float v = (z[r] + zb) * LOG2E;
        const float ls = fminf(v, 0.f) -
                         __builtin_amdgcn_logf(1.f + exp2_f(-fabsf(v)));
        b[r] = ls * (8 * g + j < lim ? a.inv_tau : 0.f);
        if (j > 0) b[r] += b[r - 1];
      }
      gs[g] = b[4 * g + 3];
      og[g] = __shfl_xor(gs[g], 32, WAVE);
    }
    float before = 0.f;          // over the tokens ahead of each four
    #pragma unroll
    for (int g = 0; g < 4; ++g) {
      const float add = before + (hi ? og[g] : 0.f);
      #pragma unroll
      for (int j = 0; j < 4; ++j) b[4 * g + j] += add;
      before += gs[g] + og[g];
    }
    return before;
  };
  // s.q / s.k rows from values per token
  auto put_rows = [&](short (*dst)[C][DP + 8], int tile, const float* f) {
    const int at = 32 * tile + (lo5 & 16) + perm16(lo5 & 15);
    #pragma unroll
    for (int r = 0; r < 16; r += 2) {
      unsigned ph, pl;
      split_pair(f[r], f[r + 1], &ph, &pl);
      dst[0][crow(r)][at] = (short)ph;
      dst[0][crow(r + 1)][at] = (short)(ph >> 16);
      dst[1][crow(r)][at] = (short)pl;
      dst[1][crow(r + 1)][at] = (short)(pl >> 16);
    }
  };
  auto do_task = [&](int c0, int task, const unsigned* a1, short8 wh,
                     short8 wl, const unsigned* rows) {
    const int tile = OUT ? task >> 1 : task, kind = OUT ? task & 1 : 1;
    const int d = 32 * tile + lo5;
    float b[16], f[16];
    const float end = logs(c0, tile, a1, wh, wl, b);
    if (kind == 0) {
      const float scale = d < a.dim ? a.qscale : 0.f;
      #pragma unroll
      for (int r = 0; r < 16; ++r)
        f[r] = value(rows[r]) * scale * exp2_f(b[r]);
      put_rows(s.q, tile, f);
      return;
    }
    const int lim = d < a.dim ? len - c0 - 4 * hi : 0;
    float k[16];
    #pragma unroll
    for (int r = 0; r < 16; ++r)
      k[r] = (r & 3) + 8 * (r >> 2) < lim
          ? value(rows[r]) : 0.f;
    #pragma unroll
    for (int r = 0; r < 16; ++r) f[r] = k[r] * exp2_f(end - b[r]);
    short8 kh, kl;
    split_rows<0>(f, &kh, &kl);
    *reinterpret_cast<short8*>(&s.kt[0][d][8 * hi]) = kh;
    *reinterpret_cast<short8*>(&s.kt[1][d][8 * hi]) = kl;
    split_rows<8>(f, &kh, &kl);
    *reinterpret_cast<short8*>(&s.kt[0][d][16 + 8 * hi]) = kh;
    *reinterpret_cast<short8*>(&s.kt[1][d][16 + 8 * hi]) = kl;
    if (OUT) {
      #pragma unroll
      for (int r = 0; r < 16; ++r) f[r] = k[r] * exp2_f(-b[r]);
      put_rows(s.k, tile, f);
    }
    if (hi == 0) {
      s.end[d] = exp2_f(end);
      if (!OUT) s.total[d] += end;
    }
    if (OUT && end < DIRECT_BELOW) s.direct[(c0 / C) & 1] = 1;
  };

  // the wave's first task comes loaded; its part of A2 stays for the segment
  const int vcol = h * a.vdim + min(col, a.vdim - 1);
  unsigned task_rows[16], vraw[16], a1[8] = {};
  short8 wh0 = {}, wl0 = {};
  if (wave < TASKS) {
    load_task(0, wave, task_rows);
    load_a2(OUT ? wave >> 1 : wave, 0, &wh0, &wl0);
  }
  load_a1(0, 0, a1);
  load16(0, a.v_off + vcol, vraw);

  for (int c0 = 0; c0 < len; c0 += C) {
    const int par = (c0 / C) & 1;
    #pragma unroll 1
    for (int task = wave; task < TASKS; task += nw) {
      short8 wh = wh0, wl = wl0;
      if (task != wave) {
        load_task(c0, task, task_rows);
        load_a2(OUT ? task >> 1 : task, 0, &wh, &wl);
      }
      do_task(c0, task, a1, wh, wl, task_rows);
    }
    // V as the second operand of both products: token order as in the
    // accumulators
    if constexpr (CONST) {
      #pragma unroll
      for (int r = 0; r < 16; ++r)
        vraw[r] = __float_as_uint(value(vraw[r])) >> 16;
    }
    const short8 vf[2] = {pack8(vraw), pack8(vraw + 8)};
    __syncthreads();
    const bool direct = OUT && s.direct[par] != 0;    // uniform
    if (OUT && tid == 0) s.direct[par ^ 1] = 0;

    if (direct) {
      // the summed logs take the place of k~
      float (*sb)[DP + 8] = reinterpret_cast<float (*)[DP + 8]>(s.k);
      for (int tile = wave; tile < DT; tile += nw) {
        float b[16];
        short8 wh, wl;
        load_a2(tile, 0, &wh, &wl);
        logs(c0, tile, a1, wh, wl, b);
        #pragma unroll
        for (int r = 0; r < 16; ++r) sb[crow(r)][32 * tile + lo5] = b[r];
      }
      __syncthreads();
      const bf16_t* x = a.x + (row0 + c0) * ld + h * a.dim;
      for (int i = tid; i < C * C; i += blockDim.x) {
        const int ks = i / C, qt = i % C;
        float acc = 0.f;
        if (ks <= qt && c0 + qt < len) {
          for (int d = 0; d < a.dim; ++d)
            acc += value(raw16(x[qt * ld + d])) * a.qscale *
                   value(raw16(x[ks * ld + a.k_off + d])) *
                   exp2_f(sb[qt][d] - sb[ks][d]);
        }
        s.score[ks][qt] = acc;
      }
      __syncthreads();
    }

    unsigned graw[16];
    if (OUT && !CONST) load16(c0, a.g_off + vcol, graw);
    if (c0 + C < len) {
      if (wave < TASKS) load_task(c0 + C, wave, task_rows);
      load_a1(c0 + C, 0, a1);
      load16(c0 + C, a.v_off + vcol, vraw);
    }

    float16v o = {};
    if (OUT) {
      float16v at = {};             // A^T: row = key token, column = query
      #pragma unroll
      for (int i = 0; i < DT; ++i) {
        #pragma unroll
        for (int g = 0; g < 2; ++g) {
          const int d = 32 * i + 16 * g + 8 * hi;
          const short8 qh = *reinterpret_cast<const short8*>(&s.q[0][lo5][d]);
          const short8 ql = *reinterpret_cast<const short8*>(&s.q[1][lo5][d]);
          short8 sh, sl;
          if (g == 0) split_rows<0>(st[i], &sh, &sl);
          else split_rows<8>(st[i], &sh, &sl);
          o = mma(qh, sh, o);
          o = mma(qh, sl, o);
          o = mma(ql, sh, o);
          const short8 kh = *reinterpret_cast<const short8*>(&s.k[0][lo5][d]);
          const short8 kl = *reinterpret_cast<const short8*>(&s.k[1][lo5][d]);
          at = mma(kh, qh, at);
          at = mma(kh, ql, at);
          at = mma(kl, qh, at);
        }
      }
      if (direct) {
        #pragma unroll
        for (int r = 0; r < 16; ++r) at[r] = s.score[crow(r)][lo5];
      }
      #pragma unroll
      for (int r = 0; r < 16; ++r)
        if (crow(r) > lo5) at[r] = 0.f;
      short8 ph, pl;
      split_rows<0>(at, &ph, &pl);
      o = mma(ph, vf[0], o);
      o = mma(pl, vf[0], o);
      split_rows<8>(at, &ph, &pl);
      o = mma(ph, vf[1], o);
      o = mma(pl, vf[1], o);
    }

    #pragma unroll
    for (int i = 0; i < DT; ++i) {
      #pragma unroll
      for (int g = 0; g < 4; ++g) {
        const float4 f = *reinterpret_cast<const float4*>(
            &s.end[32 * i + 8 * g + 4 * hi]);
        st[i][4 * g] *= f.x; st[i][4 * g + 1] *= f.y;
        st[i][4 * g + 2] *= f.z; st[i][4 * g + 3] *= f.w;
      }
      #pragma unroll
      for (int g = 0; g < 2; ++g) {
        const short8 kh = *reinterpret_cast<const short8*>(
            &s.kt[0][32 * i + lo5][16 * g + 8 * hi]);
        const short8 kl = *reinterpret_cast<const short8*>(
            &s.kt[1][32 * i + lo5][16 * g + 8 * hi]);
        st[i] = mma(kh, vf[g], st[i]);
        st[i] = mma(kl, vf[g], st[i]);
      }
    }

    if (OUT && !CONST) {
      // sum of squares of each token over the wave's 32 columns: halve the
      // set of tokens a lane holds at every exchange
      float q[16];
      #pragma unroll
      for (int r = 0; r < 16; ++r) q[r] = col_ok ? o[r] * o[r] : 0.f;
      #pragma unroll
      for (int w = 8; w >= 1; w >>= 1) {
        #pragma unroll
        for (int r = 0; r < w; ++r) {
          const bool up = (lane & w) != 0;
          const float give = up ? q[r] : q[r + w];
          q[r] = (up ? q[r + w] : q[r]) + __shfl_xor(give, w, WAVE);
        }
      }
      // lane now holds accumulator row lane & 15, over 16 of 32 columns
      q[0] += __shfl_xor(q[0], 16, WAVE);
      if ((lane & 16) == 0) s.ssq[wave][crow(lane & 15)] = q[0];
    }
    __syncthreads();
    if constexpr (OUT && !CONST) {
      float ss[16];
      #pragma unroll
      for (int r = 0; r < 16; ++r) ss[r] = 0.f;
      #pragma unroll 2
      for (int w = 0; w < nw; ++w)
        #pragma unroll
        for (int g = 0; g < 4; ++g) {
          const float4 f = *reinterpret_cast<const float4*>(
              &s.ssq[w][8 * g + 4 * hi]);
          ss[4 * g] += f.x; ss[4 * g + 1] += f.y;
          ss[4 * g + 2] += f.z; ss[4 * g + 3] += f.w;
        }
      #pragma unroll
      for (int r = 0; r < 16; ++r) {
        const float g = __uint_as_float(graw[r] << 16);
        o[r] *= __builtin_amdgcn_rsqf(ss[r] * inv_vdim + a.eps) * nweight *
                g * __builtin_amdgcn_rcpf(1.f + exp2_f(-g * LOG2E));
      }
    }
    if constexpr (OUT) {
      const int off = col_ok
          ? ((c0 + 4 * hi) * out_ld + h * a.vdim + col) * 2 : OUT_OF_RANGE;
      #pragma unroll
      for (int r = 0; r < 16; ++r)
        __builtin_amdgcn_raw_buffer_store_b16(
            cvt_pk_bf16(o[r], o[r]), rows_out,
            col_ok ? off + ((r & 3) + 8 * (r >> 2)) * out_ld * 2 : off, 0, 0);
      // ssq is written again only after the next chunk's barrier
    }
  }

  float* fin = !OUT ? ws + (((long)e * nseg + seg + 1) * a.heads + h) * hstate
      : last ? slot_state : nullptr;
  if (fin != nullptr && col_ok) {
    #pragma unroll
    for (int i = 0; i < DT; ++i)
      #pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int d = 32 * i + crow(r);
        if (d < a.dim) fin[(long)d * a.vdim + col] = st[i][r];
      }
  }
  if (!OUT) {
    for (int d = tid; d < a.dim; d += blockDim.x)
      ws_decay[(((long)e * nseg + seg) * a.heads + h) * a.dim + d] =
          exp2_f(s.total[d]);
  }
}

// ws[e][c] (c >= 1) holds the own state of segment c - 1; afterwards ws[e][c]
// is the state at the start of segment c.
__global__ __launch_bounds__(256)
void gla_scan_kernel(Gla<bf16_t> a, int nseg, int seg_len,
                     float* __restrict__ ws,
                     const float* __restrict__ ws_decay) {
  const int e = blockIdx.y, h = blockIdx.z;
  const int hstate = a.dim * a.vdim;
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i >= hstate) return;
  const Entry en = entry_of(a.seq_start, e);
  const int slot = a.state_slots[e];
  float s = slot >= 0 && a.positions[en.row0] > 0
      ? a.state[((long)slot * a.heads + h) * hstate + i] : 0.f;
  for (int c = 0; c < nseg && c * seg_len < en.n; ++c) {
    const long at = ((long)e * nseg + c) * a.heads + h;
    if (c > 0)
      s = s * ws_decay[(at - a.heads) * a.dim + i / a.vdim] +
          ws[at * hstate + i];
    ws[at * hstate + i] = s;
  }
}

template <int DT, bool CONST>
void run(const Gla<bf16_t>& a, int entries, int max_len, int nseg, float* ws,
         float* ws_decay, hipStream_t stream) {
  const int waves = (a.vdim + 31) / 32;
  int seg_len = (max_len + nseg - 1) / nseg;
  seg_len = (seg_len + C - 1) / C * C;
  const dim3 grid(entries * nseg, a.heads), block(waves * WAVE);
  if (nseg > 1) {
    gla_chunk_kernel<DT, false, CONST><<<grid, block, 0, stream>>>(
        a, nseg, seg_len, ws, ws_decay);
    gla_scan_kernel<<<dim3((a.dim * a.vdim + 255) / 256, entries, a.heads),
                      dim3(256), 0, stream>>>(a, nseg, seg_len, ws, ws_decay);
  }
  gla_chunk_kernel<DT, true, CONST><<<grid, block, 0, stream>>>(
      a, nseg, seg_len, ws, ws_decay);
}

}  // namespace

bool gla_chunk_supported(int dim, int vdim, int rank) {
  return dim <= 256 && vdim <= 32 * MAXW && rank <= MAXRANK;
}

// Segments per portion: enough workgroups for two per CU, segments of at
// least 256 tokens.
int gla_chunk_segments(int entries, int heads, int max_len) {
  int n = 1;
  while ((long)entries * heads * n < 512 && max_len >= n * 2 * 256) n *= 2;
  return n;
}

void launch_gla_chunk(const Gla<bf16_t>& a, int entries, int max_len, int nseg,
                      float* ws, float* ws_decay, hipStream_t stream) {
  auto go = [&](auto dt) {
    constexpr int DT = decltype(dt)::value;
    if (a.decay != nullptr)
      run<DT, true>(a, entries, max_len, nseg, ws, ws_decay, stream);
    else
      run<DT, false>(a, entries, max_len, nseg, ws, ws_decay, stream);
  };
  using std::integral_constant;
  if (a.dim <= 32) go(integral_constant<int, 1>{});
  else if (a.dim <= 64) go(integral_constant<int, 2>{});
  else if (a.dim <= 128) go(integral_constant<int, 4>{});
  else go(integral_constant<int, 8>{});
}
