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
#include "gla.h"

typedef __attribute__((ext_vector_type(8))) short short8;
typedef __attribute__((ext_vector_type(4))) short short4v;
typedef __attribute__((ext_vector_type(16))) float float16v;

namespace {

constexpr int C = 32;               // tokens per chunk
constexpr int MAXW = 8;             // waves per workgroup
constexpr int MAXRANK = 64;
constexpr float DIRECT_BELOW = -60.f;

// place of element i (of 16) so that a lane half reads 8 in a row
DEV_INLINE int perm16(int i) {
  return (i & ~12) | (i & 4) << 1 | (i & 8) >> 1;
}

DEV_INLINE short bf_bits(float f) {
  const bf16_t b = f2bf(f);
  return *reinterpret_cast<const short*>(&b);
}

DEV_INLINE float bits_f(short s) {
  return __uint_as_float((unsigned)(unsigned short)s << 16);
}

DEV_INLINE void split_bf(float f, short* hi, short* lo) {
  *hi = bf_bits(f);
  *lo = bf_bits(f - bits_f(*hi));
}

DEV_INLINE unsigned cvt_pk_bf16(float lo, float hi) {
  unsigned r;
  asm("v_cvt_pk_bf16_f32 %0, %1, %2" : "=v"(r) : "v"(lo), "v"(hi));
  return r;
}

// 8 consecutive accumulator rows as bf16 high and low operand parts
template <int AT>
DEV_INLINE void split_rows(const float16v& f, short8* hi, short8* lo) {
  unsigned h[4], l[4];
  #pragma unroll
  for (int i = 0; i < 4; ++i) {
    const float f0 = f[AT + 2 * i], f1 = f[AT + 2 * i + 1];
    h[i] = cvt_pk_bf16(f0, f1);
    const float2 back = unpack_bf16x2(h[i]);
    l[i] = cvt_pk_bf16(f0 - back.x, f1 - back.y);
  }
  *hi = *reinterpret_cast<const short8*>(h);
  *lo = *reinterpret_cast<const short8*>(l);
}

DEV_INLINE float16v mma(short8 a, short8 b, float16v c) {
  return __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b, c, 0, 0, 0);
}

template <int DT>
struct Lds {
  static constexpr int DP = DT * 32;
  alignas(16) short q[2][C][DP + 8];      // [hi|lo][token][channel, permuted]
  alignas(16) short k[2][C][DP + 8];
  alignas(16) short kt[2][DP][C + 8];     // [hi|lo][channel][token, permuted]
  float end[DP];                          // e^(b_end)
  float total[DP];                        // b_end summed over the segment
  float a1[C][MAXRANK + 4];
  float ssq[MAXW][C];
  int direct[2];
};

// OUT: write outputs and the final state; else leave the segment's own state
// and decay in the workspace.
template <int DT, bool OUT>
__global__ __launch_bounds__(MAXW * WAVE)
void gla_chunk_kernel(Gla<bf16_t> a, int nseg, int seg_len,
                      float* __restrict__ ws, float* __restrict__ ws_decay) {
  constexpr int DP = DT * 32;
  __shared__ Lds<DT> s;
  const int e = blockIdx.x / nseg, seg = blockIdx.x % nseg, h = blockIdx.y;
  const Entry en = entry_of(a.seq_start, e);
  const int t0 = seg * seg_len;
  if (t0 >= en.n || (!OUT && t0 + seg_len >= en.n)) return;
  const int len = min(seg_len, en.n - t0);
  const bool last = t0 + seg_len >= en.n;
  const int nw = blockDim.x / WAVE, tid = threadIdx.x;
  const int wave = tid / WAVE, lane = tid % WAVE;
  const int lo5 = lane & 31, hi = lane >> 5;
  const int col = wave * 32 + lo5;
  const bool col_ok = col < a.vdim;
  const long row0 = en.row0 + t0;
  const int slot = a.state_slots[e];
  const long hstate = (long)a.dim * a.vdim;
  float* slot_state = slot < 0 ? nullptr
      : a.state + ((long)slot * a.heads + h) * hstate;
  float* seg_state =
      ws + (((long)e * nseg + seg) * a.heads + h) * hstate;

  // accumulator row r of channel tile i is channel 32i + crow(r)
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
          ? init[(long)d * a.vdim + col] : 0.f;
    }
  const float nweight = OUT && col_ok ? a.norm[col] : 0.f;
  if (tid < 2) s.direct[tid] = 0;
  for (int d = tid; d < DP; d += blockDim.x) s.total[d] = 0.f;

  auto stage_a1 = [&](int c0) {
    for (int i = tid; i < C * a.rank; i += blockDim.x) {
      const int t = i / a.rank, r = i % a.rank;
      s.a1[t][r] = c0 + t < len
          ? bf2f(a.x[(row0 + c0 + t) * a.ld + a.a_off + r]) : 0.f;
    }
  };
  stage_a1(0);
  __syncthreads();

  // Logs of decays, summed along the chunk, for 16 channels at a time:
  // lane = (channel, quarter of the tokens); f(d, tq, b[8], b_end).
  auto decays = [&](int c0, auto f) {
    const int dl = lane & 15, tq = lane >> 4;
    for (int d0 = wave * 16; d0 < DP; d0 += nw * 16) {
      const int d = d0 + dl;
      float b[8];
      if (d < a.dim) {
        const int c = h * a.dim + d;
        const float z0 = a.a2b[c];
        #pragma unroll
        for (int i = 0; i < 8; ++i) b[i] = z0;
        for (int r = 0; r < a.rank; ++r) {
          const float w = a.a2[(long)c * a.rank + r];
          #pragma unroll
          for (int i = 0; i < 8; ++i) b[i] += s.a1[tq * 8 + i][r] * w;
        }
        #pragma unroll
        for (int i = 0; i < 8; ++i) {
          const float z = b[i];
          const float ls = fminf(z, 0.f) -
                           __logf(1.f + __expf(-fabsf(z)));
          b[i] = c0 + tq * 8 + i < len ? ls * a.inv_tau : 0.f;
        }
      } else {
        #pragma unroll
        for (int i = 0; i < 8; ++i) b[i] = 0.f;
      }
      #pragma unroll
      for (int i = 1; i < 8; ++i) b[i] += b[i - 1];
      float before = 0.f;             // sum over earlier quarters
      const float mine = b[7];
      #pragma unroll
      for (int k = 1; k < 4; ++k) {
        const float u = __shfl(mine, dl + 16 * (k - 1), WAVE);
        if (tq >= k) before += u;
      }
      #pragma unroll
      for (int i = 0; i < 8; ++i) b[i] += before;
      const float end = __shfl(b[7], 48 + dl, WAVE);
      f(d, tq, b, end);
    }
  };

  for (int c0 = 0; c0 < len; c0 += C) {
    const int par = (c0 / C) & 1;
    // V as the second operand of both products, straight from the rows:
    // token order as in the accumulators
    short8 vf[2];
    #pragma unroll
    for (int g = 0; g < 2; ++g)
      #pragma unroll
      for (int j = 0; j < 8; ++j) {
        const int t = c0 + 16 * g + crow(j);
        vf[g][j] = t < len && col_ok
            ? *reinterpret_cast<const short*>(
                  a.x + (row0 + t) * a.ld + a.v_off + h * a.vdim + col)
            : (short)0;
      }

    decays(c0, [&](int d, int tq, const float* b, float end) {
      const int c = h * a.dim + d;
      const int dpos = (d & ~15) | perm16(d & 15);
      short kh[8], kl[8];
      #pragma unroll
      for (int i = 0; i < 8; ++i) {
        const int t = tq * 8 + i;
        const bool ok = c0 + t < len && d < a.dim;
        const bf16_t* x = a.x + (row0 + (ok ? c0 + t : 0)) * a.ld;
        const float k = ok ? bf2f(x[a.k_off + c]) : 0.f;
        split_bf(k * __expf(end - b[i]), &kh[i], &kl[i]);
        if (OUT) {
          const float q = ok ? bf2f(x[c]) * a.qscale : 0.f;
          short ph, pl;
          split_bf(q * __expf(b[i]), &ph, &pl);
          s.q[0][t][dpos] = ph;
          s.q[1][t][dpos] = pl;
          split_bf(k * __expf(-b[i]), &ph, &pl);
          s.k[0][t][dpos] = ph;
          s.k[1][t][dpos] = pl;
        }
      }
      // tokens 8tq..8tq+7 of the permuted order: two runs of four
      const int at = (tq >> 1) * 16 + (tq & 1) * 4;
      #pragma unroll
      for (int u = 0; u < 2; ++u) {
        *reinterpret_cast<short4v*>(&s.kt[0][d][at + 8 * u]) =
            (short4v){kh[4 * u], kh[4 * u + 1], kh[4 * u + 2], kh[4 * u + 3]};
        *reinterpret_cast<short4v*>(&s.kt[1][d][at + 8 * u]) =
            (short4v){kl[4 * u], kl[4 * u + 1], kl[4 * u + 2], kl[4 * u + 3]};
      }
      if (tq == 3) {
        s.end[d] = __expf(end);
        if (!OUT) s.total[d] += end;
        if (OUT && end < DIRECT_BELOW) s.direct[par] = 1;
      }
    });
    __syncthreads();
    const bool direct = OUT && s.direct[par] != 0;    // uniform
    if (OUT && tid == 0) s.direct[par ^ 1] = 0;

    float16v o = {};
    if (OUT) {
      float16v at = {};             // A^T: row = key token, column = query
      if (direct) {
        // the summed logs take the place of k~
        float (*sb)[DP + 8] = reinterpret_cast<float (*)[DP + 8]>(s.k);
        decays(c0, [&](int d, int tq, const float* b, float) {
          #pragma unroll
          for (int i = 0; i < 8; ++i) sb[tq * 8 + i][d] = b[i];
        });
        __syncthreads();
        if (c0 + lo5 < len) {
          const bf16_t* q = a.x + (row0 + c0 + lo5) * a.ld + h * a.dim;
          #pragma unroll
          for (int r = 0; r < 16; ++r) {
            const int ks = crow(r);
            if (ks > lo5) continue;
            const bf16_t* k =
                a.x + (row0 + c0 + ks) * a.ld + a.k_off + h * a.dim;
            float acc = 0.f;
            for (int d = 0; d < a.dim; ++d)
              acc += bf2f(q[d]) * a.qscale * bf2f(k[d]) *
                     __expf(sb[lo5][d] - sb[ks][d]);
            at[r] = acc;
          }
        }
      }
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
          if (!direct) {
            const short8 kh =
                *reinterpret_cast<const short8*>(&s.k[0][lo5][d]);
            const short8 kl =
                *reinterpret_cast<const short8*>(&s.k[1][lo5][d]);
            at = mma(kh, qh, at);
            at = mma(kh, ql, at);
            at = mma(kl, qh, at);
          }
        }
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
      for (int r = 0; r < 16; ++r) st[i][r] *= s.end[32 * i + crow(r)];
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
    if (c0 + C < len) stage_a1(c0 + C);

    if (OUT) {
      // sum of squares of each token over the wave's 32 columns: halve the
      // set of tokens a lane holds at every exchange
      float q[16];
      #pragma unroll
      for (int r = 0; r < 16; ++r) q[r] = o[r] * o[r];
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
    if (OUT) {
      #pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int t = crow(r);
        float ss = 0.f;
        for (int w = 0; w < nw; ++w) ss += s.ssq[w][t];
        if (c0 + t < len && col_ok) {
          const long row = row0 + c0 + t;
          const float g =
              bf2f(a.x[row * a.ld + a.g_off + h * a.vdim + col]);
          const float inv = 1.f / sqrtf(ss / (float)a.vdim + a.eps);
          a.out[(row * a.heads + h) * a.vdim + col] =
              f2bf(o[r] * inv * nweight * (g / (1.f + __expf(-g))));
        }
      }
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
          expf(s.total[d]);
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

template <int DT>
void run(const Gla<bf16_t>& a, int entries, int max_len, int nseg, float* ws,
         float* ws_decay, hipStream_t stream) {
  const int waves = (a.vdim + 31) / 32;
  int seg_len = (max_len + nseg - 1) / nseg;
  seg_len = (seg_len + C - 1) / C * C;
  const dim3 grid(entries * nseg, a.heads), block(waves * WAVE);
  if (nseg > 1) {
    gla_chunk_kernel<DT, false><<<grid, block, 0, stream>>>(
        a, nseg, seg_len, ws, ws_decay);
    gla_scan_kernel<<<dim3((a.dim * a.vdim + 255) / 256, entries, a.heads),
                      dim3(256), 0, stream>>>(a, nseg, seg_len, ws, ws_decay);
  }
  gla_chunk_kernel<DT, true><<<grid, block, 0, stream>>>(
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
  if (a.dim <= 32) run<1>(a, entries, max_len, nseg, ws, ws_decay, stream);
  else if (a.dim <= 64) run<2>(a, entries, max_len, nseg, ws, ws_decay, stream);
  else if (a.dim <= 128) run<4>(a, entries, max_len, nseg, ws, ws_decay, stream);
  else run<8>(a, entries, max_len, nseg, ws, ws_decay, stream);
}
