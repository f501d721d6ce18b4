// The gated delta rule over prompt portions, 32 tokens at a time on the matrix
// cores (formulas in delta.h).
//
// With b_t the decays' logarithms summed over the chunk's tokens up to t (per
// key channel), S the state at the chunk's start and k, q the unit vectors,
//
//   q~_t = q_t e^(b_t)    k~_t = k_t e^(b_t)    k^_s = k_s e^(b_end - b_s)
//   A = tril(k~ (k e^-b)^T, -1)    P = tril(q~ (k e^-b)^T)
//
// a chunk's updates u solve u_t = beta_t (v_t - S^T k~_t - sum_s A_ts u_s):
//
//   U = T (V - k~ S),  T = (1 + diag(beta) A)^-1 diag(beta)
//   O = q~ S + P U,    S <- diag(e^(b_end)) S + k^^T U
//
// Only products with S have to wait for the chunk before. So a first kernel
// makes q~, k~, k^, P and T of all chunks side by side, and leaves them as
// matrix-core operands. The second kernel walks a portion's chunks with a
// workgroup per (portion, head), a wave per 32 value columns, its columns of S
// in accumulators; the next chunk's operands are in flight meanwhile, and go
// through LDS as they are.
//
// Factors are split into bf16 high and low parts (2^-16 relative), V is bf16
// already. Contraction indices run in the order in which accumulators hold
// their rows ({0-3, 8-11 | 4-7, 12-15} of every 16), so S, V - k~ S and U
// feed the next product without a lane exchange.
//
// e^(-b) overflows when a channel decays by more than about e^-88 within the
// chunk. Beyond e^-60 A and P are summed directly, where no exponent is
// positive.
#include "chunk.h"
#include "delta.h"

#include <algorithm>

namespace {

constexpr int PREP = 256;           // threads of the first kernel

// Operands of one chunk and head: [..][high | low][lane][8]. Lane l has row
// l % 32 of the 32; with hi = l / 32, its 8 are 16 g + 4 hi + {0-3, 8-11} of
// the contraction index.
template <int DT>
struct Operands {
  short q[2 * DT][2][WAVE][8];      // tokens x channels, by 16 channels
  short k[2 * DT][2][WAVE][8];
  short kt[2 * DT][2][WAVE][8];     // channels x tokens, [2 tile + g]
  short p[2][2][WAVE][8];           // tokens x tokens, by 16
  short t[2][2][WAVE][8];
  float end[32 * DT];               // e^(b_end)
};

template <int DT>
struct PrepLds {
  static constexpr int DP = 32 * DT;
  struct Rows {
    alignas(16) float b[C][DP + 4];   // summed logs, base 2
    alignas(16) float k[C][DP + 4];   // unit keys
  };
  struct Scores {
    alignas(16) float l[C][C + 4];    // beta A
    float part[4][C][C + 1];          // A, P of the channels' halves; T, P
  };
  union {
    Rows rows;
    Scores scores;                    // once the rows are done with
  };
  float iq[C], beta[C];
  int direct;
};

// the place of a chunk among all of the batch's: entries' chunks never meet
DEV_INLINE long chunk_at(int row0, int e, int c) { return row0 / C + e + c; }

DEV_INLINE int ctr(int g, int hi, int j) {
  return 16 * g + 8 * (j >> 2) + 4 * hi + (j & 3);
}

DEV_INLINE void put_split(const float* f, short (*dst)[WAVE][8], int lane) {
  short8 h, l;
  split_rows<0>(f, &h, &l);
  *reinterpret_cast<short8*>(dst[0][lane]) = h;
  *reinterpret_cast<short8*>(dst[1][lane]) = l;
}

template <int DT>
__global__ __launch_bounds__(PREP)
void delta_prep_kernel(Delta<bf16_t> a, int h0,
                       Operands<DT>* __restrict__ ws) {
  constexpr int DP = 32 * DT;
  __shared__ PrepLds<DT> s;
  auto& b = s.rows.b;
  auto& k = s.rows.k;
  const int c = blockIdx.x, e = blockIdx.y, h = h0 + blockIdx.z;
  const Entry en = entry_of(a.seq_start, e);
  if (c * C >= en.n) return;
  const int len = min(C, en.n - c * C);
  const long row0 = en.row0 + c * C;
  Operands<DT>* w = ws + chunk_at(en.row0, e, c) * gridDim.z + blockIdx.z;
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid % WAVE;
  const int lo5 = lane & 31, hi = lane >> 5;
  const int nq = a.kv_heads * a.dim;
  const int head = h / (a.heads / a.kv_heads) * a.dim;
  const bf16_t* x = a.qkv + row0 * a.ld + head;
  const float rate = -a.rate[h];

  if (tid == 0) s.direct = 0;
  if (tid < C)
    s.beta[tid] = tid < len
        ? sigmoid_f(ld1(a.beta + (row0 + tid) * a.b_ld + h)) : 0.f;
  {
    // lengths of the vectors, four threads each: all of q, then all of k
    constexpr int PER = DP / 4;
    const int t = tid / 4 % C, at = tid % 4 * PER;
    const bool key = tid / 4 >= C;
    float f[PER], ss = 0.f;
    #pragma unroll
    for (int j = 0; j < PER; j += 4) {
      if (t < len && at + j < a.dim) {
        ldv<4>(x + t * a.ld + (key ? nq : 0) + at + j, f + j);
      } else {
        f[j] = f[j + 1] = f[j + 2] = f[j + 3] = 0.f;
      }
      ss += f[j] * f[j] + f[j + 1] * f[j + 1] + f[j + 2] * f[j + 2] +
            f[j + 3] * f[j + 3];
    }
    ss += __shfl_xor(ss, 1, WAVE);
    ss += __shfl_xor(ss, 2, WAVE);
    const float inv = 1.f / sqrtf(ss + UNIT_EPS);
    if (key) {
      #pragma unroll
      for (int j = 0; j < PER; ++j) k[t][at + j] = f[j] * inv;
    } else if (tid % 4 == 0) {
      s.iq[t] = inv / sqrtf((float)a.dim);
    }
  }
  {
    // summed logs: a few tokens per thread, then what lies ahead of them
    constexpr int N = C * DP / PREP;
    const int d = tid % DP, grp = tid / DP;
    const long at = (long)h * a.dim + min(d, a.dim - 1);
    const long ld = (long)a.heads * a.dim;
    const float zb = a.zb[at];
    float z[N], sum = 0.f, ahead = 0.f;
    #pragma unroll
    for (int j = 0; j < N; ++j)
      z[j] = a.z[(row0 + min(grp * N + j, len - 1)) * ld + at];
    #pragma unroll
    for (int j = 0; j < N; ++j) {
      if (grp * N + j < len && d < a.dim)
        sum += fmaxf(rate * softplus2_f(z[j] + zb), -160.f);   // 0 in float
      z[j] = sum;
    }
    b[grp * N + N - 1][d] = sum;
    __syncthreads();
    for (int p = 0; p < grp; ++p) ahead += b[p * N + N - 1][d];
    __syncthreads();
    #pragma unroll
    for (int j = 0; j < N; ++j) b[grp * N + j][d] = z[j] + ahead;
    if (grp == PREP / DP - 1) {
      w->end[d] = exp2_f(sum + ahead);
      if (sum + ahead < DIRECT_BELOW) s.direct = 1;
    }
  }
  __syncthreads();
  const bool direct = s.direct != 0;

  // k^: a channel per lane
  for (int it = wave; it < 2 * DT; it += PREP / WAVE) {
    const int d = 32 * (it >> 1) + lo5;
    const float end = b[C - 1][d];
    float f[8];
    #pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int t = ctr(it & 1, hi, j);
      f[j] = k[t][d] * exp2_f(end - b[t][d]);
    }
    put_split(f, w->kt[it], lane);
  }
  // q~ and P (odd waves) or k~ and A: a token per lane, every other 16
  // channels
  float16v acc = {};
  {
    const bool odd = wave & 1;
    for (int it = wave >> 1; it < 2 * DT; it += 2) {
      float f[8], n[8];
      #pragma unroll
      for (int g = 0; g < 8; g += 4) {
        const int d = ctr(it, hi, g);
        float sum[4], key[4], own[4] = {};
        ldv<4>(&b[lo5][d], sum);
        ldv<4>(&k[lo5][d], key);
        if (odd && lo5 < len && d < a.dim) ldv<4>(x + lo5 * a.ld + d, own);
        #pragma unroll
        for (int j = 0; j < 4; ++j) {
          const float y = odd ? own[j] * s.iq[lo5] : key[j];
          f[g + j] = y * exp2_f(sum[j]);
          n[g + j] = direct ? 0.f : key[j] * exp2_f(-sum[j]);
        }
      }
      short8 fh, fl, nh, nl;
      split_rows<0>(f, &fh, &fl);
      split_rows<0>(n, &nh, &nl);
      short (*dst)[WAVE][8] = odd ? w->q[it] : w->k[it];
      *reinterpret_cast<short8*>(dst[0][lane]) = fh;
      *reinterpret_cast<short8*>(dst[1][lane]) = fl;
      acc = mma(fh, nh, acc);
      acc = mma(fh, nl, acc);
      acc = mma(fl, nh, acc);
    }
  }
  constexpr int PAIRS = C * C / PREP;   // scores per thread
  float av[PAIRS], pv[PAIRS];
  if (direct) {
    #pragma unroll 1
    for (int i = 0; i < PAIRS; ++i) {
      const int t = (tid + i * PREP) / C, j = tid % C;
      float sa = 0.f, sp = 0.f;
      if (j <= t && t < len) {
        for (int d = 0; d < a.dim; ++d) {
          const float f = k[j][d] * exp2_f(b[t][d] - b[j][d]);
          sa += f * k[t][d];
          sp += f * ld1(x + t * a.ld + d);
        }
      }
      #pragma unroll
      for (int n = 0; n < PAIRS; ++n)
        if (n == i) { av[n] = sa; pv[n] = sp * s.iq[t]; }
    }
  }
  __syncthreads();
  auto& part = s.scores.part;
  auto& l = s.scores.l;
  #pragma unroll
  for (int r = 0; r < 16; ++r)
    part[wave][(r & 3) + 8 * (r >> 2) + 4 * hi][lo5] = acc[r];
  __syncthreads();
  #pragma unroll
  for (int i = 0; i < PAIRS; ++i) {
    const int t = (tid + i * PREP) / C, j = tid % C;
    if (!direct) {
      av[i] = part[0][t][j] + part[2][t][j];
      pv[i] = part[1][t][j] + part[3][t][j];
    }
    l[t][j] = j < t ? s.beta[t] * av[i] : 0.f;
    part[1][t][j] = j <= t ? pv[i] : 0.f;
  }
  __syncthreads();
  if (wave == 0) {
    // a column of the inverse per lane, from the top
    float inv[C];
    #pragma unroll
    for (int t = 0; t < C; ++t) {
      float v = t == lo5 ? 1.f : 0.f;
      #pragma unroll
      for (int j = 0; j < t; ++j) v -= l[t][j] * inv[j];
      inv[t] = v;
    }
    if (hi == 0) {
      #pragma unroll
      for (int t = 0; t < C; ++t) part[0][t][lo5] = inv[t] * s.beta[lo5];
    }
  } else if (wave < 3) {
    float f[8];
    #pragma unroll
    for (int j = 0; j < 8; ++j) f[j] = part[1][lo5][ctr(wave - 1, hi, j)];
    put_split(f, w->p[wave - 1], lane);
  }
  __syncthreads();
  if (wave < 2) {
    float f[8];
    #pragma unroll
    for (int j = 0; j < 8; ++j) f[j] = part[0][lo5][ctr(wave, hi, j)];
    put_split(f, w->t[wave], lane);
  }
}

// LDS written before is seen after; loads from memory may stay in flight.
DEV_INLINE void lds_barrier() {
  asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
}

DEV_INLINE short8 operand(const short* p, int lane) {
  return *reinterpret_cast<const short8*>(p + 8 * lane);
}

// NW waves; those past the value columns only help to load.
template <int DT, int NW>
__global__ __launch_bounds__(NW * WAVE, 2)
void delta_chunk_kernel(Delta<bf16_t> a, int h0,
                        const Operands<DT>* __restrict__ ws) {
  constexpr int THREADS = NW * WAVE, PIECES = sizeof(Operands<DT>) / 16;
  constexpr int MINE = (PIECES + THREADS - 1) / THREADS;
  __shared__ struct {
    alignas(16) Operands<DT> in;
    float ssq[NW][C];
  } s;
  const int e = blockIdx.x, h = h0 + blockIdx.y;
  const Entry en = entry_of(a.seq_start, e);
  if (en.n <= 0) return;
  const int tid = threadIdx.x;
  const int wave = __builtin_amdgcn_readfirstlane(tid / WAVE);
  const int lane = tid % WAVE, lo5 = lane & 31, hi = lane >> 5;
  const int col = wave * 32 + lo5;
  const bool col_ok = col < a.vdim;
  const int vcol = h * a.vdim + min(col, a.vdim - 1);
  const int slot = a.state_slots[e];
  float* state = slot < 0 ? nullptr
      : a.state + ((long)slot * a.heads + h) * a.dim * a.vdim;
  const bool held = state != nullptr && a.positions[en.row0] > 0;
  auto crow = [&](int r) { return (r & 3) + 8 * (r >> 2) + 4 * hi; };

  float16v st[DT];
  #pragma unroll
  for (int i = 0; i < DT; ++i)
    #pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int d = 32 * i + crow(r);
      st[i][r] = held && d < a.dim && col_ok ? state[d * a.vdim + col] : 0.f;
    }
  const float nweight = col_ok ? a.norm[col] * a.mult : 0.f;
  const float inv_vdim = 1.f / (float)a.vdim;
  // The portion's rows as bounded buffers: rows past its end read as zero and
  // are not written.
  auto buffer = [&](const bf16_t* p, long ld) {
    return __builtin_amdgcn_make_buffer_rsrc(
        const_cast<bf16_t*>(p) + en.row0 * ld, 0, (int)(en.n * ld * 2),
        BUFFER_FLAGS);
  };
  const auto v_in = buffer(a.qkv, a.ld), g_in = buffer(a.gate, a.g_ld);
  const auto out = buffer(a.out, a.out_ld);
  const int v_at = 2 * a.kv_heads * a.dim + vcol;
  auto load16 = [&](auto from, int ld, int at, int c0, unsigned* f) {
    const int off = ((c0 + 4 * hi) * ld + at) * 2;
    #pragma unroll
    for (int r = 0; r < 16; ++r)
      f[r] = __builtin_amdgcn_raw_buffer_load_b16(
          from, off + ((r & 3) + 8 * (r >> 2)) * ld * 2, 0, 0);
  };

  const Operands<DT>* w = ws + chunk_at(en.row0, e, 0) * gridDim.y +
                          blockIdx.y;
  short8 next[MINE];
  unsigned vn[16];
  auto load = [&](int c0) {
    const auto from = __builtin_amdgcn_make_buffer_rsrc(
        const_cast<Operands<DT>*>(w), 0, sizeof(Operands<DT>), BUFFER_FLAGS);
    #pragma unroll
    for (int i = 0; i < MINE; ++i)
      next[i] = __builtin_bit_cast(
          short8, __builtin_amdgcn_raw_buffer_load_b128(
              from, tid * 16, i * THREADS * 16, 0));
    load16(v_in, a.ld, v_at, c0, vn);
    w += gridDim.y;
  };
  auto to_lds = [&]() {
    short8* to = reinterpret_cast<short8*>(&s.in);
    #pragma unroll
    for (int i = 0; i < MINE; ++i)
      if (tid + i * THREADS < PIECES) to[tid + i * THREADS] = next[i];
  };
  load(0);
  to_lds();
  lds_barrier();

  for (int c0 = 0; c0 < en.n; c0 += C) {
    float16v ks, o = {};            // k~ S - V
    #pragma unroll
    for (int r = 0; r < 16; ++r) ks[r] = -__uint_as_float(vn[r] << 16);
    if (c0 + C < en.n) load(c0 + C);

    #pragma unroll
    for (int i = 0; i < DT; ++i) {
      #pragma unroll
      for (int y = 0; y < 2; ++y) {
        const int it = 2 * i + y;
        short8 sh, sl;
        if (y == 0) split_rows<0>(st[i], &sh, &sl);
        else split_rows<8>(st[i], &sh, &sl);
        const short8 kh = operand(s.in.k[it][0][0], lane);
        const short8 qh = operand(s.in.q[it][0][0], lane);
        ks = mma(kh, sh, ks);
        o = mma(qh, sh, o);
        ks = mma(kh, sl, ks);
        o = mma(qh, sl, o);
        ks = mma(operand(s.in.k[it][1][0], lane), sh, ks);
        o = mma(operand(s.in.q[it][1][0], lane), sh, o);
      }
      __builtin_amdgcn_sched_barrier(0);
    }
    unsigned g[16];
    load16(g_in, a.g_ld, vcol, c0, g);
    #pragma unroll
    for (int r = 0; r < 16; ++r) ks[r] = -ks[r];
    float16v u = {};
    #pragma unroll
    for (int y = 0; y < 2; ++y) {
      short8 rh, rl;
      if (y == 0) split_rows<0>(ks, &rh, &rl);
      else split_rows<8>(ks, &rh, &rl);
      const short8 th = operand(s.in.t[y][0][0], lane);
      u = mma(th, rh, u);
      u = mma(th, rl, u);
      u = mma(operand(s.in.t[y][1][0], lane), rh, u);
    }
    short8 uh[2], ul[2];
    split_rows<0>(u, &uh[0], &ul[0]);
    split_rows<8>(u, &uh[1], &ul[1]);
    #pragma unroll
    for (int y = 0; y < 2; ++y) {
      const short8 ph = operand(s.in.p[y][0][0], lane);
      o = mma(ph, uh[y], o);
      o = mma(ph, ul[y], o);
      o = mma(operand(s.in.p[y][1][0], lane), uh[y], o);
    }
    #pragma unroll
    for (int i = 0; i < DT; ++i) {
      #pragma unroll
      for (int r = 0; r < 16; r += 4) {
        float end[4];
        ldv<4>(&s.in.end[32 * i + crow(r)], end);
        #pragma unroll
        for (int j = 0; j < 4; ++j) st[i][r + j] *= end[j];
      }
      #pragma unroll
      for (int y = 0; y < 2; ++y) {
        const short8 kh = operand(s.in.kt[2 * i + y][0][0], lane);
        st[i] = mma(kh, uh[y], st[i]);
        st[i] = mma(kh, ul[y], st[i]);
        st[i] = mma(operand(s.in.kt[2 * i + y][1][0], lane), uh[y], st[i]);
      }
      __builtin_amdgcn_sched_barrier(0);
    }

    // sum of squares of each token over the wave's 32 columns: halve the set
    // of tokens a lane holds at every exchange
    float q[16];
    #pragma unroll
    for (int r = 0; r < 16; ++r) q[r] = col_ok ? o[r] * o[r] : 0.f;
    #pragma unroll
    for (int n = 8; n >= 1; n >>= 1) {
      #pragma unroll
      for (int r = 0; r < n; ++r) {
        const bool up = (lane & n) != 0;
        const float give = up ? q[r] : q[r + n];
        q[r] = (up ? q[r + n] : q[r]) + __shfl_xor(give, n, WAVE);
      }
    }
    q[0] += __shfl_xor(q[0], 16, WAVE);
    if ((lane & 16) == 0) s.ssq[wave][crow(lane & 15)] = q[0];
    lds_barrier();                  // the chunk's operands have been read
    if (c0 + C < en.n) to_lds();
    float ss[16];
    #pragma unroll
    for (int r = 0; r < 16; ++r) ss[r] = 0.f;
    #pragma unroll 1
    for (int n = 0; n < NW; ++n)
      #pragma unroll
      for (int r = 0; r < 16; r += 4) {
        float f[4];
        ldv<4>(&s.ssq[n][crow(r)], f);
        #pragma unroll
        for (int j = 0; j < 4; ++j) ss[r + j] += f[j];
      }
    lds_barrier();
    const int off = ((c0 + 4 * hi) * (int)a.out_ld + vcol) * 2;
    #pragma unroll
    for (int r = 0; r < 16; ++r) {
      const float f = o[r] * __builtin_amdgcn_rsqf(ss[r] * inv_vdim + a.eps) *
          nweight * __builtin_amdgcn_rcpf(
              1.f + exp2_f(-__uint_as_float(g[r] << 16) * LOG2E));
      __builtin_amdgcn_raw_buffer_store_b16(
          cvt_pk_bf16(f, f), out, col_ok
              ? off + ((r & 3) + 8 * (r >> 2)) * (int)a.out_ld * 2
              : OUT_OF_RANGE, 0, 0);
    }
  }
  if (state != nullptr && col_ok) {
    // addresses are formed anew: those of the beginning would have to stay in
    // registers all the while
    int to = col, dim = a.dim;
    asm volatile("" : "+v"(to), "+s"(dim));
    #pragma unroll
    for (int i = 0; i < DT; ++i)
      #pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int d = 32 * i + crow(r);
        if (d < dim) state[d * a.vdim + to] = st[i][r];
      }
  }
}

template <int DT>
void run(const Delta<bf16_t>& a, int entries, int max_len, int h0, int heads,
         void* ws, hipStream_t stream) {
  auto* ops = static_cast<Operands<DT>*>(ws);
  delta_prep_kernel<DT>
      <<<dim3((max_len + C - 1) / C, entries, heads), PREP, 0, stream>>>(
          a, h0, ops);
  const dim3 grid(entries, heads);
  if (a.vdim <= 128)
    delta_chunk_kernel<DT, 4><<<grid, 4 * WAVE, 0, stream>>>(a, h0, ops);
  else
    delta_chunk_kernel<DT, 8><<<grid, 8 * WAVE, 0, stream>>>(a, h0, ops);
}

int tiles(int dim) { return dim <= 32 ? 1 : dim <= 64 ? 2 : 4; }

}  // namespace

bool delta_chunk_supported(const Delta<bf16_t>& a, int max_len) {
  // a portion's rows are addressed with 32-bit offsets
  const long far = (max_len + C) * std::max({a.ld, a.out_ld, a.g_ld}) * 2;
  return a.dim <= 128 && a.dim % 4 == 0 && a.vdim <= 256 && a.ld % 4 == 0 &&
         reinterpret_cast<uintptr_t>(a.qkv) % 8 == 0 && far < OUT_OF_RANGE;
}

long delta_chunk_bytes(int dim, long rows, int entries) {
  const long chunks = rows / C + entries + 1;
  switch (tiles(dim)) {
    case 1: return chunks * sizeof(Operands<1>);
    case 2: return chunks * sizeof(Operands<2>);
    default: return chunks * sizeof(Operands<4>);
  }
}

void launch_delta_chunk(const Delta<bf16_t>& a, int entries, int max_len,
                        int h0, int heads, void* ws, hipStream_t stream) {
  switch (tiles(a.dim)) {
    case 1: run<1>(a, entries, max_len, h0, heads, ws, stream); break;
    case 2: run<2>(a, entries, max_len, h0, heads, ws, stream); break;
    default: run<4>(a, entries, max_len, h0, heads, ws, stream);
  }
}
