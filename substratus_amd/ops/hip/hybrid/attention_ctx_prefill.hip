// Attention of prompt portions over the paged bf16 cache (which already holds
// the portion's own keys and values), with a distance bias, a chunk mask,
// unequal key and value head sizes, a gated output, and softmax or sigmoid
// weights; the formulas are in attention_ctx.hip. Rows of a portion carry
// their absolute positions, so a prompt can be cut anywhere.
//
// The structure is that of attention_v5.hip: every wave owns 32 query rows
// kept in registers, 64 keys per step go through LDS, S^T = K Q^T leaves a
// lane with scores of its own query row only, and softmax stays in registers.
// Differences:
//   * K and V rows are gathered through the block table, page numbers one
//     step ahead of the rows they point at;
//   * a step's biases depend only on i - j: one window of the bias row per
//     step and workgroup in LDS;
//   * the weights enter the second product as bf16 high and low parts, i.e.
//     with 16 mantissa bits, so softmax weights keep more than bf16 carries;
//   * keys and values may also lie unpaged, projected for this step from what
//     the cache holds (FLAT), with a key part that all heads share;
//   * V is staged with keys 4..7 and 8..11 of every 16 exchanged, which is
//     the order in which the score accumulators hold them: weights need no
//     lane exchange before the second product.
#include "attention_ctx.h"

typedef __attribute__((ext_vector_type(8))) short short8;
typedef __attribute__((ext_vector_type(4))) short short4v;
typedef __attribute__((ext_vector_type(16))) float float16v;

namespace {

constexpr int CH = 64;          // keys per step
constexpr int PAGE = 16;

DEV_INLINE short4v tr16_read(const short* p) {
  return __builtin_amdgcn_ds_read_tr16_b64_v4i16(
      (__attribute__((address_space(3))) short4v*)p);
}

// KK: 16-wide steps of the key size; DC: 32-wide tiles of the value size
enum Kind {
  PLAIN,
  CAP,        // scores are capped
  SIGMOID,    // weights are sigmoids: no maximum, no sum
};

template <int KK, int DC, int WAVES, bool FLAT, Kind KIND>
__global__ __launch_bounds__(WAVES * WAVE)
void attn_ctx_prefill_kernel(AttnCtx<bf16_t> a) {
  constexpr int THREADS = WAVES * WAVE;
  constexpr int QT = WAVES * 32;            // query rows per workgroup
  constexpr int KROW = KK * 16 + 8;         // padded LDS row, in elements
  constexpr int BW = QT + CH - 1;           // distances met in one step
  constexpr int LK = (CH * KK * 2 + THREADS - 1) / THREADS;
  constexpr int LV = (CH * DC * 4 + THREADS - 1) / THREADS;
  static_assert(BW <= THREADS, "one bias per thread");

  __shared__ alignas(16) short s_k[2][CH][KROW];
  __shared__ alignas(16) short s_v[2][DC][CH / 32][2][2][16][16];
  __shared__ float s_b[2][THREADS];

  const int e = blockIdx.x, head = blockIdx.y;
  const int tile = gridDim.z - 1 - blockIdx.z;   // longest rows first
  const Entry en = entry_of(a.seq_start, e);
  const int q0_tile = tile * QT;
  if (q0_tile >= en.n) return;
  const int kvh = head / (a.heads / a.kv_heads);
  const int* bt = FLAT ? nullptr : a.block_table + (long)e * a.max_blocks;
  const int kd = a.dim - a.shared;               // a head's own key elements

  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid % WAVE;
  const int lo5 = lane & 31, hi = lane >> 5;
  const int pos0 = a.positions[en.row0];
  const int total = pos0 + en.n;                 // keys in the cache
  const int from = FLAT ? flat_from(a.window, pos0) : 0;
  const long flat0 = FLAT ? (long)a.ctx_start[e] - from : 0;
  const int qa0 = pos0 + q0_tile;                // first position of the tile
  const int qw0 = qa0 + wave * 32;               // first position of the wave
  const bool wave_live = qw0 < total;
  const int qpos = qw0 + lo5;
  const int row = min(q0_tile + wave * 32 + lo5, en.n - 1);
  const int lo = first_seen(a, qpos), lo_wave = first_seen(a, qw0);
  const int hi_wave = min(qw0 + 31, total - 1);
  // lo of the wave's last row: keys at or above it are inside every range
  const int lo_last = first_seen(a, qw0 + 31);
  const Pieces part(a.keep, first_seen(a, qa0),
                    (min(qa0 + QT, total) + CH - 1) / CH, CH);

  short8 qreg[KK];
  {
    const bf16_t* qp = a.q + (long)(en.row0 + row) * a.q_ld +
                       (long)head * a.dim;
    #pragma unroll
    for (int kk = 0; kk < KK; ++kk) {
      const int d = kk * 16 + hi * 8;
      qreg[kk] = d < a.dim ? *reinterpret_cast<const short8*>(qp + d)
                           : (short8){0, 0, 0, 0, 0, 0, 0, 0};
    }
  }
  float m = -INFINITY, l = 0.f;
  if (a.sink != nullptr) { m = a.sink[head] * LOG2E; l = 1.f; }
  float16v o_t[DC];
  #pragma unroll
  for (int c = 0; c < DC; ++c) o_t[c] = (float16v){};

  const float scale2 = a.scale * LOG2E;
  const float cap2 = a.cap * LOG2E;
  const float cscale = a.cap > 0.f ? 2.f * scale2 / a.cap : 0.f;
  int pgk[LK], pgv[LV];                          // page bases, -1: no key
  uint4 st_k[LK], st_v[LV];
  float st_b = 0.f;
  const float wb2 = KIND == SIGMOID ? a.wbias[head] * LOG2E : 0.f;

  auto pages = [&](int it) {
    const int st = part.at(it);
    #pragma unroll
    for (int i = 0; i < LK; ++i) {
      const int key = st * CH + (i * THREADS + tid) / (KK * 2);
      pgk[i] = it < part.n && key >= from && key < total &&
               key < st * CH + CH
          ? (FLAT ? key : bt[key / PAGE]) : -1;
    }
    #pragma unroll
    for (int i = 0; i < LV; ++i) {
      const int key = st * CH + (i * THREADS + tid) / (DC * 4);
      pgv[i] = it < part.n && key >= from && key < total &&
               key < st * CH + CH
          ? (FLAT ? key : bt[key / PAGE]) : -1;
    }
  };
  auto stage_load = [&](int it) {
    const int st = part.at(it);
    #pragma unroll
    for (int i = 0; i < LK; ++i) {
      const int f = i * THREADS + tid;
      const int r = f / (KK * 2), d = f % (KK * 2) * 8;
      st_k[i] = make_uint4(0, 0, 0, 0);
      if constexpr (FLAT) {
        const long at = flat0 + pgk[i];
        if (pgk[i] >= 0 && d < a.dim)
          st_k[i] = *reinterpret_cast<const uint4*>(
              d < kd ? a.kc + at * a.v_ld + (long)head * kd + d
                     : a.kr + at * a.shared + d - kd);
      } else if (pgk[i] >= 0 && d < a.dim)
        st_k[i] = *reinterpret_cast<const uint4*>(
            a.kc + (((long)pgk[i] * a.kv_heads + kvh) * PAGE +
                    (st * CH + r) % PAGE) * a.dim + d);
    }
    #pragma unroll
    for (int i = 0; i < LV; ++i) {
      const int f = i * THREADS + tid;
      const int r = f / (DC * 4), d = f % (DC * 4) * 8;
      st_v[i] = make_uint4(0, 0, 0, 0);
      if constexpr (FLAT) {
        if (pgv[i] >= 0 && d < a.vdim)
          st_v[i] = *reinterpret_cast<const uint4*>(
              a.vc + (flat0 + pgv[i]) * a.v_ld + (long)head * a.vdim + d);
      } else if (pgv[i] >= 0 && d < a.vdim)
        st_v[i] = *reinterpret_cast<const uint4*>(
            a.vc + (((long)pgv[i] * a.kv_heads + kvh) * PAGE +
                    (st * CH + r) % PAGE) * a.v_ld + d);
    }
    if (a.bias != nullptr || a.r1 != nullptr)
      st_b = distance_bias2(a, head, qa0 - (st * CH + CH - 1) + tid);
    if constexpr (KIND == SIGMOID) st_b += wb2;
  };
  auto stage_write = [&](int buf) {
    #pragma unroll
    for (int i = 0; i < LK; ++i) {
      const int f = i * THREADS + tid;
      const int r = f / (KK * 2), d = f % (KK * 2) * 8;
      if (r < CH) *reinterpret_cast<uint4*>(&s_k[buf][r][d]) = st_k[i];
    }
    #pragma unroll
    for (int i = 0; i < LV; ++i) {
      const int f = i * THREADS + tid;
      const int r = f / (DC * 4), col = f % (DC * 4) * 8;
      if (r < CH) {
        // bits 2 and 3 of the key exchanged
        const int kx = (r & 3) | (r & 4) << 1 | (r & 8) >> 1;
        const int ir = ((kx & 8) ? 8 : 0) + ((col % 32) / 16) * 4 + (kx & 3);
        *reinterpret_cast<uint4*>(
            &s_v[buf][col / 32][r / 32][(r % 32) / 16][(kx >> 2) & 1][ir]
                [col % 16]) = st_v[i];
      }
    }
    s_b[buf][tid] = st_b;
  };

  pages(0);
  stage_load(0);
  pages(1);
  stage_write(0);
  __syncthreads();

  for (int it = 0; it < part.n; ++it) {
    const int cur = it & 1;
    if (it + 1 < part.n) {
      stage_load(it + 1);
      pages(it + 2);
    }
    const int kbase = part.at(it) * CH;
    if (wave_live && kbase <= hi_wave &&
        (kbase + CH > lo_wave || kbase < a.keep)) {
      float16v sacc[CH / 32];
      #pragma unroll
      for (int sc = 0; sc < CH / 32; ++sc) {
        sacc[sc] = (float16v){};
        #pragma unroll
        for (int kk = 0; kk < KK; ++kk) {
          const short8 ka = *reinterpret_cast<const short8*>(
              &s_k[cur][sc * 32 + lo5][kk * 16 + hi * 8]);
          sacc[sc] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(
              ka, qreg[kk], sacc[sc], 0, 0, 0);
        }
      }
      float sv[CH / 32][16];
      const float* bw = &s_b[cur][wave * 32 + lo5 + CH - 1 - 4 * hi];
      #pragma unroll
      for (int sc = 0; sc < CH / 32; ++sc)
        #pragma unroll
        for (int r = 0; r < 16; ++r)
          sv[sc][r] = (KIND == CAP ? cap2 * tanh_exp2(sacc[sc][r] * cscale)
                                   : sacc[sc][r] * scale2) +
                      bw[-(sc * 32 + (r & 3) + 8 * (r >> 2))];
      // steps inside every row's range need no mask
      if (kbase < lo_last || kbase + CH - 1 > qw0 || qw0 + 31 >= total) {
        #pragma unroll
        for (int sc = 0; sc < CH / 32; ++sc)
          #pragma unroll
          for (int r = 0; r < 16; ++r) {
            const int kpos =
                kbase + sc * 32 + (r & 3) + 8 * (r >> 2) + 4 * hi;
            if (!(kpos <= qpos && (kpos >= lo || kpos < a.keep) &&
                  qpos < total))
              sv[sc][r] = -INFINITY;
          }
      }
      if constexpr (KIND != SIGMOID) {
        float mloc = -INFINITY;
        #pragma unroll
        for (int sc = 0; sc < CH / 32; ++sc)
          #pragma unroll
          for (int r = 0; r < 16; ++r) mloc = fmaxf(mloc, sv[sc][r]);
        mloc = fmaxf(mloc, __shfl_xor(mloc, 32, WAVE));
        // the running maximum moves only when a score exceeds it by 2^8
        if (!__all(mloc == -INFINITY || mloc - m <= 8.f)) {
          const float mn = fmaxf(m, mloc);
          const float keep = m == -INFINITY ? 0.f
                                            : __builtin_amdgcn_exp2f(m - mn);
          m = mn;
          l *= keep;
          #pragma unroll
          for (int c = 0; c < DC; ++c)
            #pragma unroll
            for (int r = 0; r < 16; ++r) o_t[c][r] *= keep;
        }
      }
      float sum = 0.f;
      #pragma unroll
      for (int sc = 0; sc < CH / 32; ++sc) {
        #pragma unroll
        for (int g = 0; g < 2; ++g) {
          unsigned wh[4], wl[4];
          #pragma unroll
          for (int i = 0; i < 4; ++i) {
            const float s0 = sv[sc][8 * g + 2 * i];
            const float s1 = sv[sc][8 * g + 2 * i + 1];
            float p0, p1;
            if constexpr (KIND == SIGMOID) {
              p0 = sigmoid_exp2(s0);
              p1 = sigmoid_exp2(s1);
            } else {
              p0 = s0 == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(s0 - m);
              p1 = s1 == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(s1 - m);
              sum += p0 + p1;
            }
            wh[i] = cvt_pk_bf16(p0, p1);
            const float2 back = unpack_bf16x2(wh[i]);
            wl[i] = cvt_pk_bf16(p0 - back.x, p1 - back.y);
          }
          const short8 ph = *reinterpret_cast<const short8*>(wh);
          const short8 pl = *reinterpret_cast<const short8*>(wl);
          #pragma unroll
          for (int c = 0; c < DC; ++c) {
            const short4v v0 =
                tr16_read(&s_v[cur][c][sc][g][0][0][0] + lane * 4);
            const short4v v1 =
                tr16_read(&s_v[cur][c][sc][g][1][0][0] + lane * 4);
            short8 vt;
            #pragma unroll
            for (int j = 0; j < 4; ++j) { vt[j] = v0[j]; vt[4 + j] = v1[j]; }
            o_t[c] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vt, ph, o_t[c],
                                                             0, 0, 0);
            o_t[c] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vt, pl, o_t[c],
                                                             0, 0, 0);
          }
        }
      }
      if constexpr (KIND != SIGMOID) l += sum + __shfl_xor(sum, 32, WAVE);
    }
    if (it + 1 < part.n) stage_write(cur ^ 1);
    __syncthreads();
  }

  if (wave_live && qpos < total) {
    const long r = en.row0 + row;
    float f = KIND == SIGMOID ? a.mult : a.mult / l;
    if (!(FLAT && a.gate_each) && a.gate != nullptr)
      f *= sigmoid_f(bf2f(a.gate[r * a.g_ld + head]));
    bf16_t* op = a.out + r * a.out_ld + (long)head * a.vdim;
    #pragma unroll
    for (int c = 0; c < DC; ++c) {
      #pragma unroll
      for (int rr = 0; rr < 4; ++rr) {
        const int d0 = c * 32 + 8 * rr + 4 * hi;
        if (d0 < a.vdim) {
          float o[4];
          #pragma unroll
          for (int j = 0; j < 4; ++j) o[j] = o_t[c][rr * 4 + j] * f;
          if (FLAT && a.gate_each && a.gate != nullptr) {
            float g[4];
            ldv<4>(a.gate + r * a.g_ld + (long)head * a.vdim + d0, g);
            #pragma unroll
            for (int j = 0; j < 4; ++j) o[j] *= sigmoid_f(g[j]);
          }
          if (a.quads) {
            stv<4>(op + d0, o);
          } else {
            #pragma unroll
            for (int j = 0; j < 4; ++j) st1(op + d0 + j, o[j]);
          }
        }
      }
    }
  }
}

}  // namespace

bool attn_ctx_prefill_supported(int dim, int vdim, int block_size) {
  return dim % 8 == 0 && vdim % 8 == 0 && dim <= 256 && vdim <= 256 &&
         block_size == PAGE;
}

void launch_attn_ctx_prefill(const AttnCtx<bf16_t>& a, int entries,
                             int max_len, hipStream_t stream) {
  auto go = [&](auto kk, auto dc, auto waves) {
    constexpr int W = decltype(waves)::value;
    const dim3 grid(entries, a.heads, (max_len + W * 32 - 1) / (W * 32));
    constexpr int K = decltype(kk)::value, D = decltype(dc)::value;
    const dim3 block(W * WAVE);
    if (a.ctx_start != nullptr)
      attn_ctx_prefill_kernel<K, D, W, true, PLAIN>
          <<<grid, block, 0, stream>>>(a);
    else if (a.wbias != nullptr)
      attn_ctx_prefill_kernel<K, D, W, false, SIGMOID>
          <<<grid, block, 0, stream>>>(a);
    else if (a.cap > 0.f)
      attn_ctx_prefill_kernel<K, D, W, false, CAP>
          <<<grid, block, 0, stream>>>(a);
    else
      attn_ctx_prefill_kernel<K, D, W, false, PLAIN>
          <<<grid, block, 0, stream>>>(a);
  };
  using std::integral_constant;
  auto by_dc = [&](auto kk) {
    if (a.vdim <= 64)
      go(kk, integral_constant<int, 2>{}, integral_constant<int, 8>{});
    else if (a.vdim <= 128)
      go(kk, integral_constant<int, 4>{}, integral_constant<int, 8>{});
    else
      go(kk, integral_constant<int, 8>{}, integral_constant<int, 4>{});
  };
  if (a.dim <= 64) by_dc(integral_constant<int, 4>{});
  else if (a.dim <= 96) by_dc(integral_constant<int, 6>{});
  else if (a.dim <= 128) by_dc(integral_constant<int, 8>{});
  else if (a.dim <= 192) by_dc(integral_constant<int, 12>{});
  else by_dc(integral_constant<int, 16>{});
}
