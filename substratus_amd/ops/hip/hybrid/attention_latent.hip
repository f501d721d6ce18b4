// Attention in the latent space over the paged bf16 cache: all query heads
// share one key per token, and its first `vdim` columns are the value. For
// single tokens and portions of prompts: an entry's queries are its rows
// times its heads, in that order, and a workgroup takes 16 * MT of them.
//
// A step is 64 keys, four pages, one per wave. A page is one contiguous piece
// of memory and goes to LDS as it is (direct loads, the next step's in
// flight), except that the 16-byte pieces of a row are permuted by the row,
// so that neither of the two products meets bank conflicts:
//   scores   S^T = K Q^T: each wave its own page's 16 keys, queries in
//            registers throughout;
//   values   O^T = V^T P^T: each wave a quarter of the columns, for all 64
//            keys. V^T is read by the transposing LDS loads from the same
//            rows; weights come from the other waves through LDS, as bf16
//            high and low parts, so they keep 16 bits.
// Maximum and sum of a query are shared by the waves through LDS. Long
// contexts are split over workgroups and merged by attn_ctx_merge.
#include "attention_ctx.h"

namespace {

typedef __attribute__((ext_vector_type(8))) short short8;
typedef __attribute__((ext_vector_type(4))) short short4v;
typedef __attribute__((ext_vector_type(4))) float float4v;

constexpr int NW = 4;
constexpr int PAGE = 16;
constexpr int CH = NW * PAGE;
constexpr float NEG = -1e30f;   // "no key yet": finite, so differences are too

DEV_INLINE void load_to_lds(const void* g, void* lds) {
  __builtin_amdgcn_global_load_lds(
      (const __attribute__((address_space(1))) unsigned int*)g,
      (__attribute__((address_space(3))) unsigned int*)lds, 16, 0, 0);
}

// Waits for LDS only: the next step's loads stay in flight.
DEV_INLINE void lds_barrier() {
  asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
}

// KS: 32-wide steps of the key size (even); CT: 16-wide column tiles per wave
template <int KS, int CT, int MT>
__global__ __launch_bounds__(NW * WAVE, 1)
void attn_latent_kernel(AttnCtx<bf16_t> a, int splits,
                        float* __restrict__ part_o,
                        float* __restrict__ part_ml) {
  constexpr int QT = MT * 16;
  constexpr int RC = KS * 4;                     // 16-byte pieces per LDS row
  constexpr int PP = CH + 8;                     // padded row of weights
  __shared__ alignas(16) uint4 s_c[2][CH * RC];
  __shared__ alignas(16) short s_p[2][QT][PP];   // high and low parts
  __shared__ float s_m[NW][QT];

  const int e = blockIdx.x, split = blockIdx.z;
  const Entry en = entry_of(a.seq_start, e);
  const int q0 = blockIdx.y * QT, nq = en.n * a.heads;
  if (q0 >= nq) return;
  const int* bt = a.block_table + (long)e * a.max_blocks;
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
  const int lo = lane & 15, grp = lane >> 4;
  const int pos0 = a.positions[en.row0];
  const int last = pos0 + (min(q0 + QT, nq) - 1) / a.heads;  // of the tile
  const int pages = last / PAGE + 1;
  const int steps = (pages + NW - 1) / NW;
  const int st0 = (int)((long)steps * split / splits),
            st1 = (int)((long)steps * (split + 1) / splits);

  // queries: lane = query, 8 consecutive elements
  short8 q[MT][KS];
  int qpos[MT];
  #pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    const int qi = min(q0 + mt * 16 + lo, nq - 1);
    const int r = qi / a.heads, h = qi % a.heads;
    qpos[mt] = pos0 + r;
    const bf16_t* qp = a.q + (long)(en.row0 + r) * a.q_ld + (long)h * a.dim;
    #pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const int d = ks * 32 + grp * 8;
      q[mt][ks] = d < a.dim ? *reinterpret_cast<const short8*>(qp + d)
                            : (short8){0, 0, 0, 0, 0, 0, 0, 0};
    }
  }

  const int pieces = a.dim / 8;
  auto load = [&](int st, int buf) {
    const long page = bt[min(st * NW + wave, pages - 1)];
    const bf16_t* base = a.kc + page * PAGE * a.dim;
    #pragma unroll
    for (int i = 0; i < PAGE * RC / WAVE; ++i) {
      const int at = i * WAVE + lane;            // piece of the LDS image
      const int row = at / RC, c = (at % RC) ^ (row & 7);
      // pieces past the row's end meet zeros of the queries
      load_to_lds(base + (long)row * a.dim + min(c, pieces - 1) * 8,
                  &s_c[buf][wave * PAGE * RC + i * WAVE]);
    }
  };
  constexpr int LOADS = PAGE * RC / WAVE;
  static_assert(PAGE * RC % WAVE == 0);

  float m[MT], l[MT];
  float4v o[CT][MT];
  #pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    m[mt] = NEG; l[mt] = 0.f;
    #pragma unroll
    for (int c = 0; c < CT; ++c) o[c][mt] = (float4v){0.f, 0.f, 0.f, 0.f};
  }
  const float scale2 = a.scale * LOG2E;

  if (st0 < st1) load(st0, 0);
  for (int st = st0; st < st1; ++st) {
    const int buf = (st - st0) & 1;
    // the barrier at the end of the last step has released the other buffer
    if (st + 1 < st1) {
      load(st + 1, buf ^ 1);
      asm volatile("s_waitcnt vmcnt(%0)" :: "i"(LOADS) : "memory");
    } else {
      asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    }
    // scores of the wave's own page, which no other wave has loaded
    float4v s[MT];
    #pragma unroll
    for (int mt = 0; mt < MT; ++mt) s[mt] = (float4v){0.f, 0.f, 0.f, 0.f};
    const uint4* krow = &s_c[buf][(wave * PAGE + lo) * RC];
    #pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const short8 k = *reinterpret_cast<const short8*>(
          &krow[(ks * 4 + grp) ^ (lo & 7)]);
      #pragma unroll
      for (int mt = 0; mt < MT; ++mt)
        s[mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k, q[mt][ks], s[mt],
                                                        0, 0, 0);
    }
    const int key0 = st * CH + wave * PAGE + grp * 4;
    #pragma unroll
    for (int mt = 0; mt < MT; ++mt) {
      float mx = NEG;
      #pragma unroll
      for (int i = 0; i < 4; ++i) {
        s[mt][i] = key0 + i <= qpos[mt] ? s[mt][i] * scale2 : -INFINITY;
        mx = fmaxf(mx, s[mt][i]);
      }
      mx = fmaxf(mx, __shfl_xor(mx, 16, WAVE));
      mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE));
      if (grp == 0) s_m[wave][mt * 16 + lo] = mx;
    }
    lds_barrier();
    #pragma unroll
    for (int mt = 0; mt < MT; ++mt) {
      float mn = m[mt];
      #pragma unroll
      for (int w = 0; w < NW; ++w) mn = fmaxf(mn, s_m[w][mt * 16 + lo]);
      const float keep = __builtin_amdgcn_exp2f(m[mt] - mn);
      m[mt] = mn;
      short4v hi, low;
      float sum = 0.f;
      #pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float p = s[mt][i] == -INFINITY
            ? 0.f : __builtin_amdgcn_exp2f(s[mt][i] - mn);
        sum += p;
        const bf16_t ph = f2bf(p), pl = f2bf(p - bf2f(ph));
        hi[i] = *reinterpret_cast<const short*>(&ph);
        low[i] = *reinterpret_cast<const short*>(&pl);
      }
      const int at = wave * PAGE + grp * 4;
      *reinterpret_cast<short4v*>(&s_p[0][mt * 16 + lo][at]) = hi;
      *reinterpret_cast<short4v*>(&s_p[1][mt * 16 + lo][at]) = low;
      sum += __shfl_xor(sum, 16, WAVE);
      sum += __shfl_xor(sum, 32, WAVE);
      l[mt] = l[mt] * keep + sum;                // of the wave's own keys
      if (!__all(keep == 1.f)) {
        #pragma unroll
        for (int c = 0; c < CT; ++c) o[c][mt] *= keep;
      }
    }
    lds_barrier();
    #pragma unroll
    for (int half = 0; half < CH / 32; ++half) {
      short8 ph[MT], pl[MT];
      #pragma unroll
      for (int mt = 0; mt < MT; ++mt) {
        ph[mt] = *reinterpret_cast<const short8*>(
            &s_p[0][mt * 16 + lo][half * 32 + grp * 8]);
        pl[mt] = *reinterpret_cast<const short8*>(
            &s_p[1][mt * 16 + lo][half * 32 + grp * 8]);
      }
      // the lane's place in a transposing load: a key's four columns
      const int key = half * 32 + grp * 8 + (lo >> 2);
      #pragma unroll
      for (int c = 0; c < CT; ++c) {
        const int col = (wave * CT + c) * 16 + (lo & 3) * 4;
        short4v v[2];
        #pragma unroll
        for (int t = 0; t < 2; ++t) {
          const int kk = key + 4 * t;
          const short* p = reinterpret_cast<const short*>(
              &s_c[buf][kk * RC + ((col / 8) ^ (kk & 7))]) + col % 8;
          v[t] = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
              (__attribute__((address_space(3))) short4v*)p);
        }
        short8 vt;
        #pragma unroll
        for (int j = 0; j < 4; ++j) { vt[j] = v[0][j]; vt[4 + j] = v[1][j]; }
        #pragma unroll
        for (int mt = 0; mt < MT; ++mt) {
          o[c][mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              vt, ph[mt], o[c][mt], 0, 0, 0);
          o[c][mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              vt, pl[mt], o[c][mt], 0, 0, 0);
        }
      }
    }
    lds_barrier();
  }

  // sums of all waves' keys
  #pragma unroll
  for (int mt = 0; mt < MT; ++mt)
    if (grp == 0) s_m[wave][mt * 16 + lo] = l[mt];
  __syncthreads();
  #pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    float sum = 0.f;
    #pragma unroll
    for (int w = 0; w < NW; ++w) sum += s_m[w][mt * 16 + lo];
    const int qi = q0 + mt * 16 + lo;
    if (qi >= nq) continue;
    const long row = (long)en.row0 * a.heads + qi;   // row and head
    const long at = row * splits + split;
    const float f = splits == 1 ? 1.f / sum : 1.f;
    #pragma unroll
    for (int c = 0; c < CT; ++c) {
      const int col = (wave * CT + c) * 16 + grp * 4;
      if (col >= a.vdim) continue;
      float v[4];
      #pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = o[c][mt][j] * f;
      if (splits == 1) stv<4>(a.out + row * a.vdim + col, v);
      else stv<4>(part_o + at * a.vdim + col, v);
    }
    if (splits > 1 && wave == 0 && grp == 0) {
      part_ml[at * 2] = m[mt];
      part_ml[at * 2 + 1] = sum;
    }
  }
}

}  // namespace

bool attn_latent_supported(int dim, int vdim, int block_size) {
  return dim % 8 == 0 && vdim % 8 == 0 && vdim <= dim && dim <= 576 &&
         vdim <= 512 && block_size == PAGE;
}

// Workgroups that share one context: enough for every CU, but at least two
// steps for each. `span`: most keys a row can see.
int attn_latent_splits(int entries, int max_len, int heads, int span) {
  const long groups = (long)entries * (((long)max_len * heads + 31) / 32);
  const int steps = (span + CH - 1) / CH;
  int s = 1;
  while (s < 32 && groups * s < 256 && steps >= s * 4) s *= 2;
  return s;
}

void launch_attn_latent(const AttnCtx<bf16_t>& a, int entries, int max_len,
                        int splits, float* part_o, float* part_ml,
                        hipStream_t stream) {
  auto go = [&](auto ks, auto ct, auto mt) {
    constexpr int QT = decltype(mt)::value * 16;
    attn_latent_kernel<decltype(ks)::value, decltype(ct)::value,
                       decltype(mt)::value>
        <<<dim3(entries, ((long)max_len * a.heads + QT - 1) / QT, splits),
           dim3(NW * WAVE), 0, stream>>>(a, splits, part_o, part_ml);
  };
  using std::integral_constant;
  auto by_mt = [&](auto ks, auto ct) {
    if ((long)max_len * a.heads <= 16) go(ks, ct, integral_constant<int, 1>{});
    else go(ks, ct, integral_constant<int, 2>{});
  };
  if (a.dim <= 192 && a.vdim <= 128)
    by_mt(integral_constant<int, 6>{}, integral_constant<int, 2>{});
  else if (a.dim <= 320 && a.vdim <= 256)
    by_mt(integral_constant<int, 10>{}, integral_constant<int, 4>{});
  else
    by_mt(integral_constant<int, 18>{}, integral_constant<int, 8>{});
}
