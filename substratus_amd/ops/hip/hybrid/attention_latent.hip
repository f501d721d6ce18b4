// Attention in the latent space over the paged bf16 cache: all query heads
// share one key per token, and its first `vdim` columns are the value. For
// single tokens and portions of prompts: an entry's queries are its rows
// times its heads, in that order, and a workgroup takes 16 * MT of them.
//
// A step is 64 keys, four pages. A page is one contiguous piece of memory and
// goes to LDS as it is (direct loads, the next step's in flight, page numbers
// another step ahead), except that the 16-byte pieces of a row are permuted
// by the row, so that neither of the two products meets bank conflicts:
//   scores   S^T = K Q^T: each of eight waves has one page's 16 keys and, of
//            the queries, half (MT 2) or half of their elements (MT 1), in
//            registers throughout. Scores meet in LDS;
//   values   O^T = V^T P^T: each wave has an eighth of the columns, for all
//            64 keys. V^T is read by the transposing LDS loads from the same
//            rows. Every wave forms all weights for itself, in the registers
//            where the product wants them, as bf16 high and low parts, so
//            they keep 16 bits.
// Long contexts are split over workgroups and merged by attn_ctx_merge.
#include "attention_ctx.h"

namespace {

typedef __attribute__((ext_vector_type(8))) short short8;
typedef __attribute__((ext_vector_type(4))) short short4v;
typedef __attribute__((ext_vector_type(4))) float float4v;

constexpr int NW = 8;
constexpr int PAGE = 16;
constexpr int PAGES = 4;        // per step
constexpr int CH = PAGES * PAGE;
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
__global__ __launch_bounds__(NW * WAVE)
void attn_latent_kernel(AttnCtx<bf16_t> a, int splits,
                        float* __restrict__ part_o,
                        float* __restrict__ part_ml) {
  constexpr int QT = MT * 16;
  constexpr int RC = KS * 4;                     // 16-byte pieces per LDS row
  constexpr int QS = MT == 2 ? KS : KS / 2;      // key steps of one wave
  constexpr int SS = MT == 2 ? 1 : 2;            // parts of a score
  constexpr int LOADS = PAGE * RC / WAVE / 2;    // of one wave per step
  static_assert(PAGE * RC % (2 * WAVE) == 0 && KS % 2 == 0);
  // one array: beside a second one the compiler guards every LDS read
  // against the direct loads in flight, and waits for them
  __shared__ alignas(16) uint4 s_all[2 * CH * RC + SS * QT * (CH + 4) / 4];
  auto& s_c = *reinterpret_cast<uint4(*)[2][CH * RC]>(s_all);
  auto& s_s = *reinterpret_cast<float(*)[SS][QT][CH + 4]>(
      s_all + 2 * CH * RC);

  const int e = blockIdx.x, split = blockIdx.z;
  const Entry en = entry_of(a.seq_start, e);
  const int q0 = blockIdx.y * QT, nq = en.n * a.heads;
  if (q0 >= nq) return;
  // page numbers come by scalar loads, which the counted waits do not see
  const auto* bt = (const __attribute__((address_space(4))) int*)(
      a.block_table + (long)e * a.max_blocks);
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / WAVE);
  const int lane = threadIdx.x % WAVE;
  const int lo = lane & 15, grp = lane >> 4;
  const int page = wave % PAGES, part = wave / PAGES;
  const int pos0 = a.positions[en.row0];
  const int last = pos0 + (min(q0 + QT, nq) - 1) / a.heads;  // of the tile
  const int pages = last / PAGE + 1;
  const int steps = (pages + PAGES - 1) / PAGES;
  const int st0 = (int)((long)steps * split / splits),
            st1 = (int)((long)steps * (split + 1) / splits);
  auto page_at = [&](int st) {
    return bt[min(st * PAGES + page, pages - 1)];
  };
  int pg = page_at(st0);                         // of the step to load next

  // queries: lane = query, 8 consecutive elements
  short8 q[QS];
  const int ks0 = MT == 2 ? 0 : part * QS;
  {
    const int qi = min(q0 + (MT == 2 ? part * 16 : 0) + lo, nq - 1);
    const bf16_t* qp = a.q + (long)(en.row0 + qi / a.heads) * a.q_ld +
                       (long)(qi % a.heads) * a.dim;
    #pragma unroll
    for (int ks = 0; ks < QS; ++ks) {
      const int d = (ks0 + ks) * 32 + grp * 8;
      q[ks] = d < a.dim ? *reinterpret_cast<const short8*>(qp + d)
                        : (short8){0, 0, 0, 0, 0, 0, 0, 0};
    }
  }
  int qpos[MT];
  #pragma unroll
  for (int mt = 0; mt < MT; ++mt)
    qpos[mt] = pos0 + min(q0 + mt * 16 + lo, nq - 1) / a.heads;

  // the lane's pieces of its wave's half page
  const int pieces = a.dim / 8;
  int off[LOADS];
  #pragma unroll
  for (int i = 0; i < LOADS; ++i) {
    const int at = (part * LOADS + i) * WAVE + lane;
    const int row = at / RC, c = (at % RC) ^ (row & 7);
    // pieces past the row's end meet zeros of the queries
    off[i] = row * a.dim + min(c, pieces - 1) * 8;
  }
  auto load = [&](int buf) {
    const bf16_t* base =
        a.kc + (long)pg * PAGE * a.dim;
    #pragma unroll
    for (int i = 0; i < LOADS; ++i)
      load_to_lds(base + off[i],
                  &s_c[buf][page * PAGE * RC + (part * LOADS + i) * WAVE]);
  };

  float m[MT], l[MT];
  float4v o[CT][MT];
  #pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    m[mt] = NEG; l[mt] = 0.f;
    #pragma unroll
    for (int c = 0; c < CT; ++c) o[c][mt] = (float4v){0.f, 0.f, 0.f, 0.f};
  }
  const float scale2 = a.scale * LOG2E;

  if (st0 < st1) load(0);
  pg = page_at(st0 + 1);
  // queries are there before the loop, so that it never waits for them
  #pragma unroll
  for (int ks = 0; ks < QS; ++ks) asm volatile("" : "+v"(q[ks]));
  for (int st = st0; st < st1; ++st) {
    const int buf = (st - st0) & 1;
    // the barrier at the end of the last step has released the other buffer
    if (st + 1 < st1) {
      const int next = page_at(st + 2);
      load(buf ^ 1);
      pg = next;
      asm volatile("s_waitcnt vmcnt(%0)" :: "i"(LOADS) : "memory");
    } else {
      asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    }
    asm volatile("s_barrier" ::: "memory");
    float4v s[2];
    s[0] = s[1] = (float4v){0.f, 0.f, 0.f, 0.f};
    const uint4* krow = &s_c[buf][(page * PAGE + lo) * RC];
    #pragma unroll
    for (int ks = 0; ks < QS; ++ks) {
      const short8 k = *reinterpret_cast<const short8*>(
          &krow[((ks0 + ks) * 4 + grp) ^ (lo & 7)]);
      s[ks & 1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k, q[ks], s[ks & 1],
                                                          0, 0, 0);
    }
    *reinterpret_cast<float4v*>(
        &s_s[MT == 2 ? 0 : part][(MT == 2 ? part * 16 : 0) + lo]
            [page * PAGE + grp * 4]) = s[0] + s[1];
    lds_barrier();

    short8 ph[MT][2], pl[MT][2];                 // weights of keys
    #pragma unroll
    for (int mt = 0; mt < MT; ++mt) {            //   half * 32 + grp * 8 + j
      float v[2][8];
      float mx = NEG;
      #pragma unroll
      for (int half = 0; half < 2; ++half)
        #pragma unroll
        for (int j4 = 0; j4 < 2; ++j4) {
          const int k = half * 32 + grp * 8 + j4 * 4;
          float4v f =
              *reinterpret_cast<const float4v*>(&s_s[0][mt * 16 + lo][k]);
          if constexpr (SS == 2)
            f += *reinterpret_cast<const float4v*>(&s_s[1][mt * 16 + lo][k]);
          #pragma unroll
          for (int j = 0; j < 4; ++j) {
            const float x = st * CH + k + j <= qpos[mt] ? f[j] * scale2
                                                        : -INFINITY;
            v[half][j4 * 4 + j] = x;
            mx = fmaxf(mx, x);
          }
        }
      mx = fmaxf(mx, __shfl_xor(mx, 16, WAVE));
      mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE));
      const float mn = fmaxf(m[mt], mx);
      const float keep = __builtin_amdgcn_exp2f(m[mt] - mn);
      m[mt] = mn;
      float sum = 0.f;
      #pragma unroll
      for (int half = 0; half < 2; ++half)
        #pragma unroll
        for (int j = 0; j < 8; ++j) {
          const float p = __builtin_amdgcn_exp2f(v[half][j] - mn);
          sum += p;                              // exp2(-inf) is 0
          const bf16_t h = f2bf(p), w = f2bf(p - bf2f(h));
          ph[mt][half][j] = *reinterpret_cast<const short*>(&h);
          pl[mt][half][j] = *reinterpret_cast<const short*>(&w);
        }
      sum += __shfl_xor(sum, 16, WAVE);
      sum += __shfl_xor(sum, 32, WAVE);
      l[mt] = l[mt] * keep + sum;
      if (!__all(keep == 1.f)) {
        #pragma unroll
        for (int c = 0; c < CT; ++c) o[c][mt] *= keep;
      }
    }
    #pragma unroll
    for (int half = 0; half < 2; ++half) {
      // the lane's place in a transposing load: a key's four columns
      const int key = half * 32 + grp * 8 + (lo >> 2);
      short8 vt[CT];
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
        #pragma unroll
        for (int j = 0; j < 4; ++j) {
          vt[c][j] = v[0][j];
          vt[c][4 + j] = v[1][j];
        }
      }
      #pragma unroll
      for (int c = 0; c < CT; ++c)
        #pragma unroll
        for (int mt = 0; mt < MT; ++mt) {
          o[c][mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              vt[c], ph[mt][half], o[c][mt], 0, 0, 0);
          o[c][mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              vt[c], pl[mt][half], o[c][mt], 0, 0, 0);
        }
    }
    lds_barrier();
  }

  #pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    const int qi = q0 + mt * 16 + lo;
    if (qi >= nq) continue;
    const long row = (long)en.row0 * a.heads + qi;   // row and head
    const long at = row * splits + split;
    const float f = splits == 1 ? 1.f / l[mt] : 1.f;
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
      part_ml[at * 2 + 1] = l[mt];
    }
  }
}

// Queries per workgroup: 32 where that leaves enough of them.
int query_tile(int entries, int max_len, int heads) {
  const long q = (long)max_len * heads;
  return q > 16 && entries * ((q + 31) / 32) >= 192 ? 32 : 16;
}

}  // namespace

bool attn_latent_supported(int dim, int vdim, int block_size) {
  return dim % 8 == 0 && vdim % 8 == 0 && vdim <= dim && dim <= 576 &&
         vdim <= 512 && block_size == PAGE;
}

// Workgroups that share one context: enough for every CU, but at least two
// steps for each. `span`: most keys a row can see.
int attn_latent_splits(int entries, int max_len, int heads, int span) {
  const int qt = query_tile(entries, max_len, heads);
  const long groups = (long)entries * (((long)max_len * heads + qt - 1) / qt);
  const int steps = (span + CH - 1) / CH;
  int s = 1;
  while (s < 32 && groups * s * 3 < 512 && steps >= s * 4) s *= 2;
  return s;
}

void launch_attn_latent(const AttnCtx<bf16_t>& a, int entries, int max_len,
                        int splits, float* part_o, float* part_ml,
                        hipStream_t stream) {
  const int qt = query_tile(entries, max_len, a.heads);
  const dim3 grid(entries, ((long)max_len * a.heads + qt - 1) / qt, splits);
  auto go = [&](auto ks, auto ct) {
    constexpr int KS = decltype(ks)::value, CT = decltype(ct)::value;
    if (qt == 16)
      attn_latent_kernel<KS, CT, 1><<<grid, dim3(NW * WAVE), 0, stream>>>(
          a, splits, part_o, part_ml);
    else
      attn_latent_kernel<KS, CT, 2><<<grid, dim3(NW * WAVE), 0, stream>>>(
          a, splits, part_o, part_ml);
  };
  using std::integral_constant;
  if (a.dim <= 192 && a.vdim <= 128)
    go(integral_constant<int, 6>{}, integral_constant<int, 1>{});
  else if (a.dim <= 320 && a.vdim <= 256)
    go(integral_constant<int, 10>{}, integral_constant<int, 2>{});
  else
    go(integral_constant<int, 18>{}, integral_constant<int, 4>{});
}
