// Attention in the latent space over the paged bf16 cache: all query heads
// share one key per token, and its first `vdim` columns are the value. For
// single tokens and portions of prompts: an entry's queries are its rows
// times its heads, in that order, and a workgroup takes 16 * MT of them. With
// a window, it begins at the step with the first key that any of them sees.
//
// A step is 64 keys, four pages. A page is one contiguous piece of memory and
// goes to LDS as it is (direct loads, the next step's in flight, page numbers
// another step ahead), except that the 16-byte pieces of a row are permuted
// by the row, so that neither of the two products meets bank conflicts:
//   scores   S^T = K Q^T: each wave has one page's 16 keys and 16 queries, in
//            registers throughout (with 16 queries in all, half the waves).
//            It forms their weights, once the waves have exchanged maxima;
//   values   O^T = V^T P^T: each of the eight waves has an eighth of the
//            columns, for all 64 keys. V^T is read by the transposing LDS
//            loads from the same rows, weights through LDS as bf16 high and
//            low parts, so they keep 16 bits.
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
void attn_latent_kernel(AttnCtx<bf16_t> a, int entries, int splits,
                        float* __restrict__ part_o,
                        float* __restrict__ part_ml) {
  constexpr int QT = MT * 16;
  constexpr int RC = KS * 4;                     // 16-byte pieces per LDS row
  constexpr int PP = CH + 8;                     // padded row of weights
  constexpr int LOADS = PAGE * RC / WAVE / 2;    // of one wave per step
  static_assert(PAGE * RC % (2 * WAVE) == 0 && KS % 2 == 0);
  // one array: beside a second one the compiler guards every LDS read
  // against the direct loads in flight, and waits for them
  __shared__ alignas(16) uint4
      s_all[2 * CH * RC + 2 * QT * PP / 8 + PAGES * QT / 4];
  auto& s_c = *reinterpret_cast<uint4(*)[2][CH * RC]>(s_all);
  auto& s_p = *reinterpret_cast<short(*)[2][QT][PP]>(   // high and low parts
      s_all + 2 * CH * RC);
  auto& s_m = *reinterpret_cast<float(*)[PAGES][QT]>(
      s_all + 2 * CH * RC + 2 * QT * PP / 8);

  const int e = blockIdx.x % entries, split = blockIdx.y;
  const Entry en = entry_of(a.seq_start, e);
  const int q0 = blockIdx.x / entries * QT, nq = en.n * a.heads;
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
  const int sb = first_seen(a, pos0 + q0 / a.heads) / CH;
  const int steps = (pages + PAGES - 1) / PAGES - sb;
  const int st0 = sb + (int)((long)steps * split / splits),
            st1 = sb + (int)((long)steps * (split + 1) / splits);
  auto page_at = [&](int st) {
    return bt[min(st * PAGES + page, pages - 1)];
  };
  int pg = page_at(st0);                         // of the step to load next

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

  if (st0 < st1) load(0);
  pg = page_at(st0 + 1);

  // queries: lane = query, 8 consecutive elements
  const bool scoring = part < MT;
  const int mine = (scoring ? part : 0) * 16;
  short8 q[KS];
  int qpos, qlo;                                 // first and last key seen
  {
    const int qi = min(q0 + mine + lo, nq - 1);
    qpos = pos0 + qi / a.heads;
    qlo = first_seen(a, qpos);
    const bf16_t* qp = a.q + (long)(en.row0 + qi / a.heads) * a.q_ld +
                       (long)(qi % a.heads) * a.dim;
    #pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const int d = ks * 32 + grp * 8;
      q[ks] = scoring && d < a.dim
          ? *reinterpret_cast<const short8*>(qp + d)
          : (short8){0, 0, 0, 0, 0, 0, 0, 0};
    }
  }

  float m[MT], l = 0.f;                          // l: of the wave's own keys
  float4v o[CT][MT];
  #pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    m[mt] = NEG;
    #pragma unroll
    for (int c = 0; c < CT; ++c) o[c][mt] = (float4v){0.f, 0.f, 0.f, 0.f};
  }
  const float scale2 = a.scale * LOG2E;
  // queries are there before the loop, so that it never waits for them
  #pragma unroll
  for (int ks = 0; ks < KS; ++ks) asm volatile("" : "+v"(q[ks]));
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
    float s[4];
    if (scoring) {
      float4v acc[2];
      acc[0] = acc[1] = (float4v){0.f, 0.f, 0.f, 0.f};
      const uint4* krow = &s_c[buf][(page * PAGE + lo) * RC];
      #pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        const short8 k = *reinterpret_cast<const short8*>(
            &krow[(ks * 4 + grp) ^ (lo & 7)]);
        acc[ks & 1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            k, q[ks], acc[ks & 1], 0, 0, 0);
      }
      const int key = st * CH + page * PAGE + grp * 4;
      float mx = NEG;
      #pragma unroll
      for (int i = 0; i < 4; ++i) {
        s[i] = key + i <= qpos && key + i >= qlo
            ? (acc[0][i] + acc[1][i]) * scale2 : -INFINITY;
        mx = fmaxf(mx, s[i]);
      }
      mx = fmaxf(mx, __shfl_xor(mx, 16, WAVE));
      mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE));
      if (grp == 0) s_m[page][mine + lo] = mx;
    }
    lds_barrier();
    float keep[MT];
    #pragma unroll
    for (int mt = 0; mt < MT; ++mt) {
      float mn = m[mt];
      #pragma unroll
      for (int p = 0; p < PAGES; ++p) mn = fmaxf(mn, s_m[p][mt * 16 + lo]);
      keep[mt] = __builtin_amdgcn_exp2f(m[mt] - mn);
      m[mt] = mn;
    }
    if (scoring) {
      const float mn = MT == 2 && part == 1 ? m[MT - 1] : m[0];
      float p[4], sum = 0.f;
      #pragma unroll
      for (int i = 0; i < 4; ++i) {
        p[i] = __builtin_amdgcn_exp2f(s[i] - mn);    // exp2(-inf) is 0
        sum += p[i];
      }
      l = l * (MT == 2 && part == 1 ? keep[MT - 1] : keep[0]) + sum;
      uint2 hi, low;
      hi.x = cvt_pk_bf16(p[0], p[1]);
      hi.y = cvt_pk_bf16(p[2], p[3]);
      const float2 b0 = unpack_bf16x2(hi.x), b1 = unpack_bf16x2(hi.y);
      low.x = cvt_pk_bf16(p[0] - b0.x, p[1] - b0.y);
      low.y = cvt_pk_bf16(p[2] - b1.x, p[3] - b1.y);
      const int at = page * PAGE + grp * 4;
      *reinterpret_cast<uint2*>(&s_p[0][mine + lo][at]) = hi;
      *reinterpret_cast<uint2*>(&s_p[1][mine + lo][at]) = low;
    }
    #pragma unroll
    for (int mt = 0; mt < MT; ++mt)
      if (!__all(keep[mt] == 1.f)) {
        #pragma unroll
        for (int c = 0; c < CT; ++c) o[c][mt] *= keep[mt];
      }
    lds_barrier();
    #pragma unroll
    for (int half = 0; half < 2; ++half) {
      // the lane's place in a transposing load: a key's four columns
      const int key = half * 32 + grp * 8 + (lo >> 2);
      short8 vt[CT], ph[MT], pl[MT];
      #pragma unroll
      for (int mt = 0; mt < MT; ++mt) {
        ph[mt] = *reinterpret_cast<const short8*>(
            &s_p[0][mt * 16 + lo][half * 32 + grp * 8]);
        pl[mt] = *reinterpret_cast<const short8*>(
            &s_p[1][mt * 16 + lo][half * 32 + grp * 8]);
      }
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
              vt[c], ph[mt], o[c][mt], 0, 0, 0);
          o[c][mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              vt[c], pl[mt], o[c][mt], 0, 0, 0);
        }
    }
    lds_barrier();
  }

  // sums of all waves' keys
  l += __shfl_xor(l, 16, WAVE);
  l += __shfl_xor(l, 32, WAVE);
  if (scoring && grp == 0) s_m[page][mine + lo] = l;
  lds_barrier();
  #pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    float sum = 0.f;
    #pragma unroll
    for (int p = 0; p < PAGES; ++p) sum += s_m[p][mt * 16 + lo];
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

// Queries per workgroup: 32, which reads the latents once for as many heads,
// where that leaves enough workgroups (or steps to split between them).
int query_tile(int entries, int max_len, int heads, int span) {
  const long q = (long)max_len * heads, groups = entries * ((q + 31) / 32);
  if (q <= 16) return 16;
  return groups >= 192 || (groups >= 64 && span >= 24 * CH) ? 32 : 16;
}

}  // namespace

bool attn_latent_supported(int dim, int vdim, int block_size) {
  return dim % 8 == 0 && vdim % 8 == 0 && vdim <= dim && dim <= 576 &&
         vdim <= 512 && block_size == PAGE;
}

// Workgroups that share one context: enough for every CU, but at least two
// steps for each. `span`: most keys a row can see.
int attn_latent_splits(int entries, int max_len, int heads, int span) {
  const int qt = query_tile(entries, max_len, heads, span);
  const long groups = (long)entries * (((long)max_len * heads + qt - 1) / qt);
  const int steps = (span + CH - 1) / CH;
  int s = 1;
  while (s < 32 && groups * s < 256 && steps >= s * 4) s *= 2;
  return s;
}

void launch_attn_latent(const AttnCtx<bf16_t>& a, int entries, int max_len,
                        int span, int splits, float* part_o, float* part_ml,
                        hipStream_t stream) {
  const int qt = query_tile(entries, max_len, a.heads, span);
  const dim3 grid(entries * (((long)max_len * a.heads + qt - 1) / qt), splits);
  auto go = [&](auto ks, auto ct) {
    constexpr int KS = decltype(ks)::value, CT = decltype(ct)::value;
    if (qt == 16)
      attn_latent_kernel<KS, CT, 1><<<grid, dim3(NW * WAVE), 0, stream>>>(
          a, entries, splits, part_o, part_ml);
    else
      attn_latent_kernel<KS, CT, 2><<<grid, dim3(NW * WAVE), 0, stream>>>(
          a, entries, splits, part_o, part_ml);
  };
  using std::integral_constant;
  if (a.dim <= 192 && a.vdim <= 128)
    go(integral_constant<int, 6>{}, integral_constant<int, 1>{});
  else if (a.dim <= 320 && a.vdim <= 256)
    go(integral_constant<int, 10>{}, integral_constant<int, 2>{});
  else
    go(integral_constant<int, 18>{}, integral_constant<int, 4>{});
}
