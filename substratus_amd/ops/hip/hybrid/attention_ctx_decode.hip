// Single-token attention over the paged bf16 cache with a distance bias, a
// chunk mask, unequal key and value head sizes, a gated output, and softmax or
// sigmoid weights (the formulas are in attention_ctx.hip). HBM-bound: every K
// and V row is read once per group of GQ query heads.
//
// One page of 16 keys is a wave's unit of work. Scores: 4 lanes per key, each
// with every fourth 16-byte piece of the row. Values: CL lanes across the
// columns (8 each), 64/CL rows side by side. The next page's K, V and bias
// are in flight while the current page is computed. Queries stay bf16 and
// scores are sums of v_dot2_f32_bf16 (two products added to a float), so K
// needs no unpacking. Four waves take pages in turn and merge through LDS;
// `splits` workgroups share one long context and a second kernel merges those.
#include "attention_ctx.h"

namespace {

constexpr int NW = 4;         // waves per workgroup
constexpr int PAGE = 16;
constexpr float NEG = -1e30f; // "no key yet": finite, so differences are too

typedef __attribute__((ext_vector_type(2))) __bf16 bf16x2_t;

DEV_INLINE float dot2(unsigned a, unsigned b, float c) {
  return __builtin_amdgcn_fdot2_f32_bf16(
      __builtin_bit_cast(bf16x2_t, a), __builtin_bit_cast(bf16x2_t, b), c,
      false);
}

// SIG: sigmoid weights, so partial results add up as they are
template <int DCH, int CL, int GQ, bool SIG>
__global__ __launch_bounds__(NW * WAVE)
void attn_ctx_decode_kernel(AttnCtx<bf16_t> a, int splits,
                            float* __restrict__ part_o,
                            float* __restrict__ part_ml) {
  constexpr int RPI = WAVE / CL;          // V rows per instruction
  constexpr int NV = PAGE / RPI;          // V instructions per page
  __shared__ alignas(16) unsigned s_q[GQ][DCH * 16];
  __shared__ float s_o[NW][GQ][CL * 8];
  __shared__ float s_ml[NW][GQ][2];
  const int b = blockIdx.x, kvh = blockIdx.y;
  const int split = blockIdx.z % splits;
  const int per = a.heads / a.kv_heads;
  const int g0 = blockIdx.z / splits * GQ;
  const int h0 = kvh * per + g0;
  const int nh = min(GQ, per - g0);
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
  const int pos = a.positions[b];
  const int lo = first_seen(a, pos);
  const Pieces part(a.keep, lo, pos / PAGE + 1, PAGE);
  const int* bt = a.block_table + (long)b * a.max_blocks;

  for (int i = threadIdx.x; i < GQ * DCH * 16; i += NW * WAVE) {
    const int g = i / (DCH * 16), d = i % (DCH * 16) * 2;
    const unsigned short* q = reinterpret_cast<const unsigned short*>(a.q) +
                              (long)b * a.q_ld + (long)(h0 + g) * a.dim + d;
    s_q[g][d / 2] = g < nh && d < a.dim ? q[0] | (unsigned)q[1] << 16 : 0u;
  }
  __syncthreads();

  const int key = lane >> 2, sub = lane & 3;
  const int col = lane % CL, rg = lane / CL;
  const int kch = a.dim / 8, vch = a.vdim / 8;
  const int first = split * NW + wave, stride = splits * NW;
  // a capped score: cap tanh(s scale / cap), by tanh_exp2
  const float scale2 = a.scale * LOG2E;
  const float cap2 = a.cap * LOG2E;
  const float cscale = a.cap > 0.f ? 2.f * scale2 / a.cap : 0.f;

  float r1[GQ], r2[GQ], wb[GQ];
  #pragma unroll
  for (int g = 0; g < GQ; ++g) {
    const int h = h0 + min(g, nh - 1);
    r1[g] = a.r1 != nullptr ? a.r1[h] : 0.f;
    r2[g] = a.r1 != nullptr ? a.r2[h] : 0.f;
    wb[g] = SIG ? a.wbias[h] * LOG2E : 0.f;
  }
  uint4v kr[DCH], vr[NV];
  float br[GQ];
  auto load = [&](int pg) {
    const long page = (long)bt[pg] * a.kv_heads + kvh;
    const bf16_t* kp = a.kc + (page * PAGE + key) * a.dim;
    const bf16_t* vp = a.vc + page * PAGE * a.v_ld;
    #pragma unroll
    for (int i = 0; i < DCH; ++i)
      kr[i] = sub + 4 * i < kch ? nt_load_u4(kp + (sub + 4 * i) * 8)
                                : (uint4v){0, 0, 0, 0};
    #pragma unroll
    for (int i = 0; i < NV; ++i)
      vr[i] = col < vch
          ? nt_load_u4(vp + (long)(rg + RPI * i) * a.v_ld + col * 8)
          : (uint4v){0, 0, 0, 0};
    #pragma unroll
    for (int g = 0; g < GQ; ++g) {
      const int n = min(max(pos - (pg * PAGE + key), 0), a.nbias - 1);
      br[g] = a.bias != nullptr && g < nh
          ? a.bias[(long)(h0 + g) * a.nbias + n] * LOG2E : 0.f;
    }
  };

  float m[GQ], l[GQ], acc[GQ][8];
  #pragma unroll
  for (int g = 0; g < GQ; ++g) {
    m[g] = NEG; l[g] = 0.f;
    #pragma unroll
    for (int j = 0; j < 8; ++j) acc[g][j] = 0.f;
  }
  if (first < part.n) load(part.at(first));
  for (int it = first; it < part.n; it += stride) {
    const int pg = part.at(it);
    uint4v kn[DCH], vn[NV];
    float bn[GQ];
    #pragma unroll
    for (int i = 0; i < DCH; ++i) kn[i] = kr[i];
    #pragma unroll
    for (int i = 0; i < NV; ++i) vn[i] = vr[i];
    #pragma unroll
    for (int g = 0; g < GQ; ++g) bn[g] = br[g];
    if (it + stride < part.n) load(part.at(it + stride));

    float s[GQ];
    #pragma unroll
    for (int g = 0; g < GQ; ++g) s[g] = 0.f;
    #pragma unroll
    for (int i = 0; i < DCH; ++i) {
      #pragma unroll
      for (int g = 0; g < GQ; ++g) {
        const uint4 qp =
            *reinterpret_cast<const uint4*>(&s_q[g][(sub + 4 * i) * 4]);
        s[g] = dot2(kn[i][0], qp.x, s[g]);
        s[g] = dot2(kn[i][1], qp.y, s[g]);
        s[g] = dot2(kn[i][2], qp.z, s[g]);
        s[g] = dot2(kn[i][3], qp.w, s[g]);
      }
    }
    const int kpos = pg * PAGE + key;
    const bool live = kpos <= pos && (kpos >= lo || kpos < a.keep);
    const float dist = (float)(pos - kpos);
    #pragma unroll
    for (int g = 0; g < GQ; ++g) {
      s[g] += __shfl_xor(s[g], 1, WAVE);
      s[g] += __shfl_xor(s[g], 2, WAVE);
      s[g] = a.cap > 0.f ? cap2 * tanh_exp2(s[g] * cscale) : s[g] * scale2;
      if (a.r1 != nullptr)
        s[g] -= r1[g] * __builtin_amdgcn_logf(1.f + r2[g] * dist);
      if constexpr (SIG) {
        s[g] = live ? sigmoid_exp2(s[g] + bn[g] + wb[g]) : 0.f;
        continue;
      }
      s[g] = live ? s[g] + bn[g] : NEG;
      float mx = s[g];
      #pragma unroll
      for (int off = 4; off < WAVE; off <<= 1)
        mx = fmaxf(mx, __shfl_xor(mx, off, WAVE));
      if (mx > m[g]) {                     // uniform over the wave
        const float keep = __builtin_amdgcn_exp2f(m[g] - mx);
        l[g] *= keep;
        #pragma unroll
        for (int j = 0; j < 8; ++j) acc[g][j] *= keep;
        m[g] = mx;
      }
      s[g] = live ? __builtin_amdgcn_exp2f(s[g] - m[g]) : 0.f;
      l[g] += s[g];                        // lanes hold 4 copies of each key
    }
    #pragma unroll
    for (int i = 0; i < NV; ++i) {
      float vf[8];
      #pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float2 t = unpack_bf16x2(vn[i][j]);
        vf[2 * j] = t.x; vf[2 * j + 1] = t.y;
      }
      #pragma unroll
      for (int g = 0; g < GQ; ++g) {
        const float p = __shfl(s[g], (rg + RPI * i) * 4, WAVE);
        #pragma unroll
        for (int j = 0; j < 8; ++j) acc[g][j] += p * vf[j];
      }
    }
  }

  #pragma unroll
  for (int g = 0; g < GQ; ++g) {
    #pragma unroll
    for (int j = 0; j < 8; ++j) {
      #pragma unroll
      for (int off = CL; off < WAVE; off <<= 1)
        acc[g][j] += __shfl_xor(acc[g][j], off, WAVE);
      if (rg == 0) s_o[wave][g][col * 8 + j] = acc[g][j];
    }
    const float lt = wave_sum(l[g]) * 0.25f;
    if (lane == 0) { s_ml[wave][g][0] = m[g]; s_ml[wave][g][1] = lt; }
  }
  __syncthreads();

  for (int i = threadIdx.x; i < nh * a.vdim; i += NW * WAVE) {
    const int g = i / a.vdim, c = i % a.vdim, h = h0 + g;
    if constexpr (SIG) {
      float o = 0.f;
      #pragma unroll
      for (int w = 0; w < NW; ++w) o += s_o[w][g][c];
      if (splits == 1) {
        float f = a.mult;
        if (a.gate != nullptr)
          f *= sigmoid_f(bf2f(a.gate[(long)b * a.g_ld + h]));
        a.out[(long)b * a.out_ld + (long)h * a.vdim + c] = f2bf(o * f);
      } else {
        part_o[(((long)b * a.heads + h) * splits + split) * a.vdim + c] = o;
      }
      continue;
    }
    float M = s_ml[0][g][0];
    #pragma unroll
    for (int w = 1; w < NW; ++w) M = fmaxf(M, s_ml[w][g][0]);
    float L = 0.f, o = 0.f;
    if (a.sink != nullptr && splits == 1) {
      const float s = a.sink[h] * LOG2E;
      M = fmaxf(M, s);
      L = __builtin_amdgcn_exp2f(s - M);
    }
    #pragma unroll
    for (int w = 0; w < NW; ++w) {
      const float f = __builtin_amdgcn_exp2f(s_ml[w][g][0] - M);
      L += s_ml[w][g][1] * f;
      o += s_o[w][g][c] * f;
    }
    if (splits == 1) {
      float f = a.mult / L;
      if (a.gate != nullptr)
        f *= sigmoid_f(bf2f(a.gate[(long)b * a.g_ld + h]));
      a.out[(long)b * a.out_ld + (long)h * a.vdim + c] = f2bf(o * f);
    } else {
      const long at = ((long)b * a.heads + h) * splits + split;
      part_o[at * a.vdim + c] = o;
      if (c == 0) { part_ml[at * 2] = M; part_ml[at * 2 + 1] = L; }
    }
  }
}

// VEC columns per thread
template <int VEC>
__global__
void attn_ctx_merge_kernel(AttnCtx<bf16_t> a, int splits,
                           const float* __restrict__ part_o,
                           const float* __restrict__ part_ml) {
  const int h = blockIdx.x;
  const long b = blockIdx.y, at = (b * a.heads + h) * splits;
  const int c = threadIdx.x * VEC;
  if (c >= a.vdim) return;
  const bool sig = a.wbias != nullptr;          // sums only, no part_ml
  float M = sig ? 0.f : NEG;
  for (int s = 0; s < splits && !sig; ++s)
    M = fmaxf(M, part_ml[(at + s) * 2]);
  float L = sig ? 1.f : 0.f, o[VEC];
  if (a.sink != nullptr) {
    const float s = a.sink[h] * LOG2E;
    M = fmaxf(M, s);
    L = __builtin_amdgcn_exp2f(s - M);
  }
  #pragma unroll
  for (int j = 0; j < VEC; ++j) o[j] = 0.f;
  #pragma unroll 4
  for (int s = 0; s < splits; ++s) {
    const float f =
        sig ? 1.f : __builtin_amdgcn_exp2f(part_ml[(at + s) * 2] - M);
    float p[VEC];
    ldv<VEC>(part_o + (at + s) * a.vdim + c, p);
    if (!sig) L += part_ml[(at + s) * 2 + 1] * f;
    #pragma unroll
    for (int j = 0; j < VEC; ++j) o[j] += p[j] * f;
  }
  float f = a.mult / L;
  if (a.gate != nullptr) f *= sigmoid_f(bf2f(a.gate[b * a.g_ld + h]));
  #pragma unroll
  for (int j = 0; j < VEC; ++j) o[j] *= f;
  bf16_t* out = a.out + b * a.out_ld + (long)h * a.vdim + c;
  if (a.quads) {
    stv<VEC>(out, o);
  } else {
    #pragma unroll
    for (int j = 0; j < VEC; ++j) st1(out + j, o[j]);
  }
}

constexpr int pick_gq(int per) { return per >= 4 ? 4 : per >= 2 ? 2 : 1; }

}  // namespace

bool attn_ctx_decode_supported(int dim, int vdim, int block_size) {
  return dim % 8 == 0 && vdim % 8 == 0 && dim <= 256 && vdim <= 256 &&
         block_size == PAGE;
}

// Workgroups that share one context: enough to fill 256 CUs four deep, but
// at least two pages for every wave. `span`: most keys a token can see.
int attn_ctx_decode_splits(int entries, int heads, int kv_heads, int span) {
  const int per = heads / kv_heads, gq = pick_gq(per);
  const long groups = (long)entries * kv_heads * ((per + gq - 1) / gq);
  const int pages = (span + PAGE - 1) / PAGE;
  int s = 1;
  while (s < 32 && groups * s < 1024 && pages >= s * 2 * NW * 2) s *= 2;
  return s;
}

void launch_attn_ctx_decode(const AttnCtx<bf16_t>& a, int entries, int splits,
                            float* part_o, float* part_ml,
                            hipStream_t stream) {
  const int per = a.heads / a.kv_heads, gq = pick_gq(per);
  const dim3 grid(entries, a.kv_heads, (per + gq - 1) / gq * splits);
  auto go = [&](auto dch, auto cl, auto g) {
    constexpr int D = decltype(dch)::value, C = decltype(cl)::value,
                  G = decltype(g)::value;
    if (a.wbias != nullptr)
      attn_ctx_decode_kernel<D, C, G, true>
          <<<grid, dim3(NW * WAVE), 0, stream>>>(a, splits, part_o, part_ml);
    else
      attn_ctx_decode_kernel<D, C, G, false>
          <<<grid, dim3(NW * WAVE), 0, stream>>>(a, splits, part_o, part_ml);
  };
  using std::integral_constant;
  auto by_g = [&](auto dch, auto cl) {
    if (gq == 1) go(dch, cl, integral_constant<int, 1>{});
    else if (gq == 2) go(dch, cl, integral_constant<int, 2>{});
    else go(dch, cl, integral_constant<int, 4>{});
  };
  auto by_cl = [&](auto dch) {
    if (a.vdim <= 64) by_g(dch, integral_constant<int, 8>{});
    else if (a.vdim <= 128) by_g(dch, integral_constant<int, 16>{});
    else by_g(dch, integral_constant<int, 32>{});
  };
  if (a.dim <= 64) by_cl(integral_constant<int, 2>{});
  else if (a.dim <= 96) by_cl(integral_constant<int, 3>{});
  else if (a.dim <= 128) by_cl(integral_constant<int, 4>{});
  else by_cl(integral_constant<int, 8>{});
  if (splits > 1)
    launch_attn_ctx_merge(a, entries, splits, part_o, part_ml, stream);
}

void launch_attn_ctx_merge(const AttnCtx<bf16_t>& a, long rows, int splits,
                           const float* part_o, const float* part_ml,
                           hipStream_t stream) {
  // value sizes of the split kernels are multiples of 8, at most 512
  attn_ctx_merge_kernel<4><<<dim3(a.heads, rows), (a.vdim / 4 + 63) / 64 * 64,
                             0, stream>>>(a, splits, part_o, part_ml);
}
