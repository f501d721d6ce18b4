// Gated linear attention, token by token, in float or bf16 (formulas in
// gla.h). One workgroup per (entry, head) walks the entry's rows; for single
// tokens it is the decode step: the state is read once, updated, used and
// written once, with the decay, the group norm and the gate in the same
// kernel, so a step moves two states' worth of bytes and little else.
//
// LPR lanes cover a state row (VEC columns each); the workgroup's lane groups
// take key channels in turn.
#include "gla.h"

#include <type_traits>

namespace {

constexpr int BLOCK = 256;
constexpr int UNROLL = 8;    // state rows in flight per lane group

typedef __attribute__((ext_vector_type(4))) float float4v;

template <int VEC>
DEV_INLINE void ld_state(const float* p, float* f) {
  if constexpr (VEC == 4) {
    const float4v u =
        __builtin_nontemporal_load(reinterpret_cast<const float4v*>(p));
    #pragma unroll
    for (int j = 0; j < 4; ++j) f[j] = u[j];
  } else {
    f[0] = *p;
  }
}

template <int VEC>
DEV_INLINE void st_state(float* p, const float* f) {
  if constexpr (VEC == 4) {
    const float4v u = {f[0], f[1], f[2], f[3]};
    __builtin_nontemporal_store(u, reinterpret_cast<float4v*>(p));
  } else {
    *p = f[0];
  }
}

// CONST: constant decays
template <class T, int VEC, bool CONST>
__global__ __launch_bounds__(BLOCK)
void gla_recurrent_kernel(Gla<T> a, int lpr) {
  extern __shared__ float smem[];
  __shared__ float scratch[BLOCK / WAVE];
  float* s_a = smem;                  // [dim] decay
  float* s_k = s_a + a.dim;           // [dim]
  float* s_q = s_k + a.dim;           // [dim]
  float* s_o = s_q + a.dim;           // [groups][vdim]
  const int e = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const Entry en = entry_of(a.seq_start, e);
  const int slot = a.state_slots[e];
  const int groups = BLOCK / lpr, grp = tid / lpr, li = tid % lpr;
  float* state = slot < 0 ? nullptr
      : a.state + ((long)slot * a.heads + h) * a.dim * a.vdim;

  for (int t = 0; t < en.n; ++t) {
    const long row = en.row0 + t;
    const T* x = a.x + row * a.ld;
    const bool fresh = state == nullptr || a.positions[row] == 0;
    for (int d = tid; d < a.dim; d += BLOCK) {
      const int c = h * a.dim + d;
      if constexpr (CONST) {
        s_a[d] = a.decay[h];
        s_q[d] = silu_as<T>(ld1(x + c));
        s_k[d] = silu_as<T>(ld1(x + a.k_off + c));
        continue;
      }
      float z = a.a2b[c];
      for (int r = 0; r < a.rank; ++r)
        z += a.a2[(long)c * a.rank + r] * ld1(x + a.a_off + r);
      s_a[d] = expf(log_sigmoid_f(z) * a.inv_tau);
      s_q[d] = ld1(x + c) * a.qscale;
      s_k[d] = ld1(x + a.k_off + c);
    }
    __syncthreads();
    for (int c0 = li * VEC; c0 < a.vdim; c0 += lpr * VEC) {
      float v[VEC], o[VEC];
      ldv<VEC>(x + a.v_off + h * a.vdim + c0, v);
      #pragma unroll
      for (int j = 0; j < VEC; ++j) {
        if constexpr (CONST) v[j] = silu_as<T>(v[j]);
        o[j] = 0.f;
      }
      for (int d0 = grp; d0 < a.dim; d0 += groups * UNROLL) {
        float s[UNROLL][VEC];
        #pragma unroll
        for (int u = 0; u < UNROLL; ++u) {
          const int d = d0 + u * groups;
          if (!fresh && d < a.dim) {
            ld_state<VEC>(state + (long)d * a.vdim + c0, s[u]);
          } else {
            #pragma unroll
            for (int j = 0; j < VEC; ++j) s[u][j] = 0.f;
          }
        }
        #pragma unroll
        for (int u = 0; u < UNROLL; ++u) {
          const int d = d0 + u * groups;
          if (d < a.dim) {
            const float al = s_a[d], k = s_k[d], q = s_q[d];
            #pragma unroll
            for (int j = 0; j < VEC; ++j) {
              s[u][j] = al * s[u][j] + k * v[j];
              o[j] += q * s[u][j];
            }
            if (state != nullptr)
              st_state<VEC>(state + (long)d * a.vdim + c0, s[u]);
          }
        }
      }
      #pragma unroll
      for (int j = 0; j < VEC; ++j) s_o[grp * a.vdim + c0 + j] = o[j];
    }
    __syncthreads();
    float ss = 0.f;
    for (int c = tid; c < a.vdim; c += BLOCK) {
      float o = 0.f;
      for (int g = 0; g < groups; ++g) o += s_o[g * a.vdim + c];
      if constexpr (CONST) {
        st1(a.out + (row * a.heads + h) * a.vdim + c, o);
        continue;
      }
      s_o[c] = o;                     // column c of group 0: this thread's
      ss += o * o;
    }
    if constexpr (CONST) {
      __syncthreads();
      continue;
    }
    ss = block_sum<BLOCK / WAVE>(ss, scratch);
    const float inv = 1.f / sqrtf(ss / (float)a.vdim + a.eps);
    for (int c = tid; c < a.vdim; c += BLOCK) {
      const float g = ld1(x + a.g_off + h * a.vdim + c);
      st1(a.out + (row * a.heads + h) * a.vdim + c,
          s_o[c] * inv * a.norm[c] * (g * sigmoid_f(g)));
    }
    __syncthreads();
  }
}

}  // namespace

template <class T>
void launch_gla_recurrent(const Gla<T>& a, int entries, hipStream_t stream) {
  const bool vec = a.vdim % 4 == 0 && a.v_off % 4 == 0 && a.ld % 4 == 0;
  const int pieces = (a.vdim + (vec ? 3 : 0)) / (vec ? 4 : 1);
  int lpr = 1;                        // power of two, at most a wave
  while (lpr < pieces && lpr < WAVE) lpr *= 2;
  // partial outputs of all lane groups must fit the LDS
  while (lpr < BLOCK && (BLOCK / lpr) * a.vdim > 8192) lpr *= 2;
  const size_t lds = sizeof(float) * (3 * a.dim + (BLOCK / lpr) * a.vdim);
  const dim3 grid(entries, a.heads);
  auto go = [&](auto v, auto constant) {
    gla_recurrent_kernel<T, decltype(v)::value, decltype(constant)::value>
        <<<grid, dim3(BLOCK), lds, stream>>>(a, lpr);
  };
  auto by_vec = [&](auto constant) {
    if (vec) go(std::integral_constant<int, 4>{}, constant);
    else go(std::integral_constant<int, 1>{}, constant);
  };
  if (a.decay != nullptr) by_vec(std::true_type{});
  else by_vec(std::false_type{});
}

template void launch_gla_recurrent<float>(const Gla<float>&, int, hipStream_t);
template void launch_gla_recurrent<bf16_t>(const Gla<bf16_t>&, int,
                                           hipStream_t);
