// The gated delta rule, token by token, in float or bf16 (formulas in
// delta.h). One workgroup per (entry, head) walks the entry's rows; for
// single tokens it is the decode step: the state is read once, before
// anything else, and written once.
//
// `lpr` lanes cover a state row (VEC columns each); the workgroup's lane
// groups take key channels in turn and hold them in registers (R rows each;
// R 0: heads too large for that, the state is read again after each of the
// rule's two halves). S^T k and S^T q of the decayed state are summed in one
// pass: S_new^T q = S^T q + (k . q) u.
#include "delta.h"

namespace {

constexpr int BLOCK = 512;

template <class T, int VEC, int R>
__global__ __launch_bounds__(BLOCK)
void delta_recurrent_kernel(Delta<T> a, int lpr) {
  extern __shared__ float smem[];
  __shared__ float scratch[4][BLOCK / WAVE];
  const int groups = BLOCK / lpr;
  float* s_k = smem;                    // [dim]
  float* s_q = s_k + a.dim;             // [dim]
  float* s_g = s_q + a.dim;             // [dim]
  float* s_u = s_g + a.dim;             // [vdim]
  float* s_pk = s_u + a.vdim;           // [groups][vdim]
  float* s_pq = s_pk + groups * a.vdim; // [groups][vdim]
  const int e = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const Entry en = entry_of(a.seq_start, e);
  if (en.n <= 0) return;
  const int slot = a.state_slots[e];
  const int grp = tid / lpr, li = tid % lpr;
  const int hk = h / (a.heads / a.kv_heads);
  const int nq = a.kv_heads * a.dim;
  const float qscale = 1.f / sqrtf((float)a.dim), rate = a.rate[h];
  float* state = slot < 0 ? nullptr
      : a.state + ((long)slot * a.heads + h) * a.dim * a.vdim;
  const bool held = state != nullptr && a.positions[en.row0] > 0;

  constexpr int RR = R > 0 ? R : 1;
  float s[RR][VEC];
  const int c0 = li * VEC;              // R > 0: the thread's only columns
  if constexpr (R > 0) {
    #pragma unroll
    for (int i = 0; i < R; ++i) {
      const int d = grp + i * groups;
      #pragma unroll
      for (int j = 0; j < VEC; ++j) s[i][j] = 0.f;
      if (held && d < a.dim && c0 < a.vdim)
        ldv<VEC>(state + (long)d * a.vdim + c0, s[i]);
    }
  }

  for (int t = 0; t < en.n; ++t) {
    const long row = en.row0 + t;
    const T* x = a.qkv + row * a.ld;
    const T* v = x + 2 * nq + h * a.vdim;
    float qq = 0.f, kk = 0.f, kq = 0.f;
    for (int d = tid; d < a.dim; d += BLOCK) {
      const float q = ld1(x + hk * a.dim + d);
      const float k = ld1(x + nq + hk * a.dim + d);
      const long c = (long)h * a.dim + d;
      qq += q * q; kk += k * k; kq += k * q;
      s_q[d] = q; s_k[d] = k;
      s_g[d] = expf(-rate * softplus_f(a.z[row * a.heads * a.dim + c] +
                                       a.zb[c]));
    }
    qq = block_sum<BLOCK / WAVE>(qq, scratch[0]);
    kk = block_sum<BLOCK / WAVE>(kk, scratch[1]);
    kq = block_sum<BLOCK / WAVE>(kq, scratch[2]);
    const float iq = qscale / sqrtf(qq + UNIT_EPS);
    const float ik = 1.f / sqrtf(kk + UNIT_EPS);
    kq *= iq * ik;

    for (int c = c0; c < a.vdim; c += lpr * VEC) {
      float pk[VEC], pq[VEC];
      #pragma unroll
      for (int j = 0; j < VEC; ++j) pk[j] = pq[j] = 0.f;
      auto add = [&](int d, float* f) {
        const float g = s_g[d], k = s_k[d], q = s_q[d];
        #pragma unroll
        for (int j = 0; j < VEC; ++j) {
          f[j] *= g;
          pk[j] += k * f[j];
          pq[j] += q * f[j];
        }
      };
      if constexpr (R > 0) {
        #pragma unroll
        for (int i = 0; i < R; ++i)
          if (grp + i * groups < a.dim) add(grp + i * groups, s[i]);
      } else if (state != nullptr && (held || t > 0)) {
        for (int d = grp; d < a.dim; d += groups) {
          float f[VEC];
          ldv<VEC>(state + (long)d * a.vdim + c, f);
          add(d, f);
        }
      }
      #pragma unroll
      for (int j = 0; j < VEC; ++j) {
        s_pk[grp * a.vdim + c + j] = pk[j] * ik;
        s_pq[grp * a.vdim + c + j] = pq[j] * iq;
      }
    }
    __syncthreads();
    const float beta = sigmoid_f(ld1(a.beta + row * a.b_ld + h));
    float ss = 0.f;
    for (int c = tid; c < a.vdim; c += BLOCK) {
      float pk = 0.f, o = 0.f;
      for (int g = 0; g < groups; ++g) {
        pk += s_pk[g * a.vdim + c];
        o += s_pq[g * a.vdim + c];
      }
      const float u = beta * (ld1(v + c) - pk);
      o += kq * u;
      s_u[c] = u;
      s_pq[c] = o;                      // column c of group 0: this thread's
      ss += o * o;
    }
    ss = block_sum<BLOCK / WAVE>(ss, scratch[3]);
    const float inv = a.mult / sqrtf(ss / (float)a.vdim + a.eps);
    for (int c = tid; c < a.vdim; c += BLOCK)
      st1(a.out + row * a.out_ld + (long)h * a.vdim + c,
          s_pq[c] * inv * a.norm[c] *
              sigmoid_f(ld1(a.gate + row * a.g_ld + (long)h * a.vdim + c)));
    for (int c = c0; c < a.vdim; c += lpr * VEC) {
      if constexpr (R > 0) {
        #pragma unroll
        for (int i = 0; i < R; ++i) {
          const int d = grp + i * groups;
          if (d < a.dim) {
            const float k = s_k[d] * ik;
            #pragma unroll
            for (int j = 0; j < VEC; ++j) s[i][j] += k * s_u[c + j];
          }
        }
      } else if (state != nullptr) {
        for (int d = grp; d < a.dim; d += groups) {
          float f[VEC];
          const float k = s_k[d] * ik, g = s_g[d];
          if (held || t > 0) {
            ldv<VEC>(state + (long)d * a.vdim + c, f);
          } else {
            #pragma unroll
            for (int j = 0; j < VEC; ++j) f[j] = 0.f;
          }
          #pragma unroll
          for (int j = 0; j < VEC; ++j) f[j] = g * f[j] + k * s_u[c + j];
          stv<VEC>(state + (long)d * a.vdim + c, f);
        }
      }
    }
    __syncthreads();
  }
  if constexpr (R > 0) {
    if (state != nullptr && c0 < a.vdim) {
      #pragma unroll
      for (int i = 0; i < R; ++i) {
        const int d = grp + i * groups;
        if (d < a.dim) stv<VEC>(state + (long)d * a.vdim + c0, s[i]);
      }
    }
  }
}

}  // namespace

template <class T>
void launch_delta_recurrent(const Delta<T>& a, int entries,
                            hipStream_t stream) {
  const bool vec = a.vdim % 4 == 0;
  const int pieces = vec ? a.vdim / 4 : a.vdim;
  int lpr = 1;                          // power of two
  while (lpr < pieces && lpr < WAVE) lpr *= 2;
  // partial sums of all lane groups must fit the LDS
  while (lpr < BLOCK && (BLOCK / lpr) * a.vdim > 4096) lpr *= 2;
  const int groups = BLOCK / lpr, rows = (a.dim + groups - 1) / groups;
  const bool fits = pieces <= lpr;      // one piece of columns per thread
  const size_t lds =
      sizeof(float) * (3 * a.dim + a.vdim + 2 * groups * a.vdim);
  auto go = [&](auto v, auto r) {
    delta_recurrent_kernel<T, decltype(v)::value, decltype(r)::value>
        <<<dim3(entries, a.heads), dim3(BLOCK), lds, stream>>>(a, lpr);
  };
  using std::integral_constant;
  auto by_rows = [&](auto v) {
    if (fits && rows <= 8) go(v, integral_constant<int, 8>{});
    else if (fits && rows <= 32) go(v, integral_constant<int, 32>{});
    else go(v, integral_constant<int, 0>{});
  };
  if (vec) by_rows(integral_constant<int, 4>{});
  else by_rows(integral_constant<int, 1>{});
}

template void launch_delta_recurrent<float>(const Delta<float>&, int,
                                            hipStream_t);
template void launch_delta_recurrent<bf16_t>(const Delta<bf16_t>&, int,
                                             hipStream_t);
