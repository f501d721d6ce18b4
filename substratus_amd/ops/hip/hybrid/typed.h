// Loads and stores of float and bf16 activations as float, one or VEC at a
// time; the hybrid kernels are templates over the activation type.
#pragma once

#include "../common.h"

DEV_INLINE float ld1(const float* p) { return *p; }
DEV_INLINE float ld1(const bf16_t* p) { return bf2f(*p); }
DEV_INLINE void st1(float* p, float v) { *p = v; }
DEV_INLINE void st1(bf16_t* p, float v) { *p = f2bf(v); }

template <int VEC>
DEV_INLINE void ldv(const float* p, float* f) {
  if constexpr (VEC == 4) {
    const float4 u = *reinterpret_cast<const float4*>(p);
    f[0] = u.x; f[1] = u.y; f[2] = u.z; f[3] = u.w;
  } else {
    #pragma unroll
    for (int i = 0; i < VEC; ++i) f[i] = p[i];
  }
}

template <int VEC>
DEV_INLINE void ldv(const bf16_t* p, float* f) {
  if constexpr (VEC == 4) {
    const uint2 u = *reinterpret_cast<const uint2*>(p);
    const float2 a = unpack_bf16x2(u.x), b = unpack_bf16x2(u.y);
    f[0] = a.x; f[1] = a.y; f[2] = b.x; f[3] = b.y;
  } else {
    #pragma unroll
    for (int i = 0; i < VEC; ++i) f[i] = bf2f(p[i]);
  }
}

template <int VEC>
DEV_INLINE void stv(float* p, const float* f) {
  if constexpr (VEC == 4) {
    *reinterpret_cast<float4*>(p) = make_float4(f[0], f[1], f[2], f[3]);
  } else if constexpr (VEC == 2) {
    *reinterpret_cast<float2*>(p) = make_float2(f[0], f[1]);
  } else {
    #pragma unroll
    for (int i = 0; i < VEC; ++i) p[i] = f[i];
  }
}

template <int VEC>
DEV_INLINE void stv(bf16_t* p, const float* f) {
  if constexpr (VEC == 4) {
    *reinterpret_cast<uint2*>(p) =
        make_uint2(pack_bf16x2(f[0], f[1]), pack_bf16x2(f[2], f[3]));
  } else if constexpr (VEC == 2) {
    *reinterpret_cast<unsigned*>(p) = pack_bf16x2(f[0], f[1]);
  } else {
    #pragma unroll
    for (int i = 0; i < VEC; ++i) p[i] = f2bf(f[i]);
  }
}

// Two bf16 in one instruction. Not by inline assembly: the compiler does not
// see what that reads, and leaves out the wait that the result of an
// exponential or a reciprocal needs ahead of its first use.
DEV_INLINE unsigned cvt_pk_bf16(float lo, float hi) {
  typedef __attribute__((ext_vector_type(2))) __bf16 bf16x2;
  typedef __attribute__((ext_vector_type(2))) float floatx2;
  return __builtin_bit_cast(
      unsigned, __builtin_convertvector((floatx2){lo, hi}, bf16x2));
}

DEV_INLINE float sigmoid_f(float z) { return 1.f / (1.f + expf(-z)); }

// ln(sigmoid(z)) without overflow at either end
DEV_INLINE float log_sigmoid_f(float z) {
  return fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
}

// Hidden values of a gated feed-forward.
enum class Glu {
  SILU,      // silu(g) u
  RELU,      // max(g, 0) u
  CLAMPED,   // g sigmoid(1.702 g) (u + 1), g up to limit, u within it
};

DEV_INLINE float glu_f(Glu kind, float g, float u, float limit) {
  if (kind == Glu::RELU) return fmaxf(g, 0.f) * u;
  float s = 1.f;
  if (kind == Glu::CLAMPED) {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit) + 1.f;
    s = 1.702f;
  }
  return g * sigmoid_f(s * g) * u;
}

DEV_INLINE float softplus_f(float z) {
  return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z)));
}

// log2(1 + e^z) and z sigmoid(z) in a few instructions, to 2e-6 relative
DEV_INLINE float softplus2_f(float z) {
  constexpr float log2e = 1.44269504088896340736f;
  const float x = __builtin_amdgcn_exp2f(-fabsf(z) * log2e);
  const float small = x * (1.f - x * (0.5f - x * (1.f / 3.f - x *
                          (0.25f - x * 0.2f)))) * log2e;
  return fmaxf(z, 0.f) * log2e +
         (x < 0.1f ? small : __builtin_amdgcn_logf(1.f + x));
}

DEV_INLINE float fast_silu_f(float z) {
  constexpr float log2e = 1.44269504088896340736f;
  return z * __builtin_amdgcn_rcpf(
      1.f + __builtin_amdgcn_exp2f(-z * log2e));
}

// One request's place in the batch, for kernels over single tokens and over
// portions of prompts alike: rows [row0, row0 + n) of the packed activations.
struct Entry {
  int row0, n;
};

// seq_start null: entry e is the single row e.
DEV_INLINE Entry entry_of(const int* seq_start, int e) {
  if (seq_start == nullptr) return {e, 1};
  const int a = seq_start[e];
  return {a, seq_start[e + 1] - a};
}
