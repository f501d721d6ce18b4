// What recurrences over chunks of tokens on the matrix cores share
// (gla_chunk.hip, delta_chunk.hip): 32x32x16 products whose factors are split
// into bf16 high and low parts.
#pragma once

#include "typed.h"

typedef __attribute__((ext_vector_type(8))) short short8;
typedef __attribute__((ext_vector_type(4))) short short4v;
typedef __attribute__((ext_vector_type(16))) float float16v;

namespace {

constexpr int C = 32;               // tokens per chunk
constexpr float DIRECT_BELOW = -86.f;      // in powers of two: e^-60
constexpr float LOG2E = 1.44269504088896340736f;
constexpr int BUFFER_FLAGS = 0x00020000;   // untyped, offset-checked
constexpr int OUT_OF_RANGE = 0x7ffffff0;   // beyond any buffer's end

DEV_INLINE float exp2_f(float x) { return __builtin_amdgcn_exp2f(x); }

// two floats as bf16 high parts and low parts, each pair in one word
DEV_INLINE void split_pair(float f0, float f1, unsigned* hi, unsigned* lo) {
  *hi = cvt_pk_bf16(f0, f1);
  const float2 back = unpack_bf16x2(*hi);
  *lo = cvt_pk_bf16(f0 - back.x, f1 - back.y);
}

// 8 consecutive accumulator rows as bf16 high and low operand parts
template <int AT, class F>
DEV_INLINE void split_rows(const F& f, short8* hi, short8* lo) {
  unsigned h[4], l[4];
  #pragma unroll
  for (int i = 0; i < 4; ++i)
    split_pair(f[AT + 2 * i], f[AT + 2 * i + 1], &h[i], &l[i]);
  *hi = *reinterpret_cast<const short8*>(h);
  *lo = *reinterpret_cast<const short8*>(l);
}

DEV_INLINE float16v mma(short8 a, short8 b, float16v c) {
  return __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b, c, 0, 0, 0);
}

}  // namespace
