// hyb_mfma.cuh -- what the matrix-core kernels of layer-list decoders share: operand types, base-two exponentials, f32 numbers as three bf16 operands.
#pragma once
#include "common.cuh"

namespace mrs {
namespace mfma {

typedef short bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x16 __attribute__((ext_vector_type(16)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
__device__ __forceinline__ float exp2_f(float v) { return __builtin_amdgcn_exp2f(v); }
constexpr float LOG2E = 1.4426950408889634f;

// a pair of f32 numbers as three packed pairs of bf16 that add up to them: every term takes the top sixteen bits of what is left
__device__ __forceinline__ void split3_pair(float a, float b, unsigned *w) {
#pragma unroll
  for (int c = 0; c < 3; ++c) {
    const unsigned ua = __float_as_uint(a) & 0xffff0000u, ub = __float_as_uint(b) & 0xffff0000u;
    w[c] = (ua >> 16) | ub;
    a -= __uint_as_float(ua);
    b -= __uint_as_float(ub);
  }
}
// eight f32 numbers as three bf16 operands whose sum is the numbers
__device__ __forceinline__ void split3(const float *p, bf16x8 *out) {
  unsigned w[4][3];
#pragma unroll
  for (int j = 0; j < 4; ++j) split3_pair(p[2 * j], p[2 * j + 1], w[j]);
#pragma unroll
  for (int c = 0; c < 3; ++c) out[c] = __builtin_bit_cast(bf16x8, make_int4((int)w[0][c], (int)w[1][c], (int)w[2][c], (int)w[3][c]));
}

}  // namespace mfma
}  // namespace mrs
