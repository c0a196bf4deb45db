// Device helpers of the recurrent kernels. Sums over 4, 8 or 16 neighbouring lanes of a wave on the VALU (DPP operands of the add, no LDS round trip). Every lane of
// the group receives the same bits: each step adds a value to its mirror image, which is symmetric.
#pragma once

#include "common.h"

namespace die {

template <int CTRL> __device__ __forceinline__ float dpp_add(float x) {
  return x + __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, x), CTRL, 0xf, 0xf, true));
}

// LN in {4, 8, 16}: the sum over the LN lanes of the group lane / LN
template <int LN> __device__ __forceinline__ float group_sum(float x) {
  static_assert(LN == 4 || LN == 8 || LN == 16, "group size");
  if constexpr (LN == 16) x = dpp_add<0x140>(x);   // row_mirror: lane i and 15 - i
  if constexpr (LN >= 8) x = dpp_add<0x141>(x);    // row_half_mirror: i and 7 - i
  x = dpp_add<0xB1>(x);                            // quad_perm 1, 0, 3, 2
  return dpp_add<0x4E>(x);                         // quad_perm 2, 3, 0, 1
}

// softplus; FAST (bf16 steps): hardware exponential and logarithm (v_exp_f32 / v_log_f32), a series where 1 + e^z rounds
template <bool FAST> __device__ __forceinline__ float softplus_of(float z) {
  if constexpr (FAST) {
    const float e = __expf(-fabsf(z));
    const float l = e < 9.765625e-4f ? e - 0.5f * e * e : __logf(1.0f + e);
    return fmaxf(z, 0.f) + l;
  } else {
    return z > 20.f ? z : log1pf(expf(z));
  }
}
// e^x; FAST: 2^(x log2 e) on the hardware's 2^x
template <bool FAST> __device__ __forceinline__ float exp_of(float x) {
  if constexpr (FAST)
    return __builtin_amdgcn_exp2f(x * 1.4426950408889634f);
  else
    return expf(x);
}

}  // namespace die
