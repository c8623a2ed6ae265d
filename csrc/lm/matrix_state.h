// Device helpers of the kernels with a matrix state per head (hgrn2.hip, rule.hip): fp32 values as a bf16 value plus its bf16
// remainder in matrix products.
#pragma once
#include "lm_device.h"

namespace shai_lm {

constexpr float kInvLn2 = 1.4426950408889634f;

__device__ __forceinline__ float silu_exact(float x) { return x / (1.f + expf(-x)); }
__device__ __forceinline__ float silu_fast(float x) {
  return x * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-x * kInvLn2));
}
// value | remainder of two floats as packed words (value in the upper half)
__device__ __forceinline__ void pack_pair(float a, float b, uint32_t& pa, uint32_t& pb) {
  const uint32_t ua = __float_as_uint(a), ub = __float_as_uint(b);
  const uint32_t lo = pack2(a - __uint_as_float(ua & 0xffff0000u), b - __uint_as_float(ub & 0xffff0000u));
  pa = __builtin_amdgcn_perm(ua, lo, 0x07060100u);
  pb = __builtin_amdgcn_perm(ub, lo, 0x07060302u);
}
struct Split {                                    // 8 values of a matrix operand and their remainders
  bf16x8 hi, lo;
};
__device__ __forceinline__ Split unpack(uint4_ a, uint4_ b) {
  uint4_ h, l;
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    h[i] = __builtin_amdgcn_perm(a[2 * i + 1], a[2 * i], 0x07060302u);
    l[i] = __builtin_amdgcn_perm(a[2 * i + 1], a[2 * i], 0x05040100u);
    h[2 + i] = __builtin_amdgcn_perm(b[2 * i + 1], b[2 * i], 0x07060302u);
    l[2 + i] = __builtin_amdgcn_perm(b[2 * i + 1], b[2 * i], 0x05040100u);
  }
  return Split{__builtin_bit_cast(bf16x8, h), __builtin_bit_cast(bf16x8, l)};
}
__device__ __forceinline__ Split split8(float4_ a, float4_ b) {
  uint4_ h, l;
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const float4_ x = i ? b : a;
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const uint32_t u0 = __float_as_uint(x[2 * j]), u1 = __float_as_uint(x[2 * j + 1]);
      h[2 * i + j] = __builtin_amdgcn_perm(u1, u0, 0x07060302u);
      l[2 * i + j] = pack2(x[2 * j] - __uint_as_float(u0 & 0xffff0000u), x[2 * j + 1] - __uint_as_float(u1 & 0xffff0000u));
    }
  }
  return Split{__builtin_bit_cast(bf16x8, h), __builtin_bit_cast(bf16x8, l)};
}
__device__ __forceinline__ float4_ mac(bf16x8 a, bf16x8 b, float4_ c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ float4_ mac(const Split& a, const Split& b, float4_ c) {
  return mac(a.hi, b.lo, mac(a.lo, b.hi, mac(a.hi, b.hi, c)));
}

// stored head sizes
#define SHAI_LM_STATE(FN, ...)                                      \
  do {                                                              \
    if (a.dk == 64 && a.dv == 64) FN(64, 64, __VA_ARGS__);          \
    else if (a.dk == 64 && a.dv == 128) FN(64, 128, __VA_ARGS__);   \
    else if (a.dk == 128 && a.dv == 64) FN(128, 64, __VA_ARGS__);   \
    else if (a.dk == 128 && a.dv == 128) FN(128, 128, __VA_ARGS__); \
    else FN(256, 256, __VA_ARGS__);                                 \
  } while (0)

}  // namespace shai_lm
