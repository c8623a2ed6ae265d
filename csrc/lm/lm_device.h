// Device helpers of the decoder-block kernels: element access for bf16 / fp32 tensors.
#pragma once
#include "../kernels/common.h"
#include "lm.h"

namespace shai_lm {
using namespace shai;
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));

// 4 consecutive elements as fp32
__device__ __forceinline__ float4_ load4(const float* p) { return *reinterpret_cast<const float4_*>(p); }
__device__ __forceinline__ float4_ load4(const bf16_t* p) {
  const uint2_ v = *reinterpret_cast<const uint2_*>(p);
  return float4_{__uint_as_float(v[0] << 16), __uint_as_float(v[0] & 0xffff0000u), __uint_as_float(v[1] << 16),
                 __uint_as_float(v[1] & 0xffff0000u)};
}
__device__ __forceinline__ void store4(float* p, float4_ v) { *reinterpret_cast<float4_*>(p) = v; }
__device__ __forceinline__ void store4(bf16_t* p, float4_ v) {
  *reinterpret_cast<uint2_*>(p) = uint2_{pack2(v[0], v[1]), pack2(v[2], v[3])};
}
__device__ __forceinline__ float load1(const float* p) { return *p; }
__device__ __forceinline__ float load1(const bf16_t* p) { return bf2f(*p); }
__device__ __forceinline__ void store1(float* p, float v) { *p = v; }
__device__ __forceinline__ void store1(bf16_t* p, float v) { *p = f2bf(v); }

__device__ __forceinline__ float sigmoid_f(float x) { return 1.f / (1.f + expf(-x)); }
// clamped GLU: value (u + 1), gate g sigmoid(1.702 g), both limited
__device__ __forceinline__ float clamp_glu(float g, float u, float lim) {
  g = fminf(g, lim);
  u = fminf(fmaxf(u, -lim), lim);
  return g * sigmoid_f(1.702f * g) * (u + 1.f);
}
// sum over a 256-thread workgroup; every thread returns the same value
__device__ __forceinline__ float block_sum256(float v, float* red) {
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  return (red[0] + red[1]) + (red[2] + red[3]);
}

// Store 4 consecutive columns n .. n + 3 of row m after the epilogue.
template <typename O>
__device__ __forceinline__ void store_cols(const GemmArgs& p, long m, int n, float4_ c) {
  O* out = static_cast<O*>(p.C);
  if (n >= p.n_main) {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (n + i < p.N) p.side[m * (p.N - p.n_main) + n + i - p.n_main] = c[i];
    return;
  }
  if (p.epi == EPI_CLAMP_GLU) {
    const int ld = p.n_main >> 1, j = n >> 1;
    if (n < p.N) store1(out + m * ld + j, clamp_glu(c[0], c[1], p.param));
    if (n + 2 < p.N) store1(out + m * ld + j + 1, clamp_glu(c[2], c[3], p.param));
    return;
  }
  if (p.epi == EPI_SOFTCAP) {
#pragma unroll
    for (int i = 0; i < 4; ++i) c[i] = p.param * tanhf(c[i] / p.param);
  }
  O* o = out + m * p.N + n;
  if ((p.N & 3) == 0) {
    if (n < p.N) store4(o, c);
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (n + i < p.N) store1(o + i, c[i]);
  }
}

}  // namespace shai_lm
