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

// DMA to LDS: 16 bytes a lane, lane-linear from a wave-uniform LDS address; a buffer's range check zero-fills past its end
typedef __attribute__((address_space(3))) void lds_void;
typedef __attribute__((address_space(1))) void glb_void;
__device__ __forceinline__ __amdgpu_buffer_rsrc_t rsrc(const void* b, long bytes) {
  return __builtin_amdgcn_make_buffer_rsrc(const_cast<void*>(b), (short)0, (int)bytes, 0x00020000);
}
__device__ __forceinline__ void dma16(__amdgpu_buffer_rsrc_t r, bf16_t* lds_wave_base, uint32_t voff) {
  __builtin_amdgcn_raw_ptr_buffer_load_lds(r, (lds_void*)lds_wave_base, 16, voff, 0, 0, 0);
}
__device__ __forceinline__ void dma16(const bf16_t* src, bf16_t* lds_wave_base) {
  __builtin_amdgcn_global_load_lds((glb_void*)src, (lds_void*)lds_wave_base, 16, 0, 0);
}

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
// the same with `red` changing between two buffers (`turn`), so that calls may follow each other with one barrier each
__device__ __forceinline__ float block_sum256(float v, float (*red)[4], int& turn) {
  v = wave_sum(v);
  float* r = red[turn];
  turn ^= 1;
  if ((threadIdx.x & 63) == 0) r[threadIdx.x >> 6] = v;
  __syncthreads();
  return (r[0] + r[1]) + (r[2] + r[3]);
}

// xIELU: ap z^2 + z / 2 above zero, an (exp(z) - 1 - z) + z / 2 below.  `fast` (results that are rounded to bf16): the
// hardware exponential, a short series near zero.
__device__ __forceinline__ float xielu(float z, float ap, float an, bool fast) {
  float e;
  if (fast) {
    const float series = z * z * (0.5f + z * (1.f / 6.f + z * (1.f / 24.f + z * (1.f / 120.f))));
    e = z > -0.3f ? series : __builtin_amdgcn_exp2f(z * 1.4426950408889634f) - 1.f - z;
  } else {
    e = expm1f(z) - z;
  }
  return (z > 0.f ? ap * z * z : an * e) + 0.5f * z;
}

// the tanh form of gelu: z / (1 + exp(-2 u)) = z (1 + tanh u) / 2.  `fast`: the hardware exponential and reciprocal.
__device__ __forceinline__ float gelu_tanh(float z, bool fast) {
  const float u = 0.7978845608028654f * (z + 0.044715f * z * z * z);
  if (fast) return z * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-2.f * 1.4426950408889634f * u));
  return z / (1.f + expf(-2.f * u));
}

// Epilogue of 4 consecutive columns n .. n + 3 of row m, in place (a GLU's two results: c[0], c[1]).
template <typename O, int EC>
__device__ __forceinline__ void epilogue_cols(const GemmArgs& p, long m, int n, float4_& c) {
  constexpr bool fast = sizeof(O) == 2;
  const auto is = [&](int epi) { return epi_in(EC, epi) && p.epi == epi; };
  if (is(EPI_CLAMP_GLU)) {
    c[0] = clamp_glu(c[0], c[1], p.param);
    c[1] = clamp_glu(c[2], c[3], p.param);
  } else if (is(EPI_SOFTCAP)) {
#pragma unroll
    for (int i = 0; i < 4; ++i) c[i] = p.param * tanhf(c[i] / p.param);
  } else if (is(EPI_XIELU)) {
    const float ap = p.vec[0], an = p.vec[1];
#pragma unroll
    for (int i = 0; i < 4; ++i) c[i] = xielu(c[i], ap, an, fast);
  } else if (is(EPI_GELU_GLU)) {
    c[0] = gelu_tanh(c[0], fast) * c[1];
    c[1] = gelu_tanh(c[2], fast) * c[3];
  } else if (is(EPI_RELU2)) {
#pragma unroll
    for (int i = 0; i < 4; ++i) c[i] = n >= p.n_act ? c[i] : c[i] > 0.f ? c[i] * c[i] : 0.f;
  } else if (is(EPI_GELU_ROWS)) {
    if (n < p.N) {
      const long at = (long)min(max(p.ids[m], 0), p.table_rows - 1) * p.table_ld + n;
      const float4_ e = p.table_f32 ? load4(static_cast<const float*>(p.table) + at)
                                    : load4(static_cast<const bf16_t*>(p.table) + at);
#pragma unroll
      for (int i = 0; i < 4; ++i) c[i] = gelu_tanh(c[i], fast) * e[i];
    }
  } else if (is(EPI_ROTARY)) {
    const int d = n % p.head - p.rot0;
    if (d >= 0 && d < p.rot && n < p.N) {
      const float* t = p.rope + m * p.rot + d;
      const float u = c[0], v = c[1];
      c[0] = u * t[0] - v * t[1];
      c[1] = v * t[0] + u * t[1];
      if (d + 2 < p.rot) {
        const float u2 = c[2], v2 = c[3];
        c[2] = u2 * t[2] - v2 * t[3];
        c[3] = v2 * t[2] + u2 * t[3];
      }
    }
  }
}

// Store 4 consecutive columns n .. n + 3 of row m after the epilogue.  `out`: C of this product.
template <typename O, int EC>
__device__ __forceinline__ void store_cols(const GemmArgs& p, O* out, long m, int n, float4_ c) {
  if (n >= p.n_main) {
    const int ld = p.N - p.n_main, j = n - p.n_main;
    float* o = p.side + m * ld + j;
    if ((ld & 3) == 0) {
      if (n < p.N) store4(o, c);
      return;
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (n + i < p.N) o[i] = c[i];
    return;
  }
  epilogue_cols<O, EC>(p, m, n, c);
  if (glu_class(EC) && glu_epi(p.epi)) {
    const int j = n >> 1;
    if (n < p.N) store1(out + m * p.ldc + j, c[0]);
    if (n + 2 < p.N) store1(out + m * p.ldc + j + 1, c[1]);
    return;
  }
  O* o = out + m * p.ldc + n;
  if (((p.n_main | (int)p.ldc) & 3) == 0) {
    if (n < p.N) store4(o, c);
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (n + i < p.N) store1(o + i, c[i]);
  }
}

}  // namespace shai_lm
