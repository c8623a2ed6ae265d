// Embedding + first norm, and residual add (+ expert combine) + norm, on the fp32 residual stream.
// One 256-thread workgroup per row; the row stays in registers between the add and the norm (width <= 16384).
#include "lm_device.h"
#include "lm.h"

namespace shai_lm {

template <typename T, int NV>
__global__ void __launch_bounds__(256) embed_norm_kernel(const EmbedNormArgs p) {
  __shared__ float red[4];
  const long t = blockIdx.x;
  const int id = min(max(p.ids[t], 0), p.V - 1), pv = p.prev ? p.prev[t] : -1;
  const T* e = static_cast<const T*>(p.table) + (long)id * p.Dp;
  const T* g = nullptr;
  if (p.bigram) {
    const long row = pv < 0 ? p.buckets : (long)((unsigned long)((long)pv * p.mul_prev + (long)id * p.mul_cur) %
                                                 (unsigned long)p.buckets);
    g = static_cast<const T*>(p.bigram) + row * p.Dp;
  }
  float4_ v[NV];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * 256 + threadIdx.x) * 4;
    v[i] = float4_{0.f, 0.f, 0.f, 0.f};
    if (c < p.Dp) {
      v[i] = load4(e + c);
      if (g) v[i] += load4(g + c);
      store4(p.x + t * p.Dp + c, v[i]);
      ss += v[i][0] * v[i][0] + v[i][1] * v[i][1] + v[i][2] * v[i][2] + v[i][3] * v[i][3];
    }
  }
  ss = block_sum256(ss, red);
  const float r = 1.f / sqrtf(ss / (float)p.width + p.eps);
  T* h = static_cast<T*>(p.h) + t * p.Dp;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * 256 + threadIdx.x) * 4;
    if (c < p.Dp) store4(h + c, v[i] * r * (load4(p.w + c) + 1.f));
  }
}

template <typename T, int NV>
__global__ void __launch_bounds__(256) add_norm_kernel(const AddNormArgs p) {
  __shared__ float red[4];
  const long row = p.rows ? p.rows[blockIdx.x] : blockIdx.x;
  const bool keep = p.rows == nullptr;
  float* x = p.x + row * p.Dp;
  float4_ v[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * 256 + threadIdx.x) * 4;
    v[i] = c < p.Dp ? load4(x + c) : float4_{0.f, 0.f, 0.f, 0.f};
  }
  if (p.ye) {
#pragma unroll 4
    for (int k = 0; k < p.top; ++k) {
      const float wk = p.wts[row * p.top + k];
      const T* y = static_cast<const T*>(p.ye) + (long)p.slot_of[row * p.top + k] * p.Dp;
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int c = (i * 256 + threadIdx.x) * 4;
        if (c < p.Dp) v[i] += wk * load4(y + c);
      }
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * 256 + threadIdx.x) * 4;
    if (c < p.Dp) {
      if (p.dense) v[i] += load4(static_cast<const T*>(p.dense) + row * p.Dp + c);
      if (p.inject) v[i] += load4(p.inject + row * p.Dp + c);
      if (keep) store4(x + c, v[i]);
      ss += v[i][0] * v[i][0] + v[i][1] * v[i][1] + v[i][2] * v[i][2] + v[i][3] * v[i][3];
    }
  }
  if (!p.w) return;
  ss = block_sum256(ss, red);
  const float r = 1.f / sqrtf(ss / (float)p.width + p.eps);
  T* h = static_cast<T*>(p.h) + (long)blockIdx.x * p.Dp;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * 256 + threadIdx.x) * 4;
    if (c < p.Dp) store4(h + c, v[i] * r * (load4(p.w + c) + 1.f));
  }
}

#define SHAI_LM_ROWS(KERNEL, a, f32, s)                                                            \
  do {                                                                                             \
    const int nv = ((a).Dp + 1023) / 1024;                                                         \
    auto go = [&](auto tag) {                                                                      \
      using T = decltype(tag);                                                                     \
      if (nv <= 1) KERNEL<T, 1><<<(a).T, 256, 0, s>>>(a);                                          \
      else if (nv <= 2) KERNEL<T, 2><<<(a).T, 256, 0, s>>>(a);                                     \
      else if (nv <= 4) KERNEL<T, 4><<<(a).T, 256, 0, s>>>(a);                                     \
      else if (nv <= 8) KERNEL<T, 8><<<(a).T, 256, 0, s>>>(a);                                     \
      else KERNEL<T, 16><<<(a).T, 256, 0, s>>>(a);                                                 \
    };                                                                                             \
    if (f32) go(float{});                                                                          \
    else go(bf16_t{});                                                                             \
    SHAI_CHECK_LAUNCH();                                                                           \
  } while (0)

void launch_embed_norm(const EmbedNormArgs& a, bool f32, hipStream_t s) { SHAI_LM_ROWS(embed_norm_kernel, a, f32, s); }
void launch_add_norm(const AddNormArgs& a, bool f32, hipStream_t s) { SHAI_LM_ROWS(add_norm_kernel, a, f32, s); }

}  // namespace shai_lm
