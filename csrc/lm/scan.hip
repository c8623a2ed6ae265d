// Gated linear recurrence over time (minGRU), channel by channel and in fp32:
//   z = sigmoid(zx[.., c] + bias),  c = u + 1/2 for u >= 0, sigmoid(u) below, u = zx[.., W + c] + bias,
//   S_t = (1 - z) S_(t-1) + z c,  out = S_t silu(g).
// S is kept per sequence slot; a sequence's first token starts from zero whatever the slot holds.
//
// Prefill: a sequence longer than `len` is cut into chunks.  scan_totals composes every chunk but the last into one step
// (S -> A S + B; the first chunk's is applied to the stored state already), scan folds the chunks before its own and
// walks its rows.  Only totals are exchanged between workgroups, in two launches.  Decode: scan alone.
#include "lm_device.h"

namespace shai_lm {

constexpr int kAhead = 8;                        // rows loaded ahead of the recurrence

__device__ __forceinline__ void scan_gate(float z, float u, float& a, float& b) {
  // 1 - sigmoid(z) as sigmoid(-z): no cancellation
  const float e = expf(-fabsf(z)), r = 1.f / (1.f + e), hi = r, lo = e * r;
  a = z >= 0.f ? lo : hi;
  b = (z >= 0.f ? hi : lo) * (u >= 0.f ? u + 0.5f : sigmoid_f(u));
}

template <typename F>
__device__ __forceinline__ void scan_rows(const ScanArgs& p, long t0, int n, int c, F&& f) {
  const float bz = p.bias[c], bu = p.bias[p.W + c];
  const float* src = p.zx + t0 * 2 * p.W + c;
  auto one = [&](int i, float z, float u) {
    float a, b;
    scan_gate(z + bz, u + bu, a, b);
    f(t0 + i, a, b);
  };
  int i0 = 0;
  for (; i0 + kAhead <= n; i0 += kAhead) {
    float z[kAhead], u[kAhead];
#pragma unroll
    for (int i = 0; i < kAhead; ++i) {
      z[i] = src[(long)(i0 + i) * 2 * p.W];
      u[i] = src[(long)(i0 + i) * 2 * p.W + p.W];
    }
#pragma unroll
    for (int i = 0; i < kAhead; ++i) one(i0 + i, z[i], u[i]);
  }
  for (; i0 < n; ++i0) one(i0, src[(long)i0 * 2 * p.W], src[(long)i0 * 2 * p.W + p.W]);
}

__device__ __forceinline__ float scan_start(const ScanArgs& p, long t0, int b, int c) {
  const int slot = p.slots[b];
  return slot >= 0 && p.pos[t0] > 0 ? p.state[(long)slot * p.W + c] : 0.f;
}

__global__ void __launch_bounds__(128) scan_totals_kernel(const ScanArgs p) {
  const int c = blockIdx.x * 128 + threadIdx.x, k = blockIdx.y, b = blockIdx.z;
  const int n = p.q_lens[b];
  if (c >= p.W || (k + 1) * p.len >= n) return;  // the last chunk's total is not needed
  const long q0 = p.q_start[b];
  const float start = k == 0 ? scan_start(p, q0, b, c) : 0.f;
  float A = 1.f, B = start;
  scan_rows(p, q0 + (long)k * p.len, p.len, c, [&](long, float a, float bb) {
    A *= a;
    B = a * B + bb;
  });
  float* w = p.ws + ((long)b * p.chunks + k) * 2 * p.W + c;
  w[0] = k == 0 ? start : A;                     // the first chunk's own factor is in B already
  w[p.W] = B;
}

template <typename T>
__global__ void __launch_bounds__(128) scan_kernel(const ScanArgs p) {
  const int c = blockIdx.x * 128 + threadIdx.x, k = blockIdx.y, b = blockIdx.z;
  const int n = p.q_lens ? p.q_lens[b] : 1;
  if (c >= p.W || k * p.len >= n) return;
  const long q0 = p.q_start ? p.q_start[b] : b;
  const int rows = min(p.len, n - k * p.len);
  const float* w = p.ws + (long)b * p.chunks * 2 * p.W + c;
  float S;
  if (n <= p.len) {
    S = scan_start(p, q0, b, c);
  } else if (k == 0) {
    S = w[0];                                    // not the slot: the last chunk's workgroup writes it in this launch
  } else {
    S = w[p.W];
#pragma unroll 4
    for (int j = 1; j < k; ++j) S = w[(long)j * 2 * p.W] * S + w[(long)j * 2 * p.W + p.W];
  }
  const T* g = static_cast<const T*>(p.g);
  T* out = static_cast<T*>(p.out);
  scan_rows(p, q0 + (long)k * p.len, rows, c, [&](long t, float a, float bb) {
    S = a * S + bb;
    const float gv = load1(g + t * p.W + c);
    store1(out + t * p.W + c, S * (gv * sigmoid_f(gv)));
  });
  const int slot = p.slots[b];
  if (slot >= 0 && (k + 1) * p.len >= n) p.state[(long)slot * p.W + c] = S;
}

void launch_mingru_scan(const ScanArgs& a, bool f32, hipStream_t s) {
  const dim3 grid((a.W + 127) / 128, a.chunks, a.B);
  if (a.chunks > 1) scan_totals_kernel<<<dim3(grid.x, a.chunks - 1, a.B), 128, 0, s>>>(a);
  if (f32) scan_kernel<float><<<grid, 128, 0, s>>>(a);
  else scan_kernel<bf16_t><<<grid, 128, 0, s>>>(a);
  SHAI_CHECK_LAUNCH();
}

}  // namespace shai_lm
