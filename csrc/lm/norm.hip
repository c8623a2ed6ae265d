// Embedding + first norm, residual add (+ expert combine) + norm, and normed residual add + norm + input convolution,
// on the fp32 residual stream.
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

// sum over a workgroup of NT threads; `red` alternates between two buffers, one barrier per call
template <int NT>
__device__ __forceinline__ float block_sum(float v, float (*red)[NT / 64], int& turn) {
  v = wave_sum(v);
  float* r = red[turn];
  turn ^= 1;
  if ((threadIdx.x & 63) == 0) r[threadIdx.x >> 6] = v;
  __syncthreads();
  float x = r[0];
#pragma unroll
  for (int i = 1; i < NT / 64; ++i) x += r[i];
  return x;
}

// 4 elements as they lie in memory: converted when they are used, so that a load issued ahead is not waited for early
__device__ __forceinline__ float4_ raw4(const float* p) { return load4(p); }
__device__ __forceinline__ uint2_ raw4(const bf16_t* p) { return *reinterpret_cast<const uint2_*>(p); }
__device__ __forceinline__ float4_ wide4(float4_ v) { return v; }
__device__ __forceinline__ float4_ wide4(uint2_ v) {
  return float4_{__uint_as_float(v[0] << 16), __uint_as_float(v[0] & 0xffff0000u), __uint_as_float(v[1] << 16),
                 __uint_as_float(v[1] & 0xffff0000u)};
}

// The row stays in registers through both norms (RMS norms, or layer norms where there is a bias).  With a convolution a
// workgroup walks `run` consecutive rows, two of them loaded ahead, and keeps the last taps - 1 inputs in registers; the ones before its first row are recomputed from their
// residual rows (which is why x_out is not x then) or, before the step's first row of a sequence, come from the sequence's
// state.  Whatever the rows share (gains, taps, the rows' places) is read before the first row: a load inside the loop
// would wait for the rows ahead of it.  TD: the type of delta.
constexpr int conv_waves(int taps, int nt, int nv) { return taps > 0 && taps <= 4 && nt <= 512 && nv <= 2 ? 4 : 1; }   // per SIMD
template <typename T, typename TD, int NT, int NV, int TAPS>
__global__ void __launch_bounds__(NT, conv_waves(TAPS, NT, NV)) residual_norm_kernel(const ResidualNormArgs p) {
  constexpr bool CONV = TAPS > 0, KEEP = CONV && TAPS <= 4 && NV <= 2;   // KEEP: taps in registers
  constexpr int KN = KEEP ? NV : 1, KT = KEEP ? TAPS : 1;
  using Raw = decltype(raw4(static_cast<const TD*>(nullptr)));
  __shared__ float red[2][NT / 64];
  __shared__ __attribute__((aligned(16))) float sw[CONV ? 2 : 1][CONV ? NT * NV * 4 : 4];   // w (without it: bb), wb
  int turn = 0;
  const int c0 = threadIdx.x * 4;
  const float inv_w = 1.f / (float)p.width;
  const float4_ zero = float4_{0.f, 0.f, 0.f, 0.f};
  const bool has_delta = p.delta || p.ye;
  struct Row {
    float4_ x[NV];
    Raw d[NV];
  };
  auto fetch = [&](long row, Row& q) {
    const float* x = p.x ? p.x + row * p.Dp : nullptr;
    const T* e = x ? nullptr : static_cast<const T*>(p.table) + (long)min(max(p.ids[row], 0), p.V - 1) * p.Dp;
    const TD* d = static_cast<const TD*>(p.delta) + row * p.Dp;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = i * NT * 4 + c0;
      q.x[i] = zero;
      q.d[i] = Raw{};
      if (c < p.Dp) {
        q.x[i] = x ? load4(x + c) : load4(e + c) * p.scale;
        if (p.delta) q.d[i] = raw4(d + c);
        if constexpr (sizeof(TD) == 4) {
          if (p.ye) {                                      // (the only part then: no other delta)
            float4_ s = zero;
#pragma unroll 4
            for (int k = 0; k < p.top; ++k)
              s += p.wts[row * p.top + k] * load4(static_cast<const T*>(p.ye) + (long)p.slot_of[row * p.top + k] * p.Dp + c);
            q.d[i] = s;
          }
          for (int k = 1; k < p.parts; k += 3) {           // three loads at a time, none of them waited for alone
            float4_ e[3];
#pragma unroll
            for (int j = 0; j < 3; ++j) e[j] = raw4(d + min(k + j, p.parts - 1) * p.part_stride + c);
            q.d[i] += e[0] + (k + 1 < p.parts ? e[1] : zero) + (k + 2 < p.parts ? e[2] : zero);
          }
        }
      }
    }
  };
  auto gain = [&](const float* g, int which, int i) {      // gains of this thread's columns
    const int c = i * NT * 4 + c0;
    if constexpr (CONV) return *reinterpret_cast<const float4_*>(&sw[which][c]);
    else return load4(g + c);
  };
  // 1 / root of the mean square of d; with `centre` its mean is taken off first (pad columns stay out of both)
  auto scale_of = [&](float4_(&d)[NV], bool centre) {
    float ss = 0.f;
    if (centre) {
      float s = 0.f;
#pragma unroll
      for (int i = 0; i < NV; ++i) s += (d[i][0] + d[i][1]) + (d[i][2] + d[i][3]);
      const float mean = block_sum<NT>(s, red, turn) * inv_w;
#pragma unroll
      for (int i = 0; i < NV; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) d[i][j] = i * NT * 4 + c0 + j < p.width ? d[i][j] - mean : 0.f;
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) ss += d[i][0] * d[i][0] + d[i][1] * d[i][1] + d[i][2] * d[i][2] + d[i][3] * d[i][3];
    return 1.f / sqrtf(block_sum<NT>(ss, red, turn) * inv_w + p.eps);
  };
  auto add = [&](const Row& q, float4_(&v)[NV]) {
    float r = 0.f;
    float4_ d[NV];
    if (has_delta) {
#pragma unroll
      for (int i = 0; i < NV; ++i) d[i] = wide4(q.d[i]);
      r = p.wb ? p.mult * scale_of(d, p.bb != nullptr) : p.mult;
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = i * NT * 4 + c0;
      v[i] = q.x[i];
      if (c < p.Dp) {
        if (has_delta) {
          v[i] += p.wb ? d[i] * r * gain(p.wb, 1, i) : d[i] * r;
          if (p.bb) v[i] += p.mult * (CONV && !p.w ? gain(p.bb, 0, i) : load4(p.bb + c));
        }
        if (p.step) v[i] += load4(p.step + c);
      }
    }
  };
  auto norm = [&](float4_(&v)[NV]) {
    if (!p.w) return;
    const float r = scale_of(v, p.b != nullptr);
#pragma unroll
    for (int i = 0; i < NV; ++i)
      if (i * NT * 4 + c0 < p.Dp) {
        v[i] = v[i] * r * gain(p.w, 0, i);
        if (p.b) v[i] += load4(p.b + i * NT * 4 + c0);
      }
  };
  auto put = [&](auto* dst, const float4_(&v)[NV]) {
#pragma unroll
    for (int i = 0; i < NV; ++i)
      if (i * NT * 4 + c0 < p.Dp) store4(dst + i * NT * 4 + c0, v[i]);
  };

  float4_ v[NV];
  if constexpr (!CONV) {
    Row q;
    const long row = p.rows ? p.rows[blockIdx.x] : blockIdx.x;
    fetch(row, q);
    add(q, v);
    if (p.x_out) put(p.x_out + row * p.Dp, v);
    if (!p.h) return;
    norm(v);
    put(static_cast<T*>(p.h) + (long)blockIdx.x * p.Dp, v);
  } else {
    const int row0 = blockIdx.x * p.run, row1 = min(row0 + p.run, p.T);
    // lane i of every wave holds row i's place: its sequence, offset in the step, position, state slot, rows after it
    const int mt = min(row0 + (int)(threadIdx.x & 63), row1 - 1);
    const int m_b = p.row_seq ? p.row_seq[mt] : mt, m_pos = p.pos[mt], m_slot = p.slots[m_b];
    const int m_at = p.row_seq ? mt - p.q_start[m_b] : 0, m_left = p.row_seq ? p.q_lens[m_b] - 1 - m_at : 0;
    Row q0, q1;
    fetch(row0, q0);
    if (row0 + 1 < row1) fetch(row0 + 1, q1);
    float4_ hist[TAPS - 1][NV];                  // hist[j]: input of the row j + 1 before
    // the inputs before the step's first row of a sequence, `at` rows before this one
    auto past = [&](int slot, int at, int pos) {
      const float* st = p.state + (long)slot * (p.taps - 1) * p.Dp;
#pragma unroll
      for (int j = 0; j < TAPS - 1; ++j) {
        const bool in = j + 1 < p.taps && j + 1 > at && j + 1 <= pos && slot >= 0;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
          const int c = i * NT * 4 + c0;
          hist[j][i] = in && c < p.Dp ? load4(st + (long)(p.taps - 2 - j + at) * p.Dp + c) : zero;
        }
      }
    };
    int seq = -1;
    if (!p.row_seq) {                            // decode: this row's state in flight with the rest
      seq = row0;
      past(__builtin_amdgcn_readlane(m_slot, 0), 0, __builtin_amdgcn_readlane(m_pos, 0));
    }
    float4_ kc[KT][KN];                          // kc[j]: tap of the input j rows before
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = i * NT * 4 + c0;
      const bool in = c < p.Dp;
      const float* first = p.w ? p.w : p.bb;
      store4(&sw[0][c], in && first ? load4(first + c) : zero);     // read back by this thread only
      store4(&sw[1][c], in && has_delta ? load4(p.wb + c) : zero);
      if constexpr (KEEP) {
#pragma unroll
        for (int j = 0; j < TAPS; ++j)
          kc[j][i] = in && j < p.taps ? load4(p.cw + (long)(p.taps - 1 - j) * p.Dp + c) : zero;
      }
    }
    for (int t = row0; t < row1; ++t) {
      const int b = __builtin_amdgcn_readlane(m_b, t - row0), at = __builtin_amdgcn_readlane(m_at, t - row0);
      const int slot = __builtin_amdgcn_readlane(m_slot, t - row0);
      float* st = p.state + (long)max(slot, 0) * (p.taps - 1) * p.Dp;
      if (b != seq) {
        seq = b;
        past(slot, at, __builtin_amdgcn_readlane(m_pos, t - row0));
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j)
          if (j + 1 < p.taps && j + 1 <= at) {   // a row of this step
            Row o;
            fetch(t - j - 1, o);
            add(o, hist[j]);
            norm(hist[j]);
          }
      }
      add(q0, v);
      q0 = q1;
      if (t + 2 < row1) fetch(t + 2, q1);
      put(p.x_out + (long)t * p.Dp, v);
      norm(v);
      float4_ y[NV];
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int c = i * NT * 4 + c0;
        y[i] = v[i];
        if constexpr (KEEP) {
          y[i] += kc[0][i] * v[i];
#pragma unroll
          for (int j = 0; j < TAPS - 1; ++j) y[i] += kc[j + 1][i] * hist[j][i];
        } else if (c < p.Dp) {
          y[i] += load4(p.cw + (long)(p.taps - 1) * p.Dp + c) * v[i];
#pragma unroll
          for (int j = 0; j < TAPS - 1; ++j)
            if (j + 1 < p.taps) y[i] += load4(p.cw + (long)(p.taps - 2 - j) * p.Dp + c) * hist[j][i];
        }
      }
      put(static_cast<T*>(p.h) + (long)t * p.Dp, y);
      if (p.row_seq) {
        const int left = __builtin_amdgcn_readlane(m_left, t - row0);
        if (left < p.taps - 1) put(p.tail + ((long)b * (p.taps - 1) + p.taps - 2 - left) * p.Dp, v);
      } else if (slot >= 0 && p.taps > 1) {      // the only workgroup that reads this state
        put(st + (long)(p.taps - 2) * p.Dp, v);
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j)
          if (j + 2 < p.taps) put(st + (long)(p.taps - 3 - j) * p.Dp, hist[j]);
      }
#pragma unroll
      for (int j = TAPS - 2; j > 0; --j)
#pragma unroll
        for (int i = 0; i < NV; ++i) hist[j][i] = hist[j - 1][i];
#pragma unroll
      for (int i = 0; i < NV; ++i) hist[0][i] = v[i];
    }
  }
}

// Newest inputs first come from the step's tail, older ones move down inside the state (a portion shorter than the window).
__global__ void __launch_bounds__(256) conv_commit_kernel(const ConvCommitArgs p) {
  const int b = blockIdx.y, run = blockIdx.z, c = (blockIdx.x * 256 + threadIdx.x) * 4;
  const int slot = p.slots[b], n = p.q_lens[b], k = p.taps - 1;
  if (c >= p.Dp || slot < 0 || slot >= p.n_slots) return;
  float* st = p.state + ((long)run * p.n_slots + slot) * k * p.Dp + c;
  const float* tail = p.tail + ((long)run * p.B + b) * k * p.Dp + c;
  for (int j = 0; j < k; ++j)
    store4(st + (long)j * p.Dp, k - 1 - j < n ? load4(tail + (long)j * p.Dp) : load4(st + (long)(j + n) * p.Dp));
}

void launch_conv_commit(const ConvCommitArgs& a, hipStream_t s) {
  conv_commit_kernel<<<dim3((a.Dp + 1023) / 1024, a.B, a.runs), 256, 0, s>>>(a);
  SHAI_CHECK_LAUNCH();
}

// The angle is a float pair: position * frequency and its rounding error plus the frequency's remainder.
__global__ void __launch_bounds__(256) rope_rows_kernel(const RopeRowsArgs p) {
  const long id = (long)blockIdx.x * 256 + threadIdx.x;
  if (id >= (long)p.T * p.n) return;
  const int t = id / p.n, i = id % p.n;
  const float x = (float)p.pos[t], f = p.freq[2 * i], a = x * f;
  const float e = fmaf(x, f, -a) + x * p.freq[2 * i + 1];
  float s, c;
  sincosf(a, &s, &c);
  const float ce = 1.f - 0.5f * e * e, se = e - e * e * e * (1.f / 6.f);   // e is small: below 0.1 up to position 2^20
  p.out[2 * id] = c * ce - s * se;
  p.out[2 * id + 1] = s * ce + c * se;
}

void launch_rope_rows(const RopeRowsArgs& a, hipStream_t s) {
  rope_rows_kernel<<<((long)a.T * a.n + 255) / 256, 256, 0, s>>>(a);
  SHAI_CHECK_LAUNCH();
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

template <typename T, typename TD, int NT, int NV>
static void residual_norm(const ResidualNormArgs& a, hipStream_t s) {
  const int grid = a.cw ? (a.T + a.run - 1) / a.run : a.T;
  if (!a.cw) residual_norm_kernel<T, TD, NT, NV, 0><<<grid, NT, 0, s>>>(a);
  else if (a.taps <= 2) residual_norm_kernel<T, TD, NT, NV, 2><<<grid, NT, 0, s>>>(a);
  else if (a.taps <= 4) residual_norm_kernel<T, TD, NT, NV, 4><<<grid, NT, 0, s>>>(a);
  else residual_norm_kernel<T, TD, NT, NV, 16><<<grid, NT, 0, s>>>(a);
}

template <typename T, typename TD>
static void residual_norm(const ResidualNormArgs& a, hipStream_t s) {
  if (a.Dp <= 1024) residual_norm<T, TD, 256, 1>(a, s);
  else if (a.Dp <= 2048) residual_norm<T, TD, 256, 2>(a, s);
  else if (a.Dp <= 4096) residual_norm<T, TD, 512, 2>(a, s);
  else if (a.Dp <= 8192) residual_norm<T, TD, 1024, 2>(a, s);
  else residual_norm<T, TD, 1024, 4>(a, s);
}

void launch_residual_norm(const ResidualNormArgs& a, bool f32, hipStream_t s) {
  if (f32) residual_norm<float, float>(a, s);
  else if (a.parts || a.ye) residual_norm<bf16_t, float>(a, s);
  else residual_norm<bf16_t, bf16_t>(a, s);
  SHAI_CHECK_LAUNCH();
}

}  // namespace shai_lm
