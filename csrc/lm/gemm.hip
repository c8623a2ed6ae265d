// C = epi(A W^T), streaming form: a workgroup owns NT x 16 rows of W and up to MT x 16 rows of A, its waves split K and
// fold their fp32 partials through LDS.  W goes straight from memory to the matrix cores (no LDS round trip), so the
// kernel runs at the speed the weights arrive: decode steps, routers, and expert products with few rows per expert.
// bf16: v_mfma_f32_16x16x32_bf16; fp32: v_mfma_f32_16x16x4_f32 (full fp32 products).
//
// Operands are swapped (C^T = W A^T): a lane ends up with 4 consecutive output columns of one row, so a (gate, up) row
// pair of W is folded in registers.  A k-step covers 64 values; lane group g = lane / 16 takes values 16 g .. 16 g + 15
// of it in both operands (the order of k inside a dot product is free), i.e. every W row is read 128 bytes at a time.
//
// Dense: row tiles of A are blockIdx.y, products of a batch (one per attention head, say) or parts of K (partial sums for
// the consumer to add) blockIdx.z.  Grouped (experts): blockIdx.y is an entry of the tile list and blockIdx.z a 16 MT-row
// part of it; rows past the expert's last slot are computed on a clamped row and not stored.
#include "lm_device.h"
#include "lm.h"

namespace shai_lm {

template <typename T>
struct Frag;
template <>
struct Frag<bf16_t> {
  uint4_ v[2];
  __device__ __forceinline__ void load(const bf16_t* p) {
    v[0] = *reinterpret_cast<const uint4_*>(p);
    v[1] = *reinterpret_cast<const uint4_*>(p + 8);
  }
  static __device__ __forceinline__ float4_ mac(const Frag& w, const Frag& a, float4_ c) {
#pragma unroll
    for (int i = 0; i < 2; ++i)
      c = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, w.v[i]),
                                                  __builtin_bit_cast(bf16x8, a.v[i]), c, 0, 0, 0);
    return c;
  }
};
template <>
struct Frag<float> {
  float4_ v[4];
  __device__ __forceinline__ void load(const float* p) {
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = *reinterpret_cast<const float4_*>(p + 4 * i);
  }
  static __device__ __forceinline__ float4_ mac(const Frag& w, const Frag& a, float4_ c) {
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) c = __builtin_amdgcn_mfma_f32_16x16x4f32(w.v[i][j], a.v[i][j], c, 0, 0, 0);
    return c;
  }
};

template <typename T, typename O, int EC, int MT, int NT, int NW, int D>
__global__ void __launch_bounds__(NW * 64) gemm_stream_kernel(const GemmArgs p) {
  __shared__ float4_ red[NW][MT][64];
  const int lane = threadIdx.x & 63;
  const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int r = lane & 15, g = lane >> 4;
  const int n0 = blockIdx.x * 16 * NT;
  int row0 = blockIdx.y * 16 * MT, rows_end = p.M, expert = 0;
  if (p.tiles) {
    expert = p.tiles[2 * blockIdx.y];
    if (expert < 0) return;
    row0 = p.tiles[2 * blockIdx.y + 1];
    rows_end = min(p.offsets[expert + 1], row0 + p.bm);
    row0 += blockIdx.z * 16 * MT;
  }
  if (row0 >= rows_end) return;
  const T* W = static_cast<const T*>(p.W) + (long)expert * p.N * p.K;
  const T* A = static_cast<const T*>(p.A);
  O* C = static_cast<O*>(p.C);
  if (p.batch > 1) {
    W += blockIdx.z * p.w_batch;
    A += blockIdx.z * p.a_batch;
    C += blockIdx.z * p.c_batch;
  }
  const T* wp[NT];
  const T* ap[MT];
#pragma unroll
  for (int i = 0; i < NT; ++i) wp[i] = W + (long)min(n0 + 16 * i + r, p.N - 1) * p.K + g * 16;
#pragma unroll
  for (int j = 0; j < MT; ++j) {
    int m = min(row0 + 16 * j + r, rows_end - 1);
    if (p.gather) m = p.gather[m];
    ap[j] = A + m * p.lda + g * 16;
  }
  float4_ acc[NT][MT];
#pragma unroll
  for (int i = 0; i < NT; ++i)
#pragma unroll
    for (int j = 0; j < MT; ++j) acc[i][j] = float4_{0.f, 0.f, 0.f, 0.f};
  // this wave's k-steps are first + wid, first + wid + NW, ...; D of them are in flight
  int steps = p.K / 64, first = 0;
  if (p.splits > 1) {
    first = (int)(blockIdx.z * (long)steps / p.splits);
    steps = (int)((blockIdx.z + 1L) * steps / p.splits);
    C += (long)blockIdx.z * p.M * p.N;
  }
  Frag<T> w[D][NT], x[D][MT];
  auto fetch = [&](int u, int s) {
    if (s < steps) {
      const long k = (long)s * 64;
#pragma unroll
      for (int i = 0; i < NT; ++i) w[u][i].load(wp[i] + k);
#pragma unroll
      for (int j = 0; j < MT; ++j) x[u][j].load(ap[j] + k);
    }
  };
#pragma unroll
  for (int u = 0; u < D; ++u) fetch(u, first + wid + u * NW);
  for (int s0 = first + wid; s0 < steps; s0 += NW * D) {
#pragma unroll
    for (int u = 0; u < D; ++u) {
      if (s0 + u * NW < steps) {
#pragma unroll
        for (int j = 0; j < MT; ++j)
#pragma unroll
          for (int i = 0; i < NT; ++i) acc[i][j] = Frag<T>::mac(w[u][i], x[u][j], acc[i][j]);
        fetch(u, s0 + (u + D) * NW);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < NT; ++i) {
    if (i > 0) __syncthreads();
#pragma unroll
    for (int j = 0; j < MT; ++j) red[wid][j][lane] = acc[i][j];
    __syncthreads();
    for (int t = wid; t < MT; t += NW) {
      float4_ c = red[0][t][lane];
#pragma unroll
      for (int w = 1; w < NW; ++w) c += red[w][t][lane];
      const int m = row0 + 16 * t + r;
      if (m < rows_end) store_cols<O, EC>(p, C, m, n0 + 16 * i + 4 * g, c);
    }
  }
}

// Workgroup shapes (16 MT rows of A x 16 NT rows of W, NW waves along K, D k-steps in flight), from a sweep at decode
// sizes: enough workgroups to fill the chip come first, then fewer passes over W (MT), then fewer re-reads of A (NT).
template <typename T, typename O, int EC>
static void stream(const GemmArgs& a, hipStream_t s) {
  auto go = [&](auto kernel, int mt, int nt, int nw) {
    const dim3 grid((a.N + 16 * nt - 1) / (16 * nt), a.tiles ? a.n_tiles : (a.M + 16 * mt - 1) / (16 * mt),
                    a.tiles ? (a.bm + 16 * mt - 1) / (16 * mt) : a.splits > 1 ? a.splits : a.batch);
    kernel<<<grid, 64 * nw, 0, s>>>(a);
  };
  constexpr bool H = sizeof(T) == 2;              // fp32 fragments are twice the registers
#define GO(MT_, NT_, NW_, D_) go(gemm_stream_kernel<T, O, EC, MT_, NT_, NW_, H ? D_ : 1>, MT_, NT_, NW_)
  const int rows = a.tiles ? a.bm : a.M;
  if (a.splits > 1) {
    if constexpr (epi_in(EC, EPI_NONE)) {         // partial sums
      if (rows <= 16) GO(1, 1, 4, 4);
      else if (rows <= 32) GO(2, 2, 4, 4);
      else if (a.N < 2560 && a.K < 16384) GO(4, 2, 4, 3);
      else GO(4, 4, 4, 2);
    }
  } else if (!a.tiles && a.K <= 256) {            // too few k-steps to split over many waves
    if (rows <= 16) GO(1, 2, 2, 2);
    else if (rows <= 32) GO(2, 2, 2, 2);
    else GO(4, 2, 2, 2);
  } else if (rows <= 16 || a.N < 512) GO(1, 1, 8, 4);
  else if (a.tiles) GO(4, 2, 4, 2);
  else if (a.N < 3072 || (rows <= 32 && a.N < 5120)) GO(2, 1, 8, 4);
  else if (a.N < 5120) GO(2, 2, 8, 2);
  else if (rows <= 32) GO(2, 4, 4, 3);
  else if (a.N < 8192) GO(4, 2, 4, 2);
  else if (H && a.N <= 12288) GO(4, 3, 4, 2);    // up to 20480 columns: as few as give every CU one workgroup
  else if (a.N <= 16384) GO(4, 4, 4, 3);
  else if (H && a.N <= 20480) GO(4, 5, 4, 2);
  else GO(4, 4, 2, 3);
#undef GO
  SHAI_CHECK_LAUNCH();
}

void launch_gemm(const GemmArgs& a, bool f32, hipStream_t s) {
  const int ec = epi_class(a.epi);
  if (f32) stream<float, float, EC_ANY>(a, s);
  else if (a.out_f32 && ec == EC_PLAIN) stream<bf16_t, float, EC_PLAIN>(a, s);
  else if (a.out_f32) stream<bf16_t, float, EC_ANY>(a, s);
  else if (ec == EC_PLAIN) stream<bf16_t, bf16_t, EC_PLAIN>(a, s);
  else if (ec == EC_CLAMP) stream<bf16_t, bf16_t, EC_CLAMP>(a, s);
  else if (ec == EC_GELU) stream<bf16_t, bf16_t, EC_GELU>(a, s);
  else stream<bf16_t, bf16_t, EC_OTHER>(a, s);
}

}  // namespace shai_lm
