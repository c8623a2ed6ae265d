// C = epi(A W^T), LDS-tiled bf16 form for many rows (prefill): 64 x 64 or 128 x 128 tiles of 4 waves or 256 x 256 tiles of
// 8, 64-wide k-tiles moved global -> LDS by DMA (buffer_load ... lds, 16 bytes per lane) into two stages; the load of
// k-tile t + 1 is issued before the MFMAs of t.  The bank swizzle is applied to the per-lane source chunk.  Buffer range checks zero-fill
// rows past the ends.  Dense or grouped by expert: the row tiles of a grouped product come from the tile list, each with
// its own W and with A rows gathered per lane.  Tiles are walked XCD by XCD in groups of 8 row tiles that share their W
// columns.
#include "lm_device.h"
#include "lm.h"

namespace shai_lm {

constexpr uint32_t kOob = 0x80000000u;

__device__ __forceinline__ int swz(int row, int ch) { return row * 64 + ((ch ^ ((row >> 1) & 7)) << 3); }

template <typename O, int EC, int BM, int BN, int WM, int WN>
__global__ void __launch_bounds__(WM * WN * 64, WM * WN == 4 ? 2 : 1) gemm_tile_kernel(const GemmArgs p) {
  constexpr int NW = WM * WN, TM = BM / WM, TN = BN / WN, IM = TM / 32, JN = TN / 32;
  constexpr int JA = BM / 8 / NW, JB = BN / 8 / NW, STAGE = (BM + BN) * 64;
  extern __shared__ __attribute__((aligned(16))) bf16_t smem[];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int wm = wid / WN, wn = wid % WN;

  const int tiles_m = p.tiles ? p.n_tiles : (p.M + BM - 1) / BM, tiles_n = (p.N + BN - 1) / BN;
  const int total = tiles_m * tiles_n;
  int bid = blockIdx.x;
  {
    const int xcd = bid & 7, q = total >> 3, r = total & 7;
    bid = (xcd < r ? xcd * (q + 1) : r * (q + 1) + (xcd - r) * q) + (bid >> 3);
  }
  constexpr int GROUP = 8;
  const int group = bid / (GROUP * tiles_n), first_m = group * GROUP;
  const int gsize = min(tiles_m - first_m, GROUP);
  const int in_group = bid - group * GROUP * tiles_n;
  const int mt = first_m + in_group % gsize, n0 = (in_group / gsize) * BN;
  int m0 = mt * BM, m_end = p.M, expert = 0;
  if (p.tiles) {
    expert = p.tiles[2 * mt];
    if (expert < 0) return;
    m0 = p.tiles[2 * mt + 1];
    m_end = min(p.offsets[expert + 1], m0 + BM);
  }
  const bf16_t* Wt = static_cast<const bf16_t*>(p.W) + (long)expert * p.N * p.K;
  const __amdgpu_buffer_rsrc_t rW = rsrc(Wt, (long)p.N * p.K * 2), rA = rsrc(p.A, ((long)(p.a_rows - 1) * p.lda + p.K) * 2);

  // byte offset of this lane's 16-byte chunk of every staged row at k = 0 (kOob: the row does not exist)
  const int lrow = lane >> 3, lpos = lane & 7;
  uint32_t offA[JA], offW[JB];
#pragma unroll
  for (int j = 0; j < JA; ++j) {
    const int r = (wid * JA + j) * 8 + lrow, m = m0 + r;
    const long src = m < m_end ? (p.gather ? p.gather[m] : m) : -1;
    offA[j] = src < 0 ? kOob : (uint32_t)((src * p.lda + (lpos ^ ((r >> 1) & 7)) * 8) * 2);
  }
#pragma unroll
  for (int j = 0; j < JB; ++j) {
    const int r = (wid * JB + j) * 8 + lrow, n = n0 + r;
    offW[j] = n < p.N ? (uint32_t)(((long)n * p.K + (lpos ^ ((r >> 1) & 7)) * 8) * 2) : kOob;
  }
  auto stage = [&](int buf, int kt) {
    bf16_t* sa = smem + buf * STAGE;
    bf16_t* sw = sa + BM * 64;
    const uint32_t kb = (uint32_t)kt * 128u;
#pragma unroll
    for (int j = 0; j < JB; ++j)
      dma16(rW, sw + (wid * JB + j) * 512, offW[j] == kOob ? kOob : offW[j] + kb);
#pragma unroll
    for (int j = 0; j < JA; ++j)
      dma16(rA, sa + (wid * JA + j) * 512, offA[j] == kOob ? kOob : offA[j] + kb);
  };

  float16_ acc[IM][JN];
#pragma unroll
  for (int i = 0; i < IM; ++i)
#pragma unroll
    for (int j = 0; j < JN; ++j)
#pragma unroll
      for (int r = 0; r < 16; ++r) acc[i][j][r] = 0.f;

  int nk = p.K / 64, k0 = 0;
  O* C = static_cast<O*>(p.C);
  if (p.splits > 1) {                            // this workgroup's part of K, its own partial sums
    k0 = (int)(blockIdx.y * (long)nk / p.splits);
    nk = (int)((blockIdx.y + 1L) * nk / p.splits) - k0;
    C += (long)blockIdx.y * p.M * p.N;
  }
  const int fr = lane & 31, fh = lane >> 5;
  stage(0, k0);
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  __syncthreads();
  for (int kt = 0; kt < nk; ++kt) {
    const int cur = kt & 1;
    if (kt + 1 < nk) stage(cur ^ 1, k0 + kt + 1);
    const bf16_t* sa = smem + cur * STAGE;
    const bf16_t* sw = sa + BM * 64;
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      bf16x8 af[IM], wf[JN];
#pragma unroll
      for (int i = 0; i < IM; ++i)
        af[i] = *reinterpret_cast<const bf16x8*>(sa + swz(wm * TM + i * 32 + fr, 2 * s + fh));
#pragma unroll
      for (int j = 0; j < JN; ++j)
        wf[j] = *reinterpret_cast<const bf16x8*>(sw + swz(wn * TN + j * 32 + fr, 2 * s + fh));
#pragma unroll
      for (int i = 0; i < IM; ++i)
#pragma unroll
        for (int j = 0; j < JN; ++j)
          acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(wf[j], af[i], acc[i][j], 0, 0, 0);
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
  }
  // bf16 results go through LDS, so that rows are stored 16 bytes a lane, whole lines at a time
  const bool glu = glu_class(EC) && glu_epi(p.epi);
  if (sizeof(O) == 2 && p.ldc % 8 == 0 && (glu || p.n_main % 8 == 0) && (p.n_main == p.N || n0 + BN <= p.n_main)) {
    constexpr int LD = BN + 8;
    __syncthreads();
#pragma unroll
    for (int i = 0; i < IM; ++i) {
      const int r = wm * TM + i * 32 + fr;
      const bool live = m0 + r < m_end;          // a row past the end has no angles to read
#pragma unroll
      for (int j = 0; j < JN; ++j)
#pragma unroll
        for (int g = 0; g < 4; ++g) {
          const int n = wn * TN + j * 32 + 8 * g + 4 * fh;
          float4_ c = float4_{acc[i][j][4 * g], acc[i][j][4 * g + 1], acc[i][j][4 * g + 2], acc[i][j][4 * g + 3]};
          if (live) epilogue_cols<O, EC>(p, m0 + r, n0 + n, c);
          if (glu) *reinterpret_cast<uint32_t*>(smem + r * LD + (n >> 1)) = pack2(c[0], c[1]);
          else store4(smem + r * LD + n, c);
        }
    }
    __syncthreads();
    const int cols = glu ? BN / 2 : BN, c0 = glu ? n0 >> 1 : n0, per = cols / 8, end = glu ? p.n_main >> 1 : p.n_main;
    bf16_t* out = reinterpret_cast<bf16_t*>(C);
    for (int id = tid; id < BM * per; id += NW * 64) {
      const int r = id / per, ch = (id % per) * 8;
      if (m0 + r < m_end && c0 + ch < end)
        *reinterpret_cast<uint4_*>(out + (long)(m0 + r) * p.ldc + c0 + ch) =
            *reinterpret_cast<const uint4_*>(smem + r * LD + ch);
    }
    return;
  }
#pragma unroll
  for (int i = 0; i < IM; ++i) {
    const int m = m0 + wm * TM + i * 32 + fr;
    if (m >= m_end) continue;
#pragma unroll
    for (int j = 0; j < JN; ++j)
#pragma unroll
      for (int g = 0; g < 4; ++g)
        store_cols<O, EC>(p, C, m, n0 + wn * TN + j * 32 + 8 * g + 4 * fh,
                      float4_{acc[i][j][4 * g], acc[i][j][4 * g + 1], acc[i][j][4 * g + 2], acc[i][j][4 * g + 3]});
  }
}

template <int BM, int BN, int WM, int WN>
static void tile(const GemmArgs& a, hipStream_t s) {
  const int tiles_m = a.tiles ? a.n_tiles : (a.M + BM - 1) / BM;
  const int grid = tiles_m * ((a.N + BN - 1) / BN);
  constexpr int lds = 2 * (BM + BN) * 64 * 2 > BM * (BN + 8) * 2 ? 2 * (BM + BN) * 64 * 2 : BM * (BN + 8) * 2;
  auto go = [&](auto k) {
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(k), hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    k<<<dim3(grid, a.splits > 1 ? a.splits : 1), WM * WN * 64, lds, s>>>(a);
  };
  const int ec = epi_class(a.epi);
  if (a.out_f32 && ec == EC_PLAIN) go(gemm_tile_kernel<float, EC_PLAIN, BM, BN, WM, WN>);
  else if (a.out_f32) go(gemm_tile_kernel<float, EC_ANY, BM, BN, WM, WN>);
  else if (ec == EC_PLAIN) go(gemm_tile_kernel<bf16_t, EC_PLAIN, BM, BN, WM, WN>);
  else if (ec == EC_CLAMP) go(gemm_tile_kernel<bf16_t, EC_CLAMP, BM, BN, WM, WN>);
  else if (ec == EC_GELU) go(gemm_tile_kernel<bf16_t, EC_GELU, BM, BN, WM, WN>);
  else go(gemm_tile_kernel<bf16_t, EC_OTHER, BM, BN, WM, WN>);
  SHAI_CHECK_LAUNCH();
}

void launch_gemm_tile(const GemmArgs& a, hipStream_t s) {
  // 256 x 256 tiles (8 waves) once they fill the chip, 128 x 128 (4 waves, two workgroups per CU) below and for narrow
  // outputs and short K (a second workgroup computes while the first one stores), 64 x 64 where those would leave most of
  // the chip idle
  const long m128 = (a.M + 127) / 128, n128 = (a.N + 127) / 128;
  const bool fills = a.N > 128 && a.K > 1536 && (long)((a.M + 255) / 256) * ((a.N + 255) / 256) >= 192;
  const bool big = a.tiles ? a.bm == 256 : a.splits <= 1 && fills;
  if (big) tile<256, 256, 2, 4>(a, s);
  else if (!a.tiles && a.splits <= 1 && m128 * n128 < 256 && a.K <= 2048) tile<64, 64, 2, 2>(a, s);
  else tile<128, 128, 2, 2>(a, s);
}

}  // namespace shai_lm
