// Weight-quantized linear layers for gfx950 (MI355X).
//
//   y[m, n] = (sum_k x[m, k] * q[n, k]) * scale[n] (+ bias[n])      q in {e4m3fn, int8, bf16}
//
// Replaces the NxDI quantized Column/RowParallel linears the reference reaches through
// /root/reference/vllm_neuron/worker/neuronx_distributed_model_loader.py:339-348, with the
// quantization keys of loader.py:886-898.
//
// Storage: the library owns the weights, so they are kept in the shape the matrix cores
// want.  A tile is 16 output rows x 64 bytes of K (fp8/int8; 32 elements for bf16) = 1 KiB
// laid out lane-linear: lane l holds the 16 bytes of row (l & 15), k-chunk (l >> 4).  One
// 16-byte load per lane is then (a) a perfectly coalesced 1 KiB wave read and (b) exactly
// the A operand of v_mfma_f32_16x16x32_bf16 after an in-register fp8->bf16 decode (two
// k-steps per load for the 1-byte types).  Tiles of one 16-row group are contiguous along K,
// so a wave streams a dense byte range.
//
// Decode (M <= 16): gemv_kernel — pure weight streaming, HBM-bound.  x lives in LDS in
//   fragment order; every wave streams a K-slice of one row-tile with 2 x 8 KiB in flight;
//   the MFMA does the dot products AND the cross-lane reduction; waves combine through LDS
//   in a fixed order (deterministic, no atomics).
// Prefill (M > 16): gemm_kernel — 128 x 128 tile, x through swizzled LDS, W straight
//   from global in fragment order.
//
// Both share one epilogue on D[n = 4g + r][m = c] (lane = 16 g + c): dequant scale, bias,
// then fp32 store | RoPE + q/KV-pool scatter | SwiGLU.

#include "linear_kernels.h"

#include "linear_device.h"

namespace mi {

// instantiated in gemv_bf16.hip / gemv_f8.hip / gemv_i8.hip
template <int WD>
int launch_gemv_wd(const LinearW& w, int M, int pro, const ProArgs& p, int epi, const EpiArgs& e, hipStream_t s);
extern template int launch_gemv_wd<MI_W_BF16>(const LinearW&, int, int, const ProArgs&, int, const EpiArgs&, hipStream_t);
extern template int launch_gemv_wd<MI_W_F8E4M3>(const LinearW&, int, int, const ProArgs&, int, const EpiArgs&, hipStream_t);
extern template int launch_gemv_wd<MI_W_INT8>(const LinearW&, int, int, const ProArgs&, int, const EpiArgs&, hipStream_t);

size_t gemv_lds_bytes(int M, int K) { return gemv_image_lds_bytes(M, K); }
bool gemv_fits(int M, int K) { (void)K; return gemv_rows_fit(M); }

int launch_gemv(const LinearW& w, int M, int pro, const ProArgs& p, int epi, const EpiArgs& e, hipStream_t s) {
  MI_CHECK(M >= 1 && M <= 32, "gemv: M must be 1..32");
  MI_CHECK(w.N % 16 == 0 && w.K % 64 == 0, "gemv: N % 16 == 0 and K % 64 == 0 required");
  switch (w.wd) {
    case MI_W_BF16: return launch_gemv_wd<MI_W_BF16>(w, M, pro, p, epi, e, s);
    case MI_W_F8E4M3: return launch_gemv_wd<MI_W_F8E4M3>(w, M, pro, p, epi, e, s);
    case MI_W_INT8: return launch_gemv_wd<MI_W_INT8>(w, M, pro, p, epi, e, s);
  }
  set_error("gemv: bad weight dtype");
  return MI_EINVAL;
}

// =====================================================================================
// GEMM (context encoding)
// =====================================================================================
// Work-group tile 128 (n) x 128 (m); 4 waves as 2 (n) x 2 (m), each 64 x 64 = 4 x 4 MFMA tiles.
// x tile [128 m][64 k] bf16 through LDS (16-byte chunks XOR-swizzled by row); W fragments
// straight from the pre-tiled global image.
constexpr int kBM = 128, kBN = 128, kBK = 64;

// XOR swizzle of the 16-byte chunks of a 128-byte activation row in LDS.  A ds_read_b128 is
// serviced in four groups of 16 lanes ({0-3,12-15,20-27}, ...: MI355X_MICROARCH.md, LDS); with the
// fragment addressing of the MFMA B operand (lane (g, c): row c, chunk 2g / 2g+1 for 1-byte weights,
// g / 4+g for bf16 weights) the plain `chunk ^ (row & 7)` image is conflict-free for the bf16-weight
// chunk order but puts every group of the 1-byte order two-deep on its banks; folding row bit 3 into
// the key makes that order conflict-free too (enumerated over the lane groups).
template <int WD>
__device__ __forceinline__ int xs_swz(int r) { return WD == MI_W_BF16 ? (r & 7) : ((r & 7) ^ ((r >> 3) & 1)); }

// SPLIT: grid.z K-slices write raw fp32 accumulators to slab[z][m][n] (see gemm_a8_kernel).
// Registers are kept under 170 per lane so that three work-groups share a CU (the same lesson as
// the FP8 GEMM): the weight tiles of a K-step are decoded once into their A fragments, the raw
// registers are refilled with the next K-step's tiles straight away, and the activation
// fragments are read per 16-token tile instead of all at once.
template <int WD, int EPI, bool SPLIT>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(WD == MI_W_BF16 ? 2 : 3, WD == MI_W_BF16 ? 2 : 3))) void gemm_kernel(const uint4* __restrict__ W, int NT, int KT, int T, int K,
                                                   const uint16_t* __restrict__ x, int ldx, EpiArgs e,
                                                   float* __restrict__ slab) {
  __shared__ __attribute__((aligned(16))) uint4 xs[kBM * 8];  // 16 KiB
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int g = lane >> 4, c = lane & 15;
  const int wn = wave >> 1, wm = wave & 1;
  // XCD-aware tile order (see gemm_a8_kernel): XCD = linear id % 8 owns every eighth weight slab
  // and walks all token blocks of a slab back to back
  const int mtiles = ceil_div(T, kBM), ntiles = ceil_div(NT, kBN / 16);
  const int xcd = blockIdx.x & 7, seq = blockIdx.x >> 3;
  const int mblk = seq % mtiles, nblk = (seq / mtiles) * 8 + xcd;
  if (nblk >= ntiles) return;
  const int m0 = mblk * kBM, nt0 = nblk * (kBN / 16) + wn * 4;
  const int nks_all = K / kBK;
  const int ks_per = SPLIT ? ceil_div(nks_all, (int)gridDim.z) : nks_all;
  const int ks_beg = SPLIT ? (int)blockIdx.z * ks_per : 0;
  const int nks = min(ks_beg + ks_per, nks_all);
  constexpr int WPK = (WD == MI_W_BF16) ? 2 : 1;  // weight tiles per K-step

  f32x4_t acc[4][4];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = f32x4_t{0.f, 0.f, 0.f, 0.f};

  // x staging: thread -> rows (tid/8 + 32 i), 16-byte chunk tid%8
  const int srow = tid >> 3, sch = tid & 7;
  u32x4_t xr[4], wr[4][WPK];
  auto load_x = [&](int ks) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int m = min(m0 + srow + 32 * i, T - 1);   // rows past T: a copy of the last row, never stored
      xr[i] = *reinterpret_cast<const u32x4_t*>(x + (size_t)m * ldx + ks * kBK + sch * 8);
    }
  };
  auto load_w = [&](int ks) {
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int t = 0; t < WPK; ++t)
        wr[i][t] = *reinterpret_cast<const u32x4_t*>(W + ((size_t)min(nt0 + i, NT - 1) * KT + ks * WPK + t) * 64 + lane);
  };

  if (ks_beg < nks) {
    load_x(ks_beg);
    load_w(ks_beg);
  }
  for (int ks = ks_beg; ks < nks; ++ks) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int r = srow + 32 * i;
      *reinterpret_cast<u32x4_t*>(&xs[r * 8 + (sch ^ xs_swz<WD>(r))]) = xr[i];
    }
    bf16x8_t a0[4], a1[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      if constexpr (WD == MI_W_BF16) {
        a0[i] = __builtin_bit_cast(bf16x8_t, wr[i][0]);
        a1[i] = __builtin_bit_cast(bf16x8_t, wr[i][1]);
      } else {
        const u32x4_t w4 = wr[i][0];
        a0[i] = decode8<WD>(w4[0], w4[1]);
        a1[i] = decode8<WD>(w4[2], w4[3]);
      }
    }
    __syncthreads();
    if (ks + 1 < nks) {      // the raw registers are free again: next K-step's operands
      load_x(ks + 1);
      load_w(ks + 1);
    }
#pragma unroll
    for (int mt = 0; mt < 4; ++mt) {
      const int r = wm * 64 + mt * 16 + c;
      const int ch0 = (WD == MI_W_BF16) ? g : 2 * g, ch1 = (WD == MI_W_BF16) ? 4 + g : 2 * g + 1;
      const bf16x8_t b0 = __builtin_bit_cast(bf16x8_t, xs[r * 8 + (ch0 ^ xs_swz<WD>(r))]);
      const bf16x8_t b1 = __builtin_bit_cast(bf16x8_t, xs[r * 8 + (ch1 ^ xs_swz<WD>(r))]);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        acc[i][mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a0[i], b0, acc[i][mt], 0, 0, 0);
        acc[i][mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a1[i], b1, acc[i][mt], 0, 0, 0);
      }
    }
    __syncthreads();
  }

#pragma unroll
  for (int i = 0; i < 4; ++i) {
    if (nt0 + i >= NT) continue;
#pragma unroll
    for (int mt = 0; mt < 4; ++mt) {
      const int m = m0 + wm * 64 + mt * 16 + c;
      if (m >= T) continue;
      const int n0 = (nt0 + i) * 16 + g * 4;
      if constexpr (SPLIT) {
        *reinterpret_cast<float4*>(slab + ((size_t)blockIdx.z * T + m) * (NT * 16) + n0) =
            make_float4(acc[i][mt][0], acc[i][mt][1], acc[i][mt][2], acc[i][mt][3]);
      } else {
        epilogue<EPI>(e, m, n0, acc[i][mt]);
      }
    }
  }
}

template <int EPI>
__global__ __launch_bounds__(256) void splitk_reduce_kernel(const float* __restrict__ slab, int KS, int T, int N, EpiArgs e);

// K-split for grids too small to occupy the chip (768 work-groups are resident at once): below 256
// tiles aim for 512 work-groups, below 384 for 768 (rule measured on the FP8 GEMM).
static int gemm_pick_splitk(int tiles, int nks, int T, int N, size_t ws_bytes) {
  if (!ws_bytes || tiles >= 384) return 1;
  int KS = min(min(8, nks), ceil_div(tiles < 256 ? 512 : 768, tiles));
  while (KS > 1 && (size_t)KS * T * N * sizeof(float) > ws_bytes) --KS;
  return KS;
}

template <int WD>
static int launch_gemm_wd(const LinearW& w, int T, const uint16_t* x, int ldx, int epi, const EpiArgs& e, hipStream_t s,
                          float* splitk_ws, size_t splitk_ws_bytes, SlabSum* defer) {
  const int NT = w.N / 16, KT = w.K / tile_k(WD);
  const int mtiles = ceil_div(T, kBM), ntiles = ceil_div(w.N, kBN);
  const int KS = gemm_pick_splitk(mtiles * ntiles, w.K / kBK, T, w.N, splitk_ws ? splitk_ws_bytes : 0);
  dim3 grid(8 * mtiles * ceil_div(ntiles, 8), 1, KS);
  const uint4* W = reinterpret_cast<const uint4*>(w.w);
#define MI_G(EPI_) \
  do { \
    if (KS == 1) { \
      hipLaunchKernelGGL((gemm_kernel<WD, EPI_, false>), grid, dim3(256), 0, s, W, NT, KT, T, w.K, x, ldx, e, nullptr); \
    } else { \
      hipLaunchKernelGGL((gemm_kernel<WD, EPI_, true>), grid, dim3(256), 0, s, W, NT, KT, T, w.K, x, ldx, e, splitk_ws); \
      if (defer && (EPI_ == EPI_RESID || EPI_ == EPI_F32)) { *defer = SlabSum{splitk_ws, KS, T, w.N, e.scale, e.bias, e.row_scale}; } \
      else hipLaunchKernelGGL((splitk_reduce_kernel<EPI_>), dim3(ceil_div(T * (w.N / 4), 256)), dim3(256), 0, s, splitk_ws, KS, T, w.N, e); \
    } \
  } while (0)
  if (epi == EPI_QKV) MI_G(EPI_QKV);
  else if (epi == EPI_SWIGLU) MI_G(EPI_SWIGLU);
  else if (epi == EPI_RESID) MI_G(EPI_RESID);
  else if (epi >= EPI_RELU2) {
    if constexpr (WD == MI_W_BF16) {
      if (epi == EPI_RELU2) MI_G(EPI_RELU2);
      else if (epi == EPI_GLU_CLIP) MI_G(EPI_GLU_CLIP);
      else if (epi == EPI_SOFTCAP) MI_G(EPI_SOFTCAP);
      else MI_G(EPI_HEADS_KV);
    } else { set_error("gemm: this epilogue is built for bf16 weights"); return MI_EINVAL; }
  } else MI_G(EPI_F32);
#undef MI_G
  MI_HIP(hipGetLastError());
  return MI_OK;
}


// =====================================================================================
// GEMM, wide-N tile with an LDS-DMA ring and two wave groups half a K-step apart (context encoding, 1-byte weights)
// =====================================================================================
// The 128 x 128 kernel above is L1-fill bound: per 64-deep K-step a work-group pulls
// 16 KiB of bf16 activations + 8 KiB of fp8 weights for 2.1 MFLOP.  Weights are half the bytes per
// element of the activations, so the tile grows along N: 128 tokens x 256 weight rows = 16 + 16 KiB
// for 4.2 MFLOP (1.5 x the flops per byte), 256 x 256 = 32 + 16 KiB for 8.4.  Eight waves as 2 (tokens) x 4 (weight
// rows): activation fragments are shared by four waves, weight fragments by two.  Both operands arrive by LDS-DMA
// (global_load_lds, 1 KiB per wave-instruction: the weight tiles land lane-linear = fragment
// order; the activation rows land in the XOR-swizzled image of the kernel above, the swizzle being
// applied to the per-lane SOURCE address) into a ring of three stages: two K-steps are in
// flight while one is multiplied, retired by counted vmcnt waits in front of raw barriers -- no ordinary global
// load in the loop, so hipcc has nothing to drain.  Round 3: a wave's K-step is a READ phase (fragments LDS -> registers,
// weight codes decoded on the way) and a MULTIPLY phase (MFMAs only), and the two waves of a SIMD are in opposite phases
// (see "Schedule" in the kernel): gate|up at 2048 tokens 436.6 -> 373.4 us (1.10 -> 1.29 PF/s), down 220 -> 198 us.
constexpr int kWideBN = 256, kWideWBytes = 16 * 1024, kWideStages = 3;


// BM = 128: each wave 64 x 64 (64 accumulator registers).  BM = 256: each 128 x 64 (128 accumulator registers, 246 VGPRs
// with the decoded fragments of one K-step).
// SPLIT: grid.z K-slices write raw fp32 accumulators to slab[z][m][n] (see gemm_a8_kernel); K / 64 is a multiple of grid.z.
template <int WD, int EPI, int BM, bool SPLIT>
__global__ __launch_bounds__(512) void gemm_wide_kernel(const uint4* __restrict__ W, int NT, int KT, int T, int K,
                                                        const uint16_t* __restrict__ x, int ldx, EpiArgs e,
                                                        float* __restrict__ slab) {
  static_assert(WD != MI_W_BF16, "1-byte weight tiles (64 k per tile)");
  static_assert(BM == 128 || BM == 256, "token block");
  // waves as 2 (tokens) x 4 (weight rows), each MT 16-token tiles x 4 16-row weight tiles.  (4 x 2 waves of 64 x 128 read
  // 16 instead of 20 KiB of fragments per K-step but decode every weight code four times instead of twice: measured slower,
  // 401 against 387 us on the gate-up shape -- the decode, not the LDS read, is what the schedule has to hide.)
  constexpr int MT = BM / 32;                 // 16-token tiles per wave
  constexpr int WM = 2, NTW = 4;
  constexpr int XP = BM / 64;                 // 8-row activation pieces per wave and stage
  constexpr int kStage = kWideWBytes + BM * 128;
  constexpr int kDma = 2 + XP;                // DMAs per wave and stage
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int g = lane >> 4, c = lane & 15;
  const int wm = wave % WM, wn = wave / WM;
  // XCD-aware tile order (see gemm_a8_kernel): an XCD walks all token blocks of a weight slab back to back
  const int mtiles = ceil_div(T, BM), ntiles = ceil_div(NT, kWideBN / 16);
  const int xcd = blockIdx.x & 7, seq = blockIdx.x >> 3;
  const int mblk = seq % mtiles, nblk = (seq / mtiles) * 8 + xcd;
  if (nblk >= ntiles) return;
  const int m0 = mblk * BM, ntb = nblk * (kWideBN / 16);
  const int nks = SPLIT ? K / 64 / (int)gridDim.z : K / 64;     // this slice's K-steps, from K-step ks0 on
  const int ks0 = SPLIT ? (int)blockIdx.z * nks : 0;

  // this lane's DMA sources: wave w brings weight tiles 2w, 2w + 1 of the work-group's 16 (fragment
  // order) and XP 8-row pieces of the activation tile
  const uint4* wsrc[2];
  const uint16_t* xsrc[XP];
#pragma unroll
  for (int i = 0; i < 2; ++i) wsrc[i] = W + ((size_t)min(ntb + 2 * wave + i, NT - 1) * KT + ks0) * 64 + lane;
#pragma unroll
  for (int i = 0; i < XP; ++i) {
    const int r = (XP * wave + i) * 8 + (lane >> 3), sl = lane & 7;
    xsrc[i] = x + (size_t)min(m0 + r, T - 1) * ldx + (size_t)ks0 * 64 + ((sl ^ xs_swz<WD>(r)) * 8);   // LDS slot sl of row r holds chunk sl ^ swz(r)
  }
  auto issue = [&](int ks) {
    unsigned char* st = smem + (ks % kWideStages) * kStage;
#pragma unroll
    for (int i = 0; i < 2; ++i) glds16(wsrc[i] + (size_t)ks * 64, st + (2 * wave + i) * 1024);
#pragma unroll
    for (int i = 0; i < XP; ++i) glds16(xsrc[i] + (size_t)ks * 64, st + kWideWBytes + (XP * wave + i) * 1024);
  };

  f32x4_t acc[NTW][MT];
#pragma unroll
  for (int i = 0; i < NTW; ++i)
#pragma unroll
    for (int j = 0; j < MT; ++j) acc[i][j] = f32x4_t{0.f, 0.f, 0.f, 0.f};

  // Schedule.  A K-step of a wave is two phases: READ (its fragments, 20 KiB at BM = 256, from LDS into registers, the weight codes decoded to bf16 on the way) and MULTIPLY
  // (2 NTW MT MFMAs from registers).  With one barrier per K-step every wave is in the same phase at the same time, the two waves
  // of a SIMD included, and LDS-read time and MFMA time add up: 1.7 us per K-step at BM = 256 against 1.0 us of MFMAs.  Here
  // the two wave groups (waves 0-3 / 4-7 = the two waves of every SIMD) run half a K-step apart -- group 1 executes one
  // barrier more at the start -- so one group multiplies while the other reads:
  //     physical barrier:      P0        P1        P2        P3        P4  ...
  //     group 0 (waves 0-3):   | READ 0  | MUL 0   | READ 1  | MUL 1   | ...
  //     group 1 (waves 4-7):   |         | READ 0  | MUL 0   | READ 1  | MUL 1 ...
  // Stage k is read in [P2k, P2k+2]; K-step k + 2 goes into the stage of K-step k - 1 (read until P2k), requested by every wave
  // behind its top barrier of iteration k: two K-steps ahead of its first read, as before.  A wave waits for ITS pieces of a
  // stage before the barrier in front of the stage's first read by anyone (group 0: its top barrier; group 1: its second one).
  const int grp = __builtin_amdgcn_readfirstlane(wave >> 2);
  issue(0);
  if (nks > 1) issue(1);
  if (grp == 1) {   // its pieces of stage 0 are in before P0
    if (nks > 1) asm volatile("s_waitcnt vmcnt(%0)" ::"n"(kDma) : "memory");
    else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();           // P0
  }
  for (int ks = 0; ks < nks; ++ks) {
    if (grp == 0) {   // own pieces of stage ks (at most those of stage ks + 1 are younger)
      if (ks + 1 < nks) asm volatile("s_waitcnt vmcnt(%0)" ::"n"(kDma) : "memory");
      else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    }
    __builtin_amdgcn_s_barrier();           // group 0: P2ks | group 1: P2ks+1 -- either way nobody reads stage ks - 1 any more
    if (ks + 2 < nks) issue(ks + 2);
    const unsigned char* st = smem + (ks % kWideStages) * kStage;
    const uint4* xs = reinterpret_cast<const uint4*>(st + kWideWBytes);
    u32x4_t b0[MT], b1[MT];
    bf16x8_t a0[NTW], a1[NTW];
#pragma unroll
    for (int mt = 0; mt < MT; ++mt) {
      const int r = wm * (BM / 2) + mt * 16 + c;
      b0[mt] = *reinterpret_cast<const u32x4_t*>(&xs[r * 8 + ((2 * g) ^ xs_swz<WD>(r))]);
      b1[mt] = *reinterpret_cast<const u32x4_t*>(&xs[r * 8 + ((2 * g + 1) ^ xs_swz<WD>(r))]);
    }
#pragma unroll
    for (int i = 0; i < NTW; ++i) {   // decoded here, in the READ phase, while the SIMD's other wave multiplies: the MULTIPLY phase is MFMAs only
      const u32x4_t w4 = *reinterpret_cast<const u32x4_t*>(st + (wn * NTW + i) * 1024 + lane * 16);
      a0[i] = decode8<WD>(w4[0], w4[1]);
      a1[i] = decode8<WD>(w4[2], w4[3]);
    }
    // the fragments are in registers (the empty asm takes them as operands: the compiler's wait for the reads sits in front of it)
#pragma unroll
    for (int mt = 0; mt < MT; ++mt) { asm volatile("" : "+v"(b0[mt])); asm volatile("" : "+v"(b1[mt])); }
#pragma unroll
    for (int i = 0; i < NTW; ++i) { asm volatile("" : "+v"(a0[i])); asm volatile("" : "+v"(a1[i])); }
    if (grp == 1 && ks + 1 < nks) {   // own pieces of stage ks + 1: group 0 reads it behind the next barrier
      if (ks + 2 < nks) asm volatile("s_waitcnt vmcnt(%0)" ::"n"(kDma) : "memory");
      else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    }
    __builtin_amdgcn_s_barrier();           // group 0: P2ks+1 | group 1: P2ks+2
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int i = 0; i < NTW; ++i) {
#pragma unroll
      for (int mt = 0; mt < MT; ++mt) {
        acc[i][mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a0[i], __builtin_bit_cast(bf16x8_t, b0[mt]), acc[i][mt], 0, 0, 0);
        acc[i][mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a1[i], __builtin_bit_cast(bf16x8_t, b1[mt]), acc[i][mt], 0, 0, 0);
      }
    }
  }
  if (grp == 0) __builtin_amdgcn_s_barrier();   // the barrier group 1 executed first
#pragma unroll
  for (int i = 0; i < NTW; ++i) {
    const int nt = ntb + wn * NTW + i;
    if (nt >= NT) continue;
#pragma unroll
    for (int mt = 0; mt < MT; ++mt) {
      const int m = m0 + wm * (BM / 2) + mt * 16 + c;
      if (m >= T) continue;
      if constexpr (SPLIT) {
        *reinterpret_cast<float4*>(slab + ((size_t)blockIdx.z * T + m) * (NT * 16) + nt * 16 + g * 4) =
            make_float4(acc[i][mt][0], acc[i][mt][1], acc[i][mt][2], acc[i][mt][3]);
      } else {
        epilogue<EPI>(e, m, nt * 16 + g * 4, acc[i][mt]);
      }
    }
  }
}

template <int WD, int BM>
static int launch_gemm_wide_bm(const LinearW& w, int T, const uint16_t* x, int ldx, int epi, const EpiArgs& e, hipStream_t s,
                               int KS, float* splitk_ws, SlabSum* defer) {
  const int NT = w.N / 16, KT = w.K / 64;
  const int mtiles = ceil_div(T, BM), ntiles = ceil_div(w.N, kWideBN);
  dim3 grid(8 * mtiles * ceil_div(ntiles, 8), 1, KS);
  const uint4* W = reinterpret_cast<const uint4*>(w.w);
  constexpr int lds = kWideStages * (kWideWBytes + BM * 128);
#define MI_GW(EPI_) \
  do { \
    if (KS == 1) { \
      MI_TRY_(ensure_dynamic_lds(reinterpret_cast<const void*>(gemm_wide_kernel<WD, EPI_, BM, false>), lds)); \
      hipLaunchKernelGGL((gemm_wide_kernel<WD, EPI_, BM, false>), grid, dim3(512), lds, s, W, NT, KT, T, w.K, x, ldx, e, nullptr); \
    } else { \
      MI_TRY_(ensure_dynamic_lds(reinterpret_cast<const void*>(gemm_wide_kernel<WD, EPI_, BM, true>), lds)); \
      hipLaunchKernelGGL((gemm_wide_kernel<WD, EPI_, BM, true>), grid, dim3(512), lds, s, W, NT, KT, T, w.K, x, ldx, e, splitk_ws); \
      if (defer && EPI_ == EPI_RESID) { *defer = SlabSum{splitk_ws, KS, T, w.N, e.scale, e.bias, e.row_scale}; } \
      else hipLaunchKernelGGL((splitk_reduce_kernel<EPI_>), dim3(ceil_div(T * (w.N / 4), 256)), dim3(256), 0, s, splitk_ws, KS, T, w.N, e); \
    } \
  } while (0)
  if (epi == EPI_QKV) MI_GW(EPI_QKV);
  else if (epi == EPI_SWIGLU) MI_GW(EPI_SWIGLU);
  else if (epi == EPI_RESID) MI_GW(EPI_RESID);
  else MI_GW(EPI_F32);
#undef MI_GW
  MI_HIP(hipGetLastError());
  return MI_OK;
}
// The wide kernel runs ONE work-group per CU (96 / 144 KiB of LDS), so what decides is how full its rounds of the chip are,
// and between the two token blocks, rounds x time per K-step (measured on full grids: 0.90 us at 128 tokens, 1.45 us at 256 --
// twice the flops).  Measured on the Llama-8B shapes (round 3, staggered schedule; wide against the 128 x 128 kernel, us):
//     gate|up  256 tokens: 224 work-groups of 128 tokens (one round, 88 %)   62.0 vs  73.4      512: 448 (two rounds)  115.3 vs 141.6
//     gate|up 1024 tokens: 896 (3.5 rounds)                                 224.5 vs 227.6      QKV 1024: 192 (one round, 75 %) 66.6 vs 84.2
//     QKV  512: 96 work-groups   64.6 vs 40.1      O / down 1024: 128   57.1 vs 40.7 / 166.6 vs 116.2 (K-split on the other side)
//     QKV 2048: 384 (1.5 rounds, 75 %)  134.5 vs 112.4;  gate|up 2048: 403.6 at 128 tokens (7 rounds), 373.4 at 256 (3.5)
// -> a shape is eligible with one partial round from 70 % of the CUs on or several rounds at 80 % fill; the cheapest eligible
// (token block, K-split) runs: rounds x K-steps x time per K-step, plus, for a K-split, the slabs written and read once more
// (~4 bytes/ns) and the launch that sums them.
struct WidePlan { int bm, ks; };   // bm 0: not wanted
static WidePlan gemm_wide_plan(int T, int N, int K, size_t ws_bytes, int wd) {
  int cus = 256;
  if (device_num_cu(&cus) != MI_OK || cus < 1) cus = 256;
  const int nks = K / 64;
  WidePlan best{0, 1};
  double best_cost = 0.;
  for (int bm = 128; bm <= 256; bm *= 2) {
    for (int ks = 1; ks <= 8; ks *= 2) {
      if (nks % ks != 0 || nks / ks < 8) continue;
      if (ks > 1 && (size_t)ks * T * N * sizeof(float) > ws_bytes) continue;
      const int wgs = ceil_div(T, bm) * ceil_div(N, kWideBN) * ks, rounds = ceil_div(wgs, cus);
      const bool ok = wgs < cus ? wgs * 10 >= cus * 7 : wgs * 5 >= rounds * cus * 4;
      if (!ok) continue;
      // INT8 codes cost the READ phase ~6 x the VALU work of the fp8 hardware convert: 1.38 / 1.73 us per K-step measured on
      // the Qwen2.5-7B shapes (gate|up at 1024 tokens 387.8 us at 128-token blocks against 303.5 on the 128 x 128 kernel;
      // at 2048 tokens 485 at 256-token blocks against 592) -- there the wide tile must also beat what the 128 x 128 kernel
      // holds: 0.9 PF/s on grids that keep three work-groups per CU resident, 0.65 on its K-split grids
      const bool i8 = wd == MI_W_INT8;
      double cost = (double)rounds * (nks / ks) * (bm == 128 ? (i8 ? 1.38 : 0.90) : (i8 ? 1.73 : 1.45));
      if (ks > 1) cost += 4.0 + (double)(ks + 1) * T * N * 4.0 / 4.0e6 * 1.0;   // slabs out and in, the sum out
      const double alt_pf = ceil_div(T, 128) * ceil_div(N, 128) >= 3 * cus ? 0.9e9 : 0.65e9;   // flops per us: full residency / a K-split grid
      if (i8 && cost > 2.0 * T * N * (double)K / alt_pf) continue;
      if (best.bm == 0 || cost < best_cost) { best = WidePlan{bm, ks}; best_cost = cost; }
    }
  }
  return best;
}
static int gemm_wide_mode() {   // MI355X_GEMM_WIDE: 0 never, 1 whenever the shape allows, unset: by size
  static const int m = [] { const char* v = getenv("MI355X_GEMM_WIDE"); return v ? atoi(v) : -1; }();
  return m;
}
static int gemm_wide_bm() {      // MI355X_GEMM_WIDE_BM: 128 / 256 forces the token block (default: by grid size)
  static const int m = [] { const char* v = getenv("MI355X_GEMM_WIDE_BM"); return v ? atoi(v) : 0; }();
  return m;
}
static int gemm_wide_ks() {      // MI355X_GEMM_WIDE_KS: 1 = never split K in the wide kernel
  static const int m = [] { const char* v = getenv("MI355X_GEMM_WIDE_KS"); return v ? atoi(v) : 0; }();
  return m;
}
template <int WD>
static int launch_gemm_wide_wd(const LinearW& w, int T, const uint16_t* x, int ldx, int epi, const EpiArgs& e, hipStream_t s,
                               float* splitk_ws, size_t splitk_ws_bytes, SlabSum* defer, int force_bm, int force_ks) {
  WidePlan pl = gemm_wide_plan(T, w.N, w.K, gemm_wide_ks() == 1 || !splitk_ws ? 0 : splitk_ws_bytes, w.wd);
  const int forced_bm = force_bm ? force_bm : gemm_wide_bm();
  if (forced_bm == 128 || forced_bm == 256) pl = WidePlan{forced_bm, 1};
  if (pl.bm == 0) pl = WidePlan{ceil_div(T, 256) * ceil_div(w.N, kWideBN) >= 512 ? 256 : 128, 1};   // forced onto a shape the plan would not take
  if (force_ks) {
    MI_CHECK(force_ks >= 1 && (w.K / 64) % force_ks == 0 && (force_ks == 1 || (splitk_ws && (size_t)force_ks * T * w.N * 4 <= splitk_ws_bytes)),
             "gemm_wide: forced K-split must divide K / 64 and fit the workspace");
    pl.ks = force_ks;
  }
  if (pl.bm == 256) return launch_gemm_wide_bm<WD, 256>(w, T, x, ldx, epi, e, s, pl.ks, splitk_ws, defer);
  return launch_gemm_wide_bm<WD, 128>(w, T, x, ldx, epi, e, s, pl.ks, splitk_ws, defer);
}
// the wide tile needs 1-byte weights
static bool gemm_wide_wanted(const LinearW& w, int T, size_t ws_bytes) {
  if (w.wd == MI_W_BF16 || w.K % 64 != 0 || (w.N / 16) < 2) return false;
  const int mode = gemm_wide_mode();
  if (mode == 1) return true;
  if (mode == 0) return false;
  if (T <= 128) return false;   // up to one 128-token block: the 128 x 128 kernel and its K-split (also the 33 .. 128-row decode batches)
  return gemm_wide_plan(T, w.N, w.K, gemm_wide_ks() == 1 ? 0 : ws_bytes, w.wd).bm != 0;
}
int launch_gemm_wide(const LinearW& w, int T, const uint16_t* x, int ldx, int epi, const EpiArgs& e, hipStream_t s,
                     float* splitk_ws, size_t splitk_ws_bytes, SlabSum* defer, int force_bm, int force_ks) {
  if (defer) *defer = SlabSum();
  MI_CHECK(w.wd != MI_W_BF16 && w.K % 64 == 0 && ldx % 8 == 0, "gemm_wide: 1-byte weights, K % 64 == 0");
  if (w.wd == MI_W_F8E4M3)
    return launch_gemm_wide_wd<MI_W_F8E4M3>(w, T, x, ldx, epi, e, s, splitk_ws, splitk_ws_bytes, defer, force_bm, force_ks);
  return launch_gemm_wide_wd<MI_W_INT8>(w, T, x, ldx, epi, e, s, splitk_ws, splitk_ws_bytes, defer, force_bm, force_ks);
}

int launch_gemm(const LinearW& w, int T, const uint16_t* x, int ldx, int epi, const EpiArgs& e, hipStream_t s,
                float* splitk_ws, size_t splitk_ws_bytes, SlabSum* defer) {
  if (defer) *defer = SlabSum();
  MI_CHECK(T >= 1, "gemm: T must be >= 1");
  if (epi < EPI_RELU2 && gemm_wide_wanted(w, T, splitk_ws ? splitk_ws_bytes : 0) && ldx % 8 == 0)
    return launch_gemm_wide(w, T, x, ldx, epi, e, s, splitk_ws, splitk_ws_bytes, defer);
  MI_CHECK(w.N % 16 == 0 && w.K % 64 == 0, "gemm: N % 16 == 0 and K % 64 == 0 required");
  MI_CHECK(ldx % 8 == 0, "gemm: x row stride must be a multiple of 8 elements");
  switch (w.wd) {
    case MI_W_BF16: return launch_gemm_wd<MI_W_BF16>(w, T, x, ldx, epi, e, s, splitk_ws, splitk_ws_bytes, defer);
    case MI_W_F8E4M3: return launch_gemm_wd<MI_W_F8E4M3>(w, T, x, ldx, epi, e, s, splitk_ws, splitk_ws_bytes, defer);
    case MI_W_INT8: return launch_gemm_wd<MI_W_INT8>(w, T, x, ldx, epi, e, s, splitk_ws, splitk_ws_bytes, defer);
  }
  set_error("gemm: bad weight dtype");
  return MI_EINVAL;
}

// =====================================================================================
// GEMM with FP8 activations (context encoding, the MFMA-bound contraction)
// =====================================================================================
// y[m, n] = (sum_k q_x[m, k] * q_w[n, k]) * s_w[n] * s_x[m]   both operands OCP e4m3.
// v_mfma_scale_f32_16x16x128_f8f6f4 with every block scale = 2^0 runs at twice the rate of
// the bf16 (and of the unscaled fp8) MFMA.  Its lane (g = lane >> 4, r = lane & 15) holds 32
// bytes of row r: they are taken as the lane's 16 bytes of weight tile 2s and of tile 2s + 1
// (the contraction order inside an MFMA is free as long as both operands agree), so the
// weight image is the same one the GEMV streams.  Work-group = 4 waves, tile 256 (n) x 128 (m):
// wave w owns n-tiles 4w..4w+3 against all 8 m-tiles (128 fp32 accumulators per lane, one wave
// per SIMD); W fragments come straight from global (every wave reads distinct rows), x8 goes
// through LDS; the next K-step's operands are fetched into registers under the MFMAs.
typedef __attribute__((ext_vector_type(8))) int i32x8_t;
constexpr int kA8BM = 128, kA8BK = 128;   // tile: (64 NTW) weight rows x 128 tokens x 128 K bytes
constexpr int kA8Pitch = kA8BK + 32;   // LDS row pitch in bytes: 160 makes the fragment reads (row c, 16 B at g * 16 / + 64) conflict-free
                                       // over the ds_read_b128 lane groups; 144 left every group two-deep on its banks

// SPLIT: grid.z K-slices each write their raw fp32 accumulators to slab[z][m][n]; splitk_reduce
// sums the slabs in slice order (deterministic) and applies the epilogue.  Used when a short
// prompt leaves the (m-tile x n-tile) grid too small to pull the weights at HBM rate.
template <int EPI, bool SPLIT, int NTW>   // NTW 16-row weight tiles per wave: the tile is (64 NTW) x 128
__global__ __launch_bounds__(256) void gemm_a8_kernel(const uint4* __restrict__ W, int NT, int KT, int T, int K,
                                                      const uint8_t* __restrict__ x8, int ldx, EpiArgs e,
                                                      float* __restrict__ slab) {
  __shared__ __attribute__((aligned(16))) unsigned char xs[kA8BM * kA8Pitch];   // 20 KiB
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int g = lane >> 4, c = lane & 15;
  // XCD-aware tile order.  Work-groups go round-robin over the 8 XCDs (own 4 MiB L2 each), so
  // linear id L runs on XCD L % 8.  An XCD takes every eighth 256-row weight slab and walks ALL
  // token blocks of a slab back to back: the slab (and the K-step the co-resident work-groups
  // are at) is fetched over the fabric once per XCD instead of once per XCD per token block.
  constexpr int BN = 64 * NTW;
  const int mtiles = ceil_div(T, kA8BM), ntiles = ceil_div(NT, BN / 16);
  const int xcd = blockIdx.x & 7, seq = blockIdx.x >> 3;
  const int mblk = seq % mtiles, nblk = (seq / mtiles) * 8 + xcd;
  if (nblk >= ntiles) return;
  const int m0 = mblk * kA8BM, nt0 = nblk * (BN / 16) + wave * NTW;
  const int nks_all = K / kA8BK;
  const int ks_per = SPLIT ? ceil_div(nks_all, (int)gridDim.z) : nks_all;
  const int ks_beg = SPLIT ? (int)blockIdx.z * ks_per : 0;
  const int nks = min(ks_beg + ks_per, nks_all);   // exclusive end of this slice
  constexpr int kUnit = 0x7f7f7f7f;   // E8M0 block scales: 2^0

  f32x4_t acc[NTW][8];
#pragma unroll
  for (int i = 0; i < NTW; ++i)
#pragma unroll
    for (int j = 0; j < 8; ++j) acc[i][j] = f32x4_t{0.f, 0.f, 0.f, 0.f};

  // x staging: 128 rows x 128 B per K-step = 1024 chunks of 16 B, 4 per thread.  The fp8 image
  // is K-step-major, [K / 128][ldx = T rows][128 B]: a work-group's K-step is 16 KiB contiguous.
  u32x4_t xr[4], wr[NTW][2], wn[NTW][2];
  auto load_x = [&](int ks) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int idx = tid + i * 256, row = idx >> 3, ch = idx & 7;
      const int m = min(m0 + row, T - 1);   // rows past T are computed on a copy of the last row, never stored
      xr[i] = *reinterpret_cast<const u32x4_t*>(x8 + ((size_t)ks * ldx + m) * kA8BK + ch * 16);
    }
  };
  auto load_w = [&](u32x4_t (&dst)[NTW][2], int ks) {
#pragma unroll
    for (int i = 0; i < NTW; ++i) {
      const int nt = min(nt0 + i, NT - 1);
#pragma unroll
      for (int t = 0; t < 2; ++t)
        dst[i][t] = *reinterpret_cast<const u32x4_t*>(W + ((size_t)nt * KT + ks * 2 + t) * 64 + lane);
    }
  };
  MI_TRACE_BEGIN();
  MI_STAMP(0);
  if (ks_beg < nks) {
    load_x(ks_beg);
    load_w(wr, ks_beg);
  }
  for (int ks = ks_beg; ks < nks; ++ks) {
    if (ks == ks_beg + 4) MI_STAMP(1);     // tools/trace_gemm.py: phases of the fifth K-step
    if (ks == ks_beg + 5) MI_STAMP(6);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int idx = tid + i * 256, row = idx >> 3, ch = idx & 7;
      *reinterpret_cast<u32x4_t*>(&xs[row * kA8Pitch + ch * 16]) = xr[i];
    }
    __syncthreads();
    if (ks == ks_beg + 4) MI_STAMP(2);
    if (ks + 1 < nks) {
      load_x(ks + 1);
      load_w(wn, ks + 1);
    }
    if (ks == ks_beg + 4) MI_STAMP(3);
#pragma unroll
    for (int mt = 0; mt < 8; ++mt) {
      const unsigned char* xrow = &xs[(mt * 16 + c) * kA8Pitch + g * 16];
      const u32x4_t b0 = *reinterpret_cast<const u32x4_t*>(xrow);        // k-tile 2ks,   chunk g
      const u32x4_t b1 = *reinterpret_cast<const u32x4_t*>(xrow + 64);   // k-tile 2ks+1, chunk g
      const i32x8_t b = {(int)b0[0], (int)b0[1], (int)b0[2], (int)b0[3], (int)b1[0], (int)b1[1], (int)b1[2], (int)b1[3]};
#pragma unroll
      for (int i = 0; i < NTW; ++i) {
        const i32x8_t a = {(int)wr[i][0][0], (int)wr[i][0][1], (int)wr[i][0][2], (int)wr[i][0][3],
                           (int)wr[i][1][0], (int)wr[i][1][1], (int)wr[i][1][2], (int)wr[i][1][3]};
        acc[i][mt] = __builtin_amdgcn_mfma_scale_f32_16x16x128_f8f6f4(a, b, acc[i][mt], 0, 0, 0, kUnit, 0, kUnit);
      }
    }
    if (ks == ks_beg + 4) MI_STAMP(4);
    __syncthreads();
    if (ks == ks_beg + 4) MI_STAMP(5);
    if (ks + 1 < nks) {
#pragma unroll
      for (int i = 0; i < NTW; ++i) {
        wr[i][0] = wn[i][0];
        wr[i][1] = wn[i][1];
      }
    }
  }
#pragma unroll
  for (int i = 0; i < NTW; ++i) {
    if (nt0 + i >= NT) continue;
#pragma unroll
    for (int mt = 0; mt < 8; ++mt) {
      const int m = m0 + mt * 16 + c;
      if (m >= T) continue;
      const int n0 = (nt0 + i) * 16 + g * 4;
      if constexpr (SPLIT) {
        *reinterpret_cast<float4*>(slab + ((size_t)blockIdx.z * T + m) * (NT * 16) + n0) =
            make_float4(acc[i][mt][0], acc[i][mt][1], acc[i][mt][2], acc[i][mt][3]);
      } else {
        epilogue<EPI>(e, m, n0, acc[i][mt]);
      }
    }
  }
  MI_STAMP(7);
  MI_TRACE_END();
}

// ---- FP8 activations on the wide tile ------------------------------------------------------------
// The kernel above keeps three work-groups of 128 x 128 on a CU and takes in 32 KiB per 4.2 MFLOP; this one is
// gemm_wide_kernel's schedule (LDS-DMA ring of three stages, the two wave groups half a K-step apart) on 128 tokens x 256
// weight rows x 128 K bytes: 16 + 32 KiB per 8.4 MFLOP, half the bytes per flop.  (256 x 256 would halve them again but is
// 64 KiB a stage: two stages in 160 KiB, and two stages cannot carry the stagger -- profiles/r03_a8_wide_experiment.txt.)
// A stage: [16 n-tiles][2 k-tiles][64 lanes x 16 B] weight fragments as stored, then 128 activation rows x 128 B with
// 16-byte chunk ch of row r at slot ch ^ (r & 7) (the lane reads chunks g and 4 + g: conflict-free with that key).
constexpr int kA8wStage = 32 * 1024 + 128 * 128, kA8wDma = 6;
// (A ninth wave touching the lines of the K-step four ahead, to make the ring's DMAs L2 hits, cost 27 %: 260 -> 330 us on
// gate|up at 2048 tokens -- profiles/r03_a8_wide_experiment.txt.)
template <int EPI, bool SPLIT>
__global__ __launch_bounds__(512) void gemm_a8_wide_kernel(const uint4* __restrict__ W, int NT, int KT, int T, int K,
                                                           const uint8_t* __restrict__ x8, int ldx, EpiArgs e,
                                                           float* __restrict__ slab) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int g = lane >> 4, c = lane & 15;
  const int wm = wave & 1, wn = wave >> 1;      // waves 2 (tokens) x 4 (weight rows), each 64 x 64
  const int mtiles = ceil_div(T, 128), ntiles = ceil_div(NT, 16);
  const int xcd = blockIdx.x & 7, seq = blockIdx.x >> 3;
  const int mblk = seq % mtiles, nblk = (seq / mtiles) * 8 + xcd;
  if (nblk >= ntiles) return;
  const int m0 = mblk * 128, ntb = nblk * 16;
  const int nks = SPLIT ? K / 128 / (int)gridDim.z : K / 128;
  const int ks0 = SPLIT ? (int)blockIdx.z * nks : 0;
  constexpr int kUnit = 0x7f7f7f7f;   // E8M0 block scales: 2^0

  // DMA sources of this lane: weight n-tiles 2w, 2w + 1 (two k-tiles each, adjacent in the image), activation pieces 2w, 2w + 1
  const uint4* wsrc[2];
  const uint8_t* xsrc[2];
#pragma unroll
  for (int i = 0; i < 2; ++i) wsrc[i] = W + ((size_t)min(ntb + 2 * wave + i, NT - 1) * KT + 2 * ks0) * 64 + lane;
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int r = (2 * wave + i) * 8 + (lane >> 3), sl = lane & 7;
    xsrc[i] = x8 + ((size_t)ks0 * ldx + min(m0 + r, T - 1)) * 128 + ((sl ^ (r & 7)) * 16);
  }
  auto issue = [&](int ks) {
    unsigned char* st = smem + (ks % kWideStages) * kA8wStage;
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int t = 0; t < 2; ++t) glds16(wsrc[i] + ((size_t)ks * 2 + t) * 64, st + ((2 * wave + i) * 2 + t) * 1024);
#pragma unroll
    for (int i = 0; i < 2; ++i) glds16(xsrc[i] + (size_t)ks * ldx * 128, st + 32 * 1024 + (2 * wave + i) * 1024);
  };

  f32x4_t acc[4][4];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = f32x4_t{0.f, 0.f, 0.f, 0.f};

  // the schedule of gemm_wide_kernel: READ (fragments to registers) / MULTIPLY (MFMAs only), the groups in opposite phases
  const int grp = __builtin_amdgcn_readfirstlane(wave >> 2);
  issue(0);
  if (nks > 1) issue(1);
  if (grp == 1) {
    if (nks > 1) asm volatile("s_waitcnt vmcnt(%0)" ::"n"(kA8wDma) : "memory");
    else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
  }
  for (int ks = 0; ks < nks; ++ks) {
    if (grp == 0) {
      if (ks + 1 < nks) asm volatile("s_waitcnt vmcnt(%0)" ::"n"(kA8wDma) : "memory");
      else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    }
    __builtin_amdgcn_s_barrier();
    if (ks + 2 < nks) issue(ks + 2);
    const unsigned char* st = smem + (ks % kWideStages) * kA8wStage;
    const uint4* xs = reinterpret_cast<const uint4*>(st + 32 * 1024);
    u32x4_t b0[4], b1[4], a0[4], a1[4];
#pragma unroll
    for (int mt = 0; mt < 4; ++mt) {
      const int r = wm * 64 + mt * 16 + c;
      b0[mt] = *reinterpret_cast<const u32x4_t*>(&xs[r * 8 + (g ^ (r & 7))]);
      b1[mt] = *reinterpret_cast<const u32x4_t*>(&xs[r * 8 + ((4 + g) ^ (r & 7))]);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      a0[i] = *reinterpret_cast<const u32x4_t*>(st + ((wn * 4 + i) * 2) * 1024 + lane * 16);
      a1[i] = *reinterpret_cast<const u32x4_t*>(st + ((wn * 4 + i) * 2 + 1) * 1024 + lane * 16);
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      asm volatile("" : "+v"(b0[j])); asm volatile("" : "+v"(b1[j]));
      asm volatile("" : "+v"(a0[j])); asm volatile("" : "+v"(a1[j]));
    }
    if (grp == 1 && ks + 1 < nks) {
      if (ks + 2 < nks) asm volatile("s_waitcnt vmcnt(%0)" ::"n"(kA8wDma) : "memory");
      else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    }
    __builtin_amdgcn_s_barrier();
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int mt = 0; mt < 4; ++mt) {
      const i32x8_t b = {(int)b0[mt][0], (int)b0[mt][1], (int)b0[mt][2], (int)b0[mt][3], (int)b1[mt][0], (int)b1[mt][1], (int)b1[mt][2], (int)b1[mt][3]};
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const i32x8_t a = {(int)a0[i][0], (int)a0[i][1], (int)a0[i][2], (int)a0[i][3], (int)a1[i][0], (int)a1[i][1], (int)a1[i][2], (int)a1[i][3]};
        acc[i][mt] = __builtin_amdgcn_mfma_scale_f32_16x16x128_f8f6f4(a, b, acc[i][mt], 0, 0, 0, kUnit, 0, kUnit);
      }
    }
  }
  if (grp == 0) __builtin_amdgcn_s_barrier();
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int nt = ntb + wn * 4 + i;
    if (nt >= NT) continue;
#pragma unroll
    for (int mt = 0; mt < 4; ++mt) {
      const int m = m0 + wm * 64 + mt * 16 + c;
      if (m >= T) continue;
      if constexpr (SPLIT) {
        *reinterpret_cast<float4*>(slab + ((size_t)blockIdx.z * T + m) * (NT * 16) + nt * 16 + g * 4) =
            make_float4(acc[i][mt][0], acc[i][mt][1], acc[i][mt][2], acc[i][mt][3]);
      } else {
        epilogue<EPI>(e, m, nt * 16 + g * 4, acc[i][mt]);
      }
    }
  }
}

template <int EPI>
__global__ __launch_bounds__(256) void splitk_reduce_kernel(const float* __restrict__ slab, int KS, int T, int N, EpiArgs e) {
  const int q = blockIdx.x * 256 + threadIdx.x;      // one (m, 4 consecutive n) per thread
  const int nq = N >> 2;
  if (q >= T * nq) return;
  const int m = q / nq, n0 = (q - m * nq) * 4;
  f32x4_t v = {0.f, 0.f, 0.f, 0.f};
  for (int z = 0; z < KS; ++z) {
    const float4 p = *reinterpret_cast<const float4*>(slab + ((size_t)z * T + m) * N + n0);
    v[0] += p.x; v[1] += p.y; v[2] += p.z; v[3] += p.w;
  }
  epilogue<EPI>(e, m, n0, v);
}

// sum a deferred K-split (SlabSum) the plain way: splitk_reduce + residual epilogue
int launch_splitk_flush(const SlabSum& sl, const float* resid_in, float* out, int ld_out, hipStream_t s) {
  EpiArgs e{};
  e.scale = sl.scale; e.bias = sl.bias; e.row_scale = sl.row_scale;
  e.out_f32 = out; e.resid_in = resid_in; e.ld_out = ld_out;
  hipLaunchKernelGGL((splitk_reduce_kernel<EPI_RESID>), dim3(ceil_div(sl.T * (sl.N / 4), 256)), dim3(256), 0, s, sl.slab, sl.KS,
                     sl.T, sl.N, e);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

bool gemm_a8_supported(const LinearW& w) {
  return w.wd == MI_W_F8E4M3 && w.K % kA8BK == 0 && w.N % 16 == 0;
}

int launch_gemm_a8(const LinearW& w, int T, const uint8_t* x8, int ldx, int epi, const EpiArgs& e, hipStream_t s,
                   float* splitk_ws, size_t splitk_ws_bytes, SlabSum* defer) {
  if (defer) *defer = SlabSum();
  MI_CHECK(T >= 1, "gemm_a8: T must be >= 1");
  MI_CHECK(gemm_a8_supported(w), "gemm_a8: needs fp8 weights, K % 128 == 0, N % 16 == 0");
  MI_CHECK(ldx >= T && e.row_scale != nullptr, "gemm_a8: x8 is the K-step-major image of >= T rows, with its row scales");
  const int NT = w.N / 16, KT = w.K / 64, nks = w.K / kA8BK;
  {   // The wide tile (MI355X_A8_WIDE: 0 never, 1 always, unset: by plan) where its one-work-group-per-CU grid fills one or two
      // rounds of the chip.  Measured on the Llama-8B shapes against the kernel below (us): 256 tokens gate|up 43.6 vs 45.9,
      // down 24.0 vs 25.6, QKV 17.3 vs 19.4; 512: 76.9 vs 86.0, 34.8 vs 39.6, 23.5 vs 28.0; 1024: down 58.4 vs 68.2, QKV 48.8 vs
      // 51.9 but gate|up (3.5 rounds) 145.0 vs 135.9; 2048: down 121.0 vs 136.1, O 46.2 vs 49.3, gate|up (7 rounds) 260.4 vs
      // 254.2 -- on long grids the three resident work-groups of the 128 x 128 kernel hide more latency than the ring does.
    static const int mode = [] { const char* v = getenv("MI355X_A8_WIDE"); return v ? atoi(v) : -1; }();
    int cus = 256;
    if (device_num_cu(&cus) != MI_OK || cus < 1) cus = 256;
    int best_ks = 0;
    double best_cost = 0.;
    for (int ks = 1; ks <= 8; ks *= 2) {
      if (nks % ks != 0 || nks / ks < 4) continue;
      if (ks > 1 && (!splitk_ws || (size_t)ks * T * w.N * sizeof(float) > splitk_ws_bytes)) continue;
      const int wgs = ceil_div(T, 128) * ceil_div(w.N, 256) * ks, rounds = ceil_div(wgs, cus);
      const bool ok = mode == 1 || (rounds <= 2 && (wgs < cus ? wgs * 10 >= cus * 7 : wgs * 5 >= rounds * cus * 4));
      if (!ok) continue;
      double cost = (double)rounds * (nks / ks) * 1.0;
      if (ks > 1) cost += 4.0 + (double)(ks + 1) * T * w.N * 4.0 / 4.0e6;
      if (best_ks == 0 || cost < best_cost) { best_ks = ks; best_cost = cost; }
    }
    if (mode != 0 && best_ks && T > 128) {
      const int KS = best_ks;
      dim3 grid(8 * ceil_div(T, 128) * ceil_div(ceil_div(w.N, 256), 8), 1, KS);
      const uint4* W = reinterpret_cast<const uint4*>(w.w);
      constexpr int lds = kWideStages * kA8wStage;
#define MI_A8W_L(EPI_, SPLIT_, WS_) \
  do { \
    MI_TRY_(ensure_dynamic_lds(reinterpret_cast<const void*>(gemm_a8_wide_kernel<EPI_, SPLIT_>), lds)); \
    hipLaunchKernelGGL((gemm_a8_wide_kernel<EPI_, SPLIT_>), grid, dim3(512), lds, s, W, NT, KT, T, w.K, x8, ldx, e, WS_); \
  } while (0)
#define MI_A8W(EPI_) \
  do { \
    if (KS == 1) { \
      MI_A8W_L(EPI_, false, nullptr); \
    } else { \
      MI_A8W_L(EPI_, true, splitk_ws); \
      if (defer && EPI_ == EPI_RESID) { *defer = SlabSum{splitk_ws, KS, T, w.N, e.scale, e.bias, e.row_scale}; } \
      else hipLaunchKernelGGL((splitk_reduce_kernel<EPI_>), dim3(ceil_div(T * (w.N / 4), 256)), dim3(256), 0, s, splitk_ws, KS, T, w.N, e); \
    } \
  } while (0)
      if (epi == EPI_QKV) MI_A8W(EPI_QKV);
      else if (epi == EPI_SWIGLU) MI_A8W(EPI_SWIGLU);
      else if (epi == EPI_RESID) MI_A8W(EPI_RESID);
      else MI_A8W(EPI_F32);
#undef MI_A8W
#undef MI_A8W_L
      MI_HIP(hipGetLastError());
      return MI_OK;
    }
  }
  // 128 x 128 tiles: 64 accumulator registers per lane leave room for three work-groups per CU,
  // which hide each other's load latency (the 256 x 128 tile ran one work-group per CU at 24 % of
  // the matrix-core rate: 29.7 ms for the 2048 bucket against 22.5 ms; forcing a fourth wave per
  // SIMD spills inside the K loop: 122 ms)
  constexpr int ntw = 2;
  const int bn = 64 * ntw;
  const int mtiles = ceil_div(T, kA8BM), ntiles = ceil_div(w.N, bn);
  // K-split only when the tile grid cannot occupy the chip and the slabs stay small
  // (768 work-groups are resident at once.  Measured on the Llama-8B shapes: below 256 tiles aim
  // for 512 work-groups, below 384 for 768; splitting larger grids costs more in slab traffic
  // than it wins -- 6.2 / 8.8 / 13.5 ms for the 256 / 512 / 1024 buckets.)
  const int KS = gemm_pick_splitk(mtiles * ntiles, nks, T, w.N, splitk_ws ? splitk_ws_bytes : 0);
  const uint4* W = reinterpret_cast<const uint4*>(w.w);
  dim3 grid(8 * mtiles * ceil_div(ntiles, 8), 1, KS);   // see the kernel: XCD-aware tile order
#define MI_A8(EPI_) \
  do { \
    if (KS == 1) { \
      hipLaunchKernelGGL((gemm_a8_kernel<EPI_, false, ntw>), grid, dim3(256), 0, s, W, NT, KT, T, w.K, x8, ldx, e, nullptr); \
    } else { \
      hipLaunchKernelGGL((gemm_a8_kernel<EPI_, true, ntw>), grid, dim3(256), 0, s, W, NT, KT, T, w.K, x8, ldx, e, splitk_ws); \
      if (defer && EPI_ == EPI_RESID) { *defer = SlabSum{splitk_ws, KS, T, w.N, e.scale, e.bias, e.row_scale}; } \
      else hipLaunchKernelGGL((splitk_reduce_kernel<EPI_>), dim3(ceil_div(T * (w.N / 4), 256)), dim3(256), 0, s, splitk_ws, KS, T, w.N, e); \
    } \
  } while (0)
  if (epi == EPI_QKV) MI_A8(EPI_QKV);
  else if (epi == EPI_SWIGLU) MI_A8(EPI_SWIGLU);
  else if (epi == EPI_RESID) MI_A8(EPI_RESID);
  else MI_A8(EPI_F32);
#undef MI_A8
  MI_HIP(hipGetLastError());
  return MI_OK;
}

// =====================================================================================
// Load-time quantize + tile
// =====================================================================================
__global__ void rowmax_kernel(const float* __restrict__ w, int ld, float* __restrict__ rowmax) {
  const float* r = w + (size_t)blockIdx.x * ld;
  float m = 0.f;
  for (int i = threadIdx.x; i < ld; i += blockDim.x) m = fmaxf(m, fabsf(r[i]));
  __shared__ float sm[256];
  sm[threadIdx.x] = m;
  __syncthreads();
  for (int s = 128; s > 0; s >>= 1) {
    if (threadIdx.x < s) sm[threadIdx.x] = fmaxf(sm[threadIdx.x], sm[threadIdx.x + s]);
    __syncthreads();
  }
  if (threadIdx.x == 0) rowmax[blockIdx.x] = sm[0];
}
__global__ void allmax_kernel(const float* __restrict__ rowmax, int n, float* __restrict__ out) {
  float m = 0.f;
  for (int i = threadIdx.x; i < n; i += blockDim.x) m = fmaxf(m, rowmax[i]);
  __shared__ float sm[256];
  sm[threadIdx.x] = m;
  __syncthreads();
  for (int s = 128; s > 0; s >>= 1) {
    if (threadIdx.x < s) sm[threadIdx.x] = fmaxf(sm[threadIdx.x], sm[threadIdx.x + s]);
    __syncthreads();
  }
  if (threadIdx.x == 0) *out = sm[0];
}

// bf16 activations -> e4m3 + per-token scale: s = amax / 448 (all-zero row: 1), q = rne(x / s).
// One work-group per row.
// The row stays in registers between the amax pass and the quantize pass (up to kRqMax 16-byte
// chunks per thread, K <= 16384); longer rows are re-read.
constexpr int kRqMax = 8;
__global__ __launch_bounds__(256) void rowquant_fp8_kernel(const uint16_t* __restrict__ x, int K, int ldx,
                                                           uint8_t* __restrict__ x8, float* __restrict__ row_scale) {
  __shared__ float red[4];
  const int t = blockIdx.x, tid = threadIdx.x;
  const uint16_t* row = x + (size_t)t * ldx;
  const int nchunk = K / 8;
  u32x4_t v[kRqMax];
  float amax = 0.f;
#pragma unroll
  for (int q = 0; q < kRqMax; ++q) {
    const int c8 = tid + q * 256;
    v[q] = c8 < nchunk ? *reinterpret_cast<const u32x4_t*>(row + c8 * 8) : u32x4_t{0, 0, 0, 0};
  }
#pragma unroll
  for (int q = 0; q < kRqMax; ++q)
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const uint32_t w = v[q][k];
      amax = fmaxf(amax, fmaxf(fabsf(bf16lo_to_f32(w)), fabsf(bf16hi_to_f32(w))));
    }
  for (int c8 = tid + kRqMax * 256; c8 < nchunk; c8 += 256) {
    const u32x4_t r = *reinterpret_cast<const u32x4_t*>(row + c8 * 8);
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const uint32_t w = r[k];
      amax = fmaxf(amax, fmaxf(fabsf(bf16lo_to_f32(w)), fabsf(bf16hi_to_f32(w))));
    }
  }
  amax = fmaxf(amax, __shfl_xor(amax, 1));
  amax = fmaxf(amax, __shfl_xor(amax, 2));
  amax = fmaxf(amax, __shfl_xor(amax, 4));
  amax = fmaxf(amax, __shfl_xor(amax, 8));
  amax = fmaxf(amax, __shfl_xor(amax, 16));
  amax = fmaxf(amax, __shfl_xor(amax, 32));
  if ((tid & 63) == 0) red[tid >> 6] = amax;
  __syncthreads();
  amax = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
  const float scale = amax > 0.f ? amax / 448.f : 1.f;
  if (tid == 0) row_scale[t] = scale;
  auto emit = [&](const u32x4_t r, int c8) {
    uint32_t o[2] = {0, 0};
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const uint32_t w = r[k];
      const float a = fminf(fmaxf(bf16lo_to_f32(w) / scale, -448.f), 448.f);
      const float b = fminf(fmaxf(bf16hi_to_f32(w) / scale, -448.f), 448.f);
      o[k >> 1] |= (f32_to_e4m3fn(a) | (f32_to_e4m3fn(b) << 8)) << (16 * (k & 1));
    }
    // K-step-major image: [K / 128][T][128 B] (see gemm_a8_kernel: load_x)
    const int k0 = c8 * 8;
    *reinterpret_cast<uint2*>(x8 + ((size_t)(k0 >> 7) * gridDim.x + t) * 128 + (k0 & 127)) = make_uint2(o[0], o[1]);
  };
#pragma unroll
  for (int q = 0; q < kRqMax; ++q) {
    const int c8 = tid + q * 256;
    if (c8 < nchunk) emit(v[q], c8);
  }
  for (int c8 = tid + kRqMax * 256; c8 < nchunk; c8 += 256) emit(*reinterpret_cast<const u32x4_t*>(row + c8 * 8), c8);
}

int launch_rowquant_fp8(const uint16_t* x, int T, int K, int ldx, uint8_t* x8, float* row_scale, hipStream_t s) {
  MI_CHECK(K % 8 == 0 && ldx % 8 == 0, "rowquant: K and the row stride must be multiples of 8");
  hipLaunchKernelGGL(rowquant_fp8_kernel, dim3(T), dim3(256), 0, s, x, K, ldx, x8, row_scale);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

__device__ __forceinline__ int dst_to_src_row(const QuantJob& j, int r) {
  const int rel = r - j.dst_row0;
  if (rel < 0) return -1;
  int i;
  if (j.rowmap == ROWMAP_PLAIN) {
    i = rel;
  } else if (j.rowmap == ROWMAP_ROPE_PAIRS) {
    const int head = rel / j.hd, jj = rel % j.hd;
    i = head * j.hd + ((jj & 1) ? (jj >> 1) + (j.hd >> 1) : (jj >> 1));
  } else {
    if (rel & 1) return -1;
    i = rel >> 1;
  }
  return i < j.n_rows ? i : -1;
}

// one wave per destination tile
template <int WD>
__global__ __launch_bounds__(256) void quant_tile_kernel(QuantJob j, int nt_lo, int nt_cnt, int KT) {
  const int wave = (blockIdx.x * blockDim.x + threadIdx.x) >> 6, lane = threadIdx.x & 63;
  if (wave >= nt_cnt * KT) return;
  const int nt = nt_lo + wave / KT, kt = wave % KT;
  const int r = nt * 16 + (lane & 15), gq = lane >> 4;
  const int i = dst_to_src_row(j, r);
  if (i < 0) return;
  constexpr int EPL = (WD == MI_W_BF16) ? 8 : 16;  // elements per lane
  const int col0 = kt * (EPL * 4) + gq * EPL;      // first of the lane's columns, relative to src_col0
  const bool pad_row = i >= j.n_rows - j.pad_rows;
  const int k_src = j.K - j.pad_cols;
  if (pad_row || col0 >= k_src) {                  // EPL divides every head size: a lane is all padding or none
    if (pad_row && kt == 0 && gq == 0) j.dst_scale[r] = 1.f;
    if (!pad_row && kt == 0 && gq == 0) {
      float sc = 1.f;
      if constexpr (WD != MI_W_BF16) {
        const float qm = (WD == MI_W_INT8) ? 127.f : 448.f;
        const float am = (j.quant_type == MI_Q_PER_TENSOR_SYMMETRIC) ? j.tmp_rowmax[j.src_rows_total] : j.tmp_rowmax[j.src_row0 + i];
        sc = am > 0.f ? am / qm : 1.f;
      }
      j.dst_scale[r] = sc;
    }
    reinterpret_cast<uint4*>(j.dst)[((size_t)nt * KT + kt) * 64 + lane] = make_uint4(0, 0, 0, 0);
    return;
  }
  const int srow = j.src_row0 + i;
  const float* src = j.src + (size_t)srow * j.ld + j.src_col0 + col0;
  float scale = 1.f;
  if constexpr (WD != MI_W_BF16) {
    const float qmax = (WD == MI_W_INT8) ? 127.f : 448.f;
    const float amax = (j.quant_type == MI_Q_PER_TENSOR_SYMMETRIC) ? j.tmp_rowmax[j.src_rows_total] : j.tmp_rowmax[srow];
    scale = amax > 0.f ? amax / qmax : 1.f;
  }
  if (kt == 0 && gq == 0) j.dst_scale[r] = scale;
  uint4 out;
  if constexpr (WD == MI_W_BF16) {
    uint32_t o[4];
#pragma unroll
    for (int k = 0; k < 4; ++k) o[k] = pack_bf16x2(src[2 * k], src[2 * k + 1]);
    out = make_uint4(o[0], o[1], o[2], o[3]);
  } else {
    const float qmax = (WD == MI_W_INT8) ? 127.f : 448.f;
    uint32_t o[4] = {0, 0, 0, 0};
#pragma unroll
    for (int k = 0; k < 16; ++k) {
      float t = src[k] / scale;
      t = fminf(fmaxf(t, -qmax), qmax);
      uint32_t b;
      if constexpr (WD == MI_W_INT8) b = (uint32_t)(int)rintf(t) & 0xffu;
      else b = f32_to_e4m3fn(t);
      o[k >> 2] |= b << (8 * (k & 3));
    }
    out = make_uint4(o[0], o[1], o[2], o[3]);
  }
  reinterpret_cast<uint4*>(j.dst)[((size_t)nt * KT + kt) * 64 + lane] = out;
}

int run_quant_job(const QuantJob& j, hipStream_t s) {
  MI_CHECK(j.K % 64 == 0, "quantize: K % 64 == 0 required");
  if (j.wd != MI_W_BF16) {
    hipLaunchKernelGGL(rowmax_kernel, dim3(j.src_rows_total), dim3(256), 0, s, j.src, j.ld, j.tmp_rowmax);
    hipLaunchKernelGGL(allmax_kernel, dim3(1), dim3(256), 0, s, j.tmp_rowmax, j.src_rows_total, j.tmp_rowmax + j.src_rows_total);
  }
  // destination rows touched: [dst_row0, dst_row0 + span)
  const int span = (j.rowmap == ROWMAP_EVERY_OTHER) ? 2 * j.n_rows : j.n_rows;
  const int nt_lo = j.dst_row0 / 16, nt_hi = ceil_div(j.dst_row0 + span, 16);
  const int KT = j.K / tile_k(j.wd);
  const int waves = (nt_hi - nt_lo) * KT;
  const dim3 grid(ceil_div(waves, 4)), block(256);
  if (j.wd == MI_W_BF16) hipLaunchKernelGGL((quant_tile_kernel<MI_W_BF16>), grid, block, 0, s, j, nt_lo, nt_hi - nt_lo, KT);
  else if (j.wd == MI_W_F8E4M3) hipLaunchKernelGGL((quant_tile_kernel<MI_W_F8E4M3>), grid, block, 0, s, j, nt_lo, nt_hi - nt_lo, KT);
  else hipLaunchKernelGGL((quant_tile_kernel<MI_W_INT8>), grid, block, 0, s, j, nt_lo, nt_hi - nt_lo, KT);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

// tiled -> row-major (inspection / tests)
__global__ void untile_kernel(const uint4* __restrict__ tiled, int NT, int KT, int K, int eb, unsigned char* __restrict__ out) {
  const int wave = (blockIdx.x * blockDim.x + threadIdx.x) >> 6, lane = threadIdx.x & 63;
  if (wave >= NT * KT) return;
  const int nt = wave / KT, kt = wave % KT;
  const uint4 v = tiled[(size_t)wave * 64 + lane];
  const int r = nt * 16 + (lane & 15);
  // 16 bytes = 16 elements (1-byte types) or 8 elements (bf16)
  const size_t byte_col = (size_t)kt * 64 + (lane >> 4) * 16;
  *reinterpret_cast<uint4*>(out + (size_t)r * K * eb + byte_col) = v;
}

int launch_untile(const void* tiled, int N, int K, int wd, void* out, hipStream_t s) {
  MI_CHECK(N % 16 == 0 && K % 64 == 0, "untile: N % 16 == 0 and K % 64 == 0 required");
  const int NT = N / 16, KT = K / tile_k(wd);
  hipLaunchKernelGGL(untile_kernel, dim3(ceil_div(NT * KT, 4)), dim3(256), 0, s,
                     reinterpret_cast<const uint4*>(tiled), NT, KT, K, elem_bytes(wd), reinterpret_cast<unsigned char*>(out));
  MI_HIP(hipGetLastError());
  return MI_OK;
}

__global__ void bf16_to_f32_kernel(const uint16_t* __restrict__ in, float* __restrict__ out, size_t n) {
  for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (size_t)gridDim.x * blockDim.x)
    out[i] = bf16_to_f32(in[i]);
}
int launch_bf16_to_f32(const uint16_t* in, float* out, size_t n, hipStream_t s) {
  hipLaunchKernelGGL(bf16_to_f32_kernel, dim3(2048), dim3(256), 0, s, in, out, n);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

}  // namespace mi
