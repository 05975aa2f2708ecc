// Row-wise kernels of the layer-stack decoders (stack.hip): embedding with learned positions, layer norm with up to
// two affine outputs, the looped stack's input, per-head unit norm with the KV scatter, and the 32-bit linear layer.
// Every kernel takes its activations as bf16 (`f32 = false`) or fp32 (`f32 = true`: the 32-bit compute mode).
#pragma once
#include "linear_kernels.h"

namespace mi {

// resid[t, :] = E[ids[t], :] + P[pos[t], :] in fp32, also to x0 when given; columns D .. ld - 1 are zero
int launch_embed_pos(const int32_t* ids, const int32_t* pos, const void* table, const void* ptable, bool f32, int T,
                     int D, int ld, float* resid, float* x0, hipStream_t s);

struct NormOut {
  const float* w = nullptr;   // [ld], zero beyond D
  const float* b = nullptr;   // [ld], zero beyond D
  void* y = nullptr;          // [T, ldy]; null = this output is not wanted
};
// y = (x - mean) / sqrt(mean squared deviation + eps) * w + b for one or two (w, b) pairs over the same row.
// slabs: as launch_norm_rows -- the row is resid_in + the unsummed K-split projection, and goes to resid_out
int launch_layernorm_rows(const float* resid_in, float* resid_out, int T, int D, int ld, float eps, const NormOut& a,
                          const NormOut& b, int ldy, bool f32, hipStream_t s, const SlabSum* slabs = nullptr);
// y[t] = [x ; x0] in the compute type, the second half at column half
int launch_pair_rows(const float* x, const float* x0, int T, int D, int ld, int half, void* y, bool f32, hipStream_t s);

// geometry of one attention layer's pool rows: rows padded to 16 elements, zeros in the padding
struct HeadGeom {
  int H = 0, G = 0, dk = 0, dv = 0, dkp = 0, dvp = 0;
};
// qkv [T, ldq] fp32 (q heads, k heads, v heads) -> q [T, H, dkp], K / V pool rows at slots (-1: not written).
// unit_norm: q and k heads over sqrt(mean square + eps)
int launch_qkv_scatter(const float* qkv, int ldq, int T, const HeadGeom& g, bool unit_norm, float eps, const int32_t* slots,
                       int block_size, void* q, void* kpool, void* vpool, bool f32, hipStream_t s);

// y[m, n] = scale[n] sum_k x[m, k] w[n, k] in true fp32, epilogues EPI_F32 / EPI_RESID / EPI_RELU2 (act_out is fp32 here)
int launch_linear_f32(const float* w, int N, int K, const float* x, int ldx, int T, int epi, const EpiArgs& e, hipStream_t s);

// weight placement: src fp32 [rows, ld], columns src_col0 .. + cols, into rows row0.. / columns col0.. of a
// zero-filled matrix of K columns -- 16 x 32 bf16 tiles (linear_kernels.hip) or row-major fp32
int launch_place(const float* src, int ld, int src_col0, int rows, int cols, void* dst, int K, bool f32, int row0, int col0, hipStream_t s);
// dst[t, :V] = src[t, :V] with row strides lds_src / V (a vocabulary that is no multiple of 16)
int launch_pack_rows(const float* src, int ld_src, int T, int V, float* dst, hipStream_t s);

}  // namespace mi
