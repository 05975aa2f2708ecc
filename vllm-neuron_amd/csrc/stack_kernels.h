// Row-wise kernels of the layer-stack decoders (stack.hip): embedding with learned or sinusoidal positions, layer norm with up to
// two affine outputs, the sandwich block's row (post-norm, residual sum, pre-norm, causal convolution), the looped stack's
// input, per-head norms with the KV scatter, and the 32-bit linear layer.
// Every kernel takes its activations as bf16 (`f32 = false`) or fp32 (`f32 = true`: the 32-bit compute mode).
#pragma once
#include "linear_kernels.h"

namespace mi {

struct AttnSeg { int row0, n, pos0, seq; };   // rows row0 .. + n of the batch = positions pos0 .. of the sequence in block-table row seq

// resid[t, :] = scale E[ids[t], :] (+ P[pos[t], :], ptable not null) in fp32, also to x0 when given; columns D .. ld - 1 are zero.
// turns [ceil(D / 2)] (not null): + sin / cos of 2 pi pos[t] turns[i] at elements 2 i / 2 i + 1.  y [T, ldy] (not null): the same row in the compute type
int launch_embed_pos(const int32_t* ids, const int32_t* pos, const void* table, const void* ptable, float scale, bool f32, int T,
                     int D, int ld, float* resid, float* x0, hipStream_t s, const double* turns = nullptr, void* y = nullptr, int ldy = 0);

struct NormOut {
  const float* w = nullptr;   // [ld], zero beyond D
  const float* b = nullptr;   // [ld], zero beyond D
  void* y = nullptr;          // [T, ldy]; null = this output is not wanted
};
// y = (x - mean) / sqrt(mean squared deviation + eps) * w + b for one or two (w, b) pairs over the same row.
// slabs: as launch_norm_rows -- the row is resid_in + the unsummed K-split projection, and goes to resid_out
int launch_layernorm_rows(const float* resid_in, float* resid_out, int T, int D, int ld, float eps, const NormOut& a,
                          const NormOut& b, int ldy, bool f32, hipStream_t s, const SlabSum* slabs = nullptr);

// ---- sandwich blocks: x <- x + post_norm(sublayer output); h = pre_norm(x); a = h + causal convolution of h ----------
// Norms are RMS norms over `groups` equal parts of the row, each over its own sqrt(mean square + eps).
// A sublayer's output, in whatever form the sublayer leaves it (slabs and pairs: their sum):
struct RowSource {
  const float* y = nullptr;        // [T, ld] fp32 ...
  const uint16_t* y16 = nullptr;   // ... or (experts) bf16
  int ld = 0;
  SlabSum slabs;                   // slabs.slab: the K-split sum of a projection, not summed yet
  const float* pair_w = nullptr;   // experts: row t is sum_j pair_w[t top + j] y(16)[t top + j]
  int top = 0;
  __host__ __device__ bool any() const { return y || y16 || slabs.slab; }
};
// The convolution and its state.  The state lives in the KV blocks: every block keeps the last `keep` inputs h of its
// positions, position p at row (p % block_size) % keep, so pages that are freed, shared or used again carry it along.
struct ConvState {
  const float* w = nullptr;        // [taps][ld]: row taps - 1 meets the token itself; null: no convolution
  int taps = 0, keep = 0;
  void* ring = nullptr;            // [blocks][keep][ldy] in the compute type
  int block_size = 0, MB = 0;
  const int32_t *bt = nullptr, *pos = nullptr, *slots = nullptr;
};
// resid_out = resid_in (+ post-normed src; w_post null: + src as it is); then, with w_pre, y [T, ldy] = h in the compute type, or (conv, every row its own
// sequence: block-table row = row) a with the state read and renewed.  Without w_pre only the residual sum, or (as_is) y = that row itself.
int launch_sandwich_rows(const float* resid_in, float* resid_out, const RowSource& src, const float* w_post, const float* w_pre, int T,
                         int D, int ld, int groups, float eps, const ConvState* conv, void* y, int ldy, bool f32, hipStream_t s, bool as_is = false);
// a = h + conv(h) over a ragged batch: h [T, ldy] as launch_sandwich_rows leaves it
int launch_conv_rows(const void* h, const ConvState& conv, const AttnSeg* segs_dev, const AttnSeg* segs_host, int nseg, int D, int ld,
                     void* y, int ldy, bool f32, hipStream_t s);

// y [T, ldy] = columns col .. col + n of x [T, ld] fp32 in the compute type, zeros behind them; w [n]: over their root mean square, times w
struct Columns { int col = 0, n = 0; const float* w = nullptr; void* y = nullptr; };      // w null: no norm
int launch_columns(const float* x, int ld, Columns a, Columns b, float eps, int T, int ldy, bool f32, hipStream_t s);   // b.y null: a alone
// y[t, h dv + d] *= sigmoid(g[t, ...]): one gate per head, or (per_element) per element; g [T, ldg] fp32, y [T, ldy] in the compute type
int launch_gate_rows(void* y, int ldy, int T, int H, int dv, const float* g, int ldg, bool per_element, bool f32, hipStream_t s);
// dst = src + offset;  dst = src factor
int launch_offset_copy(const float* src, int n, float offset, float* dst, hipStream_t s);
int launch_scaled_copy(const float* src, int n, float factor, float* dst, hipStream_t s);

// y[t] = [x ; x0] in the compute type, the second half at column half
int launch_pair_rows(const float* x, const float* x0, int T, int D, int ld, int half, void* y, bool f32, hipStream_t s);

// geometry of one attention layer's pool rows: rows padded to 16 elements, zeros in the padding
struct HeadGeom {
  int H = 0, G = 0, dk = 0, dv = 0, dkp = 0, dvp = 0;
};
// What happens to the projected heads on their way to the query buffer and the pools
struct HeadRule {
  bool unit_norm = false;          // q and k heads over sqrt(mean square + eps) ...
  const float *q_norm = nullptr, *k_norm = nullptr;   // ... times a weight per element [dk] (null: 1)
  const float* bias = nullptr;     // [H dk + G dk] added to the q and k heads first (null: none)
  bool keys_as_values = false;     // no v heads: a value is the key ahead of its norm (dv = dk)
};
// qkv [T, ldq] fp32 (q heads, k heads, v heads) -> q [T, H, dkp], K / V pool rows at slots (-1: not written)
int launch_qkv_scatter(const float* qkv, int ldq, int T, const HeadGeom& g, const HeadRule& rule, float eps, const int32_t* slots,
                       int block_size, void* q, void* kpool, void* vpool, bool f32, hipStream_t s);

// y[m, n] = scale[n] sum_k x[m, k] w[n, k] in true fp32, epilogues EPI_F32 / EPI_RESID / EPI_RELU2 / EPI_GLU_CLIP / EPI_SOFTCAP
// (act_out is fp32 here)
int launch_linear_f32(const float* w, int N, int K, const float* x, int ldx, int T, int epi, const EpiArgs& e, hipStream_t s);

// weight placement: src fp32 [rows, ld], columns src_col0 .. + cols, into rows row0.. / columns col0.. of a
// zero-filled matrix of K columns -- 16 x 32 bf16 tiles (linear_kernels.hip) or row-major fp32.  Source row r lands in
// row row0 + r row_step (2: gate / up rows interleaved)
int launch_place(const float* src, int ld, int src_col0, int rows, int cols, void* dst, int K, bool f32, int row0, int col0, hipStream_t s,
                 int row_step = 1);
// the same into a zero-filled row-major matrix of K columns, bf16 or fp32
int launch_place_rows(const float* src, int rows, int cols, void* dst, int K, bool f32, hipStream_t s);
// dst[c * ld_dst + r] = src[r * cols + c]
int launch_transpose(const float* src, int rows, int cols, float* dst, int ld_dst, hipStream_t s);
// dst[t, :V] = src[t, :V] with row strides lds_src / V (a vocabulary that is no multiple of 16)
int launch_pack_rows(const float* src, int ld_src, int T, int V, float* dst, hipStream_t s);

}  // namespace mi
