// Latent attention of the layer-stack decoders (stack.hip): what a token leaves in the cache is one latent c [rank] per
// layer; per head k = W_uk c, v = W_uv c.
//
//   s_ij = scale q_i.k_j for 0 <= i - j < window;  o_i = softmax_j(s_ij) v_j
//
// Scores and outputs are taken in the latent space: q.k = (W_uk^T q).c and o = W_uv (sum_j p_j c_j), so that every head reads
// the same cached row.  Pool: [num_blocks][block_size][rp]; head rows and latents are padded to 32 elements with zeros.
#pragma once
#include "window_attn.h"

namespace mi {

struct LatentGeom {
  int H = 0, dk = 0, dv = 0, rank = 0;
  int dkp = 0, dvp = 0, rp = 0;      // padded to 32
};
// qd [T, ldq] fp32 (q heads, then the latent's projection where c_norm is given) -> q [T, H, dkp]; latent over its root mean
// square times c_norm [rank] into the pool at slots (-1: not written).  slabs (slabs->slab): the projection as a K-split of row
// stride ldq that is not summed yet, instead of qd
int launch_latent_scatter(const float* qd, int ldq, int T, const LatentGeom& g, const float* c_norm, float eps, const int32_t* slots,
                          int block_size, void* q, void* pool, bool f32, hipStream_t s, const SlabSum* slabs = nullptr);
// token generation: qa [rows, H, rp] = W_uk^T q (bf16) from the same projection, and the latents' scatter, in one launch
inline bool latent_token_supported(const LatentGeom& g) { return g.dk % 4 == 0; }
int launch_latent_token(const float* qd, int ldq, int rows, const LatentGeom& g, const void* w_uk, const float* c_norm, float eps, const int32_t* slots,
                        uint16_t* qa, uint16_t* pool, hipStream_t s);
// The rows of a batch that a kernel takes: every row (token generation: segs null, row = block-table row), or the rows of the
// segments with fewer than below_n rows.
struct LatentRows {
  const AttnSeg* segs = nullptr;   // device
  int nseg = 0, below_n = 0;
  int rows = 0;                    // how many rows that is
};
// per head y[t, h] = W_h x[t, h]: x [T, H, K], W [H][N, K] (16 x 32 bf16 tiles or row-major fp32; K % 32 == 0, N % 16 == 0);
// columns n < n_valid go to y[t * ldy + h * y_head + n]
int launch_head_linear(const void* w, int H, int N, int K, const void* x, int T, void* y, int ldy, int y_head, int n_valid, bool f32, hipStream_t s);
int launch_head_linear_rows(const void* w, int H, int N, int K, const uint16_t* x, const LatentRows& rows, uint16_t* y, int ldy, int y_head,
                            int n_valid, hipStream_t s);      // bf16, the listed rows only
// ---- attention over latents, MFMA form (bf16)
bool latent_attn_supported(const LatentGeom& g);      // rank <= 512
size_t latent_attn_scratch_bytes(const LatentGeom& g);
// qa [T, H, rp] = W_uk^T q; lat [T, H, rp] scratch; out [T, ldo]: head h at column h dv
int launch_latent_attn_rows(const LatentGeom& g, float scale, int window, const uint16_t* qa, const uint16_t* pool, int block_size,
                            const int32_t* block_table, int MB, const int32_t* pos, const LatentRows& rows, int max_ctx, const void* w_uv,
                            uint16_t* lat, uint16_t* out, int ldo, void* scratch, hipStream_t s);

// ---- prompts: keys and values of the tokens in sight written out per head, for the windowed context-encoding kernel ---------------
// Of every segment with at least min_n rows: the latents of positions kv_first .. end, padded to whole kKvBlock rows, gathered into
// x [rows, ldx] (zero beyond the rank); kv_bt row = the segment's block-table row: position p -> block of kKvBlock gathered rows
constexpr int kKvBlock = 64;
__host__ __device__ inline int latent_kv_first(const AttnSeg& s, int window) {
  const int lo = window > 0 && s.pos0 - window + 1 > 0 ? s.pos0 - window + 1 : 0;
  return lo / kKvBlock * kKvBlock;
}
__host__ __device__ inline int latent_kv_rows(const AttnSeg& s, int window) {
  return (s.pos0 + s.n - latent_kv_first(s, window) + kKvBlock - 1) / kKvBlock * kKvBlock;
}
int launch_latent_gather(const LatentGeom& g, int window, const uint16_t* pool, int block_size, const int32_t* block_table, int MB, const AttnSeg* segs,
                         int nseg, int min_n, int rows, uint16_t* x, int ldx, int32_t* kv_bt, int kv_mb, hipStream_t s);

}  // namespace mi
