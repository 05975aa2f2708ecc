// Latent attention of the layer-stack decoders (stack.hip): what a token leaves in the cache is one latent c [rank] per
// layer; per head k = W_uk c, v = W_uv c.
//
// and, where queries and keys have a rotated part, one rotated key part for all heads beside it.
//
//   s_ij = scale (q_i.k_j + rot(q'_i).rot(k'_j)) for 0 <= i - j < window;  o_i = softmax_j(s_ij) v_j
//
// Scores and outputs are taken in the latent space: q.k = (W_uk^T q).c and o = W_uv (sum_j p_j c_j), so that every head reads
// the same cached row.  Pool rows hold [latent, rp | rotated part, cp - rp]; head rows, latents and rotated parts are padded to 32
// elements with zeros.  W_uk^T is kept as a [cp, dkp] matrix per head that passes the rotated part of a query row through (ones on
// a diagonal), so a row W_uk^T q meets a pool row in one product.
#pragma once
#include "window_attn.h"

namespace mi {

struct LatentGeom {
  int H = 0, dk = 0, dv = 0, rank = 0;
  int dkp = 0, dvp = 0, rp = 0;      // padded to 32; dkp: of dk + nr
  int nr = 0, dims = 0, cp = 0;      // rotated part (0: none), its leading elements that turn, a pool row
  int dq() const { return dk + nr; }
};
inline LatentGeom latent_geom(int H, int dk, int dv, int rank, int nr = 0, int dims = 0) {
  auto pad = [](int v) { return (v + 31) / 32 * 32; };
  return LatentGeom{H, dk, dv, rank, pad(dk + nr), pad(dv), pad(rank), nr, dims, pad(rank) + pad(nr)};
}
struct Rotation {
  const float2* table = nullptr;     // [positions][dims / 2]: cosine, sine
  const int32_t* pos = nullptr;      // [rows]
};
// What a layer's projections leave for a row: H query heads of dq() elements, and (lat not null) rank + nr elements of the token's own.
struct LatentRowsIn {
  const float *q = nullptr, *lat = nullptr;
  int ldq = 0, ldl = 0;
};
// q heads -> q [T, H, dkp], their last nr elements rotated; latent over its root mean square times c_norm [rank], and the rotated key
// part, into the pool at slots (-1: not written).  slabs (slabs->slab): in.q is a K-split of that row stride that is not summed yet,
// with the latent's columns behind the heads'
int launch_latent_scatter(const LatentRowsIn& in, int T, const LatentGeom& g, const Rotation& rot, const float* c_norm, float eps, const int32_t* slots,
                          int block_size, void* q, void* pool, bool f32, hipStream_t s, const SlabSum* slabs = nullptr);
// token generation: qa [rows, H, cp] = W_uk^T q (bf16) from the same projections, and the latents' scatter, in one launch
inline bool latent_token_supported(const LatentGeom& g) { return g.dk % 4 == 0 && g.nr % 4 == 0; }
int launch_latent_token(const LatentRowsIn& in, int rows, const LatentGeom& g, const Rotation& rot, const void* w_uk, const float* c_norm, float eps,
                        const int32_t* slots, uint16_t* qa, uint16_t* pool, hipStream_t s);
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
                            int n_valid, hipStream_t s, OutGate gate = OutGate());      // bf16, the listed rows only
// ---- attention over latents, MFMA form (bf16)
bool latent_attn_supported(const LatentGeom& g);      // rank <= 512, rotated part <= 64
size_t latent_attn_scratch_bytes(const LatentGeom& g);
// qa [T, H, cp] = W_uk^T q; lat [T, H, rp] scratch; out [T, ldo]: head h at column h dv
int launch_latent_attn_rows(const LatentGeom& g, float scale, int window, const uint16_t* qa, const uint16_t* pool, int block_size,
                            const int32_t* block_table, int MB, const int32_t* pos, const LatentRows& rows, int max_ctx, const void* w_uv,
                            uint16_t* lat, uint16_t* out, int ldo, void* scratch, hipStream_t s, OutGate gate = OutGate());

// ---- prompts: keys and values of the tokens in sight written out per head, for the windowed context-encoding kernel ---------------
// Of every segment with at least min_n rows: the latents of positions kv_first .. end, padded to whole kKvBlock rows, gathered into
// x [rows, ldx] (zero beyond the pool row); kv_bt row = the segment's block-table row: position p -> block of kKvBlock gathered rows
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
