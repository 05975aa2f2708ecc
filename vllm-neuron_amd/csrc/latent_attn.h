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
// square times c_norm [rank] into the pool at slots (-1: not written)
int launch_latent_scatter(const float* qd, int ldq, int T, const LatentGeom& g, const float* c_norm, float eps, const int32_t* slots,
                          int block_size, void* q, void* pool, bool f32, hipStream_t s);
// per head y[t, h] = W_h x[t, h]: x [T, H, K], W [H][N, K] (16 x 32 bf16 tiles or row-major fp32; K % 32 == 0, N % 16 == 0);
// columns n < n_valid go to y[t * ldy + h * y_head + n]
int launch_head_linear(const void* w, int H, int N, int K, const void* x, int T, void* y, int ldy, int y_head, int n_valid, bool f32, hipStream_t s);

}  // namespace mi
