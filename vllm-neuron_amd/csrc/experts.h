// Mixture-of-experts feed-forward of the layer-stack decoders: router and the experts' linear layers.
//   z = W_router x + b (fp32);  chosen = the `top` largest logits;  weights = softmax over the chosen logits
//   pair (t, j) = row t and its j-th expert, number t top + j
#pragma once
#include "mi_common.h"

namespace mi {

// x [T, ldx], w [E, K] in the compute type, b [E] fp32 -> ids [T, top], weights [T, top] (largest logit first; ties: lowest expert)
int launch_route(const void* x, int ldx, int T, const void* w, const float* b, int E, int K, int top, int32_t* ids, float* weights, bool f32, hipStream_t s);

struct ExpertsLinear {
  const void* w = nullptr;      // [E][N, K]: 16 x 32 bf16 tiles or row-major fp32
  int E = 0, N = 0, K = 0;      // N % 16 == 0, K % 64 == 0
};
// y of every pair through its expert.  x row of pair p: p / x_div.  glu: rows of W interleaved (gate, up), y [P, ldy] in the compute
// type = silu(gate) up; else y [P, ldy] fp32
int launch_experts_linear(const ExpertsLinear& w, const int32_t* ids, int P, const void* x, int ldx, int x_div, bool glu, void* y, int ldy,
                          bool f32, hipStream_t s);

}  // namespace mi
