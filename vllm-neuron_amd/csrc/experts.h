// Mixture-of-experts feed-forward of the layer-stack decoders: router and the experts' linear layers.
//   z = W_router x + b (fp32);  chosen = the `top` largest logits;  weights = softmax over the chosen logits
// pair (t, j) = row t and its j-th expert, number t top + j
#pragma once
#include "mi_common.h"

namespace mi {

struct RouterRule {
  bool sigmoid = false;
  const float* b = nullptr;      // [E]: softmax, added to the logits (may be null: given logits hold it); sigmoid, the correction
  int groups = 1, keep = 1;
};
// x [T, ldx], w [E, K] row-major in the compute type -> ids [T, top], weights [T, top] (largest logit first; ties:
// lowest expert).  With z [T, E] and tickets [T] (zero, and left zero) a row's experts are shared out to several work-groups.
int launch_route(const void* x, int ldx, int T, const void* w, const RouterRule& rule, int E, int K, int top, int32_t* ids, float* weights, bool f32, hipStream_t s,
                 float* z = nullptr, uint32_t* tickets = nullptr);
// the same choice over given logits z [T, ldz] (softmax: nothing is added to them)
int launch_route_pick(const float* z, int ldz, int T, const RouterRule& rule, int E, int top, int32_t* ids, float* weights, hipStream_t s);

struct ExpertsLinear {
  const void* w = nullptr;      // [E][N, K]: 16 x 32 bf16 tiles or row-major fp32
  int E = 0, N = 0, K = 0;      // N % 16 == 0, K % 64 == 0
};
enum { EXPERT_LINEAR = 0, EXPERT_SILU_GLU = 1, EXPERT_RELU2 = 2 };
// y of every pair through its expert.  x row of pair p: p / x_div.  EXPERT_SILU_GLU: rows of W interleaved (gate, up), y [P, ldy] in
// the compute type = silu(gate) up; EXPERT_RELU2: y in the compute type = max(., 0)^2; EXPERT_LINEAR: y [P, ldy] fp32
int launch_experts_linear(const ExpertsLinear& w, const int32_t* ids, int P, const void* x, int ldx, int x_div, int act, void* y, int ldy,
                          bool f32, hipStream_t s);

// Many rows (bf16): the pairs are grouped by expert once, then every linear layer is one MFMA launch over (expert, block of its
// pairs, block of its rows).
struct ExpertPlan {
  int32_t* order = nullptr;     // [P] pairs, expert by expert
  int32_t* tiles = nullptr;     // [max_tiles][3] (expert, first place in order, pairs); then the number of tiles
  int block = 0;                // pairs per tile: 64 or 128
  int max_tiles = 0;
};
size_t experts_plan_ints(int P, int E);                                             // int32s of device memory behind a plan
ExpertPlan experts_plan(int32_t* mem, int P, int E);
int launch_experts_sort(const ExpertPlan& plan, const int32_t* ids, int P, int E, hipStream_t s);
// y bf16 in every case
int launch_experts_gemm(const ExpertsLinear& w, const ExpertPlan& plan, int P, const uint16_t* x, int ldx, int x_div, int act, uint16_t* y, int ldy, hipStream_t s);

}  // namespace mi
