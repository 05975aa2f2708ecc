// Layer-stack decoders behind the same context, KV addressing and model calls as the Llama-family layers of model.hip:
// what mi_ctx_create_stack adds to an mi_ctx.
#pragma once
#include <string>
#include <vector>

#include "delta_rule.h"
#include "experts.h"
#include "latent_attn.h"
#include "model_internal.h"
#include "ssm.h"

namespace mi {

struct StackMat {   // a projection in the compute type: 16-row bf16 tiles (Linear) or row-major fp32
  Linear L;
  int N = 0, K = 0;   // padded: N % 16 == 0, K % 64 == 0
};
struct StackNorm { float *w = nullptr, *b = nullptr; };   // [ld], zero beyond the width

struct StackLayer {
  mi_layer_spec s{};
  HeadGeom g;
  AttnSpec attn;
  int attn_cols = 0, ff_cols = 0;   // columns of the concatenated output projection's input: [heads x v_dim | feed-forward]
  StackMat qkv, up, out;            // out = residual_mult [W_o | W_down]
  StackNorm n1, n2;
  float* slopes = nullptr;
  // sandwich blocks: qkv = [W_q | W_dkv], out = W_o, up = gate / up rows interleaved, down
  StackNorm n1b, n2b;                            // post-norms
  float *conv1 = nullptr, *conv2 = nullptr;      // [taps][ld]
  StackMat down;
  LatentGeom lg;
  AttnSpec latent;                               // the attention over latents: one shared key / value row for all heads
  float* c_norm = nullptr;                       // [rank]; null where the latents are another layer's
  void *w_uk = nullptr, *w_uv = nullptr;         // per head: W_uk^T [rp, dkp], W_uv [dvp, rp]
  StackMat ukv;                                  // [W_uk ; W_uv], heads padded to dkp / dvp rows: keys and values of a prompt (bf16)
  HeadGeom kvg;                                  // ... as the context-encoding attention sees them: every head its own
  bool fast() const { return ukv.L.w != nullptr; }   // the MFMA forms are built for the layer's sizes
  // one-norm blocks: qkv = every product with h the mixer needs, columns at col_*; latent mixer: [dkv | dq (or q) | g]; delta rule:
  // [q | k | v | b | a1 | g1]
  int col_q = 0, col_g = 0, col_b = 0, col_a = 0;
  StackMat uq, a2, g2;
  float *q_norm = nullptr, *conv = nullptr, *a_log = nullptr, *dt = nullptr, *o_norm = nullptr;
  DeltaGeom dg;
  // post-norm blocks: qkv = every product with x the mixer needs; attention: [q | k (| v) | g], beside it [z | x B C | dt]; selective scan: [x | z].
  // out = W_o, or [W_o left | W_o right] over [heads x v_dim | second mixer]; n1 / n2 the norms of the sublayers' outputs
  int col_z = 0, col_x = 0, col_dt = 0;
  HeadRule heads;
  float *qk_bias = nullptr, *k_norm = nullptr, *sinks = nullptr, *table = nullptr;
  std::vector<int> table_rows;                   // row of the checkpoint's distance table by distance
  StackMat low_in, dt_mat;                       // selective scan: x -> [low | B | C], low -> step sizes of the channels
  int col_B = 0, col_C = 0;
  void* w_dt = nullptr;                          // dt_mat row-major [C][rank_p]: token generation
  float *conv_b = nullptr, *decay = nullptr, *ssm_d = nullptr;   // (decay, bias and norm: a_log, dt, o_norm)
  ScanGeom scan;
  SsdGeom ssd;
  bool has_scan() const { return s.mixer_kind == MI_MIX_SCAN; }
  bool has_ssd() const { return s.beside_kind == MI_MIX_SSD; }
  int conv_channels() const { return has_scan() ? scan.C : ssd.channels(); }
  size_t ssm_state_floats() const { return has_scan() ? scan.state_floats() : has_ssd() ? ssd.state_floats() : 0; }
  size_t ssm_ring_floats() const { return ssm_state_floats() ? (size_t)s.conv_taps * conv_channels() : 0; }
  const float2* rot = nullptr;                   // cosines and sines of the layer's rotation (Stack::rot)
  int ff_act() const { return s.ff_act == MI_ACT_RELU2 ? EXPERT_RELU2 : EXPERT_SILU_GLU; }
  RouterRule rule() const {
    RouterRule r;
    r.sigmoid = s.router_score == MI_ROUTE_SIGMOID; r.b = router_b;
    if (r.sigmoid) { r.groups = s.router_groups; r.keep = s.router_keep; }
    return r;
  }
  void *router = nullptr, *expert_gu = nullptr, *expert_down = nullptr;
  float* router_b = nullptr;                     // [experts padded to 16]
  StackMat router_t;                             // the router as tiles: many rows (bf16)
  int ffk = 0;                                   // padded ff_size: contraction length of the experts' down projection
  ExpertsLinear expert_up() const { return ExpertsLinear{expert_gu, s.experts, ((s.ff_act == MI_ACT_RELU2 ? 1 : 2) * s.ff_size + 15) / 16 * 16, up.K}; }
  ExpertsLinear expert_dn() const { return ExpertsLinear{expert_down, s.experts, out.N, ffk}; }
};
struct StackRun { int layer; bool pass_start; };   // pass_start: the looped layers' input projection runs first

struct Stack {
  mi_stack_config cfg{};
  std::vector<StackLayer> layers;
  std::vector<StackRun> runs;
  bool f32 = false;
  int D = 0, ld = 0, Kd = 0;          // width; residual row stride (multiple of 16); activation row stride (multiple of 64)
  void *embed = nullptr, *pos = nullptr;
  StackMat loop_in, head;
  StackNorm final_norm;
  std::vector<size_t> kv_at;          // pool offset (elements) of every run's K (V follows) or latents (its own, or the layer's it reads)
  std::vector<size_t> conv_at;        // sandwich blocks: offset of every run's first convolution's state, the second's follows
  int conv_keep = 0;                  // convolution inputs a block keeps
  std::vector<std::string> missing;   // tensors not loaded yet
  // activations
  float *x0 = nullptr, *qkv_out = nullptr, *logits_pad = nullptr;
  void *n1 = nullptr, *n2 = nullptr, *q = nullptr, *cat = nullptr, *pair = nullptr;
  int qkv_ld = 0, q_cols = 0, cat_ld = 0;
  // sandwich blocks
  float *y = nullptr, *pair_w = nullptr;       // a sublayer's output rows (experts: of every pair); the pairs' weights
  int32_t *pair_ids = nullptr, *plan = nullptr;
  uint32_t* tickets = nullptr;
  float* route_z = nullptr;
  int max_experts = 0;
  void *hb = nullptr, *act = nullptr, *qa = nullptr, *lat = nullptr;   // convolution inputs; gated units; queries / outputs in latent space
  int act_ld = 0, lat_cols = 0, max_top = 0;
  // keys and values of a prompt, written out per head
  void *kv_x = nullptr, *kv_k = nullptr, *kv_v = nullptr;
  int32_t* kv_bt = nullptr;
  int kv_rows = 0, kv_mb = 0, kv_ldx = 0;
  size_t kv_k_cols = 0, kv_v_cols = 0;
  // one-norm blocks
  struct RotTable { float base; int dims; float2* t; };
  std::vector<RotTable> rot;
  std::vector<float*> state_at;       // every run's recurrent state, then its ring (null: none)
  int state_slots = 0;                // 0: no layer has any
  int z_ld = 0, z_gate = 0, low_ld = 0, cq_ld = 0, q2_ld = 0, delta_chunks = 0;
  size_t chunk_floats = 0;
  void *cq = nullptr, *low = nullptr; // normed query latents; the inputs of the decay's and the gate's second product [2][rows][low_ld]
  float *q2 = nullptr, *z = nullptr, *delta_records = nullptr;
  // post-norm blocks
  double* turns = nullptr;             // sinusoidal positions: turns per position [ceil(width / 2)]
  void *xc = nullptr;                  // convolution outputs [rows][xc_ld]
  float *xp = nullptr, *dtp = nullptr, *yssm = nullptr, *ssd_records = nullptr;   // [low | B | C]; step sizes; outputs ahead of gate and norm
  int xc_ld = 0, xp_ld = 0, dtp_ld = 0, yssm_ld = 0, ssd_chunks = 0;
  size_t ssd_chunk_floats = 0;
  bool post_norm() const { return cfg.block_kind == MI_BLOCK_POST_NORM; }
  bool parallel() const { return cfg.block_kind == MI_BLOCK_PARALLEL; }
  bool one_norm() const { return cfg.block_kind == MI_BLOCK_ONE_NORM; }
  bool sandwich() const { return cfg.block_kind == MI_BLOCK_SANDWICH; }
  void* attn_scratch = nullptr;
  SlabSum pend;                        // K-split sum of the last output projection, left for the next norm
  float* residuals = nullptr;          // mi_layer_residuals: [runs][max_rows][ld]
  size_t elem() const { return f32 ? 4 : 2; }
};

// *turns [ceil(width / 2)] (device, allocated): base^(-2 i / width) / 2 pi
int stack_position_turns(int width, float base, double** turns, hipStream_t s);
// table [H][rows.size()] = rel [rel_rows, H] (device) by distance
int stack_distance_table(const float* rel, const std::vector<int>& rows, int rel_rows, int H, float* table, hipStream_t s);
int stack_create(mi_ctx* c, const mi_stack_config& cfg);      // geometry + weight images (zeroed)
void stack_destroy(mi_ctx* c);
int stack_load_tensor(mi_ctx* c, const std::string& name, const float* dev, int rows, int cols);   // cols 0: a vector of `rows`
int stack_synthetic(mi_ctx* c, uint64_t seed, float std);
void stack_artifact_tensors(mi_ctx* c, std::vector<std::pair<void*, size_t>>& out);
int stack_geometry_hash(const mi_ctx* c);
size_t stack_kv_bytes_per_block(const mi_ctx* c);
size_t stack_workspace_estimate(const mi_ctx* c);               // recurrent state included
bool stack_has_state(const mi_ctx* c);
int stack_alloc(mi_ctx* c);                                    // KV pool + activations (mi_finalize)
// the layers over `rows` rows; leaves the residual stream in c->resid[c->tail_cur]
int stack_trunk(mi_ctx* c, int rows, bool decode, int MB, const AttnSeg* segs, int nseg);
// final norm + head over nrows contiguous residual rows -> c->logits
int stack_head(mi_ctx* c, const float* resid, int nrows);

}  // namespace mi
