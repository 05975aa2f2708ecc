// Layer-stack decoders (mi_ctx_create_stack): geometry, weights and the layer loop.  Sampling, block tables, input
// staging, hipGraph capture and the model calls are model.hip's, shared with the Llama-family layers.
//
// One layer run (token generation: 5 or 6 launches):
//   layer norm, both affine outputs from one pass over the row           layernorm_rows_kernel
//   norm1 -> [q | k | v] projection                                       GEMV / GEMM
//   unit norm of q and k heads, q buffer, KV scatter                      qkv_scatter_kernel
//   windowed attention -> left part of the concatenated row               window_attn.hip
//   norm2 -> up projection, squared relu -> right part of the same row    GEMV / GEMM
//   [W_o | W_down] x concatenated row, residual_mult in its row scale, + residual
// The last one is both branches' output projection and the residual sum in one matrix product.
//
// A sandwich block's run (RMS norms around both sublayers, causal convolutions, latent attention, gated or expert feed-forward):
//   row: x += post-norm of the previous sublayer's output; pre-norm; convolution    sandwich_rows / conv_rows
//   [q | latent] projection; latent norm into the pool; W_uk^T q                    GEMV / GEMM, latent_scatter, head_linear
//   attention over latents; W_uv; output projection
//   row, as above; gated feed-forward, or router and experts                        experts.hip
//
// A one-norm block's run (RMS norm, then mixer and experts of the same row):
//   row: x += what the previous run left unsummed; norm                             sandwich_rows
//   router, experts                                                                 experts.hip
//   latent attention: [dkv | dq | g] product; query latent's norm; W_uq; rotation, scatter, attention as above; output gate
//   delta rule: [q | k | v | b | a1 | g1] product; a2, g2; recurrence               delta_rule.hip
//   output projection + residual; the experts' weighted sum and a K-split's are left to the next row kernel
//
// A post-norm block's run (the sublayers read the stream itself, RMS norms on their outputs):
//   row: x += norm of the previous sublayer's output; x in the compute type         sandwich_rows
//   attention: [q | k | g] product, beside it [z | x B C | dt]; norms and scatter; attention with gate; short convolution, recurrence,
//   gate and norm into the same row (ssm.hip); one output projection for both
//   selective scan: [x | z] product; short convolution; [low | B | C] product; step sizes; scan (ssm.hip); output projection
//   up, squared relu, down

#include "stack.h"

#include <cmath>
#include <cstring>

#include "misc_kernels.h"

namespace mi {

#define MI_TRY(expr)             \
  do {                           \
    int _rc = (expr);            \
    if (_rc != MI_OK) return _rc; \
  } while (0)

namespace {

int pad_to(int v, int m) { return (v + m - 1) / m * m; }

template <typename T>
int alloc0(mi_ctx* c, T** p, size_t bytes, size_t* tally) {
  MI_HIP(hipMalloc(reinterpret_cast<void**>(p), bytes));
  MI_HIP(hipMemsetAsync(*p, 0, bytes, c->stream));
  if (tally) *tally += bytes;
  return MI_OK;
}

int alloc_mat(mi_ctx* c, StackMat& m, int n, int k, float row_scale) {
  m.N = pad_to(n, 16);
  m.K = pad_to(k, 64);
  m.L.N = m.N; m.L.K = m.K; m.L.wd = MI_W_BF16;
  MI_TRY(alloc0(c, &m.L.w, (size_t)m.N * m.K * c->stack->elem(), &c->weight_bytes));
  MI_HIP(hipMalloc(reinterpret_cast<void**>(&m.L.scale), (size_t)m.N * 4));
  c->weight_bytes += (size_t)m.N * 4;
  return launch_fill_f32(m.L.scale, (size_t)m.N, row_scale, c->stream);
}
int alloc_norm(mi_ctx* c, StackNorm& n) {
  MI_TRY(alloc0(c, &n.w, (size_t)c->stack->ld * 4, &c->weight_bytes));
  return alloc0(c, &n.b, (size_t)c->stack->ld * 4, &c->weight_bytes);
}
void free_mat(StackMat& m) { hipFree(m.L.w); hipFree(m.L.scale); }
void free_norm(StackNorm& n) { hipFree(n.w); hipFree(n.b); }

// activations x [rows, ldx] through a projection
int apply(mi_ctx* c, const StackMat& m, int rows, const void* x, int ldx, int epi, EpiArgs e, SlabSum* defer = nullptr) {
  Stack* S = c->stack;
  e.scale = m.L.scale;
  if (S->f32) {
    Scope sc(c, MI_K_GEMM);
    return launch_linear_f32((const float*)m.L.w, m.N, m.K, (const float*)x, ldx, rows, epi, e, c->stream);
  }
  if (gemv_fits(rows, m.K)) {
    if (!c->runs(MI_K_GEMV)) return MI_OK;
    Scope sc(c, MI_K_GEMV);
    if (c->prof.on) c->prof.gemv_bytes += (double)m.N * m.K * 2;
    ProArgs p{};
    p.x = (const uint16_t*)x;
    p.ldx = ldx;
    return launch_gemv(m.L.view(), rows, PRO_BF16, p, epi, e, c->stream);
  }
  Scope sc(c, MI_K_GEMM);
  return launch_gemm(m.L.view(), rows, (const uint16_t*)x, ldx, epi, e, c->stream, c->splitk_ws, c->splitk_ws_bytes, defer);
}

// the residual sum a K-split output projection still owes: c->resid[cur ^ 1] + slabs -> c->resid[cur]
int flush(mi_ctx* c, int cur) {
  Stack* S = c->stack;
  if (!S->pend.slab) return MI_OK;
  Scope sc(c, MI_K_GEMM);
  const SlabSum sl = S->pend;
  S->pend = SlabSum();
  return launch_splitk_flush(sl, c->resid[cur ^ 1], c->resid[cur], S->ld, c->stream);
}

int norm_rows(mi_ctx* c, int cur, int rows, const NormOut& a, const NormOut& b) {
  Stack* S = c->stack;
  Scope sc(c, MI_K_OTHER);
  const SlabSum sl = S->pend;
  S->pend = SlabSum();
  if (sl.slab) return launch_layernorm_rows(c->resid[cur ^ 1], c->resid[cur], rows, S->D, S->ld, S->cfg.norm_eps, a, b, S->Kd, S->f32, c->stream, &sl);
  return launch_layernorm_rows(c->resid[cur], nullptr, rows, S->D, S->ld, S->cfg.norm_eps, a, b, S->Kd, S->f32, c->stream);
}

bool runs_other(mi_ctx* c) { return c->runs(MI_K_OTHER); }

int attention(mi_ctx* c, const StackLayer& W, size_t kv_at, int ldq, int rows, bool decode, int MB, const AttnSeg* segs, int nseg, const OutGate& gate = OutGate()) {
  Stack* S = c->stack;
  const mi_model_config& k = c->cfg;
  unsigned char* base = reinterpret_cast<unsigned char*>(c->kv_pool);
  const size_t kn = (size_t)k.num_blocks * W.g.G * k.block_size * W.g.dkp;
  unsigned char *kp = base + kv_at * S->elem(), *vp = base + (kv_at + kn) * S->elem();
  if (runs_other(c)) {
    Scope sc(c, MI_K_OTHER);
    MI_TRY(launch_qkv_scatter(S->qkv_out, ldq, rows, W.g, W.heads, S->cfg.norm_eps, c->d_slots, k.block_size, S->q, kp, vp, S->f32, c->stream));
  }
  const int ldo = S->cat_ld;
  if (S->f32 || !attn_window_supported(W.g) || (W.attn.table && !attn_table_supported(W.g, W.attn.table_n))) {
    if (!c->runs(decode ? MI_K_ATTN_DECODE : MI_K_ATTN_PREFILL)) return MI_OK;
    Scope sc(c, decode ? MI_K_ATTN_DECODE : MI_K_ATTN_PREFILL);
    return launch_attn_plain(W.attn, S->q, kp, vp, k.block_size, c->d_bt, MB, c->d_pos, decode ? nullptr : reinterpret_cast<const AttnSeg*>(c->d_segs),
                             nseg, rows, S->cat, ldo, S->f32, c->stream, gate);
  }
  const uint16_t* q = reinterpret_cast<const uint16_t*>(S->q);
  const uint16_t *kb = reinterpret_cast<const uint16_t*>(kp), *vb = reinterpret_cast<const uint16_t*>(vp);
  uint16_t* out = reinterpret_cast<uint16_t*>(S->cat);
  const size_t qrow = (size_t)W.g.H * W.g.dkp;
  if (decode) {
    if (!c->runs(MI_K_ATTN_DECODE)) return MI_OK;
    Scope sc(c, MI_K_ATTN_DECODE);
    return launch_attn_window_decode(W.attn, q, kb, vb, k.block_size, c->d_bt, MB, c->d_ctx, rows, k.max_model_len, out, ldo, S->attn_scratch, c->stream, gate);
  }
  Scope sc(c, MI_K_ATTN_PREFILL);
  MI_TRY(launch_attn_window_prefill(W.attn, q, kb, vb, k.block_size, c->d_bt, MB, reinterpret_cast<const AttnSeg*>(c->d_segs), segs, nseg, out, ldo, c->stream, 2, gate));
  for (int i = 0; i < nseg;) {   // runs of requests with one token: one token-generation launch each
    int j = i;
    while (j < nseg && segs[j].n == 1) ++j;
    if (j > i)
      MI_TRY(launch_attn_window_decode(W.attn, q + segs[i].row0 * qrow, kb, vb, k.block_size, c->d_bt + (size_t)i * MB, MB, c->d_seg_ctx + i, j - i,
                                       k.max_model_len, out + (size_t)segs[i].row0 * ldo, ldo, S->attn_scratch, c->stream,
                                       OutGate{gate.z ? gate.z + (size_t)segs[i].row0 * gate.ld : nullptr, gate.ld, false, gate.mult}));
    i = j > i ? j : i + 1;
  }
  return MI_OK;
}

// what latent attention needs in either block: W_uk, W_uv, W_o and the workspace's columns
int latent_layer_create(mi_ctx* c, StackLayer& W) {
  Stack* S = c->stack;
  const mi_layer_spec& s = W.s;
  size_t* wb = &c->weight_bytes;
  const LatentGeom& g = W.lg = latent_geom(s.num_heads, s.qk_dim, s.v_dim, s.kv_rank, s.rot_dim, s.rot_dims);
  W.latent = AttnSpec{HeadGeom{s.num_heads, 1, g.cp, g.rp, g.cp, g.cp}, s.scale, s.window, nullptr, 0, 0};
  MI_TRY(alloc_mat(c, W.out, S->D, s.num_heads * s.v_dim, 1.f));
  MI_TRY(alloc0(c, &W.w_uk, (size_t)s.num_heads * g.cp * g.dkp * S->elem(), wb));
  MI_TRY(alloc0(c, &W.w_uv, (size_t)s.num_heads * g.dvp * g.rp * S->elem(), wb));
  W.kvg = HeadGeom{s.num_heads, s.num_heads, g.dq(), s.v_dim, g.dkp, g.dvp};
  if (!S->f32 && latent_attn_supported(g) && attn_window_supported(W.kvg)) {
    MI_TRY(alloc_mat(c, W.ukv, s.num_heads * (g.dkp + g.dvp), g.nr ? g.rp + g.nr : s.kv_rank, 1.f));
    S->kv_ldx = std::max(S->kv_ldx, W.ukv.K);
    S->kv_k_cols = std::max(S->kv_k_cols, (size_t)s.num_heads * g.dkp);
    S->kv_v_cols = std::max(S->kv_v_cols, (size_t)s.num_heads * g.dvp);
  }
  S->q_cols = std::max(S->q_cols, s.num_heads * g.dkp);
  S->lat_cols = std::max(S->lat_cols, s.num_heads * g.cp);
  S->cat_ld = std::max(S->cat_ld, W.out.K);
  return MI_OK;
}

int experts_create(mi_ctx* c, StackLayer& W, const std::string& p) {
  Stack* S = c->stack;
  const mi_layer_spec& s = W.s;
  size_t* wb = &c->weight_bytes;
  auto want = [&](const char* n) { S->missing.push_back(p + n); };
  W.up.K = S->Kd;
  W.ffk = pad_to(s.ff_size, 64);
  S->max_top = std::max(S->max_top, s.experts_top);
  const ExpertsLinear gu = W.expert_up(), dn = W.expert_dn();
  MI_TRY(alloc0(c, &W.expert_gu, (size_t)gu.E * gu.N * gu.K * S->elem(), wb));
  MI_TRY(alloc0(c, &W.expert_down, (size_t)dn.E * dn.N * dn.K * S->elem(), wb));
  MI_TRY(alloc0(c, &W.router, (size_t)s.experts * S->Kd * S->elem(), wb));
  MI_TRY(alloc0(c, &W.router_b, (size_t)pad_to(s.experts, 16) * 4, wb));
  if (!S->f32) MI_TRY(alloc_mat(c, W.router_t, s.experts, S->D, 1.f));
  S->max_experts = std::max(S->max_experts, pad_to(s.experts, 16));
  want("mlp.router");
  want(s.router_score == MI_ROUTE_SIGMOID ? "mlp.correction" : "mlp.router.b");
  for (int e = 0; e < s.experts; ++e)
    for (const char* n : {".gate", ".up", ".down"})
      if (n[1] != 'g' || s.ff_act != MI_ACT_RELU2) want(("mlp.e" + std::to_string(e) + n).c_str());
  S->act_ld = std::max(S->act_ld, W.ffk);
  return MI_OK;
}

// ---- sandwich blocks: geometry and weights of one layer --------------------------------------------------------------------
int sandwich_layer_create(mi_ctx* c, StackLayer& W, const std::string& p) {
  Stack* S = c->stack;
  const mi_layer_spec& s = W.s;
  size_t* wb = &c->weight_bytes;
  auto want = [&](const char* n) { S->missing.push_back(p + n); };
  auto norm = [&](StackNorm& n) { return alloc0(c, &n.w, (size_t)S->ld * 4, wb); };
  const int taps = S->cfg.conv_taps;
  const bool own = s.kv_from < 0;
  MI_TRY(alloc_mat(c, W.qkv, s.num_heads * s.qk_dim + (own ? s.kv_rank : 0), S->D, 1.f));
  MI_TRY(latent_layer_create(c, W));
  if (own) MI_TRY(alloc0(c, &W.c_norm, (size_t)s.kv_rank * 4, wb));
  MI_TRY(norm(W.n1)); MI_TRY(norm(W.n1b));
  MI_TRY(alloc0(c, &W.conv1, (size_t)taps * S->ld * 4, wb));
  for (const char* n : {"norm1", "norm1b", "canon1", "mix.q", "mix.uk", "mix.uv", "mix.o"}) want(n);
  if (own) { want("mix.dkv"); want("mix.dkv.norm"); }
  S->qkv_ld = std::max(S->qkv_ld, W.qkv.N);
  if (s.ff_kind == MI_FF_NONE) return MI_OK;
  MI_TRY(norm(W.n2)); MI_TRY(norm(W.n2b));
  MI_TRY(alloc0(c, &W.conv2, (size_t)taps * S->ld * 4, wb));
  for (const char* n : {"norm2", "norm2b", "canon2"}) want(n);
  if (s.ff_kind == MI_FF_GLU) {
    MI_TRY(alloc_mat(c, W.up, 2 * s.ff_size, S->D, 1.f));
    MI_TRY(alloc_mat(c, W.down, S->D, s.ff_size, 1.f));
    W.ffk = W.down.K;
    for (const char* n : {"mlp.gate", "mlp.up", "mlp.down"}) want(n);
  } else {
    MI_TRY(experts_create(c, W, p));
  }
  S->act_ld = std::max(S->act_ld, W.ffk);
  return MI_OK;
}

void experts_tensor_shape(const Stack* S, const mi_layer_spec& s, const std::string& t, int* rows, int* cols) {
  int e = -1, at = 0;
  auto is = [&](int r, int k) { *rows = r; *cols = k; };
  const bool sigmoid = s.router_score == MI_ROUTE_SIGMOID;
  if (t == "mlp.router") is(s.experts, S->D);
  else if (t == (sigmoid ? "mlp.correction" : "mlp.router.b")) is(s.experts, 0);
  else if (sscanf(t.c_str(), "mlp.e%d.%n", &e, &at) == 1 && at > 0 && e >= 0 && e < s.experts) {
    const std::string m = t.substr(at);
    if ((m == "gate" && s.ff_act != MI_ACT_RELU2) || m == "up") is(s.ff_size, S->D);
    else if (m == "down") is(S->D, s.ff_size);
  }
}

// shape of a tensor of a sandwich block's layer by its name behind "l<i>."; rows 0: not one of its tensors
void sandwich_tensor_shape(const Stack* S, const StackLayer& W, const std::string& t, int* rows, int* cols) {
  const mi_layer_spec& s = W.s;
  *rows = *cols = 0;
  const bool ff = s.ff_kind != MI_FF_NONE;
  auto is = [&](int r, int k) { *rows = r; *cols = k; };
  if (t == "norm1" || t == "norm1b" || (ff && (t == "norm2" || t == "norm2b"))) is(S->D, 0);
  else if (t == "canon1" || (ff && t == "canon2")) is(S->D, S->cfg.conv_taps);
  else if (t == "mix.q") is(s.num_heads * s.qk_dim, S->D);
  else if (t == "mix.dkv" && s.kv_from < 0) is(s.kv_rank, S->D);
  else if (t == "mix.dkv.norm" && s.kv_from < 0) is(s.kv_rank, 0);
  else if (t == "mix.uk") is(s.num_heads * s.qk_dim, s.kv_rank);
  else if (t == "mix.uv") is(s.num_heads * s.v_dim, s.kv_rank);
  else if (t == "mix.o") is(S->D, s.num_heads * s.v_dim);
  else if (s.ff_kind == MI_FF_GLU) {
    if (t == "mlp.gate" || t == "mlp.up") is(s.ff_size, S->D);
    else if (t == "mlp.down") is(S->D, s.ff_size);
  } else if (s.ff_kind == MI_FF_MOE) {
    experts_tensor_shape(S, s, t, rows, cols);
  }
}

// W_uk: transposed, with ones on the rotated part's diagonal; and, as W_uv, a block of rows of the prompts' matrix
int latent_place(mi_ctx* c, StackLayer& W, bool k, const float* dev, int cols) {
  Stack* S = c->stack;
  const LatentGeom& g = W.lg;
  hipStream_t st = c->stream;
  const int n = k ? g.dk : g.dv, dq = g.dq();
  auto at = [&](void* base, size_t elems) -> void* { return reinterpret_cast<unsigned char*>(base) + elems * S->elem(); };
  float *tmp = nullptr, *ones = nullptr;      // [rank][dq]: W_uk^T, zeros behind it; [nr][dq]: zeros, then the unit matrix
  int rc = MI_OK;
  if (k) {
    std::vector<float> u((size_t)std::max(g.nr, 1) * dq, 0.f);
    for (int i = 0; i < g.nr; ++i) u[(size_t)i * dq + g.dk + i] = 1.f;
    MI_HIP(hipMalloc(reinterpret_cast<void**>(&tmp), (size_t)cols * dq * 4));
    MI_HIP(hipMalloc(reinterpret_cast<void**>(&ones), u.size() * 4));
    MI_HIP(hipMemcpyAsync(ones, u.data(), u.size() * 4, hipMemcpyHostToDevice, st));
    MI_HIP(hipMemsetAsync(tmp, 0, (size_t)cols * dq * 4, st));
    MI_HIP(hipStreamSynchronize(st));
  }
  for (int h = 0; h < g.H && rc == MI_OK; ++h) {
    const float* src = dev + (size_t)h * n * cols;
    if (k) {
      void* dst = at(W.w_uk, (size_t)h * g.cp * g.dkp);
      rc = launch_transpose(src, n, cols, tmp, dq, st);
      if (rc == MI_OK) rc = launch_place(tmp, dq, 0, cols, dq, dst, g.dkp, S->f32, 0, 0, st);
      if (rc == MI_OK && g.nr) rc = launch_place(ones, dq, 0, g.nr, dq, dst, g.dkp, S->f32, g.rp, 0, st);
    } else {
      rc = launch_place(src, cols, 0, n, cols, at(W.w_uv, (size_t)h * g.dvp * g.rp), g.rp, S->f32, 0, 0, st);
    }
    if (rc == MI_OK && W.fast()) {
      const int row0 = k ? h * g.dkp : g.H * g.dkp + h * g.dvp;
      rc = launch_place(src, cols, 0, n, cols, W.ukv.L.w, W.ukv.K, false, row0, 0, st);
      if (rc == MI_OK && k && g.nr) rc = launch_place(ones, dq, g.dk, g.nr, g.nr, W.ukv.L.w, W.ukv.K, false, row0 + g.dk, g.rp, st);
    }
  }
  hipStreamSynchronize(st);
  hipFree(tmp);
  hipFree(ones);
  return rc;
}

int experts_place(mi_ctx* c, StackLayer& W, const std::string& t, const float* dev, int rows, int cols) {
  Stack* S = c->stack;
  const mi_layer_spec& s = W.s;
  hipStream_t st = c->stream;
  auto at = [&](void* base, size_t elems) -> void* { return reinterpret_cast<unsigned char*>(base) + elems * S->elem(); };
  auto place = [&](void* dst, int K, int row0 = 0, int step = 1) { return launch_place(dev, cols, 0, rows, cols, dst, K, S->f32, row0, 0, st, step); };
  if (t == "mlp.router" && !S->f32) MI_TRY(place(W.router_t.L.w, W.router_t.K));
  if (t == "mlp.router") return launch_place_rows(dev, rows, cols, W.router, S->Kd, S->f32, st);
  if (t == "mlp.router.b" || t == "mlp.correction") return launch_offset_copy(dev, rows, 0.f, W.router_b, st);
  int e = -1, off = 0;
  sscanf(t.c_str(), "mlp.e%d.%n", &e, &off);
  const std::string m = t.substr(off);
  const ExpertsLinear gu = W.expert_up(), dn = W.expert_dn();
  if (m == "down") return place(at(W.expert_down, (size_t)e * dn.N * dn.K), dn.K);
  if (s.ff_act == MI_ACT_RELU2) return place(at(W.expert_gu, (size_t)e * gu.N * gu.K), gu.K);
  return place(at(W.expert_gu, (size_t)e * gu.N * gu.K), gu.K, m == "up" ? 1 : 0, 2);
}

int sandwich_place(mi_ctx* c, StackLayer& W, const std::string& t, const float* dev, int rows, int cols) {
  Stack* S = c->stack;
  const mi_layer_spec& s = W.s;
  hipStream_t st = c->stream;
  auto vec = [&](float* dst) -> int {
    MI_HIP(hipMemcpyAsync(dst, dev, (size_t)rows * 4, hipMemcpyDeviceToDevice, st));
    return MI_OK;
  };
  auto place = [&](void* dst, int K, int row0 = 0, int step = 1) { return launch_place(dev, cols, 0, rows, cols, dst, K, S->f32, row0, 0, st, step); };
  if (t == "norm1") return vec(W.n1.w);
  if (t == "norm1b") return vec(W.n1b.w);
  if (t == "norm2") return vec(W.n2.w);
  if (t == "norm2b") return vec(W.n2b.w);
  if (t == "canon1" || t == "canon2") return launch_transpose(dev, rows, cols, t == "canon1" ? W.conv1 : W.conv2, S->ld, st);
  if (t == "mix.q") return place(W.qkv.L.w, W.qkv.K);
  if (t == "mix.dkv") return place(W.qkv.L.w, W.qkv.K, s.num_heads * s.qk_dim);
  if (t == "mix.dkv.norm") return vec(W.c_norm);
  if (t == "mix.o") return place(W.out.L.w, W.out.K);
  if (t == "mix.uk" || t == "mix.uv") return latent_place(c, W, t == "mix.uk", dev, cols);
  if (t == "mlp.gate") return place(W.up.L.w, W.up.K, 0, 2);
  if (t == "mlp.up") return place(W.up.L.w, W.up.K, 1, 2);
  if (t == "mlp.down") return place(W.down.L.w, W.down.K);
  return experts_place(c, W, t, dev, rows, cols);
}

// ---- one-norm blocks: geometry and weights of one layer ----------------------------------------------------------------------
int delta_layer_create(mi_ctx* c, StackLayer& W) {
  Stack* S = c->stack;
  const mi_layer_spec& s = W.s;
  size_t* wb = &c->weight_bytes;
  DeltaGeom& g = W.dg;
  g = DeltaGeom{s.num_heads, s.num_kv_heads, s.qk_dim, s.v_dim, pad_to(s.qk_dim, 16), pad_to(s.v_dim, 16), s.conv_taps};
  W.col_b = pad_to(g.channels(), 16);
  W.col_a = W.col_b + pad_to(g.H, 16);
  W.col_g = W.col_a + pad_to(s.decay_rank, 16);
  MI_TRY(alloc_mat(c, W.qkv, W.col_g + s.gate_rank, S->D, 1.f));
  MI_TRY(alloc_mat(c, W.a2, g.H * g.dk, s.decay_rank, 1.f));
  MI_TRY(alloc_mat(c, W.g2, g.H * g.dv, s.gate_rank, 1.f));
  MI_TRY(alloc_mat(c, W.out, S->D, g.H * g.dv, 1.f));
  MI_TRY(alloc0(c, &W.conv, (size_t)g.taps * g.channels() * 4, wb));
  MI_TRY(alloc0(c, &W.a_log, (size_t)g.H * 4, wb));
  MI_TRY(alloc0(c, &W.dt, (size_t)g.H * g.dk * 4, wb));
  MI_TRY(alloc0(c, &W.o_norm, (size_t)g.dv * 4, wb));
  S->z_ld = std::max(S->z_ld, W.a2.N + W.g2.N);
  S->low_ld = std::max(S->low_ld, std::max(W.a2.K, W.g2.K));
  S->chunk_floats = std::max(S->chunk_floats, delta_chunk_floats(g));
  S->cat_ld = std::max(S->cat_ld, W.out.K);
  S->state_slots = c->cfg.max_num_seqs;
  return MI_OK;
}

int one_norm_layer_create(mi_ctx* c, StackLayer& W, const std::string& p) {
  Stack* S = c->stack;
  const mi_layer_spec& s = W.s;
  size_t* wb = &c->weight_bytes;
  auto want = [&](const char* n) { S->missing.push_back(p + n); };
  MI_TRY(alloc0(c, &W.n1.w, (size_t)S->ld * 4, wb));
  want("norm1");
  if (s.mixer_kind == MI_MIX_DELTA) {
    MI_TRY(delta_layer_create(c, W));
    for (const char* n : {"q", "q.conv", "k", "k.conv", "v", "v.conv", "b", "A_log", "a1", "a2", "dt_bias", "g1", "g2", "norm", "o"}) want((std::string("mix.") + n).c_str());
  } else {
    const int dq = s.num_heads * (s.qk_dim + s.rot_dim), gates = s.out_gate == MI_GATE_HEAD ? s.num_heads : s.out_gate == MI_GATE_ELEMENT ? s.num_heads * s.v_dim : 0;
    W.col_q = pad_to(s.kv_rank + s.rot_dim, 16);
    W.col_g = W.col_q + pad_to(s.q_rank ? s.q_rank : dq, 16);
    MI_TRY(alloc_mat(c, W.qkv, W.col_g + gates, S->D, 1.f));
    MI_TRY(latent_layer_create(c, W));
    MI_TRY(alloc0(c, &W.c_norm, (size_t)s.kv_rank * 4, wb));
    if (s.q_rank) {
      MI_TRY(alloc_mat(c, W.uq, dq, s.q_rank, 1.f));
      MI_TRY(alloc0(c, &W.q_norm, (size_t)s.q_rank * 4, wb));
      S->cq_ld = std::max(S->cq_ld, W.uq.K);
      S->q2_ld = std::max(S->q2_ld, W.uq.N);
      for (const char* n : {"mix.dq", "mix.dq.norm", "mix.uq"}) want(n);
    } else {
      want("mix.q");
    }
    for (const char* n : {"mix.dkv", "mix.dkv.norm", "mix.uk", "mix.uv", "mix.o"}) want(n);
    if (gates) want("mix.g");
  }
  S->qkv_ld = std::max(S->qkv_ld, W.qkv.N);
  return s.ff_kind == MI_FF_MOE ? experts_create(c, W, p) : MI_OK;
}

void one_norm_tensor_shape(const Stack* S, const StackLayer& W, const std::string& t, int* rows, int* cols) {
  const mi_layer_spec& s = W.s;
  *rows = *cols = 0;
  auto is = [&](int r, int k) { *rows = r; *cols = k; };
  if (t == "norm1") return is(S->D, 0);
  if (s.ff_kind == MI_FF_MOE && t.compare(0, 4, "mlp.") == 0) return experts_tensor_shape(S, s, t, rows, cols);
  if (t.compare(0, 4, "mix.") != 0) return;
  const std::string m = t.substr(4);
  const int H = s.num_heads, G = s.num_kv_heads;
  if (s.mixer_kind == MI_MIX_DELTA) {
    const int qk = G * s.qk_dim, v = H * s.v_dim;
    if (m == "q" || m == "k") is(qk, S->D);
    else if (m == "q.conv" || m == "k.conv") is(qk, s.conv_taps);
    else if (m == "v") is(v, S->D);
    else if (m == "v.conv") is(v, s.conv_taps);
    else if (m == "b") is(H, S->D);
    else if (m == "A_log") is(H, 0);
    else if (m == "a1") is(s.decay_rank, S->D);
    else if (m == "a2") is(H * s.qk_dim, s.decay_rank);
    else if (m == "dt_bias") is(H * s.qk_dim, 0);
    else if (m == "g1") is(s.gate_rank, S->D);
    else if (m == "g2") is(v, s.gate_rank);
    else if (m == "norm") is(s.v_dim, 0);
    else if (m == "o") is(S->D, v);
    return;
  }
  const int dq = H * (s.qk_dim + s.rot_dim);
  if (m == "dq" && s.q_rank) is(s.q_rank, S->D);
  else if (m == "dq.norm" && s.q_rank) is(s.q_rank, 0);
  else if (m == "uq" && s.q_rank) is(dq, s.q_rank);
  else if (m == "q" && !s.q_rank) is(dq, S->D);
  else if (m == "dkv") is(s.kv_rank + s.rot_dim, S->D);
  else if (m == "dkv.norm") is(s.kv_rank, 0);
  else if (m == "uk") is(H * s.qk_dim, s.kv_rank);
  else if (m == "uv") is(H * s.v_dim, s.kv_rank);
  else if (m == "g" && s.out_gate != MI_GATE_NONE) is(s.out_gate == MI_GATE_HEAD ? H : H * s.v_dim, S->D);
  else if (m == "o") is(S->D, H * s.v_dim);
}

int one_norm_place(mi_ctx* c, StackLayer& W, const std::string& t, const float* dev, int rows, int cols) {
  Stack* S = c->stack;
  const mi_layer_spec& s = W.s;
  hipStream_t st = c->stream;
  auto vec = [&](float* dst, float offset = 0.f) { return launch_offset_copy(dev, rows, offset, dst, st); };
  auto place = [&](const StackMat& m, int row0 = 0) { return launch_place(dev, cols, 0, rows, cols, m.L.w, m.K, S->f32, row0, 0, st); };
  if (t == "norm1") return vec(W.n1.w, S->cfg.norm_offset);
  if (t.compare(0, 4, "mlp.") == 0) return experts_place(c, W, t, dev, rows, cols);
  const std::string m = t.substr(4);
  if (m == "o") return place(W.out);
  if (s.mixer_kind == MI_MIX_DELTA) {
    const DeltaGeom& g = W.dg;
    const int part = m[0] == 'q' ? 0 : m[0] == 'k' ? g.G * g.dk : 2 * g.G * g.dk;      // the tensor's channels
    if (m == "q" || m == "k" || m == "v") return place(W.qkv, part);
    if (m == "q.conv" || m == "k.conv" || m == "v.conv") return launch_transpose(dev, rows, cols, W.conv + part, g.channels(), st);
    if (m == "b") return place(W.qkv, W.col_b);
    if (m == "a1") return place(W.qkv, W.col_a);
    if (m == "g1") return place(W.qkv, W.col_g);
    if (m == "a2") return place(W.a2);
    if (m == "g2") return place(W.g2);
    return vec(m == "A_log" ? W.a_log : m == "dt_bias" ? W.dt : W.o_norm);
  }
  if (m == "uk" || m == "uv") return latent_place(c, W, m == "uk", dev, cols);
  if (m == "dkv") return place(W.qkv);
  if (m == "dq" || m == "q") return place(W.qkv, W.col_q);
  if (m == "g") return place(W.qkv, W.col_g);
  if (m == "uq") return place(W.uq);
  return vec(m == "dq.norm" ? W.q_norm : W.c_norm);
}

// ---- post-norm blocks: geometry and weights of one layer ---------------------------------------------------------------------
// name of a layer's tensor behind "mix." within the mixer it belongs to: 0 the only or the left one, 1 the right one, -1 neither's
int mixer_of(const StackLayer& W, const std::string& t, std::string* name) {
  if (t.compare(0, 4, "mix.") != 0) return -1;
  *name = t.substr(4);
  if (!W.s.beside_kind) return 0;
  for (int i = 0; i < 2; ++i) {
    const std::string p = i ? "right." : "left.";
    if (name->compare(0, p.size(), p) == 0) { *name = name->substr(p.size()); return i; }
  }
  return -1;
}

int post_norm_layer_create(mi_ctx* c, StackLayer& W, const std::string& p) {
  Stack* S = c->stack;
  const mi_layer_spec& s = W.s;
  size_t* wb = &c->weight_bytes;
  auto want = [&](const std::string& n) { S->missing.push_back(p + n); };
  auto vec = [&](float** v, size_t n) { return alloc0(c, v, n * 4, wb); };
  MI_TRY(vec(&W.n1.w, S->ld));
  want("norm1");
  if (s.ff_kind != MI_FF_NONE) {
    MI_TRY(vec(&W.n2.w, S->ld));
    MI_TRY(alloc_mat(c, W.up, s.ff_size, S->D, 1.f));
    MI_TRY(alloc_mat(c, W.down, S->D, s.ff_size, 1.f));
    W.ffk = W.down.K;
    S->act_ld = std::max(S->act_ld, W.ffk);
    for (const char* n : {"norm2", "mlp.up", "mlp.down"}) want(n);
  }
  if (W.has_scan()) {
    const ScanGeom& g = W.scan = scan_geom(s.ssm_inner, s.ssm_state, s.dt_rank);
    W.col_z = pad_to(g.C, 16);
    W.col_B = pad_to(g.rank, 16);
    W.col_C = W.col_B + pad_to(g.N, 16);
    MI_TRY(alloc_mat(c, W.qkv, W.col_z + g.C, S->D, 1.f));
    MI_TRY(alloc_mat(c, W.low_in, W.col_C + g.N, g.C, 1.f));
    MI_TRY(alloc_mat(c, W.dt_mat, g.C, g.rank, 1.f));
    MI_TRY(alloc_mat(c, W.out, S->D, g.C, 1.f));
    MI_TRY(alloc0(c, &W.w_dt, (size_t)g.C * g.rank_p * S->elem(), wb));
    MI_TRY(vec(&W.decay, (size_t)g.C * g.Np));
    MI_TRY(vec(&W.dt, g.C));
    MI_TRY(vec(&W.ssm_d, g.C));
    S->xc_ld = std::max(S->xc_ld, W.low_in.K);
    S->xp_ld = std::max(S->xp_ld, W.low_in.N);
    S->low_ld = std::max(S->low_ld, W.dt_mat.K);
    S->dtp_ld = std::max(S->dtp_ld, W.dt_mat.N);
    for (const char* n : {"in", "conv", "conv.b", "x", "dt", "dt.b", "A_log", "D", "o"}) want(std::string("mix.") + n);
  } else {
    const std::string m = s.beside_kind ? "mix.left." : "mix.";
    const int qk = (s.num_heads + s.num_kv_heads) * s.qk_dim;
    W.g = HeadGeom{s.num_heads, s.num_kv_heads, s.qk_dim, s.v_dim, pad_to(s.qk_dim, 16), pad_to(s.v_dim, 16)};
    W.attn_cols = pad_to(s.num_heads * s.v_dim, 16);
    int n = pad_to(qk + (s.keys_as_values ? 0 : s.num_kv_heads * s.v_dim), 16);
    W.col_g = n;
    if (s.out_gate) n = W.col_g + pad_to(s.num_heads, 16);
    if (W.has_ssd()) {
      const SsdGeom& g = W.ssd = ssd_geom(s.ssm_heads, s.ssm_dim, s.ssm_state, s.ssm_groups);
      W.col_z = n;
      W.col_x = W.col_z + pad_to(g.inner(), 16);
      W.col_dt = W.col_x + pad_to(g.channels(), 16);
      n = W.col_dt + pad_to(g.H, 16);
      MI_TRY(vec(&W.a_log, g.H));
      MI_TRY(vec(&W.dt, g.H));
      MI_TRY(vec(&W.ssm_d, g.H));
      MI_TRY(vec(&W.o_norm, g.inner()));
      S->xc_ld = std::max(S->xc_ld, pad_to(g.channels(), 16));
      S->yssm_ld = std::max(S->yssm_ld, pad_to(g.inner(), 16));
      S->ssd_chunk_floats = std::max(S->ssd_chunk_floats, ssd_chunk_floats(g));
      for (const char* t : {"in", "conv", "conv.b", "dt_bias", "A_log", "D", "norm", "o"}) want(std::string("mix.right.") + t);
    }
    MI_TRY(alloc_mat(c, W.qkv, n, S->D, 1.f));
    MI_TRY(alloc_mat(c, W.out, S->D, W.attn_cols + (W.has_ssd() ? W.ssd.inner() : 0), 1.f));
    for (const char* t : {"q", "k", "o"}) want(m + t);
    if (!s.keys_as_values) want(m + "v");
    W.heads = HeadRule{s.qk_norm || s.qk_unit_norm, nullptr, nullptr, nullptr, s.keys_as_values != 0};
    if (s.qk_bias) {
      MI_TRY(vec(&W.qk_bias, qk));
      W.heads.bias = W.qk_bias;
      want(m + "q.b"); want(m + "k.b");
    }
    if (s.qk_norm) {
      MI_TRY(vec(&W.q_norm, s.qk_dim));
      MI_TRY(vec(&W.k_norm, s.qk_dim));
      W.heads.q_norm = W.q_norm; W.heads.k_norm = W.k_norm;
      want(m + "q.norm"); want(m + "k.norm");
    }
    if (s.out_gate) want(m + "g");
    if (s.softmax_sink == MI_SINK_LEARNED) {
      MI_TRY(vec(&W.sinks, s.num_heads));
      want(m + "sink");
    }
    if (s.distance_bias == MI_BIAS_TABLE) {
      W.table_rows = distance_rows(s.rel_rows, s.rel_far, s.chunk);
      MI_TRY(vec(&W.table, (size_t)s.num_heads * W.table_rows.size()));
      want(m + "rel");
    }
    W.attn = AttnSpec{W.g, s.scale, s.window, nullptr, 0, s.softmax_sink != MI_SINK_NONE, s.chunk, W.sinks, W.table, (int)W.table_rows.size()};
    S->q_cols = std::max(S->q_cols, s.num_heads * W.g.dkp);
  }
  if (W.ssm_state_floats()) {
    const int C = W.conv_channels();
    MI_TRY(vec(&W.conv, (size_t)s.conv_taps * C));
    MI_TRY(vec(&W.conv_b, C));
    S->state_slots = c->cfg.max_num_seqs;
  }
  S->qkv_ld = std::max(S->qkv_ld, W.qkv.N);
  S->cat_ld = std::max(S->cat_ld, W.out.K);
  return MI_OK;
}

void post_norm_tensor_shape(const Stack* S, const StackLayer& W, const std::string& t, int* rows, int* cols) {
  const mi_layer_spec& s = W.s;
  *rows = *cols = 0;
  auto is = [&](int r, int k) { *rows = r; *cols = k; };
  const bool ff = s.ff_kind != MI_FF_NONE;
  if (t == "norm1" || (ff && t == "norm2")) return is(S->D, 0);
  if (ff && t == "mlp.up") return is(s.ff_size, S->D);
  if (ff && t == "mlp.down") return is(S->D, s.ff_size);
  std::string m;
  const int part = mixer_of(W, t, &m);
  if (part < 0) return;
  if (part == 0 && !W.has_scan()) {
    const int H = s.num_heads, G = s.num_kv_heads, d = s.qk_dim;
    if (m == "q") is(H * d, S->D);
    else if (m == "k") is(G * d, S->D);
    else if (m == "v" && !s.keys_as_values) is(G * s.v_dim, S->D);
    else if (m == "q.b" && s.qk_bias) is(H * d, 0);
    else if (m == "k.b" && s.qk_bias) is(G * d, 0);
    else if ((m == "q.norm" || m == "k.norm") && s.qk_norm) is(d, 0);
    else if (m == "rel" && s.distance_bias == MI_BIAS_TABLE) is(s.rel_rows, H);
    else if (m == "sink" && s.softmax_sink == MI_SINK_LEARNED) is(H, 0);
    else if (m == "g" && s.out_gate) is(H, S->D);
    else if (m == "o") is(S->D, H * s.v_dim);
    return;
  }
  const int C = W.conv_channels();
  if (m == "conv") return is(C, s.conv_taps);
  if (m == "conv.b") return is(C, 0);
  if (W.has_scan()) {
    const ScanGeom& g = W.scan;
    if (m == "in") is(2 * g.C, S->D);
    else if (m == "x") is(g.rank + 2 * g.N, g.C);
    else if (m == "dt") is(g.C, g.rank);
    else if (m == "dt.b" || m == "D") is(g.C, 0);
    else if (m == "A_log") is(g.C, g.N);
    else if (m == "o") is(S->D, g.C);
    return;
  }
  const SsdGeom& g = W.ssd;
  if (m == "in") is(g.inner() + C + g.H, S->D);
  else if (m == "dt_bias" || m == "A_log" || m == "D") is(g.H, 0);
  else if (m == "norm") is(g.inner(), 0);
  else if (m == "o") is(S->D, g.inner());
}

int post_norm_place(mi_ctx* c, StackLayer& W, const std::string& t, const float* dev, int rows, int cols) {
  Stack* S = c->stack;
  const mi_layer_spec& s = W.s;
  hipStream_t st = c->stream;
  auto vec = [&](float* dst) { return launch_offset_copy(dev, rows, 0.f, dst, st); };
  // rows r0 .. + n of the tensor to row0 of the matrix
  auto part = [&](const StackMat& m, int r0, int n, int row0, int col0 = 0) {
    return launch_place(dev + (size_t)r0 * cols, cols, 0, n, cols, m.L.w, m.K, S->f32, row0, col0, st);
  };
  if (t == "norm1") return vec(W.n1.w);
  if (t == "norm2") return vec(W.n2.w);
  if (t == "mlp.up") return part(W.up, 0, rows, 0);
  if (t == "mlp.down") return part(W.down, 0, rows, 0);
  std::string m;
  const int which = mixer_of(W, t, &m);
  if (which == 0 && !W.has_scan()) {
    const int qn = s.num_heads * s.qk_dim, kn = s.num_kv_heads * s.qk_dim;
    if (m == "q") return part(W.qkv, 0, rows, 0);
    if (m == "k") return part(W.qkv, 0, rows, qn);
    if (m == "v") return part(W.qkv, 0, rows, qn + kn);
    if (m == "g") return part(W.qkv, 0, rows, W.col_g);
    if (m == "o") return part(W.out, 0, rows, 0);
    if (m == "q.b") return vec(W.qk_bias);
    if (m == "k.b") return vec(W.qk_bias + qn);
    if (m == "q.norm") return vec(W.q_norm);
    if (m == "k.norm") return vec(W.k_norm);
    if (m == "sink") return vec(W.sinks);
    return stack_distance_table(dev, W.table_rows, s.rel_rows, s.num_heads, W.table, st);
  }
  if (m == "conv") return launch_transpose(dev, rows, cols, W.conv, rows, st);
  if (m == "conv.b") return vec(W.conv_b);
  if (m == "D") return vec(W.ssm_d);
  if (W.has_scan()) {
    const ScanGeom& g = W.scan;
    if (m == "in") { MI_TRY(part(W.qkv, 0, g.C, 0)); return part(W.qkv, g.C, g.C, W.col_z); }
    if (m == "x") {
      MI_TRY(part(W.low_in, 0, g.rank, 0));
      MI_TRY(part(W.low_in, g.rank, g.N, W.col_B));
      return part(W.low_in, g.rank + g.N, g.N, W.col_C);
    }
    if (m == "dt") { MI_TRY(launch_place_rows(dev, rows, cols, W.w_dt, g.rank_p, S->f32, st)); return part(W.dt_mat, 0, rows, 0); }
    if (m == "dt.b") return vec(W.dt);
    if (m == "A_log") return launch_scan_decay(dev, g, W.decay, st);
    return part(W.out, 0, rows, 0);
  }
  const SsdGeom& g = W.ssd;
  if (m == "in") {
    MI_TRY(part(W.qkv, 0, g.inner(), W.col_z));
    MI_TRY(part(W.qkv, g.inner(), g.channels(), W.col_x));
    return part(W.qkv, g.inner() + g.channels(), g.H, W.col_dt);
  }
  if (m == "o") return part(W.out, 0, rows, 0, W.attn_cols);
  if (m == "norm") return launch_scaled_copy(dev, rows, s.beside_mult, W.o_norm, st);
  return vec(m == "A_log" ? W.a_log : W.dt);
}

}  // namespace

int stack_distance_table(const float* rel, const std::vector<int>& rows, int rel_rows, int H, float* table, hipStream_t s) {
  std::vector<float> r((size_t)rel_rows * H), t((size_t)H * rows.size());
  MI_HIP(hipMemcpyAsync(r.data(), rel, r.size() * 4, hipMemcpyDeviceToHost, s));
  MI_HIP(hipStreamSynchronize(s));
  for (int h = 0; h < H; ++h)
    for (size_t n = 0; n < rows.size(); ++n) t[h * rows.size() + n] = r[(size_t)rows[n] * H + h];
  MI_HIP(hipMemcpyAsync(table, t.data(), t.size() * 4, hipMemcpyHostToDevice, s));
  MI_HIP(hipStreamSynchronize(s));
  return MI_OK;
}

int stack_create(mi_ctx* c, const mi_stack_config& cfg) {
  Stack* S = c->stack = new Stack();
  S->cfg = cfg;
  S->cfg.layers = nullptr;
  S->f32 = cfg.compute_dtype == MI_F32;
  S->D = cfg.width;
  S->ld = pad_to(S->D, 16);
  S->Kd = pad_to(S->D, 64);
  c->H = S->ld;
  c->V_l = cfg.vocab_size;
  const bool loop = cfg.loop_times > 0;
  for (int i = 0; i < cfg.num_layers; ++i) {
    if (S->one_norm()) {
      int j = i;
      while (cfg.layers[j].weights_of >= 0) j = cfg.layers[j].weights_of;     // (checked by mi_ctx_create_stack)
      S->runs.push_back({j, false});
      continue;
    }
    if (!loop || i < cfg.loop_start || i >= cfg.loop_stop) {
      S->runs.push_back({i, false});
      continue;
    }
    if (i > cfg.loop_start) continue;
    for (int t = 0; t < cfg.loop_times; ++t)
      for (int l = cfg.loop_start; l < cfg.loop_stop; ++l) S->runs.push_back({l, l == cfg.loop_start});
  }
  auto want = [&](const std::string& n) { S->missing.push_back(n); };
  size_t* wb = &c->weight_bytes;
  MI_TRY(alloc0(c, &S->embed, (size_t)cfg.vocab_size * S->D * S->elem(), wb));
  want("embed");
  if (cfg.max_positions > 0) {
    MI_TRY(alloc0(c, &S->pos, (size_t)cfg.max_positions * S->D * S->elem(), wb));
    want("pos");
  }
  S->conv_keep = cfg.conv_taps > 1 ? std::min(c->cfg.block_size, cfg.conv_taps - 1 + cfg.state_lookahead) : 0;
  if (loop) {
    MI_TRY(alloc_mat(c, S->loop_in, S->D, 2 * S->Kd, 1.f));
    want("loop.in");
  }
  S->layers.resize(cfg.num_layers);
  for (int i = 0; i < cfg.num_layers; ++i) {
    StackLayer& W = S->layers[i];
    W.s = cfg.layers[i];
    const mi_layer_spec& s = W.s;
    if (S->post_norm()) {
      MI_TRY(post_norm_layer_create(c, W, "l" + std::to_string(i) + "."));
      continue;
    }
    if (S->one_norm()) {
      if (s.weights_of < 0) MI_TRY(one_norm_layer_create(c, W, "l" + std::to_string(i) + "."));
      continue;
    }
    if (S->sandwich()) {
      MI_TRY(sandwich_layer_create(c, W, "l" + std::to_string(i) + "."));
      continue;
    }
    W.g = HeadGeom{s.num_heads, s.num_kv_heads, s.qk_dim, s.v_dim, pad_to(s.qk_dim, 16), pad_to(s.v_dim, 16)};
    W.attn_cols = pad_to(s.num_heads * s.v_dim, 16);
    W.ff_cols = s.ff_kind == MI_FF_NONE ? 0 : pad_to(s.ff_size, 16);
    MI_TRY(alloc_mat(c, W.qkv, (s.num_heads + s.num_kv_heads) * s.qk_dim + s.num_kv_heads * s.v_dim, S->D, 1.f));
    if (W.ff_cols) MI_TRY(alloc_mat(c, W.up, s.ff_size, S->D, 1.f));
    MI_TRY(alloc_mat(c, W.out, S->D, W.attn_cols + W.ff_cols, cfg.residual_mult));
    MI_TRY(alloc_norm(c, W.n1));
    if (W.ff_cols) MI_TRY(alloc_norm(c, W.n2));
    if (s.distance_bias) {
      std::vector<float> sl(s.num_heads);
      for (int h = 0; h < s.num_heads; ++h) sl[h] = (float)std::exp2(-8.0 * (h + 1) / s.num_heads);
      MI_TRY(alloc0(c, &W.slopes, sl.size() * 4, wb));
      MI_HIP(hipMemcpyAsync(W.slopes, sl.data(), sl.size() * 4, hipMemcpyHostToDevice, c->stream));
      MI_HIP(hipStreamSynchronize(c->stream));
    }
    W.attn = AttnSpec{W.g, s.scale, s.window, W.slopes, s.qk_unit_norm ? 1 : 0, s.softmax_sink ? 1 : 0};
    W.heads.unit_norm = s.qk_unit_norm != 0;
    S->qkv_ld = std::max(S->qkv_ld, W.qkv.N);
    S->q_cols = std::max(S->q_cols, s.num_heads * W.g.dkp);
    S->cat_ld = std::max(S->cat_ld, W.out.K);
    const std::string p = "l" + std::to_string(i) + ".";
    for (const char* n : {"norm1", "norm1.b", "mix.q", "mix.k", "mix.v", "mix.o"}) want(p + n);
    if (W.ff_cols)
      for (const char* n : {"norm2", "norm2.b", "mlp.up", "mlp.down"}) want(p + n);
  }
  MI_TRY(alloc_norm(c, S->final_norm));
  MI_TRY(alloc_mat(c, S->head, cfg.vocab_size, S->D, cfg.logit_scale));
  want("final.norm"); want("head");
  if (cfg.norm_groups == 0) want("final.norm.b");
  MI_HIP(hipStreamSynchronize(c->stream));
  return MI_OK;
}

void stack_destroy(mi_ctx* c) {
  Stack* S = c->stack;
  for (StackLayer& W : S->layers) {
    free_mat(W.qkv); free_mat(W.up); free_mat(W.out);
    free_mat(W.down); free_mat(W.ukv); free_mat(W.router_t);
    free_norm(W.n1); free_norm(W.n2); free_norm(W.n1b); free_norm(W.n2b);
    free_mat(W.low_in); free_mat(W.dt_mat);
    free_mat(W.uq); free_mat(W.a2); free_mat(W.g2);
    void* ps[] = {W.q_norm, W.conv, W.a_log, W.dt, W.o_norm, W.slopes, W.conv1, W.conv2, W.c_norm, W.w_uk, W.w_uv, W.router, W.router_b, W.expert_gu, W.expert_down,
                  W.qk_bias, W.k_norm, W.sinks, W.table, W.w_dt, W.conv_b, W.decay, W.ssm_d};
    for (void* p : ps) hipFree(p);
  }
  free_mat(S->loop_in); free_mat(S->head);
  free_norm(S->final_norm);
  void* ptrs[] = {S->embed, S->pos, S->x0, S->qkv_out, S->logits_pad, S->n1, S->n2, S->q, S->cat, S->pair, S->attn_scratch, S->residuals,
                  S->y, S->pair_w, S->pair_ids, S->hb, S->act, S->qa, S->lat, S->kv_x, S->kv_k, S->kv_v, S->kv_bt, S->plan,
                  S->tickets, S->route_z, S->cq, S->low, S->q2, S->z, S->delta_records,
                  S->turns, S->xc, S->xp, S->dtp, S->yssm, S->ssd_records};
  for (void* p : ptrs) hipFree(p);
  for (float* p : S->state_at) hipFree(p);
  for (Stack::RotTable& r : S->rot) hipFree(r.t);
  delete S;
  c->stack = nullptr;
}

int stack_load_tensor(mi_ctx* c, const std::string& name, const float* dev, int rows, int cols) {
  Stack* S = c->stack;
  const mi_stack_config& k = S->cfg;
  hipStream_t s = c->stream;
  auto bad = [&]() -> int {
    set_error("tensor " + name + " [" + std::to_string(rows) + (cols ? ", " + std::to_string(cols) : std::string()) + "] has another shape than the configuration gives it");
    return MI_EINVAL;
  };
  auto done = [&](int rc) -> int {
    if (rc == MI_OK)
      for (size_t i = 0; i < S->missing.size(); ++i)
        if (S->missing[i] == name) { S->missing.erase(S->missing.begin() + i); break; }
    return rc;
  };
  auto place = [&](const StackMat& m, int n, int kk, int row0 = 0, int col0 = 0) -> int {
    if (rows != n || cols != kk) return bad();
    return done(launch_place(dev, cols, 0, rows, cols, m.L.w, m.K, S->f32, row0, col0, s));
  };
  auto vec = [&](float* dst) -> int {
    if (rows != S->D || cols != 0) return bad();
    MI_HIP(hipMemcpyAsync(dst, dev, (size_t)rows * 4, hipMemcpyDeviceToDevice, s));
    return done(MI_OK);
  };
  auto table = [&](void* dst, int n) -> int {
    if (rows != n || cols != S->D) return bad();
    if (S->f32) {
      MI_HIP(hipMemcpyAsync(dst, dev, (size_t)rows * cols * 4, hipMemcpyDeviceToDevice, s));
    } else {
      MI_TRY(launch_f32_to_bf16(dev, (uint16_t*)dst, (size_t)rows * cols, s));
    }
    return done(MI_OK);
  };
  if (name == "embed") return table(S->embed, k.vocab_size);
  if (name == "pos" && k.max_positions > 0) return table(S->pos, k.max_positions);
  if (name == "head") return place(S->head, k.vocab_size, S->D);
  if (name == "final.norm" && k.norm_offset != 0.f)
    return rows == S->D && cols == 0 ? done(launch_offset_copy(dev, rows, k.norm_offset, S->final_norm.w, s)) : bad();
  if (name == "final.norm") return vec(S->final_norm.w);
  if (name == "final.norm.b" && k.norm_groups == 0) return vec(S->final_norm.b);
  if (name == "loop.in" && k.loop_times > 0) {   // [x ; x0]: the halves at columns 0 and Kd
    if (rows != S->D || cols != 2 * S->D) return bad();
    for (int h = 0; h < 2; ++h) MI_TRY(launch_place(dev, cols, h * S->D, rows, S->D, S->loop_in.L.w, S->loop_in.K, S->f32, 0, h * S->Kd, s));
    return done(MI_OK);
  }
  int l = -1, at = 0;
  if (sscanf(name.c_str(), "l%d.%n", &l, &at) == 1 && at > 0 && l >= 0 && l < k.num_layers) {
    StackLayer& W = S->layers[l];
    const mi_layer_spec& p = W.s;
    const std::string t = name.substr(at);
    if (S->post_norm()) {
      int r = 0, cl = 0;
      post_norm_tensor_shape(S, W, t, &r, &cl);
      if (r > 0) return rows == r && cols == cl ? done(post_norm_place(c, W, t, dev, rows, cols)) : bad();
      set_error("tensor " + name + " is not part of this model's configuration");
      return MI_EINVAL;
    }
    if (S->one_norm()) {
      int r = 0, cl = 0;
      if (p.weights_of < 0) one_norm_tensor_shape(S, W, t, &r, &cl);
      if (r > 0) return rows == r && cols == cl ? done(one_norm_place(c, W, t, dev, rows, cols)) : bad();
      set_error("tensor " + name + " is not part of this model's configuration");
      return MI_EINVAL;
    }
    if (S->sandwich()) {
      int r = 0, cl = 0;
      sandwich_tensor_shape(S, W, t, &r, &cl);
      if (r > 0) return rows == r && cols == cl ? done(sandwich_place(c, W, t, dev, rows, cols)) : bad();
    }
    const int qn = p.num_heads * p.qk_dim, kn = p.num_kv_heads * p.qk_dim;
    if (!S->sandwich()) {
      if (t == "norm1") return vec(W.n1.w);
      if (t == "norm1.b") return vec(W.n1.b);
      if (t == "mix.q") return place(W.qkv, qn, S->D);
      if (t == "mix.k") return place(W.qkv, kn, S->D, qn);
      if (t == "mix.v") return place(W.qkv, p.num_kv_heads * p.v_dim, S->D, qn + kn);
      if (t == "mix.o") return place(W.out, S->D, p.num_heads * p.v_dim);
    }
    if (W.ff_cols) {
      if (t == "norm2") return vec(W.n2.w);
      if (t == "norm2.b") return vec(W.n2.b);
      if (t == "mlp.up") return place(W.up, p.ff_size, S->D);
      if (t == "mlp.down") return place(W.out, S->D, p.ff_size, 0, W.attn_cols);
    }
  }
  set_error("tensor " + name + " is not part of this model's configuration");
  return MI_EINVAL;
}

int stack_synthetic(mi_ctx* c, uint64_t seed, float std) {
  Stack* S = c->stack;
  const mi_stack_config& k = S->cfg;
  uint64_t tid = 1;
  float* buf = nullptr;
  size_t cap = 0;
  int rc = MI_OK;
  const std::vector<std::string> names = S->missing;
  for (const std::string& n : names) {
    int rows = S->D, cols = 0;
    float sd = std;
    bool is_norm = n.find("norm") != std::string::npos || (n.size() > 2 && n.compare(n.size() - 2, 2, ".b") == 0);
    if (is_norm && S->sandwich() && n[0] == 'l') {
      int r = 0, k0 = 0;
      sandwich_tensor_shape(S, S->layers[atoi(n.c_str() + 1)], n.substr(n.find('.') + 1), &r, &k0);
      rows = r;
    }
    if (n == "embed" || n == "head") { rows = k.vocab_size; cols = S->D; if (n == "embed") sd = 1.f; }
    else if (n == "pos") { rows = k.max_positions; cols = S->D; sd = 0.1f; }
    else if (n == "loop.in") cols = 2 * S->D;
    else if ((S->one_norm() || S->post_norm()) && n[0] == 'l') {
      const StackLayer& W = S->layers[atoi(n.c_str() + 1)];
      if (S->one_norm()) one_norm_tensor_shape(S, W, n.substr(n.find('.') + 1), &rows, &cols);
      else post_norm_tensor_shape(S, W, n.substr(n.find('.') + 1), &rows, &cols);
      if (n.find(".conv") != std::string::npos) sd = 0.3f;
      is_norm = cols == 0;
    } else if (!is_norm) {
      const int l = atoi(n.c_str() + 1);
      const mi_layer_spec& p = S->layers[l].s;
      const std::string t = n.substr(n.find('.') + 1);
      cols = S->D;
      if (S->sandwich()) {
        sandwich_tensor_shape(S, S->layers[l], t, &rows, &cols);
        if (t.compare(0, 5, "canon") == 0) sd = 0.3f;
      } else if (t == "mix.q") rows = p.num_heads * p.qk_dim;
      else if (t == "mix.k") rows = p.num_kv_heads * p.qk_dim;
      else if (t == "mix.v") rows = p.num_kv_heads * p.v_dim;
      else if (t == "mlp.up") rows = p.ff_size;
      else cols = t == "mix.o" ? p.num_heads * p.v_dim : p.ff_size;
    }
    const size_t elems = (size_t)rows * (cols ? cols : 1);
    if (elems > cap) {
      hipFree(buf);
      MI_HIP(hipMalloc(reinterpret_cast<void**>(&buf), elems * 4));
      cap = elems;
    }
    if (is_norm && S->one_norm())     // norms around zero; plain ones; decays, biases and corrections zero
      rc = launch_fill_f32(buf, elems, n.find(".mix.") != std::string::npos && n.find("norm") != std::string::npos ? 1.f : 0.f, c->stream);
    else if (is_norm && S->post_norm()) rc = launch_fill_f32(buf, elems, n.find("norm") != std::string::npos ? 1.f : 0.f, c->stream);
    else if (is_norm) rc = launch_fill_f32(buf, elems, n.size() > 2 && n.compare(n.size() - 2, 2, ".b") == 0 ? 0.f : 1.f, c->stream);
    else rc = launch_randn(buf, elems, seed, tid, sd, c->stream);
    ++tid;
    if (rc == MI_OK) rc = stack_load_tensor(c, n, buf, rows, cols);
    if (rc != MI_OK) break;
  }
  hipStreamSynchronize(c->stream);
  hipFree(buf);
  return rc;
}

void stack_artifact_tensors(mi_ctx* c, std::vector<std::pair<void*, size_t>>& out) {
  Stack* S = c->stack;
  const size_t nb = (size_t)S->ld * 4;
  auto mat = [&](StackMat& m) { out.push_back({m.L.w, (size_t)m.N * m.K * S->elem()}); };
  auto norm = [&](StackNorm& n) { out.push_back({n.w, nb}); out.push_back({n.b, nb}); };   // (an RMS norm's bias is zero)
  out.push_back({S->embed, (size_t)S->cfg.vocab_size * S->D * S->elem()});
  if (S->pos) out.push_back({S->pos, (size_t)S->cfg.max_positions * S->D * S->elem()});
  if (S->cfg.loop_times > 0) mat(S->loop_in);
  for (StackLayer& W : S->layers) {
    if (S->one_norm() && W.s.weights_of >= 0) continue;
    if (S->post_norm()) {
      auto put = [&](void* q, size_t elems) { if (q) out.push_back({q, elems * 4}); };
      const mi_layer_spec& p = W.s;
      mat(W.qkv); mat(W.out); put(W.n1.w, S->ld); put(W.n2.w, S->ld);
      for (StackMat* m : {&W.up, &W.down, &W.low_in, &W.dt_mat})
        if (m->L.w) mat(*m);
      if (W.w_dt) out.push_back({W.w_dt, (size_t)W.scan.C * W.scan.rank_p * S->elem()});
      const size_t heads = W.has_scan() ? W.scan.C : W.ssd.H;
      put(W.decay, (size_t)W.scan.C * W.scan.Np); put(W.dt, heads); put(W.ssm_d, heads); put(W.a_log, heads); put(W.o_norm, W.ssd.inner());
      put(W.conv, W.ssm_ring_floats()); put(W.conv_b, W.ssm_state_floats() ? W.conv_channels() : 0);
      put(W.qk_bias, (size_t)(p.num_heads + p.num_kv_heads) * p.qk_dim); put(W.q_norm, p.qk_dim); put(W.k_norm, p.qk_dim);
      put(W.sinks, p.num_heads); put(W.table, (size_t)p.num_heads * W.table_rows.size());
      continue;
    }
    if (S->parallel()) {
      mat(W.qkv); mat(W.out); norm(W.n1);
      if (W.ff_cols) { mat(W.up); norm(W.n2); }
      continue;
    }
    {
      const mi_layer_spec& p = W.s;
      auto put = [&](void* q, size_t bytes) { if (q) out.push_back({q, bytes}); };
      const size_t el = S->elem(), cb = (size_t)S->cfg.conv_taps * S->ld * 4;
      mat(W.qkv); mat(W.out);
      put(W.n1.w, nb); put(W.n1b.w, nb); put(W.n2.w, nb); put(W.n2b.w, nb);
      put(W.conv1, cb); put(W.conv2, cb); put(W.c_norm, (size_t)p.kv_rank * 4);
      put(W.w_uk, (size_t)p.num_heads * W.lg.cp * W.lg.dkp * el);
      put(W.w_uv, (size_t)p.num_heads * W.lg.dvp * W.lg.rp * el);
      if (W.fast()) mat(W.ukv);
      for (StackMat* m : {&W.uq, &W.a2, &W.g2})
        if (m->L.w) mat(*m);
      put(W.q_norm, (size_t)p.q_rank * 4);
      put(W.conv, (size_t)W.dg.taps * W.dg.channels() * 4); put(W.a_log, (size_t)W.dg.H * 4);
      put(W.dt, (size_t)W.dg.H * W.dg.dk * 4); put(W.o_norm, (size_t)W.dg.dv * 4);
      if (p.ff_kind == MI_FF_GLU) { mat(W.up); mat(W.down); }
      if (p.ff_kind == MI_FF_MOE) {
        const ExpertsLinear gu = W.expert_up(), dn = W.expert_dn();
        put(W.router, (size_t)p.experts * S->Kd * el); put(W.router_b, (size_t)p.experts * 4);
        if (!S->f32) mat(W.router_t);
        put(W.expert_gu, (size_t)gu.E * gu.N * gu.K * el); put(W.expert_down, (size_t)dn.E * dn.N * dn.K * el);
      }
    }
  }
  norm(S->final_norm);
  mat(S->head);
}

int stack_geometry_hash(const mi_ctx* c) {
  const Stack* S = c->stack;
  uint32_t h = 2166136261u;
  auto mix = [&](const void* p, size_t n) {
    for (size_t i = 0; i < n; ++i) h = (h ^ reinterpret_cast<const unsigned char*>(p)[i]) * 16777619u;
  };
  const mi_stack_config& k = S->cfg;
  const int32_t g[9] = {k.num_layers, k.width, k.vocab_size, k.max_positions, k.loop_times > 0, k.compute_dtype, k.block_kind, k.norm_groups, k.conv_taps};
  mix(g, sizeof g);
  const float f[2] = {k.embed_scale, k.norm_offset};
  if (S->one_norm()) mix(f, sizeof f);
  const float pf[3] = {k.embed_scale, k.pos_base, k.logit_scale};
  if (S->post_norm()) mix(pf, sizeof pf);
  for (const StackLayer& W : S->layers) mix(&W.s, sizeof W.s);
  return (int)(h & 0x7fffffff);
}

static size_t kv_run_elems_per_block(const mi_ctx* c, const StackLayer& W) {
  const Stack* S = c->stack;
  if (W.has_scan()) return 0;
  if (S->one_norm()) return W.s.mixer_kind == MI_MIX_LATENT ? (size_t)c->cfg.block_size * W.lg.cp : 0;
  if (S->sandwich())   // latents (own ones) and both convolutions' state
    return (W.s.kv_from < 0 ? (size_t)c->cfg.block_size * W.lg.cp : 0) + (size_t)S->conv_keep * S->Kd * (W.s.ff_kind == MI_FF_NONE ? 1 : 2);
  return (size_t)W.g.G * c->cfg.block_size * (W.g.dkp + W.g.dvp);
}
size_t stack_kv_bytes_per_block(const mi_ctx* c) {
  size_t e = 0;
  for (const StackRun& r : c->stack->runs) e += kv_run_elems_per_block(c, c->stack->layers[r.layer]);
  return e * c->stack->elem();
}

static size_t stack_scratch(const mi_ctx* c) {
  size_t b = 16;
  if (c->stack->sandwich() || c->stack->one_norm()) {
    for (const StackLayer& W : c->stack->layers)
      if (W.fast()) b = std::max(b, latent_attn_scratch_bytes(W.lg));
    return b;
  }
  for (const StackLayer& W : c->stack->layers)
    if (W.g.H) b = std::max(b, attn_window_scratch_bytes(c->cfg.max_num_seqs, W.g));
  return b;
}

// rows of the written-out keys and values: the longest sequence, and as much again for batches of several prompts
static int kv_work_rows(const mi_ctx* c) {
  return c->stack->kv_ldx ? 2 * pad_to(std::max(c->max_rows, c->cfg.max_model_len), kKvBlock) + 2 * kKvBlock : 0;
}

bool stack_has_state(const mi_ctx* c) { return c->stack && c->stack->state_slots > 0; }

static size_t state_floats(const mi_ctx* c, const StackLayer& W) {
  if (c->stack->post_norm()) return c->stack->state_slots * (W.ssm_state_floats() + W.ssm_ring_floats());
  return W.s.mixer_kind == MI_MIX_DELTA ? c->stack->state_slots * (W.dg.state_floats() + W.dg.ring_floats()) : 0;
}
// chunks of prompts whose factors are in memory at a time
static int delta_chunks(const mi_ctx* c) { return std::min(512, c->max_rows / kDeltaChunk + c->cfg.max_num_seqs); }

static int ssd_chunks(const mi_ctx* c) { return std::min(256, c->max_rows / kSsdChunk + c->cfg.max_num_seqs); }

size_t stack_workspace_estimate(const mi_ctx* c) {
  const Stack* S = c->stack;
  const size_t R = (size_t)c->max_rows;
  size_t extra = 0;
  if (S->post_norm()) {
    for (const StackRun& r : S->runs) extra += state_floats(c, S->layers[r.layer]) * 4;
    extra += R * (size_t)(S->xc_ld + S->low_ld) * S->elem() + R * (size_t)(S->xp_ld + S->dtp_ld + S->yssm_ld) * 4 + (size_t)ssd_chunks(c) * S->ssd_chunk_floats * 4;
  }
  if (S->one_norm()) {
    for (const StackRun& r : S->runs) extra += state_floats(c, S->layers[r.layer]) * 4;
    if (S->state_slots) extra += (size_t)delta_chunks(c) * S->chunk_floats * 4;
    extra += R * ((size_t)S->z_ld + S->q2_ld) * 4 + R * (2 * (size_t)S->low_ld + S->cq_ld) * S->elem();
    for (const StackLayer& W : S->layers) extra += W.s.mixer_kind == MI_MIX_LATENT ? (size_t)c->cfg.max_model_len * W.s.rot_dims * 4 : 0;
  }
  size_t b = 3 * R * S->ld * 4 + R * S->qkv_ld * 4 + R * (4 * (size_t)S->Kd + S->q_cols + S->cat_ld) * S->elem();
  b += extra;
  if (!S->parallel()) {
    const size_t pairs = R * std::max(1, S->max_top);
    b += (size_t)kv_work_rows(c) * (S->kv_ldx + S->kv_k_cols + S->kv_v_cols) * 2;
    b += pairs * S->ld * 4 + pairs * 16 + R * (S->max_experts + 1) * 4 + R * S->Kd * S->elem() + pairs * S->act_ld * S->elem() + 2 * R * S->lat_cols * S->elem();
  }
  b += (size_t)64 << 20;
  b += 2 * (size_t)c->cfg.max_num_seqs * pad_to(c->V_l, 16) * 4;
  return b + stack_scratch(c) + ((size_t)8 << 20);
}

// recurrent state, rotation tables and the workspace only one-norm blocks have
static int one_norm_alloc(mi_ctx* c) {
  Stack* S = c->stack;
  const size_t R = (size_t)c->max_rows;
  size_t* ws = &c->workspace_bytes;
  for (const StackRun& r : S->runs) {
    float* p = nullptr;
    if (const size_t n = state_floats(c, S->layers[r.layer])) MI_TRY(alloc0(c, &p, n * 4, &c->kv_bytes));
    S->state_at.push_back(p);
  }
  for (StackLayer& W : S->layers) {
    if (W.s.weights_of >= 0 || W.s.mixer_kind != MI_MIX_LATENT || W.s.rot_dim == 0) continue;
    for (const Stack::RotTable& r : S->rot)
      if (r.base == W.s.rot_base && r.dims == W.s.rot_dims) W.rot = r.t;
    if (W.rot) continue;
    const int half = W.s.rot_dims / 2, P = c->cfg.max_model_len;
    std::vector<float2> t(std::max<size_t>((size_t)P * half, 1));
    for (int i = 0; i < half; ++i) {
      const double f = std::pow((double)W.s.rot_base, -2.0 * i / W.s.rot_dims);
      for (int p = 0; p < P; ++p) t[(size_t)p * half + i] = make_float2((float)std::cos(p * f), (float)std::sin(p * f));
    }
    float2* d = nullptr;
    MI_TRY(alloc0(c, &d, t.size() * sizeof(float2), ws));
    S->rot.push_back({W.s.rot_base, W.s.rot_dims, d});
    MI_HIP(hipMemcpyAsync(d, t.data(), t.size() * sizeof(float2), hipMemcpyHostToDevice, c->stream));
    MI_HIP(hipStreamSynchronize(c->stream));
    W.rot = d;
  }
  if (S->cq_ld) {
    MI_TRY(alloc0(c, &S->cq, R * S->cq_ld * S->elem(), ws));
    MI_TRY(alloc0(c, &S->q2, R * S->q2_ld * 4, ws));
  }
  if (S->state_slots) {
    S->delta_chunks = delta_chunks(c);
    MI_TRY(alloc0(c, &S->low, 2 * R * S->low_ld * S->elem(), ws));
    MI_TRY(alloc0(c, &S->z, R * S->z_ld * 4, ws));
    MI_TRY(alloc0(c, &S->delta_records, (size_t)S->delta_chunks * S->chunk_floats * 4, ws));
  }
  return MI_OK;
}

// recurrent state, position table and the workspace only post-norm blocks have
static int post_norm_alloc(mi_ctx* c) {
  Stack* S = c->stack;
  const size_t R = (size_t)c->max_rows;
  size_t* ws = &c->workspace_bytes;
  for (const StackRun& r : S->runs) {
    float* p = nullptr;
    if (const size_t n = state_floats(c, S->layers[r.layer])) MI_TRY(alloc0(c, &p, n * 4, &c->kv_bytes));
    S->state_at.push_back(p);
  }
  if (S->cfg.pos_base > 0.f) MI_TRY(stack_position_turns(S->D, S->cfg.pos_base, &S->turns, c->stream));
  if (S->xc_ld) MI_TRY(alloc0(c, &S->xc, R * S->xc_ld * S->elem(), ws));
  if (S->low_ld) {
    MI_TRY(alloc0(c, &S->low, R * S->low_ld * S->elem(), ws));
    MI_TRY(alloc0(c, &S->xp, R * S->xp_ld * 4, ws));
    MI_TRY(alloc0(c, &S->dtp, R * S->dtp_ld * 4, ws));
  }
  if (S->yssm_ld) {
    S->ssd_chunks = ssd_chunks(c);
    MI_TRY(alloc0(c, &S->yssm, R * S->yssm_ld * 4, ws));
    MI_TRY(alloc0(c, &S->ssd_records, (size_t)S->ssd_chunks * S->ssd_chunk_floats * 4, ws));
  }
  return MI_OK;
}

int stack_position_turns(int width, float base, double** turns, hipStream_t s) {
  std::vector<double> t((size_t)(width + 1) / 2);
  for (size_t i = 0; i < t.size(); ++i) t[i] = std::pow((double)base, -2.0 * (double)i / width) / 6.283185307179586476925286766559;
  MI_HIP(hipMalloc(reinterpret_cast<void**>(turns), t.size() * 8));
  MI_HIP(hipMemcpyAsync(*turns, t.data(), t.size() * 8, hipMemcpyHostToDevice, s));
  MI_HIP(hipStreamSynchronize(s));
  return MI_OK;
}

int stack_alloc(mi_ctx* c) {
  Stack* S = c->stack;
  if (!S->missing.empty()) {
    std::string m;
    for (size_t i = 0; i < S->missing.size() && i < 4; ++i) m += (i ? ", " : "") + S->missing[i];
    set_error(std::to_string(S->missing.size()) + " weight tensors were never loaded: " + m + (S->missing.size() > 4 ? ", ..." : ""));
    return MI_ESTATE;
  }
  const mi_model_config& k = c->cfg;
  const size_t kv_bytes = stack_kv_bytes_per_block(c) * k.num_blocks;
  size_t fr = 0, tot = 0;
  MI_HIP(hipMemGetInfo(&fr, &tot));
  if (kv_bytes + stack_workspace_estimate(c) > fr) {
    set_error("KV pool of " + std::to_string(k.num_blocks) + " blocks (" + std::to_string(kv_bytes >> 20) + " MiB over " + std::to_string(S->runs.size()) +
              " layer runs) + workspace do not fit the " + std::to_string(fr >> 20) + " MiB free on the device: lower num_gpu_blocks_override / gpu_memory_utilization");
    return MI_ENOMEM;
  }
  // zero-filled: rows that were never written must hold finite values
  MI_TRY(alloc0(c, &c->kv_pool, std::max<size_t>(kv_bytes, 16), &c->kv_bytes));
  size_t at = 0;
  for (const StackRun& r : S->runs) {
    const StackLayer& W = S->layers[r.layer];
    const bool shared = S->sandwich() && W.s.kv_from >= 0;
    S->kv_at.push_back(shared ? S->kv_at[W.s.kv_from] : at);
    if (S->sandwich()) S->conv_at.push_back(at + (shared ? 0 : (size_t)k.num_blocks * k.block_size * W.lg.cp));
    at += kv_run_elems_per_block(c, W) * k.num_blocks;
  }
  if (S->one_norm()) MI_TRY(one_norm_alloc(c));
  if (S->post_norm()) MI_TRY(post_norm_alloc(c));
  const size_t R = (size_t)c->max_rows;
  size_t* ws = &c->workspace_bytes;
  MI_TRY(alloc0(c, &c->resid[0], R * S->ld * 4, ws));
  MI_TRY(alloc0(c, &c->resid[1], R * S->ld * 4, ws));
  MI_TRY(alloc0(c, &S->n1, R * S->Kd * S->elem(), ws));
  if (!S->parallel()) {
    const size_t pairs = R * std::max(1, S->max_top);   // (a dense feed-forward: one "pair" per row)
    MI_TRY(alloc0(c, &S->y, pairs * S->ld * 4, ws));
    MI_TRY(alloc0(c, &S->hb, R * S->Kd * S->elem(), ws));
    if (S->act_ld) MI_TRY(alloc0(c, &S->act, pairs * S->act_ld * S->elem(), ws));
    MI_TRY(alloc0(c, &S->qa, std::max<size_t>(R * S->lat_cols * S->elem(), 16), ws));
    MI_TRY(alloc0(c, &S->lat, std::max<size_t>(R * S->lat_cols * S->elem(), 16), ws));
    if (S->kv_ldx) {
      S->kv_rows = kv_work_rows(c);
      S->kv_mb = ceil_div(k.max_model_len, kKvBlock) + 1;
      MI_TRY(alloc0(c, &S->kv_x, (size_t)S->kv_rows * S->kv_ldx * 2, ws));
      MI_TRY(alloc0(c, &S->kv_k, (size_t)S->kv_rows * S->kv_k_cols * 2, ws));
      MI_TRY(alloc0(c, &S->kv_v, (size_t)S->kv_rows * S->kv_v_cols * 2, ws));
      MI_TRY(alloc0(c, &S->kv_bt, (size_t)k.max_num_seqs * S->kv_mb * 4, ws));
    }
    if (S->max_top) {
      MI_TRY(alloc0(c, &S->pair_w, pairs * 4, ws));
      MI_TRY(alloc0(c, &S->pair_ids, pairs * 4, ws));
      MI_TRY(alloc0(c, &S->route_z, R * S->max_experts * 4, ws));
      MI_TRY(alloc0(c, &S->tickets, R * 4, ws));
      MI_TRY(alloc0(c, &S->plan, experts_plan_ints((int)pairs, S->max_experts) * 4, ws));
    }
  } else {
    MI_TRY(alloc0(c, &S->n2, R * S->Kd * S->elem(), ws));
  }
  MI_TRY(alloc0(c, &S->qkv_out, R * S->qkv_ld * 4, ws));
  MI_TRY(alloc0(c, &S->q, std::max<size_t>(R * S->q_cols * S->elem(), 16), ws));
  MI_TRY(alloc0(c, &S->cat, R * S->cat_ld * S->elem(), ws));
  if (S->cfg.loop_times > 0) {
    MI_TRY(alloc0(c, &S->x0, R * S->ld * 4, ws));
    MI_TRY(alloc0(c, &S->pair, R * 2 * S->Kd * S->elem(), ws));
  }
  if (c->V_l % 16) MI_TRY(alloc0(c, &S->logits_pad, (size_t)k.max_num_seqs * S->head.N * 4, ws));
  MI_TRY(alloc0(c, &S->attn_scratch, stack_scratch(c), ws));
  return MI_OK;
}

namespace {

// ---- sandwich blocks ---------------------------------------------------------------------------------------------------------
struct Batch { int rows; bool decode; int MB; const AttnSeg* segs; int nseg; };

// x += post-norm of src; pre-norm and convolution -> S->n1.  cur: which residual buffer holds x
int sandwich_norm(mi_ctx* c, int& cur, const Batch& b, RowSource& src, const float* w_post, const float* w_pre, const float* conv_w, size_t conv_at) {
  Stack* S = c->stack;
  if (!runs_other(c)) { if (src.any()) cur ^= 1; src = RowSource(); return MI_OK; }
  Scope sc(c, MI_K_OTHER);
  ConvState cs;
  cs.w = conv_w;
  cs.taps = S->cfg.conv_taps;
  cs.keep = S->conv_keep;
  cs.ring = reinterpret_cast<unsigned char*>(c->kv_pool) + conv_at * S->elem();
  cs.block_size = c->cfg.block_size;
  cs.MB = b.MB;
  cs.bt = c->d_bt; cs.pos = c->d_pos; cs.slots = c->d_slots;
  const bool fused = b.decode || !w_pre;
  MI_TRY(launch_sandwich_rows(c->resid[cur], c->resid[cur ^ 1], src, w_post, w_pre, b.rows, S->D, S->ld, S->cfg.norm_groups, S->cfg.norm_eps,
                              fused && w_pre ? &cs : nullptr, fused ? S->n1 : S->hb, S->Kd, S->f32, c->stream));
  if (src.any()) cur ^= 1;
  src = RowSource();
  if (fused) return MI_OK;
  return launch_conv_rows(S->hb, cs, reinterpret_cast<const AttnSeg*>(c->d_segs), b.segs, b.nseg, S->D, S->ld, S->n1, S->Kd, S->f32, c->stream);
}

// any sizes, bf16 or fp32
int latent_attention_plain(mi_ctx* c, const StackLayer& W, const void* pool, const Batch& b) {
  Stack* S = c->stack;
  const LatentGeom& g = W.lg;
  Scope sc(c, b.decode ? MI_K_ATTN_DECODE : MI_K_ATTN_PREFILL);
  MI_TRY(launch_head_linear(W.w_uk, g.H, g.cp, g.dkp, S->q, b.rows, S->qa, g.H * g.cp, g.cp, g.cp, S->f32, c->stream));
  MI_TRY(launch_attn_plain(W.latent, S->qa, pool, pool, c->cfg.block_size, c->d_bt, b.MB, c->d_pos,
                           b.decode ? nullptr : reinterpret_cast<const AttnSeg*>(c->d_segs), b.nseg, b.rows, S->lat, g.H * g.rp, S->f32, c->stream));
  return launch_head_linear(W.w_uv, g.H, g.dvp, g.rp, S->lat, b.rows, S->cat, S->cat_ld, g.dv, g.dv, S->f32, c->stream);
}

// Rows of short portions (and token generation) stay in the latent space; longer ones get the keys and values in their sight
// written out per head, which costs a matrix product over those tokens and then a quarter of the attention arithmetic or less.
constexpr int kLatentRowsBelow = 64;
int latent_attention(mi_ctx* c, const StackLayer& W, const uint16_t* pool, const Batch& b, const OutGate& gate = OutGate()) {
  Stack* S = c->stack;
  const mi_model_config& k = c->cfg;
  const LatentGeom& g = W.lg;
  hipStream_t s = c->stream;
  const uint16_t* q = reinterpret_cast<const uint16_t*>(S->q);
  uint16_t *qa = reinterpret_cast<uint16_t*>(S->qa), *out = reinterpret_cast<uint16_t*>(S->cat);
  const AttnSeg* segs_dev = reinterpret_cast<const AttnSeg*>(c->d_segs);
  LatentRows lr;
  lr.rows = b.rows;
  if (!b.decode) {
    lr = LatentRows{segs_dev, b.nseg, kLatentRowsBelow, 0};
    for (int i = 0; i < b.nseg; ++i) lr.rows += b.segs[i].n < kLatentRowsBelow ? b.segs[i].n : 0;
  }
  const int cls = b.decode ? MI_K_ATTN_DECODE : MI_K_ATTN_PREFILL;
  if (!c->runs(cls)) return MI_OK;
  if (lr.rows > 0) {
    Scope sc(c, cls);
    if (!b.decode || !latent_token_supported(g))   // (token generation: done with the scatter)
      MI_TRY(launch_head_linear_rows(W.w_uk, g.H, g.cp, g.dkp, q, lr, qa, g.H * g.cp, g.cp, g.cp, s));
    MI_TRY(launch_latent_attn_rows(g, W.s.scale, W.s.window, qa, pool, k.block_size, c->d_bt, b.MB, c->d_pos, lr, k.max_model_len, W.w_uv,
                                   reinterpret_cast<uint16_t*>(S->lat), out, S->cat_ld, S->attn_scratch, s, gate));
  }
  const AttnSpec a{W.kvg, W.s.scale, W.s.window, nullptr, 0, 0};
  uint16_t *kk = reinterpret_cast<uint16_t*>(S->kv_k), *vv = reinterpret_cast<uint16_t*>(S->kv_v);
  for (int i = 0, j; i < b.nseg; i = j) {      // as many segments at a time as the written-out keys and values have room for
    int rows = 0;
    for (j = i; j < b.nseg; ++j) {
      const int n = b.segs[j].n < kLatentRowsBelow ? 0 : latent_kv_rows(b.segs[j], W.s.window);
      if (j > i && rows + n > S->kv_rows) break;
      rows += n;
    }
    if (rows == 0) continue;
    MI_CHECK(rows <= S->kv_rows, "latent attention: a sequence longer than the workspace");
    {
      Scope sc(c, MI_K_OTHER);
      MI_TRY(launch_latent_gather(g, W.s.window, pool, k.block_size, c->d_bt, b.MB, segs_dev + i, j - i, kLatentRowsBelow, rows,
                                  reinterpret_cast<uint16_t*>(S->kv_x), W.ukv.K, S->kv_bt, S->kv_mb, s));
    }
    {
      Scope sc(c, MI_K_GEMM);
      EpiArgs e{};
      e.scale = W.ukv.L.scale;
      e.q_dim = g.H * g.dkp; e.hd = g.dkp; e.kv_dim = g.dvp; e.nkv = g.H; e.block_size = kKvBlock;
      e.kpool = kk; e.vpool = vv;
      MI_TRY(launch_gemm(W.ukv.L.view(), rows, reinterpret_cast<const uint16_t*>(S->kv_x), W.ukv.K, EPI_HEADS_KV, e, s, c->splitk_ws, c->splitk_ws_bytes));
    }
    Scope sc(c, cls);
    MI_TRY(launch_attn_window_prefill(a, q, kk, vv, kKvBlock, S->kv_bt, S->kv_mb, segs_dev + i, b.segs + i, j - i, out, S->cat_ld, s, kLatentRowsBelow));
  }
  return MI_OK;
}

int latent_mixer(mi_ctx* c, const StackLayer& W, size_t kv_at, const Batch& b, RowSource& out) {
  Stack* S = c->stack;
  const mi_model_config& k = c->cfg;
  const LatentGeom& g = W.lg;
  hipStream_t s = c->stream;
  EpiArgs e{};
  e.out_f32 = S->qkv_out; e.ld_out = W.qkv.N;
  SlabSum slabs;       // (many rows: a K-split's sum is left to the scatter)
  MI_TRY(apply(c, W.qkv, b.rows, S->n1, S->Kd, EPI_F32, e, b.rows >= 384 ? &slabs : nullptr));
  unsigned char* pool = reinterpret_cast<unsigned char*>(c->kv_pool) + kv_at * S->elem();
  const LatentRowsIn in{S->qkv_out, S->qkv_out + g.H * g.dk, W.qkv.N, W.qkv.N};
  if (b.decode && W.fast() && latent_token_supported(g)) {
    if (runs_other(c)) {
      Scope sc(c, MI_K_OTHER);
      MI_TRY(launch_latent_token(in, b.rows, g, Rotation(), W.w_uk, W.c_norm, S->cfg.norm_eps, c->d_slots, reinterpret_cast<uint16_t*>(S->qa),
                                 reinterpret_cast<uint16_t*>(pool), s));
    }
  } else if (runs_other(c)) {
    Scope sc(c, MI_K_OTHER);
    MI_TRY(launch_latent_scatter(in, b.rows, g, Rotation(), W.c_norm, S->cfg.norm_eps, c->d_slots, k.block_size, S->q, pool, S->f32, s, &slabs));
  }
  MI_TRY(W.fast() ? latent_attention(c, W, reinterpret_cast<const uint16_t*>(pool), b) : latent_attention_plain(c, W, pool, b));
  EpiArgs o{};
  o.out_f32 = S->y; o.ld_out = S->ld;
  out.y = S->y; out.ld = S->ld;
  return apply(c, W.out, b.rows, S->cat, S->cat_ld, EPI_F32, o, b.rows >= 384 ? &out.slabs : nullptr);
}

int gated_ff(mi_ctx* c, const StackLayer& W, int rows, RowSource& out) {
  Stack* S = c->stack;
  EpiArgs e{};
  e.act_out = reinterpret_cast<uint16_t*>(S->act); e.ld_act = S->act_ld;
  e.glu_limit = W.s.ff_limit; e.glu_alpha = W.s.ff_alpha;
  MI_TRY(apply(c, W.up, rows, S->n1, S->Kd, EPI_GLU_CLIP, e));
  EpiArgs o{};
  o.out_f32 = S->y; o.ld_out = S->ld;
  out.y = S->y; out.ld = S->ld;
  return apply(c, W.down, rows, S->act, S->act_ld, EPI_F32, o, rows >= 384 ? &out.slabs : nullptr);
}

// few rows stream the weights of the experts they chose; many are grouped by expert
constexpr int kExpertStreamRows = 32;
int expert_ff(mi_ctx* c, const StackLayer& W, int rows, RowSource& out) {
  Stack* S = c->stack;
  const mi_layer_spec& p = W.s;
  const int pairs = rows * p.experts_top;
  const bool grouped = rows > kExpertStreamRows && !S->f32;
  hipStream_t s = c->stream;
  const ExpertPlan plan = experts_plan(S->plan, pairs, p.experts);
  out.ld = S->ld;
  out.pair_w = S->pair_w; out.top = p.experts_top;
  if (grouped) {
    {
      Scope sc(c, MI_K_GEMM);
      EpiArgs e{};
      e.scale = W.router_t.L.scale; e.bias = W.rule().sigmoid ? nullptr : W.router_b;
      e.out_f32 = S->route_z; e.ld_out = W.router_t.N;
      MI_TRY(launch_gemm(W.router_t.L.view(), rows, reinterpret_cast<const uint16_t*>(S->n1), S->Kd, EPI_F32, e, s, c->splitk_ws, c->splitk_ws_bytes));
    }
    if (runs_other(c)) {
      Scope sc(c, MI_K_OTHER);
      MI_TRY(launch_route_pick(S->route_z, W.router_t.N, rows, W.rule(), p.experts, p.experts_top, S->pair_ids, S->pair_w, s));
      MI_TRY(launch_experts_sort(plan, S->pair_ids, pairs, p.experts, s));
    }
    Scope sc(c, MI_K_GEMM);
    uint16_t *act = reinterpret_cast<uint16_t*>(S->act), *y = reinterpret_cast<uint16_t*>(S->y);
    MI_TRY(launch_experts_gemm(W.expert_up(), plan, pairs, reinterpret_cast<const uint16_t*>(S->n1), S->Kd, p.experts_top, W.ff_act(), act, S->act_ld, s));
    MI_TRY(launch_experts_gemm(W.expert_dn(), plan, pairs, act, S->act_ld, 1, EXPERT_LINEAR, y, S->ld, s));
    out.y16 = y;
    return MI_OK;
  }
  if (runs_other(c)) {
    Scope sc(c, MI_K_OTHER);
    MI_TRY(launch_route(S->n1, S->Kd, rows, W.router, W.rule(), p.experts, S->Kd, p.experts_top, S->pair_ids, S->pair_w, S->f32, s,
                        S->f32 ? nullptr : S->route_z, S->f32 ? nullptr : S->tickets));
  }
  const int cls = S->f32 ? MI_K_GEMM : MI_K_GEMV;
  if (c->runs(cls)) {
    Scope sc(c, cls);
    MI_TRY(launch_experts_linear(W.expert_up(), S->pair_ids, pairs, S->n1, S->Kd, p.experts_top, W.ff_act(), S->act, S->act_ld, S->f32, s));
  }
  if (c->runs(cls)) {
    Scope sc(c, cls);
    MI_TRY(launch_experts_linear(W.expert_dn(), S->pair_ids, pairs, S->act, S->act_ld, 1, EXPERT_LINEAR, S->y, S->ld, S->f32, s));
  }
  out.y = S->y;
  return MI_OK;
}

int sandwich_trunk(mi_ctx* c, const Batch& b, int& cur) {
  Stack* S = c->stack;
  RowSource src;
  const float* w_post = nullptr;
  auto keep = [&](size_t run) -> int {   // the stream behind layer run `run` is complete once its last sublayer is added
    if (S->residuals)
      MI_HIP(hipMemcpyAsync(S->residuals + run * c->max_rows * S->ld, c->resid[cur], (size_t)b.rows * S->ld * 4, hipMemcpyDeviceToDevice, c->stream));
    return MI_OK;
  };
  for (size_t i = 0; i < S->runs.size(); ++i) {
    const StackLayer& W = S->layers[S->runs[i].layer];
    MI_TRY(sandwich_norm(c, cur, b, src, w_post, W.n1.w, W.conv1, S->conv_at[i]));
    if (i > 0) MI_TRY(keep(i - 1));
    MI_TRY(latent_mixer(c, W, S->kv_at[i], b, src));
    w_post = W.n1b.w;
    if (W.s.ff_kind == MI_FF_NONE) continue;
    MI_TRY(sandwich_norm(c, cur, b, src, w_post, W.n2.w, W.conv2, S->conv_at[i] + (size_t)c->cfg.num_blocks * S->conv_keep * S->Kd));
    MI_TRY(W.s.ff_kind == MI_FF_MOE ? expert_ff(c, W, b.rows, src) : gated_ff(c, W, b.rows, src));
    w_post = W.n2b.w;
  }
  MI_TRY(sandwich_norm(c, cur, b, src, w_post, nullptr, nullptr, 0));
  return keep(S->runs.size() - 1);
}

// ---- one-norm blocks -----------------------------------------------------------------------------------------------------------
int one_norm_latent(mi_ctx* c, const StackLayer& W, size_t kv_at, const Batch& b) {
  Stack* S = c->stack;
  const LatentGeom& g = W.lg;
  hipStream_t s = c->stream;
  EpiArgs e{};
  e.out_f32 = S->qkv_out; e.ld_out = W.qkv.N;
  MI_TRY(apply(c, W.qkv, b.rows, S->n1, S->Kd, EPI_F32, e));
  LatentRowsIn in{S->qkv_out + W.col_q, S->qkv_out, W.qkv.N, W.qkv.N};
  if (W.s.q_rank) {
    if (runs_other(c)) {
      Scope sc(c, MI_K_OTHER);
      MI_TRY(launch_columns(S->qkv_out, W.qkv.N, {W.col_q, W.s.q_rank, W.q_norm, S->cq}, {}, S->cfg.norm_eps, b.rows, W.uq.K, S->f32, s));
    }
    EpiArgs u{};
    u.out_f32 = S->q2; u.ld_out = W.uq.N;
    MI_TRY(apply(c, W.uq, b.rows, S->cq, W.uq.K, EPI_F32, u));
    in.q = S->q2; in.ldq = W.uq.N;
  }
  const Rotation rot{W.rot, c->d_pos};
  unsigned char* pool = reinterpret_cast<unsigned char*>(c->kv_pool) + kv_at * S->elem();
  if (runs_other(c)) {
    Scope sc(c, MI_K_OTHER);
    if (b.decode && W.fast() && latent_token_supported(g))
      MI_TRY(launch_latent_token(in, b.rows, g, rot, W.w_uk, W.c_norm, S->cfg.norm_eps, c->d_slots, reinterpret_cast<uint16_t*>(S->qa),
                                 reinterpret_cast<uint16_t*>(pool), s));
    else
      MI_TRY(launch_latent_scatter(in, b.rows, g, rot, W.c_norm, S->cfg.norm_eps, c->d_slots, c->cfg.block_size, S->q, pool, S->f32, s));
  }
  // (token generation: the gate goes onto the heads' outputs before they are rounded)
  const OutGate gate{b.decode && W.fast() && W.s.out_gate != MI_GATE_NONE ? S->qkv_out + W.col_g : nullptr, W.qkv.N, W.s.out_gate == MI_GATE_ELEMENT};
  MI_TRY(W.fast() ? latent_attention(c, W, reinterpret_cast<const uint16_t*>(pool), b, gate) : latent_attention_plain(c, W, pool, b));
  if (W.s.out_gate == MI_GATE_NONE || gate.z || !runs_other(c)) return MI_OK;
  Scope sc(c, MI_K_OTHER);
  return launch_gate_rows(S->cat, S->cat_ld, b.rows, g.H, g.dv, S->qkv_out + W.col_g, W.qkv.N, W.s.out_gate == MI_GATE_ELEMENT, S->f32, s);
}

int one_norm_delta(mi_ctx* c, const StackLayer& W, float* state, const Batch& b) {
  Stack* S = c->stack;
  const DeltaGeom& g = W.dg;
  hipStream_t s = c->stream;
  EpiArgs e{};
  e.out_f32 = S->qkv_out; e.ld_out = W.qkv.N;
  MI_TRY(apply(c, W.qkv, b.rows, S->n1, S->Kd, EPI_F32, e));
  void* low2 = reinterpret_cast<unsigned char*>(S->low) + (size_t)c->max_rows * S->low_ld * S->elem();
  if (runs_other(c)) {
    Scope sc(c, MI_K_OTHER);
    MI_TRY(launch_columns(S->qkv_out, W.qkv.N, {W.col_a, W.s.decay_rank, nullptr, S->low}, {W.col_g, W.s.gate_rank, nullptr, low2}, 0.f, b.rows, S->low_ld,
                          S->f32, s));
  }
  const int ldz = W.a2.N + W.g2.N;
  EpiArgs z{};
  z.out_f32 = S->z; z.ld_out = ldz;
  MI_TRY(apply(c, W.a2, b.rows, S->low, S->low_ld, EPI_F32, z));
  z.out_f32 = S->z + W.a2.N;
  MI_TRY(apply(c, W.g2, b.rows, low2, S->low_ld, EPI_F32, z));
  DeltaIn in;
  in.proj = S->qkv_out; in.ldp = W.qkv.N; in.beta = W.col_b;
  in.z = S->z; in.ldz = ldz; in.gate = W.a2.N;
  in.conv = W.conv; in.a_log = W.a_log; in.dt = W.dt; in.norm = W.o_norm;
  in.eps = S->cfg.norm_eps;
  in.state = state; in.ring = state + (size_t)S->state_slots * g.state_floats();
  in.slots = c->d_state; in.pos = c->d_pos;
  const int cls = b.decode ? MI_K_ATTN_DECODE : MI_K_ATTN_PREFILL;
  if (!c->runs(cls)) return MI_OK;
  Scope sc(c, cls);
  if (b.decode) return launch_delta_token(g, in, b.rows, nullptr, S->cat, S->cat_ld, S->f32, s);
  int ones = 0;
  for (int i = 0; i < b.nseg; ++i) ones += b.segs[i].n == 1;
  const AttnSeg* segs = reinterpret_cast<const AttnSeg*>(c->d_segs);
  if (ones) MI_TRY(launch_delta_token(g, in, b.nseg, segs, S->cat, S->cat_ld, S->f32, s));
  if (ones < b.nseg) MI_TRY(launch_delta_prompt(g, in, segs, b.segs, b.nseg, S->delta_records, S->delta_chunks, S->cat, S->cat_ld, S->f32, s));
  return MI_OK;
}

// The feed-forward runs ahead of the mixer: the mixer's output projection may leave a K-split's sum in the workspace that the
// router's product uses too.
int one_norm_trunk(mi_ctx* c, const Batch& b, int& cur) {
  Stack* S = c->stack;
  RowSource src;
  auto keep = [&](size_t run) -> int {
    if (S->residuals)
      MI_HIP(hipMemcpyAsync(S->residuals + run * c->max_rows * S->ld, c->resid[cur], (size_t)b.rows * S->ld * 4, hipMemcpyDeviceToDevice, c->stream));
    return MI_OK;
  };
  auto row = [&](const float* w_norm) -> int {
    const bool add = src.any();
    if (runs_other(c) && (add || w_norm)) {
      Scope sc(c, MI_K_OTHER);
      MI_TRY(launch_sandwich_rows(c->resid[cur], c->resid[cur ^ 1], src, nullptr, w_norm, b.rows, S->D, S->ld, 1, S->cfg.norm_eps, nullptr, S->n1, S->Kd, S->f32, c->stream));
    }
    if (add) cur ^= 1;
    src = RowSource();
    return MI_OK;
  };
  for (size_t i = 0; i < S->runs.size(); ++i) {
    const StackLayer& W = S->layers[S->runs[i].layer];
    MI_TRY(row(W.n1.w));
    if (i > 0) MI_TRY(keep(i - 1));
    if (W.s.ff_kind == MI_FF_MOE) MI_TRY(expert_ff(c, W, b.rows, src));
    MI_TRY(W.s.mixer_kind == MI_MIX_DELTA ? one_norm_delta(c, W, S->state_at[i], b) : one_norm_latent(c, W, S->kv_at[i], b));
    EpiArgs e{};
    e.out_f32 = c->resid[cur ^ 1]; e.resid_in = c->resid[cur]; e.ld_out = S->ld;
    MI_TRY(apply(c, W.out, b.rows, S->cat, S->cat_ld, EPI_RESID, e, b.rows >= 384 ? &src.slabs : nullptr));
    if (!src.slabs.slab) cur ^= 1;
  }
  MI_TRY(row(nullptr));
  return keep(S->runs.size() - 1);
}

// ---- post-norm blocks ----------------------------------------------------------------------------------------------------------
ShortConv short_conv(const mi_ctx* c, const StackLayer& W, float* state) {
  return ShortConv{W.conv, W.conv_b, W.s.conv_taps, W.conv_channels(), state + (size_t)c->stack->state_slots * W.ssm_state_floats(), c->d_state};
}
int post_norm_conv(mi_ctx* c, const StackLayer& W, float* state, const Batch& b, int col, int ldc) {
  Stack* S = c->stack;
  if (!runs_other(c)) return MI_OK;
  Scope sc(c, MI_K_OTHER);
  const ShortConv cv = short_conv(c, W, state);
  return launch_short_conv(S->qkv_out + col, W.qkv.N, cv, c->d_pos, reinterpret_cast<const AttnSeg*>(c->d_segs), b.segs, b.decode ? 0 : b.nseg, b.rows, S->xc, ldc,
                           S->f32, c->stream);
}

int post_norm_scan(mi_ctx* c, const StackLayer& W, float* state, const Batch& b) {
  Stack* S = c->stack;
  const ScanGeom& g = W.scan;
  hipStream_t s = c->stream;
  EpiArgs e{};
  e.out_f32 = S->qkv_out; e.ld_out = W.qkv.N;
  MI_TRY(apply(c, W.qkv, b.rows, S->n1, S->Kd, EPI_F32, e));
  MI_TRY(post_norm_conv(c, W, state, b, 0, W.low_in.K));
  EpiArgs x{};
  x.out_f32 = S->xp; x.ld_out = W.low_in.N;
  MI_TRY(apply(c, W.low_in, b.rows, S->xc, W.low_in.K, EPI_F32, x));
  ScanIn in;
  in.x = S->xc; in.ldx = W.low_in.K;
  in.low = S->xp; in.ldl = W.low_in.N; in.col_b = W.col_B; in.col_c = W.col_C;
  in.dt = S->dtp; in.ldt = W.dt_mat.N; in.w_dt = W.w_dt;
  in.dt_bias = W.dt; in.a2 = W.decay; in.d = W.ssm_d;
  in.z = S->qkv_out + W.col_z; in.ldz = W.qkv.N;
  in.state = state; in.slots = c->d_state; in.pos = c->d_pos;
  int ones = 0;
  for (int i = 0; i < b.nseg; ++i) ones += b.segs[i].n == 1;
  const bool prompts = !b.decode && ones < b.nseg;
  if (prompts) {
    if (runs_other(c)) {
      Scope sc(c, MI_K_OTHER);
      MI_TRY(launch_columns(S->xp, W.low_in.N, {0, g.rank, nullptr, S->low}, {}, 0.f, b.rows, W.dt_mat.K, S->f32, s));
    }
    EpiArgs z{};
    z.out_f32 = S->dtp; z.ld_out = W.dt_mat.N;
    MI_TRY(apply(c, W.dt_mat, b.rows, S->low, W.dt_mat.K, EPI_F32, z));
  }
  const int cls = b.decode ? MI_K_ATTN_DECODE : MI_K_ATTN_PREFILL;
  if (!c->runs(cls)) return MI_OK;
  Scope sc(c, cls);
  if (b.decode) return launch_scan_token(g, in, b.rows, nullptr, S->cat, S->cat_ld, S->f32, s);
  const AttnSeg* segs = reinterpret_cast<const AttnSeg*>(c->d_segs);
  if (ones) MI_TRY(launch_scan_token(g, in, b.nseg, segs, S->cat, S->cat_ld, S->f32, s));
  if (prompts) MI_TRY(launch_scan_prompt(g, in, segs, b.nseg, S->cat, S->cat_ld, S->f32, s));
  return MI_OK;
}

// the second mixer of x beside attention: columns attn_cols .. of the concatenated row
int post_norm_ssd(mi_ctx* c, const StackLayer& W, float* state, const Batch& b) {
  Stack* S = c->stack;
  const SsdGeom& g = W.ssd;
  hipStream_t s = c->stream;
  const int ldc = pad_to(g.channels(), 16), ldy = pad_to(g.inner(), 16);
  if (!b.decode) MI_TRY(post_norm_conv(c, W, state, b, W.col_x, ldc));
  SsdIn in;
  in.xbc = S->xc; in.ldx = ldc;
  in.dt = S->qkv_out + W.col_dt; in.ldt = W.qkv.N;
  in.dt_bias = W.dt; in.a_log = W.a_log; in.d = W.ssm_d;
  in.state = state; in.slots = c->d_state; in.pos = c->d_pos;
  const int cls = b.decode ? MI_K_ATTN_DECODE : MI_K_ATTN_PREFILL;
  if (c->runs(cls)) {
    Scope sc(c, cls);
    if (b.decode) {
      const ShortConv cv = short_conv(c, W, state);
      MI_TRY(launch_ssd_token(g, in, b.rows, nullptr, S->yssm, ldy, S->f32, s, &cv, S->qkv_out + W.col_x, W.qkv.N));
    } else {
      int ones = 0;
      for (int i = 0; i < b.nseg; ++i) ones += b.segs[i].n == 1;
      const AttnSeg* segs = reinterpret_cast<const AttnSeg*>(c->d_segs);
      if (ones) MI_TRY(launch_ssd_token(g, in, b.nseg, segs, S->yssm, ldy, S->f32, s));
      if (ones < b.nseg) MI_TRY(launch_ssd_prompt(g, in, segs, b.segs, b.nseg, S->ssd_records, S->ssd_chunks, S->yssm, ldy, S->f32, s));
    }
  }
  if (!runs_other(c)) return MI_OK;
  Scope sc(c, MI_K_OTHER);
  void* out = reinterpret_cast<unsigned char*>(S->cat) + (size_t)W.attn_cols * S->elem();
  return launch_gated_norm(S->yssm, ldy, S->qkv_out + W.col_z, W.qkv.N, W.o_norm, g.inner(), W.s.ssm_parts, S->cfg.norm_eps, b.rows, out, S->cat_ld, S->f32, s);
}

int post_norm_trunk(mi_ctx* c, const Batch& b, int& cur) {
  Stack* S = c->stack;
  RowSource src;
  const float* w_post = nullptr;
  auto keep = [&](size_t run) -> int {
    if (S->residuals)
      MI_HIP(hipMemcpyAsync(S->residuals + run * c->max_rows * S->ld, c->resid[cur], (size_t)b.rows * S->ld * 4, hipMemcpyDeviceToDevice, c->stream));
    return MI_OK;
  };
  // x += norm of the sublayer's output; x in the compute type -> S->n1
  auto row = [&]() -> int {
    if (runs_other(c)) {
      Scope sc(c, MI_K_OTHER);
      MI_TRY(launch_sandwich_rows(c->resid[cur], c->resid[cur ^ 1], src, w_post, nullptr, b.rows, S->D, S->ld, 1, S->cfg.norm_eps, nullptr, S->n1, S->Kd, S->f32,
                                  c->stream, true));
    }
    cur ^= 1;
    src = RowSource();
    return MI_OK;
  };
  // a sublayer's output rows -> src
  auto project = [&](const StackMat& m, const void* x, int ldx, const float* w) -> int {
    EpiArgs e{};
    e.out_f32 = S->y; e.ld_out = S->ld;
    src.y = S->y; src.ld = S->ld;
    w_post = w;
    return apply(c, m, b.rows, x, ldx, EPI_F32, e, b.rows >= 384 ? &src.slabs : nullptr);
  };
  for (size_t i = 0; i < S->runs.size(); ++i) {
    const StackLayer& W = S->layers[S->runs[i].layer];
    if (i > 0) {
      MI_TRY(row());
      MI_TRY(keep(i - 1));
    }
    if (W.has_scan()) {
      MI_TRY(post_norm_scan(c, W, S->state_at[i], b));
    } else {
      EpiArgs e{};
      e.out_f32 = S->qkv_out; e.ld_out = W.qkv.N;
      MI_TRY(apply(c, W.qkv, b.rows, S->n1, S->Kd, EPI_F32, e));
      const OutGate gate{W.s.out_gate ? S->qkv_out + W.col_g : nullptr, W.qkv.N, false, W.s.mix_mult};
      MI_TRY(attention(c, W, S->kv_at[i], W.qkv.N, b.rows, b.decode, b.MB, b.segs, b.nseg, gate));
      if (W.has_ssd()) MI_TRY(post_norm_ssd(c, W, S->state_at[i], b));
    }
    MI_TRY(project(W.out, S->cat, S->cat_ld, W.n1.w));
    if (W.s.ff_kind == MI_FF_NONE) continue;
    MI_TRY(row());
    EpiArgs u{};
    u.act_out = reinterpret_cast<uint16_t*>(S->act); u.ld_act = S->act_ld;
    MI_TRY(apply(c, W.up, b.rows, S->n1, S->Kd, EPI_RELU2, u));
    MI_TRY(project(W.down, S->act, S->act_ld, W.n2.w));
  }
  MI_TRY(row());
  return keep(S->runs.size() - 1);
}

}  // namespace

int stack_trunk(mi_ctx* c, int rows, bool decode, int MB, const AttnSeg* segs, int nseg) {
  Stack* S = c->stack;
  hipStream_t s = c->stream;
  S->pend = SlabSum();
  int cur = 0;
  if (runs_other(c)) {
    Scope sc(c, MI_K_OTHER);
    MI_TRY(launch_embed_pos(c->d_ids, c->d_pos, S->embed, S->pos, S->cfg.embed_scale, S->f32, rows, S->D, S->ld, c->resid[0], S->x0, s, S->turns,
                            S->post_norm() ? S->n1 : nullptr, S->Kd));
  }
  if (S->post_norm()) {
    MI_TRY(post_norm_trunk(c, Batch{rows, decode, MB, segs, nseg}, cur));
    c->tail_cur = cur;
    return MI_OK;
  }
  if (S->one_norm()) {
    MI_TRY(one_norm_trunk(c, Batch{rows, decode, MB, segs, nseg}, cur));
    c->tail_cur = cur;
    return MI_OK;
  }
  if (S->sandwich()) {
    MI_TRY(sandwich_trunk(c, Batch{rows, decode, MB, segs, nseg}, cur));
    c->tail_cur = cur;
    return MI_OK;
  }
  for (size_t i = 0; i < S->runs.size(); ++i) {
    const StackRun& run = S->runs[i];
    const StackLayer& W = S->layers[run.layer];
    if (run.pass_start) {
      MI_TRY(flush(c, cur));
      if (runs_other(c)) {
        Scope sc(c, MI_K_OTHER);
        MI_TRY(launch_pair_rows(c->resid[cur], S->x0, rows, S->D, S->ld, S->Kd, S->pair, S->f32, s));
      }
      EpiArgs e{};
      e.out_f32 = c->resid[cur]; e.ld_out = S->ld;
      MI_TRY(apply(c, S->loop_in, rows, S->pair, 2 * S->Kd, EPI_F32, e));
    }
    if (runs_other(c)) {
      NormOut a{W.n1.w, W.n1.b, S->n1}, b{};
      if (W.ff_cols) b = NormOut{W.n2.w, W.n2.b, S->n2};
      MI_TRY(norm_rows(c, cur, rows, a, b));
    }
    {
      EpiArgs e{};
      e.out_f32 = S->qkv_out; e.ld_out = S->qkv_ld;
      MI_TRY(apply(c, W.qkv, rows, S->n1, S->Kd, EPI_F32, e));
    }
    MI_TRY(attention(c, W, S->kv_at[i], S->qkv_ld, rows, decode, MB, segs, nseg));
    if (W.ff_cols) {
      EpiArgs e{};
      e.act_out = reinterpret_cast<uint16_t*>(reinterpret_cast<unsigned char*>(S->cat) + (size_t)W.attn_cols * S->elem());
      e.ld_act = S->cat_ld;
      MI_TRY(apply(c, W.up, rows, S->n2, S->Kd, EPI_RELU2, e));
    }
    {
      EpiArgs e{};
      e.out_f32 = c->resid[cur ^ 1]; e.resid_in = c->resid[cur]; e.ld_out = S->ld;
      // (many rows: the K-split sum is left to the next norm, which passes over the row anyway)
      MI_TRY(apply(c, W.out, rows, S->cat, S->cat_ld, EPI_RESID, e, rows >= 384 && !S->residuals ? &S->pend : nullptr));
      cur ^= 1;
    }
    if (S->residuals)
      MI_HIP(hipMemcpyAsync(S->residuals + i * c->max_rows * S->ld, c->resid[cur], (size_t)rows * S->ld * 4, hipMemcpyDeviceToDevice, s));
  }
  MI_TRY(flush(c, cur));
  c->tail_cur = cur;
  return MI_OK;
}

int stack_head(mi_ctx* c, const float* resid, int nrows) {
  Stack* S = c->stack;
  if (runs_other(c)) {
    Scope sc(c, MI_K_OTHER);
    if (S->cfg.norm_groups > 0)
      MI_TRY(launch_sandwich_rows(resid, nullptr, RowSource(), nullptr, S->final_norm.w, nrows, S->D, S->ld, S->cfg.norm_groups, S->cfg.norm_eps, nullptr, S->n1, S->Kd, S->f32, c->stream));
    else
      MI_TRY(launch_layernorm_rows(resid, nullptr, nrows, S->D, S->ld, S->cfg.norm_eps, NormOut{S->final_norm.w, S->final_norm.b, S->n1}, NormOut{}, S->Kd, S->f32, c->stream));
  }
  const bool direct = c->V_l % 16 == 0;
  EpiArgs e{};
  e.out_f32 = direct ? c->logits : S->logits_pad;
  e.ld_out = S->head.N;
  e.softcap = S->cfg.logit_softcap;
  MI_TRY(apply(c, S->head, nrows, S->n1, S->Kd, e.softcap > 0.f ? EPI_SOFTCAP : EPI_F32, e));
  if (!direct) {
    Scope sc(c, MI_K_OTHER);
    MI_TRY(launch_pack_rows(S->logits_pad, S->head.N, nrows, c->V_l, c->logits, c->stream));
  }
  return MI_OK;
}

}  // namespace mi
