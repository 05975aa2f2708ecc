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

int attention(mi_ctx* c, const StackLayer& W, size_t kv_at, int rows, bool decode, int MB, const AttnSeg* segs, int nseg) {
  Stack* S = c->stack;
  const mi_model_config& k = c->cfg;
  unsigned char* base = reinterpret_cast<unsigned char*>(c->kv_pool);
  const size_t kn = (size_t)k.num_blocks * W.g.G * k.block_size * W.g.dkp;
  unsigned char *kp = base + kv_at * S->elem(), *vp = base + (kv_at + kn) * S->elem();
  if (runs_other(c)) {
    Scope sc(c, MI_K_OTHER);
    MI_TRY(launch_qkv_scatter(S->qkv_out, S->qkv_ld, rows, W.g, W.s.qk_unit_norm != 0, S->cfg.norm_eps, c->d_slots, k.block_size, S->q, kp, vp, S->f32, c->stream));
  }
  const int ldo = S->cat_ld;
  if (S->f32 || !attn_window_supported(W.g)) {
    Scope sc(c, decode ? MI_K_ATTN_DECODE : MI_K_ATTN_PREFILL);
    return launch_attn_plain(W.attn, S->q, kp, vp, k.block_size, c->d_bt, MB, c->d_pos, decode ? nullptr : reinterpret_cast<const AttnSeg*>(c->d_segs),
                             nseg, rows, S->cat, ldo, S->f32, c->stream);
  }
  const uint16_t* q = reinterpret_cast<const uint16_t*>(S->q);
  const uint16_t *kb = reinterpret_cast<const uint16_t*>(kp), *vb = reinterpret_cast<const uint16_t*>(vp);
  uint16_t* out = reinterpret_cast<uint16_t*>(S->cat);
  const size_t qrow = (size_t)W.g.H * W.g.dkp;
  if (decode) {
    if (!c->runs(MI_K_ATTN_DECODE)) return MI_OK;
    Scope sc(c, MI_K_ATTN_DECODE);
    return launch_attn_window_decode(W.attn, q, kb, vb, k.block_size, c->d_bt, MB, c->d_ctx, rows, k.max_model_len, out, ldo, S->attn_scratch, c->stream);
  }
  Scope sc(c, MI_K_ATTN_PREFILL);
  MI_TRY(launch_attn_window_prefill(W.attn, q, kb, vb, k.block_size, c->d_bt, MB, reinterpret_cast<const AttnSeg*>(c->d_segs), segs, nseg, out, ldo, c->stream));
  for (int i = 0; i < nseg;) {   // runs of requests with one token: one token-generation launch each
    int j = i;
    while (j < nseg && segs[j].n == 1) ++j;
    if (j > i)
      MI_TRY(launch_attn_window_decode(W.attn, q + segs[i].row0 * qrow, kb, vb, k.block_size, c->d_bt + (size_t)i * MB, MB, c->d_seg_ctx + i, j - i,
                                       k.max_model_len, out + (size_t)segs[i].row0 * ldo, ldo, S->attn_scratch, c->stream));
    i = j > i ? j : i + 1;
  }
  return MI_OK;
}

}  // namespace

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
  MI_TRY(alloc0(c, &S->pos, (size_t)cfg.max_positions * S->D * S->elem(), wb));
  want("embed"); want("pos");
  if (loop) {
    MI_TRY(alloc_mat(c, S->loop_in, S->D, 2 * S->Kd, 1.f));
    want("loop.in");
  }
  S->layers.resize(cfg.num_layers);
  for (int i = 0; i < cfg.num_layers; ++i) {
    StackLayer& W = S->layers[i];
    W.s = cfg.layers[i];
    const mi_layer_spec& s = W.s;
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
    S->qkv_ld = std::max(S->qkv_ld, W.qkv.N);
    S->q_cols = std::max(S->q_cols, s.num_heads * W.g.dkp);
    S->cat_ld = std::max(S->cat_ld, W.out.K);
    const std::string p = "l" + std::to_string(i) + ".";
    for (const char* n : {"norm1", "norm1.b", "mix.q", "mix.k", "mix.v", "mix.o"}) want(p + n);
    if (W.ff_cols)
      for (const char* n : {"norm2", "norm2.b", "mlp.up", "mlp.down"}) want(p + n);
  }
  MI_TRY(alloc_norm(c, S->final_norm));
  MI_TRY(alloc_mat(c, S->head, cfg.vocab_size, S->D, 1.f));
  want("final.norm"); want("final.norm.b"); want("head");
  MI_HIP(hipStreamSynchronize(c->stream));
  return MI_OK;
}

void stack_destroy(mi_ctx* c) {
  Stack* S = c->stack;
  for (StackLayer& W : S->layers) {
    free_mat(W.qkv); free_mat(W.up); free_mat(W.out);
    free_norm(W.n1); free_norm(W.n2);
    hipFree(W.slopes);
  }
  free_mat(S->loop_in); free_mat(S->head);
  free_norm(S->final_norm);
  void* ptrs[] = {S->embed, S->pos, S->x0, S->qkv_out, S->logits_pad, S->n1, S->n2, S->q, S->cat, S->pair, S->attn_scratch, S->residuals};
  for (void* p : ptrs) hipFree(p);
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
  if (name == "pos") return table(S->pos, k.max_positions);
  if (name == "head") return place(S->head, k.vocab_size, S->D);
  if (name == "final.norm") return vec(S->final_norm.w);
  if (name == "final.norm.b") return vec(S->final_norm.b);
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
    const int qn = p.num_heads * p.qk_dim, kn = p.num_kv_heads * p.qk_dim;
    if (t == "norm1") return vec(W.n1.w);
    if (t == "norm1.b") return vec(W.n1.b);
    if (t == "mix.q") return place(W.qkv, qn, S->D);
    if (t == "mix.k") return place(W.qkv, kn, S->D, qn);
    if (t == "mix.v") return place(W.qkv, p.num_kv_heads * p.v_dim, S->D, qn + kn);
    if (t == "mix.o") return place(W.out, S->D, p.num_heads * p.v_dim);
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
    bool is_norm = n.find("norm") != std::string::npos;
    if (n == "embed" || n == "head") { rows = k.vocab_size; cols = S->D; if (n == "embed") sd = 1.f; }
    else if (n == "pos") { rows = k.max_positions; cols = S->D; sd = 0.1f; }
    else if (n == "loop.in") cols = 2 * S->D;
    else if (!is_norm) {
      const int l = atoi(n.c_str() + 1);
      const mi_layer_spec& p = S->layers[l].s;
      const std::string t = n.substr(n.find('.') + 1);
      cols = S->D;
      if (t == "mix.q") rows = p.num_heads * p.qk_dim;
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
    if (is_norm) rc = launch_fill_f32(buf, elems, n.size() > 2 && n.compare(n.size() - 2, 2, ".b") == 0 ? 0.f : 1.f, c->stream);
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
  auto norm = [&](StackNorm& n) { out.push_back({n.w, nb}); out.push_back({n.b, nb}); };
  out.push_back({S->embed, (size_t)S->cfg.vocab_size * S->D * S->elem()});
  out.push_back({S->pos, (size_t)S->cfg.max_positions * S->D * S->elem()});
  if (S->cfg.loop_times > 0) mat(S->loop_in);
  for (StackLayer& W : S->layers) {
    mat(W.qkv); mat(W.out); norm(W.n1);
    if (W.ff_cols) { mat(W.up); norm(W.n2); }
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
  const int32_t g[7] = {k.num_layers, k.width, k.vocab_size, k.max_positions, k.loop_times > 0, k.compute_dtype, 0};
  mix(g, sizeof g);
  for (const StackLayer& W : S->layers) mix(&W.s, sizeof W.s);
  return (int)(h & 0x7fffffff);
}

static size_t kv_run_elems_per_block(const mi_ctx* c, const StackLayer& W) { return (size_t)W.g.G * c->cfg.block_size * (W.g.dkp + W.g.dvp); }
size_t stack_kv_bytes_per_block(const mi_ctx* c) {
  size_t e = 0;
  for (const StackRun& r : c->stack->runs) e += kv_run_elems_per_block(c, c->stack->layers[r.layer]);
  return e * c->stack->elem();
}

static size_t stack_scratch(const mi_ctx* c) {
  size_t b = 16;
  for (const StackLayer& W : c->stack->layers) b = std::max(b, attn_window_scratch_bytes(c->cfg.max_num_seqs, W.g));
  return b;
}

size_t stack_workspace_estimate(const mi_ctx* c) {
  const Stack* S = c->stack;
  const size_t R = (size_t)c->max_rows;
  size_t b = 3 * R * S->ld * 4 + R * S->qkv_ld * 4 + R * (4 * (size_t)S->Kd + S->q_cols + S->cat_ld) * S->elem();
  b += (size_t)64 << 20;
  b += 2 * (size_t)c->cfg.max_num_seqs * pad_to(c->V_l, 16) * 4;
  return b + stack_scratch(c) + ((size_t)8 << 20);
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
  MI_TRY(alloc0(c, &c->kv_pool, kv_bytes, &c->kv_bytes));
  size_t at = 0;
  for (const StackRun& r : S->runs) {
    S->kv_at.push_back(at);
    at += kv_run_elems_per_block(c, S->layers[r.layer]) * k.num_blocks;
  }
  const size_t R = (size_t)c->max_rows;
  size_t* ws = &c->workspace_bytes;
  MI_TRY(alloc0(c, &c->resid[0], R * S->ld * 4, ws));
  MI_TRY(alloc0(c, &c->resid[1], R * S->ld * 4, ws));
  MI_TRY(alloc0(c, &S->n1, R * S->Kd * S->elem(), ws));
  MI_TRY(alloc0(c, &S->n2, R * S->Kd * S->elem(), ws));
  MI_TRY(alloc0(c, &S->qkv_out, R * S->qkv_ld * 4, ws));
  MI_TRY(alloc0(c, &S->q, R * S->q_cols * S->elem(), ws));
  MI_TRY(alloc0(c, &S->cat, R * S->cat_ld * S->elem(), ws));
  if (S->cfg.loop_times > 0) {
    MI_TRY(alloc0(c, &S->x0, R * S->ld * 4, ws));
    MI_TRY(alloc0(c, &S->pair, R * 2 * S->Kd * S->elem(), ws));
  }
  if (c->V_l % 16) MI_TRY(alloc0(c, &S->logits_pad, (size_t)k.max_num_seqs * S->head.N * 4, ws));
  MI_TRY(alloc0(c, &S->attn_scratch, stack_scratch(c), ws));
  return MI_OK;
}

int stack_trunk(mi_ctx* c, int rows, bool decode, int MB, const AttnSeg* segs, int nseg) {
  Stack* S = c->stack;
  hipStream_t s = c->stream;
  S->pend = SlabSum();
  int cur = 0;
  if (runs_other(c)) {
    Scope sc(c, MI_K_OTHER);
    MI_TRY(launch_embed_pos(c->d_ids, c->d_pos, S->embed, S->pos, S->f32, rows, S->D, S->ld, c->resid[0], S->x0, s));
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
    MI_TRY(attention(c, W, S->kv_at[i], rows, decode, MB, segs, nseg));
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
    MI_TRY(launch_layernorm_rows(resid, nullptr, nrows, S->D, S->ld, S->cfg.norm_eps, NormOut{S->final_norm.w, S->final_norm.b, S->n1}, NormOut{}, S->Kd, S->f32, c->stream));
  }
  const bool direct = c->V_l % 16 == 0;
  EpiArgs e{};
  e.out_f32 = direct ? c->logits : S->logits_pad;
  e.ld_out = S->head.N;
  MI_TRY(apply(c, S->head, nrows, S->n1, S->Kd, EPI_F32, e));
  if (!direct) {
    Scope sc(c, MI_K_OTHER);
    MI_TRY(launch_pack_rows(S->logits_pad, S->head.N, nrows, c->V_l, c->logits, c->stream));
  }
  return MI_OK;
}

}  // namespace mi
