// Per-kernel entry points of the sandwich, one-norm and post-norm blocks' mechanisms (include/mi355x_vllm.h: tests and micro-benchmarks): weights are
// placed here the way stack.hip places a layer's, then the launchers the model call uses run on the caller's data.
#include <algorithm>
#include <cstring>
#include <vector>

#include "misc_kernels.h"
#include "stack.h"

namespace mi {
namespace {

#define MI_TRY(expr)             \
  do {                           \
    int _rc = (expr);            \
    if (_rc != MI_OK) return _rc; \
  } while (0)

int pad_to(int v, int m) { return (v + m - 1) / m * m; }

// device memory of one call, zero-filled
struct Arena {
  std::vector<void*> ps;
  ~Arena() { for (void* p : ps) hipFree(p); }
  template <typename T>
  int take(T** p, size_t bytes, hipStream_t s) {
    MI_HIP(hipMalloc(reinterpret_cast<void**>(p), bytes));
    ps.push_back(*p);
    MI_HIP(hipMemsetAsync(*p, 0, bytes, s));
    return MI_OK;
  }
};

int take_segs(Arena& a, const int32_t* segs_host, int nseg, int T, int block_size, int MB, std::vector<AttnSeg>& segs, AttnSeg** dev, hipStream_t s) {
  segs.resize((size_t)nseg);
  memcpy(segs.data(), segs_host, (size_t)nseg * sizeof(AttnSeg));
  int row = 0;
  for (const AttnSeg& g : segs) {
    MI_CHECK(g.row0 == row && g.n >= 1 && g.pos0 >= 0 && g.seq >= 0 && ceil_div(g.pos0 + g.n, block_size) <= MB, "segments: contiguous rows, contexts within the block table");
    row += g.n;
  }
  MI_CHECK(row == T, "segments do not add up to the rows");
  MI_TRY(a.take(dev, (size_t)nseg * sizeof(AttnSeg), s));
  MI_HIP(hipMemcpyAsync(*dev, segs.data(), (size_t)nseg * sizeof(AttnSeg), hipMemcpyHostToDevice, s));
  MI_HIP(hipStreamSynchronize(s));
  return MI_OK;
}

int latent_op(const mi_layer_spec& p, const float* uk, const float* uv, const void* q, const void* pool, int bs, const int32_t* bt, int MB,
              const int32_t* pos, const int32_t* segs_host, int nseg, int T, int max_ctx, void* out, int ldo, bool f32, int path, hipStream_t s) {
  Arena mem;
  const int H = p.num_heads;
  const LatentGeom g = latent_geom(H, p.qk_dim, p.v_dim, p.kv_rank, p.rot_dim, p.rot_dims);
  const HeadGeom kvg{H, H, g.dq(), g.dv, g.dkp, g.dvp};
  const size_t el = f32 ? 4 : 2;
  const int dq = g.dq(), Kc = pad_to(g.nr ? g.rp + g.nr : g.rank, 64), nkv = H * (g.dkp + g.dvp);
  std::vector<AttnSeg> segs;
  AttnSeg* sd = nullptr;
  MI_TRY(take_segs(mem, segs_host, nseg, T, bs, MB, segs, &sd, s));
  int max_seq = 0;
  for (const AttnSeg& x : segs) {
    MI_CHECK(x.pos0 + x.n <= max_ctx, "segments: max_ctx");
    max_seq = std::max(max_seq, x.seq);
  }
  unsigned char *w_uk, *w_uv, *qa, *lat;
  uint16_t* ukv;
  float *tmp, *ones, *unit;
  MI_TRY(mem.take(&w_uk, (size_t)H * g.cp * g.dkp * el, s));
  MI_TRY(mem.take(&w_uv, (size_t)H * g.dvp * g.rp * el, s));
  MI_TRY(mem.take(&ukv, (size_t)nkv * Kc * 2, s));
  MI_TRY(mem.take(&tmp, (size_t)dq * g.rank * 4, s));
  MI_TRY(mem.take(&ones, (size_t)nkv * 4, s));
  MI_TRY(mem.take(&qa, (size_t)T * H * g.cp * el, s));
  MI_TRY(mem.take(&lat, (size_t)T * H * g.cp * el, s));
  MI_TRY(launch_fill_f32(ones, nkv, 1.f, s));
  std::vector<float> u((size_t)std::max(g.nr, 1) * dq, 0.f);
  for (int i = 0; i < g.nr; ++i) u[(size_t)i * dq + g.dk + i] = 1.f;
  MI_TRY(mem.take(&unit, u.size() * 4, s));
  MI_HIP(hipMemcpyAsync(unit, u.data(), u.size() * 4, hipMemcpyHostToDevice, s));
  MI_HIP(hipStreamSynchronize(s));
  for (int h = 0; h < H; ++h) {
    const float *k = uk + (size_t)h * g.dk * g.rank, *v = uv + (size_t)h * g.dv * g.rank;
    MI_TRY(launch_transpose(k, g.dk, g.rank, tmp, dq, s));
    MI_TRY(launch_place(tmp, dq, 0, g.rank, dq, w_uk + (size_t)h * g.cp * g.dkp * el, g.dkp, f32, 0, 0, s));
    if (g.nr) {
      MI_TRY(launch_place(unit, dq, 0, g.nr, dq, w_uk + (size_t)h * g.cp * g.dkp * el, g.dkp, f32, g.rp, 0, s));
      MI_TRY(launch_place(unit, dq, g.dk, g.nr, g.nr, ukv, Kc, false, h * g.dkp + g.dk, g.rp, s));
    }
    MI_TRY(launch_place(v, g.rank, 0, g.dv, g.rank, w_uv + (size_t)h * g.dvp * g.rp * el, g.rp, f32, 0, 0, s));
    MI_TRY(launch_place(k, g.rank, 0, g.dk, g.rank, ukv, Kc, false, h * g.dkp, 0, s));
    MI_TRY(launch_place(v, g.rank, 0, g.dv, g.rank, ukv, Kc, false, H * g.dkp + h * g.dvp, 0, s));
  }
  if (f32 || path == 1) {
    const AttnSpec a{HeadGeom{H, 1, g.cp, g.rp, g.cp, g.cp}, p.scale, p.window, nullptr, 0, 0};
    MI_TRY(launch_head_linear(w_uk, H, g.cp, g.dkp, q, T, qa, H * g.cp, g.cp, g.cp, f32, s));
    MI_TRY(launch_attn_plain(a, qa, pool, pool, bs, bt, MB, pos, sd, nseg, T, lat, H * g.rp, f32, s));
    MI_TRY(launch_head_linear(w_uv, H, g.dvp, g.rp, lat, T, out, ldo, g.dv, g.dv, f32, s));
  } else if (path == 2) {
    MI_CHECK(latent_attn_supported(g), "latent rows: rank up to 512");
    void* scratch = nullptr;
    MI_TRY(mem.take(&scratch, latent_attn_scratch_bytes(g), s));
    const LatentRows lr{sd, nseg, 1 << 30, T};
    MI_TRY(launch_head_linear_rows(w_uk, H, g.cp, g.dkp, (const uint16_t*)q, lr, (uint16_t*)qa, H * g.cp, g.cp, g.cp, s));
    MI_TRY(launch_latent_attn_rows(g, p.scale, p.window, (const uint16_t*)qa, (const uint16_t*)pool, bs, bt, MB, pos, lr, max_ctx, w_uv, (uint16_t*)lat,
                                   (uint16_t*)out, ldo, scratch, s));
  } else {
    MI_CHECK(attn_window_supported(kvg), "written-out keys: heads up to 256");
    int rows = 0;
    const int kv_mb = ceil_div(max_ctx, kKvBlock) + 1;
    for (const AttnSeg& x : segs) rows += x.n >= 2 ? latent_kv_rows(x, p.window) : 0;
    MI_CHECK(rows > 0, "written-out keys: no segment of two rows");
    uint16_t *x, *k, *v;
    int32_t* kv_bt;
    MI_TRY(mem.take(&x, (size_t)rows * Kc * 2, s));
    MI_TRY(mem.take(&k, (size_t)rows * H * g.dkp * 2, s));
    MI_TRY(mem.take(&v, (size_t)rows * H * g.dvp * 2, s));
    MI_TRY(mem.take(&kv_bt, (size_t)(max_seq + 1) * kv_mb * 4, s));
    MI_TRY(launch_latent_gather(g, p.window, (const uint16_t*)pool, bs, bt, MB, sd, nseg, 2, rows, x, Kc, kv_bt, kv_mb, s));
    EpiArgs e{};
    e.scale = ones;
    e.q_dim = H * g.dkp; e.hd = g.dkp; e.kv_dim = g.dvp; e.nkv = H; e.block_size = kKvBlock;
    e.kpool = k; e.vpool = v;
    MI_TRY(launch_gemm(LinearW{ukv, nkv, Kc, MI_W_BF16}, rows, x, Kc, EPI_HEADS_KV, e, s));
    const AttnSpec a{kvg, p.scale, p.window, nullptr, 0, 0};
    MI_TRY(launch_attn_window_prefill(a, (const uint16_t*)q, k, v, kKvBlock, kv_bt, kv_mb, sd, segs.data(), nseg, (uint16_t*)out, ldo, s));
  }
  MI_HIP(hipStreamSynchronize(s));
  return MI_OK;
}

}  // namespace
}  // namespace mi

using namespace mi;

extern "C" {

int mi_op_sandwich_rows(const float* resid_in, float* resid_out, const float* y, const float* pair_w, int32_t top, const float* w_post,
                        const float* w_pre, int32_t T, int32_t D, int32_t ld, int32_t groups, float eps, const float* conv_w, int32_t taps,
                        void* ring, int32_t keep, int32_t block_size, const int32_t* block_table, int32_t MB, const int32_t* pos,
                        const int32_t* slots, const int32_t* segs_host, int32_t nseg, void* out, int32_t ldy, int32_t f32, void* stream) {
  MI_CHECK(resid_in && T >= 1 && (w_pre == nullptr || out), "null argument");
  hipStream_t s = (hipStream_t)stream;
  RowSource src;
  src.y = y; src.ld = ld; src.pair_w = pair_w; src.top = top;
  ConvState cs;
  cs.w = conv_w; cs.taps = taps; cs.keep = keep; cs.ring = ring; cs.block_size = block_size; cs.MB = MB;
  cs.bt = block_table; cs.pos = pos; cs.slots = slots;
  if (nseg == 0 || !conv_w) {
    MI_TRY(launch_sandwich_rows(resid_in, resid_out, src, w_post, w_pre, T, D, ld, groups, eps, conv_w ? &cs : nullptr, out, ldy, f32 != 0, s));
    MI_HIP(hipStreamSynchronize(s));
    return MI_OK;
  }
  Arena mem;
  std::vector<AttnSeg> segs;
  AttnSeg* sd = nullptr;
  void* h = nullptr;
  MI_TRY(take_segs(mem, segs_host, nseg, T, block_size, MB, segs, &sd, s));
  MI_TRY(mem.take(&h, (size_t)T * ldy * (f32 ? 4 : 2), s));
  MI_TRY(launch_sandwich_rows(resid_in, resid_out, src, w_post, w_pre, T, D, ld, groups, eps, nullptr, h, ldy, f32 != 0, s));
  MI_TRY(launch_conv_rows(h, cs, sd, segs.data(), nseg, D, ld, out, ldy, f32 != 0, s));
  MI_HIP(hipStreamSynchronize(s));
  return MI_OK;
}

int mi_op_latent_scatter(const float* qd, int32_t ldq, int32_t T, const mi_layer_spec* spec, const float* rot, const int32_t* pos, const float* c_norm,
                         float eps, const int32_t* slots, int32_t block_size, void* q, void* pool, int32_t f32, void* stream) {
  MI_CHECK(qd && spec && slots && q && pool, "null argument");
  const mi_layer_spec& p = *spec;
  const LatentGeom g = latent_geom(p.num_heads, p.qk_dim, p.v_dim, p.kv_rank, p.rot_dim, p.rot_dims);
  MI_CHECK(!c_norm || ldq >= g.H * g.dq() + g.rank + g.nr, "latent scatter: columns");
  const LatentRowsIn in{qd, qd + g.H * g.dq(), ldq, ldq};
  return launch_latent_scatter(in, T, g, Rotation{(const float2*)rot, pos}, c_norm, eps, slots, block_size, q, pool, f32 != 0, (hipStream_t)stream);
}

int mi_op_delta_rule(const mi_layer_spec* spec, const float* proj, int32_t ldp, int32_t beta, const float* z, int32_t ldz, int32_t gate, const float* conv,
                     const float* a_log, const float* dt, const float* norm, float eps, float* state, float* ring, int32_t num_slots, const int32_t* slots_host,
                     const int32_t* pos_host, const int32_t* segs_host, int32_t nseg, int32_t T, int32_t max_chunks, void* out, int32_t ldo, int32_t f32,
                     void* stream) {
  MI_CHECK(spec && proj && z && conv && a_log && dt && norm && state && ring && slots_host && pos_host && out && T >= 1 && nseg >= 0, "null argument");
  MI_CHECK(max_chunks >= 1 && (nseg == 0 || segs_host), "delta rule: segments");
  const mi_layer_spec& p = *spec;
  hipStream_t s = (hipStream_t)stream;
  Arena mem;
  const DeltaGeom g{p.num_heads, p.num_kv_heads, p.qk_dim, p.v_dim, pad_to(p.qk_dim, 16), pad_to(p.v_dim, 16), p.conv_taps};
  MI_CHECK(delta_supported(g), "delta rule: sizes");
  const int seqs = nseg ? nseg : T;
  for (int i = 0; i < seqs; ++i) MI_CHECK(slots_host[i] >= 0 && slots_host[i] < num_slots, "delta rule: slot out of range");
  for (int i = 0; i < T; ++i) MI_CHECK(pos_host[i] >= 0, "delta rule: position");
  std::vector<AttnSeg> segs;
  AttnSeg* sd = nullptr;
  if (nseg) {
    MI_TRY(take_segs(mem, segs_host, nseg, T, 16, 1 << 20, segs, &sd, s));
    for (const AttnSeg& x : segs) MI_CHECK(x.seq < seqs, "segments: sequence");
  }
  int32_t *slots, *pos;
  float* records;
  MI_TRY(mem.take(&slots, (size_t)seqs * 4, s));
  MI_TRY(mem.take(&pos, (size_t)T * 4, s));
  MI_TRY(mem.take(&records, (size_t)max_chunks * delta_chunk_floats(g) * 4, s));
  MI_HIP(hipMemcpyAsync(slots, slots_host, (size_t)seqs * 4, hipMemcpyHostToDevice, s));
  MI_HIP(hipMemcpyAsync(pos, pos_host, (size_t)T * 4, hipMemcpyHostToDevice, s));
  DeltaIn in;
  in.proj = proj; in.ldp = ldp; in.beta = beta; in.z = z; in.ldz = ldz; in.gate = gate;
  in.conv = conv; in.a_log = a_log; in.dt = dt; in.norm = norm; in.eps = eps;
  in.state = state; in.ring = ring; in.slots = slots; in.pos = pos;
  if (!nseg) {
    MI_TRY(launch_delta_token(g, in, T, nullptr, out, ldo, f32 != 0, s));
  } else {
    MI_TRY(launch_delta_token(g, in, nseg, sd, out, ldo, f32 != 0, s));
    MI_TRY(launch_delta_prompt(g, in, sd, segs.data(), nseg, records, max_chunks, out, ldo, f32 != 0, s));
  }
  MI_HIP(hipStreamSynchronize(s));
  return MI_OK;
}

// sequences of a recurrent mixer's step: slots and positions on the device
static int take_sequences(Arena& mem, int32_t num_slots, const int32_t* slots_host, const int32_t* pos_host, const int32_t* segs_host, int nseg, int T,
                          std::vector<AttnSeg>& segs, AttnSeg** sd, int32_t** slots, int32_t** pos, hipStream_t s) {
  MI_CHECK(slots_host && pos_host && T >= 1 && nseg >= 0 && (nseg == 0 || segs_host), "sequences: null argument");
  const int seqs = nseg ? nseg : T;
  for (int i = 0; i < seqs; ++i) MI_CHECK(slots_host[i] >= 0 && slots_host[i] < num_slots, "state slot out of range");
  for (int i = 0; i < T; ++i) MI_CHECK(pos_host[i] >= 0, "position");
  if (nseg) {
    MI_TRY(take_segs(mem, segs_host, nseg, T, 16, 1 << 20, segs, sd, s));
    for (const AttnSeg& x : segs) MI_CHECK(x.seq < seqs, "segments: sequence");
  }
  MI_TRY(mem.take(slots, (size_t)seqs * 4, s));
  MI_TRY(mem.take(pos, (size_t)T * 4, s));
  MI_HIP(hipMemcpyAsync(*slots, slots_host, (size_t)seqs * 4, hipMemcpyHostToDevice, s));
  MI_HIP(hipMemcpyAsync(*pos, pos_host, (size_t)T * 4, hipMemcpyHostToDevice, s));
  return MI_OK;
}

int mi_op_embed_sinusoid(const int32_t* ids, const int32_t* pos, const void* table, float scale, float pos_base, int32_t T, int32_t D, int32_t ld,
                         float* resid, void* out, int32_t ldy, int32_t f32, void* stream) {
  MI_CHECK(ids && pos && table && resid && out && T >= 1 && D >= 1 && ld >= D && ld % 4 == 0 && pos_base > 0.f, "bad argument");
  hipStream_t s = (hipStream_t)stream;
  double* turns = nullptr;
  int rc = stack_position_turns(D, pos_base, &turns, s);
  if (rc == MI_OK) rc = launch_embed_pos(ids, pos, table, nullptr, scale, f32 != 0, T, D, ld, resid, nullptr, s, turns, out, ldy);
  hipStreamSynchronize(s);
  hipFree(turns);
  return rc;
}

int mi_op_head_scatter(const float* qkv, int32_t ldq, int32_t T, const mi_layer_spec* spec, const float* bias, const float* q_norm, const float* k_norm,
                       float eps, const int32_t* slots, int32_t block_size, void* q, void* kpool, void* vpool, int32_t f32, void* stream) {
  MI_CHECK(qkv && spec && slots && q && kpool && vpool && T >= 1, "null argument");
  const mi_layer_spec& p = *spec;
  const HeadGeom g{p.num_heads, p.num_kv_heads, p.qk_dim, p.v_dim, pad_to(p.qk_dim, 16), pad_to(p.v_dim, 16)};
  return launch_qkv_scatter(qkv, ldq, T, g, HeadRule{p.qk_norm || p.qk_unit_norm, q_norm, k_norm, bias, p.keys_as_values != 0}, eps, slots, block_size, q, kpool, vpool,
                            f32 != 0, (hipStream_t)stream);
}

int mi_op_short_conv(const float* x, int32_t ldx, const float* w, const float* b, int32_t C, int32_t taps, float* ring, int32_t num_slots,
                     const int32_t* slots_host, const int32_t* pos_host, const int32_t* segs_host, int32_t nseg, int32_t T, void* y, int32_t ldy,
                     int32_t f32, void* stream) {
  hipStream_t s = (hipStream_t)stream;
  Arena mem;
  std::vector<AttnSeg> segs;
  AttnSeg* sd = nullptr;
  int32_t *slots, *pos;
  MI_TRY(take_sequences(mem, num_slots, slots_host, pos_host, segs_host, nseg, T, segs, &sd, &slots, &pos, s));
  MI_TRY(launch_short_conv(x, ldx, ShortConv{w, b, taps, C, ring, slots}, pos, sd, segs.data(), nseg, T, y, ldy, f32 != 0, s));
  MI_HIP(hipStreamSynchronize(s));
  return MI_OK;
}

int32_t mi_op_scan_state(int32_t state) { return scan_geom(1, state, 1).Np; }

int mi_op_scan(const mi_layer_spec* spec, const void* x, int32_t ldx, const float* low, int32_t ldl, int32_t col_b, int32_t col_c, const float* w_dt,
               const float* dt_bias, const float* a_log, const float* d, const float* z, int32_t ldz, float* state, int32_t num_slots,
               const int32_t* slots_host, const int32_t* pos_host, const int32_t* segs_host, int32_t nseg, int32_t T, void* y, int32_t ldy, int32_t f32,
               void* stream) {
  MI_CHECK(spec && x && low && w_dt && a_log && state && scan_supported(spec->ssm_state) && spec->ssm_inner >= 1 && spec->dt_rank >= 1, "selective scan: arguments");
  hipStream_t s = (hipStream_t)stream;
  Arena mem;
  std::vector<AttnSeg> segs;
  AttnSeg* sd = nullptr;
  int32_t *slots, *pos;
  MI_TRY(take_sequences(mem, num_slots, slots_host, pos_host, segs_host, nseg, T, segs, &sd, &slots, &pos, s));
  const ScanGeom g = scan_geom(spec->ssm_inner, spec->ssm_state, spec->dt_rank);
  const size_t el = f32 ? 4 : 2;
  const int N = pad_to(g.C, 16), K = pad_to(g.rank, 64);
  unsigned char *wr, *wt, *lo;
  float *a2, *dt, *ones;
  MI_TRY(mem.take(&wr, (size_t)g.C * g.rank_p * el, s));
  MI_TRY(mem.take(&wt, (size_t)N * K * el, s));
  MI_TRY(mem.take(&lo, (size_t)T * K * el, s));
  MI_TRY(mem.take(&a2, (size_t)g.C * g.Np * 4, s));
  MI_TRY(mem.take(&dt, (size_t)T * N * 4, s));
  MI_TRY(mem.take(&ones, (size_t)N * 4, s));
  MI_TRY(launch_fill_f32(ones, N, 1.f, s));
  MI_TRY(launch_place_rows(w_dt, g.C, g.rank, wr, g.rank_p, f32 != 0, s));
  MI_TRY(launch_place(w_dt, g.rank, 0, g.C, g.rank, wt, K, f32 != 0, 0, 0, s));
  MI_TRY(launch_scan_decay(a_log, g, a2, s));
  ScanIn in;
  in.x = x; in.ldx = ldx; in.low = low; in.ldl = ldl; in.col_b = col_b; in.col_c = col_c;
  in.dt = dt; in.ldt = N; in.w_dt = wr; in.dt_bias = dt_bias; in.a2 = a2; in.d = d; in.z = z; in.ldz = ldz;
  in.state = state; in.slots = slots; in.pos = pos;
  if (!nseg) {
    MI_TRY(launch_scan_token(g, in, T, nullptr, y, ldy, f32 != 0, s));
  } else {
    MI_TRY(launch_columns(low, ldl, {0, g.rank, nullptr, lo}, {}, 0.f, T, K, f32 != 0, s));
    EpiArgs e{};
    e.scale = ones; e.out_f32 = dt; e.ld_out = N;
    if (f32) MI_TRY(launch_linear_f32((const float*)wt, N, K, (const float*)lo, K, T, EPI_F32, e, s));
    else MI_TRY(launch_gemm(LinearW{wt, N, K, MI_W_BF16}, T, (const uint16_t*)lo, K, EPI_F32, e, s));
    MI_TRY(launch_scan_token(g, in, nseg, sd, y, ldy, f32 != 0, s));
    MI_TRY(launch_scan_prompt(g, in, sd, nseg, y, ldy, f32 != 0, s));
  }
  MI_HIP(hipStreamSynchronize(s));
  return MI_OK;
}

int mi_op_ssd(const mi_layer_spec* spec, const void* xbc, int32_t ldx, const float* dt, int32_t ldt, const float* dt_bias, const float* a_log, const float* d,
              float* state, int32_t num_slots, const int32_t* slots_host, const int32_t* pos_host, const int32_t* segs_host, int32_t nseg, int32_t T,
              int32_t max_chunks, float* y, int32_t ldy, int32_t f32, void* stream) {
  MI_CHECK(spec && max_chunks >= 1, "state-space duality: arguments");
  hipStream_t s = (hipStream_t)stream;
  Arena mem;
  std::vector<AttnSeg> segs;
  AttnSeg* sd = nullptr;
  int32_t *slots, *pos;
  MI_TRY(take_sequences(mem, num_slots, slots_host, pos_host, segs_host, nseg, T, segs, &sd, &slots, &pos, s));
  const SsdGeom g = ssd_geom(spec->ssm_heads, spec->ssm_dim, spec->ssm_state, spec->ssm_groups);
  MI_CHECK(ssd_supported(g), "state-space duality: sizes");
  float* records;
  MI_TRY(mem.take(&records, (size_t)max_chunks * ssd_chunk_floats(g) * 4, s));
  SsdIn in;
  in.xbc = xbc; in.ldx = ldx; in.dt = dt; in.ldt = ldt; in.dt_bias = dt_bias; in.a_log = a_log; in.d = d;
  in.state = state; in.slots = slots; in.pos = pos;
  if (!nseg) {
    MI_TRY(launch_ssd_token(g, in, T, nullptr, y, ldy, f32 != 0, s));
  } else {
    MI_TRY(launch_ssd_token(g, in, nseg, sd, y, ldy, f32 != 0, s));
    MI_TRY(launch_ssd_prompt(g, in, sd, segs.data(), nseg, records, max_chunks, y, ldy, f32 != 0, s));
  }
  MI_HIP(hipStreamSynchronize(s));
  return MI_OK;
}

int mi_op_gated_norm(const float* y, int32_t ldy, const float* z, int32_t ldz, const float* w, int32_t n, int32_t parts, float eps, int32_t T, void* out,
                     int32_t ldo, int32_t f32, void* stream) {
  return launch_gated_norm(y, ldy, z, ldz, w, n, parts, eps, T, out, ldo, f32 != 0, (hipStream_t)stream);
}

int mi_op_latent_attn(const mi_layer_spec* spec, const float* uk, const float* uv, const void* q, const void* pool, int32_t block_size,
                      const int32_t* block_table, int32_t MB, const int32_t* pos, const int32_t* segs_host, int32_t nseg, int32_t T,
                      int32_t max_ctx, void* out, int32_t ldo, int32_t f32, int32_t path, void* stream) {
  MI_CHECK(spec && uk && uv && q && pool && block_table && pos && segs_host && out && nseg >= 1 && T >= 1, "null argument");
  MI_CHECK(path >= 1 && path <= 3, "path: 1 plain, 2 rows, 3 written-out keys and values");
  return latent_op(*spec, uk, uv, q, pool, block_size, block_table, MB, pos, segs_host, nseg, T, max_ctx, out, ldo, f32 != 0, path, (hipStream_t)stream);
}

int mi_op_experts(const void* x, int32_t ldx, int32_t T, int32_t D, int32_t experts, int32_t top, int32_t ff, const float* router, const float* router_b,
                  const float* gate, const float* up, const float* down, int32_t* ids, float* weights, float* y, int32_t ldy, int32_t groups, int32_t keep,
                  int32_t f32, int32_t path, void* stream) {
  const bool relu2 = groups > 0;
  MI_CHECK(x && router && router_b && (gate || relu2) && up && down && ids && weights && y && T >= 1, "null argument");
  MI_CHECK(path == 1 || path == 2, "path: 1 weight streaming (or fp32), 2 grouped");
  MI_CHECK(path == 1 || !f32, "experts: the grouped form is built for bf16");
  hipStream_t s = (hipStream_t)stream;
  Arena mem;
  const size_t el = f32 ? 4 : 2;
  const int Kd = pad_to(D, 64), N1 = pad_to((relu2 ? 1 : 2) * ff, 16), K2 = pad_to(ff, 64), N2 = pad_to(D, 16), E16 = pad_to(experts, 16), pairs = T * top;
  MI_CHECK(ldx >= Kd && ldy >= N2, "experts: strides");
  unsigned char *gu, *dn, *act, *rw;
  uint16_t *y16, *rt;
  float *z, *bias, *ones;
  uint32_t* tickets;
  int32_t* plan_mem;
  MI_TRY(mem.take(&gu, (size_t)experts * N1 * Kd * el, s));
  MI_TRY(mem.take(&dn, (size_t)experts * N2 * K2 * el, s));
  MI_TRY(mem.take(&act, (size_t)pairs * K2 * el, s));
  MI_TRY(mem.take(&rw, (size_t)experts * Kd * el, s));
  MI_TRY(mem.take(&rt, (size_t)E16 * Kd * 2, s));
  MI_TRY(mem.take(&z, (size_t)T * E16 * 4, s));
  MI_TRY(mem.take(&bias, (size_t)E16 * 4, s));
  MI_TRY(mem.take(&ones, (size_t)E16 * 4, s));
  MI_TRY(mem.take(&tickets, (size_t)T * 4, s));
  MI_TRY(mem.take(&plan_mem, experts_plan_ints(pairs, experts) * 4, s));
  MI_TRY(mem.take(&y16, (size_t)pairs * ldy * 2, s));
  MI_HIP(hipMemcpyAsync(bias, router_b, (size_t)experts * 4, hipMemcpyDeviceToDevice, s));
  MI_TRY(launch_fill_f32(ones, E16, 1.f, s));
  MI_TRY(launch_place_rows(router, experts, D, rw, Kd, f32 != 0, s));
  for (int e = 0; e < experts; ++e) {
    if (!relu2) MI_TRY(launch_place(gate + (size_t)e * ff * D, D, 0, ff, D, gu + (size_t)e * N1 * Kd * el, Kd, f32 != 0, 0, 0, s, 2));
    MI_TRY(launch_place(up + (size_t)e * ff * D, D, 0, ff, D, gu + (size_t)e * N1 * Kd * el, Kd, f32 != 0, relu2 ? 0 : 1, 0, s, relu2 ? 1 : 2));
    MI_TRY(launch_place(down + (size_t)e * D * ff, ff, 0, D, ff, dn + (size_t)e * N2 * K2 * el, K2, f32 != 0, 0, 0, s));
  }
  RouterRule rule;
  rule.b = bias;
  if (relu2) { rule.sigmoid = true; rule.groups = groups; rule.keep = keep; }
  const int a1 = relu2 ? EXPERT_RELU2 : EXPERT_SILU_GLU;
  const ExpertsLinear l1{gu, experts, N1, Kd}, l2{dn, experts, N2, K2};
  if (path == 1) {
    MI_TRY(launch_route(x, ldx, T, rw, rule, experts, Kd, top, ids, weights, f32 != 0, s, f32 ? nullptr : z, f32 ? nullptr : tickets));
    MI_TRY(launch_experts_linear(l1, ids, pairs, x, ldx, top, a1, act, K2, f32 != 0, s));
    MI_TRY(launch_experts_linear(l2, ids, pairs, act, K2, 1, EXPERT_LINEAR, y, ldy, f32 != 0, s));
  } else {
    MI_TRY(launch_place(router, D, 0, experts, D, rt, Kd, false, 0, 0, s));
    EpiArgs e{};
    e.scale = ones; e.bias = relu2 ? nullptr : bias; e.out_f32 = z; e.ld_out = E16;
    MI_TRY(launch_gemm(LinearW{rt, E16, Kd, MI_W_BF16}, T, (const uint16_t*)x, ldx, EPI_F32, e, s));
    MI_TRY(launch_route_pick(z, E16, T, rule, experts, top, ids, weights, s));
    const ExpertPlan plan = experts_plan(plan_mem, pairs, experts);
    MI_TRY(launch_experts_sort(plan, ids, pairs, experts, s));
    MI_TRY(launch_experts_gemm(l1, plan, pairs, (const uint16_t*)x, ldx, top, a1, (uint16_t*)act, K2, s));
    MI_TRY(launch_experts_gemm(l2, plan, pairs, (const uint16_t*)act, K2, 1, EXPERT_LINEAR, y16, ldy, s));
    MI_TRY(launch_bf16_to_f32(y16, y, (size_t)pairs * ldy, s));
  }
  MI_HIP(hipStreamSynchronize(s));
  return MI_OK;
}

}  // extern "C"
