// Latent attention.  See latent_attn.h.
#include "latent_attn.h"

namespace mi {

namespace {

__device__ __forceinline__ void put4(uint16_t* p, float4 v) { *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf16x2(v.x, v.y), pack_bf16x2(v.z, v.w)); }
__device__ __forceinline__ void put4(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }

// the projection's row t: summed, or slabs of a K-split still to be summed (slice order, as splitk_reduce does)
struct QdRow {
  const float* p;
  const SlabSum& sl;
  __device__ __forceinline__ float at(int c) const {
    if (!sl.slab) return p[c];
    float v = 0.f;
    for (int z = 0; z < sl.KS; ++z) v += p[(size_t)z * sl.T * sl.N + c];
    return v * sl.scale[c];
  }
  __device__ __forceinline__ float4 at4(int c) const {      // c % 4 == 0
    float4 v = *reinterpret_cast<const float4*>(p + c);
    if (!sl.slab) return v;
    for (int z = 1; z < sl.KS; ++z) {
      const float4 q = *reinterpret_cast<const float4*>(p + (size_t)z * sl.T * sl.N + c);
      v.x += q.x; v.y += q.y; v.z += q.z; v.w += q.w;
    }
    const float4 s = *reinterpret_cast<const float4*>(sl.scale + c);
    return make_float4(v.x * s.x, v.y * s.y, v.z * s.z, v.w * s.w);
  }
};

// element d of a query head with its last nr elements rotated, at(i) the unrotated ones (rotate-half pairs)
template <typename F>
__device__ __forceinline__ float rotated(int i, int dims, const float2* cs, F at) {
  if (i >= dims) return at(i);
  const int half = dims >> 1;
  if (i < half) return at(i) * cs[i].x - at(i + half) * cs[i].y;
  return at(i) * cs[i - half].x + at(i - half) * cs[i - half].y;
}

// elements i .. i + 3 (i % 4 == 0) of a rotated part of nr, zeros behind it; at4: four at a time, for vec (nr and the part's place
// multiples of 4), where no pair is split by the quads of either half
template <typename F, typename F4>
__device__ __forceinline__ float4 rotated4(int i, int nr, int dims, const float2* cs, bool vec, F at, F4 at4) {
  const int half = dims >> 1;
  if (vec && (half & 3) == 0) {
    if (i >= dims) return i < nr ? at4(i) : make_float4(0.f, 0.f, 0.f, 0.f);
    const int j = i < half ? i : i - half;
    const float4 u = at4(j), w = at4(j + half);
    const float4 a = *reinterpret_cast<const float4*>(cs + j), b = *reinterpret_cast<const float4*>(cs + j + 2);    // (cos, sin) of two pairs each
    return i < half ? make_float4(u.x * a.x - w.x * a.y, u.y * a.z - w.y * a.w, u.z * b.x - w.z * b.y, u.w * b.z - w.w * b.w)
                    : make_float4(w.x * a.x + u.x * a.y, w.y * a.z + u.y * a.w, w.z * b.x + u.z * b.y, w.w * b.z + u.w * b.w);
  }
  auto one = [&](int k) { return k < nr ? rotated(k, dims, cs, at) : 0.f; };
  return make_float4(one(i), one(i + 1), one(i + 2), one(i + 3));
}

// one latent (columns c0 .. of the row) over its root mean square times c_norm, into its pool row; 256 threads
template <typename T>
__device__ __forceinline__ void latent_norm_row(const QdRow& row, int c0, const LatentGeom& g, const float2* cs, const float* __restrict__ c_norm, float eps,
                                                int slot, T* __restrict__ pool, float* red) {
  const int tid = threadIdx.x;
  float ss = 0.f;
  for (int d = tid; d < g.rank; d += 256) { const float v = row.at(c0 + d); ss = __builtin_fmaf(v, v, ss); }
  ss = wave_sum(ss);
  if ((tid & 63) == 0) red[tid >> 6] = ss;
  __syncthreads();
  const float f = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)g.rank + eps);
  if (slot < 0) return;
  T* dst = pool + (size_t)slot * g.cp;        // (a block's rows are consecutive: slot = block * block_size + offset)
  for (int d = tid * 4; d < g.rp; d += 1024) {
    auto at = [&](int i) { return d + i < g.rank ? row.at(c0 + d + i) * f * c_norm[d + i] : 0.f; };
    put4(dst + d, make_float4(at(0), at(1), at(2), at(3)));
  }
  for (int d = tid * 4; d < g.cp - g.rp; d += 1024) {
    auto at = [&](int i) { return d + i < g.nr ? rotated(d + i, g.dims, cs, [&](int k) { return row.at(c0 + g.rank + k); }) : 0.f; };
    put4(dst + g.rp + d, make_float4(at(0), at(1), at(2), at(3)));
  }
}

// blockIdx.y < q groups: 8 heads of 32 lanes each; the last one: the latent, one work-group per row
template <typename T>
__global__ __launch_bounds__(256) void latent_scatter_kernel(LatentRowsIn in, SlabSum sl, LatentGeom g, Rotation rot, const float* __restrict__ c_norm,
                                                             float eps, const int32_t* __restrict__ slots, int bs, T* __restrict__ q,
                                                             T* __restrict__ pool) {
  __shared__ float red[4];
  const int t = blockIdx.x, tid = threadIdx.x;
  const QdRow row{sl.slab ? sl.slab + (size_t)t * sl.N : in.q + (size_t)t * in.ldq, sl};
  const float2* cs = g.nr ? rot.table + (size_t)rot.pos[t] * (g.dims / 2) : nullptr;
  if ((int)blockIdx.y < ceil_div(g.H, 8)) {
    const int h = blockIdx.y * 8 + (tid >> 5);
    if (h >= g.H) return;
    const int c0 = h * (g.dk + g.nr);
    T* dst = q + ((size_t)t * g.H + h) * g.dkp;
    const bool vec = ((g.dk | g.nr) & 3) == 0;
    for (int d = (tid & 31) * 4; d < g.dkp; d += 128) {
      float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
      if (vec && d >= g.dk && g.nr) {
        v = rotated4(d - g.dk, g.nr, g.dims, cs, true, [&](int k) { return row.at(c0 + g.dk + k); }, [&](int k) { return row.at4(c0 + g.dk + k); });
      } else if (d + 3 >= g.dk && g.nr) {
        auto at = [&](int i) {
          if (d + i < g.dk) return row.at(c0 + d + i);
          return d + i < g.dk + g.nr ? rotated(d + i - g.dk, g.dims, cs, [&](int k) { return row.at(c0 + g.dk + k); }) : 0.f;
        };
        v = make_float4(at(0), at(1), at(2), at(3));
      } else if (vec) {
        if (d < g.dk) v = row.at4(c0 + d);
      } else {
        if (d < g.dk) v.x = row.at(c0 + d);
        if (d + 1 < g.dk) v.y = row.at(c0 + d + 1);
        if (d + 2 < g.dk) v.z = row.at(c0 + d + 2);
        if (d + 3 < g.dk) v.w = row.at(c0 + d + 3);
      }
      put4(dst + d, v);
    }
    return;
  }
  if (sl.slab) { latent_norm_row(row, g.H * (g.dk + g.nr), g, cs, c_norm, eps, slots[t], pool, red); return; }
  latent_norm_row(QdRow{in.lat + (size_t)t * in.ldl, sl}, 0, g, cs, c_norm, eps, slots[t], pool, red);
}

struct RowAt { int row, seq; };
__device__ __forceinline__ RowAt latent_row(const LatentRows& r, int z) {
  if (!r.segs) return RowAt{z, z};
  for (int i = 0; i < r.nseg; ++i) {
    const AttnSeg sg = r.segs[i];
    if (sg.n >= r.below_n) continue;
    if (z < sg.n) return RowAt{sg.row0 + z, sg.seq};
    z -= sg.n;
  }
  return RowAt{0, 0};    // (not reached: the grid has LatentRows::rows rows)
}

// factors of the elements d .. d + 3 of head h
__device__ __forceinline__ float4 gate4(const OutGate& gt, int row, int h, int dv, int d) {
  if (!gt.z) return make_float4(gt.mult, gt.mult, gt.mult, gt.mult);
  const float* z = gt.z + (size_t)row * gt.ld;
  auto f = [&](int i) { return gt.mult / (1.f + expf(-z[gt.per_element ? h * dv + min(d + i, dv - 1) : h])); };
  if (gt.per_element) return make_float4(f(0), f(1), f(2), f(3));
  const float v = f(0);
  return make_float4(v, v, v, v);
}

// a wave: one 16-row tile of W_h against 16 tokens
__global__ __launch_bounds__(256) void head_linear_kernel(const uint4* __restrict__ w, int H, int NT, int KT, const uint16_t* __restrict__ x,
                                                          LatentRows lr, OutGate gt, uint16_t* __restrict__ y, int ldy, int y_head, int n_valid) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, g4 = lane >> 4, c = lane & 15;
  const int nt = blockIdx.x * 4 + wave, h = blockIdx.y, z = blockIdx.z * 16 + c, m = latent_row(lr, min(z, lr.rows - 1)).row;
  if (nt >= NT) return;
  const u32x4_t* W = reinterpret_cast<const u32x4_t*>(w) + ((size_t)h * NT + nt) * KT * 64 + lane;
  const u32x4_t* X = reinterpret_cast<const u32x4_t*>(x + ((size_t)m * H + h) * (KT * 32)) + g4;
  f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
  int kt = 0;
  for (; kt + 4 <= KT; kt += 4) {
    u32x4_t a[4], b[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) { a[u] = W[(kt + u) * 64]; b[u] = X[(kt + u) * 4]; }
#pragma unroll
    for (int u = 0; u < 4; ++u) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a[u]), __builtin_bit_cast(bf16x8_t, b[u]), acc, 0, 0, 0);
  }
  for (; kt < KT; ++kt)
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, W[kt * 64]), __builtin_bit_cast(bf16x8_t, X[kt * 4]), acc, 0, 0, 0);
  if (z >= lr.rows) return;
  const int n = nt * 16 + g4 * 4;
  uint16_t* o = y + (size_t)m * ldy + (size_t)h * y_head + n;
  const float4 f = gate4(gt, m, h, n_valid, n);
  acc[0] *= f.x; acc[1] *= f.y; acc[2] *= f.z; acc[3] *= f.w;
  if (n + 4 <= n_valid && ((y_head | ldy) & 3) == 0) {
    put4(o, make_float4(acc[0], acc[1], acc[2], acc[3]));
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (n + i < n_valid) o[i] = f32_to_bf16(acc[i]);
  }
}

// Token generation: W_uk^T q straight from the projection's fp32 rows (rounded to bf16 on the way, as latent_scatter_kernel
// leaves q), and the latents' norm and scatter in the same launch: blockIdx.y < H a head, = H the latents of row blockIdx.x.
__global__ __launch_bounds__(256) void latent_token_kernel(LatentRowsIn in, LatentGeom g, Rotation rot, const uint4* __restrict__ w_uk, int rows,
                                                           const float* __restrict__ c_norm, float eps, const int32_t* __restrict__ slots,
                                                           uint16_t* __restrict__ qa, uint16_t* __restrict__ pool) {
  __shared__ float red[4];
  const int h = blockIdx.y;
  if (h == g.H) {
    const SlabSum none;
    const int t = blockIdx.x;
    if (t < rows)
      latent_norm_row(QdRow{in.lat + (size_t)t * in.ldl, none}, 0, g, g.nr ? rot.table + (size_t)rot.pos[t] * (g.dims / 2) : nullptr, c_norm, eps, slots[t], pool, red);
    return;
  }
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, g4 = lane >> 4, c = lane & 15;
  const int NT = g.cp / 16, KT = g.dkp / 32, ntg = ceil_div(NT, 4), tt = blockIdx.x / ntg, nt = (blockIdx.x % ntg) * 4 + wave, m = tt * 16 + c;
  if (tt * 16 >= rows || nt >= NT) return;
  const float* X = in.q + (size_t)min(m, rows - 1) * in.ldq + (size_t)h * (g.dk + g.nr);
  uint16_t* dst = qa + ((size_t)m * g.H + h) * g.cp + nt * 16 + g4 * 4;
  if (nt * 16 >= g.rp) {                     // the rotated part, as it is
    if (m >= rows) return;
    const float* X1 = X + g.dk;
    put4(dst, rotated4(nt * 16 + g4 * 4 - g.rp, g.nr, g.dims, rot.table + (size_t)rot.pos[m] * (g.dims / 2), true, [&](int k) { return X1[k]; },
                       [&](int k) { return *reinterpret_cast<const float4*>(X1 + k); }));
    return;
  }
  const u32x4_t* W = reinterpret_cast<const u32x4_t*>(w_uk) + ((size_t)h * NT + nt) * KT * 64 + lane;
  X += g4 * 8;
  const int KD = ceil_div(g.dk, 32);         // (the latent's rows have zeros behind dk)
  f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < KD; k0 += 4) {       // (past the last tile: the last one's weights against zeros)
    u32x4_t a[4], x[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      a[u] = W[min(k0 + u, KD - 1) * 64];
      float4 x0 = make_float4(0.f, 0.f, 0.f, 0.f), x1 = x0;
      const int d = (k0 + u) * 32 + g4 * 8;
      if (d < g.dk) x0 = *reinterpret_cast<const float4*>(X + (k0 + u) * 32);
      if (d + 4 < g.dk) x1 = *reinterpret_cast<const float4*>(X + (k0 + u) * 32 + 4);
      x[u] = u32x4_t{pack_bf16x2(x0.x, x0.y), pack_bf16x2(x0.z, x0.w), pack_bf16x2(x1.x, x1.y), pack_bf16x2(x1.z, x1.w)};
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a[u]), __builtin_bit_cast(bf16x8_t, x[u]), acc, 0, 0, 0);
  }
  if (m < rows) put4(dst, make_float4(acc[0], acc[1], acc[2], acc[3]));
}

__global__ __launch_bounds__(64) void head_linear_f32_kernel(const float* __restrict__ w, int H, int N, int K, const float* __restrict__ x,
                                                             float* __restrict__ y, int ldy, int y_head, int n_valid) {
  const int n = blockIdx.y * 64 + threadIdx.x, h = blockIdx.z, m = blockIdx.x;
  if (n >= n_valid) return;
  const float *W = w + ((size_t)h * N + n) * K, *X = x + ((size_t)m * H + h) * K;
  float acc = 0.f;
  for (int k = 0; k < K; ++k) acc = __builtin_fmaf(W[k], X[k], acc);
  y[(size_t)m * ldy + (size_t)h * y_head + n] = acc;
}

// =====================================================================================
// attention over latents, MFMA form
// =====================================================================================
// One work-group per (context split, HG groups of 16 heads, row), four waves, 64-key tiles of latents in LDS: keys and values at
// once.  Scores transposed (S^T = C.Q^T): wave w takes keys 16 w .. of the tile against every head; the softmax reference is
// shared through LDS; O^T += C^T.P^T is split over the latent's columns, wave w takes a quarter, with C read transposed
// (ds_read_b64_tr_b16) and the score registers as the B operand.  The next tile's rows are in flight in registers meanwhile.
typedef __attribute__((ext_vector_type(4))) short s16x4_t;
constexpr float kLog2e = 1.4426950408889634f;
constexpr int kMaxSplits = 16;
__device__ __forceinline__ float fexp2(float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ float sexp2(float x, float m) { return (x == -INFINITY) ? 0.f : fexp2(x - m); }

constexpr int kCPitch = 16;
template <int RP, int RX, int HG>
constexpr size_t latent_lds() { return (size_t)64 * (RP + RX + kCPitch) * 2 + (HG == 1 ? 0 : (size_t)HG * (RP + RX) * 32) + (size_t)HG * 4 * 64 * 8 + (size_t)HG * 4 * 16 * 4; }

// RX: columns of the rotated part (behind the latent's RP in LDS; scores only)
template <int RP, int RX, int HG, bool FINAL>
__global__ __launch_bounds__(256, HG == 1 ? 2 : 1) void latent_rows_kernel(LatentGeom g, float sc2, int window, const uint16_t* __restrict__ qa,
                                                          const uint16_t* __restrict__ pool, int bs, const int32_t* __restrict__ bt, int MB,
                                                          const int32_t* __restrict__ pos, LatentRows lr, int NS, int bs_shift, float* __restrict__ o_part,
                                                          float* __restrict__ ml_part, uint16_t* __restrict__ lat) {
  constexpr int CP = RP + RX + kCPitch, KS = (RP + RX) / 32, DN = RP / 64, CCH = RP / 8, NL = 64 * CCH / 256, NX = RX / 32;
  extern __shared__ __attribute__((aligned(16))) unsigned char dsm[];
  uint16_t* Cs = reinterpret_cast<uint16_t*>(dsm);                        // [64][CP]
  u32x4_t* Qs = reinterpret_cast<u32x4_t*>(Cs + 64 * CP);                 // [HG][KS][64 lanes]; one head group: in registers
  uint2* Ps = reinterpret_cast<uint2*>(Qs + (HG == 1 ? 0 : HG * KS * 64));   // [HG][4 waves][64 lanes]
  float* Ms = reinterpret_cast<float*>(Ps + HG * 4 * 64);                 // [HG][4 waves][16]
  const int split = blockIdx.x, h0 = blockIdx.y * 16 * HG, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, g4 = lane >> 4, c = lane & 15;
  const RowAt at = latent_row(lr, blockIdx.z);
  const int ctx = pos[at.row] + 1, lo = window > 0 ? max(0, ctx - window) : 0;
  const int32_t* btr = bt + (size_t)at.seq * MB;
  const int t_lo = lo / 64, t_hi = ceil_div(ctx, 64), per = ceil_div(t_hi - t_lo, NS);
  const int t0 = t_lo + split * per, t1 = min(t0 + per, t_hi);
  const int last_ch = g.rp / 8 - 1;

  u32x4_t cr[NL], xr[NX > 0 ? NX : 1];     // (rotated part: eight chunks a row, row tid / 8 + 32 i)
  // (addresses: a uniform part per 16-token group and a per-lane part that never changes, as in window_attn.hip)
  int blk[4], off[4];
  auto fetch_ids = [&](int tt) {     // the block of every 16-token group (block_size is a multiple of 16); past the keys: the null block
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int k = tt * 64 + 16 * u;
      int bi;
      if (bs_shift >= 0) { bi = k >> bs_shift; off[u] = k & (bs - 1); }
      else { bi = k / bs; off[u] = k - bi * bs; }
      const bool in = tt < t1 && k < ctx;
      blk[u] = in ? btr[bi] : 0;
      if (!in) off[u] = 0;
    }
  };
  constexpr int R = 256 / CCH;       // rows of a load
  const int row0 = tid / CCH, lane_off = (row0 & 15) * g.cp + min(tid % CCH, last_ch) * 8;
  const int x_off = ((tid >> 3) & 15) * g.cp + g.rp + min((tid & 7) * 8, g.cp - g.rp - 8);
  auto issue = [&]() {               // the tile whose ids fetch_ids loaded last
    const uint16_t* base[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) base[u] = pool + ((size_t)blk[u] * bs + off[u]) * g.cp;
#pragma unroll
    for (int i = 0; i < NL; ++i) {
      const uint16_t* b = base[i * R / 16];
      if constexpr (R == 32) b = row0 >= 16 ? base[i * 2 + 1] : base[i * 2];
      cr[i] = *reinterpret_cast<const u32x4_t*>(b + (R < 16 ? (i * R % 16) * g.cp : 0) + lane_off);
    }
    if constexpr (NX > 0) {
#pragma unroll
      for (int i = 0; i < NX; ++i) xr[i] = *reinterpret_cast<const u32x4_t*>((tid >= 128 ? base[2 * i + 1] : base[2 * i]) + x_off);
    }
  };
  if (t0 < t1) {
    fetch_ids(t0);
    issue();
    fetch_ids(t0 + 1);
  }
  u32x4_t qr[KS];
  auto q_frag = [&](int hg, int ks, int l) {
    const int h = h0 + hg * 16 + (l & 15), e = ks * 32 + (l >> 4) * 8, d = e < RP ? e : g.rp + e - RP;
    return h < g.H && d < (e < RP ? g.rp : g.cp) ? *reinterpret_cast<const u32x4_t*>(qa + ((size_t)at.row * g.H + h) * g.cp + d) : u32x4_t{0, 0, 0, 0};
  };
  if constexpr (HG == 1) {
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) qr[ks] = q_frag(0, ks, lane);
  } else {
    for (int i = tid; i < HG * KS * 64; i += 256) Qs[i] = q_frag((i >> 6) / KS, (i >> 6) % KS, i & 63);
  }
  f32x4_t acc[HG][DN];
  float mrow[HG], lrow[HG];
#pragma unroll
  for (int hg = 0; hg < HG; ++hg) {
    mrow[hg] = -INFINITY;
    lrow[hg] = 0.f;
#pragma unroll
    for (int dn = 0; dn < DN; ++dn) acc[hg][dn] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  }
  const int tr_row = (lane & 15) >> 2, tr_col = (lane & 3) * 4, d_w = wave * (RP / 4);

  for (int tt = t0; tt < t1; ++tt) {
    __syncthreads();                       // the previous tile is used up
#pragma unroll
    for (int i = 0; i < NL; ++i) {
      const int idx = tid + 256 * i;
      *reinterpret_cast<u32x4_t*>(&Cs[(idx / CCH) * CP + (idx % CCH) * 8]) = cr[i];
    }
    if constexpr (NX > 0) {
#pragma unroll
      for (int i = 0; i < NX; ++i) *reinterpret_cast<u32x4_t*>(&Cs[((tid >> 3) + 32 * i) * CP + RP + (tid & 7) * 8]) = xr[i];
    }
    __syncthreads();
    if (tt + 1 < t1) {
      issue();
      fetch_ids(tt + 2);
    }
    f32x4_t st[HG];
#pragma unroll
    for (int hg = 0; hg < HG; ++hg) st[hg] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    {   // fragments requested kAhead MFMAs ahead of their use
      constexpr int kAhead = KS < 8 ? KS : 8;
      bf16x8_t kf[KS];
      auto kread = [&](int ks) { kf[ks] = *reinterpret_cast<const bf16x8_t*>(&Cs[(16 * wave + c) * CP + ks * 32 + g4 * 8]); };
#pragma unroll
      for (int ks = 0; ks < kAhead; ++ks) kread(ks);
      f32x4_t s2[HG];                    // two chains of sums, added at the end
#pragma unroll
      for (int hg = 0; hg < HG; ++hg) s2[hg] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
#pragma unroll
        for (int hg = 0; hg < HG; ++hg) {
          const bf16x8_t qf = __builtin_bit_cast(bf16x8_t, HG == 1 ? qr[ks] : Qs[(hg * KS + ks) * 64 + lane]);
          if (ks & 1) s2[hg] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[ks], qf, s2[hg], 0, 0, 0);
          else st[hg] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[ks], qf, st[hg], 0, 0, 0);
        }
        if (ks + kAhead < KS) kread(ks + kAhead);
      }
      if constexpr (HG == 1) {
        __builtin_amdgcn_sched_group_barrier(0x100, kAhead, 0);
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
          __builtin_amdgcn_sched_group_barrier(0x8, 1, 0);
          if (ks + kAhead < KS) __builtin_amdgcn_sched_group_barrier(0x100, 1, 0);
        }
      }
#pragma unroll
      for (int hg = 0; hg < HG; ++hg) { st[hg][0] += s2[hg][0]; st[hg][1] += s2[hg][1]; st[hg][2] += s2[hg][2]; st[hg][3] += s2[hg][3]; }
    }
    const int j0 = tt * 64 + 16 * wave + 4 * g4;
#pragma unroll
    for (int hg = 0; hg < HG; ++hg) {
      float mx = -INFINITY;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        st[hg][i] = j0 + i >= lo && j0 + i < ctx ? st[hg][i] * sc2 : -INFINITY;
        mx = fmaxf(mx, st[hg][i]);
      }
      mx = fmaxf(mx, __shfl_xor(mx, 16));
      mx = fmaxf(mx, __shfl_xor(mx, 32));
      if (g4 == 0) Ms[(hg * 4 + wave) * 16 + c] = mx;
    }
    __syncthreads();
    float alpha[HG];
#pragma unroll
    for (int hg = 0; hg < HG; ++hg) {
      const float* M = Ms + hg * 64 + c;
      const float mn = fmaxf(mrow[hg], fmaxf(fmaxf(M[0], M[16]), fmaxf(M[32], M[48])));
      alpha[hg] = sexp2(mrow[hg], mn);
      mrow[hg] = mn;                       // (finite: a tile of the split's range has a key in sight)
      float e[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) e[i] = sexp2(st[hg][i], mn);
      lrow[hg] = lrow[hg] * alpha[hg] + ((e[0] + e[1]) + (e[2] + e[3]));
      Ps[(hg * 4 + wave) * 64 + lane] = make_uint2(pack_bf16x2(e[0], e[1]), pack_bf16x2(e[2], e[3]));
    }
    __syncthreads();
#pragma unroll
    for (int hg = 0; hg < HG; ++hg)
#pragma unroll
      for (int dn = 0; dn < DN; ++dn) { acc[hg][dn][0] *= alpha[hg]; acc[hg][dn][1] *= alpha[hg]; acc[hg][dn][2] *= alpha[hg]; acc[hg][dn][3] *= alpha[hg]; }
    // the k-slot (g4, j) of a 32-key half is key (j < 4 ? 4 g4 + j : 16 + 4 g4 + j - 4)
    bf16x8_t pf[2][HG];
#pragma unroll
    for (int hf = 0; hf < 2; ++hf)
#pragma unroll
      for (int hg = 0; hg < HG; ++hg) {
        const uint2 a = Ps[(hg * 4 + 2 * hf) * 64 + lane], b = Ps[(hg * 4 + 2 * hf + 1) * 64 + lane];
        pf[hf][hg] = __builtin_bit_cast(bf16x8_t, u32x4_t{a.x, a.y, b.x, b.y});
      }
    {
      constexpr int NPV = 2 * DN, kAhead = NPV < 6 ? NPV : 6;
      s16x4_t vlo[NPV], vhi[NPV];
      auto vread = [&](int i) {
        const uint16_t* r0 = &Cs[(32 * (i / DN) + 4 * g4 + tr_row) * CP + d_w + 16 * (i % DN) + tr_col];
        vlo[i] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((s16x4_t __attribute__((address_space(3)))*)r0);
        vhi[i] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((s16x4_t __attribute__((address_space(3)))*)(r0 + 16 * CP));
      };
#pragma unroll
      for (int i = 0; i < kAhead; ++i) vread(i);
#pragma unroll
      for (int i = 0; i < NPV; ++i) {
        const bf16x8_t av = {vlo[i][0], vlo[i][1], vlo[i][2], vlo[i][3], vhi[i][0], vhi[i][1], vhi[i][2], vhi[i][3]};
#pragma unroll
        for (int hg = 0; hg < HG; ++hg) acc[hg][i % DN] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(av, pf[i / DN][hg], acc[hg][i % DN], 0, 0, 0);
        if (i + kAhead < NPV) vread(i + kAhead);
      }
    }
  }

  // denominators: over the lanes of a head, then over the waves, in wave order
  __syncthreads();
#pragma unroll
  for (int hg = 0; hg < HG; ++hg) {
    lrow[hg] += __shfl_xor(lrow[hg], 16);
    lrow[hg] += __shfl_xor(lrow[hg], 32);
    if (g4 == 0) Ms[(hg * 4 + wave) * 16 + c] = lrow[hg];
  }
  __syncthreads();
#pragma unroll
  for (int hg = 0; hg < HG; ++hg) {
    const int h = h0 + hg * 16 + c;
    if (h >= g.H) continue;
    const float* M = Ms + hg * 64 + c;
    const float L = (M[0] + M[16]) + (M[32] + M[48]);
    const size_t hr = (size_t)at.row * g.H + h;
    const float inv = FINAL ? (L > 0.f ? 1.f / L : 0.f) : 1.f;
#pragma unroll
    for (int dn = 0; dn < DN; ++dn) {
      const int d = d_w + 16 * dn + 4 * g4;
      if (d >= g.rp) continue;
      const f32x4_t a = acc[hg][dn];
      if constexpr (FINAL) put4(lat + hr * g.rp + d, make_float4(a[0] * inv, a[1] * inv, a[2] * inv, a[3] * inv));
      else put4(o_part + (((size_t)blockIdx.z * g.H + h) * NS + split) * g.rp + d, make_float4(a[0], a[1], a[2], a[3]));
    }
    if (!FINAL && wave == 0 && g4 == 0) *reinterpret_cast<float2*>(ml_part + (((size_t)blockIdx.z * g.H + h) * NS + split) * 2) = make_float2(mrow[hg], L);
  }
}

// merge the context splits of one head over up to RW rows (split order), then W_uv.  A thread owns four columns of one row; the first
// weight tiles are requested ahead of the merge.
template <int RW>
__global__ __launch_bounds__(512) void latent_merge_kernel(LatentGeom g, const float* __restrict__ o_part, const float* __restrict__ ml_part, int NS,
                                                           LatentRows lr, OutGate gt, const uint4* __restrict__ w_uv, uint16_t* __restrict__ out, int ldo) {
  extern __shared__ __attribute__((aligned(16))) unsigned char dsm[];
  uint16_t* os = reinterpret_cast<uint16_t*>(dsm);           // [RW][rp + 8]
  const int h = blockIdx.x, z0 = blockIdx.y * RW, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, g4 = lane >> 4, c = lane & 15;
  const int pitch = g.rp + 8, n = min(RW, lr.rows - z0), NT = g.dvp / 16, KT = g.rp / 32;
  constexpr int PF = 8;
  const u32x4_t* W0 = reinterpret_cast<const u32x4_t*>(w_uv) + ((size_t)h * NT + min(wave, NT - 1)) * KT * 64 + lane;
  u32x4_t pre[PF];
#pragma unroll
  for (int u = 0; u < PF; ++u) pre[u] = W0[min(u, KT - 1) * 64];
  const int row = latent_row(lr, z0 + min(c, n - 1)).row;
  const float4 gate0 = gate4(gt, row, h, g.dv, wave * 16 + g4 * 4);
  for (int i = tid; i < n * (g.rp / 4); i += 512) {
    const int r = i / (g.rp / 4), d = (i % (g.rp / 4)) * 4;
    const size_t at = ((size_t)(z0 + r) * g.H + h) * NS;
    float m[kMaxSplits], l[kMaxSplits];
    float4 v[kMaxSplits];
#pragma unroll
    for (int k = 0; k < kMaxSplits; ++k) {
      const float2 ml = k < NS ? *reinterpret_cast<const float2*>(ml_part + (at + k) * 2) : make_float2(-INFINITY, 0.f);
      m[k] = ml.x; l[k] = ml.y;
      v[k] = k < NS ? *reinterpret_cast<const float4*>(o_part + (at + k) * g.rp + d) : make_float4(0.f, 0.f, 0.f, 0.f);
    }
    float M = -INFINITY, L = 0.f;
#pragma unroll
    for (int k = 0; k < kMaxSplits; ++k) M = fmaxf(M, m[k]);
    float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
    for (int k = 0; k < kMaxSplits; ++k) {
      const float f = sexp2(m[k], M);
      L += f * l[k];
      o.x = __builtin_fmaf(f, v[k].x, o.x); o.y = __builtin_fmaf(f, v[k].y, o.y); o.z = __builtin_fmaf(f, v[k].z, o.z); o.w = __builtin_fmaf(f, v[k].w, o.w);
    }
    const float inv = L > 0.f ? 1.f / L : 0.f;
    put4(os + r * pitch + d, make_float4(o.x * inv, o.y * inv, o.z * inv, o.w * inv));
  }
  __syncthreads();
  const bool live = c < n;
  const uint16_t* X = os + min(c, n - 1) * pitch + g4 * 8;
  for (int nt = wave; nt < NT; nt += 8) {
    const u32x4_t* W = reinterpret_cast<const u32x4_t*>(w_uv) + ((size_t)h * NT + nt) * KT * 64 + lane;
    f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int u = 0; u < PF; ++u) {
      if (u >= KT) break;
      const u32x4_t a = nt == wave ? pre[u] : W[u * 64];
      acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a), *reinterpret_cast<const bf16x8_t*>(X + u * 32), acc, 0, 0, 0);
    }
    int kt = PF;
    for (; kt + 8 <= KT; kt += 8) {
      u32x4_t a[8];
#pragma unroll
      for (int u = 0; u < 8; ++u) a[u] = W[(kt + u) * 64];
#pragma unroll
      for (int u = 0; u < 8; ++u)
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a[u]), *reinterpret_cast<const bf16x8_t*>(X + (kt + u) * 32), acc, 0, 0, 0);
    }
    for (; kt < KT; ++kt)
      acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, W[kt * 64]), *reinterpret_cast<const bf16x8_t*>(X + kt * 32), acc, 0, 0, 0);
    if (!live) continue;
    const int d = nt * 16 + g4 * 4;
    const float4 f = nt == wave ? gate0 : gate4(gt, row, h, g.dv, d);
    acc[0] *= f.x; acc[1] *= f.y; acc[2] *= f.z; acc[3] *= f.w;
    uint16_t* o = out + (size_t)row * ldo + (size_t)h * g.dv + d;
    if (d + 4 <= g.dv && ((g.dv | ldo) & 3) == 0) {
      put4(o, make_float4(acc[0], acc[1], acc[2], acc[3]));
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (d + i < g.dv) o[i] = f32_to_bf16(acc[i]);
    }
  }
}

// four gathered rows per work-group, a wave each
__global__ __launch_bounds__(256) void latent_gather_kernel(LatentGeom g, int window, const uint16_t* __restrict__ pool, int bs,
                                                            const int32_t* __restrict__ bt, int MB, const AttnSeg* __restrict__ segs, int nseg, int min_n,
                                                            int rows, uint16_t* __restrict__ x, int ldx, int32_t* __restrict__ kv_bt, int kv_mb) {
  const int m = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (m >= rows) return;
  int at = m, i = 0;
  AttnSeg sg{0, 0, 0, 0};
  for (; i < nseg; ++i) {
    sg = segs[i];
    if (sg.n < min_n) continue;
    const int n = latent_kv_rows(sg, window);
    if (at < n) break;
    at -= n;
  }
  if (i == nseg) return;
  const int p_row = latent_kv_first(sg, window) + at, p = min(p_row, sg.pos0 + sg.n - 1);     // (padding rows: copies, never in sight)
  if (lane == 0 && m % kKvBlock == 0) kv_bt[(size_t)sg.seq * kv_mb + p_row / kKvBlock] = m / kKvBlock;
  const uint16_t* src = pool + ((size_t)bt[(size_t)sg.seq * MB + p / bs] * bs + p % bs) * g.cp;
  for (int d = lane * 8; d < ldx; d += 512)
    *reinterpret_cast<u32x4_t*>(x + (size_t)m * ldx + d) = d < g.cp ? *reinterpret_cast<const u32x4_t*>(src + d) : u32x4_t{0, 0, 0, 0};
}

// rows of the batch -> rows of a list (NS = 1: lat holds the normalised output of every row; the other rows are left alone)
template <int RP, int RX, int HG>
int launch_rows_t(const LatentGeom& g, float scale, int window, const uint16_t* qa, const uint16_t* pool, int bs, const int32_t* bt, int MB,
                  const int32_t* pos, const LatentRows& lr, int NS, float* op, float* ml, uint16_t* lat, hipStream_t s) {
  constexpr size_t lds = latent_lds<RP, RX, HG>();
  const dim3 grid(NS, ceil_div(g.H, 16 * HG), lr.rows);
  auto kern = NS == 1 ? latent_rows_kernel<RP, RX, HG, true> : latent_rows_kernel<RP, RX, HG, false>;
  if (lds > 64 * 1024) { int rc = ensure_dynamic_lds(reinterpret_cast<const void*>(kern), (int)lds); if (rc != MI_OK) return rc; }
  hipLaunchKernelGGL(kern, grid, dim3(256), lds, s, g, scale * kLog2e, window, qa, pool, bs, bt, MB, pos, lr, NS, (bs & (bs - 1)) == 0 ? __builtin_ctz(bs) : -1, op, ml, lat);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

}  // namespace

static int check_latent(const LatentRowsIn& in, int T, const LatentGeom& g, const Rotation& rot, const float* c_norm) {
  MI_CHECK(T >= 1 && in.q && in.ldq % 4 == 0 && in.ldq >= g.H * g.dq() && g.dkp >= g.dq() && g.dkp % 32 == 0 && g.rp >= g.rank && g.rp % 32 == 0 &&
           g.cp >= g.rp + g.nr && g.cp % 32 == 0, "latent rows: geometry");
  MI_CHECK(g.nr == 0 || (rot.table && rot.pos && g.dims % 2 == 0 && g.dims <= g.nr), "latent rows: rotation");
  MI_CHECK(!c_norm || (in.lat && in.ldl >= g.rank + g.nr), "latent rows: latents");
  return MI_OK;
}

int launch_latent_scatter(const LatentRowsIn& in, int T, const LatentGeom& g, const Rotation& rot, const float* c_norm, float eps, const int32_t* slots,
                          int bs, void* q, void* pool, bool f32, hipStream_t s, const SlabSum* slabs) {
  const SlabSum sl = slabs ? *slabs : SlabSum();
  int rc = check_latent(in, T, g, rot, c_norm);
  if (rc != MI_OK) return rc;
  MI_CHECK(!sl.slab || (sl.T == T && sl.N == in.ldq && !sl.bias && !sl.row_scale && sl.N >= g.H * g.dq() + (c_norm ? g.rank + g.nr : 0)),
           "latent scatter: pending K-split sum of another shape");
  MI_CHECK(bs > 0, "latent scatter: block size");
  const dim3 grid(T, ceil_div(g.H, 8) + (c_norm ? 1 : 0));
  if (f32) hipLaunchKernelGGL((latent_scatter_kernel<float>), grid, dim3(256), 0, s, in, sl, g, rot, c_norm, eps, slots, bs, (float*)q, (float*)pool);
  else hipLaunchKernelGGL((latent_scatter_kernel<uint16_t>), grid, dim3(256), 0, s, in, sl, g, rot, c_norm, eps, slots, bs, (uint16_t*)q, (uint16_t*)pool);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_latent_token(const LatentRowsIn& in, int rows, const LatentGeom& g, const Rotation& rot, const void* w_uk, const float* c_norm, float eps,
                        const int32_t* slots, uint16_t* qa, uint16_t* pool, hipStream_t s) {
  int rc = check_latent(in, rows, g, rot, c_norm);
  if (rc != MI_OK) return rc;
  MI_CHECK(latent_token_supported(g), "latent token: head sizes must be multiples of 4");
  const int heads_x = ceil_div(rows, 16) * ceil_div(g.cp / 16, 4);
  const dim3 grid(c_norm && rows > heads_x ? rows : heads_x, g.H + (c_norm ? 1 : 0));
  hipLaunchKernelGGL(latent_token_kernel, grid, dim3(256), 0, s, in, g, rot, (const uint4*)w_uk, rows, c_norm, eps, slots, qa, pool);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_head_linear_rows(const void* w, int H, int N, int K, const uint16_t* x, const LatentRows& rows, uint16_t* y, int ldy, int y_head,
                            int n_valid, hipStream_t s, OutGate gt) {
  MI_CHECK(H >= 1 && rows.rows >= 1 && N % 16 == 0 && K % 32 == 0 && n_valid <= N && y_head >= n_valid && ldy >= (H - 1) * y_head + n_valid, "head linear: shape");
  hipLaunchKernelGGL(head_linear_kernel, dim3(ceil_div(N / 16, 4), H, ceil_div(rows.rows, 16)), dim3(256), 0, s, (const uint4*)w, H, N / 16, K / 32, x, rows, gt, y, ldy, y_head, n_valid);
  MI_HIP(hipGetLastError());
  return MI_OK;
}
int launch_head_linear(const void* w, int H, int N, int K, const void* x, int T, void* y, int ldy, int y_head, int n_valid, bool f32, hipStream_t s) {
  LatentRows all;
  all.rows = T;
  if (!f32) return launch_head_linear_rows(w, H, N, K, (const uint16_t*)x, all, (uint16_t*)y, ldy, y_head, n_valid, s);
  MI_CHECK(H >= 1 && T >= 1 && N % 16 == 0 && K % 32 == 0 && n_valid <= N && y_head >= n_valid && ldy >= (H - 1) * y_head + n_valid, "head linear: shape");
  hipLaunchKernelGGL(head_linear_f32_kernel, dim3(T, ceil_div(n_valid, 64), H), dim3(64), 0, s, (const float*)w, H, N, K, (const float*)x, (float*)y, ldy, y_head, n_valid);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

bool latent_attn_supported(const LatentGeom& g) { return g.rp <= 512 && g.cp - g.rp <= 64; }

// (rows x splits <= 512, launch_latent_attn_rows)
size_t latent_attn_scratch_bytes(const LatentGeom& g) { return (size_t)512 * g.H * (g.rp + 2) * sizeof(float); }

int launch_latent_attn_rows(const LatentGeom& g, float scale, int window, const uint16_t* qa, const uint16_t* pool, int bs, const int32_t* bt,
                            int MB, const int32_t* pos, const LatentRows& lr, int max_ctx, const void* w_uv, uint16_t* lat, uint16_t* out, int ldo,
                            void* scratch, hipStream_t s, OutGate gt) {
  MI_CHECK(latent_attn_supported(g) && lr.rows >= 1 && lr.rows <= 65535 && bs > 0 && bs % 16 == 0 && max_ctx >= 1 && window >= 0 && ldo >= g.H * g.dv, "latent attention: shape");
  const int hgs = ceil_div(g.H, 16), max_keys = window > 0 && window < max_ctx ? window : max_ctx, tiles = ceil_div(max_keys, 64) + 1;
  // head groups that share a tile: as many as leave the chip full
  int hg = 1;
  while (hg < 4 && hg < hgs && lr.rows * ceil_div(hgs, 2 * hg) >= 256) hg *= 2;
  const int groups = lr.rows * ceil_div(hgs, hg);
  // One head group: 70 KiB of LDS at the largest rank, two work-groups per CU.  The second one is worth its partial results
  // (the merge reads every split's) up to eight splits.
  const int most = hg == 1 ? min(512 / groups, max(256 / groups, 8)) : 256 / groups;
  int NS = min(min(most, tiles), kMaxSplits);
  if (NS < 1) NS = 1;
  float* ml = reinterpret_cast<float*>(scratch);
  float* op = ml + (size_t)512 * g.H * 2;
  int rc = MI_OK;
#define MI_LX(RP, RX) \
  rc = hg == 1 ? launch_rows_t<RP, RX, 1>(g, scale, window, qa, pool, bs, bt, MB, pos, lr, NS, op, ml, lat, s) \
     : hg == 2 ? launch_rows_t<RP, RX, 2>(g, scale, window, qa, pool, bs, bt, MB, pos, lr, NS, op, ml, lat, s) \
               : launch_rows_t<RP, RX, 4>(g, scale, window, qa, pool, bs, bt, MB, pos, lr, NS, op, ml, lat, s)
#define MI_LR(RP) { if (g.cp > g.rp) MI_LX(RP, 64); else MI_LX(RP, 0); }
  if (g.rp <= 64) MI_LR(64)
  else if (g.rp <= 128) MI_LR(128)
  else if (g.rp <= 256) MI_LR(256)
  else MI_LR(512)
#undef MI_LR
#undef MI_LX
  if (rc != MI_OK) return rc;
  if (NS == 1) return launch_head_linear_rows(w_uv, g.H, g.dvp, g.rp, lat, lr, out, ldo, g.dv, g.dv, s, gt);
  const int per = g.H * lr.rows / 256, rw = per <= 1 ? 1 : per <= 2 ? 2 : per <= 4 ? 4 : 16;
  const size_t lds = (size_t)rw * (g.rp + 8) * 2;
  const dim3 grid(g.H, ceil_div(lr.rows, rw));
#define MI_LM(RW) hipLaunchKernelGGL((latent_merge_kernel<RW>), grid, dim3(512), lds, s, g, op, ml, NS, lr, gt, (const uint4*)w_uv, out, ldo)
  if (rw == 1) MI_LM(1);
  else if (rw == 2) MI_LM(2);
  else if (rw == 4) MI_LM(4);
  else MI_LM(16);
#undef MI_LM
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_latent_gather(const LatentGeom& g, int window, const uint16_t* pool, int bs, const int32_t* bt, int MB, const AttnSeg* segs, int nseg,
                         int min_n, int rows, uint16_t* x, int ldx, int32_t* kv_bt, int kv_mb, hipStream_t s) {
  MI_CHECK(rows >= 1 && rows % kKvBlock == 0 && ldx % 8 == 0 && ldx >= g.cp && bs > 0 && nseg >= 1, "latent gather: shape");
  hipLaunchKernelGGL(latent_gather_kernel, dim3(ceil_div(rows, 4)), dim3(256), 0, s, g, window, pool, bs, bt, MB, segs, nseg, min_n, rows, x, ldx, kv_bt, kv_mb);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

}  // namespace mi
