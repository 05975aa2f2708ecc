// Paged attention with a sliding window or chunks, distance bias, softmax sink and output gate.  See window_attn.h.
//
// MFMA forms: a column of the 16-wide MFMA tiles is one (query, head of the kv group) pair, column = query * r + head
// with r = H / G, so the heads that share keys share the K / V tile, and a narrow window wastes little: a wave's columns
// span few queries.  Scores are computed transposed (S^T = K.Q^T); the accumulator registers are then the B operand of
// O^T += V^T.P^T as they stand, with V rows read transposed from LDS (ds_read_b64_tr_b16).  Scores, bias, softmax and
// the sink are fp32 in the exp2 domain; the sink is the running state every column starts from (max its score, sum 1).

#include "window_attn.h"

#include <algorithm>
#include <cmath>
#include <type_traits>

namespace mi {

namespace {

typedef __attribute__((ext_vector_type(4))) short s16x4_t;
constexpr float kLog2e = 1.4426950408889634f;
constexpr int kMaxSplits = 16;

__device__ __forceinline__ float fexp2(float x) { return __builtin_amdgcn_exp2f(x); }
// exp2(x - m) with the -inf conventions of online softmax (m finite or -inf)
__device__ __forceinline__ float sexp2(float x, float m) { return (x == -INFINITY) ? 0.f : fexp2(x - m); }
__device__ __forceinline__ float ld_f32(const uint16_t* p) { return bf16_to_f32(*p); }
__device__ __forceinline__ float ld_f32(const float* p) { return *p; }
__device__ __forceinline__ void st_f32(uint16_t* p, float v) { *p = f32_to_bf16(v); }
__device__ __forceinline__ void st_f32(float* p, float v) { *p = v; }
__device__ __forceinline__ float sink_score(const AttnSpec& a, int h) { return a.sinks ? a.sinks[h] : 0.f; }
__device__ __forceinline__ float gate_of(const OutGate& gt, int row, int h) { return gt.z ? gt.mult / (1.f + expf(-gt.z[(size_t)row * gt.ld + h])) : gt.mult; }
// EXT: chunks, distance tables, sinks of their own and gates; without it windows, slopes and the sink of score 0 alone (fewer registers)
bool extended(const AttnSpec& a, const OutGate& gt) { return a.chunk > 0 || a.table || a.sinks || gt.z || gt.mult != 1.f; }
template <bool EXT>
__device__ __forceinline__ int first_key(const AttnSpec& a, int p) { return EXT ? a.first_key(p) : a.window > 0 ? max(0, p - a.window + 1) : 0; }

// =====================================================================================
// plain form
// =====================================================================================
// LDS: [q dk][o dv][p 64] floats, [V row offsets 64] int64
template <typename T>
__global__ __launch_bounds__(64) void attn_plain_kernel(AttnSpec a, const T* __restrict__ q, const T* __restrict__ kpool,
                                                        const T* __restrict__ vpool, int bs, const int32_t* __restrict__ bt, int MB,
                                                        const int32_t* __restrict__ pos, const AttnSeg* __restrict__ segs, int nseg,
                                                        T* __restrict__ out, int ldo, OutGate gt) {
  extern __shared__ __attribute__((aligned(16))) unsigned char dsm[];
  const HeadGeom& g = a.g;
  long long* voff = reinterpret_cast<long long*>(dsm);
  float* p = reinterpret_cast<float*>(voff + 64);
  float* qs = p + 64;
  float* o = qs + g.dk;
  const int row = blockIdx.x, h = blockIdx.y, lane = threadIdx.x, kvh = h / (g.H / g.G);
  int seq = row;
  if (segs) {
    int i = 0;
    while (i < nseg - 1 && row >= segs[i].row0 + segs[i].n) ++i;
    seq = segs[i].seq;
  }
  const int me = pos[row], lo = a.first_key(me);
  const float slope = a.slopes ? a.slopes[h] : 0.f;
  for (int d = lane; d < g.dk; d += 64) qs[d] = ld_f32(q + ((size_t)row * g.H + h) * g.dkp + d);
  for (int d = lane; d < g.dv; d += 64) o[d] = 0.f;
  __syncthreads();
  float m = a.sink ? sink_score(a, h) : -INFINITY, l = a.sink ? 1.f : 0.f;
  for (int k0 = lo; k0 <= me; k0 += 64) {
    const int j = k0 + lane;
    float s = -INFINITY;
    if (j <= me) {
      const size_t r = ((size_t)bt[(size_t)seq * MB + j / bs] * g.G + kvh) * bs + j % bs;
      const T* kr = kpool + r * g.dkp;
      float dot = 0.f;
      for (int d = 0; d < g.dk; ++d) dot = __builtin_fmaf(qs[d], ld_f32(kr + d), dot);
      s = dot * a.scale + (a.table ? a.table[(size_t)h * a.table_n + min(me - j, a.table_n - 1)] : -slope * (float)(me - j));
      voff[lane] = (long long)(r * g.dvp);
    }
    float mx = s;
#pragma unroll
    for (int x = 32; x >= 1; x >>= 1) mx = fmaxf(mx, __shfl_xor(mx, x));
    const float mn = fmaxf(m, mx), alpha = m == -INFINITY ? 0.f : expf(m - mn);
    const float e = s == -INFINITY ? 0.f : expf(s - mn);
    p[lane] = e;
    l = l * alpha + wave_sum(e);
    m = mn;
    __syncthreads();
    const int n = min(64, me - k0 + 1);
    for (int d = lane; d < g.dv; d += 64) {
      float acc = o[d] * alpha;
      for (int k = 0; k < n; ++k) acc = __builtin_fmaf(p[k], ld_f32(vpool + voff[k] + d), acc);
      o[d] = acc;
    }
    __syncthreads();
  }
  const float gf = gate_of(gt, row, h);
  for (int d = lane; d < g.dv; d += 64) st_f32(out + (size_t)row * ldo + (size_t)h * g.dv + d, l > 0.f ? o[d] / l * gf : 0.f);
}

// =====================================================================================
// context encoding
// =====================================================================================
// 4 waves x NCG column groups of 16.  64-key tiles of K and V go through LDS (registers hold the next tile while the
// current one is multiplied; the block ids run one tile further ahead).
//
// The softmax is VALU-bound (the exponential alone costs as much as the score's MFMAs), so it is kept short:
//   * FIXED: the scores are bounded from above by s_max (unit-norm queries and keys: |q.k| <= dk; the bias only lowers a
//     score), so exp2(s - s_max) needs no running maximum, no rescaling and no cross-lane step; the reference point is folded
//     into the bias.  Taken where s_max is small enough for fp32's exponent range (fixed_reference below).
//   * The denominator is one more row of the P.V product (A = ones): it sums what the numerator multiplies.
// Row pitch dk + 16 / dv + 16 elements: fragment reads and transposed reads are bank-conflict-free (as in attn_kernels.hip).
constexpr int kPitch = 16;
template <int DK, int DV>
constexpr size_t prefill_lds() { return (size_t)64 * (DK + kPitch + DV + kPitch) * 2; }

// KS = 2: a second set of four waves takes every other key tile of the same queries (short grids, whose heaviest work-group is what
// the launch waits for); the two sets' sums meet in LDS at the end.
template <int DK, int DV, int NCG, int KS2, bool FIXED, bool EXT>
__global__ __launch_bounds__(256 * KS2) __attribute__((amdgpu_waves_per_eu(DK > 192 || DV > 128 ? KS2 : 2, DK > 192 || DV > 128 ? KS2 : 2))) void attn_window_prefill_kernel(AttnSpec a, const uint16_t* __restrict__ q, const uint16_t* __restrict__ kpool,
                                                                  const uint16_t* __restrict__ vpool, int bs, const int32_t* __restrict__ bt,
                                                                  int MB, const AttnSeg* __restrict__ segs, int nseg,
                                                                  uint16_t* __restrict__ out, int ldo, float s_max, int fold, int min_rows, int bs_shift, OutGate gt) {
  constexpr int KP = DK + kPitch, VP = DV + kPitch;    // LDS row pitches (elements)
  constexpr int KS = DK / 32, DN = DV / 16, KCH = DK / 8, VCH = DV / 8, KC0 = KCH == 24 ? 16 : KCH;   // (192 = 128 + 64: powers of two)
  constexpr int NKL = 64 * KCH / 256, NVL = 64 * VCH / 256;   // 16-byte loads per thread and tile
  extern __shared__ __attribute__((aligned(16))) unsigned char dsm[];
  const int set = KS2 == 1 ? 0 : (int)threadIdx.x >> 8;
  uint16_t* Ks = reinterpret_cast<uint16_t*>(dsm) + set * (64 * (KP + VP));
  uint16_t* Vs = Ks + 64 * KP;
  const int tid = threadIdx.x & 255, wave = tid >> 6, lane = tid & 63, g4 = lane >> 4, c = lane & 15;
  const int H = a.g.H, G = a.g.G, r = H / G, qpt = (64 * NCG) / r, kvh = blockIdx.x;

  // this work-group's tile: segments with one row belong to the token-generation kernel.  Late tiles (long contexts) first; a
  // grid that is resident at once deals its second half in ascending order, so that a CU's two work-groups add up evenly.
  const int nty = (int)gridDim.y, ty = (int)blockIdx.y;
  int t = (fold && ty >= (nty + 1) / 2) ? ty - (nty + 1) / 2 : nty - 1 - ty, si = 0;
  AttnSeg sg{0, 0, 0, 0};
  for (; si < nseg; ++si) {
    sg = segs[si];
    const int nt_s = sg.n >= min_rows ? ceil_div(sg.n, qpt) : 0;
    if (t < nt_s) break;
    t -= nt_s;
  }
  if (si == nseg) return;
  const int q0 = t * qpt, nq = min(qpt, sg.n - q0), row0 = sg.row0 + q0, pos0 = sg.pos0 + q0;
  const int32_t* btr = bt + (size_t)sg.seq * MB;
  const int win = a.window > 0 ? a.window : 0x3fffffff;
  const int klo = first_key<EXT>(a, pos0) & ~15, khi = pos0 + nq - 1;
  const int nt = ceil_div(khi + 1 - klo, 64);

  // Addresses are a uniform part per 16-token group (block_size is a multiple of 16) and a per-lane part that never changes: thread
  // load i covers rows i R .. of the tile, R = 256 / chunks per row.
  const int dkc = a.g.dkp / 8 - 1, dvc = a.g.dvp / 8 - 1;   // last 16-byte chunk of a pool row
  u32x4_t kr[NKL], vr[NVL];
  int blk[4], off[4];
  auto fetch_ids = [&](int k0) {     // block of each 16-token group; past the keys: the null block
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int k = k0 + 16 * u;
      int bi;
      if (bs_shift >= 0) { bi = k >> bs_shift; off[u] = k & (bs - 1); }
      else { bi = k / bs; off[u] = k - bi * bs; }
      const bool in = k <= khi;
      blk[u] = in ? btr[bi] : 0;
      if (!in) off[u] = 0;
    }
  };
  auto load_tile = [&](u32x4_t* reg, const uint16_t* pool, const size_t (&base)[4], int rowp, int last, auto chunks, int chunk0 = 0) {
    constexpr int CH = decltype(chunks)::value, R = 256 / CH, N = 64 / R;
    const int row0 = tid / CH, lane_off = (row0 & 15) * rowp + min(chunk0 + tid % CH, last) * 8;
#pragma unroll
    for (int i = 0; i < N; ++i) {
      if constexpr (R >= 16) {
        size_t b = base[i * R / 16];
        if constexpr (R == 32) b = row0 >= 16 ? base[i * 2 + 1] : base[i * 2];
        reg[i] = *reinterpret_cast<const u32x4_t*>(pool + b * rowp + lane_off);
      } else {
        reg[i] = *reinterpret_cast<const u32x4_t*>(pool + base[i * R / 16] * rowp + (i * R % 16) * rowp + lane_off);
      }
    }
  };
  auto issue = [&]() {               // the tile whose ids fetch_ids loaded last
    size_t base[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) base[u] = ((size_t)blk[u] * G + kvh) * bs + off[u];
    load_tile(kr, kpool, base, a.g.dkp, dkc, std::integral_constant<int, KC0>{});
    if constexpr (KCH > KC0) load_tile(kr + KC0 / 4, kpool, base, a.g.dkp, dkc, std::integral_constant<int, KCH - KC0>{}, KC0);
    load_tile(vr, vpool, base, a.g.dvp, dvc, std::integral_constant<int, VCH>{});
  };
  const int k_own = klo + 64 * set;        // this set's first tile
  fetch_ids(k_own);
  issue();
  fetch_ids(k_own + 64 * KS2);

  // distance table of the group's heads, in the exp2 domain, entries of keys ahead of the query in front (any value: they are masked)
  float* tab = reinterpret_cast<float*>(dsm + KS2 * prefill_lds<DK, DV>());
  const int front = 63 + qpt, tp = front + a.table_n;
  if (EXT && a.table)
    for (int i = threadIdx.x; i < r * tp; i += 256 * KS2) {
      const int hh = i / tp, n = i - hh * tp - front;
      tab[i] = n < 0 ? 0.f : __builtin_fmaf(a.table[(size_t)(kvh * r + hh) * a.table_n + n], kLog2e, FIXED ? -s_max : 0.f);
    }

  // columns: position, keys in sight, bias slope, query fragments (zero beyond dkp and in dead columns)
  int pc[NCG], sight[NCG];
  float sl2[NCG], mrow[NCG];
  u32x4_t qf[NCG][KS];
  f32x4_t acc[NCG][DN], den[NCG];     // den: the column's denominator, the same in every row
#pragma unroll
  for (int cg = 0; cg < NCG; ++cg) {
    const int col = (wave * NCG + cg) * 16 + c, ql = col / r, h = kvh * r + col % r;
    const bool live = ql < nq && ql < qpt;
    pc[cg] = pos0 + (live ? ql : 0);
    if constexpr (EXT) sight[cg] = pc[cg] - a.first_key(pc[cg]) + 1;
    const float sink2 = EXT ? sink_score(a, h) * kLog2e : 0.f;
    sl2[cg] = a.slopes ? a.slopes[h] * kLog2e : 0.f;
    mrow[cg] = FIXED ? s_max : (a.sink && set == 0 ? sink2 : -INFINITY);
    const float d0 = a.sink && set == 0 ? (FIXED ? fexp2(sink2 - s_max) : 1.f) : 0.f;
    den[cg] = f32x4_t{d0, d0, d0, d0};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
      qf[cg][ks] = (live && ks * 32 + g4 * 8 < a.g.dkp) ? *reinterpret_cast<const u32x4_t*>(q + ((size_t)(row0 + ql) * H + h) * a.g.dkp + ks * 32 + g4 * 8)
                                                        : u32x4_t{0, 0, 0, 0};
#pragma unroll
    for (int dn = 0; dn < DN; ++dn) acc[cg][dn] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  }
  const float sc2 = a.scale * kLog2e;
  // the wave's own query range (uniform)
  const int wq0 = (wave * NCG * 16) / r, wq1 = min(nq - 1, (wave * NCG * 16 + NCG * 16 - 1) / r);
  const bool wave_live = wq0 < nq;
  const int pmin = pos0 + wq0, pmax = pos0 + wq1, lo_min = first_key<EXT>(a, pmin), lo_max = first_key<EXT>(a, pmax);
  const int tr_row = (lane & 15) >> 2, tr_col = (lane & 3) * 4;
  const short one = 0x3f80;            // bf16 1.0
  const bf16x8_t ones = {one, one, one, one, one, one, one, one};

  for (int n = 0; n < nt; n += KS2) {
    const int k0 = k_own + 64 * n;       // (the second set's last tile may lie beyond the keys: no wave sees a key of it)
    __syncthreads();                     // the previous tile is consumed
#pragma unroll
    for (int i = 0; i < KC0 / 4; ++i) {
      const int idx = tid + 256 * i;
      *reinterpret_cast<u32x4_t*>(&Ks[(idx / KC0) * KP + (idx % KC0) * 8]) = kr[i];
    }
    if constexpr (KCH > KC0) {
#pragma unroll
      for (int i = 0; i < (KCH - KC0) / 4; ++i) {
        const int idx = tid + 256 * i;
        *reinterpret_cast<u32x4_t*>(&Ks[(idx / (KCH - KC0)) * KP + (KC0 + idx % (KCH - KC0)) * 8]) = kr[KC0 / 4 + i];
      }
    }
#pragma unroll
    for (int i = 0; i < NVL; ++i) {
      const int idx = tid + 256 * i;
      *reinterpret_cast<u32x4_t*>(&Vs[(idx / VCH) * VP + (idx % VCH) * 8]) = vr[i];
    }
    __syncthreads();
    if (n + KS2 < nt) {
      issue();
      fetch_ids(k0 + 128 * KS2);
    }
    if (!wave_live || k0 > pmax || k0 + 63 < lo_min) continue;   // no key of this tile is seen by the wave (uniform)
    // S^T = K.Q^T: the fragments of a 16-key group are requested one group ahead of the MFMAs that take them
    f32x4_t st[NCG][4];
    {
      bf16x8_t kf[KS];
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) kf[ks] = *reinterpret_cast<const bf16x8_t*>(&Ks[c * KP + ks * 32 + g4 * 8]);
#pragma unroll
      for (int u = 0; u < 4; ++u) {
#pragma unroll
        for (int cg = 0; cg < NCG; ++cg) st[cg][u] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
#pragma unroll
          for (int cg = 0; cg < NCG; ++cg)
            st[cg][u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[ks], __builtin_bit_cast(bf16x8_t, qf[cg][ks]), st[cg][u], 0, 0, 0);
          if (u < 3) kf[ks] = *reinterpret_cast<const bf16x8_t*>(&Ks[(16 * (u + 1) + c) * KP + ks * 32 + g4 * 8]);
        }
      }
      __builtin_amdgcn_sched_group_barrier(0x100, KS, 0);
#pragma unroll
      for (int i = 0; i < 3 * KS; ++i) {
        __builtin_amdgcn_sched_group_barrier(0x8, NCG, 0);
        __builtin_amdgcn_sched_group_barrier(0x100, 1, 0);
      }
#pragma unroll
      for (int i = 0; i < KS; ++i) __builtin_amdgcn_sched_group_barrier(0x8, NCG, 0);
    }
    const bool edge = k0 + 63 > pmin || k0 < lo_max;
    union { uint32_t w[4]; bf16x8_t v; } pk[NCG][2];
#pragma unroll
    for (int cg = 0; cg < NCG; ++cg) {
      if (!EXT && a.slopes) {
        // - slope (i - j) of the lane's first key (- the fixed reference)
        const float b0 = __builtin_fmaf(sl2[cg], (float)(k0 + 4 * g4 - pc[cg]), FIXED ? -s_max : 0.f);
#pragma unroll
        for (int u = 0; u < 4; ++u)
#pragma unroll
          for (int i = 0; i < 4; ++i)
            st[cg][u][i] = __builtin_fmaf(st[cg][u][i], sc2, __builtin_fmaf(sl2[cg], (float)(16 * u + i), b0));
      } else if (EXT && a.table) {
        const float* th = tab + (((wave * NCG + cg) * 16 + c) % r) * tp + front;
        const int n0 = pc[cg] - (k0 + 4 * g4), last = a.table_n - 1;       // distance of the lane's first key
        if (pos0 - (k0 + 63) >= last) {            // (uniform, as below: every distance is past the table, or none is)
          const float b = th[last];
#pragma unroll
          for (int u = 0; u < 4; ++u)
#pragma unroll
            for (int i = 0; i < 4; ++i) st[cg][u][i] = __builtin_fmaf(st[cg][u][i], sc2, b);
        } else if (pmax - k0 <= last) {
#pragma unroll
          for (int u = 0; u < 4; ++u)
#pragma unroll
            for (int i = 0; i < 4; ++i) st[cg][u][i] = __builtin_fmaf(st[cg][u][i], sc2, th[n0 - 16 * u - i]);
        } else {
#pragma unroll
          for (int u = 0; u < 4; ++u)
#pragma unroll
            for (int i = 0; i < 4; ++i) st[cg][u][i] = __builtin_fmaf(st[cg][u][i], sc2, th[min(n0 - 16 * u - i, last)]);
        }
      } else {
#pragma unroll
        for (int u = 0; u < 4; ++u)
#pragma unroll
          for (int i = 0; i < 4; ++i) st[cg][u][i] = FIXED ? __builtin_fmaf(st[cg][u][i], sc2, -s_max) : st[cg][u][i] * sc2;
      }
      if (edge) {
        const int j0 = k0 + 4 * g4;
#pragma unroll
        for (int u = 0; u < 4; ++u)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int back = pc[cg] - (j0 + 16 * u + i);
            if ((unsigned)back >= (unsigned)(EXT ? sight[cg] : win)) st[cg][u][i] = -INFINITY;   // ahead of the query, or out of its sight
          }
      }
      float ms = 0.f;
      if constexpr (!FIXED) {
        float mx = -INFINITY;
#pragma unroll
        for (int u = 0; u < 4; ++u)
          mx = fmaxf(fmaxf(fmaxf(mx, st[cg][u][0]), fmaxf(st[cg][u][1], st[cg][u][2])), st[cg][u][3]);
        mx = fmaxf(mx, __shfl_xor(mx, 16));
        mx = fmaxf(mx, __shfl_xor(mx, 32));
        const float mn = fmaxf(mrow[cg], mx);
        const float alpha = sexp2(mrow[cg], mn);
        const bool moved = mn != mrow[cg];
        mrow[cg] = mn;
        ms = mn == -INFINITY ? 0.f : mn;   // (a column without a key so far: every score is -inf, exp2 gives 0)
        if (__any(moved)) {
          den[cg][0] *= alpha; den[cg][1] *= alpha; den[cg][2] *= alpha; den[cg][3] *= alpha;
#pragma unroll
          for (int dn = 0; dn < DN; ++dn) {
            acc[cg][dn][0] *= alpha; acc[cg][dn][1] *= alpha; acc[cg][dn][2] *= alpha; acc[cg][dn][3] *= alpha;
          }
        }
      }
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        float e[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) e[i] = FIXED ? fexp2(st[cg][u][i]) : fexp2(st[cg][u][i] - ms);
        pk[cg][u >> 1].w[(u & 1) * 2] = pack_bf16x2(e[0], e[1]);
        pk[cg][u >> 1].w[(u & 1) * 2 + 1] = pack_bf16x2(e[2], e[3]);
      }
#pragma unroll
      for (int hf = 0; hf < 2; ++hf) den[cg] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ones, pk[cg][hf].v, den[cg], 0, 0, 0);
    }
    // O^T += V^T.P^T: the k-slot (g4, j) of a 32-key half is key (j < 4 ? 4 g4 + j : 16 + 4 g4 + j - 4); fragments requested
    // kAhead MFMAs ahead of their use
    {
      constexpr int NPV = 2 * DN, kAhead = NPV < 4 ? NPV : 4;
      s16x4_t vlo[NPV], vhi[NPV];
      auto vread = [&](int i) {
        const uint16_t* r0 = &Vs[(32 * (i / DN) + 4 * g4 + tr_row) * VP + 16 * (i % DN) + tr_col];
        vlo[i] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((s16x4_t __attribute__((address_space(3)))*)r0);
        vhi[i] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((s16x4_t __attribute__((address_space(3)))*)(r0 + 16 * VP));
      };
#pragma unroll
      for (int i = 0; i < kAhead; ++i) vread(i);
#pragma unroll
      for (int i = 0; i < NPV; ++i) {
        const bf16x8_t av = {vlo[i][0], vlo[i][1], vlo[i][2], vlo[i][3], vhi[i][0], vhi[i][1], vhi[i][2], vhi[i][3]};
#pragma unroll
        for (int cg = 0; cg < NCG; ++cg) acc[cg][i % DN] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(av, pk[cg][i / DN].v, acc[cg][i % DN], 0, 0, 0);
        if (i + kAhead < NPV) vread(i + kAhead);
      }
      __builtin_amdgcn_sched_group_barrier(0x100, 2 * kAhead, 0);
#pragma unroll
      for (int i = 0; i < NPV; ++i) {
        __builtin_amdgcn_sched_group_barrier(0x8, NCG, 0);
        if (i + kAhead < NPV) __builtin_amdgcn_sched_group_barrier(0x100, 2, 0);
      }
    }
  }

  if constexpr (KS2 == 2) {              // the second set hands over its sums, lane by lane
    float* x = reinterpret_cast<float*>(dsm) + (size_t)tid * 4;      // [DN + 1][256 lanes][4], one column group at a time
#pragma unroll
    for (int cg = 0; cg < NCG; ++cg) {
      __syncthreads();
      if (set == 1) {
#pragma unroll
        for (int dn = 0; dn < DN; ++dn) *reinterpret_cast<f32x4_t*>(x + dn * 1024) = acc[cg][dn];
        *reinterpret_cast<float2*>(x + DN * 1024) = make_float2(mrow[cg], den[cg][0]);
      }
      __syncthreads();
      if (set == 0) {
        const float2 ml = *reinterpret_cast<const float2*>(x + DN * 1024);
        float f0 = 1.f, f1 = 1.f;
        if constexpr (!FIXED) {
          const float M = fmaxf(mrow[cg], ml.x);
          f0 = sexp2(mrow[cg], M); f1 = sexp2(ml.x, M);
        }
        den[cg][0] = den[cg][0] * f0 + ml.y * f1;
#pragma unroll
        for (int dn = 0; dn < DN; ++dn) {
          const f32x4_t o = *reinterpret_cast<const f32x4_t*>(x + dn * 1024);
#pragma unroll
          for (int i = 0; i < 4; ++i) acc[cg][dn][i] = acc[cg][dn][i] * f0 + o[i] * f1;
        }
      }
    }
    if (set == 1) return;
  }
#pragma unroll
  for (int cg = 0; cg < NCG; ++cg) {
    const float L = den[cg][0];
    const int col = (wave * NCG + cg) * 16 + c, ql = col / r, h = kvh * r + col % r;
    if (ql >= nq || ql >= qpt) continue;
    const float inv = L > 0.f ? (EXT ? gate_of(gt, row0 + ql, h) : 1.f) / L : 0.f;
    uint16_t* o = out + (size_t)(row0 + ql) * ldo + (size_t)h * a.g.dv;
#pragma unroll
    for (int dn = 0; dn < DN; ++dn) {
      const int d = 16 * dn + 4 * g4;
      if ((a.g.dv & 3) == 0) {
        if (d < a.g.dv)
          *reinterpret_cast<uint2*>(o + d) = make_uint2(pack_bf16x2(acc[cg][dn][0] * inv, acc[cg][dn][1] * inv), pack_bf16x2(acc[cg][dn][2] * inv, acc[cg][dn][3] * inv));
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (d + i < a.g.dv) o[d + i] = f32_to_bf16(acc[cg][dn][i] * inv);
      }
    }
  }
}

// =====================================================================================
// token generation
// =====================================================================================
// One work-group per (context split, kv head and group of 16 of its heads, sequence); its waves walk 32-key tiles
// round-robin, two tiles in flight per wave.  K goes from the pool straight into A fragments, V through a wave-private LDS tile.
template <int DV, int NW>
constexpr size_t decode_lds() { return (size_t)NW * 32 * (DV + 8) * 2 + (size_t)NW * 16 * 2 * sizeof(float); }

template <int DK, int DV, int NW, bool FINAL, bool EXT>
__global__ __launch_bounds__(NW * 64) void attn_window_decode_kernel(AttnSpec a, const uint16_t* __restrict__ q, const uint16_t* __restrict__ kpool,
                                                                     const uint16_t* __restrict__ vpool, int bs, const int32_t* __restrict__ bt,
                                                                     int MB, const int32_t* __restrict__ ctx_lens, int NS,
                                                                     float* __restrict__ o_part, float* __restrict__ ml_part,
                                                                     uint16_t* __restrict__ out, int ldo, OutGate gt) {
  constexpr int VP = DV + 8, KS = DK / 32, DN = DV / 16, VCH = DV / 8;
  constexpr int NV = 32 * VCH / 64;
  constexpr int VT = 32 * VP;
  extern __shared__ __attribute__((aligned(16))) unsigned char dsm[];
  uint16_t* Vs = reinterpret_cast<uint16_t*>(dsm);                       // [NW][32][VP]
  float* sm_ml = reinterpret_cast<float*>(dsm + (size_t)NW * VT * 2);    // [NW][16][2]
  const int H = a.g.H, G = a.g.G, r = H / G;
  const int split = blockIdx.x, kvh = blockIdx.y % G, hc = blockIdx.y / G, b = blockIdx.z;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, g4 = lane >> 4, c = lane & 15;
  const int nhc = min(16, r - hc * 16), h0 = kvh * r + hc * 16;          // this work-group's heads
  const int ctx = ctx_lens[b], lo = first_key<EXT>(a, ctx - 1);
  const int32_t* btr = bt + (size_t)b * MB;
  const int t_first = lo / 32 + split * NW + wave, t_end = ceil_div(ctx, 32), stride = NS * NW;
  const int dkc = a.g.dkp / 8 - 1, dvc = a.g.dvp / 8 - 1;
  uint16_t* Vw = Vs + wave * VT;

  u32x4_t kA[2 * KS], vA[NV], kB[2 * KS], vB[NV];
  float bA[8], bB[8];                                                    // distance biases (table)
  const float* th = EXT && a.table ? a.table + (size_t)(h0 + min(c, nhc - 1)) * a.table_n : nullptr;
  auto issue = [&](u32x4_t (&kr)[2 * KS], u32x4_t (&vr)[NV], float (&br)[8], int tt) {
    if (EXT && th) {
#pragma unroll
      for (int k = 0; k < 8; ++k) br[k] = th[min(max(ctx - 1 - (tt * 32 + 16 * (k >> 2) + 4 * g4 + (k & 3)), 0), a.table_n - 1)];
    }
    size_t rowh[2];   // pool row of the first token of each 16-token half (the null block where there is none)
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int tok = tt * 32 + 16 * u;
      rowh[u] = (tt < t_end && tok < ctx) ? ((size_t)btr[tok / bs] * G + kvh) * bs + tok % bs : 0;
    }
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
      for (int ks = 0; ks < KS; ++ks)
        kr[u * KS + ks] = __builtin_nontemporal_load(reinterpret_cast<const u32x4_t*>(kpool + (rowh[u] + c) * a.g.dkp + min(ks * 4 + g4, dkc) * 8));
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int row = (lane + 64 * i) / VCH, ch = min((lane + 64 * i) % VCH, dvc);
      vr[i] = __builtin_nontemporal_load(reinterpret_cast<const u32x4_t*>(vpool + (rowh[row >> 4] + (row & 15)) * a.g.dvp + ch * 8));
    }
  };
  if (t_first < t_end) issue(kA, vA, bA, t_first);

  u32x4_t qf[KS];
#pragma unroll
  for (int ks = 0; ks < KS; ++ks)
    qf[ks] = (c < nhc && ks * 32 + g4 * 8 < a.g.dkp) ? *reinterpret_cast<const u32x4_t*>(q + ((size_t)b * H + h0 + c) * a.g.dkp + ks * 32 + g4 * 8)
                                                     : u32x4_t{0, 0, 0, 0};
  const float sl2 = (a.slopes && c < nhc) ? a.slopes[h0 + c] * kLog2e : 0.f, sc2 = a.scale * kLog2e;
  f32x4_t acc[DN];
#pragma unroll
  for (int dn = 0; dn < DN; ++dn) acc[dn] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  float mrow = -INFINITY, lrow = 0.f;
  const int tr_row = (lane & 15) >> 2, tr_col = (lane & 3) * 4;

  auto update = [&](const u32x4_t (&kr)[2 * KS], const u32x4_t (&vr)[NV], const float (&br)[8], int tt) {
    asm volatile("" ::: "memory");
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int idx = lane + 64 * i;
      *reinterpret_cast<u32x4_t*>(&Vw[(idx / VCH) * VP + (idx % VCH) * 8]) = vr[i];
    }
    asm volatile("" ::: "memory");   // LDS ops of one wave execute in order; keep the compiler from reordering them
    f32x4_t st[2];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      st[u] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < KS; ++ks)
        st[u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, kr[u * KS + ks]), __builtin_bit_cast(bf16x8_t, qf[ks]), st[u], 0, 0, 0);
    }
    s16x4_t vlo[DN], vhi[DN];
#pragma unroll
    for (int dn = 0; dn < DN; ++dn) {
      const uint16_t* r0 = &Vw[(4 * g4 + tr_row) * VP + 16 * dn + tr_col];
      vlo[dn] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((s16x4_t __attribute__((address_space(3)))*)r0);
      vhi[dn] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((s16x4_t __attribute__((address_space(3)))*)(r0 + 16 * VP));
    }
    float pv[8], mx = -INFINITY;
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int j = tt * 32 + 16 * u + 4 * g4 + i;
        float sv = __builtin_fmaf(st[u][i], sc2, EXT && th ? br[4 * u + i] * kLog2e : sl2 * (float)(j - (ctx - 1)));
        if (j >= ctx || j < lo) sv = -INFINITY;
        pv[4 * u + i] = sv;
        mx = fmaxf(mx, sv);
      }
    mx = fmaxf(mx, __shfl_xor(mx, 16));
    mx = fmaxf(mx, __shfl_xor(mx, 32));
    const float mn = fmaxf(mrow, mx);
    const float alpha = sexp2(mrow, mn);
    float ps = 0.f;
#pragma unroll
    for (int k = 0; k < 8; ++k) {
      pv[k] = sexp2(pv[k], mn);
      ps += pv[k];
    }
    const bool moved = mn != mrow;
    mrow = mn;
    lrow = lrow * alpha + ps;
    union { uint32_t w[4]; bf16x8_t v; } pk;
#pragma unroll
    for (int k = 0; k < 4; ++k) pk.w[k] = pack_bf16x2(pv[2 * k], pv[2 * k + 1]);
    if (__any(moved)) {
#pragma unroll
      for (int dn = 0; dn < DN; ++dn) {
        acc[dn][0] *= alpha; acc[dn][1] *= alpha; acc[dn][2] *= alpha; acc[dn][3] *= alpha;
      }
    }
#pragma unroll
    for (int dn = 0; dn < DN; ++dn) {
      const s16x4_t l4 = vlo[dn], h4 = vhi[dn];
      const bf16x8_t av = {l4[0], l4[1], l4[2], l4[3], h4[0], h4[1], h4[2], h4[3]};
      acc[dn] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(av, pk.v, acc[dn], 0, 0, 0);
    }
  };

  for (int tt = t_first; tt < t_end; tt += 2 * stride) {
    if (tt + stride < t_end) issue(kB, vB, bB, tt + stride);
    update(kA, vA, bA, tt);
    if (tt + 2 * stride < t_end) issue(kA, vA, bA, tt + 2 * stride);
    if (tt + stride < t_end) update(kB, vB, bB, tt + stride);
  }

  // merge the waves through their (now idle) LDS tiles, in wave order
  lrow += __shfl_xor(lrow, 16);
  lrow += __shfl_xor(lrow, 32);
  asm volatile("" ::: "memory");
  float* so = reinterpret_cast<float*>(Vw);            // [16 heads][DV] f32 <= the tile
#pragma unroll
  for (int dn = 0; dn < DN; ++dn) *reinterpret_cast<f32x4_t*>(&so[c * DV + 16 * dn + 4 * g4]) = acc[dn];
  if (g4 == 0) {
    sm_ml[(wave * 16 + c) * 2] = mrow;
    sm_ml[(wave * 16 + c) * 2 + 1] = lrow;
  }
  __syncthreads();
  for (int idx = tid; idx < nhc * DV; idx += NW * 64) {
    const int h = idx / DV, d = idx % DV;
    if (d >= a.g.dvp) continue;
    float M = sm_ml[h * 2];
#pragma unroll
    for (int w = 1; w < NW; ++w) M = fmaxf(M, sm_ml[(w * 16 + h) * 2]);
    const float sink2 = EXT && FINAL && a.sink ? sink_score(a, h0 + h) * kLog2e : 0.f;
    if (FINAL && a.sink) M = fmaxf(M, sink2);
    float o = 0.f, L = 0.f;
#pragma unroll
    for (int w = 0; w < NW; ++w) {
      const float f = sexp2(sm_ml[(w * 16 + h) * 2], M);
      o += f * reinterpret_cast<const float*>(Vs + w * VT)[h * DV + d];
      L += f * sm_ml[(w * 16 + h) * 2 + 1];
    }
    if constexpr (FINAL) {
      if (a.sink) L += fexp2(sink2 - M);
      if (d < a.g.dv) out[(size_t)b * ldo + (size_t)(h0 + h) * a.g.dv + d] = f32_to_bf16(L > 0.f ? o * (EXT ? gate_of(gt, b, h0 + h) : 1.f) / L : 0.f);
    } else {
      const size_t row = ((size_t)b * H + h0 + h) * kMaxSplits + split;
      o_part[row * a.g.dvp + d] = o;
      if (d == 0) {
        ml_part[row * 2] = M;
        ml_part[row * 2 + 1] = L;
      }
    }
  }
}

// merge the context splits of one (sequence, head) in split order, the sink last
__global__ __launch_bounds__(128) void attn_window_combine_kernel(AttnSpec a, const float* __restrict__ o_part, const float* __restrict__ ml_part,
                                                                  int NS, uint16_t* __restrict__ out, int ldo, OutGate gt) {
  const int head = blockIdx.x, b = blockIdx.y;
  const size_t row0 = ((size_t)b * a.g.H + head) * kMaxSplits;
  float mv[kMaxSplits], lv[kMaxSplits];
  const float sink2 = a.sink ? sink_score(a, head) * kLog2e : 0.f, gf = gate_of(gt, b, head);
  float M = a.sink ? sink2 : -INFINITY;
#pragma unroll
  for (int s = 0; s < kMaxSplits; ++s) {
    const float2 ml = s < NS ? *reinterpret_cast<const float2*>(ml_part + (row0 + s) * 2) : make_float2(-INFINITY, 0.f);
    mv[s] = ml.x;
    lv[s] = ml.y;
    M = fmaxf(M, ml.x);
  }
  float L = a.sink ? fexp2(sink2 - M) : 0.f;
#pragma unroll
  for (int s = 0; s < kMaxSplits; ++s) {
    mv[s] = sexp2(mv[s], M);
    L += mv[s] * lv[s];
  }
  for (int d = threadIdx.x; d < a.g.dv; d += 128) {
    float ov[kMaxSplits];
#pragma unroll
    for (int s = 0; s < kMaxSplits; ++s) ov[s] = s < NS ? o_part[(row0 + s) * a.g.dvp + d] : 0.f;
    float acc = 0.f;
#pragma unroll
    for (int s = 0; s < kMaxSplits; ++s) acc += mv[s] * ov[s];
    out[(size_t)b * ldo + (size_t)head * a.g.dv + d] = f32_to_bf16(L > 0.f ? acc * gf / L : 0.f);
  }
}

// context splits: about one work-group per CU, every wave of a split with at least a tile to walk
int decode_splits(int groups, int max_keys, int nw) {
  const int by_cu = 256 / groups, by_len = ceil_div(ceil_div(max_keys, 32) + 1, nw);
  const int ns = by_cu < by_len ? by_cu : by_len;
  return ns < 1 ? 1 : (ns > kMaxSplits ? kMaxSplits : ns);
}

int check_spec(const AttnSpec& a, int block_size) {
  MI_CHECK(a.g.H > 0 && a.g.G > 0 && a.g.H % a.g.G == 0, "attention: query heads must be a multiple of kv heads");
  MI_CHECK(a.g.dk > 0 && a.g.dv > 0 && a.g.dkp % 16 == 0 && a.g.dvp % 16 == 0 && a.g.dkp >= a.g.dk && a.g.dvp >= a.g.dv, "attention: head sizes");
  MI_CHECK(block_size > 0 && block_size % 16 == 0 && a.window >= 0, "attention: block_size % 16 == 0, window >= 0");
  MI_CHECK(a.chunk >= 0 && (!a.table || (a.table_n >= 1 && !a.slopes)), "attention: chunk / distance table");
  return MI_OK;
}

template <int DK, int DV, bool EXT>
int launch_decode_t(const AttnSpec& a, const uint16_t* q, const uint16_t* kpool, const uint16_t* vpool, int bs, const int32_t* bt, int MB,
                    const int32_t* ctx, int B, int max_ctx, uint16_t* out, int ldo, void* scratch, hipStream_t s, const OutGate& gt) {
  constexpr int NW = 4;
  const int hcs = ceil_div(a.g.H / a.g.G, 16), groups = B * a.g.G * hcs;
  const int NS = decode_splits(groups, a.most_keys(max_ctx), NW);
  constexpr size_t lds = decode_lds<DV, NW>();
  const dim3 grid(NS, a.g.G * hcs, B);
  if (NS == 1) {
    auto kern = attn_window_decode_kernel<DK, DV, NW, true, EXT>;
    if (lds > 64 * 1024) { int rc = ensure_dynamic_lds(reinterpret_cast<const void*>(kern), (int)lds); if (rc != MI_OK) return rc; }
    hipLaunchKernelGGL(kern, grid, dim3(NW * 64), lds, s, a, q, kpool, vpool, bs, bt, MB, ctx, 1, nullptr, nullptr, out, ldo, gt);
  } else {
    float* ml = reinterpret_cast<float*>(scratch);
    float* op = ml + (size_t)B * a.g.H * kMaxSplits * 2;
    auto kern = attn_window_decode_kernel<DK, DV, NW, false, EXT>;
    if (lds > 64 * 1024) { int rc = ensure_dynamic_lds(reinterpret_cast<const void*>(kern), (int)lds); if (rc != MI_OK) return rc; }
    hipLaunchKernelGGL(kern, grid, dim3(NW * 64), lds, s, a, q, kpool, vpool, bs, bt, MB, ctx, NS, op, ml, out, ldo, gt);
    hipLaunchKernelGGL(attn_window_combine_kernel, dim3(a.g.H, B), dim3(128), 0, s, a, op, ml, NS, out, ldo, gt);
  }
  MI_HIP(hipGetLastError());
  return MI_OK;
}

// FIXED softmax reference (exp2 domain): unit-norm heads bound the score by |scale| dk, 1 % for the rounding of q and k to bf16.
// Up to 2^+-60 around it every weight that matters stays a normal fp32 number: the lowest unbiased score is 2^-120 of the
// reference, and the sink (score 0) 2^-60.  0: not applicable, the running maximum is used.
float fixed_reference(const AttnSpec& a) {
  const float b = fabsf(a.scale) * (float)a.g.dk * 1.01f * kLog2e;
  return a.unit_norm && b <= 60.f && b > 0.f ? b : 0.f;
}

template <int DK, int DV, int NCG, int KS2, bool EXT>
int launch_prefill_t(const AttnSpec& a, const uint16_t* q, const uint16_t* kpool, const uint16_t* vpool, int bs, const int32_t* bt, int MB,
                     const AttnSeg* sd, const AttnSeg* sh, int nseg, uint16_t* out, int ldo, hipStream_t s, int min_rows, const OutGate& gt) {
  const int qpt = 64 * NCG / (a.g.H / a.g.G);
  int tiles = 0;
  for (int i = 0; i < nseg; ++i) tiles += sh[i].n >= min_rows ? ceil_div(sh[i].n, qpt) : 0;
  if (tiles == 0) return MI_OK;
  constexpr size_t tiles_lds = KS2 * prefill_lds<DK, DV>();
  static_assert(KS2 == 1 || tiles_lds >= (size_t)(DV / 16 + 1) * 1024 * 4, "the handed-over sums fit the tiles");
  const size_t lds = tiles_lds + (a.table ? (size_t)(a.g.H / a.g.G) * (63 + qpt + a.table_n) * 4 : 0);
  const float s_max = EXT ? 0.f : fixed_reference(a);
  int num_cu = 0;
  { int rc = device_num_cu(&num_cu); if (rc != MI_OK) return rc; }
  const int fold = KS2 == 1 && tiles * a.g.G <= 2 * num_cu;
  auto kern = attn_window_prefill_kernel<DK, DV, NCG, KS2, false, EXT>;
  if constexpr (!EXT) { if (s_max > 0.f) kern = attn_window_prefill_kernel<DK, DV, NCG, KS2, true, false>; }
  MI_CHECK(lds <= 160 * 1024, "windowed prefill attention: the distance table does not fit the LDS");
  if (lds > 64 * 1024) { int rc = ensure_dynamic_lds(reinterpret_cast<const void*>(kern), a.table ? 160 * 1024 : (int)lds); if (rc != MI_OK) return rc; }
  // kv head fastest: consecutive work-groups (one per XCD) read different heads, a head's tiles meet in one L2
  hipLaunchKernelGGL(kern, dim3(a.g.G, tiles), dim3(256 * KS2), lds, s, a, q, kpool, vpool, bs, bt, MB, sd, nseg, out, ldo, s_max, fold, min_rows, (bs & (bs - 1)) == 0 ? __builtin_ctz(bs) : -1, gt);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

// the built (dk, dv) sizes: the smallest that holds the layer's
#define MI_BY_SIZE(CALL)                                                          \
  do {                                                                            \
    const int dk_ = a.g.dkp, dv_ = a.g.dvp;                                       \
    if (dk_ <= 64 && dv_ <= 64) return CALL(64, 64, 2);                           \
    if (dk_ <= 64 && dv_ <= 128) return CALL(64, 128, 2);                         \
    if (dk_ <= 128 && dv_ <= 64) return CALL(128, 64, 2);                         \
    if (dk_ <= 128 && dv_ <= 128) return CALL(128, 128, 2);                       \
    return CALL(256, 256, 1);                                                     \
  } while (0)

}  // namespace

std::vector<int> distance_rows(int rows, double far, int limit) {
  std::vector<int> out;
  const int half = rows / 2;
  for (int n = 0; (limit <= 0 || n < limit) && out.size() < (1u << 24); ++n) {
    int b = n;
    // (a quotient that is a whole number in exact arithmetic may come out just below it)
    if (n >= half) b = half == 0 ? 0 : half + (int)std::min(std::floor(std::log((double)n / half) / std::log(far / half) * (rows - half) + 1e-9), (double)rows);
    out.push_back(std::min(b, rows - 1));
    if (out.back() == rows - 1) break;
  }
  return out;
}

bool attn_window_supported(const HeadGeom& g) { return g.dkp <= 256 && g.dvp <= 256 && g.H / g.G <= 64; }
bool attn_table_supported(const HeadGeom& g, int table_n) {
  // beside the largest tiles the size may take: two wave sets of 128-wide heads, one of 256-wide ones
  const size_t tiles = 2 * prefill_lds<128, 128>() > prefill_lds<256, 256>() ? 2 * prefill_lds<128, 128>() : prefill_lds<256, 256>();
  return tiles + (size_t)(g.H / g.G) * (63 + 128 + table_n) * 4 <= 160 * 1024;
}

size_t attn_window_scratch_bytes(int B, const HeadGeom& g) { return (size_t)B * g.H * kMaxSplits * (g.dvp + 2) * sizeof(float); }

int launch_attn_plain(const AttnSpec& a, const void* q, const void* kpool, const void* vpool, int bs, const int32_t* bt, int MB,
                      const int32_t* pos, const AttnSeg* segs, int nseg, int T, void* out, int ldo, bool f32, hipStream_t s, OutGate gate) {
  int rc = check_spec(a, bs);
  if (rc != MI_OK) return rc;
  MI_CHECK(!gate.per_element, "attention: gates per element are not built");
  MI_CHECK(T >= 1 && ldo >= a.g.H * a.g.dv && (segs == nullptr || nseg >= 1), "attention: rows / output stride");
  const size_t lds = 64 * 8 + (64 + (size_t)a.g.dk + a.g.dv) * 4;
  MI_CHECK(lds <= 64 * 1024, "attention: head sizes too large");
  const dim3 grid(T, a.g.H);
  if (f32) hipLaunchKernelGGL((attn_plain_kernel<float>), grid, dim3(64), lds, s, a, (const float*)q, (const float*)kpool, (const float*)vpool, bs, bt, MB, pos, segs, nseg, (float*)out, ldo, gate);
  else hipLaunchKernelGGL((attn_plain_kernel<uint16_t>), grid, dim3(64), lds, s, a, (const uint16_t*)q, (const uint16_t*)kpool, (const uint16_t*)vpool, bs, bt, MB, pos, segs, nseg, (uint16_t*)out, ldo, gate);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_attn_window_decode(const AttnSpec& a, const uint16_t* q, const uint16_t* kpool, const uint16_t* vpool, int bs, const int32_t* bt,
                              int MB, const int32_t* ctx, int B, int max_ctx, uint16_t* out, int ldo, void* scratch, hipStream_t s, OutGate gate) {
  int rc = check_spec(a, bs);
  if (rc != MI_OK) return rc;
  MI_CHECK(!gate.per_element, "windowed decode attention: gates per element are not built");
  MI_CHECK(attn_window_supported(a.g) && B >= 1 && max_ctx >= 1 && ldo >= a.g.H * a.g.dv, "windowed decode attention: shape");
  const bool ext = extended(a, gate);
  MI_CHECK(!ext || !a.slopes, "windowed decode attention: slopes beside chunks, tables, sinks or gates are not built");
#define MI_CALL_D(DK, DV, NCG) ext ? MI_CALL_DE(DK, DV, true) : MI_CALL_DE(DK, DV, false)
#define MI_CALL_DE(DK, DV, EXT) launch_decode_t<DK, DV, EXT>(a, q, kpool, vpool, bs, bt, MB, ctx, B, max_ctx, out, ldo, scratch, s, gate)
  MI_BY_SIZE(MI_CALL_D);
#undef MI_CALL_D
#undef MI_CALL_DE
}

int launch_attn_window_prefill(const AttnSpec& a, const uint16_t* q, const uint16_t* kpool, const uint16_t* vpool, int bs, const int32_t* bt,
                               int MB, const AttnSeg* sd, const AttnSeg* sh, int nseg, uint16_t* out, int ldo, hipStream_t s, int min_rows, OutGate gate) {
  int rc = check_spec(a, bs);
  if (rc != MI_OK) return rc;
  MI_CHECK(!gate.per_element, "windowed prefill attention: gates per element are not built");
  MI_CHECK(attn_window_supported(a.g) && nseg >= 1 && min_rows >= 2 && ldo >= a.g.H * a.g.dv && ((a.g.dv & 3) != 0 || ldo % 4 == 0), "windowed prefill attention: shape");
  // a grid that does not give every CU two work-groups takes tiles of half the queries, and two sets of waves to each
  int num_cu = 0, tiles = 0;
  rc = device_num_cu(&num_cu);
  if (rc != MI_OK) return rc;
  for (int i = 0; i < nseg; ++i) tiles += sh[i].n >= min_rows ? ceil_div(sh[i].n, 128 / (a.g.H / a.g.G)) : 0;
  const bool half = tiles * a.g.G < 2 * num_cu;
  const bool ext = extended(a, gate);
  MI_CHECK(!ext || !a.slopes, "windowed prefill attention: slopes beside chunks, tables, sinks or gates are not built");
#define MI_CALL_PE(DK, DV, NCG, EXT) \
  (half ? launch_prefill_t<DK, DV, 1, (DK > 192 || DV > 128 ? 1 : 2), EXT>(a, q, kpool, vpool, bs, bt, MB, sd, sh, nseg, out, ldo, s, min_rows, gate) \
        : launch_prefill_t<DK, DV, NCG, 1, EXT>(a, q, kpool, vpool, bs, bt, MB, sd, sh, nseg, out, ldo, s, min_rows, gate))
#define MI_CALL_P(DK, DV, NCG) ext ? MI_CALL_PE(DK, DV, NCG, true) : MI_CALL_PE(DK, DV, NCG, false)
  if (!ext && a.g.dkp > 128 && a.g.dkp <= 192 && a.g.dvp <= 128) return MI_CALL_PE(192, 128, 2, false);
  MI_BY_SIZE(MI_CALL_P);
#undef MI_CALL_PE
#undef MI_CALL_P
}

}  // namespace mi
