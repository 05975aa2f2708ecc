// Gated delta rule.  See delta_rule.h.
#include "delta_rule.h"

#include <algorithm>

namespace mi {

namespace {

constexpr int kC = kDeltaChunk;

__device__ __forceinline__ float silu(float v) { return v * __builtin_amdgcn_rcpf(1.f + __expf(-v)); }
__device__ __forceinline__ float gate(float v) { return __builtin_amdgcn_rcpf(1.f + __expf(-v)); }
__device__ __forceinline__ float sigmoid(float v) { return 1.f / (1.f + expf(-v)); }
// max(v, 0) + log(1 + w), w = exp(-|v|): the series where w is small (its first left-out term is w^5 / 5)
__device__ __forceinline__ float softplus(float v) {
  const float w = __expf(-fabsf(v)), series = w * (1.f - w * (0.5f - w * (1.f / 3.f - 0.25f * w)));
  return fmaxf(v, 0.f) + (w < 0.02f ? series : __logf(1.f + w));
}
__device__ __forceinline__ float log_decay(float z, float dt, float a_log) { return -expf(a_log) * softplus(z + dt); }
__device__ __forceinline__ void put1(uint16_t* p, float v) { *p = f32_to_bf16(v); }
__device__ __forceinline__ void put1(float* p, float v) { *p = v; }

// ---- token generation ---------------------------------------------------------------------------------------------------------
// One work-group per (head, row): the whole state of the head in registers, requested first; thread (vq, dg) owns columns
// 4 vq .. + 3 of rows dg RPT .. + RPT - 1.  Both products with the decayed state are taken in one pass (o = S^T q + (k.q) u).
constexpr int kTokenThreads = 512;
template <typename T, int VQ, int RPT>
__global__ __launch_bounds__(kTokenThreads) void delta_token_kernel(DeltaGeom g, DeltaIn in, const AttnSeg* __restrict__ segs, T* __restrict__ y, int ldy) {
  constexpr int NW = kTokenThreads / 64;
  __shared__ float qs[256], ks[256], gs[256], vs[256];
  __shared__ float norms[3];
  __shared__ __attribute__((aligned(16))) float red[2][NW][VQ * 4];
  const int h = blockIdx.x, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  int row = blockIdx.y, seq = blockIdx.y;
  if (segs) {
    const AttnSeg sg = segs[blockIdx.y];
    if (sg.n != 1) return;
    row = sg.row0; seq = sg.seq;
  }
  const int slot = in.slots[seq], p = in.pos[row], vq = tid % VQ, dg = tid / VQ;
  const bool vin = vq * 4 < g.dvp;
  float* S0 = in.state + ((size_t)slot * g.H + h) * g.dkp * g.dvp + vq * 4;
  float4 S[RPT];
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int d = dg * RPT + i;
    S[i] = p > 0 && vin && d < g.dkp ? *reinterpret_cast<const float4*>(S0 + (size_t)d * g.dvp) : make_float4(0.f, 0.f, 0.f, 0.f);
  }
  // convolutions of the head's channels; position p goes to a row of the ring that nobody reads in this launch
  const int C = g.channels(), r = g.H / g.G, kvh = h / r;
  const float* x = in.proj + (size_t)row * in.ldp;
  float* ring = in.ring + (size_t)slot * g.taps * C;
  for (int i = tid; i < 2 * g.dk + g.dv; i += kTokenThreads) {
    const int part = i < g.dk ? 0 : i < 2 * g.dk ? 1 : 2, d = i - part * g.dk;
    const int ch = part == 2 ? 2 * g.G * g.dk + h * g.dv + d : (part * g.G + kvh) * g.dk + d;
    const float now = x[ch];
    float a = 0.f;
    for (int j = 0; j + 1 < g.taps; ++j) {
      const int q = p - (g.taps - 1 - j);
      if (q >= 0) a = __builtin_fmaf(in.conv[(size_t)j * C + ch], ring[(size_t)(q % g.taps) * C + ch], a);
    }
    a = silu(__builtin_fmaf(in.conv[(size_t)(g.taps - 1) * C + ch], now, a));
    if (part == 2 || h % r == 0) ring[(size_t)(p % g.taps) * C + ch] = now;
    (part == 0 ? qs : part == 1 ? ks : vs)[d] = a;
  }
  for (int d = tid; d < g.dkp; d += kTokenThreads) {
    if (d >= g.dk) { qs[d] = ks[d] = 0.f; gs[d] = 1.f; continue; }
    gs[d] = expf(log_decay(in.z[(size_t)row * in.ldz + h * g.dk + d], in.dt[h * g.dk + d], in.a_log[h]));
  }
  for (int d = g.dv + tid; d < g.dvp; d += kTokenThreads) vs[d] = 0.f;
  const float beta = sigmoid(x[in.beta + h]);
  __syncthreads();
  if (wave < 3) {
    float s = 0.f;
    for (int d = lane; d < g.dk; d += 64) s = __builtin_fmaf(wave == 1 ? ks[d] : qs[d], wave == 0 ? qs[d] : ks[d], s);
    s = wave_sum(s);
    if (lane == 0) norms[wave] = s;
  }
  __syncthreads();
  const float fq = 1.f / sqrtf(norms[0] + 1e-6f) * (1.f / sqrtf((float)g.dk)), fk = 1.f / sqrtf(norms[1] + 1e-6f), qk = norms[2] * fq * fk;
  float4 r1 = make_float4(0.f, 0.f, 0.f, 0.f), r2 = r1;
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int d = dg * RPT + i;
    if (d >= g.dkp) continue;
    const float gd = gs[d], kd = ks[d] * fk, qd = qs[d] * fq;
    S[i].x *= gd; S[i].y *= gd; S[i].z *= gd; S[i].w *= gd;
    r1.x = __builtin_fmaf(S[i].x, kd, r1.x); r1.y = __builtin_fmaf(S[i].y, kd, r1.y); r1.z = __builtin_fmaf(S[i].z, kd, r1.z); r1.w = __builtin_fmaf(S[i].w, kd, r1.w);
    r2.x = __builtin_fmaf(S[i].x, qd, r2.x); r2.y = __builtin_fmaf(S[i].y, qd, r2.y); r2.z = __builtin_fmaf(S[i].z, qd, r2.z); r2.w = __builtin_fmaf(S[i].w, qd, r2.w);
  }
#pragma unroll
  for (int m = VQ; m < 64; m *= 2) {
    r1.x += __shfl_xor(r1.x, m); r1.y += __shfl_xor(r1.y, m); r1.z += __shfl_xor(r1.z, m); r1.w += __shfl_xor(r1.w, m);
    r2.x += __shfl_xor(r2.x, m); r2.y += __shfl_xor(r2.y, m); r2.z += __shfl_xor(r2.z, m); r2.w += __shfl_xor(r2.w, m);
  }
  if (lane < VQ) {
    *reinterpret_cast<float4*>(&red[0][wave][vq * 4]) = r1;
    *reinterpret_cast<float4*>(&red[1][wave][vq * 4]) = r2;
  }
  __syncthreads();
  r1 = make_float4(0.f, 0.f, 0.f, 0.f);
  r2 = r1;
#pragma unroll
  for (int w = 0; w < NW; ++w) {
    const float4 a = *reinterpret_cast<const float4*>(&red[0][w][vq * 4]), b = *reinterpret_cast<const float4*>(&red[1][w][vq * 4]);
    r1.x += a.x; r1.y += a.y; r1.z += a.z; r1.w += a.w;
    r2.x += b.x; r2.y += b.y; r2.z += b.z; r2.w += b.w;
  }
  if (!vin) r1 = r2 = make_float4(0.f, 0.f, 0.f, 0.f);
  float4 u = make_float4(0.f, 0.f, 0.f, 0.f);
  if (vin) u = make_float4(beta * (vs[vq * 4] - r1.x), beta * (vs[vq * 4 + 1] - r1.y), beta * (vs[vq * 4 + 2] - r1.z), beta * (vs[vq * 4 + 3] - r1.w));
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int d = dg * RPT + i;
    if (!vin || d >= g.dkp) continue;
    const float kd = ks[d] * fk;
    S[i].x = __builtin_fmaf(kd, u.x, S[i].x); S[i].y = __builtin_fmaf(kd, u.y, S[i].y); S[i].z = __builtin_fmaf(kd, u.z, S[i].z); S[i].w = __builtin_fmaf(kd, u.w, S[i].w);
    *reinterpret_cast<float4*>(S0 + (size_t)d * g.dvp) = S[i];
  }
  if (wave) return;                                  // (VQ <= 64 lanes of the first wave hold every column)
  float o[4] = {__builtin_fmaf(qk, u.x, r2.x), __builtin_fmaf(qk, u.y, r2.y), __builtin_fmaf(qk, u.z, r2.z), __builtin_fmaf(qk, u.w, r2.w)};
  float ss = lane < VQ ? (o[0] * o[0] + o[1] * o[1]) + (o[2] * o[2] + o[3] * o[3]) : 0.f;     // (padding columns are zero)
  ss = wave_sum(ss);
  const float f = 1.f / sqrtf(ss / (float)g.dv + in.eps);
  if (lane >= VQ) return;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int v = vq * 4 + i;
    if (v < g.dv) put1(y + (size_t)row * ldy + h * g.dv + v, o[i] * f * in.norm[v] * gate(in.z[(size_t)row * in.ldz + in.gate + h * g.dv + v]));
  }
}

// ---- prompts: the chunks of a ragged batch ------------------------------------------------------------------------------------
struct ChunkAt { AttnSeg sg; int t0, n; bool ok, last; };     // rows t0 .. + n of the segment
__device__ __forceinline__ ChunkAt chunk_at(const AttnSeg* segs, int nseg, int c) {
  for (int i = 0; i < nseg; ++i) {
    const AttnSeg sg = segs[i];
    if (sg.n < 2) continue;
    const int k = ceil_div(sg.n, kC);
    if (c < k) return ChunkAt{sg, c * kC, min(kC, sg.n - c * kC), true, c == k - 1};
    c -= k;
  }
  return ChunkAt{AttnSeg{0, 0, 0, 0}, 0, 0, false, false};
}

// The record of a chunk and head, in floats: -W, Q', K' as [dkp / 16] tiles of 16 x 16 (W, Q': token x channel; K': channel x token),
// exp L_end [dkp], T and P T [16][16], and [dvp / 16] tiles (token x column) of values that the scan replaces by outputs.  A head's
// records follow each other: the scan reads on without a gap.
struct Factors { float *w, *q, *k, *e, *t, *m, *v; };
__host__ __device__ __forceinline__ size_t record_floats(int dkp, int dvp) { return (size_t)49 * dkp + 512 + 16 * dvp; }
__device__ __forceinline__ Factors factors_at(float* base, size_t index, int dkp, int dvp) {
  float* p = base + index * record_floats(dkp, dvp);
  return Factors{p, p + 16 * dkp, p + 32 * dkp, p + 48 * dkp, p + 49 * dkp, p + 49 * dkp + 256, p + 49 * dkp + 512};
}

// where the input of a convolution `i` rows behind the segment's start lies (negative: ahead of it; ahead of the sequence: anywhere
// valid, conv_known is false).  Addresses are selected, not branched over: loads stay in flight together.
__device__ __forceinline__ const float* conv_at(const DeltaIn& in, const AttnSeg& sg, const float* ring, int taps, int C, int ch, int i) {
  const int p = max(sg.pos0 + i, 0) % taps;
  const float *a = in.proj + (size_t)(sg.row0 + max(i, 0)) * in.ldp + ch, *b = ring + (size_t)p * C + ch;
  return i >= 0 ? a : b;
}
__device__ __forceinline__ bool conv_known(const AttnSeg& sg, int i) { return sg.pos0 + i >= 0; }
__device__ __forceinline__ float conv_in(const DeltaIn& in, const AttnSeg& sg, const float* ring, int taps, int C, int ch, int i) {
  const float v = *conv_at(in, sg, ring, taps, C, ch, i);
  return conv_known(sg, i) ? v : 0.f;
}

// LDS written by some lanes of a wave, read by others of it
__device__ __forceinline__ void wave_order() {
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  __builtin_amdgcn_wave_barrier();
}
constexpr int kPairTiles = 36, kPairParts = 7;

template <int TAPS>
__global__ __launch_bounds__(256) void delta_factors_kernel(DeltaGeom g, DeltaIn in, const AttnSeg* __restrict__ segs, int nseg, int c0, float* __restrict__ out) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int pitch = g.dkp + 4;
  float *qs = sm, *ks = qs + kC * pitch, *Ls = ks + kC * pitch, *gs = Ls + kC * pitch, *red = gs;   // (red: in place of gs once that is used up)
  __shared__ float As[kC][kC + 1], Ps[kC][kC + 1], Ts[kC][kC + 1], Ms[kC][kC + 1], bs[kC], rn[2 * kC];
  const ChunkAt at = chunk_at(segs, nseg, c0 + blockIdx.x);
  if (!at.ok) return;
  const int h = blockIdx.y, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, n = at.n, C = g.channels(), kvh = h / (g.H / g.G);
  const Factors F = factors_at(out, (size_t)h * gridDim.x + blockIdx.x, g.dkp, g.dvp);
  const float* ring = in.ring + (size_t)in.slots[at.sg.seq] * g.taps * C;
  const float* rows = in.proj + (size_t)(at.sg.row0 + at.t0) * in.ldp;
  // Convolutions: a thread walks channels of q, k and v down half the chunk, kItems of them at a time; their inputs and the decays' are
  // requested together.
  constexpr int kHalf = kC / 2, kItems = 3, kZ = 8, NX = TAPS > 0 ? kHalf + TAPS - 1 : 1, NW = TAPS > 0 ? TAPS : 1;
  const int cols = 2 * g.dkp + g.dvp;
  struct Item { int t0, d, ch, size; bool v; float* dst; int step; };
  auto item = [&](int i) {
    Item x;
    x.t0 = i < cols ? 0 : kHalf;
    const int col = i < cols ? i : min(i - cols, cols - 1), part = col < g.dkp ? 0 : col < 2 * g.dkp ? 1 : 2;
    x.d = col - part * g.dkp;
    x.v = part == 2;
    x.size = x.v ? g.dv : g.dk;
    x.ch = (x.v ? 2 * g.G * g.dk + h * g.dv : (part * g.G + kvh) * g.dk) + min(x.d, x.size - 1);
    x.dst = x.v ? F.v + (x.d >> 4) * 256 + (x.d & 15) : (part ? ks : qs) + x.d;
    x.step = x.v ? 16 : pitch;
    return x;
  };
  // decays: thread = channel zd of tokens zt0, zt0 + zn, ...
  const float decay = expf(in.a_log[h]);
  const int zn = 256 / g.dkp, zt0 = tid / g.dkp, zd = tid - zt0 * g.dkp, zdc = min(zd, g.dk - 1);
  const bool zin = zt0 < zn;
  const float* zr = in.z + (size_t)(at.sg.row0 + at.t0) * in.ldz + h * g.dk;
  const float zdt = in.dt[h * g.dk + zdc];
  auto put_decay = [&](int t, float z) { Ls[t * pitch + zd] = zd < g.dk && t < n ? -decay * softplus(z + zdt) : 0.f; };
  float z0[kZ];
#pragma unroll
  for (int u = 0; u < kZ; ++u) z0[u] = zr[(uint32_t)min(zt0 + u * zn, n - 1) * in.ldz + zdc];
  const bool inside = at.t0 >= TAPS - 1 && n == kC;      // every input is a row of the batch: no clamps, no ring
  for (int base = 0; base < 2 * cols; base += kItems * 256) {
    float x[kItems][NX], w[kItems][NW];
    if constexpr (TAPS > 0) {
      if (inside) {
        const float* from = rows - (size_t)(TAPS - 1) * in.ldp;
#pragma unroll
        for (int p = 0; p < kItems; ++p) {
          const Item it = item(base + p * 256 + tid);
          uint32_t off = (uint32_t)it.t0 * in.ldp + it.ch;
#pragma unroll
          for (int k = 0; k < NX; ++k, off += in.ldp) x[p][k] = *reinterpret_cast<const float*>(reinterpret_cast<const unsigned char*>(from) + off * 4);
        }
      } else {
#pragma unroll
        for (int p = 0; p < kItems; ++p) {
          const Item it = item(base + p * 256 + tid);
#pragma unroll
          for (int k = 0; k < NX; ++k) x[p][k] = conv_in(in, at.sg, ring, TAPS, C, it.ch, at.t0 + min(it.t0 + k - (TAPS - 1), n - 1));
        }
      }
#pragma unroll
      for (int p = 0; p < kItems; ++p) {
        const int ch = item(base + p * 256 + tid).ch;
#pragma unroll
        for (int j = 0; j < TAPS; ++j) w[p][j] = in.conv[(uint32_t)j * C + ch];
      }
    }
#pragma unroll
    for (int p = 0; p < kItems; ++p) {
      const int i = base + p * 256 + tid;
      if (i >= 2 * cols) continue;
      const Item it = item(i);
#pragma unroll
      for (int t = 0; t < kHalf; ++t) {
        float a = 0.f;
        if constexpr (TAPS > 0) {
#pragma unroll
          for (int j = 0; j < TAPS; ++j) a = __builtin_fmaf(w[p][j], x[p][t + j], a);
        } else {
          for (int j = 0; j < g.taps; ++j)
            a = __builtin_fmaf(in.conv[(size_t)j * C + it.ch], conv_in(in, at.sg, ring, g.taps, C, it.ch, at.t0 + min(it.t0 + t, n - 1) - (g.taps - 1 - j)), a);
        }
        it.dst[(it.t0 + t) * it.step] = it.t0 + t < n && it.d < it.size ? silu(a) : 0.f;
      }
    }
  }
  if (zin) {
#pragma unroll
    for (int u = 0; u < kZ; ++u)
      if (zt0 + u * zn < kC) put_decay(zt0 + u * zn, z0[u]);
    for (int t = zt0 + kZ * zn; t < kC; t += zn) put_decay(t, zr[(uint32_t)min(t, n - 1) * in.ldz + zdc]);
  }
  if (tid < kC) bs[tid] = tid < n ? sigmoid(rows[(size_t)tid * in.ldp + in.beta + h]) : 0.f;
  __syncthreads();
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const int v = wave * 8 + i;
    const float* r = (v < kC ? qs : ks) + (v & (kC - 1)) * pitch;
    float s = 0.f;
    for (int d = lane; d < g.dkp; d += 64) s = __builtin_fmaf(r[d], r[d], s);
    s = wave_sum(s);
    if (lane == 0) rn[v] = 1.f / sqrtf(s + 1e-6f) * (v < kC ? 1.f / sqrtf((float)g.dk) : 1.f);
  }
  for (int d = tid; d < g.dkp; d += 256) {           // running sums of the decays' logarithms, the decays beside them
    float L = 0.f, lg[kC];
#pragma unroll
    for (int t = 0; t < kC; ++t) lg[t] = Ls[t * pitch + d];
#pragma unroll
    for (int t = 0; t < kC; ++t) {
      L += lg[t];
      Ls[t * pitch + d] = L;
      gs[t * pitch + d] = __expf(lg[t]);
    }
  }
  __syncthreads();
  for (int i = tid; i < 2 * kC * (g.dkp / 4); i += 256) {
    const int v = i / (g.dkp / 4), d = (i % (g.dkp / 4)) * 4;
    float4* r = reinterpret_cast<float4*>((v < kC ? qs : ks) + (v & (kC - 1)) * pitch + d);
    float4 x = *r;
    const float f = rn[v];
    *r = make_float4(x.x * f, x.y * f, x.z * f, x.w * f);
  }
  __syncthreads();
  // pairs: a thread takes one of the 36 tiles of tokens (2 I, 2 I + 1) x (2 J, 2 J + 1), J <= I, and every seventh group of four channels
  float a[4] = {0.f, 0.f, 0.f, 0.f}, p[4] = {0.f, 0.f, 0.f, 0.f};        // (i0,j0) (i0,j1) (i1,j0) (i1,j1)
  const int part = tid / kPairTiles, tl = tid - part * kPairTiles;
  if (part < kPairParts) {
    int I = 0;
#pragma unroll
    for (int k = 1; k < 8; ++k) I += tl >= k * (k + 1) / 2 ? 1 : 0;
    const int J = tl - I * (I + 1) / 2, i0 = 2 * I, j0 = 2 * J;
    const bool diag = I == J;
    for (int d = part * 4; d < g.dkp; d += 4 * kPairParts) {
      const float4 ki0 = *reinterpret_cast<const float4*>(ks + i0 * pitch + d), ki1 = *reinterpret_cast<const float4*>(ks + (i0 + 1) * pitch + d);
      const float4 qi0 = *reinterpret_cast<const float4*>(qs + i0 * pitch + d), qi1 = *reinterpret_cast<const float4*>(qs + (i0 + 1) * pitch + d);
      const float4 kj0 = *reinterpret_cast<const float4*>(ks + j0 * pitch + d), kj1 = *reinterpret_cast<const float4*>(ks + (j0 + 1) * pitch + d);
      const float4 Li = *reinterpret_cast<const float4*>(Ls + i0 * pitch + d), Lj = *reinterpret_cast<const float4*>(Ls + (j0 + 1) * pitch + d);
      const float4 gi = *reinterpret_cast<const float4*>(gs + (i0 + 1) * pitch + d), gj = *reinterpret_cast<const float4*>(gs + (j0 + 1) * pitch + d);
      auto one = [&](float k0, float k1, float q0, float q1, float c0, float c1, float li, float lj, float g1, float h1) {
        const float e = __expf(li - lj);                   // (diagonal tiles: the entry above the diagonal, left out below)
        const float e11 = diag ? 1.f : e * g1, e00 = diag ? 1.f : e * h1;
        const float x00 = c0 * e00, x01 = c1 * e, x10 = x00 * g1, x11 = c1 * e11;
        a[0] = __builtin_fmaf(k0, x00, a[0]); a[1] = __builtin_fmaf(k0, x01, a[1]); a[2] = __builtin_fmaf(k1, x10, a[2]); a[3] = __builtin_fmaf(k1, x11, a[3]);
        p[0] = __builtin_fmaf(q0, x00, p[0]); p[1] = __builtin_fmaf(q0, x01, p[1]); p[2] = __builtin_fmaf(q1, x10, p[2]); p[3] = __builtin_fmaf(q1, x11, p[3]);
      };
      one(ki0.x, ki1.x, qi0.x, qi1.x, kj0.x, kj1.x, Li.x, Lj.x, gi.x, gj.x);
      one(ki0.y, ki1.y, qi0.y, qi1.y, kj0.y, kj1.y, Li.y, Lj.y, gi.y, gj.y);
      one(ki0.z, ki1.z, qi0.z, qi1.z, kj0.z, kj1.z, Li.z, Lj.z, gi.z, gj.z);
      one(ki0.w, ki1.w, qi0.w, qi1.w, kj0.w, kj1.w, Li.w, Lj.w, gi.w, gj.w);
    }
  }
  __syncthreads();
  if (part < kPairParts) {
    float4* r = reinterpret_cast<float4*>(red + tid * 8);
    r[0] = make_float4(a[0], a[1], a[2], a[3]);
    r[1] = make_float4(p[0], p[1], p[2], p[3]);
  }
  // k exp L and q exp L in place of k and q, K' out: a thread takes eight tokens of a channel
  for (int u = tid; u < 2 * g.dkp; u += 256) {
    const int d = u < g.dkp ? u : u - g.dkp, t0 = u < g.dkp ? 0 : 8;
    const float end = Ls[(kC - 1) * pitch + d];
    float o[8];
#pragma unroll
    for (int t = 0; t < 8; ++t) {
      const int r = (t0 + t) * pitch + d;
      const float L = Ls[r], e = __expf(L), k = ks[r];
      o[t] = k * __expf(end - L);
      ks[r] = k * e;
      qs[r] *= e;
    }
    float* kt = F.k + (d >> 4) * 256 + (d & 15) * 16 + t0;
    *reinterpret_cast<float4*>(kt) = make_float4(o[0], o[1], o[2], o[3]);
    *reinterpret_cast<float4*>(kt + 4) = make_float4(o[4], o[5], o[6], o[7]);
    if (t0 == 0) F.e[d] = __expf(end);
  }
  __syncthreads();
  {
    const int i = tid >> 4, j = tid & 15, I = i >> 1, J = j >> 1, at8 = (I * (I + 1) / 2 + J) * 8 + (i & 1) * 2 + (j & 1);
    float av = 0.f, pv = 0.f;
    if (j <= i) {
#pragma unroll
      for (int w = 0; w < kPairParts; ++w) { av += red[w * kPairTiles * 8 + at8]; pv += red[w * kPairTiles * 8 + at8 + 4]; }
    }
    As[i][j] = j < i ? av * bs[i] : 0.f;
    Ps[i][j] = j <= i ? pv : 0.f;
    Ts[i][j] = 0.f;
  }
  __syncthreads();
  if (wave == 0) {   // X = (I + A)^-1: the two diagonal blocks by forward substitution, a lane per column; X21 = -X22 A21 X11
    if (lane < kC) {
      const int b8 = lane & 8, j = lane & 7;
      float x[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        float v = i == j ? 1.f : 0.f;
#pragma unroll
        for (int m = 0; m < i; ++m) v = __builtin_fmaf(-As[b8 + i][b8 + m], x[m], v);
        x[i] = v;
      }
#pragma unroll
      for (int i = 0; i < 8; ++i) Ts[b8 + i][b8 + j] = x[i];
    }
    wave_order();
    const int i = lane >> 3, j = lane & 7;
    float y = 0.f;
#pragma unroll
    for (int m = 0; m < 8; ++m) y = __builtin_fmaf(As[8 + i][m], Ts[m][j], y);
    Ms[i][j] = y;
    wave_order();
    y = 0.f;
#pragma unroll
    for (int m = 0; m < 8; ++m) y = __builtin_fmaf(-Ts[8 + i][8 + m], Ms[m][j], y);
    wave_order();
    Ts[8 + i][j] = y;
  }
  __syncthreads();
  if (tid < kC * kC) Ts[tid >> 4][tid & 15] *= bs[tid & 15];
  __syncthreads();
  {
    const int i = tid >> 4, j = tid & 15;
    float m = 0.f;
#pragma unroll
    for (int k = 0; k < kC; ++k) m = __builtin_fmaf(Ps[i][k], Ts[k][j], m);
    Ms[i][j] = m;
    F.t[tid] = Ts[i][j];
    F.m[tid] = m;
  }
  __syncthreads();
  const int g4 = lane >> 4, c = lane & 15;
  for (int t = wave; t < g.dkp / 16; t += 4) {
    f32x4_t w = {0.f, 0.f, 0.f, 0.f}, q = w;
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      const float b = ks[(4 * s + g4) * pitch + 16 * t + c];
      w = __builtin_amdgcn_mfma_f32_16x16x4f32(Ts[c][4 * s + g4], b, w, 0, 0, 0);
      q = __builtin_amdgcn_mfma_f32_16x16x4f32(Ms[c][4 * s + g4], b, q, 0, 0, 0);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 4 * g4 + r;
      F.w[t * 256 + i * 16 + c] = -w[r];
      F.q[t * 256 + i * 16 + c] = qs[i * pitch + 16 * t + c] - q[r];
    }
  }
}

// One work-group per (head, 16 value columns, segment): the chunks of the segment in order.  A wave holds NT 16-channel tiles of the
// state as MFMA accumulators, which are the B operands of the next chunk's products as they stand; the partial sums of u and
// o over the channels meet in LDS, once per chunk.
template <int NT>
__global__ __launch_bounds__(256) void delta_scan_kernel(DeltaGeom g, float* __restrict__ state, const int32_t* __restrict__ slots,
                                                         const AttnSeg* __restrict__ segs, int c0, int nchunks, int nvt, float* __restrict__ records) {
  __shared__ f32x4_t ps[2][2][4][64];
  int id = blockIdx.x, h, vt;
  if (g.H % 8 == 0) {        // the column blocks of a head on one XCD: they read the same factors
    const int k = id >> 3;
    h = (id & 7) + 8 * (k / nvt);
    vt = k % nvt;
  } else {
    h = id / nvt;
    vt = id % nvt;
  }
  const int si = blockIdx.y;
  const AttnSeg sg = segs[si];
  if (sg.n < 2) return;
  int first = 0;             // the segment's first chunk among all
  for (int i = 0; i < si; ++i) first += segs[i].n < 2 ? 0 : ceil_div(segs[i].n, kC);
  const int k0 = max(c0 - first, 0), k1 = min(c0 + nchunks - first, ceil_div(sg.n, kC));
  if (k0 >= k1) return;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63, g4 = lane >> 4, c = lane & 15, tiles = g.dkp / 16;
  float* S0 = state + ((size_t)slots[sg.seq] * g.H + h) * g.dkp * g.dvp + vt * 16 + c;
  f32x4_t S[NT];
  // Factors and values of the next kAhead chunks are in flight.  Addresses: a uniform part that moves from chunk to chunk and lane
  // offsets (bytes) that do not.
  constexpr int kAhead = NT <= 2 ? 4 : 2;
  struct Frag { f32x4_t w[NT], q[NT], k[NT], e[NT]; float t, m, x; };
  uint32_t off[NT], eoff[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const int tile = wave * NT + t, tl = min(tile, tiles - 1);            // (past the last tile: S stays zero)
    off[t] = (tl * 256 + c * 16 + 4 * g4) * 4;
    eoff[t] = (tl * 16 + 4 * g4) * 4;
#pragma unroll
    for (int r = 0; r < 4; ++r) S[t][r] = sg.pos0 + k0 > 0 && tile < tiles ? S0[(size_t)(tile * 16 + 4 * g4 + r) * g.dvp] : 0.f;
  }
  const uint32_t toff = (c * 16 + 4 * wave + g4) * 4, xoff = ((4 * wave + g4) * 16 + c) * 4, ooff = ((4 * g4 + wave) * 16 + c) * 4;
  auto at = [](float* base, uint32_t bytes) { return reinterpret_cast<unsigned char*>(base) + bytes; };
  auto record = [&](int k) { return factors_at(records, (size_t)h * nchunks + (first + k - c0), g.dkp, g.dvp); };
  auto load_w = [&](const Factors& F, Frag& f, int t) { f.w[t] = *reinterpret_cast<const f32x4_t*>(at(F.w, off[t])); };
  auto load_q = [&](const Factors& F, Frag& f, int t) { f.q[t] = *reinterpret_cast<const f32x4_t*>(at(F.q, off[t])); };
  auto load_k = [&](const Factors& F, Frag& f, int t) { f.k[t] = *reinterpret_cast<const f32x4_t*>(at(F.k, off[t])); };
  auto load_e = [&](const Factors& F, Frag& f, int t) { f.e[t] = *reinterpret_cast<const f32x4_t*>(at(F.e, eoff[t])); };
  auto load_rest = [&](const Factors& F, Frag& f, int i) {
    if (i == 0) f.t = *reinterpret_cast<const float*>(at(F.t, toff));
    if (i == 1) f.m = *reinterpret_cast<const float*>(at(F.m, toff));
    if (i == 2) f.x = *reinterpret_cast<const float*>(at(F.v + vt * 256, xoff));
  };
  auto load = [&](int k, Frag& f) {
    const Factors F = record(k);
#pragma unroll
    for (int t = 0; t < NT; ++t) { load_w(F, f, t); load_q(F, f, t); load_k(F, f, t); load_e(F, f, t); }
#pragma unroll
    for (int i = 0; i < 3; ++i) load_rest(F, f, i);
  };
  auto meet = [] {      // one barrier a chunk, for LDS alone: the loads of later chunks stay in flight across it
    __builtin_amdgcn_sched_barrier(0);
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
    __builtin_amdgcn_sched_barrier(0);
  };
  auto emit = [&](int k, int b) {      // a chunk's output in place of its values: its partial sums lie in ps[b][1]
    const float* po = reinterpret_cast<const float*>(&ps[b][1][0][0]);
    float s = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) s += po[(w * 64 + lane) * 4 + wave];
    *reinterpret_cast<float*>(at(record(k).v + vt * 256, ooff)) = s;
  };
  f32x4_t ov = {0.f, 0.f, 0.f, 0.f};
  // u's partial sums go out first; o's products and the scaling of S run while they do.  o's own meet at the next chunk's barrier.
  // A CU takes a wave's 16-byte loads in at one per 16 clocks: they are dealt out between the products, each as soon as what it
  // replaces is used up (K' and exp L_end of the chunk before behind the first products).
  auto pin = [] { __builtin_amdgcn_sched_barrier(0x6); };       // (ALU instructions may cross)
  auto step = [&](int k, Frag& f, Frag& before, bool more, bool more_before) {
    const int b = k & 1;
    const Factors Fn = record(k + kAhead), Fb = record(k - 1 + kAhead);
    f32x4_t u = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int t = 0; t < NT; ++t) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        u = __builtin_amdgcn_mfma_f32_16x16x4f32(f.w[t][r], S[t][r], u, 0, 0, 0);
        if (r & 1) {
          pin();
          if (more_before) { if (r == 1) load_k(Fb, before, t); else load_e(Fb, before, t); }
          pin();
        }
      }
    }
    u = __builtin_amdgcn_mfma_f32_16x16x4f32(f.t, f.x, u, 0, 0, 0);
    ps[b][1][wave][lane] = ov;
    ps[b][0][wave][lane] = u;
    pin();
    ov = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int t = 0; t < NT; ++t) {
#pragma unroll
      for (int r = 0; r < 4; ++r) ov = __builtin_amdgcn_mfma_f32_16x16x4f32(f.q[t][r], S[t][r], ov, 0, 0, 0);
      pin();
      if (more) load_w(Fn, f, t);
      pin();
    }
    ov = __builtin_amdgcn_mfma_f32_16x16x4f32(f.m, f.x, ov, 0, 0, 0);
    f32x4_t Sg[NT];
#pragma unroll
    for (int t = 0; t < NT; ++t) Sg[t] = f32x4_t{S[t][0] * f.e[t][0], S[t][1] * f.e[t][1], S[t][2] * f.e[t][2], S[t][3] * f.e[t][3]};
    meet();
    u = ps[b][0][0][lane];
#pragma unroll
    for (int w = 1; w < 4; ++w) {
      const f32x4_t a = ps[b][0][w][lane];
      u[0] += a[0]; u[1] += a[1]; u[2] += a[2]; u[3] += a[3];
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
#pragma unroll
      for (int t = 0; t < NT; ++t)     // (a tile past the last one stays zero)
        Sg[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(wave * NT + t < tiles ? f.k[t][r] : 0.f, u[r], Sg[t], 0, 0, 0);
      pin();
      if (more) {
        if (r < NT) load_q(Fn, f, r);
        if (r < 3) load_rest(Fn, f, r);
      }
      pin();
    }
#pragma unroll
    for (int t = 0; t < NT; ++t) S[t] = Sg[t];
    if (k > k0) emit(k - 1, b);
  };
  Frag f[kAhead];
#pragma unroll
  for (int i = 0; i < kAhead; ++i) load(min(k0 + i, k1 - 1), f[i]);
  int k = k0;
  for (; k + 2 * kAhead <= k1; k += kAhead) {
#pragma unroll
    for (int i = 0; i < kAhead; ++i) step(k + i, f[i], f[(i + kAhead - 1) % kAhead], true, i > 0 || k > k0);
  }
  // up to 2 kAhead - 1 chunks are left
  const bool was = k > k0;
  for (int j = 0; j < 2; ++j) {
#pragma unroll
    for (int i = 0; i < kAhead; ++i) {
      const int n = k + j * kAhead + i;
      if (n < k1) step(n, f[i], f[(i + kAhead - 1) % kAhead], n + kAhead < k1, (n > k || was) && n - 1 + kAhead < k1);
    }
  }
  ps[k1 & 1][1][wave][lane] = ov;
  __syncthreads();
  emit(k1 - 1, k1 & 1);
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r)
      if (wave * NT + t < tiles) S0[(size_t)((wave * NT + t) * 16 + 4 * g4 + r) * g.dvp] = S[t][r];
}

// norm and gate: a wave per head, eight (four) of the chunk's tokens at a time; the work-groups of a segment's last chunk renew its ring
template <typename T, int NV>
__global__ __launch_bounds__(256) void delta_out_kernel(DeltaGeom g, DeltaIn in, const AttnSeg* __restrict__ segs, int nseg, int c0, float* __restrict__ records,
                                                        T* __restrict__ y, int ldy) {
  const ChunkAt at = chunk_at(segs, nseg, c0 + blockIdx.x);
  if (!at.ok) return;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, h = blockIdx.y * 4 + wave;
  if (h < g.H) {
    float nw[NV];
#pragma unroll
    for (int i = 0; i < NV; ++i) nw[i] = in.norm[min(lane + 64 * i, g.dv - 1)];
    const size_t row0 = at.sg.row0 + at.t0;
    const float *src = factors_at(records, (size_t)h * gridDim.x + blockIdx.x, g.dkp, g.dvp).v, *zr = in.z + row0 * in.ldz + in.gate + h * g.dv;
    constexpr int TB = NV <= 2 ? 8 : 4;
    for (int t0 = 0; t0 < at.n; t0 += TB) {
      float x[TB][NV], z[TB][NV];
#pragma unroll
      for (int t = 0; t < TB; ++t)
#pragma unroll
        for (int i = 0; i < NV; ++i) {
          const int r = min(t0 + t, at.n - 1), v = min(lane + 64 * i, g.dv - 1);
          x[t][i] = src[(v >> 4) * 256 + r * 16 + (v & 15)];
          z[t][i] = zr[(size_t)r * in.ldz + v];
        }
#pragma unroll
      for (int t = 0; t < TB; ++t) {
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < NV; ++i) ss = __builtin_fmaf(x[t][i], lane + 64 * i < g.dv ? x[t][i] : 0.f, ss);
        const float f = 1.f / sqrtf(wave_sum(ss) / (float)g.dv + in.eps);
        if (t0 + t >= at.n) break;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
          const int v = lane + 64 * i;
          if (v < g.dv) put1(y + (row0 + t0 + t) * ldy + h * g.dv + v, x[t][i] * f * nw[i] * gate(z[t][i]));
        }
      }
    }
  }
  if (!at.last) return;
  const int C = g.channels();
  float* ring = in.ring + (size_t)in.slots[at.sg.seq] * g.taps * C;
  for (int ch = blockIdx.y * 256 + threadIdx.x; ch < C; ch += gridDim.y * 256)
    for (int i = max(0, at.sg.n - g.taps); i < at.sg.n; ++i)
      ring[(size_t)((at.sg.pos0 + i) % g.taps) * C + ch] = in.proj[(size_t)(at.sg.row0 + i) * in.ldp + ch];
}

int check_in(const DeltaGeom& g, const DeltaIn& in) {
  MI_CHECK(delta_supported(g), "delta rule: heads must be a multiple of the key heads, head sizes 1 .. 256, 1 .. 16 taps");
  MI_CHECK(g.dkp % 16 == 0 && g.dkp >= g.dk && g.dkp < g.dk + 16 && g.dvp % 16 == 0 && g.dvp >= g.dv && g.dvp < g.dv + 16, "delta rule: padding");
  MI_CHECK(in.proj && in.z && in.conv && in.a_log && in.dt && in.norm && in.state && in.ring && in.slots && in.pos, "delta rule: null argument");
  MI_CHECK(in.beta >= g.channels() && in.ldp >= in.beta + g.H && in.gate >= g.H * g.dk && in.ldz >= in.gate + g.H * g.dv, "delta rule: columns");
  return MI_OK;
}

}  // namespace

bool delta_supported(const DeltaGeom& g) {
  return g.H >= 1 && g.G >= 1 && g.H % g.G == 0 && g.dk >= 1 && g.dk <= 256 && g.dv >= 1 && g.dv <= 256 && g.taps >= 1 && g.taps <= 16;
}
size_t delta_chunk_floats(const DeltaGeom& g) { return (size_t)g.H * record_floats(g.dkp, g.dvp); }

int launch_delta_token(const DeltaGeom& g, const DeltaIn& in, int rows, const AttnSeg* segs, void* y, int ldy, bool f32, hipStream_t s) {
  int rc = check_in(g, in);
  if (rc != MI_OK) return rc;
  MI_CHECK(rows >= 1 && rows <= 65535 && y && ldy >= g.H * g.dv, "delta rule: rows");
  const dim3 grid(g.H, rows);
  const int vq = g.dvp <= 16 ? 4 : g.dvp <= 32 ? 8 : g.dvp <= 64 ? 16 : g.dvp <= 128 ? 32 : 64, need = ceil_div(g.dkp, kTokenThreads / vq);
#define MI_DT(VQ, RPT) \
  if (f32) hipLaunchKernelGGL((delta_token_kernel<float, VQ, RPT>), grid, dim3(kTokenThreads), 0, s, g, in, segs, (float*)y, ldy); \
  else hipLaunchKernelGGL((delta_token_kernel<uint16_t, VQ, RPT>), grid, dim3(kTokenThreads), 0, s, g, in, segs, (uint16_t*)y, ldy)
  if (vq == 4) { if (need <= 1) { MI_DT(4, 1); } else { MI_DT(4, 2); } }
  else if (vq == 8) { if (need <= 1) { MI_DT(8, 1); } else if (need <= 2) { MI_DT(8, 2); } else { MI_DT(8, 4); } }
  else if (vq == 16) { if (need <= 2) { MI_DT(16, 2); } else if (need <= 4) { MI_DT(16, 4); } else { MI_DT(16, 8); } }
  else if (vq == 32) { if (need <= 4) { MI_DT(32, 4); } else if (need <= 8) { MI_DT(32, 8); } else { MI_DT(32, 16); } }
  else { if (need <= 8) { MI_DT(64, 8); } else if (need <= 16) { MI_DT(64, 16); } else { MI_DT(64, 32); } }
#undef MI_DT
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_delta_prompt(const DeltaGeom& g, const DeltaIn& in, const AttnSeg* sd, const AttnSeg* sh, int nseg, float* records, int max_chunks,
                        void* y, int ldy, bool f32, hipStream_t s) {
  int rc = check_in(g, in);
  if (rc != MI_OK) return rc;
  MI_CHECK(nseg >= 1 && nseg <= 65535 && records && max_chunks >= 1 && y && ldy >= g.H * g.dv, "delta rule: segments / workspace");
  int chunks = 0;
  for (int i = 0; i < nseg; ++i) chunks += sh[i].n < 2 ? 0 : ceil_div(sh[i].n, kC);
  const int nvt = g.dvp / 16, nt = ceil_div(g.dkp / 16, 4);
  const size_t lds = (size_t)(3 * kC * (g.dkp + 4) + std::max(kC * (g.dkp + 4), kPairParts * kPairTiles * 8)) * sizeof(float);
  for (int c0 = 0; c0 < chunks; c0 += max_chunks) {
    const int n = std::min(max_chunks, chunks - c0);
    const dim3 gf(n, g.H), gs(g.H * nvt, nseg), go(n, ceil_div(g.H, 4));
#define MI_DF(TAPS) { \
    if (lds > 48 * 1024) { rc = ensure_dynamic_lds(reinterpret_cast<const void*>(delta_factors_kernel<TAPS>), (int)lds); if (rc != MI_OK) return rc; } \
    hipLaunchKernelGGL((delta_factors_kernel<TAPS>), gf, dim3(256), lds, s, g, in, sd, nseg, c0, records); }
#define MI_DS(NT) hipLaunchKernelGGL((delta_scan_kernel<NT>), gs, dim3(256), 0, s, g, in.state, in.slots, sd, c0, n, nvt, records)
    switch (g.taps) {
      case 1: MI_DF(1); break;
      case 2: MI_DF(2); break;
      case 3: MI_DF(3); break;
      case 4: MI_DF(4); break;
      default: MI_DF(0);
    }
#undef MI_DF
    if (nt == 1) MI_DS(1);
    else if (nt == 2) MI_DS(2);
    else if (nt == 3) MI_DS(3);
    else MI_DS(4);
#undef MI_DS
#define MI_DO(NV) \
    if (f32) hipLaunchKernelGGL((delta_out_kernel<float, NV>), go, dim3(256), 0, s, g, in, sd, nseg, c0, records, (float*)y, ldy); \
    else hipLaunchKernelGGL((delta_out_kernel<uint16_t, NV>), go, dim3(256), 0, s, g, in, sd, nseg, c0, records, (uint16_t*)y, ldy)
    if (g.dv <= 64) { MI_DO(1); } else if (g.dv <= 128) { MI_DO(2); } else { MI_DO(4); }
#undef MI_DO
    MI_HIP(hipGetLastError());
  }
  return MI_OK;
}

}  // namespace mi
