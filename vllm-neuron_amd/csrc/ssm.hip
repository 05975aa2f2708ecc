// State-space mixers.  See ssm.h.
#include "ssm.h"

#include <algorithm>

namespace mi {

namespace {

constexpr float kLog2e = 1.4426950408889634f;

__device__ __forceinline__ float silu(float v) { return v / (1.f + __expf(-v)); }
__device__ __forceinline__ float softplus(float v) { return fmaxf(v, 0.f) + log1pf(expf(-fabsf(v))); }
__device__ __forceinline__ float to_f32(uint16_t v) { return bf16_to_f32(v); }
__device__ __forceinline__ float to_f32(float v) { return v; }
__device__ __forceinline__ void put1(uint16_t* p, float v) { *p = f32_to_bf16(v); }
__device__ __forceinline__ void put1(float* p, float v) { *p = v; }
__device__ __forceinline__ float round_to(float v, const uint16_t*) { return bf16_to_f32(f32_to_bf16(v)); }
__device__ __forceinline__ float round_to(float v, const float*) { return v; }
__device__ __forceinline__ float4 get4(const uint16_t* p) {
  const uint2 v = *reinterpret_cast<const uint2*>(p);
  return make_float4(bf16lo_to_f32(v.x), bf16hi_to_f32(v.x), bf16lo_to_f32(v.y), bf16hi_to_f32(v.y));
}
__device__ __forceinline__ float4 get4(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ void put4(uint16_t* p, float4 v) { *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf16x2(v.x, v.y), pack_bf16x2(v.z, v.w)); }
__device__ __forceinline__ void put4(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }

// =====================================================================================
// short convolution
// =====================================================================================
// One work-group: up to kConvRows rows of one segment x 256 channels, a channel per thread.  Only a segment's first tile reads the
// ring (kConvRows >= taps - 1), and its threads renew their channel's ring once they have read it.
constexpr int kConvRows = 16;
template <typename T, int TAPS>
__global__ __launch_bounds__(256) void short_conv_kernel(const float* __restrict__ x, int ldx, ShortConv cv, const int32_t* __restrict__ pos,
                                                         const AttnSeg* __restrict__ segs, int nseg, T* __restrict__ y, int ldy) {
  int tile = blockIdx.x;
  AttnSeg sg{(int)blockIdx.x, 1, 0, (int)blockIdx.x};
  if (nseg > 0) {
    int si = 0;
    for (; si < nseg; ++si) {
      sg = segs[si];
      const int n = ceil_div(sg.n, kConvRows);
      if (tile < n) break;
      tile -= n;
    }
    if (si == nseg) return;
  } else {
    sg.pos0 = pos[sg.row0];
    tile = 0;
  }
  const int ch = blockIdx.y * 256 + threadIdx.x, C = cv.C, taps = TAPS > 0 ? TAPS : cv.taps;
  if (ch >= ldy) return;
  const int first = tile * kConvRows, last = min(first + kConvRows, sg.n);
  if (ch >= C) {
    for (int i = first; i < last; ++i) put1(y + (size_t)(sg.row0 + i) * ldy + ch, 0.f);
    return;
  }
  const float* xs = x + (size_t)sg.row0 * ldx + ch;
  float* ring = cv.ring + (size_t)cv.slots[sg.seq] * taps * C + ch;
  const float bias = cv.b[ch];
  // input i rows behind the segment's start (negative: ahead of it)
  auto input = [&](int i) {
    const int p = max(sg.pos0 + i, 0);
    const float* a = i >= 0 ? xs + (size_t)i * ldx : ring + (size_t)(p % taps) * C;
    const float v = *a;
    return sg.pos0 + i >= 0 ? v : 0.f;
  };
  if constexpr (TAPS > 0) {
    float in[kConvRows + TAPS - 1], w[TAPS];
#pragma unroll
    for (int j = 0; j < TAPS; ++j) w[j] = cv.w[(size_t)j * C + ch];
    if (sg.n == 1) {
#pragma unroll
      for (int k = 0; k < kConvRows + TAPS - 1; ++k) in[k] = k < TAPS ? input(k - (TAPS - 1)) : 0.f;
    } else {
#pragma unroll
      for (int k = 0; k < kConvRows + TAPS - 1; ++k) in[k] = input(min(first + k - (TAPS - 1), sg.n - 1));
    }
#pragma unroll
    for (int k = 0; k < kConvRows; ++k) {
      float a = bias;
#pragma unroll
      for (int j = 0; j < TAPS; ++j) a = __builtin_fmaf(w[j], in[k + j], a);
      if (first + k < last) put1(y + (size_t)(sg.row0 + first + k) * ldy + ch, silu(a));
    }
  } else {
    for (int i = first; i < last; ++i) {
      float a = bias;
      for (int j = 0; j < taps; ++j) a = __builtin_fmaf(cv.w[(size_t)j * C + ch], input(i - (taps - 1 - j)), a);
      put1(y + (size_t)(sg.row0 + i) * ldy + ch, silu(a));
    }
  }
  if (tile == 0)
    for (int i = max(0, sg.n - taps); i < sg.n; ++i) ring[(size_t)((sg.pos0 + i) % taps) * C] = xs[(size_t)i * ldx];
}

// =====================================================================================
// selective scan
// =====================================================================================
template <int LPC>
__device__ __forceinline__ float lanes_sum(float v) { return group_sum<LPC>(v); }

// LPC lanes per channel, R consecutive states per lane (Np = LPC R).
template <typename T, int LPC, int R>
__global__ __launch_bounds__(256) void scan_token_kernel(ScanGeom g, ScanIn in, const AttnSeg* __restrict__ segs, T* __restrict__ y, int ldy) {
  constexpr int CB = 256 / LPC;
  int row = blockIdx.y, seq = blockIdx.y;
  if (segs) {
    const AttnSeg sg = segs[blockIdx.y];
    if (sg.n != 1) return;
    row = sg.row0; seq = sg.seq;
  }
  const int l = threadIdx.x % LPC, c = blockIdx.x * CB + threadIdx.x / LPC, cc = min(c, g.C - 1);     // (lanes past the last channel repeat it)
  float* S0 = in.state + ((size_t)in.slots[seq] * g.C + cc) * g.Np + l * R;
  const float *a2 = in.a2 + (size_t)cc * g.Np + l * R, *lo = in.low + (size_t)row * in.ldl;
  const bool fresh = in.pos[row] == 0;
  float S[R], A[R], B[R], Cn[R];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    S[r] = S0[r];
    A[r] = a2[r];
    const int n = min(l * R + r, g.N - 1);           // (beyond the last state: B is taken as zero)
    B[r] = lo[in.col_b + n];
    Cn[r] = lo[in.col_c + n];
  }
  const float x = to_f32(reinterpret_cast<const T*>(in.x)[(size_t)row * in.ldx + cc]), z = in.z[(size_t)row * in.ldz + cc];
  const T* w = reinterpret_cast<const T*>(in.w_dt) + (size_t)cc * g.rank_p;
  float dot = 0.f;
  for (int k = l * 8; k < g.rank_p; k += LPC * 8) {
#pragma unroll
    for (int q = 0; q < 8; q += 4) {
      const float4 wv = get4(w + k + q);             // (zero beyond the rank)
      auto at = [&](int i) { return round_to(lo[min(k + q + i, g.rank - 1)], y); };
      dot = __builtin_fmaf(wv.x, at(0), dot); dot = __builtin_fmaf(wv.y, at(1), dot);
      dot = __builtin_fmaf(wv.z, at(2), dot); dot = __builtin_fmaf(wv.w, at(3), dot);
    }
  }
  const float dt = softplus(lanes_sum<LPC>(dot) + in.dt_bias[cc]), dx = dt * x;
  float o = 0.f;
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const float b = l * R + r < g.N ? B[r] : 0.f;
    S[r] = __builtin_fmaf(__builtin_amdgcn_exp2f(dt * A[r]), fresh ? 0.f : S[r], dx * b);
    o = __builtin_fmaf(S[r], Cn[r], o);
  }
  o = lanes_sum<LPC>(o);
  if (c >= g.C) return;
#pragma unroll
  for (int r = 0; r < R; ++r) S0[r] = S[r];
  if (l == 0) put1(y + (size_t)row * ldy + c, __builtin_fmaf(in.d[c], x, o) * silu(z));
}

// One work-group: CB channels of one segment, its tokens in order, TB at a time: their step sizes, inputs, B and C go through LDS (the next
// ones are requested ahead), token by token fastest so that a lane reads four tokens at once; outputs meet in LDS for gate and store.
template <typename T, int LPC, int R>
__global__ __launch_bounds__(256) void scan_prompt_kernel(ScanGeom g, ScanIn in, const AttnSeg* __restrict__ segs, T* __restrict__ y, int ldy) {
  constexpr int CB = 256 / LPC, Np = LPC * R, TB = Np <= 64 ? 32 : 16, PT = TB + 4, NI = TB * CB / 256, NB = TB * Np / 256;
  __shared__ __attribute__((aligned(16))) float dts[CB][PT], dxs[CB][PT], ys[CB][PT];
  __shared__ __attribute__((aligned(16))) float Bs[Np][PT], Cs[Np][PT];
  const AttnSeg sg = segs[blockIdx.y];
  if (sg.n < 2) return;
  const int tid = threadIdx.x, l = tid % LPC, cl = tid / LPC, c0 = blockIdx.x * CB, cc = min(c0 + cl, g.C - 1);
  float* S0 = in.state + ((size_t)in.slots[sg.seq] * g.C + cc) * g.Np + l * R;
  float S[R], A[R];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    A[r] = in.a2[(size_t)cc * g.Np + l * R + r];
    S[r] = sg.pos0 > 0 ? S0[r] : 0.f;
  }
  // items of a block: (token, channel), channel fastest; B / C: (token, state), state fastest
  float dt[NI], x[NI], z[NI], bv[NB], cv[NB], bias[NI], dd[NI];
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int ch = min(c0 + (tid + 256 * i) % CB, g.C - 1);
    bias[i] = in.dt_bias[ch];
    dd[i] = in.d[ch];
  }
  auto load = [&](int t0) {
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int k = tid + 256 * i, t = min(t0 + k / CB, sg.n - 1), ch = min(c0 + k % CB, g.C - 1);
      const size_t row = sg.row0 + t;
      dt[i] = in.dt[row * in.ldt + ch];
      x[i] = to_f32(reinterpret_cast<const T*>(in.x)[row * in.ldx + ch]);
      z[i] = in.z[row * in.ldz + ch];
    }
#pragma unroll
    for (int i = 0; i < NB; ++i) {
      const int k = tid + 256 * i, t = min(t0 + k / Np, sg.n - 1), n = k % Np;
      const float* lo = in.low + (size_t)(sg.row0 + t) * in.ldl + min(n, g.N - 1);
      bv[i] = n < g.N ? lo[in.col_b] : 0.f;
      cv[i] = lo[in.col_c];
    }
  };
  load(0);
  for (int t0 = 0; t0 < sg.n; t0 += TB) {
    float xk[NI], zk[NI];
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int k = tid + 256 * i, t = k / CB;
      const float s = t0 + t < sg.n ? softplus(dt[i] + bias[i]) : 0.f;       // (past the end: the state stays)
      xk[i] = x[i];
      zk[i] = z[i];
      dts[k % CB][t] = s;
      dxs[k % CB][t] = s * x[i];
    }
#pragma unroll
    for (int i = 0; i < NB; ++i) {
      const int k = tid + 256 * i;
      Bs[k % Np][k / Np] = bv[i];
      Cs[k % Np][k / Np] = cv[i];
    }
    __syncthreads();
    if (t0 + TB < sg.n) load(t0 + TB);
#pragma unroll 2
    for (int t = 0; t < TB; t += 4) {
      const float4 d4 = *reinterpret_cast<const float4*>(&dts[cl][t]), x4 = *reinterpret_cast<const float4*>(&dxs[cl][t]);
      const float da[4] = {d4.x, d4.y, d4.z, d4.w}, xa[4] = {x4.x, x4.y, x4.z, x4.w};
      float o[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int r = 0; r < R; ++r) {
        const float4 b4 = *reinterpret_cast<const float4*>(&Bs[l * R + r][t]), c4 = *reinterpret_cast<const float4*>(&Cs[l * R + r][t]);
        const float ba[4] = {b4.x, b4.y, b4.z, b4.w}, ca[4] = {c4.x, c4.y, c4.z, c4.w};
#pragma unroll
        for (int u = 0; u < 4; ++u) {
          S[r] = __builtin_fmaf(__builtin_amdgcn_exp2f(da[u] * A[r]), S[r], xa[u] * ba[u]);
          o[u] = __builtin_fmaf(S[r], ca[u], o[u]);
        }
      }
#pragma unroll
      for (int u = 0; u < 4; ++u) o[u] = lanes_sum<LPC>(o[u]);
      if (l == 0) *reinterpret_cast<float4*>(&ys[cl][t]) = make_float4(o[0], o[1], o[2], o[3]);
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int k = tid + 256 * i, t = t0 + k / CB, ch = c0 + k % CB;
      if (t < sg.n && ch < g.C) put1(y + (size_t)(sg.row0 + t) * ldy + ch, __builtin_fmaf(dd[i], xk[i], ys[k % CB][k / CB]) * silu(zk[i]));
    }
    // (the next block's first barrier is ahead of anything that writes ys)
  }
  if (c0 + cl >= g.C) return;
#pragma unroll
  for (int r = 0; r < R; ++r) S0[r] = S[r];
}

__global__ void scan_decay_kernel(const float* __restrict__ a_log, int C, int N, int Np, float* __restrict__ a2) {
  const int i = blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= C * N) return;
  a2[(size_t)(i / N) * Np + i % N] = -expf(a_log[i]) * kLog2e;
}

// =====================================================================================
// state-space duality
// =====================================================================================
constexpr int kQ = kSsdChunk;

// One work-group per (head, row): the head's state in registers, requested first; thread (vq, dg) owns columns 4 vq .. + 3 of rows
// dg RPT .. + RPT - 1.
constexpr int kTokenThreads = 512;
template <typename T, int VQ, int RPT>
__global__ __launch_bounds__(kTokenThreads) void ssd_token_kernel(SsdGeom g, SsdIn in, const AttnSeg* __restrict__ segs, float* __restrict__ y, int ldy) {
  constexpr int NW = kTokenThreads / 64;
  __shared__ float bs[256], cs[256], xs[256];
  __shared__ __attribute__((aligned(16))) float red[NW][VQ * 4];
  const int h = blockIdx.x, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  int row = blockIdx.y, seq = blockIdx.y;
  if (segs) {
    const AttnSeg sg = segs[blockIdx.y];
    if (sg.n != 1) return;
    row = sg.row0; seq = sg.seq;
  }
  const int vq = tid % VQ, dg = tid / VQ;
  const bool vin = vq * 4 < g.Pp, fresh = in.pos[row] == 0;
  float* S0 = in.state + ((size_t)in.slots[seq] * g.H + h) * g.Np * g.Pp + vq * 4;
  float4 S[RPT];
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int n = dg * RPT + i;
    S[i] = !fresh && vin && n < g.Np ? *reinterpret_cast<const float4*>(S0 + (size_t)n * g.Pp) : make_float4(0.f, 0.f, 0.f, 0.f);
  }
  const T* xr = reinterpret_cast<const T*>(in.xbc) + (size_t)row * in.ldx;
  const int inner = g.H * g.P, grp = h / (g.H / g.G);
  for (int i = tid; i < g.Np; i += kTokenThreads) {
    bs[i] = i < g.N ? to_f32(xr[inner + grp * g.N + i]) : 0.f;
    cs[i] = i < g.N ? to_f32(xr[inner + (g.G + grp) * g.N + i]) : 0.f;
  }
  for (int i = tid; i < g.Pp; i += kTokenThreads) xs[i] = i < g.P ? to_f32(xr[h * g.P + i]) : 0.f;
  const float dt = softplus(in.dt[(size_t)row * in.ldt + h] + in.dt_bias[h]), decay = expf(-expf(in.a_log[h]) * dt);
  __syncthreads();
  float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
  float4 u = make_float4(0.f, 0.f, 0.f, 0.f);
  if (vin) u = make_float4(dt * xs[vq * 4], dt * xs[vq * 4 + 1], dt * xs[vq * 4 + 2], dt * xs[vq * 4 + 3]);
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int n = dg * RPT + i;
    if (!vin || n >= g.Np) continue;
    const float b = bs[n], c = cs[n];
    S[i].x = __builtin_fmaf(decay, S[i].x, b * u.x); S[i].y = __builtin_fmaf(decay, S[i].y, b * u.y);
    S[i].z = __builtin_fmaf(decay, S[i].z, b * u.z); S[i].w = __builtin_fmaf(decay, S[i].w, b * u.w);
    *reinterpret_cast<float4*>(S0 + (size_t)n * g.Pp) = S[i];
    o.x = __builtin_fmaf(S[i].x, c, o.x); o.y = __builtin_fmaf(S[i].y, c, o.y); o.z = __builtin_fmaf(S[i].z, c, o.z); o.w = __builtin_fmaf(S[i].w, c, o.w);
  }
#pragma unroll
  for (int m = VQ; m < 64; m *= 2) { o.x += __shfl_xor(o.x, m); o.y += __shfl_xor(o.y, m); o.z += __shfl_xor(o.z, m); o.w += __shfl_xor(o.w, m); }
  if (lane < VQ) *reinterpret_cast<float4*>(&red[wave][vq * 4]) = o;
  __syncthreads();
  for (int p = tid; p < g.P; p += kTokenThreads) {
    float s = 0.f;
#pragma unroll
    for (int w = 0; w < NW; ++w) s += red[w][p];
    y[(size_t)row * ldy + h * g.P + p] = __builtin_fmaf(in.d[h], xs[p], s);
  }
}

struct ChunkAt { AttnSeg sg; int t0, n; bool ok; };     // rows t0 .. + n of the segment
__device__ __forceinline__ ChunkAt chunk_at(const AttnSeg* segs, int nseg, int c) {
  for (int i = 0; i < nseg; ++i) {
    const AttnSeg sg = segs[i];
    if (sg.n < 2) continue;
    const int k = ceil_div(sg.n, kQ);
    if (c < k) return ChunkAt{sg, c * kQ, min(kQ, sg.n - c * kQ), true};
    c -= k;
  }
  return ChunkAt{AttnSeg{0, 0, 0, 0}, 0, 0, false};
}

// What a piece of chunks leaves in memory: states [chunk][H][Np][Pp], C B^T [chunk][G][kQ][kQ], the chunk's whole decay [chunk][H]
struct Records { float *state, *cb, *decay; };
__host__ __device__ inline Records records_at(float* base, const SsdGeom& g, int chunks) {
  float* cb = base + (size_t)chunks * g.H * g.Np * g.Pp;
  return Records{base, cb, cb + (size_t)chunks * g.G * kQ * kQ};
}
// LDS row pitches: rows whose columns 16 lanes read side by side (four rows at once), and rows of which 16 lanes read one column each
__host__ __device__ inline int wide_pitch(int n) { return (n + 47) / 64 * 64 + 16; }
__host__ __device__ inline int tall_pitch(int n) { return (n + 63) / 64 * 64 + 4; }

// step sizes of the chunk and the running sum of their decays' logarithms; ends with a barrier
__device__ __forceinline__ void chunk_steps(const SsdIn& in, int h, const ChunkAt& at, double* L, float* dts) {
  if (threadIdx.x < 64) {
    const int t = threadIdx.x;
    const float dt = t < at.n ? softplus(in.dt[(size_t)(at.sg.row0 + at.t0 + min(t, at.n - 1)) * in.ldt + h] + in.dt_bias[h]) : 0.f;
    double s = (double)(-expf(in.a_log[h]) * dt);
#pragma unroll
    for (int m = 1; m < 64; m *= 2) {
      const double v = __shfl_up(s, m);
      if (t >= m) s += v;
    }
    L[t] = s;
    dts[t] = dt;
  }
  __syncthreads();
}

// columns col .. + n of the chunk's rows times weight(row) into LDS rows of `pitch`, zeros up to np and beyond the last row
template <typename T, typename F>
__device__ __forceinline__ void stage_rows(float* dst, int pitch, const T* src, int ld, int rows, int n, int np, F weight) {
  const int tid = threadIdx.x;
  if (((n | ld) & 3) == 0 && (reinterpret_cast<uintptr_t>(src) & (4 * sizeof(T) - 1)) == 0) {
    const int q = np / 4;
    for (int i = tid; i < kQ * q; i += 256) {
      const int t = i / q, c = (i - t * q) * 4;
      float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
      if (t < rows && c < n) {
        const float f = weight(t);
        v = get4(src + (size_t)t * ld + c);
        v = make_float4(v.x * f, v.y * f, v.z * f, v.w * f);
      }
      *reinterpret_cast<float4*>(dst + t * pitch + c) = v;
    }
    return;
  }
  for (int i = tid; i < kQ * np; i += 256) {
    const int t = i / np, c = i - t * np;
    dst[t * pitch + c] = t < rows && c < n ? to_f32(src[(size_t)t * ld + c]) * weight(t) : 0.f;
  }
}

// Of every chunk: what it adds to the state, per head (blockIdx.y < H), and C B^T, per group
template <typename T>
__global__ __launch_bounds__(256) void ssd_chunk_kernel(SsdGeom g, SsdIn in, const AttnSeg* __restrict__ segs, int nseg, int c0, float* __restrict__ base) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  __shared__ double L[kQ];
  __shared__ float dts[kQ];
  const ChunkAt at = chunk_at(segs, nseg, c0 + blockIdx.x);
  if (!at.ok) return;
  const Records rec = records_at(base, g, gridDim.x);
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, g4 = lane >> 4, c = lane & 15, inner = g.H * g.P;
  const T* rows = reinterpret_cast<const T*>(in.xbc) + (size_t)(at.sg.row0 + at.t0) * in.ldx;
  if ((int)blockIdx.y < g.H) {
    const int h = blockIdx.y, grp = h / (g.H / g.G), bp = wide_pitch(g.Np), xp = wide_pitch(g.Pp);
    float *Bs = sm, *xs = sm + kQ * bp;
    chunk_steps(in, h, at, L, dts);
    const double end = L[kQ - 1];
    stage_rows(Bs, bp, rows + inner + grp * g.N, in.ldx, at.n, g.N, g.Np, [&](int t) { return dts[t] * expf((float)(end - L[t])); });
    stage_rows(xs, xp, rows + h * g.P, in.ldx, at.n, g.P, g.Pp, [](int) { return 1.f; });
    if (tid == 0) rec.decay[(size_t)blockIdx.x * g.H + h] = expf((float)end);
    __syncthreads();
    float* out = rec.state + ((size_t)blockIdx.x * g.H + h) * g.Np * g.Pp;
    const int nt = g.Np / 16, pt = g.Pp / 16;
    for (int n = wave; n < nt; n += 4)
      for (int p0 = 0; p0 < pt; p0 += 4) {
        f32x4_t acc[4] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
        int off[4];
#pragma unroll
        for (int p = 0; p < 4; ++p) off[p] = 16 * min(p0 + p, pt - 1) + c;
#pragma unroll 4
        for (int s = 0; s < kQ / 4; ++s) {
          const float a = Bs[(4 * s + g4) * bp + 16 * n + c];
#pragma unroll
          for (int p = 0; p < 4; ++p) acc[p] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, xs[(4 * s + g4) * xp + off[p]], acc[p], 0, 0, 0);
        }
#pragma unroll
        for (int p = 0; p < 4; ++p) {
#pragma unroll
          for (int r = 0; r < 4; ++r)
            if (p0 + p < pt) out[(size_t)(16 * n + 4 * g4 + r) * g.Pp + off[p]] = acc[p][r];
        }
      }
    return;
  }
  const int grp = blockIdx.y - g.H, pitch = tall_pitch(g.Np);
  float *Bs = sm, *Cs = sm + kQ * pitch;
  auto one = [](int) { return 1.f; };
  stage_rows(Bs, pitch, rows + inner + grp * g.N, in.ldx, at.n, g.N, g.Np, one);
  stage_rows(Cs, pitch, rows + inner + (g.G + grp) * g.N, in.ldx, at.n, g.N, g.Np, one);
  __syncthreads();
  float* out = rec.cb + ((size_t)blockIdx.x * g.G + grp) * kQ * kQ;
  f32x4_t acc[4] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
  for (int s = 0; s < g.Np / 4; ++s) {
    const float a = Cs[(16 * wave + c) * pitch + 4 * s + g4];
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, Bs[(16 * j + c) * pitch + 4 * s + g4], acc[j], 0, 0, 0);
  }
#pragma unroll
  for (int j = 0; j < 4; ++j)
#pragma unroll
    for (int r = 0; r < 4; ++r) out[(16 * wave + 4 * g4 + r) * kQ + 16 * j + c] = acc[j][r];
}

// The chunks of a segment in order: what a chunk adds is replaced by the state ahead of it; the state behind the last one goes to the slot.
__global__ __launch_bounds__(256) void ssd_pass_kernel(SsdGeom g, SsdIn in, const AttnSeg* __restrict__ segs, int c0, int nchunks, float* __restrict__ base) {
  const int si = blockIdx.y;
  const AttnSeg sg = segs[si];
  if (sg.n < 2) return;
  int first = 0;             // the segment's first chunk among all
  for (int i = 0; i < si; ++i) first += segs[i].n < 2 ? 0 : ceil_div(segs[i].n, kQ);
  const int k0 = max(c0 - first, 0), k1 = min(c0 + nchunks - first, ceil_div(sg.n, kQ));
  if (k0 >= k1) return;
  const size_t hs = (size_t)g.Np * g.Pp, at = ((size_t)blockIdx.x * 256 + threadIdx.x) * 4;
  if (at >= g.H * hs) return;
  const Records rec = records_at(base, g, nchunks);
  const int h = (int)(at / hs);
  float* slot = in.state + (size_t)in.slots[sg.seq] * g.H * hs + at;
  float4 S = sg.pos0 + k0 > 0 ? *reinterpret_cast<const float4*>(slot) : make_float4(0.f, 0.f, 0.f, 0.f);
  constexpr int kAhead = 4;
  const int n = k1 - k0, r0 = first + k0 - c0;
  auto add_at = [&](int k) { return rec.state + (size_t)(r0 + min(k, n - 1)) * g.H * hs + at; };
  auto decay_at = [&](int k) { return rec.decay[(size_t)(r0 + min(k, n - 1)) * g.H + h]; };
  float4 add[kAhead];
  float e[kAhead];
#pragma unroll
  for (int i = 0; i < kAhead; ++i) { add[i] = *reinterpret_cast<const float4*>(add_at(i)); e[i] = decay_at(i); }
  for (int k = 0; k < n; k += kAhead) {
#pragma unroll
    for (int i = 0; i < kAhead; ++i) {
      if (k + i < n) {
      *reinterpret_cast<float4*>(add_at(k + i)) = S;
      S = make_float4(__builtin_fmaf(e[i], S.x, add[i].x), __builtin_fmaf(e[i], S.y, add[i].y), __builtin_fmaf(e[i], S.z, add[i].z), __builtin_fmaf(e[i], S.w, add[i].w));
      if (k + i + kAhead < n) { add[i] = *reinterpret_cast<const float4*>(add_at(k + i + kAhead)); e[i] = decay_at(k + i + kAhead); }
      }
    }
  }
  *reinterpret_cast<float4*>(slot) = S;
}

// Outputs of a chunk and head: wave w owns tokens 16 w .. + 15
template <typename T, int NPT>
__global__ __launch_bounds__(256) void ssd_out_kernel(SsdGeom g, SsdIn in, const AttnSeg* __restrict__ segs, int nseg, int c0, float* __restrict__ base,
                                                      float* __restrict__ y, int ldy) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  __shared__ double L[kQ];
  __shared__ float dts[kQ];
  const ChunkAt at = chunk_at(segs, nseg, c0 + blockIdx.x);
  if (!at.ok) return;
  const Records rec = records_at(base, g, gridDim.x);
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, g4 = lane >> 4, c = lane & 15, inner = g.H * g.P, h = blockIdx.y, grp = h / (g.H / g.G);
  const int mp = kQ + 4, xp = wide_pitch(g.Pp), cp = tall_pitch(g.Np);
  float *Ms = sm, *xs = Ms + kQ * mp, *Cs = xs + kQ * xp;
  const T* rows = reinterpret_cast<const T*>(in.xbc) + (size_t)(at.sg.row0 + at.t0) * in.ldx;
  const float* cb = rec.cb + ((size_t)blockIdx.x * g.G + grp) * kQ * kQ;
  chunk_steps(in, h, at, L, dts);
  stage_rows(xs, xp, rows + h * g.P, in.ldx, at.n, g.P, g.Pp, [](int) { return 1.f; });
  stage_rows(Cs, cp, rows + inner + (g.G + grp) * g.N, in.ldx, at.n, g.N, g.Np, [&](int t) { return expf((float)L[t]); });
  for (int k = tid; k < kQ * kQ; k += 256) {
    const int i = k / kQ, j = k % kQ;
    Ms[i * mp + j] = j <= i ? cb[k] * expf((float)(L[i] - L[j])) * dts[j] : 0.f;
  }
  __syncthreads();
  if (16 * wave >= at.n) return;
  f32x4_t acc[NPT];
  int off[NPT];
#pragma unroll
  for (int p = 0; p < NPT; ++p) {
    acc[p] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    off[p] = min(16 * p, g.Pp - 16) + c;
  }
  for (int s = 0; s < 4 * (wave + 1); ++s) {
    const float a = Ms[(16 * wave + c) * mp + 4 * s + g4];
#pragma unroll
    for (int p = 0; p < NPT; ++p) acc[p] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, xs[(4 * s + g4) * xp + off[p]], acc[p], 0, 0, 0);
  }
  const float* S0 = rec.state + ((size_t)blockIdx.x * g.H + h) * g.Np * g.Pp;
  for (int s = 0; s < g.Np / 4; ++s) {
    const float a = Cs[(16 * wave + c) * cp + 4 * s + g4];
#pragma unroll
    for (int p = 0; p < NPT; ++p) acc[p] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, S0[(size_t)(4 * s + g4) * g.Pp + off[p]], acc[p], 0, 0, 0);
  }
  const float d = in.d[h];
#pragma unroll
  for (int p = 0; p < NPT; ++p) {
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 16 * wave + 4 * g4 + r;
      if (i < at.n && 16 * p + c < g.P) y[(size_t)(at.sg.row0 + at.t0 + i) * ldy + h * g.P + 16 * p + c] = __builtin_fmaf(d, xs[i * xp + 16 * p + c], acc[p][r]);
    }
  }
}

// one work-group per row; a part is shared out to several waves where there are fewer parts than waves (summed in wave order)
template <typename T>
__global__ __launch_bounds__(1024) void gated_norm_kernel(const float* __restrict__ y, int ldy, const float* __restrict__ z, int ldz, const float* __restrict__ w,
                                                         int n, int parts, float eps, T* __restrict__ out, int ldo) {
  extern __shared__ __attribute__((aligned(16))) float row[];   // n padded to 4, then max(parts, 16) and parts floats
  const int np = (n + 3) / 4 * 4, tid = threadIdx.x, nthr = blockDim.x, nw = nthr >> 6, wave = tid >> 6, lane = tid & 63;
  float *red = row + np, *rstd = red + max(parts, 16);
  const float *yr = y + (size_t)blockIdx.x * ldy, *zr = z + (size_t)blockIdx.x * ldz;
  T* o = out + (size_t)blockIdx.x * ldo;
  const bool vec = ((n | ldy | ldz | ldo) & 3) == 0;
  if (vec) {
    for (int d = tid * 4; d < n; d += nthr * 4) {
      const float4 a = *reinterpret_cast<const float4*>(yr + d), b = *reinterpret_cast<const float4*>(zr + d);
      *reinterpret_cast<float4*>(row + d) = make_float4(a.x * silu(b.x), a.y * silu(b.y), a.z * silu(b.z), a.w * silu(b.w));
    }
  } else {
    for (int d = tid; d < n; d += nthr) row[d] = yr[d] * silu(zr[d]);
  }
  __syncthreads();
  const int gs = n / parts, P = max(1, nw / parts), len = ceil_div(gs, P);
  for (int u = wave; u < parts * P; u += nw) {
    const int g = u / P, lo = g * gs + (u - g * P) * len, hi = min(lo + len, (g + 1) * gs);
    float s = 0.f;
    for (int i = lo + lane; i < hi; i += 64) s = __builtin_fmaf(row[i], row[i], s);
    s = wave_sum(s);
    if (lane == 0) red[u] = s;
  }
  __syncthreads();
  for (int g = tid; g < parts; g += nthr) {
    float s = 0.f;
    for (int p = 0; p < P; ++p) s += red[g * P + p];
    rstd[g] = 1.0f / sqrtf(s / (float)gs + eps);
  }
  __syncthreads();
  if (vec && (gs & 3) == 0) {
    for (int d = tid * 4; d < n; d += nthr * 4) {
      const float4 a = *reinterpret_cast<const float4*>(row + d), k = *reinterpret_cast<const float4*>(w + d);
      const float f = parts == 1 ? rstd[0] : rstd[d / gs];
      put4(o + d, make_float4(a.x * f * k.x, a.y * f * k.y, a.z * f * k.z, a.w * f * k.w));
    }
  } else {
    for (int d = tid; d < n; d += nthr) put1(o + d, row[d] * rstd[d / gs] * w[d]);
  }
}

int check_scan(const ScanGeom& g, const ScanIn& in, const void* y, int ldy) {
  MI_CHECK(g.C >= 1 && scan_supported(g.N) && g.rank >= 1 && g.Np >= g.N && g.rank_p % 8 == 0 && g.rank_p >= g.rank, "selective scan: 1 .. 256 states");
  MI_CHECK(in.x && in.low && in.dt_bias && in.a2 && in.d && in.z && in.state && in.slots && in.pos && y, "selective scan: null argument");
  MI_CHECK(in.ldx >= g.C && in.ldz >= g.C && ldy >= g.C && in.col_b >= g.rank && in.col_c >= in.col_b + g.N && in.ldl >= in.col_c + g.N, "selective scan: columns");
  return MI_OK;
}
int check_ssd(const SsdGeom& g, const SsdIn& in, const float* y, int ldy) {
  MI_CHECK(ssd_supported(g), "state-space duality: heads must be a multiple of the groups, sizes 1 .. 256");
  MI_CHECK(g.Np % 16 == 0 && g.Np >= g.N && g.Np < g.N + 16 && g.Pp % 16 == 0 && g.Pp >= g.P && g.Pp < g.P + 16, "state-space duality: padding");
  MI_CHECK(in.xbc && in.dt && in.dt_bias && in.a_log && in.d && in.state && in.slots && in.pos && y, "state-space duality: null argument");
  MI_CHECK(in.ldx >= g.channels() && in.ldt >= g.H && ldy >= g.inner(), "state-space duality: columns");
  return MI_OK;
}

}  // namespace

int launch_short_conv(const float* x, int ldx, const ShortConv& cv, const int32_t* pos, const AttnSeg* sd, const AttnSeg* sh, int nseg, int rows, void* y,
                      int ldy, bool f32, hipStream_t s) {
  MI_CHECK(x && y && cv.w && cv.b && cv.ring && cv.slots && cv.taps >= 1 && cv.taps <= 16 && cv.C >= 1 && ldx >= cv.C && ldy >= cv.C && rows >= 1, "short convolution: 1 .. 16 taps / strides");
  MI_CHECK(nseg >= 0 && (nseg > 0 ? sd && sh : pos != nullptr), "short convolution: segments");
  int tiles = nseg > 0 ? 0 : rows;
  for (int i = 0; i < nseg; ++i) tiles += ceil_div(sh[i].n, kConvRows);
  const dim3 grid(tiles, ceil_div(ldy, 256));
#define MI_SC(TAPS) \
  if (f32) hipLaunchKernelGGL((short_conv_kernel<float, TAPS>), grid, dim3(256), 0, s, x, ldx, cv, pos, sd, nseg, (float*)y, ldy); \
  else hipLaunchKernelGGL((short_conv_kernel<uint16_t, TAPS>), grid, dim3(256), 0, s, x, ldx, cv, pos, sd, nseg, (uint16_t*)y, ldy)
  switch (cv.taps) {
    case 2: MI_SC(2); break;
    case 3: MI_SC(3); break;
    case 4: MI_SC(4); break;
    default: MI_SC(0);
  }
#undef MI_SC
  MI_HIP(hipGetLastError());
  return MI_OK;
}

bool scan_supported(int N) { return N >= 1 && N <= 256; }
ScanGeom scan_geom(int C, int N, int rank) {
  int np = 8;
  while (np < N) np *= 2;
  return ScanGeom{C, N, np, rank, (rank + 7) / 8 * 8};
}

// lanes per channel and states per lane by the padded state
#define MI_BY_STATE(CALL)          \
  switch (g.Np) {                  \
    case 8: CALL(8, 1); break;     \
    case 16: CALL(16, 1); break;   \
    case 32: CALL(16, 2); break;   \
    case 64: CALL(16, 4); break;   \
    case 128: CALL(16, 8); break;  \
    default: CALL(16, 16);         \
  }

int launch_scan_token(const ScanGeom& g, const ScanIn& in, int rows, const AttnSeg* segs, void* y, int ldy, bool f32, hipStream_t s) {
  int rc = check_scan(g, in, y, ldy);
  if (rc != MI_OK) return rc;
  MI_CHECK(rows >= 1 && rows <= 65535 && in.w_dt, "selective scan: rows");
#define MI_ST(LPC, R) { \
    const dim3 grid(ceil_div(g.C, 256 / LPC), rows); \
    if (f32) hipLaunchKernelGGL((scan_token_kernel<float, LPC, R>), grid, dim3(256), 0, s, g, in, segs, (float*)y, ldy); \
    else hipLaunchKernelGGL((scan_token_kernel<uint16_t, LPC, R>), grid, dim3(256), 0, s, g, in, segs, (uint16_t*)y, ldy); }
  MI_BY_STATE(MI_ST)
#undef MI_ST
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_scan_prompt(const ScanGeom& g, const ScanIn& in, const AttnSeg* segs, int nseg, void* y, int ldy, bool f32, hipStream_t s) {
  int rc = check_scan(g, in, y, ldy);
  if (rc != MI_OK) return rc;
  MI_CHECK(nseg >= 1 && nseg <= 65535 && segs && in.dt && in.ldt >= g.C, "selective scan: segments");
  int num_cu = 0;
  rc = device_num_cu(&num_cu);
  if (rc != MI_OK) return rc;
#define MI_SP(LPC, R) { \
    const dim3 grid(ceil_div(g.C, 256 / LPC), nseg); \
    if (f32) hipLaunchKernelGGL((scan_prompt_kernel<float, LPC, R>), grid, dim3(256), 0, s, g, in, segs, (float*)y, ldy); \
    else hipLaunchKernelGGL((scan_prompt_kernel<uint16_t, LPC, R>), grid, dim3(256), 0, s, g, in, segs, (uint16_t*)y, ldy); }
  if (g.Np == 16 && (size_t)g.C * nseg >= (size_t)num_cu * 32) {   // enough channels for two states per lane: fewer sums over lanes
    MI_SP(8, 2)
  } else {
    MI_BY_STATE(MI_SP)
  }
#undef MI_SP
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_scan_decay(const float* a_log, const ScanGeom& g, float* a2, hipStream_t s) {
  hipLaunchKernelGGL(scan_decay_kernel, dim3(ceil_div(g.C * g.N, 256)), dim3(256), 0, s, a_log, g.C, g.N, g.Np, a2);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

SsdGeom ssd_geom(int H, int P, int N, int G) { return SsdGeom{H, P, N, G, (P + 15) / 16 * 16, (N + 15) / 16 * 16}; }
bool ssd_supported(const SsdGeom& g) {
  return g.H >= 1 && g.G >= 1 && g.H % g.G == 0 && g.P >= 1 && g.P <= 256 && g.N >= 1 && g.N <= 256;
}
size_t ssd_chunk_floats(const SsdGeom& g) { return g.state_floats() + (size_t)g.G * kQ * kQ + g.H; }

int launch_ssd_token(const SsdGeom& g, const SsdIn& in, int rows, const AttnSeg* segs, float* y, int ldy, bool f32, hipStream_t s) {
  int rc = check_ssd(g, in, y, ldy);
  if (rc != MI_OK) return rc;
  MI_CHECK(rows >= 1 && rows <= 65535, "state-space duality: rows");
  const dim3 grid(g.H, rows);
  const int vq = g.Pp <= 16 ? 4 : g.Pp <= 32 ? 8 : g.Pp <= 64 ? 16 : g.Pp <= 128 ? 32 : 64, need = ceil_div(g.Np, kTokenThreads / vq);
#define MI_ST(VQ, RPT) \
  if (f32) hipLaunchKernelGGL((ssd_token_kernel<float, VQ, RPT>), grid, dim3(kTokenThreads), 0, s, g, in, segs, y, ldy); \
  else hipLaunchKernelGGL((ssd_token_kernel<uint16_t, VQ, RPT>), grid, dim3(kTokenThreads), 0, s, g, in, segs, y, ldy)
  if (vq == 4) { if (need <= 1) { MI_ST(4, 1); } else { MI_ST(4, 2); } }
  else if (vq == 8) { if (need <= 1) { MI_ST(8, 1); } else if (need <= 2) { MI_ST(8, 2); } else { MI_ST(8, 4); } }
  else if (vq == 16) { if (need <= 2) { MI_ST(16, 2); } else if (need <= 4) { MI_ST(16, 4); } else { MI_ST(16, 8); } }
  else if (vq == 32) { if (need <= 4) { MI_ST(32, 4); } else if (need <= 8) { MI_ST(32, 8); } else { MI_ST(32, 16); } }
  else { if (need <= 8) { MI_ST(64, 8); } else if (need <= 16) { MI_ST(64, 16); } else { MI_ST(64, 32); } }
#undef MI_ST
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_ssd_prompt(const SsdGeom& g, const SsdIn& in, const AttnSeg* sd, const AttnSeg* sh, int nseg, float* records, int max_chunks, float* y, int ldy,
                      bool f32, hipStream_t s) {
  int rc = check_ssd(g, in, y, ldy);
  if (rc != MI_OK) return rc;
  MI_CHECK(nseg >= 1 && nseg <= 65535 && records && max_chunks >= 1, "state-space duality: segments / workspace");
  int chunks = 0;
  for (int i = 0; i < nseg; ++i) chunks += sh[i].n < 2 ? 0 : ceil_div(sh[i].n, kQ);
  const size_t lds_c = (size_t)kQ * std::max(wide_pitch(g.Np) + wide_pitch(g.Pp), 2 * tall_pitch(g.Np)) * 4;
  const size_t lds_o = (size_t)kQ * (kQ + 4 + wide_pitch(g.Pp) + tall_pitch(g.Np)) * 4;
  const int npt = g.Pp <= 16 ? 1 : g.Pp <= 32 ? 2 : g.Pp <= 64 ? 4 : g.Pp <= 128 ? 8 : 16;
  for (int c0 = 0; c0 < chunks; c0 += max_chunks) {
    const int n = std::min(max_chunks, chunks - c0);
    const dim3 gc(n, g.H + g.G), gp((unsigned)ceil_div((int)(g.state_floats() / 4), 256), nseg), go(n, g.H);
#define MI_SSD_LDS(KERN, BYTES) \
    if (BYTES > 48 * 1024) { rc = ensure_dynamic_lds(reinterpret_cast<const void*>(KERN), (int)(BYTES)); if (rc != MI_OK) return rc; }
#define MI_SSD_CHUNK(T) { auto k = ssd_chunk_kernel<T>; MI_SSD_LDS(k, lds_c) hipLaunchKernelGGL(k, gc, dim3(256), lds_c, s, g, in, sd, nseg, c0, records); }
#define MI_SSD_OUT(T, NPT) { auto k = ssd_out_kernel<T, NPT>; MI_SSD_LDS(k, lds_o) hipLaunchKernelGGL(k, go, dim3(256), lds_o, s, g, in, sd, nseg, c0, records, y, ldy); }
#define MI_SSD_OUT_T(NPT) if (f32) MI_SSD_OUT(float, NPT) else MI_SSD_OUT(uint16_t, NPT)
    if (f32) MI_SSD_CHUNK(float) else MI_SSD_CHUNK(uint16_t)
    hipLaunchKernelGGL(ssd_pass_kernel, gp, dim3(256), 0, s, g, in, sd, c0, n, records);
    switch (npt) {
      case 1: MI_SSD_OUT_T(1); break;
      case 2: MI_SSD_OUT_T(2); break;
      case 4: MI_SSD_OUT_T(4); break;
      case 8: MI_SSD_OUT_T(8); break;
      default: MI_SSD_OUT_T(16);
    }
#undef MI_SSD_OUT_T
#undef MI_SSD_OUT
#undef MI_SSD_CHUNK
#undef MI_SSD_LDS
    MI_HIP(hipGetLastError());
  }
  return MI_OK;
}

int launch_gated_norm(const float* y, int ldy, const float* z, int ldz, const float* w, int n, int parts, float eps, int rows, void* out, int ldo, bool f32,
                      hipStream_t s) {
  MI_CHECK(y && z && w && out && rows >= 1 && n >= 1 && parts >= 1 && n % parts == 0 && ldy >= n && ldz >= n && ldo >= n, "gated norm: equal parts / strides");
  const size_t lds = ((size_t)(n + 3) / 4 * 4 + std::max(parts, 16) + parts) * sizeof(float);
  MI_CHECK(lds <= 160 * 1024, "gated norm: row too long");
  const int threads = rows <= 32 ? std::min(1024, ceil_div(ceil_div(n, 4), 64) * 64) : 256;
  const void* kern = f32 ? reinterpret_cast<const void*>(gated_norm_kernel<float>) : reinterpret_cast<const void*>(gated_norm_kernel<uint16_t>);
  if (lds > 64 * 1024) { int rc = ensure_dynamic_lds(kern, 160 * 1024); if (rc != MI_OK) return rc; }
  if (f32) hipLaunchKernelGGL((gated_norm_kernel<float>), dim3(rows), dim3(threads), lds, s, y, ldy, z, ldz, w, n, parts, eps, (float*)out, ldo);
  else hipLaunchKernelGGL((gated_norm_kernel<uint16_t>), dim3(rows), dim3(threads), lds, s, y, ldy, z, ldz, w, n, parts, eps, (uint16_t*)out, ldo);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

}  // namespace mi
