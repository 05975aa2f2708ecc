// State-space mixers.  See ssm.h.
#include "ssm.h"

#include <algorithm>
#include <type_traits>

namespace mi {

namespace {

constexpr float kLog2e = 1.4426950408889634f;

__device__ __forceinline__ float silu(float v) { return v * __builtin_amdgcn_rcpf(1.f + __expf(-v)); }
// max(v, 0) + log(1 + w), w = exp(-|v|); log(1 + w) as log(u) w / (u - 1) with u = 1 + w as it is rounded: right to the last places however small w is
__device__ __forceinline__ float softplus(float v) {
  const float w = __expf(-fabsf(v)), u = 1.f + w, d = u - 1.f;
  return fmaxf(v, 0.f) + (d > 0.f ? __logf(u) * w * __builtin_amdgcn_rcpf(d) : w);
}
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

// LPC lanes per channel, R consecutive states per lane (Np = LPC R), RB rows per work-group: the decays and the step sizes' weights are read
// once for them, and every row's state is requested before any is used.
template <typename T, int LPC, int R, int RB>
__global__ __launch_bounds__(256) void scan_token_kernel(ScanGeom g, ScanIn in, const AttnSeg* __restrict__ segs, int rows, T* __restrict__ y, int ldy) {
  constexpr int CB = 256 / LPC;
  extern __shared__ __attribute__((aligned(16))) float lows[];     // [RB][rank_p]
  int row[RB], seq[RB];
  bool live[RB], any = false;
#pragma unroll
  for (int b = 0; b < RB; ++b) {
    const int i = blockIdx.y * RB + b;
    live[b] = i < rows;
    row[b] = seq[b] = min(i, rows - 1);
    if (segs) {
      const AttnSeg sg = segs[row[b]];
      live[b] = live[b] && sg.n == 1;
      row[b] = sg.row0; seq[b] = sg.seq;
    }
    any = any || live[b];
  }
  if (!any) return;
  for (int i = threadIdx.x; i < RB * g.rank_p; i += 256) {
    const int b = i / g.rank_p, k = i - b * g.rank_p;
    int r = row[0];
#pragma unroll
    for (int q = 1; q < RB; ++q) r = b == q ? row[q] : r;
    lows[i] = k < g.rank ? round_to(in.low[(size_t)r * in.ldl + k], y) : 0.f;
  }
  const int l = threadIdx.x % LPC, c = blockIdx.x * CB + threadIdx.x / LPC, cc = min(c, g.C - 1);     // (lanes past the last channel repeat it)
  const float* a2 = in.a2 + (size_t)cc * g.Np + l * R;
  float S[RB][R], A[R], B[RB][R], Cn[RB][R], x[RB], z[RB], dot[RB];
  float* S0[RB];
#pragma unroll
  for (int r = 0; r < R; ++r) A[r] = a2[r];
#pragma unroll
  for (int b = 0; b < RB; ++b) {
    S0[b] = in.state + ((size_t)in.slots[seq[b]] * g.C + cc) * g.Np + l * R;
    const float* lo = in.low + (size_t)row[b] * in.ldl;
#pragma unroll
    for (int r = 0; r < R; ++r) S[b][r] = S0[b][r];
    if (l * R + R <= g.N) {                            // (one load where R allows)
#pragma unroll
      for (int r = 0; r < R; ++r) { B[b][r] = lo[in.col_b + l * R + r]; Cn[b][r] = lo[in.col_c + l * R + r]; }
    } else {
#pragma unroll
      for (int r = 0; r < R; ++r) {
        const int n = min(l * R + r, g.N - 1);
        B[b][r] = l * R + r < g.N ? lo[in.col_b + n] : 0.f;
        Cn[b][r] = lo[in.col_c + n];
      }
    }
    x[b] = to_f32(reinterpret_cast<const T*>(in.x)[(size_t)row[b] * in.ldx + cc]);
    z[b] = in.z[(size_t)row[b] * in.ldz + cc];
    dot[b] = 0.f;
  }
  __syncthreads();
  const T* w = reinterpret_cast<const T*>(in.w_dt) + (size_t)cc * g.rank_p;
  for (int k = l * 8; k < g.rank_p; k += LPC * 8) {
    const float4 w0 = get4(w + k), w1 = get4(w + k + 4);             // (zero beyond the rank)
#pragma unroll
    for (int b = 0; b < RB; ++b) {
      const float4 u = *reinterpret_cast<const float4*>(lows + b * g.rank_p + k), v = *reinterpret_cast<const float4*>(lows + b * g.rank_p + k + 4);
      dot[b] = __builtin_fmaf(w0.x, u.x, dot[b]); dot[b] = __builtin_fmaf(w0.y, u.y, dot[b]); dot[b] = __builtin_fmaf(w0.z, u.z, dot[b]); dot[b] = __builtin_fmaf(w0.w, u.w, dot[b]);
      dot[b] = __builtin_fmaf(w1.x, v.x, dot[b]); dot[b] = __builtin_fmaf(w1.y, v.y, dot[b]); dot[b] = __builtin_fmaf(w1.z, v.z, dot[b]); dot[b] = __builtin_fmaf(w1.w, v.w, dot[b]);
    }
  }
  const float bias = in.dt_bias[cc], skip = in.d[cc];
#pragma unroll
  for (int b = 0; b < RB; ++b) {
    const float dt = softplus(lanes_sum<LPC>(dot[b]) + bias), dx = dt * x[b];
    const bool fresh = in.pos[row[b]] == 0;
    float o = 0.f;
#pragma unroll
    for (int r = 0; r < R; ++r) {
      S[b][r] = __builtin_fmaf(__builtin_amdgcn_exp2f(dt * A[r]), fresh ? 0.f : S[b][r], dx * B[b][r]);
      o = __builtin_fmaf(S[b][r], Cn[b][r], o);
    }
    o = lanes_sum<LPC>(o);
    if (!live[b] || c >= g.C) continue;
#pragma unroll
    for (int r = 0; r < R; ++r) S0[b][r] = S[b][r];
    if (l == 0) put1(y + (size_t)row[b] * ldy + c, __builtin_fmaf(skip, x[b], o) * silu(z[b]));
  }
}

// Four values summed over the LPC lanes of a group, lane l left with the sum of value token_of(l)
template <int LPC>
__device__ __forceinline__ int token_of(int l) { return LPC == 16 ? (l >> 3) * 2 + ((l >> 2) & 1) : (l >> 2) * 2 + ((l >> 1) & 1); }
template <int CTRL>
__device__ __forceinline__ float swap_add(float a, float b, bool upper) {    // lower lanes: a + the partner's a; upper lanes: b + the partner's b
  const float send = upper ? a : b;
  return (upper ? b : a) + __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, send), CTRL, 0xf, 0xf, true));
}
template <int LPC>
__device__ __forceinline__ float sum_four(const float (&v)[4], int l) {
  if constexpr (LPC == 16) {       // partners 15 - l, then 7 - l within eight, then inside quads
    const float a = swap_add<0x140>(v[0], v[2], l & 8), b = swap_add<0x140>(v[1], v[3], l & 8);
    const float r = swap_add<0x141>(a, b, l & 4);
    return dpp_add<0x4E>(dpp_add<0xB1>(r));
  } else {                         // partners 7 - l, then l ^ 2, then l ^ 1
    const float a = swap_add<0x141>(v[0], v[2], l & 4), b = swap_add<0x141>(v[1], v[3], l & 4);
    return dpp_add<0xB1>(swap_add<0x4E>(a, b, l & 2));
  }
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
  const int tok = token_of<LPC>(l);
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
    // four tokens' operands are read while the four before them are worked off
    struct Four { float d[4], x[4], b[R][4], c[R][4]; };
    auto take = [&](Four& f, int t) {
      auto four = [](float* o, const float* p) { const float4 v = *reinterpret_cast<const float4*>(p); o[0] = v.x; o[1] = v.y; o[2] = v.z; o[3] = v.w; };
      four(f.d, &dts[cl][t]);
      four(f.x, &dxs[cl][t]);
#pragma unroll
      for (int r = 0; r < R; ++r) { four(f.b[r], &Bs[l * R + r][t]); four(f.c[r], &Cs[l * R + r][t]); }
    };
    Four f[2];
    take(f[0], 0);
#pragma unroll
    for (int t = 0; t < TB; t += 4) {
      const Four& q = f[(t >> 2) & 1];
      if (t + 4 < TB) take(f[((t >> 2) + 1) & 1], t + 4);
      float e[R][4], o[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int r = 0; r < R; ++r)
#pragma unroll
        for (int u = 0; u < 4; ++u) e[r][u] = __builtin_amdgcn_exp2f(q.d[u] * A[r]);
#pragma unroll
      for (int u = 0; u < 4; ++u)
#pragma unroll
        for (int r = 0; r < R; ++r) {
          S[r] = __builtin_fmaf(e[r][u], S[r], q.x[u] * q.b[r][u]);
          o[u] = __builtin_fmaf(S[r], q.c[r][u], o[u]);
        }
      const float sum = sum_four<LPC>(o, l);
      if ((l & (LPC / 4 - 1)) == 0) ys[cl][t + tok] = sum;
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
__global__ __launch_bounds__(kTokenThreads) void ssd_token_kernel(SsdGeom g, SsdIn in, ShortConv cv, const float* __restrict__ proj, int ldp, const AttnSeg* __restrict__ segs,
                                                                  float* __restrict__ y, int ldy) {
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
  const int inner = g.H * g.P, hpg = g.H / g.G, grp = h / hpg;
  if (proj) {      // convolutions of the head's channels and its group's B and C; position p goes to a row of the ring that nobody reads in this launch
    const int C = cv.C, p = in.pos[row];
    const float* x = proj + (size_t)row * ldp;
    float* ring = cv.ring + (size_t)cv.slots[seq] * cv.taps * C;
    for (int i = tid; i < g.Pp + 2 * g.Np; i += kTokenThreads) {
      const int part = i < g.Pp ? 0 : i < g.Pp + g.Np ? 1 : 2, d = i - (part == 0 ? 0 : g.Pp + (part - 1) * g.Np);
      float a = 0.f;
      if (d < (part ? g.N : g.P)) {
        const int ch = part == 0 ? h * g.P + d : inner + ((part - 1) * g.G + grp) * g.N + d;
        const float now = x[ch];
        a = cv.b[ch];
        for (int j = 0; j + 1 < cv.taps; ++j) {
          const int q = p - (cv.taps - 1 - j);
          const float v = ring[(size_t)(max(q, 0) % cv.taps) * C + ch];
          a = __builtin_fmaf(cv.w[(size_t)j * C + ch], q >= 0 ? v : 0.f, a);
        }
        a = round_to(silu(__builtin_fmaf(cv.w[(size_t)(cv.taps - 1) * C + ch], now, a)), (const T*)nullptr);
        if (part == 0 || h % hpg == 0) ring[(size_t)(p % cv.taps) * C + ch] = now;
      }
      (part == 0 ? xs : part == 1 ? bs : cs)[d] = a;
    }
  } else {
    const T* xr = reinterpret_cast<const T*>(in.xbc) + (size_t)row * in.ldx;
    for (int i = tid; i < g.Np; i += kTokenThreads) {
      bs[i] = i < g.N ? to_f32(xr[inner + grp * g.N + i]) : 0.f;
      cs[i] = i < g.N ? to_f32(xr[inner + (g.G + grp) * g.N + i]) : 0.f;
    }
    for (int i = tid; i < g.Pp; i += kTokenThreads) xs[i] = i < g.P ? to_f32(xr[h * g.P + i]) : 0.f;
  }
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

// What a piece of chunks leaves in memory: C B^T [chunk][G][kQ][kQ], and per head the chunk's steps [chunk][H]
struct Steps {
  float hi[kQ], lo[kQ];       // running sum of the decays' logarithms (base 2), in two parts: a difference of two sums is exact to fp32's last place
  float dt[kQ], e[kQ], w[kQ]; // step size; decay from the chunk's start; dt times the decay up to the chunk's end
};
struct Records { float* cb; Steps* steps; };
__host__ __device__ inline Records records_at(float* base, const SsdGeom& g, int chunks) {
  return Records{base, reinterpret_cast<Steps*>(base + (size_t)chunks * g.G * kQ * kQ)};
}
// LDS pitch of rows of which 16 lanes read one column each
__host__ __device__ inline int tall_pitch(int n) { return (n + 63) / 64 * 64 + 4; }

// columns col .. + n of the chunk's rows in LDS rows of `pitch`, zeros up to np and beyond the last row
template <typename T>
__device__ __forceinline__ void stage_rows(float* dst, int pitch, const T* src, int ld, int rows, int n, int np) {
  const int tid = threadIdx.x;
  if (((n | ld) & 3) == 0 && (reinterpret_cast<uintptr_t>(src) & (4 * sizeof(T) - 1)) == 0) {
    const int q = np / 4;
    constexpr int U = 8;                 // in flight together
    for (int i0 = tid; i0 < kQ * q; i0 += 256 * U) {
      float4 v[U];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int i = min(i0 + 256 * u, kQ * q - 1), t = i / q, c = (i - t * q) * 4;
        v[u] = get4(src + (size_t)min(t, rows - 1) * ld + min(c, n - 4));
      }
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int i = i0 + 256 * u, t = i / q, c = (i - t * q) * 4;
        if (i < kQ * q) *reinterpret_cast<float4*>(dst + t * pitch + c) = t < rows && c < n ? v[u] : make_float4(0.f, 0.f, 0.f, 0.f);
      }
    }
    return;
  }
  for (int i = tid; i < kQ * np; i += 256) {
    const int t = i / np, c = i - t * np;
    dst[t * pitch + c] = t < rows && c < n ? to_f32(src[(size_t)t * ld + c]) : 0.f;
  }
}

// Of every chunk: C B^T, a work-group per group (blockIdx.y < G), and the heads' steps, a wave per head
template <typename T>
__global__ __launch_bounds__(256) void ssd_chunk_kernel(SsdGeom g, SsdIn in, const AttnSeg* __restrict__ segs, int nseg, int c0, float* __restrict__ base) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const ChunkAt at = chunk_at(segs, nseg, c0 + blockIdx.x);
  if (!at.ok) return;
  const Records rec = records_at(base, g, gridDim.x);
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, g4 = lane >> 4, c = lane & 15, inner = g.H * g.P;
  if ((int)blockIdx.y >= g.G) {
    const int h = (blockIdx.y - g.G) * 4 + wave;
    if (h >= g.H) return;
    const float dt = lane < at.n ? softplus(in.dt[(size_t)(at.sg.row0 + at.t0 + min(lane, at.n - 1)) * in.ldt + h] + in.dt_bias[h]) : 0.f;
    double s = (double)(-expf(in.a_log[h]) * dt);
#pragma unroll
    for (int m = 1; m < 64; m *= 2) {
      const double v = __shfl_up(s, m);
      if (lane >= m) s += v;
    }
    const double end = __shfl(s, 63), l2 = s * 1.4426950408889634;
    Steps& st = rec.steps[(size_t)blockIdx.x * g.H + h];
    st.hi[lane] = (float)l2;
    st.lo[lane] = (float)(l2 - (double)(float)l2);
    st.dt[lane] = dt;
    st.e[lane] = expf((float)s);
    st.w[lane] = dt * expf((float)(end - s));
    return;
  }
  const T* rows = reinterpret_cast<const T*>(in.xbc) + (size_t)(at.sg.row0 + at.t0) * in.ldx;
  const int grp = blockIdx.y, pitch = tall_pitch(g.Np);
  float *Bs = sm, *Cs = sm + kQ * pitch;
  stage_rows(Bs, pitch, rows + inner + grp * g.N, in.ldx, at.n, g.N, g.Np);
  stage_rows(Cs, pitch, rows + inner + (g.G + grp) * g.N, in.ldx, at.n, g.N, g.Np);
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

// N elements as they lie in memory, in whole registers: taken apart where they are used, so that a load stays in flight until then
template <typename T, int N>
struct Words {
  static constexpr int BYTES = N * (int)sizeof(T), Q = BYTES >= 16 ? 4 : BYTES / 4, NV = BYTES / (4 * Q);
  typedef __attribute__((ext_vector_type(Q))) unsigned vec_t;
  vec_t v[NV];
  __device__ __forceinline__ void load(const T* p) {
#pragma unroll
    for (int i = 0; i < NV; ++i) v[i] = reinterpret_cast<const vec_t*>(p)[i];
  }
  __device__ __forceinline__ void store(T* p) const {
#pragma unroll
    for (int i = 0; i < NV; ++i) reinterpret_cast<vec_t*>(p)[i] = v[i];
  }
  __device__ __forceinline__ float at(int i) const {
    constexpr int E = 4 / (int)sizeof(T);
    const unsigned w = v[i / E / Q][i / E % Q];
    return E == 1 ? __builtin_bit_cast(float, w) : i & 1 ? bf16hi_to_f32(w) : bf16lo_to_f32(w);
  }
  __device__ __forceinline__ void set(int i, T x) {          // (elements in ascending order)
    constexpr int E = 4 / (int)sizeof(T);
    unsigned& w = reinterpret_cast<unsigned*>(v)[i / E];
    if constexpr (E == 1) w = __builtin_bit_cast(unsigned, x);
    else w = i & 1 ? w | (unsigned)x << 16 : (unsigned)x;
  }
};
template <typename T, int N> struct alignas(sizeof(T) * N) Pack { T v[N]; };

// LDS of the scan: the waves' shares of a chunk's outputs [2][4][4][64] f32x4, steps [2], x [2][kQ][kXPitch], and per wave B [kQ][b_pitch]
constexpr int kXPitch = 20;
template <typename T, int NT>
constexpr int b_pitch() {      // in elements; rows 4 apart fall into different banks
  constexpr int dw = 16 * NT * (int)sizeof(T) / 4;
  return (dw == 8 ? 12 : dw == 16 ? 20 : dw == 32 ? 40 : 68) * 4 / (int)sizeof(T);
}
template <typename T, int NT>
constexpr size_t scan_lds() { return 2 * 16 * 64 * 16 + 2 * sizeof(Steps) + 2 * kQ * kXPitch * 4 + 4 * kQ * b_pitch<T, NT>() * sizeof(T); }

// One work-group per (head, 16 columns, segment): the chunks of the segment in order.  A wave holds NT 16-row tiles of the state as MFMA
// accumulators, which are the B operands of the next chunk's products as they stand.  Row rho of a wave's tile t is state
// n = 16 NT wave + NT rho + t: a lane's A operands of all tiles lie side by side, in C (registers, four rows of the tiles at a time) as in
// B (through LDS, the wave's own columns).  The waves' shares of a chunk's outputs meet in LDS, one barrier per chunk; what the next
// chunk needs is in flight meanwhile.  VEC: whole 16-byte pieces of rows, aligned.
template <typename T, int NT, bool VEC>
__global__ __launch_bounds__(256) void ssd_scan_kernel(SsdGeom g, SsdIn in, const AttnSeg* __restrict__ segs, int c0, int nchunks, int nvt, float* __restrict__ base,
                                                       float* __restrict__ y, int ldy) {
  extern __shared__ __attribute__((aligned(16))) unsigned char dsm[];
  f32x4_t (*ps)[4][4][64] = reinterpret_cast<f32x4_t (*)[4][4][64]>(dsm);
  Steps* st = reinterpret_cast<Steps*>(dsm + 2 * 16 * 64 * 16);
  float* xs = reinterpret_cast<float*>(st + 2);
  constexpr int BP = b_pitch<T, NT>(), W = 16 / (int)sizeof(T), LPR = 16 * NT / W, RPL = 64 / LPR;    // elements per 16 bytes; lanes per row, rows per load of B
  int id = blockIdx.x, h, vt;
  if (g.H % 8 == 0) {        // the column blocks of a head on one XCD
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
  for (int i = 0; i < si; ++i) first += segs[i].n < 2 ? 0 : ceil_div(segs[i].n, kQ);
  const int k0 = max(c0 - first, 0), k1 = min(c0 + nchunks - first, ceil_div(sg.n, kQ));
  if (k0 >= k1) return;
  const Records rec = records_at(base, g, nchunks);
  const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, g4 = lane >> 4, c = lane & 15;
  const int grp = h / (g.H / g.G), n0 = 16 * NT * wave, p = 16 * vt + c;
  T* Bs = reinterpret_cast<T*>(xs + 2 * kQ * kXPitch) + wave * kQ * BP;
  float* S0 = in.state + ((size_t)in.slots[sg.seq] * g.H + h) * g.Np * g.Pp + p;
  f32x4_t S[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int n = n0 + NT * (4 * g4 + r) + t;
      S[t][r] = sg.pos0 + k0 > 0 && n < g.Np ? S0[(size_t)min(n, g.Np - 1) * g.Pp] : 0.f;
    }
  const T* xbc = reinterpret_cast<const T*>(in.xbc) + (size_t)sg.row0 * in.ldx;
  const int at_b = g.H * g.P + grp * g.N, at_c = at_b + g.G * g.N, at_x = h * g.P + 16 * vt, bn = n0 + (lane % LPR) * W, xn = (tid & 3) * 4;
  struct Kept { Words<T, 4 * NT> c[4]; f32x4_t cb[4]; };                             // used from registers
  struct Passed { Words<T, W> b[LPR]; Words<T, 4> x; float s[2]; };                  // passed on to LDS
  // columns n .. of a row's part of `size` columns; beyond it: anything (C: its states are zero), or zero (B)
  auto pack = [](auto& o, const T* row, int n, int size, bool zero) {
    constexpr int M = (int)(sizeof(o.v) / (sizeof(T)));
    if constexpr (VEC) {
      o.load(row + min(n, size - M));
    } else {
#pragma unroll
      for (int i = 0; i < M; ++i) {
        const T x = row[min(n + i, size - 1)];
        o.set(i, zero && n + i >= size ? T(0) : x);
      }
    }
  };
  constexpr int kSteps = sizeof(Steps) / 4;                // floats of a chunk's steps, shared out to the work-group
  auto load_passed = [&](int k, Passed& d) {
    const int n = min(kQ, sg.n - k * kQ), rc = first + k - c0;
    const T* rows = xbc + (size_t)k * kQ * in.ldx;
    const float* steps = reinterpret_cast<const float*>(rec.steps + (size_t)rc * g.H + h);
#pragma unroll
    for (int i = 0; i < 2; ++i) d.s[i] = steps[min(tid + 256 * i, kSteps - 1)];
    pack(d.x, rows + (size_t)min(tid >> 2, n - 1) * in.ldx + at_x, xn, g.P - 16 * vt, false);
#pragma unroll
    for (int i = 0; i < LPR; ++i) pack(d.b[i], rows + (size_t)min(RPL * i + lane / LPR, n - 1) * in.ldx + at_b, bn, g.N, true);
  };
  auto load_kept = [&](int k, Kept& f) {
    const int n = min(kQ, sg.n - k * kQ), rc = first + k - c0;
    const T* rows = xbc + (size_t)k * kQ * in.ldx;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      pack(f.c[i], rows + (size_t)min(16 * i + c, n - 1) * in.ldx + at_c, n0 + 4 * NT * g4, g.N, false);
      // (tiles above the diagonal are left out: the wave's own again)
      f.cb[i] = *reinterpret_cast<const f32x4_t*>(rec.cb + ((size_t)rc * g.G + grp) * kQ * kQ + (16 * wave + c) * kQ + 16 * min(i, wave) + 4 * g4);
    }
  };
  auto post = [&](const Passed& d, int b) {
    float* s = reinterpret_cast<float*>(&st[b]);
#pragma unroll
    for (int i = 0; i < 2; ++i)
      if (tid + 256 * i < kSteps) s[tid + 256 * i] = d.s[i];
    float xv[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) xv[i] = 16 * vt + xn + i < g.P ? d.x.at(i) : 0.f;
    *reinterpret_cast<float4*>(xs + (b * kQ + (tid >> 2)) * kXPitch + xn) = make_float4(xv[0], xv[1], xv[2], xv[3]);
#pragma unroll
    for (int i = 0; i < LPR; ++i) {
      Words<T, W> v = d.b[i];
      if constexpr (VEC) {
#pragma unroll
        for (int e = 0; e < 4; ++e) v.v[0][e] = bn < g.N ? v.v[0][e] : 0u;
      }
      v.store(Bs + (RPL * i + lane / LPR) * BP + (lane % LPR) * W);
    }
  };
  const float skip = in.d[h];
  auto step = [&](int k, Kept& f, Kept& next) {
    const int b = (k - k0) & 1, n = min(kQ, sg.n - k * kQ);
    const Steps& q = st[b];
    Passed d;                  // (behind the last chunk: that one again)
    load_passed(min(k + 1, k1 - 1), d);
    load_kept(min(k + 1, k1 - 1), next);
    __builtin_amdgcn_sched_barrier(0);
    float x[16];               // tokens 16 i + 4 g4 + r (past the last one: its weight and step are zero)
#pragma unroll
    for (int i = 0; i < 16; ++i) x[i] = xs[(b * kQ + 16 * (i >> 2) + 4 * g4 + (i & 3)) * kXPitch + c];
    // share of the outputs that the state holds
    f32x4_t o[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) o[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r)
#pragma unroll
        for (int i = 0; i < 4; ++i) o[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(f.c[i].at(NT * r + t), S[t][r], o[i], 0, 0, 0);
#pragma unroll
    for (int i = 0; i < 4; ++i) ps[b][wave][i][lane] = o[i];
    // the state behind the chunk
    const float end = q.e[kQ - 1];
#pragma unroll
    for (int t = 0; t < NT; ++t) S[t] = f32x4_t{S[t][0] * end, S[t][1] * end, S[t][2] * end, S[t][3] * end};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const f32x4_t w = *reinterpret_cast<const f32x4_t*>(q.w + 16 * i + 4 * g4);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float xw = x[4 * i + r] * w[r];
        const Pack<T, NT> bv = *reinterpret_cast<const Pack<T, NT>*>(Bs + (16 * i + 4 * g4 + r) * BP + NT * c);
#pragma unroll
        for (int t = 0; t < NT; ++t) S[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(to_f32(bv.v[t]), xw, S[t], 0, 0, 0);
      }
    }
    // what the chunk's own tokens add: the wave's 16 tokens
    f32x4_t own = {0.f, 0.f, 0.f, 0.f};
    const float hi = q.hi[16 * wave + c], lo = q.lo[16 * wave + c];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      if (j > wave) break;
      const f32x4_t hj = *reinterpret_cast<const f32x4_t*>(q.hi + 16 * j + 4 * g4), lj = *reinterpret_cast<const f32x4_t*>(q.lo + 16 * j + 4 * g4),
                    dj = *reinterpret_cast<const f32x4_t*>(q.dt + 16 * j + 4 * g4);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float dt = 16 * j + 4 * g4 + r <= 16 * wave + c ? dj[r] : 0.f, e = __builtin_amdgcn_exp2f(fminf((hi - hj[r]) + (lo - lj[r]), 0.f));
        own = __builtin_amdgcn_mfma_f32_16x16x4f32(f.cb[j][r] * e * dt, x[4 * j + r], own, 0, 0, 0);
      }
    }
    float xo[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) xo[r] = xs[(b * kQ + 16 * wave + 4 * g4 + r) * kXPitch + c];
    const f32x4_t e = *reinterpret_cast<const f32x4_t*>(q.e + 16 * wave + 4 * g4);
    __builtin_amdgcn_sched_barrier(0);
    post(d, b ^ 1);                     // (B: the wave's own reads of it are done)
    __syncthreads();
    f32x4_t sum = ps[b][0][wave][lane];
#pragma unroll
    for (int w = 1; w < 4; ++w) {
      const f32x4_t a = ps[b][w][wave][lane];
      sum[0] += a[0]; sum[1] += a[1]; sum[2] += a[2]; sum[3] += a[3];
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 16 * wave + 4 * g4 + r;
      if (i < n && p < g.P) y[(size_t)(sg.row0 + k * kQ + i) * ldy + h * g.P + p] = __builtin_fmaf(e[r], sum[r], __builtin_fmaf(skip, xo[r], own[r]));
    }
  };
  Kept f[2];
  {
    Passed d;
    load_passed(k0, d);
    load_kept(k0, f[0]);
    post(d, 0);
  }
  __syncthreads();
  for (int k = k0; k < k1; k += 2) {
    step(k, f[0], f[1]);
    if (k + 1 < k1) step(k + 1, f[1], f[0]);
  }
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int n = n0 + NT * (4 * g4 + r) + t;
      if (n < g.Np) S0[(size_t)n * g.Pp] = S[t][r];
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
int check_ssd(const SsdGeom& g, const SsdIn& in, const float* y, int ldy, bool convolved = false) {
  MI_CHECK(ssd_supported(g), "state-space duality: heads must be a multiple of the groups, sizes 1 .. 256");
  MI_CHECK(g.Np % 16 == 0 && g.Np >= g.N && g.Np < g.N + 16 && g.Pp % 16 == 0 && g.Pp >= g.P && g.Pp < g.P + 16, "state-space duality: padding");
  MI_CHECK((convolved || (in.xbc && in.ldx >= g.channels())) && in.dt && in.dt_bias && in.a_log && in.d && in.state && in.slots && in.pos && y, "state-space duality: null argument");
  MI_CHECK(in.ldt >= g.H && ldy >= g.inner(), "state-space duality: columns");
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
  // several rows: four of them per work-group; many: four states per lane as well (fewer, wider loads)
  const bool several = rows >= 3 && g.Np <= 64, many = several && rows > 8;
  const int rb = several ? 4 : 1;
  const size_t lds = (size_t)rb * g.rank_p * 4;
  MI_CHECK(lds <= 48 * 1024, "selective scan: the step sizes' rank is too large");
#define MI_ST_(LPC, R, RB) { \
    const dim3 grid(ceil_div(g.C, 256 / LPC), ceil_div(rows, rb)); \
    if (f32) hipLaunchKernelGGL((scan_token_kernel<float, LPC, R, RB>), grid, dim3(256), lds, s, g, in, segs, rows, (float*)y, ldy); \
    else hipLaunchKernelGGL((scan_token_kernel<uint16_t, LPC, R, RB>), grid, dim3(256), lds, s, g, in, segs, rows, (uint16_t*)y, ldy); }
#define MI_ST(LPC, R) MI_ST_(LPC, R, 1)
  if (!several) {
    MI_BY_STATE(MI_ST)
  } else if (g.Np == 8) { if (many) MI_ST_(4, 2, 4) else MI_ST_(8, 1, 4) }
  else if (g.Np == 16) { if (many) MI_ST_(4, 4, 4) else MI_ST_(16, 1, 4) }
  else if (g.Np == 32) { if (many) MI_ST_(8, 4, 4) else MI_ST_(16, 2, 4) }
  else MI_ST_(16, 4, 4)
#undef MI_ST
#undef MI_ST_
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
size_t ssd_chunk_floats(const SsdGeom& g) { return (size_t)g.G * kQ * kQ + (size_t)g.H * sizeof(Steps) / 4; }

int launch_ssd_token(const SsdGeom& g, const SsdIn& in, int rows, const AttnSeg* segs, float* y, int ldy, bool f32, hipStream_t s, const ShortConv* conv, const float* proj,
                     int ldp) {
  int rc = check_ssd(g, in, y, ldy, conv != nullptr);
  if (rc != MI_OK) return rc;
  MI_CHECK(!conv == !proj && (!conv || (conv->w && conv->b && conv->ring && conv->slots && conv->taps >= 1 && conv->taps <= 16 && conv->C == g.channels() && ldp >= conv->C)),
           "state-space duality: convolution");
  const ShortConv cv = conv ? *conv : ShortConv();
  MI_CHECK(rows >= 1 && rows <= 65535, "state-space duality: rows");
  const dim3 grid(g.H, rows);
  const int vq = g.Pp <= 16 ? 4 : g.Pp <= 32 ? 8 : g.Pp <= 64 ? 16 : g.Pp <= 128 ? 32 : 64, need = ceil_div(g.Np, kTokenThreads / vq);
#define MI_ST(VQ, RPT) \
  if (f32) hipLaunchKernelGGL((ssd_token_kernel<float, VQ, RPT>), grid, dim3(kTokenThreads), 0, s, g, in, cv, proj, ldp, segs, y, ldy); \
  else hipLaunchKernelGGL((ssd_token_kernel<uint16_t, VQ, RPT>), grid, dim3(kTokenThreads), 0, s, g, in, cv, proj, ldp, segs, y, ldy)
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
  const size_t lds = (size_t)kQ * 2 * tall_pitch(g.Np) * 4;
  const int nvt = g.Pp / 16, nt = g.Np <= 64 ? 1 : g.Np <= 128 ? 2 : 4;
  // whole packs of B, C and x, rows and groups aligned to them
  const int unit = std::max(4 * nt, 8);
  const bool vec = g.N % unit == 0 && g.inner() % unit == 0 && g.P % 4 == 0 && in.ldx % unit == 0 && (reinterpret_cast<uintptr_t>(in.xbc) & 63) == 0;
  for (int c0 = 0; c0 < chunks; c0 += max_chunks) {
    const int n = std::min(max_chunks, chunks - c0);
    const dim3 gc(n, g.G + ceil_div(g.H, 4)), gs(g.H * nvt, nseg);
#define MI_SSD_CHUNK(T) { auto k = ssd_chunk_kernel<T>; \
      if (lds > 48 * 1024) { rc = ensure_dynamic_lds(reinterpret_cast<const void*>(k), (int)lds); if (rc != MI_OK) return rc; } \
      hipLaunchKernelGGL(k, gc, dim3(256), lds, s, g, in, sd, nseg, c0, records); }
#define MI_SSD_SCAN(T, NT, VEC) { auto k = ssd_scan_kernel<T, NT, VEC>; constexpr size_t bytes = scan_lds<T, NT>(); \
      if (bytes > 64 * 1024) { rc = ensure_dynamic_lds(reinterpret_cast<const void*>(k), (int)bytes); if (rc != MI_OK) return rc; } \
      hipLaunchKernelGGL(k, gs, dim3(256), bytes, s, g, in, sd, c0, n, nvt, records, y, ldy); }
#define MI_SSD_SCAN_V(T, NT) if (vec) MI_SSD_SCAN(T, NT, true) else MI_SSD_SCAN(T, NT, false)
#define MI_SSD_SCAN_T(NT) if (f32) { MI_SSD_SCAN_V(float, NT) } else { MI_SSD_SCAN_V(uint16_t, NT) }
    if (f32) MI_SSD_CHUNK(float) else MI_SSD_CHUNK(uint16_t)
    if (nt == 1) { MI_SSD_SCAN_T(1) } else if (nt == 2) { MI_SSD_SCAN_T(2) } else { MI_SSD_SCAN_T(4) }
#undef MI_SSD_SCAN_T
#undef MI_SSD_SCAN_V
#undef MI_SSD_SCAN
#undef MI_SSD_CHUNK
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
