// Mixture-of-experts kernels.  See experts.h.
#include "experts.h"

namespace mi {

namespace {

constexpr int kMaxTop = 64, kRouteExperts = 8;

// ---- router ----------------------------------------------------
__device__ __forceinline__ float dot8(const uint16_t* w, const float* x) {
  const uint4 v = *reinterpret_cast<const uint4*>(w);
  float a = bf16lo_to_f32(v.x) * x[0];
  a = __builtin_fmaf(bf16hi_to_f32(v.x), x[1], a); a = __builtin_fmaf(bf16lo_to_f32(v.y), x[2], a);
  a = __builtin_fmaf(bf16hi_to_f32(v.y), x[3], a); a = __builtin_fmaf(bf16lo_to_f32(v.z), x[4], a);
  a = __builtin_fmaf(bf16hi_to_f32(v.z), x[5], a); a = __builtin_fmaf(bf16lo_to_f32(v.w), x[6], a);
  return __builtin_fmaf(bf16hi_to_f32(v.w), x[7], a);
}
__device__ __forceinline__ float dot8(const float* w, const float* x) {
  float a = 0.f;
#pragma unroll
  for (int i = 0; i < 8; ++i) a = __builtin_fmaf(w[i], x[i], a);
  return a;
}
__device__ __forceinline__ void load8f(const uint16_t* p, float* o) {
  const uint4 v = *reinterpret_cast<const uint4*>(p);
  o[0] = bf16lo_to_f32(v.x); o[1] = bf16hi_to_f32(v.x); o[2] = bf16lo_to_f32(v.y); o[3] = bf16hi_to_f32(v.y);
  o[4] = bf16lo_to_f32(v.z); o[5] = bf16hi_to_f32(v.z); o[6] = bf16lo_to_f32(v.w); o[7] = bf16hi_to_f32(v.w);
}
__device__ __forceinline__ void load8f(const float* p, float* o) {
#pragma unroll
  for (int i = 0; i < 8; ++i) o[i] = p[i];
}

__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
  for (int m = 32; m >= 1; m >>= 1) v = fmaxf(v, __shfl_xor(v, m));
  return v;
}
// LDS written by some lanes of a wave, read by others of it: a wave's LDS operations execute in order, the compiler must keep them so
__device__ __forceinline__ void wave_lds_order() {
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  __builtin_amdgcn_wave_barrier();
}
__host__ __device__ __forceinline__ int pick_stride(int E) { return (E + 3) / 4 * 4 + 4; }
__device__ __forceinline__ float route_sigmoid(float z) { return 1.f / (1.f + expf(-z)); }

// sigmoid rule: z [E] logits -> c [E] choice scores, -inf outside the best groups; gs [groups] is scratch
__device__ __forceinline__ void choice_scores(const float* z, float* c, float* gs, int E, const RouterRule& rule) {
  const int lane = threadIdx.x & 63, per = E / rule.groups;
  for (int e = lane; e < E; e += 64) c[e] = route_sigmoid(z[e]) + rule.b[e];
  if (rule.groups == 1 || rule.keep == rule.groups) return;
  wave_lds_order();
  for (int k = lane; k < rule.groups; k += 64) {
    float a = -INFINITY, b = -INFINITY;
    for (int e = k * per; e < (k + 1) * per; ++e) {
      const float v = c[e];
      b = fmaxf(b, fminf(a, v));
      a = fmaxf(a, v);
    }
    gs[k] = per > 1 ? a + b : a;
  }
  wave_lds_order();
  for (int e = lane; e < E; e += 64) {
    const int k = e / per;
    const float mine = gs[k];
    int ahead = 0;
    for (int i = 0; i < rule.groups; ++i) ahead += gs[i] > mine || (gs[i] == mine && i < k) ? 1 : 0;
    if (ahead >= rule.keep) c[e] = -INFINITY;
  }
}

// The `top` best of z [E] (LDS, pick_stride(E) floats and as many for each further array), by one wave; weights, best first, ties to
// the lowest expert.  Up to 256 experts: an expert's place is the number of experts ahead of it; beyond: one maximum after
// another (destroys the scores).
__device__ __forceinline__ void pick_top(float* z, int E, int top, const RouterRule& rule, int32_t* ids, float* weights) {
  const int lane = threadIdx.x & 63;
  float* c = z;
  wave_lds_order();
  if (rule.sigmoid) {
    c = z + pick_stride(E);
    choice_scores(z, c, c + pick_stride(E), E, rule);
    wave_lds_order();
  }
  if (E <= 256) {
    if (lane < 4) c[E + lane] = -INFINITY;
    wave_lds_order();
    float v[4], w[4], mx = -INFINITY, sum = 0.f;
    int place[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int e = lane + 64 * i;
      v[i] = e < E ? c[e] : -INFINITY;
      if (!(v[i] == v[i])) v[i] = -INFINITY;                    // (a NaN is refused)
      place[i] = e < E ? 0 : 1 << 20;
      mx = fmaxf(mx, v[i]);
    }
    for (int j = 0; j < E; j += 4) {
      const float4 q = *reinterpret_cast<const float4*>(c + j);
      const float u[4] = {q.x, q.y, q.z, q.w};
#pragma unroll
      for (int k = 0; k < 4; ++k)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          if (64 * i >= E) break;
          const float t = u[k] == u[k] ? u[k] : -INFINITY;
          place[i] += (t > v[i] || (t == v[i] && j + k < lane + 64 * i)) ? 1 : 0;
        }
    }
    mx = wave_max(mx);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      w[i] = place[i] >= top ? 0.f : rule.sigmoid ? route_sigmoid(z[lane + 64 * i]) : expf(v[i] - mx);
      sum += w[i];
    }
    sum = wave_sum(sum) + (rule.sigmoid ? 1e-20f : 0.f);
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (place[i] < top) { ids[place[i]] = lane + 64 * i; weights[place[i]] = w[i] / sum; }
    return;
  }
  float first = 0.f, sum = 0.f;
  float mine = 0.f;      // lane j keeps the j-th weight
  int mine_id = 0;
  for (int j = 0; j < top; ++j) {
    float best = -INFINITY;
    int at = 0x7fffffff;
    for (int e = lane; e < E; e += 64)
      if (c[e] > best) { best = c[e]; at = e; }
#pragma unroll
    for (int m = 32; m >= 1; m >>= 1) {
      const float v = __shfl_xor(best, m);
      const int i = __shfl_xor(at, m);
      if (v > best || (v == best && i < at)) { best = v; at = i; }
    }
    if (at >= E) at = j;       // (nothing but -inf or NaN left)
    if (j == 0) first = best;
    const float w = rule.sigmoid ? route_sigmoid(z[at]) : expf(best - first);
    sum += w;
    if (lane == j) { mine = w; mine_id = at; }
    if (lane == (at & 63)) c[at] = -INFINITY;     // (the lane that reads it)
  }
  if (rule.sigmoid) sum += 1e-20f;
  if (lane < top) { ids[lane] = mine_id; weights[lane] = mine / sum; }
}

// one work-group per row and kRouteExperts experts, or (no tickets) per row; a wave takes two experts at a time, their rows and x
// requested together
template <typename T>
__global__ __launch_bounds__(256) void route_kernel(const T* __restrict__ x, int ldx, const T* __restrict__ w, RouterRule rule, int E,
                                                        int K, int top, int32_t* __restrict__ ids, float* __restrict__ weights, float* __restrict__ zg,
                                                        uint32_t* __restrict__ tickets) {
  constexpr int NW = 4, EPW = 2;
  extern __shared__ __attribute__((aligned(16))) float z[];   // as pick_top
  __shared__ uint32_t arrived;
  const int e0 = blockIdx.y * kRouteExperts, e1 = tickets ? min(e0 + kRouteExperts, E) : E;
  const int t = blockIdx.x, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  for (int e = e0 + wave * EPW; e < e1; e += NW * EPW) {
    float a[EPW];
    const T* we[EPW];
#pragma unroll
    for (int i = 0; i < EPW; ++i) { a[i] = 0.f; we[i] = w + (size_t)min(e + i, e1 - 1) * K; }
#pragma unroll 4
    for (int k = lane * 8; k < K; k += 512) {
      float xv[8];
      load8f(x + (size_t)t * ldx + k, xv);
#pragma unroll
      for (int i = 0; i < EPW; ++i) a[i] += dot8(we[i] + k, xv);
    }
    float v = 0.f;
#pragma unroll
    for (int i = 0; i < EPW; ++i) {
      const float s = wave_sum(a[i]);
      v = lane == i ? s : v;
    }
    if (lane >= EPW || e + lane >= e1) continue;
    if (!rule.sigmoid) v += rule.b[e + lane];
    if (tickets) __hip_atomic_store(zg + (size_t)t * E + e + lane, v, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    else z[e + lane] = v;
  }
  if (tickets) {       // the row's last work-group to arrive picks; it leaves the ticket at zero for the next launch
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");   // every storing wave drains its write-through stores
    __syncthreads();
    if (tid == 0) arrived = __hip_atomic_fetch_add(tickets + t, 1u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    __syncthreads();
    if (arrived != gridDim.y - 1) return;
    for (int e = tid; e < E; e += NW * 64) z[e] = __hip_atomic_load(zg + (size_t)t * E + e, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    if (tid == 0) __hip_atomic_store(tickets + t, 0u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  }
  __syncthreads();
  if (wave == 0) pick_top(z, E, top, rule, ids + (size_t)t * top, weights + (size_t)t * top);
}

// a wave per row
__global__ __launch_bounds__(256) void route_pick_kernel(const float* __restrict__ zg, int ldz, int T, RouterRule rule, int E, int top, int32_t* __restrict__ ids,
                                                         float* __restrict__ weights) {
  extern __shared__ __attribute__((aligned(16))) float sm[];   // 4 x pick_top's
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, t = blockIdx.x * 4 + wave;
  if (t >= T) return;
  float* z = sm + wave * (rule.sigmoid ? 3 : 1) * pick_stride(E);            // (one wave's own: LDS operations of a wave execute in order)
  for (int e = lane; e < E; e += 64) z[e] = zg[(size_t)t * ldz + e];
  pick_top(z, E, top, rule, ids + (size_t)t * top, weights + (size_t)t * top);
}

__device__ __forceinline__ uint2 relu2x4(f32x4_t v) {
  auto f = [](float x) { x = fmaxf(x, 0.f); return x * x; };
  return make_uint2(pack_bf16x2(f(v[0]), f(v[1])), pack_bf16x2(f(v[2]), f(v[3])));
}

// ---- experts' linear layers, few rows: weight streaming -------------------------------------------------------------------
// One work-group per (16-row weight tile or KS = 1: four of them, expert).  The pairs that chose the expert are found by a scan
// over the pair list, in pair order, and taken 16 at a time as the columns of the MFMA tiles.
template <int KS, int ACT>
__global__ __launch_bounds__(256) void experts_stream_kernel(const uint4* __restrict__ w, int NT, int KT, const int32_t* __restrict__ ids, int P,
                                                             const uint16_t* __restrict__ x, int ldx, int x_div, void* __restrict__ y, int ldy) {
  __shared__ int list[256], count[4];
  __shared__ f32x4_t red[KS == 1 ? 1 : 4 * 64];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, g4 = lane >> 4, c = lane & 15, e = blockIdx.y;
  const int nt = KS == 1 ? (int)blockIdx.x * 4 + wave : (int)blockIdx.x;
  const int per = KS == 1 ? KT : ceil_div(KT, KS), k0 = KS == 1 ? 0 : wave * per, k1 = min(k0 + per, KT);
  for (int base = 0; base < P; base += 256) {
    const bool hit = base + tid < P && ids[base + tid] == e;
    const unsigned long long mask = __ballot(hit);
    __syncthreads();                                  // the previous round's list is used up
    if (lane == 0) count[wave] = __popcll(mask);
    __syncthreads();
    int before = 0, n = 0;
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      before += v < wave ? count[v] : 0;
      n += count[v];
    }
    if (hit) list[before + __popcll(mask & ((1ull << lane) - 1))] = base + tid;
    __syncthreads();
    for (int p0 = 0; p0 < n; p0 += 16) {
      const bool live = p0 + c < n;
      const int pair = list[min(p0 + c, n - 1)];
      const uint16_t* X = x + (size_t)(pair / x_div) * ldx + g4 * 8;
      f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
      if (nt < NT) {
        const u32x4_t* W = reinterpret_cast<const u32x4_t*>(w) + ((size_t)e * NT + nt) * KT * 64 + lane;
        constexpr int U = 8;
        int kt = k0;
        for (; kt + U <= k1; kt += U) {
          u32x4_t a[U], b[U];
#pragma unroll
          for (int u = 0; u < U; ++u) a[u] = __builtin_nontemporal_load(W + (size_t)(kt + u) * 64);
#pragma unroll
          for (int u = 0; u < U; ++u) b[u] = live ? *reinterpret_cast<const u32x4_t*>(X + (kt + u) * 32) : u32x4_t{0, 0, 0, 0};
#pragma unroll
          for (int u = 0; u < U; ++u) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a[u]), __builtin_bit_cast(bf16x8_t, b[u]), acc, 0, 0, 0);
        }
        for (; kt < k1; ++kt) {
          const u32x4_t a = W[(size_t)kt * 64], b = live ? *reinterpret_cast<const u32x4_t*>(X + kt * 32) : u32x4_t{0, 0, 0, 0};
          acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a), __builtin_bit_cast(bf16x8_t, b), acc, 0, 0, 0);
        }
      }
      if constexpr (KS > 1) {
        if (p0) __syncthreads();                      // the previous chunk's sums are read
        red[wave * 64 + lane] = acc;
        __syncthreads();
        if (wave == 0) {
#pragma unroll
          for (int v = 1; v < KS; ++v) {
            const f32x4_t r = red[v * 64 + lane];
            acc[0] += r[0]; acc[1] += r[1]; acc[2] += r[2]; acc[3] += r[3];
          }
        }
      }
      if ((KS == 1 || wave == 0) && live && nt < NT) {
        const int n0 = nt * 16 + g4 * 4;
        if constexpr (ACT == EXPERT_RELU2) {
          *reinterpret_cast<uint2*>(reinterpret_cast<uint16_t*>(y) + (size_t)pair * ldy + n0) = relu2x4(acc);
        } else if constexpr (ACT == EXPERT_SILU_GLU) {
          const float a0 = acc[0] / (1.f + __expf(-acc[0])) * acc[1], a1 = acc[2] / (1.f + __expf(-acc[2])) * acc[3];
          *reinterpret_cast<uint32_t*>(reinterpret_cast<uint16_t*>(y) + (size_t)pair * ldy + (n0 >> 1)) = pack_bf16x2(a0, a1);
        } else {
          *reinterpret_cast<float4*>(reinterpret_cast<float*>(y) + (size_t)pair * ldy + n0) = make_float4(acc[0], acc[1], acc[2], acc[3]);
        }
      }
    }
  }
}

// 32-bit form: a wave per output of one pair (for checking)
template <int ACT>
__global__ __launch_bounds__(256) void experts_f32_kernel(const float* __restrict__ w, int N, int K, const int32_t* __restrict__ ids,
                                                          const float* __restrict__ x, int ldx, int x_div, float* __restrict__ y, int ldy) {
  constexpr bool GLU = ACT == EXPERT_SILU_GLU;
  const int p = blockIdx.x, n = blockIdx.y * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (n >= (GLU ? N / 2 : N)) return;
  const float *X = x + (size_t)(p / x_div) * ldx, *W = w + ((size_t)ids[p] * N + (GLU ? 2 * n : n)) * K;
  float a = 0.f, b = 0.f;
  for (int k = lane; k < K; k += 64) {
    a = __builtin_fmaf(W[k], X[k], a);
    if constexpr (GLU) b = __builtin_fmaf(W[K + k], X[k], b);
  }
  a = wave_sum(a);
  if constexpr (GLU) {
    b = wave_sum(b);
    a = a / (1.f + expf(-a)) * b;
  }
  if constexpr (ACT == EXPERT_RELU2) { a = fmaxf(a, 0.f); a *= a; }
  if (lane == 0) y[(size_t)p * ldy + n] = a;
}

// ---- experts' linear layers, many rows -----------------------------------------------------------------------------------
// Group the pairs by expert: count, place, list the tiles.  One work-group.
__global__ __launch_bounds__(1024) void experts_sort_kernel(const int32_t* __restrict__ ids, int P, int E, ExpertPlan plan) {
  extern __shared__ __attribute__((aligned(16))) int cnt[];    // [E] counts, then places
  __shared__ int wsum[2][16];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  for (int e = tid; e < E; e += 1024) cnt[e] = 0;
  __syncthreads();
  for (int p = tid; p < P; p += 1024) atomicAdd(&cnt[ids[p]], 1);
  __syncthreads();
  // exclusive sums of counts and tile counts over the experts; thread i owns experts [i per, (i + 1) per)
  const int per = ceil_div(E, 1024), lo = min(tid * per, E), hi = min(lo + per, E);
  int a = 0, b = 0;
  for (int e = lo; e < hi; ++e) { a += cnt[e]; b += ceil_div(cnt[e], plan.block); }
  int ia = a, ib = b;
#pragma unroll
  for (int m = 1; m < 64; m *= 2) {
    const int va = __shfl_up(ia, m), vb = __shfl_up(ib, m);
    if (lane >= m) { ia += va; ib += vb; }
  }
  if (lane == 63) { wsum[0][wave] = ia; wsum[1][wave] = ib; }
  __syncthreads();
  int at = ia - a, tt = ib - b, total = 0;
  for (int v = 0; v < 16; ++v) {
    if (v < wave) { at += wsum[0][v]; tt += wsum[1][v]; }
    total += wsum[1][v];
  }
  for (int e = lo; e < hi; ++e) {
    const int n = cnt[e];
    for (int k = 0; k < n; k += plan.block) {
      int* t = plan.tiles + (size_t)tt * 3;
      t[0] = e; t[1] = at + k; t[2] = min(plan.block, n - k);
      ++tt;
    }
    cnt[e] = at;
    at += n;
  }
  if (tid == 0) plan.tiles[(size_t)plan.max_tiles * 3] = total;
  __syncthreads();
  for (int p = tid; p < P; p += 1024) plan.order[atomicAdd(&cnt[ids[p]], 1)] = p;    // (order inside an expert does not matter: rows are independent)
}

// 128 weight rows x BM pairs per work-group, four waves; pairs' rows through swizzled LDS, weights from their tiled image
template <int BM, int ACT>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(BM == 64 ? 4 : 2, BM == 64 ? 4 : 2))) void experts_gemm_kernel(
    const uint4* __restrict__ w, int NT, int KT, ExpertPlan plan, const uint16_t* __restrict__ x, int ldx, int x_div, uint16_t* __restrict__ y, int ldy) {
  constexpr int WM = BM / 64, WN = 4 / WM, NTW = 8 / WN, XL = BM / 32;
  __shared__ __attribute__((aligned(16))) u32x4_t xs[BM * 8];
  const int ntiles = ceil_div(NT, 8);
  int mt_id, nblk;
  if (ntiles % 8 == 0) {       // an XCD (linear id % 8) takes every eighth block of weight rows, all tiles of an expert back to back
    const int per = ntiles / 8, seq = blockIdx.x >> 3;
    mt_id = seq / per;
    nblk = (seq % per) * 8 + (blockIdx.x & 7);
  } else {
    mt_id = blockIdx.x / ntiles;
    nblk = blockIdx.x % ntiles;
  }
  if (mt_id >= plan.tiles[(size_t)plan.max_tiles * 3]) return;
  const int e = plan.tiles[mt_id * 3], first = plan.tiles[mt_id * 3 + 1], n = plan.tiles[mt_id * 3 + 2];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, g = lane >> 4, c = lane & 15;
  const int wn = wave / WM, wm = wave % WM, nt0 = nblk * 8 + wn * NTW;
  const u32x4_t* W = reinterpret_cast<const u32x4_t*>(w) + (size_t)e * NT * KT * 64 + lane;
  const int srow = tid >> 3, sch = tid & 7, nks = KT / 2;
  const uint16_t* xp[XL];
#pragma unroll
  for (int i = 0; i < XL; ++i) xp[i] = x + (size_t)(plan.order[first + min(srow + 32 * i, n - 1)] / x_div) * ldx + sch * 8;
  f32x4_t acc[NTW][4];
#pragma unroll
  for (int i = 0; i < NTW; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  u32x4_t xr[XL], wr[NTW][2];
  auto load = [&](int ks) {
#pragma unroll
    for (int i = 0; i < XL; ++i) xr[i] = *reinterpret_cast<const u32x4_t*>(xp[i] + ks * 64);
#pragma unroll
    for (int i = 0; i < NTW; ++i)
#pragma unroll
      for (int t = 0; t < 2; ++t) wr[i][t] = W[((size_t)min(nt0 + i, NT - 1) * KT + ks * 2 + t) * 64];
  };
  load(0);
  for (int ks = 0; ks < nks; ++ks) {
#pragma unroll
    for (int i = 0; i < XL; ++i) {
      const int r = srow + 32 * i;
      xs[r * 8 + (sch ^ (r & 7))] = xr[i];
    }
    bf16x8_t a0[NTW], a1[NTW];
#pragma unroll
    for (int i = 0; i < NTW; ++i) {
      a0[i] = __builtin_bit_cast(bf16x8_t, wr[i][0]);
      a1[i] = __builtin_bit_cast(bf16x8_t, wr[i][1]);
    }
    __syncthreads();
    if (ks + 1 < nks) load(ks + 1);
#pragma unroll
    for (int mt = 0; mt < 4; ++mt) {
      const int r = wm * 64 + mt * 16 + c;
      const bf16x8_t b0 = __builtin_bit_cast(bf16x8_t, xs[r * 8 + (g ^ (r & 7))]);
      const bf16x8_t b1 = __builtin_bit_cast(bf16x8_t, xs[r * 8 + ((4 + g) ^ (r & 7))]);
#pragma unroll
      for (int i = 0; i < NTW; ++i) {
        acc[i][mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a0[i], b0, acc[i][mt], 0, 0, 0);
        acc[i][mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a1[i], b1, acc[i][mt], 0, 0, 0);
      }
    }
    __syncthreads();
  }
#pragma unroll
  for (int mt = 0; mt < 4; ++mt) {
    const int m = wm * 64 + mt * 16 + c;
    if (m >= n) continue;
    uint16_t* row = y + (size_t)plan.order[first + m] * ldy;
#pragma unroll
    for (int i = 0; i < NTW; ++i) {
      if (nt0 + i >= NT) continue;
      const f32x4_t v = acc[i][mt];
      const int n0 = (nt0 + i) * 16 + g * 4;
      if constexpr (ACT == EXPERT_RELU2)
        *reinterpret_cast<uint2*>(row + n0) = relu2x4(v);
      else if constexpr (ACT == EXPERT_SILU_GLU)
        *reinterpret_cast<uint32_t*>(row + (n0 >> 1)) = pack_bf16x2(v[0] / (1.f + __expf(-v[0])) * v[1], v[2] / (1.f + __expf(-v[2])) * v[3]);
      else
        *reinterpret_cast<uint2*>(row + n0) = make_uint2(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]));
    }
  }
}

template <int KS>
int launch_stream(const ExpertsLinear& w, const int32_t* ids, int P, const uint16_t* x, int ldx, int x_div, int act, void* y, int ldy, hipStream_t s) {
  const int NT = w.N / 16, KT = w.K / 32;
  const dim3 grid(KS == 1 ? ceil_div(NT, 4) : NT, w.E);
  if (act == EXPERT_SILU_GLU) hipLaunchKernelGGL((experts_stream_kernel<KS, EXPERT_SILU_GLU>), grid, dim3(256), 0, s, (const uint4*)w.w, NT, KT, ids, P, x, ldx, x_div, y, ldy);
  else if (act == EXPERT_RELU2) hipLaunchKernelGGL((experts_stream_kernel<KS, EXPERT_RELU2>), grid, dim3(256), 0, s, (const uint4*)w.w, NT, KT, ids, P, x, ldx, x_div, y, ldy);
  else hipLaunchKernelGGL((experts_stream_kernel<KS, EXPERT_LINEAR>), grid, dim3(256), 0, s, (const uint4*)w.w, NT, KT, ids, P, x, ldx, x_div, y, ldy);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

}  // namespace

int launch_route(const void* x, int ldx, int T, const void* w, const RouterRule& rule, int E, int K, int top, int32_t* ids, float* weights, bool f32, hipStream_t s,
                 float* z, uint32_t* tickets) {
  MI_CHECK(T >= 1 && E >= 1 && top >= 1 && top <= E && top <= kMaxTop && K % 64 == 0 && ldx >= K && ldx % 8 == 0, "router: 1 <= top <= min(experts, 64), row stride");
  const size_t lds = (size_t)(rule.sigmoid ? 3 : 1) * pick_stride(E) * 4;
  MI_CHECK(rule.b && E <= (rule.sigmoid ? 1024 : 4096), "router: up to 4096 experts, 1024 with the sigmoid rule");
  MI_CHECK(rule.groups >= 1 && E % rule.groups == 0 && rule.keep >= 1 && rule.keep <= rule.groups, "router: groups");
  MI_CHECK(!tickets || z, "router: tickets without logits");
  const dim3 grid(T, tickets ? ceil_div(E, kRouteExperts) : 1);
  if (f32) hipLaunchKernelGGL((route_kernel<float>), grid, dim3(256), lds, s, (const float*)x, ldx, (const float*)w, rule, E, K, top, ids, weights, z, tickets);
  else hipLaunchKernelGGL((route_kernel<uint16_t>), grid, dim3(256), lds, s, (const uint16_t*)x, ldx, (const uint16_t*)w, rule, E, K, top, ids, weights, z, tickets);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_route_pick(const float* z, int ldz, int T, const RouterRule& rule, int E, int top, int32_t* ids, float* weights, hipStream_t s) {
  MI_CHECK(T >= 1 && E >= 1 && E <= (rule.sigmoid ? 1024 : 4096) && top >= 1 && top <= E && top <= kMaxTop && ldz >= E, "router: experts / top");
  MI_CHECK((!rule.sigmoid || rule.b) && rule.groups >= 1 && E % rule.groups == 0 && rule.keep >= 1 && rule.keep <= rule.groups, "router: groups");
  const size_t lds = (size_t)4 * (rule.sigmoid ? 3 : 1) * pick_stride(E) * 4;
  hipLaunchKernelGGL(route_pick_kernel, dim3(ceil_div(T, 4)), dim3(256), lds, s, z, ldz, T, rule, E, top, ids, weights);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

size_t experts_plan_ints(int P, int E) { return (size_t)P + 3 * ((size_t)P / 64 + min(P, E) + 1) + 1; }
ExpertPlan experts_plan(int32_t* mem, int P, int E) {
  const int block = P / E >= 96 ? 128 : 64;
  return ExpertPlan{mem, mem + P, block, P / block + min(P, E) + 1};
}
int launch_experts_sort(const ExpertPlan& plan, const int32_t* ids, int P, int E, hipStream_t s) {
  MI_CHECK(P >= 1 && E >= 1 && E <= 4096 && plan.order && plan.tiles, "experts: plan");
  hipLaunchKernelGGL(experts_sort_kernel, dim3(1), dim3(1024), (size_t)4 * E, s, ids, P, E, plan);
  MI_HIP(hipGetLastError());
  return MI_OK;
}
int launch_experts_gemm(const ExpertsLinear& w, const ExpertPlan& plan, int P, const uint16_t* x, int ldx, int x_div, int act, uint16_t* y, int ldy, hipStream_t s) {
  MI_CHECK(w.E >= 1 && w.N % 16 == 0 && w.K % 64 == 0 && ldx >= w.K && ldx % 8 == 0 && P >= 1 && x_div >= 1, "experts: shape");
  MI_CHECK(ldy % 4 == 0 && ldy >= (act == EXPERT_SILU_GLU ? w.N / 2 : w.N), "experts: output stride");
  const int NT = w.N / 16, KT = w.K / 32;
  const dim3 grid((unsigned)(plan.max_tiles * ceil_div(NT, 8)));
  const uint4* W = reinterpret_cast<const uint4*>(w.w);
#define MI_EG(BM) \
  if (act == EXPERT_SILU_GLU) hipLaunchKernelGGL((experts_gemm_kernel<BM, EXPERT_SILU_GLU>), grid, dim3(256), 0, s, W, NT, KT, plan, x, ldx, x_div, y, ldy); \
  else if (act == EXPERT_RELU2) hipLaunchKernelGGL((experts_gemm_kernel<BM, EXPERT_RELU2>), grid, dim3(256), 0, s, W, NT, KT, plan, x, ldx, x_div, y, ldy); \
  else hipLaunchKernelGGL((experts_gemm_kernel<BM, EXPERT_LINEAR>), grid, dim3(256), 0, s, W, NT, KT, plan, x, ldx, x_div, y, ldy)
  if (plan.block == 128) { MI_EG(128); } else { MI_EG(64); }
#undef MI_EG
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_experts_linear(const ExpertsLinear& w, const int32_t* ids, int P, const void* x, int ldx, int x_div, int act, void* y, int ldy,
                          bool f32, hipStream_t s) {
  MI_CHECK(w.E >= 1 && w.E <= 65535 && w.N % 16 == 0 && w.K % 64 == 0 && ldx >= w.K && ldx % 8 == 0 && P >= 1 && x_div >= 1, "experts: shape");
  MI_CHECK(ldy % 4 == 0 && ldy >= (act == EXPERT_SILU_GLU ? w.N / 2 : w.N), "experts: output stride");
  if (f32) {
    const dim3 grid(P, ceil_div(act == EXPERT_SILU_GLU ? w.N / 2 : w.N, 4));
    if (act == EXPERT_RELU2) hipLaunchKernelGGL((experts_f32_kernel<EXPERT_RELU2>), grid, dim3(256), 0, s, (const float*)w.w, w.N, w.K, ids, (const float*)x, ldx, x_div, (float*)y, ldy);
    else if (act == EXPERT_SILU_GLU) hipLaunchKernelGGL((experts_f32_kernel<EXPERT_SILU_GLU>), grid, dim3(256), 0, s, (const float*)w.w, w.N, w.K, ids, (const float*)x, ldx, x_div, (float*)y, ldy);
    else hipLaunchKernelGGL((experts_f32_kernel<EXPERT_LINEAR>), grid, dim3(256), 0, s, (const float*)w.w, w.N, w.K, ids, (const float*)x, ldx, x_div, (float*)y, ldy);
    MI_HIP(hipGetLastError());
    return MI_OK;
  }
  return w.K / 32 >= 16 ? launch_stream<4>(w, ids, P, (const uint16_t*)x, ldx, x_div, act, y, ldy, s)
                        : launch_stream<1>(w, ids, P, (const uint16_t*)x, ldx, x_div, act, y, ldy, s);
}

}  // namespace mi
