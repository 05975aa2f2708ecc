// Row-wise kernels of the layer-stack decoders.  See stack_kernels.h.
#include "stack_kernels.h"

#include <algorithm>

#include "misc_kernels.h"

namespace mi {

namespace {

__device__ __forceinline__ float to_f32(uint16_t v) { return bf16_to_f32(v); }
__device__ __forceinline__ float to_f32(float v) { return v; }
__device__ __forceinline__ void put4(uint16_t* p, float a, float b, float c, float d) {
  *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf16x2(a, b), pack_bf16x2(c, d));
}
__device__ __forceinline__ void put4(float* p, float a, float b, float c, float d) { *reinterpret_cast<float4*>(p) = make_float4(a, b, c, d); }

__device__ __forceinline__ float4 get4(const uint16_t* p) {
  const uint2 v = *reinterpret_cast<const uint2*>(p);
  return make_float4(bf16lo_to_f32(v.x), bf16hi_to_f32(v.x), bf16lo_to_f32(v.y), bf16hi_to_f32(v.y));
}
__device__ __forceinline__ float4 get4(const float* p) { return *reinterpret_cast<const float4*>(p); }

// sum over the work-group (up to 16 waves), in wave order; `red` has 16 floats and is free again after the next barrier
__device__ __forceinline__ float block_sum(float v, float* red) {
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float t = 0.f;
  for (int w = 0; w < (int)(blockDim.x >> 6); ++w) t += red[w];
  return t;
}

template <typename T>
__global__ __launch_bounds__(256) void embed_pos_kernel(const int32_t* __restrict__ ids, const int32_t* __restrict__ pos,
                                                        const T* __restrict__ table, const T* __restrict__ ptable, float sc, int D, int ld,
                                                        float* __restrict__ resid, float* __restrict__ x0, const double* __restrict__ turns,
                                                        T* __restrict__ y, int ldy) {
  const int t = blockIdx.x;
  const T* e = table + (size_t)ids[t] * D;
  const T* p = ptable ? ptable + (size_t)pos[t] * D : nullptr;
  for (int d = threadIdx.x * 4; d < ld; d += 1024) {
    float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
    if ((D & 3) == 0) {
      if (d < D) {
        const float4 a = get4(e + d), b = p ? get4(p + d) : make_float4(0.f, 0.f, 0.f, 0.f);
        v = make_float4(__builtin_fmaf(sc, a.x, b.x), __builtin_fmaf(sc, a.y, b.y), __builtin_fmaf(sc, a.z, b.z), __builtin_fmaf(sc, a.w, b.w));
      }
    } else {
      auto at = [&](int i) { return d + i < D ? __builtin_fmaf(sc, to_f32(e[d + i]), p ? to_f32(p[d + i]) : 0.f) : 0.f; };
      v = make_float4(at(0), at(1), at(2), at(3));
    }
    if (turns) {       // the angle in whole turns, its fraction exact in fp64
      const double p0 = (double)pos[t];
      float sn[2] = {0.f, 0.f}, cs[2] = {0.f, 0.f};
#pragma unroll
      for (int i = 0; i < 2; ++i)
        if (d + 2 * i < D) {
          const double a = p0 * turns[d / 2 + i];
          sincospif((float)(2.0 * (a - floor(a))), &sn[i], &cs[i]);
        }
      v = make_float4(v.x + sn[0], d + 1 < D ? v.y + cs[0] : 0.f, v.z + sn[1], d + 3 < D ? v.w + cs[1] : 0.f);
    }
    if (y) put4(y + (size_t)t * ldy + d, v.x, v.y, v.z, v.w);
    *reinterpret_cast<float4*>(resid + (size_t)t * ld + d) = v;
    if (x0) *reinterpret_cast<float4*>(x0 + (size_t)t * ld + d) = v;
  }
}

template <typename T>
__global__ __launch_bounds__(1024) void layernorm_rows_kernel(const float* __restrict__ resid_in, float* __restrict__ resid_out,
                                                             int D, int ld, float eps, NormOut na, NormOut nb, int ldy, SlabSum sl) {
  extern __shared__ __attribute__((aligned(16))) float hrow[];  // ld floats + 32
  const int t = blockIdx.x, tid = threadIdx.x, nthr = blockDim.x;
  const size_t o = (size_t)t * ld;
  float* red = hrow + ld;
  float sum = 0.f;
  for (int c4 = tid; c4 < ld / 4; c4 += nthr) {
    float4 a = *reinterpret_cast<const float4*>(resid_in + o + c4 * 4);
    if (sl.slab) {   // slabs in slice order, scale, + residual: the arithmetic of splitk_reduce + the residual epilogue
      float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
      for (int z = 0; z < sl.KS; ++z) {
        const float4 q = *reinterpret_cast<const float4*>(sl.slab + ((size_t)z * sl.T + t) * sl.N + c4 * 4);
        v.x += q.x; v.y += q.y; v.z += q.z; v.w += q.w;
      }
      const float4 sc = *reinterpret_cast<const float4*>(sl.scale + c4 * 4);
      a.x += v.x * sc.x; a.y += v.y * sc.y; a.z += v.z * sc.z; a.w += v.w * sc.w;
      *reinterpret_cast<float4*>(resid_out + o + c4 * 4) = a;
    }
    *reinterpret_cast<float4*>(hrow + c4 * 4) = a;
    sum += (a.x + a.y) + (a.z + a.w);     // columns beyond D are zero
  }
  const float mean = block_sum(sum, red) / (float)D;
  float ss = 0.f;
  for (int c4 = tid; c4 < ld / 4; c4 += nthr) {   // (a thread reads back what it wrote itself)
    float4 a = *reinterpret_cast<const float4*>(hrow + c4 * 4);
    const int d = c4 * 4;
    a.x = d < D ? a.x - mean : 0.f;
    a.y = d + 1 < D ? a.y - mean : 0.f;
    a.z = d + 2 < D ? a.z - mean : 0.f;
    a.w = d + 3 < D ? a.w - mean : 0.f;
    *reinterpret_cast<float4*>(hrow + c4 * 4) = a;
    ss += (a.x * a.x + a.y * a.y) + (a.z * a.z + a.w * a.w);
  }
  const float rstd = 1.0f / sqrtf(block_sum(ss, red + 16) / (float)D + eps);
  for (int c4 = tid; c4 < ld / 4; c4 += nthr) {
    const float4 a = *reinterpret_cast<const float4*>(hrow + c4 * 4);
    auto emit = [&](const NormOut& n) {
      const float4 w = *reinterpret_cast<const float4*>(n.w + c4 * 4), b = *reinterpret_cast<const float4*>(n.b + c4 * 4);
      put4(reinterpret_cast<T*>(n.y) + (size_t)t * ldy + c4 * 4, a.x * rstd * w.x + b.x, a.y * rstd * w.y + b.y,
           a.z * rstd * w.z + b.z, a.w * rstd * w.w + b.w);
    };
    if (na.y) emit(na);
    if (nb.y) emit(nb);
  }
}

__device__ __forceinline__ float round_to(float v, const uint16_t*) { return bf16_to_f32(f32_to_bf16(v)); }
__device__ __forceinline__ float round_to(float v, const float*) { return v; }

// 1 / sqrt(mean square + eps) of every one of G equal parts of the D floats in `row`, into rstd [G].  A part is shared out to
// several waves where there are fewer parts than waves; summed in wave order.  red: max(G, waves) floats.
__device__ __forceinline__ void group_rstd(const float* row, int D, int G, float eps, float* red, float* rstd) {
  const int nw = blockDim.x >> 6, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int gs = D / G, P = max(1, nw / G), len = ceil_div(gs, P);
  __syncthreads();                      // the row is complete
  for (int u = wave; u < G * P; u += nw) {
    const int g = u / P, lo = g * gs + (u - g * P) * len, hi = min(lo + len, (g + 1) * gs);
    float s = 0.f;
    for (int i = lo + lane; i < hi; i += 64) s = __builtin_fmaf(row[i], row[i], s);
    s = wave_sum(s);
    if (lane == 0) red[u] = s;
  }
  __syncthreads();
  for (int g = threadIdx.x; g < G; g += blockDim.x) {
    float s = 0.f;
    for (int p = 0; p < P; ++p) s += red[g * P + p];
    rstd[g] = 1.0f / sqrtf(s / (float)gs + eps);
  }
  __syncthreads();
}
// part of element d (exact: d < 2^15, the quotient is at least 0.5 / gs away from an integer)
__device__ __forceinline__ int part_of(int d, float inv_gs) { return (int)(((float)d + 0.5f) * inv_gs); }
__device__ __forceinline__ float4 part_rstd(const float* rstd, int d, int G, float inv_gs) {
  if (G == 1) return make_float4(rstd[0], rstd[0], rstd[0], rstd[0]);
  auto at = [&](int i) { return rstd[min(part_of(d + i, inv_gs), G - 1)]; };
  return make_float4(at(0), at(1), at(2), at(3));
}

__device__ __forceinline__ float4 source_row4(const RowSource& src, int t, int d) {
  float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
  if (src.slabs.slab) {
    for (int z = 0; z < src.slabs.KS; ++z) {
      const float4 q = *reinterpret_cast<const float4*>(src.slabs.slab + ((size_t)z * src.slabs.T + t) * src.slabs.N + d);
      v.x += q.x; v.y += q.y; v.z += q.z; v.w += q.w;
    }
    const float4 sc = *reinterpret_cast<const float4*>(src.slabs.scale + d);
    v.x *= sc.x; v.y *= sc.y; v.z *= sc.z; v.w *= sc.w;
  }
  if (src.pair_w) {
    for (int j = 0; j < src.top; ++j) {
      const size_t r = (size_t)t * src.top + j;
      const float w = src.pair_w[r];
      const float4 q = src.y16 ? get4(src.y16 + r * src.ld + d) : get4(src.y + r * src.ld + d);
      v.x = __builtin_fmaf(w, q.x, v.x); v.y = __builtin_fmaf(w, q.y, v.y);
      v.z = __builtin_fmaf(w, q.z, v.z); v.w = __builtin_fmaf(w, q.w, v.w);
    }
  } else if (!src.slabs.slab) {
    v = *reinterpret_cast<const float4*>(src.y + (size_t)t * src.ld + d);
  }
  return v;
}

// the convolution's sum for channels d .. d + 3 at position p; past(back) = input `back` positions earlier (called where p >= back)
template <typename F>
__device__ __forceinline__ float4 conv_sum(const ConvState& cs, int ld, int d, int p, float4 h, F past) {
  float4 a = make_float4(0.f, 0.f, 0.f, 0.f);
  for (int j = 0; j < cs.taps; ++j) {
    const int back = cs.taps - 1 - j;
    if (back > p) continue;
    const float4 v = back == 0 ? h : past(back), w = *reinterpret_cast<const float4*>(cs.w + (size_t)j * ld + d);
    a.x = __builtin_fmaf(w.x, v.x, a.x); a.y = __builtin_fmaf(w.y, v.y, a.y);
    a.z = __builtin_fmaf(w.z, v.z, a.z); a.w = __builtin_fmaf(w.w, v.w, a.w);
  }
  return make_float4(h.x + a.x, h.y + a.y, h.z + a.z, h.w + a.w);
}
template <typename T>
__device__ __forceinline__ T* ring_at(const ConvState& cs, int blk, int off, int ldy) {
  return reinterpret_cast<T*>(cs.ring) + ((size_t)blk * cs.keep + off % cs.keep) * ldy;
}
template <typename T>
__device__ __forceinline__ float4 ring_get4(const ConvState& cs, int seq, int p, int ldy, int d) {
  return get4(ring_at<T>(cs, cs.bt[(size_t)seq * cs.MB + p / cs.block_size], p % cs.block_size, ldy) + d);
}

template <typename T>
__global__ __launch_bounds__(1024) void sandwich_rows_kernel(const float* __restrict__ resid_in, float* __restrict__ resid_out, RowSource src,
                                                            const float* __restrict__ w_post, const float* __restrict__ w_pre, int D, int ld,
                                                            int G, float eps, ConvState cs, T* __restrict__ y, int ldy, bool as_is) {
  extern __shared__ __attribute__((aligned(16))) float row[];   // ld + max(G, 16) + G floats
  float *red = row + ld, *rstd = red + max(G, 16);
  const int t = blockIdx.x, tid = threadIdx.x, nthr = blockDim.x;
  const size_t o = (size_t)t * ld;
  const float inv_gs = 1.0f / (float)(D / G);
  const bool add = src.any();
  if (add && w_post) {
    for (int d = tid * 4; d < ld; d += nthr * 4) *reinterpret_cast<float4*>(row + d) = source_row4(src, t, d);
    group_rstd(row, D, G, eps, red, rstd);
  }
  for (int d = tid * 4; d < ld; d += nthr * 4) {   // (a thread reads back what it wrote itself)
    float4 x = *reinterpret_cast<const float4*>(resid_in + o + d);
    if (add && !w_post) {
      const float4 v = source_row4(src, t, d);
      x = make_float4(x.x + v.x, x.y + v.y, x.z + v.z, x.w + v.w);
      *reinterpret_cast<float4*>(resid_out + o + d) = x;
    } else if (add) {
      const float4 v = *reinterpret_cast<const float4*>(row + d), w = *reinterpret_cast<const float4*>(w_post + d), r = part_rstd(rstd, d, G, inv_gs);
      x.x = __builtin_fmaf(v.x * r.x, w.x, x.x); x.y = __builtin_fmaf(v.y * r.y, w.y, x.y);
      x.z = __builtin_fmaf(v.z * r.z, w.z, x.z); x.w = __builtin_fmaf(v.w * r.w, w.w, x.w);
      *reinterpret_cast<float4*>(resid_out + o + d) = x;
    }
    if (as_is) put4(y + (size_t)t * ldy + d, x.x, x.y, x.z, x.w);
    *reinterpret_cast<float4*>(row + d) = x;
  }
  if (!w_pre) return;
  group_rstd(row, D, G, eps, red, rstd);
  const int p = cs.w ? cs.pos[t] : 0, slot = cs.w ? cs.slots[t] : -1;
  for (int d = tid * 4; d < ld; d += nthr * 4) {
    const float4 x = *reinterpret_cast<const float4*>(row + d), w = *reinterpret_cast<const float4*>(w_pre + d), r = part_rstd(rstd, d, G, inv_gs);
    float4 h = make_float4(x.x * r.x * w.x, x.y * r.y * w.y, x.z * r.z * w.z, x.w * r.w * w.w);
    if (cs.w) {
      h = make_float4(round_to(h.x, y), round_to(h.y, y), round_to(h.z, y), round_to(h.w, y));
      const float4 a = conv_sum(cs, ld, d, p, h, [&](int back) { return ring_get4<T>(cs, t, p - back, ldy, d); });
      if (slot >= 0 && cs.keep > 0) put4(ring_at<T>(cs, slot / cs.block_size, slot % cs.block_size, ldy) + d, h.x, h.y, h.z, h.w);
      h = a;
    }
    put4(y + (size_t)t * ldy + d, h.x, h.y, h.z, h.w);
  }
}

template <typename T> struct Raw4;
template <> struct Raw4<uint16_t> { typedef uint2 type; };
template <> struct Raw4<float> { typedef float4 type; };
__device__ __forceinline__ float4 widen(uint2 v) { return make_float4(bf16lo_to_f32(v.x), bf16hi_to_f32(v.x), bf16lo_to_f32(v.y), bf16hi_to_f32(v.y)); }
__device__ __forceinline__ float4 widen(float4 v) { return v; }

// Token generation, rows of up to 4096: one float4 per thread and everything the row needs requested at once -- the sublayer's output,
// the stream, both weights, the convolution's taps and state -- so that the two norms wait for memory once.  D / G a multiple of
// 256: a wave's elements lie in one part, and a part's sum is a few waves' (in wave order).
template <typename T, int TAPS>
__global__ __launch_bounds__(1024) void sandwich_token_kernel(const float* __restrict__ resid_in, float* __restrict__ resid_out, RowSource src,
                                                             const float* __restrict__ w_post, const float* __restrict__ w_pre, int D, int ld,
                                                             int gs, float eps, ConvState cs, T* __restrict__ y, int ldy) {
  typedef typename Raw4<T>::type raw_t;
  __shared__ float red[2][16];
  const int t = blockIdx.x, tid = threadIdx.x, wave = tid >> 6, d = tid * 4;
  const bool in = d < ld, add = src.any();
  const int dd = in ? d : 0;
  const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
  float4 x = *reinterpret_cast<const float4*>(resid_in + (size_t)t * ld + dd);
  float4 v = add ? source_row4(src, t, dd) : zero;
  const float4 wp = add && w_post ? *reinterpret_cast<const float4*>(w_post + dd) : zero, wn = w_pre ? *reinterpret_cast<const float4*>(w_pre + dd) : zero;
  float4 w[TAPS > 0 ? TAPS : 1];
  raw_t past[TAPS > 1 ? TAPS - 1 : 1];
  int slot = -1;
  if constexpr (TAPS > 0) {
    const int p = cs.pos[t];
    slot = cs.slots[t];
#pragma unroll
    for (int j = 0; j < TAPS; ++j) w[j] = *reinterpret_cast<const float4*>(cs.w + (size_t)j * ld + dd);
#pragma unroll
    for (int j = 0; j + 1 < TAPS; ++j) {
      const int q = p - (TAPS - 1 - j);
      if (q >= 0) past[j] = *reinterpret_cast<const raw_t*>(ring_at<T>(cs, cs.bt[(size_t)t * cs.MB + q / cs.block_size], q % cs.block_size, ldy) + dd);
      else past[j] = raw_t{};
    }
  }
  const int wpg = gs >> 8, g0 = wave / wpg * wpg;              // waves of this element's part
  auto rstd = [&](float4 a, float* r) {
    const float s = wave_sum((a.x * a.x + a.y * a.y) + (a.z * a.z + a.w * a.w));   // (rows are whole parts: columns beyond D belong to no wave of a part)
    if ((tid & 63) == 0) r[wave] = s;
    __syncthreads();
    float sum = 0.f;
    for (int k = 0; k < wpg; ++k) sum += r[g0 + k];
    return 1.0f / sqrtf(sum / (float)gs + eps);
  };
  if (add && !w_post) {
    x = make_float4(x.x + v.x, x.y + v.y, x.z + v.z, x.w + v.w);
    if (in) *reinterpret_cast<float4*>(resid_out + (size_t)t * ld + d) = x;
  } else if (add) {
    const float r = rstd(in ? v : zero, red[0]);
    x.x = __builtin_fmaf(v.x * r, wp.x, x.x); x.y = __builtin_fmaf(v.y * r, wp.y, x.y);
    x.z = __builtin_fmaf(v.z * r, wp.z, x.z); x.w = __builtin_fmaf(v.w * r, wp.w, x.w);
    if (in) *reinterpret_cast<float4*>(resid_out + (size_t)t * ld + d) = x;
  }
  if (!w_pre) {         // (the row itself)
    if (in) put4(y + (size_t)t * ldy + d, x.x, x.y, x.z, x.w);
    return;
  }
  const float r = rstd(in ? x : zero, red[1]);
  if (!in) return;
  float4 h = make_float4(x.x * r * wn.x, x.y * r * wn.y, x.z * r * wn.z, x.w * r * wn.w);
  if constexpr (TAPS > 0) {
    h = make_float4(round_to(h.x, y), round_to(h.y, y), round_to(h.z, y), round_to(h.w, y));
    float4 a = zero;
#pragma unroll
    for (int j = 0; j < TAPS; ++j) {
      const float4 u = j + 1 < TAPS ? widen(past[j < TAPS - 1 ? j : 0]) : h;
      a.x = __builtin_fmaf(w[j].x, u.x, a.x); a.y = __builtin_fmaf(w[j].y, u.y, a.y);
      a.z = __builtin_fmaf(w[j].z, u.z, a.z); a.w = __builtin_fmaf(w[j].w, u.w, a.w);
    }
    if (TAPS > 1 && slot >= 0) put4(ring_at<T>(cs, slot / cs.block_size, slot % cs.block_size, ldy) + d, h.x, h.y, h.z, h.w);
    h = make_float4(h.x + a.x, h.y + a.y, h.z + a.z, h.w + a.w);
  }
  put4(y + (size_t)t * ldy + d, h.x, h.y, h.z, h.w);
}

// One work-group: up to ROWS rows of one segment x 256 C channels, C channels (16 bytes) per thread; a thread's rows and the inputs
// ahead of them are all requested at once.  TAPS = 0: any number of taps, inputs read where they are needed.
// The rows at a segment's start read the state of the positions ahead of it, and rows further on renew it.  Both may meet in one
// place only in the block that holds the position ahead of the segment; that block's renewal is left to the work-group of the
// segment's first rows, whose threads have read their channels' state by then (ROWS >= taps - 1).
constexpr int kConvRows = 16;
template <typename T> struct Chunk16 { static constexpr int C = 16 / sizeof(T); };

__device__ __forceinline__ void widen16(const u32x4_t& v, float (&o)[8]) {
#pragma unroll
  for (int i = 0; i < 4; ++i) { o[2 * i] = bf16lo_to_f32(v[i]); o[2 * i + 1] = bf16hi_to_f32(v[i]); }
}
__device__ __forceinline__ void widen16(const u32x4_t& v, float (&o)[4]) {
#pragma unroll
  for (int i = 0; i < 4; ++i) o[i] = __builtin_bit_cast(float, (unsigned)v[i]);
}
__device__ __forceinline__ void put16(uint16_t* p, const float (&v)[8]) {
  *reinterpret_cast<uint4*>(p) = make_uint4(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]), pack_bf16x2(v[4], v[5]), pack_bf16x2(v[6], v[7]));
}
__device__ __forceinline__ void put16(float* p, const float (&v)[4]) { *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]); }

template <typename T, int TAPS, int ROWS>
__global__ __launch_bounds__(256) void conv_rows_kernel(const T* __restrict__ hin, ConvState cs, const AttnSeg* __restrict__ segs, int nseg,
                                                        int ld, T* __restrict__ y, int ldy) {
  constexpr int C = Chunk16<T>::C;
  int tile = blockIdx.x, si = 0;
  AttnSeg sg{0, 0, 0, 0};
  for (; si < nseg; ++si) {
    sg = segs[si];
    const int n = ceil_div(sg.n, ROWS);
    if (tile < n) break;
    tile -= n;
  }
  const int d = (blockIdx.y * 256 + threadIdx.x) * C;
  if (si == nseg || d >= ld) return;
  const int bs = cs.block_size, first = tile * ROWS, last = min(first + ROWS, sg.n), end = sg.pos0 + sg.n;
  const int shared_block = sg.pos0 % bs ? sg.pos0 / bs : -1;      // holds positions on both sides of the segment's start
  const T* hs = hin + (size_t)sg.row0 * ldy + d;
  auto get = [&](const T* p) { return *reinterpret_cast<const u32x4_t*>(p); };
  auto state = [&](int p) { return get(ring_at<T>(cs, cs.bt[(size_t)sg.seq * cs.MB + p / bs], p % bs, ldy) + d); };
  auto renew = [&](int p, const u32x4_t& h) {
    const int slot = cs.slots[sg.row0 + p - sg.pos0];
    if (slot >= 0) *reinterpret_cast<u32x4_t*>(ring_at<T>(cs, slot / bs, slot % bs, ldy) + d) = h;
  };
  auto renew_own = [&](int p, const u32x4_t& h) {
    const int b = p / bs;
    if (b != shared_block && p + cs.keep >= min(end, (b + 1) * bs)) renew(p, h);
  };
  auto tap = [&](int j, float (&w)[C]) {
#pragma unroll
    for (int c = 0; c < C; c += 4) *reinterpret_cast<float4*>(w + c) = *reinterpret_cast<const float4*>(cs.w + (size_t)j * ld + d + c);
  };
  if constexpr (TAPS > 0) {
    u32x4_t in[ROWS + TAPS - 1];
    float w[TAPS][C];
#pragma unroll
    for (int k = 0; k < ROWS + TAPS - 1; ++k) {
      const int i = first + k - (TAPS - 1);                         // row of the segment; negative: ahead of it
      if (i >= 0) in[k] = get(hs + (size_t)min(i, sg.n - 1) * ldy);
      else if (sg.pos0 + i >= 0) in[k] = state(sg.pos0 + i);
      else in[k] = u32x4_t{0, 0, 0, 0};                              // (ahead of the sequence: zeros)
    }
#pragma unroll
    for (int j = 0; j < TAPS; ++j) tap(j, w[j]);
#pragma unroll
    for (int k = 0; k < ROWS; ++k) {
      if (first + k >= last) break;
      float a[C], h[C];
#pragma unroll
      for (int c = 0; c < C; ++c) a[c] = 0.f;
#pragma unroll
      for (int j = 0; j < TAPS; ++j) {
        widen16(in[k + j], h);
#pragma unroll
        for (int c = 0; c < C; ++c) a[c] = __builtin_fmaf(w[j][c], h[c], a[c]);
      }
#pragma unroll
      for (int c = 0; c < C; ++c) a[c] += h[c];                      // (the last tap met the token itself)
      put16(y + (size_t)(sg.row0 + first + k) * ldy + d, a);
      if constexpr (TAPS > 1) renew_own(sg.pos0 + first + k, in[k + TAPS - 1]);
    }
  } else {
    for (int i = first; i < last; ++i) {
      const int p = sg.pos0 + i;
      const T* r = hs + (size_t)i * ldy;
      float a[C], h[C], w[C];
#pragma unroll
      for (int c = 0; c < C; ++c) a[c] = 0.f;
      for (int j = 0; j < cs.taps; ++j) {
        const int back = cs.taps - 1 - j;
        if (back > p) continue;
        widen16(back <= i ? get(r - (size_t)back * ldy) : state(p - back), h);
        tap(j, w);
#pragma unroll
        for (int c = 0; c < C; ++c) a[c] = __builtin_fmaf(w[c], h[c], a[c]);
      }
#pragma unroll
      for (int c = 0; c < C; ++c) a[c] += h[c];
      put16(y + (size_t)(sg.row0 + i) * ldy + d, a);
      renew_own(p, get(r));
    }
  }
  if (tile == 0 && shared_block >= 0) {
    const int stop = min(end, (shared_block + 1) * bs);
    for (int p = max(sg.pos0, stop - cs.keep); p < stop; ++p) renew(p, get(hs + (size_t)(p - sg.pos0) * ldy));
  }
}

template <typename T>
__global__ __launch_bounds__(256) void columns_kernel(const float* __restrict__ x, int ld, Columns first, Columns second, float eps, int ldy) {
  __shared__ float red[4];
  const Columns k = blockIdx.y ? second : first;
  const int tid = threadIdx.x, n = k.n;
  const float *src = x + (size_t)blockIdx.x * ld + k.col, *w = k.w;
  T* y = reinterpret_cast<T*>(k.y);
  float f = 1.f;
  if (((n | k.col | ld) & 3) == 0 && ldy <= 2048) {      // the row in registers
    float4 v[2], u[2];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int d = (i * 256 + tid) * 4;
      const bool in = d < n;
      v[i] = in ? *reinterpret_cast<const float4*>(src + d) : make_float4(0.f, 0.f, 0.f, 0.f);
      u[i] = in && w ? make_float4(w[d], w[d + 1], w[d + 2], w[d + 3]) : make_float4(1.f, 1.f, 1.f, 1.f);
      ss += (v[i].x * v[i].x + v[i].y * v[i].y) + (v[i].z * v[i].z + v[i].w * v[i].w);
    }
    if (w) f = 1.0f / sqrtf(block_sum(ss, red) / (float)n + eps);
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int d = (i * 256 + tid) * 4;
      if (d < ldy) put4(y + (size_t)blockIdx.x * ldy + d, v[i].x * f * u[i].x, v[i].y * f * u[i].y, v[i].z * f * u[i].z, v[i].w * f * u[i].w);
    }
    return;
  }
  if (w) {
    float ss = 0.f;
    for (int d = tid; d < n; d += 256) ss = __builtin_fmaf(src[d], src[d], ss);
    f = 1.0f / sqrtf(block_sum(ss, red) / (float)n + eps);
  }
  for (int d = tid * 4; d < ldy; d += 1024) {
    auto at = [&](int i) { return d + i < n ? src[d + i] * f * (w ? w[d + i] : 1.f) : 0.f; };
    put4(y + (size_t)blockIdx.x * ldy + d, at(0), at(1), at(2), at(3));
  }
}
__device__ __forceinline__ void gate1(uint16_t* p, float g) { *p = f32_to_bf16(bf16_to_f32(*p) * g); }
__device__ __forceinline__ void gate1(float* p, float g) { *p *= g; }
__device__ __forceinline__ void gate_quad(uint16_t* p, float4 g) {
  const uint2 x = *reinterpret_cast<const uint2*>(p);
  put4(p, bf16_to_f32((uint16_t)x.x) * g.x, bf16_to_f32((uint16_t)(x.x >> 16)) * g.y, bf16_to_f32((uint16_t)x.y) * g.z, bf16_to_f32((uint16_t)(x.y >> 16)) * g.w);
}
__device__ __forceinline__ void gate_quad(float* p, float4 g) {
  const float4 x = *reinterpret_cast<const float4*>(p);
  put4(p, x.x * g.x, x.y * g.y, x.z * g.z, x.w * g.w);
}
template <typename T, bool ELEM>
__global__ __launch_bounds__(256) void gate_rows_kernel(T* __restrict__ y, int ldy, int n, int dv, const float* __restrict__ g, int ldg) {
  const int t = blockIdx.x;
  if (((n | dv | ldy | ldg) & 3) == 0) {
    for (int i = (blockIdx.y * 256 + threadIdx.x) * 4; i < n; i += gridDim.y * 1024) {
      auto f = [&](float z) { return 1.f / (1.f + expf(-z)); };
      T* p = y + (size_t)t * ldy + i;
      if constexpr (ELEM) {
        const float4 z = *reinterpret_cast<const float4*>(g + (size_t)t * ldg + i);
        gate_quad(p, make_float4(f(z.x), f(z.y), f(z.z), f(z.w)));
      } else {
        const float v = f(g[(size_t)t * ldg + i / dv]);
        gate_quad(p, make_float4(v, v, v, v));
      }
    }
    return;
  }
  for (int i = blockIdx.y * 256 + threadIdx.x; i < n; i += gridDim.y * 256)
    gate1(y + (size_t)t * ldy + i, 1.f / (1.f + expf(-g[(size_t)t * ldg + (ELEM ? i : i / dv)])));
}
__global__ void affine_copy_kernel(const float* __restrict__ src, int n, float factor, float offset, float* __restrict__ dst) {
  const int i = blockIdx.x * blockDim.x + threadIdx.x;
  if (i < n) dst[i] = __builtin_fmaf(src[i], factor, offset);
}

template <typename T>
__global__ __launch_bounds__(256) void pair_rows_kernel(const float* __restrict__ x, const float* __restrict__ x0, int D4, int ld,
                                                        int half, T* __restrict__ y) {
  const int t = blockIdx.x;
  T* row = y + (size_t)t * 2 * half;
  for (int c4 = threadIdx.x; c4 < D4; c4 += 256) {
    const float4 a = *reinterpret_cast<const float4*>(x + (size_t)t * ld + c4 * 4);
    const float4 b = *reinterpret_cast<const float4*>(x0 + (size_t)t * ld + c4 * 4);
    put4(row + c4 * 4, a.x, a.y, a.z, a.w);
    put4(row + half + c4 * 4, b.x, b.y, b.z, b.w);
  }
}

// 32 lanes per head: H q heads, G k heads, G v heads (keys_as_values: none, the k heads write both pools) of one token row
template <typename T>
__global__ __launch_bounds__(256) void qkv_scatter_kernel(const float* __restrict__ qkv, int ldq, HeadGeom g, HeadRule rule, float eps,
                                                          const int32_t* __restrict__ slots, int bs, T* __restrict__ q,
                                                          T* __restrict__ kpool, T* __restrict__ vpool) {
  const int t = blockIdx.x, head = blockIdx.y * 8 + (threadIdx.x >> 5), l = threadIdx.x & 31;
  if (head >= g.H + (rule.keys_as_values ? 1 : 2) * g.G) return;     // (whole 32-lane group: the shuffles below stay inside it)
  const bool is_q = head < g.H, is_v = head >= g.H + g.G;
  const int kvh = is_v ? head - g.H - g.G : head - g.H;
  const int d_n = is_v ? g.dv : g.dk, d_p = is_v ? g.dvp : g.dkp;
  const float* src = qkv + (size_t)t * ldq + (is_v ? (size_t)(g.H + g.G) * g.dk + (size_t)kvh * g.dv : (size_t)head * g.dk);
  const float* bias = rule.bias && !is_v ? rule.bias + (size_t)head * g.dk : nullptr;
  const float* w = is_v ? nullptr : is_q ? rule.q_norm : rule.k_norm;
  const bool vec = (d_n & 3) == 0 && (((is_v ? (g.H + g.G) * g.dk : 0)) & 3) == 0;
  T *dst, *raw = nullptr;
  if (is_q) {
    dst = q + ((size_t)t * g.H + head) * g.dkp;
  } else {
    const int slot = slots[t];
    if (slot < 0) return;
    const int blk = slot / bs, off = slot - blk * bs;
    const size_t r = ((size_t)blk * g.G + kvh) * bs + off;
    dst = (is_v ? vpool : kpool) + r * d_p;
    if (rule.keys_as_values) raw = vpool + r * d_p;
  }
  auto get = [&](const float* p, int d) -> float4 {
    if (vec) return d < d_n ? *reinterpret_cast<const float4*>(p + d) : make_float4(0.f, 0.f, 0.f, 0.f);
    return make_float4(d < d_n ? p[d] : 0.f, d + 1 < d_n ? p[d + 1] : 0.f, d + 2 < d_n ? p[d + 2] : 0.f, d + 3 < d_n ? p[d + 3] : 0.f);
  };
  auto value = [&](int d) -> float4 {
    float4 v = get(src, d);
    if (bias) {
      const float4 b = get(bias, d);
      v = make_float4(v.x + b.x, v.y + b.y, v.z + b.z, v.w + b.w);
    }
    return v;
  };
  float f = 1.f;
  if (!is_v && rule.unit_norm) {
    float ss = 0.f;
    for (int d = l * 4; d < d_n; d += 128) {
      const float4 v = value(d);
      ss += (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w);
    }
#pragma unroll
    for (int m = 16; m >= 1; m >>= 1) ss += __shfl_xor(ss, m);
    f = 1.0f / sqrtf(ss / (float)d_n + eps);
  }
  for (int d = l * 4; d < d_p; d += 128) {
    const float4 v = value(d), k = w ? get(w, d) : make_float4(1.f, 1.f, 1.f, 1.f);
    put4(dst + d, v.x * f * k.x, v.y * f * k.y, v.z * f * k.z, v.w * f * k.w);
    if (raw) put4(raw + d, v.x, v.y, v.z, v.w);
  }
}

// 64 x 64 tile, 4 x 4 outputs per thread, fp32 FMAs: the 32-bit mode is for checking, not for speed
template <int EPI>
__global__ __launch_bounds__(256) void linear_f32_kernel(const float* __restrict__ w, int N, int K, const float* __restrict__ x, int ldx,
                                                         int T, EpiArgs e) {
  __shared__ float xs[16][68], ws[16][68];
  const int n0 = blockIdx.x * 64, m0 = blockIdx.y * 64, tid = threadIdx.x;
  const int tn = (tid & 15) * 4, tm = (tid >> 4) * 4, lr = tid >> 2, lk = (tid & 3) * 4;
  float acc[4][4] = {};
  for (int k0 = 0; k0 < K; k0 += 16) {
    const float4 xv = *reinterpret_cast<const float4*>(x + (size_t)min(m0 + lr, T - 1) * ldx + k0 + lk);
    const float4 wv = *reinterpret_cast<const float4*>(w + (size_t)min(n0 + lr, N - 1) * K + k0 + lk);
    __syncthreads();
    xs[lk][lr] = xv.x; xs[lk + 1][lr] = xv.y; xs[lk + 2][lr] = xv.z; xs[lk + 3][lr] = xv.w;
    ws[lk][lr] = wv.x; ws[lk + 1][lr] = wv.y; ws[lk + 2][lr] = wv.z; ws[lk + 3][lr] = wv.w;
    __syncthreads();
#pragma unroll
    for (int k = 0; k < 16; ++k)
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = __builtin_fmaf(xs[k][tm + i], ws[k][tn + j], acc[i][j]);
  }
  if (n0 + tn >= N) return;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int m = m0 + tm + i;
    if (m >= T) continue;
    float v[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = acc[i][j] * e.scale[n0 + tn + j];
    if constexpr (EPI == EPI_RELU2) {
#pragma unroll
      for (int j = 0; j < 4; ++j) { v[j] = fmaxf(v[j], 0.f); v[j] *= v[j]; }
      put4(reinterpret_cast<float*>(e.act_out) + (size_t)m * e.ld_act + n0 + tn, v[0], v[1], v[2], v[3]);
    } else if constexpr (EPI == EPI_GLU_CLIP) {
      float a[2];
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        const float g = fminf(v[2 * j], e.glu_limit), u = fminf(fmaxf(v[2 * j + 1], -e.glu_limit), e.glu_limit);
        a[j] = g / (1.f + expf(-e.glu_alpha * g)) * (u + 1.f);
      }
      *reinterpret_cast<float2*>(reinterpret_cast<float*>(e.act_out) + (size_t)m * e.ld_act + ((n0 + tn) >> 1)) = make_float2(a[0], a[1]);
    } else if constexpr (EPI == EPI_SOFTCAP) {
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = e.softcap * tanhf(v[j] / e.softcap);
      put4(e.out_f32 + (size_t)m * e.ld_out + n0 + tn, v[0], v[1], v[2], v[3]);
    } else {
      if constexpr (EPI == EPI_RESID) {
        const float4 r = *reinterpret_cast<const float4*>(e.resid_in + (size_t)m * e.ld_out + n0 + tn);
        v[0] += r.x; v[1] += r.y; v[2] += r.z; v[3] += r.w;
      }
      put4(e.out_f32 + (size_t)m * e.ld_out + n0 + tn, v[0], v[1], v[2], v[3]);
    }
  }
}

__global__ void place_tiled_kernel(const float* __restrict__ src, int ld, int src_col0, int rows, int cols, uint16_t* __restrict__ dst,
                                   int KT, int row0, int col0, int row_step) {
  const int c8n = (cols + 7) / 8;
  const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= (size_t)rows * c8n) return;
  const int r = (int)(i / c8n), c = (int)(i % c8n) * 8;
  const float* p = src + (size_t)r * ld + src_col0 + c;
  float v[8];
#pragma unroll
  for (int k = 0; k < 8; ++k) v[k] = c + k < cols ? p[k] : 0.f;
  const int R = row0 + r * row_step, C = col0 + c;
  const size_t at = (((size_t)(R >> 4) * KT + (C >> 5)) * 64 + (R & 15) + 16 * ((C & 31) >> 3)) * 8;
  *reinterpret_cast<uint4*>(dst + at) = make_uint4(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]), pack_bf16x2(v[4], v[5]), pack_bf16x2(v[6], v[7]));
}
__global__ void place_f32_kernel(const float* __restrict__ src, int ld, int src_col0, int rows, int cols, float* __restrict__ dst, int K,
                                 int row0, int col0, int row_step) {
  const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= (size_t)rows * cols) return;
  const int r = (int)(i / cols), c = (int)(i % cols);
  dst[(size_t)(row0 + r * row_step) * K + col0 + c] = src[(size_t)r * ld + src_col0 + c];
}
__global__ void place_rows_bf16_kernel(const float* __restrict__ src, int rows, int cols, uint16_t* __restrict__ dst, int K) {
  const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= (size_t)rows * cols) return;
  dst[(i / cols) * K + i % cols] = f32_to_bf16(src[i]);
}
__global__ void transpose_kernel(const float* __restrict__ src, int rows, int cols, float* __restrict__ dst, int ld_dst) {
  const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= (size_t)rows * cols) return;
  dst[(i % cols) * ld_dst + i / cols] = src[i];
}
__global__ void pack_rows_kernel(const float* __restrict__ src, int ld_src, int V, float* __restrict__ dst) {
  for (int v = blockIdx.x * blockDim.x + threadIdx.x; v < V; v += gridDim.x * blockDim.x)
    dst[(size_t)blockIdx.y * V + v] = src[(size_t)blockIdx.y * ld_src + v];
}

}  // namespace

int launch_embed_pos(const int32_t* ids, const int32_t* pos, const void* table, const void* ptable, float scale, bool f32, int T, int D,
                     int ld, float* resid, float* x0, hipStream_t s, const double* turns, void* y, int ldy) {
  MI_CHECK(!y || (ldy >= ld && ldy % 4 == 0), "embedding: output stride");
  if (f32)
    hipLaunchKernelGGL((embed_pos_kernel<float>), dim3(T), dim3(256), 0, s, ids, pos, (const float*)table, (const float*)ptable, scale, D, ld, resid, x0, turns, (float*)y, ldy);
  else
    hipLaunchKernelGGL((embed_pos_kernel<uint16_t>), dim3(T), dim3(256), 0, s, ids, pos, (const uint16_t*)table, (const uint16_t*)ptable, scale, D, ld, resid, x0, turns, (uint16_t*)y, ldy);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_layernorm_rows(const float* resid_in, float* resid_out, int T, int D, int ld, float eps, const NormOut& a,
                          const NormOut& b, int ldy, bool f32, hipStream_t s, const SlabSum* slabs) {
  MI_CHECK(ld % 4 == 0 && ld >= D && ld <= 32768 && ldy >= ld, "layer norm: row stride must be a multiple of 4, at least the width, at most 32768");
  MI_CHECK(!slabs || (slabs->T == T && slabs->N == ld && resid_out && !slabs->bias && !slabs->row_scale), "layer norm: pending K-split sum of another shape");
  const size_t lds = (size_t)(ld + 32) * sizeof(float);
  // few rows (token generation): one float4 per thread, the row is one round of loads; many rows: 256 threads, several rows per CU
  const int threads = T <= 32 ? std::min(1024, ceil_div(ld / 4, 64) * 64) : 256;
  const SlabSum sl = slabs ? *slabs : SlabSum();
  if (lds > 64 * 1024)
    MI_HIP(f32 ? hipFuncSetAttribute(reinterpret_cast<const void*>(layernorm_rows_kernel<float>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds)
               : hipFuncSetAttribute(reinterpret_cast<const void*>(layernorm_rows_kernel<uint16_t>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
  if (f32) hipLaunchKernelGGL((layernorm_rows_kernel<float>), dim3(T), dim3(threads), lds, s, resid_in, resid_out, D, ld, eps, a, b, ldy, sl);
  else hipLaunchKernelGGL((layernorm_rows_kernel<uint16_t>), dim3(T), dim3(threads), lds, s, resid_in, resid_out, D, ld, eps, a, b, ldy, sl);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

static int check_conv(const ConvState& c) {
  MI_CHECK(c.taps >= 1 && c.taps <= kConvRows && c.block_size > 0 && c.bt && c.pos && c.slots && c.MB >= 1, "convolution: taps / block table");
  MI_CHECK(c.taps == 1 || (c.ring && (c.keep >= c.taps - 1 || c.keep == c.block_size)), "convolution: state rows per block");
  return MI_OK;
}

int launch_sandwich_rows(const float* resid_in, float* resid_out, const RowSource& src, const float* w_post, const float* w_pre, int T,
                         int D, int ld, int groups, float eps, const ConvState* conv, void* y, int ldy, bool f32, hipStream_t s, bool as_is) {
  MI_CHECK(!as_is || !w_pre, "sandwich rows: a pre-norm, or the row as it is");
  MI_CHECK(T >= 1 && ld % 4 == 0 && ld >= D && ld <= 32768 && groups >= 1 && D % groups == 0, "sandwich rows: row stride / norm groups");
  MI_CHECK(!src.any() || (resid_out && resid_out != resid_in), "sandwich rows: residual output");
  MI_CHECK(!src.slabs.slab || (src.slabs.T == T && src.slabs.N == ld && !src.slabs.bias && !src.slabs.row_scale), "sandwich rows: pending K-split sum of another shape");
  MI_CHECK(src.slabs.slab || !src.any() || src.ld >= ld, "sandwich rows: source stride");
  MI_CHECK(!src.y16 || src.pair_w, "sandwich rows: bf16 sources are built for experts");
  MI_CHECK(!(w_pre || as_is) || (y && ldy >= ld && ldy % 4 == 0), "sandwich rows: output stride");
  ConvState cs;
  if (conv) {
    int rc = check_conv(*conv);
    if (rc != MI_OK) return rc;
    cs = *conv;
  }
  if (T <= 32 && (w_pre || as_is) && ld <= 4096 && ld == D && (D / groups) % 256 == 0 && (!conv || conv->taps <= 4)) {
    const int threads = ceil_div(ld / 4, 64) * 64, gs = D / groups;
#define MI_TOKEN(TAPS) \
    if (f32) hipLaunchKernelGGL((sandwich_token_kernel<float, TAPS>), dim3(T), dim3(threads), 0, s, resid_in, resid_out, src, w_post, w_pre, D, ld, gs, eps, cs, (float*)y, ldy); \
    else hipLaunchKernelGGL((sandwich_token_kernel<uint16_t, TAPS>), dim3(T), dim3(threads), 0, s, resid_in, resid_out, src, w_post, w_pre, D, ld, gs, eps, cs, (uint16_t*)y, ldy)
    switch (conv ? conv->taps : 0) {
      case 0: MI_TOKEN(0); break;
      case 1: MI_TOKEN(1); break;
      case 2: MI_TOKEN(2); break;
      case 3: MI_TOKEN(3); break;
      default: MI_TOKEN(4);
    }
#undef MI_TOKEN
    MI_HIP(hipGetLastError());
    return MI_OK;
  }
  const size_t lds = (size_t)(ld + std::max(groups, 16) + groups) * sizeof(float);
  const int threads = T <= 32 ? std::min(1024, ceil_div(ld / 4, 64) * 64) : 256;
  const void* kern = f32 ? reinterpret_cast<const void*>(sandwich_rows_kernel<float>) : reinterpret_cast<const void*>(sandwich_rows_kernel<uint16_t>);
  MI_CHECK(lds <= 160 * 1024, "sandwich rows: row too long");
  if (lds > 64 * 1024) { int rc = ensure_dynamic_lds(kern, 160 * 1024); if (rc != MI_OK) return rc; }
  if (f32) hipLaunchKernelGGL((sandwich_rows_kernel<float>), dim3(T), dim3(threads), lds, s, resid_in, resid_out, src, w_post, w_pre, D, ld, groups, eps, cs, (float*)y, ldy, as_is);
  else hipLaunchKernelGGL((sandwich_rows_kernel<uint16_t>), dim3(T), dim3(threads), lds, s, resid_in, resid_out, src, w_post, w_pre, D, ld, groups, eps, cs, (uint16_t*)y, ldy, as_is);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_conv_rows(const void* h, const ConvState& conv, const AttnSeg* sd, const AttnSeg* sh, int nseg, int D, int ld, void* y, int ldy,
                     bool f32, hipStream_t s) {
  int rc = check_conv(conv);
  if (rc != MI_OK) return rc;
  MI_CHECK(nseg >= 1 && ld % 8 == 0 && ld >= D && ldy >= ld && ldy % 8 == 0 && h != y, "convolution: strides");
  const int rows = conv.taps <= 4 ? 8 : kConvRows;
  int tiles = 0;
  for (int i = 0; i < nseg; ++i) tiles += ceil_div(sh[i].n, rows);
  const dim3 grid(tiles, ceil_div(ld, f32 ? 1024 : 2048));
#define MI_CONV(TAPS, ROWS) \
  if (f32) hipLaunchKernelGGL((conv_rows_kernel<float, TAPS, ROWS>), grid, dim3(256), 0, s, (const float*)h, conv, sd, nseg, ld, (float*)y, ldy); \
  else hipLaunchKernelGGL((conv_rows_kernel<uint16_t, TAPS, ROWS>), grid, dim3(256), 0, s, (const uint16_t*)h, conv, sd, nseg, ld, (uint16_t*)y, ldy)
  switch (conv.taps) {
    case 2: MI_CONV(2, 8); break;
    case 3: MI_CONV(3, 8); break;
    case 4: MI_CONV(4, 8); break;
    case 1: MI_CONV(1, 8); break;
    default: MI_CONV(0, kConvRows);
  }
#undef MI_CONV
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_columns(const float* x, int ld, Columns a, Columns b, float eps, int T, int ldy, bool f32, hipStream_t s) {
  const bool two = b.y != nullptr;
  MI_CHECK(T >= 1 && a.y && a.n >= 1 && a.col >= 0 && ld >= a.col + a.n && ldy >= a.n && ldy % 4 == 0, "columns: strides");
  MI_CHECK(!two || (b.n >= 1 && b.col >= 0 && ld >= b.col + b.n && ldy >= b.n), "columns: strides");
  const dim3 grid(T, two ? 2 : 1);
  if (f32) hipLaunchKernelGGL((columns_kernel<float>), grid, dim3(256), 0, s, x, ld, a, b, eps, ldy);
  else hipLaunchKernelGGL((columns_kernel<uint16_t>), grid, dim3(256), 0, s, x, ld, a, b, eps, ldy);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_gate_rows(void* y, int ldy, int T, int H, int dv, const float* g, int ldg, bool per_element, bool f32, hipStream_t s) {
  const int n = H * dv;
  MI_CHECK(T >= 1 && H >= 1 && dv >= 1 && ldy >= n && ldg >= (per_element ? n : H), "gate rows: strides");
  const dim3 grid(T, std::min(ceil_div(n, 1024), 16));
  if (f32 && per_element) hipLaunchKernelGGL((gate_rows_kernel<float, true>), grid, dim3(256), 0, s, (float*)y, ldy, n, dv, g, ldg);
  else if (f32) hipLaunchKernelGGL((gate_rows_kernel<float, false>), grid, dim3(256), 0, s, (float*)y, ldy, n, dv, g, ldg);
  else if (per_element) hipLaunchKernelGGL((gate_rows_kernel<uint16_t, true>), grid, dim3(256), 0, s, (uint16_t*)y, ldy, n, dv, g, ldg);
  else hipLaunchKernelGGL((gate_rows_kernel<uint16_t, false>), grid, dim3(256), 0, s, (uint16_t*)y, ldy, n, dv, g, ldg);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_offset_copy(const float* src, int n, float offset, float* dst, hipStream_t s) {
  MI_CHECK(n >= 1, "offset copy: size");
  hipLaunchKernelGGL(affine_copy_kernel, dim3(ceil_div(n, 256)), dim3(256), 0, s, src, n, 1.f, offset, dst);
  MI_HIP(hipGetLastError());
  return MI_OK;
}
int launch_scaled_copy(const float* src, int n, float factor, float* dst, hipStream_t s) {
  MI_CHECK(n >= 1, "scaled copy: size");
  hipLaunchKernelGGL(affine_copy_kernel, dim3(ceil_div(n, 256)), dim3(256), 0, s, src, n, factor, 0.f, dst);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_pair_rows(const float* x, const float* x0, int T, int D, int ld, int half, void* y, bool f32, hipStream_t s) {
  MI_CHECK(ld % 4 == 0 && half % 4 == 0 && half >= ld && ld >= D, "pair rows: strides");
  if (f32) hipLaunchKernelGGL((pair_rows_kernel<float>), dim3(T), dim3(256), 0, s, x, x0, ld / 4, ld, half, (float*)y);
  else hipLaunchKernelGGL((pair_rows_kernel<uint16_t>), dim3(T), dim3(256), 0, s, x, x0, ld / 4, ld, half, (uint16_t*)y);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_qkv_scatter(const float* qkv, int ldq, int T, const HeadGeom& g, const HeadRule& rule, float eps, const int32_t* slots,
                       int block_size, void* q, void* kpool, void* vpool, bool f32, hipStream_t s) {
  MI_CHECK(!rule.keys_as_values || (g.dv == g.dk && g.dvp == g.dkp), "qkv scatter: values that are the keys have their size");
  MI_CHECK(rule.unit_norm || (!rule.q_norm && !rule.k_norm), "qkv scatter: norm weights without a norm");
  MI_CHECK(ldq % 4 == 0 && ldq >= (g.H + g.G) * g.dk + (rule.keys_as_values ? 0 : g.G * g.dv) && g.dkp % 16 == 0 && g.dvp % 16 == 0 && g.dkp >= g.dk && g.dvp >= g.dv,
           "qkv scatter: geometry");
  const dim3 grid(T, ceil_div(g.H + 2 * g.G, 8));
  if (f32) hipLaunchKernelGGL((qkv_scatter_kernel<float>), grid, dim3(256), 0, s, qkv, ldq, g, rule, eps, slots, block_size, (float*)q, (float*)kpool, (float*)vpool);
  else hipLaunchKernelGGL((qkv_scatter_kernel<uint16_t>), grid, dim3(256), 0, s, qkv, ldq, g, rule, eps, slots, block_size, (uint16_t*)q, (uint16_t*)kpool, (uint16_t*)vpool);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_linear_f32(const float* w, int N, int K, const float* x, int ldx, int T, int epi, const EpiArgs& e, hipStream_t s) {
  MI_CHECK(N % 16 == 0 && K % 16 == 0 && ldx % 4 == 0 && T >= 1, "linear_f32: N % 16 == 0, K % 16 == 0, ldx % 4 == 0");
  const dim3 grid(ceil_div(N, 64), ceil_div(T, 64));
  if (epi == EPI_F32) hipLaunchKernelGGL((linear_f32_kernel<EPI_F32>), grid, dim3(256), 0, s, w, N, K, x, ldx, T, e);
  else if (epi == EPI_RESID) hipLaunchKernelGGL((linear_f32_kernel<EPI_RESID>), grid, dim3(256), 0, s, w, N, K, x, ldx, T, e);
  else if (epi == EPI_RELU2) hipLaunchKernelGGL((linear_f32_kernel<EPI_RELU2>), grid, dim3(256), 0, s, w, N, K, x, ldx, T, e);
  else if (epi == EPI_GLU_CLIP) hipLaunchKernelGGL((linear_f32_kernel<EPI_GLU_CLIP>), grid, dim3(256), 0, s, w, N, K, x, ldx, T, e);
  else if (epi == EPI_SOFTCAP) hipLaunchKernelGGL((linear_f32_kernel<EPI_SOFTCAP>), grid, dim3(256), 0, s, w, N, K, x, ldx, T, e);
  else { set_error("linear_f32: epilogue"); return MI_EINVAL; }
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_place(const float* src, int ld, int src_col0, int rows, int cols, void* dst, int K, bool f32, int row0, int col0, hipStream_t s,
                 int row_step) {
  MI_CHECK(col0 % 8 == 0 && K % 32 == 0 && col0 + cols <= K && src_col0 + cols <= ld, "place: columns");
  if (f32) {
    const size_t n = (size_t)rows * cols;
    hipLaunchKernelGGL(place_f32_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, s, src, ld, src_col0, rows, cols, (float*)dst, K, row0, col0, row_step);
  } else {
    const size_t n = (size_t)rows * ((cols + 7) / 8);
    hipLaunchKernelGGL(place_tiled_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, s, src, ld, src_col0, rows, cols, (uint16_t*)dst, K / 32, row0, col0, row_step);
  }
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_place_rows(const float* src, int rows, int cols, void* dst, int K, bool f32, hipStream_t s) {
  MI_CHECK(rows > 0 && cols > 0 && cols <= K, "place rows: columns");
  const dim3 grid((unsigned)(((size_t)rows * cols + 255) / 256));
  if (f32) hipLaunchKernelGGL(place_f32_kernel, grid, dim3(256), 0, s, src, cols, 0, rows, cols, (float*)dst, K, 0, 0, 1);
  else hipLaunchKernelGGL(place_rows_bf16_kernel, grid, dim3(256), 0, s, src, rows, cols, (uint16_t*)dst, K);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_transpose(const float* src, int rows, int cols, float* dst, int ld_dst, hipStream_t s) {
  MI_CHECK(ld_dst >= rows && rows > 0 && cols > 0, "transpose: strides");
  const size_t n = (size_t)rows * cols;
  hipLaunchKernelGGL(transpose_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, s, src, rows, cols, dst, ld_dst);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_pack_rows(const float* src, int ld_src, int T, int V, float* dst, hipStream_t s) {
  hipLaunchKernelGGL(pack_rows_kernel, dim3(ceil_div(V, 1024), T), dim3(256), 0, s, src, ld_src, V, dst);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

}  // namespace mi
