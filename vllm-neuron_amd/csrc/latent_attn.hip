// Latent attention.  See latent_attn.h.
#include "latent_attn.h"

namespace mi {

namespace {

__device__ __forceinline__ void put4(uint16_t* p, float4 v) { *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf16x2(v.x, v.y), pack_bf16x2(v.z, v.w)); }
__device__ __forceinline__ void put4(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }

// blockIdx.y < q groups: 8 heads of 32 lanes each; the last one: the latent, one work-group per row
template <typename T>
__global__ __launch_bounds__(256) void latent_scatter_kernel(const float* __restrict__ qd, int ldq, LatentGeom g, const float* __restrict__ c_norm,
                                                             float eps, const int32_t* __restrict__ slots, int bs, T* __restrict__ q,
                                                             T* __restrict__ pool) {
  __shared__ float red[4];
  const int t = blockIdx.x, tid = threadIdx.x;
  if ((int)blockIdx.y < ceil_div(g.H, 8)) {
    const int h = blockIdx.y * 8 + (tid >> 5);
    if (h >= g.H) return;
    const float* src = qd + (size_t)t * ldq + (size_t)h * g.dk;
    T* dst = q + ((size_t)t * g.H + h) * g.dkp;
    const bool vec = (g.dk & 3) == 0;
    for (int d = (tid & 31) * 4; d < g.dkp; d += 128) {
      float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
      if (vec) {
        if (d < g.dk) v = *reinterpret_cast<const float4*>(src + d);
      } else {
        if (d < g.dk) v.x = src[d];
        if (d + 1 < g.dk) v.y = src[d + 1];
        if (d + 2 < g.dk) v.z = src[d + 2];
        if (d + 3 < g.dk) v.w = src[d + 3];
      }
      put4(dst + d, v);
    }
    return;
  }
  const float* src = qd + (size_t)t * ldq + (size_t)g.H * g.dk;
  float ss = 0.f;
  for (int d = tid; d < g.rank; d += 256) ss = __builtin_fmaf(src[d], src[d], ss);
  ss = wave_sum(ss);
  if ((tid & 63) == 0) red[tid >> 6] = ss;
  __syncthreads();
  const float f = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)g.rank + eps);
  const int slot = slots[t];
  if (slot < 0) return;
  T* dst = pool + (size_t)slot * g.rp;        // (a block's rows are consecutive: slot = block * block_size + offset)
  for (int d = tid * 4; d < g.rp; d += 1024) {
    auto at = [&](int i) { return d + i < g.rank ? src[d + i] * f * c_norm[d + i] : 0.f; };
    put4(dst + d, make_float4(at(0), at(1), at(2), at(3)));
  }
}

// a wave: one 16-row tile of W_h against 16 tokens
__global__ __launch_bounds__(256) void head_linear_kernel(const uint4* __restrict__ w, int H, int NT, int KT, const uint16_t* __restrict__ x,
                                                          int T, uint16_t* __restrict__ y, int ldy, int y_head, int n_valid) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, g4 = lane >> 4, c = lane & 15;
  const int nt = blockIdx.x * 4 + wave, h = blockIdx.y, m = blockIdx.z * 16 + c;
  if (nt >= NT) return;
  const u32x4_t* W = reinterpret_cast<const u32x4_t*>(w) + ((size_t)h * NT + nt) * KT * 64 + lane;
  const u32x4_t* X = reinterpret_cast<const u32x4_t*>(x + ((size_t)min(m, T - 1) * H + h) * (KT * 32)) + g4;
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
  if (m >= T) return;
  const int n = nt * 16 + g4 * 4;
  uint16_t* o = y + (size_t)m * ldy + (size_t)h * y_head + n;
  if (n + 4 <= n_valid && ((y_head | ldy) & 3) == 0) {
    put4(o, make_float4(acc[0], acc[1], acc[2], acc[3]));
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (n + i < n_valid) o[i] = f32_to_bf16(acc[i]);
  }
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

}  // namespace

int launch_latent_scatter(const float* qd, int ldq, int T, const LatentGeom& g, const float* c_norm, float eps, const int32_t* slots,
                          int bs, void* q, void* pool, bool f32, hipStream_t s) {
  MI_CHECK(T >= 1 && ldq % 4 == 0 && ldq >= g.H * g.dk + (c_norm ? g.rank : 0) && g.dkp >= g.dk && g.dkp % 32 == 0 && g.rp >= g.rank && g.rp % 32 == 0 && bs > 0,
           "latent scatter: geometry");
  const dim3 grid(T, ceil_div(g.H, 8) + (c_norm ? 1 : 0));
  if (f32) hipLaunchKernelGGL((latent_scatter_kernel<float>), grid, dim3(256), 0, s, qd, ldq, g, c_norm, eps, slots, bs, (float*)q, (float*)pool);
  else hipLaunchKernelGGL((latent_scatter_kernel<uint16_t>), grid, dim3(256), 0, s, qd, ldq, g, c_norm, eps, slots, bs, (uint16_t*)q, (uint16_t*)pool);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_head_linear(const void* w, int H, int N, int K, const void* x, int T, void* y, int ldy, int y_head, int n_valid, bool f32, hipStream_t s) {
  MI_CHECK(H >= 1 && T >= 1 && N % 16 == 0 && K % 32 == 0 && n_valid <= N && y_head >= n_valid && ldy >= (H - 1) * y_head + n_valid, "head linear: shape");
  if (f32) hipLaunchKernelGGL(head_linear_f32_kernel, dim3(T, ceil_div(n_valid, 64), H), dim3(64), 0, s, (const float*)w, H, N, K, (const float*)x, (float*)y, ldy, y_head, n_valid);
  else hipLaunchKernelGGL(head_linear_kernel, dim3(ceil_div(N / 16, 4), H, ceil_div(T, 16)), dim3(256), 0, s, (const uint4*)w, H, N / 16, K / 32, (const uint16_t*)x, T, (uint16_t*)y, ldy, y_head, n_valid);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

}  // namespace mi
