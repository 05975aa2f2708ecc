// Paged attention with separate query/key and value sizes, a sliding window, a per-head distance bias and a softmax
// sink -- the attention of the layer-stack decoders (stack.hip).  Same pool addressing as attn_kernels.h, rows padded to
// 16 elements:  K [num_blocks][G][block_size][dkp], V [num_blocks][G][block_size][dvp].
//
//   s_ij = scale q_i.k_j - slope_h (i - j)      for 0 <= i - j < window
//   o_i  = sum_j exp(s_ij) v_j / (sink + sum_j exp(s_ij))
#pragma once
#include "stack_kernels.h"

namespace mi {

struct AttnSpec {
  HeadGeom g;
  float scale = 1.f;
  int window = 0;                  // keys a query sees, itself included; 0 = every earlier token
  const float* slopes = nullptr;   // [H] or null: no distance bias
  int unit_norm = 0;               // q and k heads have unit root mean square: |q.k| <= dk
  int sink = 0;                    // 1: one more score of 0 in the denominator, without a value
};

// Plain form (one wave per row and head, any sizes, bf16 or fp32 pool): the 32-bit mode, and sizes the MFMA kernels are not built for.
// segs [nseg] on the device; null: row r is block-table row r (token generation).
int launch_attn_plain(const AttnSpec& a, const void* q, const void* kpool, const void* vpool, int block_size, const int32_t* block_table,
                      int MB, const int32_t* pos, const AttnSeg* segs, int nseg, int T, void* out, int ldo, bool f32, hipStream_t s);

// MFMA forms (bf16).  Built for dk, dv <= 256 and at most 64 query heads per kv head:
bool attn_window_supported(const HeadGeom& g);
// token generation: ctx_lens[b] keys incl. the new one; max_ctx bounds them (sizes the context split).
size_t attn_window_scratch_bytes(int B, const HeadGeom& g);
int launch_attn_window_decode(const AttnSpec& a, const uint16_t* q, const uint16_t* kpool, const uint16_t* vpool, int block_size,
                              const int32_t* block_table, int MB, const int32_t* ctx_lens, int B, int max_ctx, uint16_t* out, int ldo,
                              void* scratch, hipStream_t s);
// context encoding of every segment with at least min_rows (>= 2) rows (host copy of segs sizes the grid); others are left alone
int launch_attn_window_prefill(const AttnSpec& a, const uint16_t* q, const uint16_t* kpool, const uint16_t* vpool, int block_size,
                               const int32_t* block_table, int MB, const AttnSeg* segs_dev, const AttnSeg* segs_host, int nseg,
                               uint16_t* out, int ldo, hipStream_t s, int min_rows = 2);

}  // namespace mi
