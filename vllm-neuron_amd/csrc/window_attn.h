// Paged attention with separate query/key and value sizes, a sliding window or chunks, a per-head distance bias, a softmax
// sink and an output gate -- the attention of the layer-stack decoders (stack.hip).  Same pool addressing as attn_kernels.h, rows
// padded to 16 elements:  K [num_blocks][G][block_size][dkp], V [num_blocks][G][block_size][dvp].
//
//   s_ij = scale q_i.k_j - slope_h (i - j)      for 0 <= i - j < window and floor(i / chunk) = floor(j / chunk)
//          (or + table_h[min(i - j, table_n - 1)] in place of the slope)
//   o_i  = sum_j exp(s_ij) v_j / (sink + sum_j exp(s_ij)), sink = 1 or exp(a number per head);  times the gate
#pragma once
#include <vector>

#include "stack_kernels.h"

namespace mi {

struct AttnSpec {
  HeadGeom g;
  float scale = 1.f;
  int window = 0;                  // keys a query sees, itself included; 0 = every earlier token
  const float* slopes = nullptr;   // [H] or null: no distance bias
  int unit_norm = 0;               // q and k heads have unit root mean square: |q.k| <= dk
  int sink = 0;                    // 1: one more score in the denominator, without a value: ...
  int chunk = 0;                   // a query sees keys of its own chunk of this many positions (from 0 on); 0 = no chunks
  const float* sinks = nullptr;    // ... [H], null: 0
  const float* table = nullptr;    // [H][table_n] or null: bias by distance, the last entry from there on
  int table_n = 0;
  // the first key that the query at position p sees
  __host__ __device__ int first_key(int p) const {
    const int lo = window > 0 && p >= window ? p - window + 1 : 0, at = chunk > 0 ? p - p % chunk : 0;
    return lo > at ? lo : at;
  }
  // the most keys a query sees when a sequence has up to n
  int most_keys(int n) const {
    if (window > 0 && window < n) n = window;
    return chunk > 0 && chunk < n ? chunk : n;
  }
};
// Row of a distance table of `rows` rows for every distance from 0 on, up to the first one of the last row or `limit` (> 0) entries: distances
// below half the rows have a row each, from there on rows are spaced by logarithm up to distance `far`.
std::vector<int> distance_rows(int rows, double far, int limit);
// mult sigmoid(z) on the heads' outputs: row t at z + t ld, an element per head or per element of the heads; z null: none
struct OutGate {
  const float* z = nullptr;
  int ld = 0;
  bool per_element = false;
  float mult = 1.f;
};

// Plain form (one wave per row and head, any sizes, bf16 or fp32 pool): the 32-bit mode, and sizes the MFMA kernels are not built for.
// segs [nseg] on the device; null: row r is block-table row r (token generation).
int launch_attn_plain(const AttnSpec& a, const void* q, const void* kpool, const void* vpool, int block_size, const int32_t* block_table,
                      int MB, const int32_t* pos, const AttnSeg* segs, int nseg, int T, void* out, int ldo, bool f32, hipStream_t s,
                      OutGate gate = OutGate());

// MFMA forms (bf16; gates per head).  Built for dk, dv <= 256 and at most 64 query heads per kv head:
bool attn_window_supported(const HeadGeom& g);
// ... and for distance tables that fit the LDS beside the tiles:
bool attn_table_supported(const HeadGeom& g, int table_n);
// token generation: ctx_lens[b] keys incl. the new one; max_ctx bounds them (sizes the context split).
size_t attn_window_scratch_bytes(int B, const HeadGeom& g);
int launch_attn_window_decode(const AttnSpec& a, const uint16_t* q, const uint16_t* kpool, const uint16_t* vpool, int block_size,
                              const int32_t* block_table, int MB, const int32_t* ctx_lens, int B, int max_ctx, uint16_t* out, int ldo,
                              void* scratch, hipStream_t s, OutGate gate = OutGate());
// context encoding of every segment with at least min_rows (>= 2) rows (host copy of segs sizes the grid); others are left alone
int launch_attn_window_prefill(const AttnSpec& a, const uint16_t* q, const uint16_t* kpool, const uint16_t* vpool, int block_size,
                               const int32_t* block_table, int MB, const AttnSeg* segs_dev, const AttnSeg* segs_host, int nseg,
                               uint16_t* out, int ldo, hipStream_t s, int min_rows = 2, OutGate gate = OutGate());

}  // namespace mi
