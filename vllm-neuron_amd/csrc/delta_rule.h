// Gated delta rule with one decay per head and key channel: a recurrent mixer of the layer-stack decoders (stack.hip).
//   x = silu(causal convolution of the projected row, per channel);  q, k = unit(x_q) d^-1/2, unit(x_k)
//   g = exp(-exp(A) softplus(z + dt)),  b = sigmoid(.)
//   S <- diag(g) S;  u = b (v - S^T k);  S <- S + k u^T;  o = S^T q
//   y = RMSnorm(o) w sigmoid(z_gate), per head
// Everything here is fp32 whatever the model's compute type; y is written in the compute type.
//
// Prompts run in chunks of kDeltaChunk tokens.  With L the running sum of log g inside a chunk and S0 the state ahead of it,
//   A_ij = b_i sum_d k_i k_j exp(L_i - L_j) (j < i),  P_ij = sum_d q_i k_j exp(L_i - L_j) (j <= i),  T = (I + A)^-1 diag(b)
//   u = T v - T (k exp L) S0
//   o = (q exp L - P T (k exp L)) S0 + P T v
//   S = diag(exp L_end) S0 + (k exp(L_end - L))^T u
// every exponent is of a number <= 0.  The factors do not depend on the state: one kernel makes them for all chunks at once, a second
// one walks a sequence's chunks with the state in registers.
#pragma once
#include "stack_kernels.h"

namespace mi {

struct DeltaGeom {
  int H = 0, G = 0, dk = 0, dv = 0;   // heads, query / key heads, sizes (up to 256)
  int dkp = 0, dvp = 0;               // padded to 16: zeros in the state and the factors
  int taps = 0;
  __host__ __device__ int channels() const { return 2 * G * dk + H * dv; }     // of the convolution: q heads, k heads, v heads
  size_t state_floats() const { return (size_t)H * dkp * dvp; }                 // of a slot
  size_t ring_floats() const { return (size_t)taps * channels(); }
};
struct DeltaIn {
  const float* proj = nullptr;        // [rows, ldp]: the convolution's channels at column 0, H rows of beta's projection at column beta
  int ldp = 0, beta = 0;
  const float* z = nullptr;           // [rows, ldz]: decays [H dk] at column 0, output gates [H dv] at column gate
  int ldz = 0, gate = 0;
  const float *conv = nullptr, *a_log = nullptr, *dt = nullptr, *norm = nullptr;   // [taps][channels] (last row: the token itself), [H], [H dk], [dv]
  float eps = 0.f;
  float *state = nullptr, *ring = nullptr;   // [slots][H][dkp][dvp], [slots][taps][channels]: position p at row p % taps
  const int32_t* slots = nullptr;     // [sequences] slot of the sequence in block-table row i
  const int32_t* pos = nullptr;       // [rows]
};
bool delta_supported(const DeltaGeom& g);
constexpr int kDeltaChunk = 16;
size_t delta_chunk_floats(const DeltaGeom& g);         // device memory behind a chunk of a prompt: factors, values, outputs
// token generation: row = sequence (segs null), or the one-row segments of a ragged batch
int launch_delta_token(const DeltaGeom& g, const DeltaIn& in, int rows, const AttnSeg* segs, void* y, int ldy, bool f32, hipStream_t s);
// the segments of two rows and more; records: memory for max_chunks chunks, more of them go in pieces
int launch_delta_prompt(const DeltaGeom& g, const DeltaIn& in, const AttnSeg* segs_dev, const AttnSeg* segs_host, int nseg, float* records,
                        int max_chunks, void* y, int ldy, bool f32, hipStream_t s);

}  // namespace mi
