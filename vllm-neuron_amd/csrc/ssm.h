// State-space mixers of the layer-stack decoders (stack.hip): a recurrent state per sequence that decays and takes up inputs.
//
//   short convolution   y_t = silu(b + sum_j w_j x_(t - taps + 1 + j)) per channel; the last inputs are part of the state
//   selective scan      per channel c and state n:  S <- exp(dt_c A_cn) S + dt_c x_c B_n;  y_c = sum_n S_cn C_n + D_c x_c,  times silu(z_c)
//   state-space duality per head, with B and C shared by a group's heads:  S <- exp(dt A) S + dt B x^T;  y = S^T C + D x
//                       (S: state x head size), then y silu(z) in equal parts over their root mean square, times a weight
//
// dt = softplus(projection + bias).  States, step sizes, decays and what enters them are fp32 whatever the model's compute type; the
// convolution's output and the mixer's are in the compute type.
#pragma once
#include "stack_kernels.h"

namespace mi {

// ---- short convolution ----------------------------------------------------------------------------------------------------------
struct ShortConv {
  const float *w = nullptr, *b = nullptr;   // [taps][C] (last row: the token itself), [C]
  int taps = 0, C = 0;                      // up to 16 taps
  float* ring = nullptr;                    // [slots][taps][C]: position p at row p % taps
  const int32_t* slots = nullptr;           // [sequences] slot of the sequence in block-table row i
};
// x [rows, ldx] fp32 -> y [rows, ldy] in the compute type, zero beyond C; the ring read and renewed.  nseg 0: token generation, row = sequence
int launch_short_conv(const float* x, int ldx, const ShortConv& cv, const int32_t* pos, const AttnSeg* segs_dev, const AttnSeg* segs_host, int nseg, int rows,
                      void* y, int ldy, bool f32, hipStream_t s);

// ---- selective scan -------------------------------------------------------------------------------------------------------------
struct ScanGeom {
  int C = 0, N = 0, Np = 0, rank = 0, rank_p = 0;   // channels; states, padded; low rank of the step size, padded to 8
  size_t state_floats() const { return (size_t)C * Np; }   // of a slot
};
ScanGeom scan_geom(int C, int N, int rank);
bool scan_supported(int N);                          // up to 256 states
struct ScanIn {
  const void* x = nullptr;                           // [rows, ldx] compute type: the convolution's output
  int ldx = 0;
  const float* low = nullptr;                        // [rows, ldl]: dt's low-rank input at column 0, B at col_b, C at col_c
  int ldl = 0, col_b = 0, col_c = 0;
  const float* dt = nullptr;                         // prompts: [rows, ldt] projected step sizes, without their bias
  int ldt = 0;
  const void* w_dt = nullptr;                        // tokens: [C][rank_p] compute type
  const float *dt_bias = nullptr, *a2 = nullptr, *d = nullptr;   // [C], [C][Np] = -exp(A_log) log2 e (zero beyond N), [C]
  const float* z = nullptr;                          // [rows, ldz]
  int ldz = 0;
  float* state = nullptr;                            // [slots][C][Np]
  const int32_t *slots = nullptr, *pos = nullptr;
};
// y [rows, ldy] compute type.  Token generation: row = sequence (segs null), or the one-row segments of a ragged batch
int launch_scan_token(const ScanGeom& g, const ScanIn& in, int rows, const AttnSeg* segs, void* y, int ldy, bool f32, hipStream_t s);
// the segments of two rows and more
int launch_scan_prompt(const ScanGeom& g, const ScanIn& in, const AttnSeg* segs, int nseg, void* y, int ldy, bool f32, hipStream_t s);
// a2 [C][Np] (zero-filled) of A_log [C, N]
int launch_scan_decay(const float* a_log, const ScanGeom& g, float* a2, hipStream_t s);

// ---- state-space duality --------------------------------------------------------------------------------------------------------
// Prompts run in chunks of kSsdChunk tokens.  With L the running sum of dt A inside a chunk and S0 the state ahead of it,
//   y_i = e^(L_i) S0^T C_i + sum_(j <= i) (C_i.B_j) e^(L_i - L_j) dt_j x_j;   S = e^(L_end) S0 + sum_j e^(L_end - L_j) dt_j B_j x_j^T
// every exponent is of a number <= 0; L is summed in fp64 and kept in two fp32 parts, so that a strong decay leaves the following ones exact.
// One kernel makes C B^T and the steps of all chunks at once, a second one walks a sequence's chunks with the state in registers.
struct SsdGeom {
  int H = 0, P = 0, N = 0, G = 0;   // heads, head size, states, groups (sizes up to 256)
  int Pp = 0, Np = 0;               // padded to 16: zeros in the state
  int inner() const { return H * P; }
  int channels() const { return H * P + 2 * G * N; }       // of the convolution: x, B, C
  size_t state_floats() const { return (size_t)H * Np * Pp; }
};
SsdGeom ssd_geom(int H, int P, int N, int G);
bool ssd_supported(const SsdGeom& g);
struct SsdIn {
  const void* xbc = nullptr;        // [rows, ldx] compute type: the convolution's output
  int ldx = 0;
  const float* dt = nullptr;        // [rows, ldt] projected step sizes, without their bias
  int ldt = 0;
  const float *dt_bias = nullptr, *a_log = nullptr, *d = nullptr;   // [H]
  float* state = nullptr;           // [slots][H][Np][Pp]
  const int32_t *slots = nullptr, *pos = nullptr;
};
constexpr int kSsdChunk = 64;
size_t ssd_chunk_floats(const SsdGeom& g);               // device memory behind a chunk of a prompt
// y [rows, ldy] fp32, heads concatenated.  conv: the convolution in the same launch, from proj [rows, ldp] (in.xbc is not read)
int launch_ssd_token(const SsdGeom& g, const SsdIn& in, int rows, const AttnSeg* segs, float* y, int ldy, bool f32, hipStream_t s, const ShortConv* conv = nullptr,
                     const float* proj = nullptr, int ldp = 0);
int launch_ssd_prompt(const SsdGeom& g, const SsdIn& in, const AttnSeg* segs_dev, const AttnSeg* segs_host, int nseg, float* records, int max_chunks,
                      float* y, int ldy, bool f32, hipStream_t s);
// out [rows, ldo] compute type = (y silu(z)), every one of `parts` equal parts of the n columns over its root mean square, times w [n]
int launch_gated_norm(const float* y, int ldy, const float* z, int ldz, const float* w, int n, int parts, float eps, int rows, void* out, int ldo, bool f32,
                      hipStream_t s);

}  // namespace mi
