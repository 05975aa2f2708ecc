/* mi355x_vllm.h — C ABI of libmi355x_vllm.so
 *
 * The inner drop-in boundary of the MI355X vLLM plugin: everything the reference
 * (vllm-project/vllm-neuron @ 2025-11-21) obtains from the third-party NxDI model
 * object is obtained from this library instead.  Plain pointers and sizes only, no
 * torch / C++ types.  All calls arrive on ONE host thread (vLLM's "uni" executor,
 * reference platform.py:120-121,166-167); a context is not thread-safe.
 *
 * Every function returns 0 on success and a negative MI_E* code on failure;
 * mi_last_error() then describes the failure (the Python mirror raises it as
 * RuntimeError / ValueError exactly where the reference raises).
 *
 * Reference interface each entry point replaces (paths relative to /root/reference):
 *   mi_ctx_create      NxDI model-class ctor + neuron_config
 *                      vllm_neuron/worker/neuronx_distributed_model_loader.py:216-218,236
 *                      (fields: _get_default_neuron_config :725-793, overrides :870-900)
 *   mi_load_weight     checkpoint load + save_quantized_state_dict      loader.py:234-241
 *   mi_init_synthetic_weights   (bench only: no checkpoints exist offline)
 *   mi_finalize        model.compile() + model.load()                    loader.py:240-241
 *   mi_forward         NxDI model __call__ + logits[:, -1, :]            loader.py:339-363
 *   mi_kv_stats        torch.classes.neuron.Runtime().get_vnc_memory_stats()
 *                      vllm_neuron/worker/neuron_worker.py:51-63
 *   mi_tp_*            NxDI tp_degree collectives                        loader.py:752-753
 *   mi_op_*            (no reference counterpart: per-kernel entry points for the
 *                      parity tests and micro-benchmarks; device pointers)
 */
#ifndef MI355X_VLLM_H
#define MI355X_VLLM_H

#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

#define MI_OK 0
#define MI_EINVAL (-1)   /* bad argument / unsupported shape            */
#define MI_EHIP (-2)     /* HIP runtime error (message has the string) */
#define MI_ESTATE (-3)   /* call order violated (e.g. forward before finalize) */
#define MI_ENOMEM (-4)
#define MI_ECOMM (-5)    /* RCCL error */

/* element types for host/device tensors crossing the ABI */
enum { MI_F32 = 0, MI_BF16 = 1, MI_F8E4M3 = 2, MI_I8 = 3, MI_I64 = 4, MI_I32 = 5 };
/* weight storage dtypes ("quantization_dtype", loader.py:895-896) */
enum { MI_W_BF16 = 0, MI_W_F8E4M3 = 1, MI_W_INT8 = 2 };
/* "quantization_type" (loader.py:892-894) */
enum { MI_Q_PER_TENSOR_SYMMETRIC = 0, MI_Q_PER_CHANNEL_SYMMETRIC = 1 };
enum { MI_ROPE_DEFAULT = 0, MI_ROPE_LLAMA3 = 1 };

typedef struct mi_ctx mi_ctx;

typedef struct mi_model_config {
  /* decoder geometry (HF config; loader.py:612-631 derives nkv / head_dim the same way) */
  int32_t num_layers, hidden_size, num_heads, num_kv_heads, head_dim;
  int32_t intermediate_size, vocab_size;
  float rms_norm_eps;
  float rope_theta;
  int32_t rope_type; /* MI_ROPE_* */
  float rope_factor, rope_low_freq_factor, rope_high_freq_factor;
  int32_t rope_original_max_position;
  int32_t qkv_bias;            /* Qwen2 */
  int32_t tie_word_embeddings; /* lm_head shares embed_tokens */
  /* KV pool ("pa_num_blocks" incl. the null block 0, "pa_block_size": loader.py:741-745,775-778) */
  int32_t num_blocks, block_size;
  int32_t max_num_seqs;  /* "batch_size"  loader.py:738,756 */
  int32_t max_model_len; /* "seq_len"     loader.py:760-761 */
  /* "context_encoding_buckets" (README.md:80); 0 entries = one bucket of max_model_len */
  int32_t num_ctx_buckets;
  int32_t ctx_buckets[8];
  /* quantization keys (loader.py:886-898) */
  int32_t weight_dtype; /* MI_W_* ; MI_W_BF16 = not quantized */
  int32_t quant_type;   /* MI_Q_* */
  int32_t quantize_lm_head; /* 0 = "lm_head" listed in modules_to_not_convert */
  /* tensor parallelism ("tp_degree" loader.py:752-753): one process per GPU */
  int32_t tp_degree, tp_rank;
  int32_t device_id;
  int32_t use_graphs; /* capture token-generation steps into hipGraphs */
  /* Context-encoding GEMMs (rows > 16) on FP8 weights take per-token dynamically quantized FP8
   * activations and run on the MX-scaled MFMA at twice the bf16 rate; token generation (HBM-bound)
   * keeps bf16 activations.  0 = weight-only everywhere. */
  int32_t prefill_fp8_activations;
  /* Tensor parallelism inside ONE process, the reference's process model (a single worker drives
   * every core: platform.py:166-167, neuron_worker.py:106-121): tp_rank = MI_TP_ALL_RANKS makes the
   * context a group of tp_degree rank shards, rank r on GPU tp_device_ids[r] with a host thread of
   * its own; every entry point below fans out and rank 0's result is returned.  All ids equal =
   * every shard on one GPU (the single-GPU tests).  tp_transport picks the exchange between the
   * shards: the library's own all-reduce over peer-mapped memory (xGMI), or RCCL. */
  int32_t tp_device_ids[16];
  int32_t tp_transport; /* MI_TP_TRANSPORT_* */
} mi_model_config;
#define MI_TP_ALL_RANKS (-1)
enum { MI_TP_TRANSPORT_P2P = 0, MI_TP_TRANSPORT_RCCL = 1 };

/* ---- layer-stack decoders: a decoder given layer by layer, every size and constant a parameter ----
 * (Vimesun, Rapodra, Bokulorn and Nusovik are such designs; the worker's model registry fills this from their config.json.)
 *     x = embed_scale embed[token] (+ pos[position])          fp32 residual stream
 *         pos_base > 0: + sin / cos of position * pos_base^(-2 i / width) at elements 2 i / 2 i + 1
 *     block MI_BLOCK_PARALLEL:  x <- x + residual_mult (mixer(norm1 x) + ff(norm2 x))     both of the same x
 *     block MI_BLOCK_SANDWICH:  x <- x + norm1b(mixer(C1(norm1 x))); x <- x + norm2b(ff(C2(norm2 x)))
 *             C(h) = h + causal convolution of h over time, conv_taps taps per channel; the last conv_taps - 1 inputs h
 *             are part of a sequence's state
 *     block MI_BLOCK_ONE_NORM:  h = norm1 x;  x <- x + mixer(h) + ff(h)
 *     block MI_BLOCK_POST_NORM: x <- x + norm1(mixer(x));  x <- x + norm2(ff(x))
 *     norms:  norm_groups = 0: layer norm with weight and bias; else RMS norm of norm_groups equal parts, each over its
 *             own sqrt(mean square + norm_eps), times a weight (norm_offset = 1: times 1 + weight, also the final norm)
 *     loop:   layers loop_start .. loop_stop - 1 run loop_times times in a row with the same weights, each pass with a
 *             KV pool of its own; ahead of a pass's first layer  x <- W_in [x ; embedding output]
 *     weights_of >= 0: the layer has no tensors of its own, it runs that other layer's with a cache and state of its own
 *     logits = logit_scale head final_norm(x); logit_softcap > 0: softcap tanh(logits / softcap)
 * Mixers: MI_MIX_ATTENTION, grouped heads with K / V pools; MI_MIX_LATENT, per head k = W_uk c, v = W_uv c of a cached latent
 *     c = RMSnorm(W_dkv h) [kv_rank]; kv_from >= 0: the latents of that earlier layer instead of own ones.
 *     q_rank > 0: queries q = W_uq RMSnorm(W_dq h) [q_rank] instead of W_q h.  rot_dim > 0: a head's query has rot_dim more
 *     elements behind its qk_dim, W_dkv that many more rows (one more key part for all heads, not normed); both parts rotate over their
 *     first rot_dims elements, pair (i, i + rot_dims / 2) by position * rot_base^(-2 i / rot_dims), and their product joins the
 *     score.  out_gate: MI_GATE_HEAD, a head's output times sigmoid(W_g h)_head; MI_GATE_ELEMENT, every element of the heads'.
 *   MI_MIX_DELTA, a gated delta rule with one decay per head and key channel, num_kv_heads query / key heads shared by
 *     num_heads heads with a state S [qk_dim, v_dim] each: q, k, v = W h through a causal convolution of conv_taps taps and
 *     silu; q and k over sqrt(sum of squares + 1e-6), q times qk_dim^-1/2; beta = sigmoid(W_b h); g = exp(-exp(A_log)
 *     softplus(W_a2 W_a1 h + dt_bias)) (decay_rank rows in W_a1);  S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q;
 *     output W_o (RMSnorm(o) sigmoid(W_g2 W_g1 h)) (gate_rank rows in W_g1).  Everything fp32 but the projections.  S and the
 *     last inputs of the convolution live in a state slot per sequence (seq_ids of the model calls).
 *   MI_MIX_ATTENTION in post-norm blocks: qk_norm, q and k heads over sqrt(mean square + eps) times a weight per element; qk_bias, biases of
 *     their projections; keys_as_values, no W_v: a value is the key as projected (ahead of its norm); chunk > 0: a query sees keys of its own
 *     chunk of that many positions; distance_bias MI_BIAS_TABLE, rel[bucket(i - j), head] joins the score, bucket(n) = n below rel_rows / 2, else
 *     min(rel_rows - 1, rel_rows / 2 + floor(ln(n / (rel_rows / 2)) / ln(rel_far / (rel_rows / 2)) (rel_rows - rel_rows / 2)));
 *     softmax_sink MI_SINK_LEARNED, exp(sink[head]) in the denominator; out_gate MI_GATE_HEAD.  beside_kind MI_MIX_SSD: a second mixer of the same x
 *     beside it, the result mix_mult attention + beside_mult second.
 *   MI_MIX_SSD (Mamba-2), ssm_heads heads of ssm_dim with a state of ssm_state x ssm_dim each, B and C shared by ssm_groups groups of heads: W_in x =
 *     [z | x | B | C | dt]; x, B, C through a causal convolution of conv_taps taps with bias and silu; dt = softplus(dt + dt_bias);
 *     S <- exp(-exp(A_log) dt) S + dt B x^T;  y = S^T C + D x;  y silu(z) in ssm_parts equal parts over their root mean square, times norm; W_o.
 *   MI_MIX_SCAN (Mamba), ssm_inner channels with ssm_state states each: W_in x = [x | z]; x through the convolution and silu; W_x x = [low, dt_rank | B |
 *     C]; dt = softplus(W_dt low + bias) per channel; S <- exp(-exp(A_log) dt) S + dt x B;  y = sum S C + D x;  W_o (y silu(z)).
 *     States and convolution inputs of both live in the sequence's slot, in fp32.
 * Feed-forwards: MI_FF_RELU2 down(max(up x, 0)^2); MI_FF_GLU down(act(gate x, up x)); MI_FF_MOE the softmax-weighted sum of the
 *     experts_top experts with the largest router logits (W_router x + b), each down(act(gate x, up x)).
 *     router_score MI_ROUTE_SIGMOID: s = sigmoid(W_router x); choice scores s + correction; the experts lie in router_groups equal
 *     groups, of which the router_keep with the largest sum of their two best choice scores are eligible; weights s over their sum.
 * Gated activations: MI_ACT_SILU g sigmoid(g) u; MI_ACT_SWISH_CLIP, g = min(g, limit), u within +-limit: g sigmoid(alpha g) (u + 1).
 * MI_ACT_RELU2 (experts): no gate, max(up x, 0)^2.
 * Built: parallel blocks of MI_MIX_ATTENTION with layer norms, sandwich blocks of MI_MIX_LATENT with RMS norms and no loop,
 * one-norm blocks of MI_MIX_LATENT (every earlier token in sight) and MI_MIX_DELTA with RMS norms, experts or no feed-forward and no loop,
 * post-norm blocks of MI_MIX_ATTENTION (alone or beside MI_MIX_SSD) and MI_MIX_SCAN with RMS norms, MI_FF_RELU2 or no feed-forward and no loop.
 * Tensor names ("l<i>." = layer i): embed, pos, loop.in, l<i>.norm1(.b), l<i>.norm2(.b), l<i>.mix.{q,k,v,o},
 * l<i>.mlp.{up,down}, final.norm(.b), head; sandwich blocks: l<i>.norm1, .norm1b, .norm2, .norm2b, .canon1, .canon2
 * [width, taps], l<i>.mix.{q,dkv,dkv.norm,uk,uv,o}, l<i>.mlp.{gate,up,down}, l<i>.mlp.router(.b), l<i>.mlp.e<n>.{gate,up,down};
 * one-norm blocks: l<i>.norm1, l<i>.mix.{dq,dq.norm,uq | q}, l<i>.mix.{dkv,dkv.norm,uk,uv,g,o}, or l<i>.mix.{q,k,v,q.conv,k.conv,v.conv,
 * b,A_log,a1,a2,dt_bias,g1,g2,norm,o}, l<i>.mlp.router, .correction (or .router.b), l<i>.mlp.e<n>.{gate,up,down};
 * post-norm blocks: l<i>.norm1, .norm2, l<i>.mlp.{up,down}, l<i>.mix.{q,k,v,q.b,k.b,q.norm,k.norm,rel,sink,g,o} (those the layer has; beside a second
 * mixer l<i>.mix.left.*, and l<i>.mix.right.{in,conv,conv.b,dt_bias,A_log,D,norm,o}), or l<i>.mix.{in,conv,conv.b,x,dt,dt.b,A_log,D,o}. */
enum { MI_BLOCK_PARALLEL = 0, MI_BLOCK_SANDWICH = 1, MI_BLOCK_ONE_NORM = 2, MI_BLOCK_POST_NORM = 3 };
enum { MI_MIX_ATTENTION = 0, MI_MIX_LATENT = 1, MI_MIX_DELTA = 2, MI_MIX_SCAN = 3, MI_MIX_SSD = 4 };
enum { MI_BIAS_NONE = 0, MI_BIAS_SLOPE = 1, MI_BIAS_TABLE = 2 };
enum { MI_SINK_NONE = 0, MI_SINK_ONE = 1, MI_SINK_LEARNED = 2 };
enum { MI_FF_NONE = 0, MI_FF_RELU2 = 1, MI_FF_GLU = 2, MI_FF_MOE = 3 };
enum { MI_ACT_SILU = 0, MI_ACT_SWISH_CLIP = 1, MI_ACT_RELU2 = 2 };
enum { MI_GATE_NONE = 0, MI_GATE_HEAD = 1, MI_GATE_ELEMENT = 2 };
enum { MI_ROUTE_SOFTMAX = 0, MI_ROUTE_SIGMOID = 1 };
typedef struct mi_layer_spec {
  int32_t num_heads, num_kv_heads, qk_dim, v_dim;
  int32_t window;         /* a query sees keys with 0 <= i - j < window; 0 = every earlier token */
  float scale;            /* of q . k */
  int32_t qk_unit_norm;   /* q and k heads divided by sqrt(mean square + norm_eps) */
  int32_t distance_bias;  /* MI_BIAS_*; SLOPE: 2^(-8 (h + 1) / num_heads) (i - j) taken off the score of head h */
  int32_t softmax_sink;   /* MI_SINK_*; ONE: one added to the softmax denominator */
  int32_t ff_kind, ff_size;   /* ff_size: of one expert where there are experts */
  int32_t mixer_kind;
  int32_t kv_rank, kv_from;   /* MI_MIX_LATENT; kv_from = -1: own latents */
  int32_t ff_act;             /* MI_ACT_*, gated feed-forwards and experts */
  float ff_limit, ff_alpha;   /* MI_ACT_SWISH_CLIP */
  int32_t experts, experts_top;
  int32_t router_score, router_groups, router_keep;   /* MI_ROUTE_SIGMOID: groups >= 1, 1 <= keep <= groups */
  int32_t weights_of;         /* -1: tensors of its own (one-norm blocks) */
  int32_t q_rank;             /* MI_MIX_LATENT: 0 = W_q h */
  int32_t rot_dim, rot_dims;
  float rot_base;
  int32_t out_gate;           /* MI_GATE_* */
  int32_t conv_taps, decay_rank, gate_rank;   /* MI_MIX_DELTA (conv_taps: MI_MIX_SCAN and MI_MIX_SSD too) */
  int32_t qk_norm, qk_bias, keys_as_values, chunk, rel_rows;   /* post-norm blocks, MI_MIX_ATTENTION */
  float rel_far;
  int32_t beside_kind;        /* 0 or MI_MIX_SSD */
  float mix_mult, beside_mult;
  int32_t ssm_state, ssm_heads, ssm_dim, ssm_groups, ssm_parts;   /* MI_MIX_SSD (ssm_state: MI_MIX_SCAN too) */
  int32_t ssm_inner, dt_rank;                                      /* MI_MIX_SCAN */
} mi_layer_spec;
typedef struct mi_stack_config {
  int32_t num_layers;
  const mi_layer_spec* layers;
  int32_t width, vocab_size, max_positions;    /* max_positions = 0: no learned positions, no bound on the sequence */
  float norm_eps, residual_mult;
  int32_t loop_start, loop_stop, loop_times;   /* loop_times = 0: no loop (and no loop.in) */
  int32_t compute_dtype;   /* MI_BF16: bf16 matrix products and KV; MI_F32: everything in fp32 (plain kernels: for checking) */
  int32_t block_kind, norm_groups;
  int32_t conv_taps;       /* sandwich blocks: 1 .. 16 */
  float logit_softcap;     /* 0 = none */
  int32_t state_lookahead; /* sandwich blocks: a step may write this many positions behind the last accepted one (speculation: k - 1) */
  float embed_scale, norm_offset;
  float pos_base, logit_scale;   /* post-norm blocks: pos_base 0 = no sinusoidal positions; logit_scale 1 elsewhere */
} mi_stack_config;

const char* mi_last_error(void);
int mi_version(void);   /* 8 = this header (+ post-norm blocks, chunks / distance tables / learned sinks, selective scan and state-space duality); 7 (+ one-norm blocks, recurrent mixers and their state slots: seq_ids of mi_forward_chunked / mi_forward_rows); 6 (+ sandwich blocks, latent attention, experts in mi_layer_spec / mi_stack_config and their mi_op_*); 5 (+ mi_ctx_create_stack, mi_forward_rows, mi_layer_residuals, mi_op_* of the stack kernels); 4 (+ mi_tp_plan, mi_tp_info); 3 lacked them; 2 lacked tp_device_ids / tp_transport / MI_TP_ALL_RANKS; 1 lacked mi_forward_tokens, mi_op_sample, mi_tp_init_transport */

int mi_ctx_create(const mi_model_config* cfg, mi_ctx** out);
/* The same context around a layer stack.  Of cfg only the serving fields are read (pool, batch, buckets, device, graphs);
 * geometry comes from `stack` (copied).  One GPU, unquantized weights. */
int mi_ctx_create_stack(const mi_model_config* cfg, const mi_stack_config* stack, mi_ctx** out);
int mi_ctx_destroy(mi_ctx* ctx);

/* One HF-named tensor ("model.layers.3.self_attn.q_proj.weight", "lm_head.weight", ...),
 * row-major on the host, dtype MI_F32 or MI_BF16, FULL (unsharded) shape.  The library
 * slices its TP shard, quantizes (weight_dtype / quant_type) and re-tiles for the kernels. */
int mi_load_weight(mi_ctx* ctx, const char* name, const void* host, int32_t dtype,
                   const int64_t* shape, int32_t ndim);
/* Bench/smoke only: N(0, std) matrices from a counter-based RNG in LOGICAL coordinates
 * (identical values whatever the sharding); norm gains 1. */
int mi_init_synthetic_weights(mi_ctx* ctx, uint64_t seed, float std);
/* Weight artifacts -- the counterpart of the reference's compiled-artifact directory
 * (loader.py:160-226, keyed by a config hash there; the Python mirror keys the directory the same
 * way).  mi_save_weights writes this context's device images (quantized, tiled, sharded: what
 * mi_load_weight made) to <dir>/rank<r>_of<T>.miw; mi_load_weights_file streams such a file back
 * into HBM in place of every mi_load_weight call, and returns MI_EINVAL when the file is missing
 * or was made for another model, quantization, sharding or tile format (the caller then loads the
 * checkpoint the long way and saves again).  Also the home of quantized_checkpoints_path
 * (loader.py:888-891). */
int mi_save_weights(mi_ctx* ctx, const char* dir);
int mi_load_weights_file(mi_ctx* ctx, const char* dir);

/* Re-size the KV pool before mi_finalize: vLLM decides the block count after the weights
 * are resident (worker.determine_available_memory -> KVCacheConfig.num_blocks; the reference's
 * NxDI takes it at compile time as pa_num_blocks, loader.py:775-776). */
int mi_set_num_blocks(mi_ctx* ctx, int32_t num_blocks);
int mi_finalize(mi_ctx* ctx);

/* One model call.  Host arrays, caller-owned, int64 like the reference's CPU tensors:
 *   input_ids, position_ids [B, S]; seq_ids [B]; block_table [B, MB];
 *   slot_mapping [B, SM]; full_context_lens, computed_context_lens [B];
 *   logits_out [B, vocab_size] fp32 (last-token logits, loader.py:363).
 * seq_ids: models with recurrent mixers keep a sequence's state in slot seq_ids[b] (0 .. max_num_seqs - 1, no two rows
 * alike; a sequence whose first token is in the call starts from a zero state, whatever the slot held); otherwise not read.
 * S == 1 -> token generation;  S > 1 -> context encoding of tokens
 * computed..full-1 of each row (the FULL prompt is passed, runner.py:721-726,754).
 * Slot -1 = no write; block-table entries past full_context_lens are never read. */
int mi_forward(mi_ctx* ctx, int32_t B, int32_t S, const int64_t* input_ids,
               const int64_t* position_ids, const int64_t* seq_ids, const int64_t* block_table,
               int32_t MB, const int64_t* slot_mapping, int32_t SM,
               const int64_t* full_context_lens, const int64_t* computed_context_lens,
               float* logits_out);

/* The same call with on-device sampling (the reference's on_device_sampling_config path: the model
 * returns sampled ids instead of logits, loader.py:352-356, 367-375).  sampling_params: [B, 3] fp32
 * rows (top_k, top_p, temperature) as the reference packs them (runner.py:1106-1140; greedy
 * requests arrive as top_k = 1), or NULL for all-greedy.  top_k is capped at 256.  top_k == 1 is
 * argmax with the lowest index on ties (== torch.argmax on the logits mi_forward would return);
 * otherwise the id is drawn from the temperature-scaled softmax over the top_k logits cut to the
 * top_p nucleus, with u = splitmix64(seed, row) -- a pure function of (logits, params, seed, row),
 * restated in oracle/sampling.py.  tokens_out [B] int64. */
int mi_forward_tokens(mi_ctx* ctx, int32_t B, int32_t S, const int64_t* input_ids,
                      const int64_t* position_ids, const int64_t* seq_ids, const int64_t* block_table,
                      int32_t MB, const int64_t* slot_mapping, int32_t SM,
                      const int64_t* full_context_lens, const int64_t* computed_context_lens,
                      const float* sampling_params, uint64_t seed, int64_t* tokens_out);

/* Chunked prefill (the reference's path under vLLM's native scheduler: runner.py:938-1051,
 * loader.py:357-361): ONE ragged batch of `total` tokens = the concatenated chunks of n_req
 * requests -- request i contributes tokens computed_context_lens[i] .. full_context_lens[i] - 1
 * (a prompt chunk, or the single next token of a request that is generating).  input_ids,
 * position_ids, slot_mapping: [total] in request order; block_table [n_req, MB].  Every token's
 * K/V is written through slot_mapping, each request attends to its own blocks, the projections run
 * once over all rows.  logits_out [n_req, vocab_size] = logits of each request's LAST scheduled
 * token (the caller ignores rows whose prompt is not complete: prefill_completion_state);
 * or tokens_out [n_req] with sampling_params as in mi_forward_tokens.  total may not exceed the
 * largest context-encoding bucket (pass max_num_batched_tokens as a bucket).  seq_ids [n_req]: as mi_forward; may be NULL for
 * models without recurrent mixers. */
int mi_forward_chunked(mi_ctx* ctx, int32_t n_req, int32_t total, const int64_t* input_ids,
                       const int64_t* position_ids, const int64_t* seq_ids, const int64_t* slot_mapping, const int64_t* block_table,
                       int32_t MB, const int64_t* full_context_lens, const int64_t* computed_context_lens,
                       float* logits_out, const float* sampling_params, uint64_t seed, int64_t* tokens_out);

/* The same ragged batch with the logits of chosen places: rows [n_rows] = indices into the token batch (any order, any
 * number, none at all); logits_out [n_rows, vocab_size] in that order. */
int mi_forward_rows(mi_ctx* ctx, int32_t n_req, int32_t total, const int64_t* input_ids, const int64_t* position_ids,
                    const int64_t* seq_ids, const int64_t* slot_mapping, const int64_t* block_table, int32_t MB, const int64_t* full_context_lens,
                    const int64_t* computed_context_lens, int32_t n_rows, const int64_t* rows, float* logits_out);

/* Layer-stack contexts: keep a copy of the residual stream behind every layer run of the following ragged batches
 * (on != 0).  mi_layer_residuals_read copies it out: [layer runs][rows of the last batch][width] fp32.  For checking. */
int mi_layer_residuals(mi_ctx* ctx, int32_t on);
int mi_layer_residuals_read(mi_ctx* ctx, int32_t rows, float* out);

/* Fused speculation (the reference reaches it through NxDI's fused draft + target graph:
 * loader.py:349-355; output contract re-masked by _remask_fused_spec_output, loader.py:308-333; slots
 * of the speculated positions, runner.py:825-830).  One call = `k - 1` greedy token-generation steps of
 * the DRAFT context chained on the device, ONE token-generation pass of the TARGET context over the
 * B * k candidate rows, greedy acceptance.  input_ids / position_ids [B]: the last accepted token
 * of every sequence and its position; block_table [B, MB] must back positions up to
 * position + k - 1 (clipped at max_model_len) in BOTH contexts (same block ids, separate pools).
 * accepted_out [B, k]: the 1..k tokens generated this step, 0-padded (NxDI's
 * accepted_tokens_with_padding); next_pos_out [B] = position + number of tokens generated.  The
 * tokens are exactly those the target alone would generate greedily, one per step.
 * draft_catchup_ids [B] or NULL: the draft runs k - 1 steps, so after a step that generated k tokens
 * the token at position - 1 has not been through the draft; pass it here (-1 = nothing to catch up)
 * and the draft's first step takes it as an extra row.  Leaving it out never changes the output,
 * only the quality of the draft's proposals.  Needs
 * target max_num_seqs >= B * k, draft max_num_seqs >= B + catch-up rows (2 B), and both contexts created with the same
 * device (the target's rank 0 GPU when the target is an in-process tensor-parallel group; the draft is never
 * sharded), block_size, num_blocks, vocab_size and max_model_len.  From the first call on the
 * draft context runs on the target's stream: destroy the draft before the target. */
int mi_forward_spec(mi_ctx* target, mi_ctx* draft, int32_t B, int32_t k, const int64_t* input_ids,
                    const int64_t* position_ids, const int64_t* block_table, int32_t MB,
                    const int64_t* draft_catchup_ids, int64_t* accepted_out, int64_t* next_pos_out);

/* Replay the LAST token-generation call `steps` times with its inputs left resident in HBM
 * (no host round trip in between) and return the elapsed time measured with HIP events on the
 * context's stream.  For benchmarking the hot path itself: mi_forward adds one small H2D copy
 * and a [B, V] fp32 D2H copy per step. */
int mi_replay_decode(mi_ctx* ctx, int32_t steps, float* elapsed_ms);

/* The same replay with only the kernel classes of `class_mask` (bit MI_K_*) launched: e.g.
 * 1 << MI_K_GEMV replays the weight-streaming launches of a step back to back, in a graph of their
 * own -- elapsed / (steps x launches) is the average launch duration of that kernel, boundary
 * included, which is how rocprofv3's kernel trace counts it.  Timing only: the step's results are
 * not meaningful.  Single-GPU contexts. */
int mi_replay_decode_classes(mi_ctx* ctx, int32_t steps, uint32_t class_mask, float* elapsed_ms);

typedef struct mi_kv_stats_t {
  int64_t kv_bytes, weight_bytes;
  int64_t workspace_bytes;   /* before mi_finalize: what it will allocate besides the KV pool; after: what it did */
  int64_t device_free_bytes, device_total_bytes;
  int32_t num_blocks, block_size, num_kv_heads_local, head_dim, num_layers;
  /* token-generation block tables are device-resident: rows re-sent because the caller's row
   * changed (new request, block appended) vs rows found unchanged since the previous step */
  int64_t block_table_rows_sent, block_table_rows_kept;
} mi_kv_stats_t;
int mi_kv_stats(mi_ctx* ctx, mi_kv_stats_t* out);
/* Bytes ONE block costs on a GPU across all layers (K and V, this rank's kv heads): vLLM sizes the
 * cache from a single-layer spec (runner.get_kv_cache_spec), the pool holds num_layers of them. */
int64_t mi_kv_bytes_per_block(mi_ctx* ctx);

/* The pinned host buffer [max_num_seqs][vocab_size] fp32 the logits land in.  Passing it as
 * mi_forward's logits_out skips the final host copy: the caller reads the logits in place, valid
 * until the next call on this context.  NULL for tensor-parallel contexts (their shards fill the
 * caller's rows directly) and before mi_finalize. */
float* mi_logits_buffer(mi_ctx* ctx);

/* hipStream_t the context launches on (for event timing by the caller). */
void* mi_stream(mi_ctx* ctx);

/* Per-kernel-class HIP-event timing of the following mi_forward calls (eager launches,
 * no graph).  mi_profile_read returns, per class, launches and summed milliseconds. */
enum { MI_K_GEMV = 0, MI_K_GEMM = 1, MI_K_ATTN_DECODE = 2, MI_K_ATTN_PREFILL = 3, MI_K_OTHER = 4,
       MI_K_COMM = 5, MI_K_NUM = 6 };
int mi_profile_enable(mi_ctx* ctx, int32_t on);
int mi_profile_read(mi_ctx* ctx, int32_t* launches /*[MI_K_NUM]*/, float* ms /*[MI_K_NUM]*/,
                    double* gemv_weight_bytes);

/* Tensor parallel bring-up: rank 0 calls mi_tp_unique_id, the host layer broadcasts the
 * 128 bytes, every rank calls mi_tp_init (ncclCommInitRank on the context's device). */
int mi_tp_unique_id(void* out128);
int mi_tp_init(mi_ctx* ctx, const void* id128);

/* The same, with the two collectives supplied by the caller instead of RCCL (a custom xGMI
 * transport; the single-GPU loopback that tests/test_tp_loopback_gpu.py uses to run every
 * rank's shard on one device).  all_reduce: in-place fp32 sum of buf[count] over the ranks;
 * all_gather: recv[rank * count .. ] = rank's send[count].  Both are called from mi_forward on
 * the calling thread, must be ordered after the work already queued on `stream` and must leave
 * their result visible to work queued on it afterwards; return 0 on success.  Decode steps are
 * launched eagerly (no graph capture) on a context with collectives. */
typedef int (*mi_allreduce_fn)(void* user, void* buf, size_t count, void* stream);
typedef int (*mi_allgather_fn)(void* user, const void* send, void* recv, size_t count, void* stream);
int mi_tp_init_transport(mi_ctx* ctx, mi_allreduce_fn all_reduce, mi_allgather_fn all_gather, void* user);

/* The sharding plan of rank `rank` of cfg->tp_degree: which slices of the UNSHARDED checkpoint tensors the rank holds
 * (tp_degree = tensor_parallel_size, loader.py:752-753; head counts that do not divide are allowed, the reference skips
 * vLLM's divisibility check at platform.py:58-64).  Host only: no device, no context -- the same function mi_ctx_create
 * runs.  q heads [q_head0, q_head0 + q_heads_real) are real; the rank computes q_heads_local >= q_heads_real heads, the
 * surplus being zero-weight padding heads (q rows, q bias and o_proj columns zero).  kv heads [kv_head0, + kv_heads_local);
 * gate / up rows and down_proj columns [inter0, + inter_local); lm_head rows (logit columns) [vocab0, + vocab_local). */
typedef struct mi_tp_plan {
  int32_t q_head0, q_heads_real, q_heads_local;
  int32_t kv_head0, kv_heads_local;
  int32_t inter0, inter_local;
  int32_t vocab0, vocab_local;
} mi_tp_plan_t;
int mi_tp_plan(const mi_model_config* cfg, int32_t rank, mi_tp_plan_t* out);

/* What an in-process tensor-parallel context (tp_rank = MI_TP_ALL_RANKS, finalized) actually runs on -- so that a benchmark
 * record can tell "N ranks over peer memory, in hipGraphs" from "fell back to RCCL, eager". */
typedef struct mi_tp_info {
  int32_t tp_degree;
  int32_t transport;       /* MI_TP_TRANSPORT_* in use after the self-test */
  int32_t selftest;        /* 1: passed on the transport in use; -1: the peer-memory exchange failed it (transport is RCCL now); 0: not run */
  int32_t graphs;          /* 1: token-generation steps, exchange kernels included, replay from a hipGraph per shard */
  int32_t mode;            /* 0: one GPU per rank; 1: every shard on one GPU in lockstep (one stream, host barriers between the
                              exchange kernels); 2: every shard on one GPU, one stream per shard, the kernels wait on device flags */
  int32_t timeout_ms;      /* bound of a flag wait; on expiry the output is poisoned with NaN and MI_ECOMM is reported */
  int32_t device_ids[16];
  int32_t peer_access[16]; /* bit p of word r: rank r's device maps rank p's memory */
} mi_tp_info_t;
int mi_tp_info(mi_ctx* ctx, mi_tp_info_t* out);

/* ---- per-kernel entry points (device pointers; stream may be NULL) -------------------- */

/* The exchange step of an in-process tensor-parallel context (tp_rank = MI_TP_ALL_RANKS, finalized) on
 * caller-supplied data: bufs[r] = rank r's fp32 [count] on rank r's GPU, count % 8 == 0 and at most
 * max rows x hidden_size.  In place: every rank ends with the fp32 sum over ranks, taken in rank
 * order (bit-identical on every rank); messages of 512 KiB (as bf16) and more -- context encoding --
 * travel as bf16, go reduce-scatter + all-gather and round the sum to bf16 once more.  Returns
 * after the exchange has completed on every rank. */
int mi_op_tp_all_reduce(mi_ctx* ctx, float* const* bufs, size_t count);

/* The sampler of mi_forward_tokens on caller-supplied logits: logits [B, V] fp32, sampling_params
 * [B, 3] fp32 (top_k, top_p, temperature) or NULL = greedy, tokens_out [B] int32 -- all device. */
int mi_op_sample(const float* logits, int32_t B, int32_t V, const float* sampling_params, uint64_t seed,
                 int32_t* tokens_out, void* stream);
/* The same with the engine's scratch buffer (mi_op_sample_scratch_bytes(B) bytes of device memory): the form
 * mi_forward_tokens runs -- all-greedy batches split the argmax over the chip, top-k / top-p rows have the
 * vocabulary pre-selected by 32 work-groups per row.  Same ids as mi_op_sample. */
size_t mi_op_sample_scratch_bytes(int32_t B);
int mi_op_sample_ws(const float* logits, int32_t B, int32_t V, const float* sampling_params, uint64_t seed,
                    int32_t* tokens_out, void* scratch, size_t scratch_bytes, void* stream);


/* Quantize + re-tile a row-major fp32 [N, K] device matrix.  scale_out [N] fp32.
 * tiled_out: N*K bytes (fp8/int8) or 2*N*K (bf16), kernel-native 16-row tiles. */
int mi_op_quantize_weight(const float* w, int32_t N, int32_t K, int32_t weight_dtype,
                          int32_t quant_type, void* tiled_out, float* scale_out, void* stream);
/* Inverse of the tiling for inspection: q_out row-major [N, K] (1 or 2 bytes/elem). */
int mi_op_untile_weight(const void* tiled, int32_t N, int32_t K, int32_t weight_dtype,
                        void* q_out, void* stream);
/* y[M, N] fp32 = (x[M, K] bf16 . Wq^T) * scale (+ bias).  M <= 16: weight-streaming GEMV;
 * else MFMA GEMM.  force_path: 0 auto, 1 GEMV, 2 GEMM (picked by size), 3 the wide-N LDS-DMA GEMM (1-byte weights),
 * 4 / 5 that GEMM with K split over 2 / 4 slices at 128-token blocks, 6 / 7 at 256-token blocks (K / 64 a multiple of the slices). */
int mi_op_qlinear(const void* x_bf16, int32_t M, const void* w_tiled, const float* scale,
                  const float* bias, int32_t N, int32_t K, int32_t weight_dtype, float* y,
                  int32_t force_path, void* stream);
/* FP8-activation form (M > 16, fp8 weights, K % 128 == 0): x is quantized per token to e4m3
 * (scale amax/448) and multiplied on v_mfma_scale_f32_16x16x128_f8f6f4. */
int mi_op_qlinear_a8(const void* x_bf16, int32_t M, const void* w_tiled, const float* scale,
                     const float* bias, int32_t N, int32_t K, float* y, void* stream);
/* y[T, H] bf16 = rmsnorm(x[T, H] fp32) * g */
int mi_op_rmsnorm(const float* x, const float* g, int32_t T, int32_t H, float eps, void* y_bf16,
                  void* stream);
/* Paged KV write.  k, v [T, nkv, hd] bf16; slots [T] (int64; -1 skips).
 * pool layout (library-native): [2][num_blocks][nkv][block_size][hd] bf16. */
int mi_op_kv_write(const void* k, const void* v, const int64_t* slots, int32_t T, int32_t nkv,
                   int32_t hd, void* pool, int32_t num_blocks, int32_t block_size, void* stream);
/* Token-generation attention.  q [B, nh, hd] bf16; block_table [B, MB] int32;
 * ctx_lens [B] int32; out [B, nh*hd] bf16.  scratch: >= mi_op_attn_scratch_bytes. */
int64_t mi_op_attn_scratch_bytes(int32_t B, int32_t nh, int32_t hd);
int mi_op_paged_attn_decode(const void* q, const void* pool, int32_t num_blocks,
                            int32_t block_size, const int32_t* block_table, int32_t MB,
                            const int32_t* ctx_lens, int32_t B, int32_t nh, int32_t nkv,
                            int32_t hd, void* out, void* scratch, void* stream);
/* Context-encoding attention for ONE sequence.  q [T, nh, hd] bf16 are the new tokens at
 * absolute positions q_pos0 .. q_pos0+T-1; keys 0 .. q_pos0+T-1 are read from the pool
 * through block_table [MB] int32 (the new tokens' K/V must already be written). */
int mi_op_paged_attn_prefill(const void* q, int32_t T, int32_t q_pos0, const void* pool,
                             int32_t num_blocks, int32_t block_size, const int32_t* block_table,
                             int32_t MB, int32_t nh, int32_t nkv, int32_t hd, void* out,
                             void* stream);

/* ---- kernels of the layer-stack decoders.  f32 != 0: activations / pools are fp32, else bf16 ----
 * y1 / y2 [T, ldy] = layer norm of x [T, ld] fp32 over its first D columns (w, b [ld] fp32, zero beyond D; y2 may be NULL) */
int mi_op_layernorm2(const float* x, int32_t T, int32_t D, int32_t ld, float eps, const float* w1, const float* b1, void* y1,
                     const float* w2, const float* b2, void* y2, int32_t ldy, int32_t f32, void* stream);
/* resid[t] (and x0[t], may be NULL) [T, ld] fp32 = table[ids[t]] + ptable[pos[t]], columns beyond D zero */
int mi_op_embed_pos(const int32_t* ids, const int32_t* pos, const void* table, const void* ptable, int32_t T, int32_t D, int32_t ld,
                    float* resid, float* x0, int32_t f32, void* stream);
/* qkv [T, ldq] fp32 -> q [T, H, pad16(dk)], K pool [blocks][G][block_size][pad16(dk)], V pool [..][pad16(dv)] at slots (-1: skip) */
int mi_op_qkv_scatter(const float* qkv, int32_t ldq, int32_t T, const mi_layer_spec* spec, float eps, const int32_t* slots,
                      int32_t block_size, void* q, void* kpool, void* vpool, int32_t f32, void* stream);
/* Windowed attention of a ragged batch over those pools.  segs_host [nseg][4] = (first row, rows, first position, block-table
 * row); pos [T]; ctx_lens [block-table rows] (keys incl. the row's own) for one-row segments.  slopes [H] or NULL.
 * path: 0 the model's choice, 1 the plain kernel.  out [T, H v_dim] (row stride ldo).  All device pointers but segs_host. */
int mi_op_window_attn(const mi_layer_spec* spec, const float* slopes, const void* q, const void* kpool, const void* vpool,
                      int32_t block_size, const int32_t* block_table, int32_t MB, const int32_t* pos, const int32_t* ctx_lens,
                      const int32_t* segs_host, int32_t nseg, int32_t T, int32_t max_ctx, void* out, int32_t ldo, int32_t f32,
                      int32_t path, void* stream);

/* ---- kernels of the sandwich blocks (device pointers but segs_host; segs_host [nseg][4] as above) ----
 * resid_out [T, ld] = resid_in + RMS-norm(w_post) of y (may be NULL: nothing added); y [T, ld] fp32, or with pair_w [T, top] the sum over
 * j of pair_w[t, j] y[t top + j].  Then, with w_pre, out [T, ldy] = RMS-norm(w_pre) of that row and, with conv_w [taps][ld] (row taps - 1
 * meets the token itself), h + its causal convolution.  ring [blocks][keep][ldy]: the convolution's state, position p of a block at row
 * (p % block_size) % keep, keep >= taps - 1 or block_size.  nseg = 0: token generation, row = block-table row. */
int mi_op_sandwich_rows(const float* resid_in, float* resid_out, const float* y, const float* pair_w, int32_t top, const float* w_post,
                        const float* w_pre, int32_t T, int32_t D, int32_t ld, int32_t groups, float eps, const float* conv_w, int32_t taps,
                        void* ring, int32_t keep, int32_t block_size, const int32_t* block_table, int32_t MB, const int32_t* pos,
                        const int32_t* slots, const int32_t* segs_host, int32_t nseg, void* out, int32_t ldy, int32_t f32, void* stream);
/* qd [T, ldq] fp32 = [q heads | W_dkv h] -> q [T, H, pad32(dk + rot_dim)]; with c_norm [kv_rank] the RMS-normed latent and the rotated
 * key part into pool [blocks][block_size][pad32(kv_rank) + pad32(rot_dim)] at slots (-1: skip).  rot [positions][rot_dims / 2][2]: cosines and
 * sines, pos [T]; both NULL without a rotated part */
int mi_op_latent_scatter(const float* qd, int32_t ldq, int32_t T, const mi_layer_spec* spec, const float* rot, const int32_t* pos, const float* c_norm,
                         float eps, const int32_t* slots, int32_t block_size, void* q, void* pool, int32_t f32, void* stream);
/* Gated delta rule of a ragged batch (spec: MI_MIX_DELTA).  proj [T, ldp] fp32: [q | k | v] at column 0, beta's projection at column beta; z
 * [T, ldz]: decays at column 0, output gates at column gate; conv [taps][channels]; state [num_slots][H][pad16(dk)][pad16(dv)], ring
 * [num_slots][taps][channels], row p % taps = the inputs of position p.  slots_host: slot of every block-table row (segs_host's last column; nseg = 0: of
 * every row, token generation).  max_chunks: chunks of 16 tokens whose factors are kept at a time.  out [T, ldo] in the compute type. */
int mi_op_delta_rule(const mi_layer_spec* spec, const float* proj, int32_t ldp, int32_t beta, const float* z, int32_t ldz, int32_t gate, const float* conv,
                     const float* a_log, const float* dt, const float* norm, float eps, float* state, float* ring, int32_t num_slots,
                     const int32_t* slots_host, const int32_t* pos_host, const int32_t* segs_host, int32_t nseg, int32_t T, int32_t max_chunks,
                     void* out, int32_t ldo, int32_t f32, void* stream);
/* ---- kernels of the post-norm blocks (device pointers but those named host; segs_host, slots_host as above, nseg = 0: token generation) ----
 * resid [T, ld] = scale table[ids[t]] + sinusoid of pos[t] (base pos_base); out [T, ldy]: the same in the compute type */
int mi_op_embed_sinusoid(const int32_t* ids, const int32_t* pos, const void* table, float scale, float pos_base, int32_t T, int32_t D, int32_t ld,
                         float* resid, void* out, int32_t ldy, int32_t f32, void* stream);
/* mi_op_qkv_scatter with biases [H dk + G dk], norm weights [dk] (any may be NULL) and spec's qk_norm / keys_as_values */
int mi_op_head_scatter(const float* qkv, int32_t ldq, int32_t T, const mi_layer_spec* spec, const float* bias, const float* q_norm, const float* k_norm,
                       float eps, const int32_t* slots, int32_t block_size, void* q, void* kpool, void* vpool, int32_t f32, void* stream);
/* mi_op_window_attn with spec's chunk, sinks [H] (NULL: spec's softmax_sink is a score of 0), rel [rel_rows, H] (NULL: no bias), and the heads' outputs
 * times mult sigmoid(gate [T, ldg]) (NULL: mult alone) */
int mi_op_chunk_attn(const mi_layer_spec* spec, const float* sinks, const float* rel, const float* gate, int32_t ldg, float mult, const void* q,
                     const void* kpool, const void* vpool, int32_t block_size, const int32_t* block_table, int32_t MB, const int32_t* pos,
                     const int32_t* ctx_lens, const int32_t* segs_host, int32_t nseg, int32_t T, int32_t max_ctx, void* out, int32_t ldo, int32_t f32,
                     int32_t path, void* stream);
/* y [T, ldy] = silu(bias + causal convolution of x [T, ldx] over C channels); w [taps][C] (last row: the token itself), ring [slots][taps][C] */
int mi_op_short_conv(const float* x, int32_t ldx, const float* w, const float* b, int32_t C, int32_t taps, float* ring, int32_t num_slots,
                     const int32_t* slots_host, const int32_t* pos_host, const int32_t* segs_host, int32_t nseg, int32_t T, void* y, int32_t ldy,
                     int32_t f32, void* stream);
/* Selective scan (spec: MI_MIX_SCAN).  x [T, ldx] compute type; low [T, ldl] fp32: dt's low-rank input at column 0, B at col_b, C at col_c; w_dt
 * [inner, dt_rank], dt_bias, a_log [inner, state], d fp32; z [T, ldz]; state [num_slots][inner][padded state].  y [T, ldy] compute type */
int mi_op_scan(const mi_layer_spec* spec, const void* x, int32_t ldx, const float* low, int32_t ldl, int32_t col_b, int32_t col_c, const float* w_dt,
               const float* dt_bias, const float* a_log, const float* d, const float* z, int32_t ldz, float* state, int32_t num_slots,
               const int32_t* slots_host, const int32_t* pos_host, const int32_t* segs_host, int32_t nseg, int32_t T, void* y, int32_t ldy, int32_t f32,
               void* stream);
int32_t mi_op_scan_state(int32_t state);    /* the padded state */
/* State-space duality (spec: MI_MIX_SSD).  xbc [T, ldx] compute type: [x | B | C] behind the convolution; dt [T, ldt]; state [num_slots][H]
 * [pad16(state)][pad16(dim)]; max_chunks: chunks of 64 tokens in memory at a time.  y [T, ldy] fp32, ahead of gate and norm */
int mi_op_ssd(const mi_layer_spec* spec, const void* xbc, int32_t ldx, const float* dt, int32_t ldt, const float* dt_bias, const float* a_log, const float* d,
              float* state, int32_t num_slots, const int32_t* slots_host, const int32_t* pos_host, const int32_t* segs_host, int32_t nseg, int32_t T,
              int32_t max_chunks, float* y, int32_t ldy, int32_t f32, void* stream);
/* out [T, ldo] = y silu(z), in `parts` equal parts over their root mean square, times w [n] */
int mi_op_gated_norm(const float* y, int32_t ldy, const float* z, int32_t ldz, const float* w, int32_t n, int32_t parts, float eps, int32_t T, void* out,
                     int32_t ldo, int32_t f32, void* stream);
/* Latent attention of a ragged batch over that pool: uk [H dk, rank], uv [H dv, rank] fp32.  path: 1 plain, 2 rows in the latent space,
 * 3 keys and values written out (segments of two rows and more).  out [T, H v_dim] (row stride ldo). */
int mi_op_latent_attn(const mi_layer_spec* spec, const float* uk, const float* uv, const void* q, const void* pool, int32_t block_size,
                      const int32_t* block_table, int32_t MB, const int32_t* pos, const int32_t* segs_host, int32_t nseg, int32_t T,
                      int32_t max_ctx, void* out, int32_t ldo, int32_t f32, int32_t path, void* stream);
/* Router and experts: x [T, ldx]; router [E, D], router_b [E], gate / up [E, ff, D], down [E, D, ff] fp32 -> ids, weights [T, top],
 * y [T top, ldy] fp32 = every pair's expert output, unweighted.  path: 1 weight streaming (or fp32), 2 pairs grouped by expert.
 * groups > 0: the sigmoid rule over that many groups, `keep` of them eligible, router_b its correction; squared-relu experts, gate NULL. */
int mi_op_experts(const void* x, int32_t ldx, int32_t T, int32_t D, int32_t experts, int32_t top, int32_t ff, const float* router, const float* router_b,
                  const float* gate, const float* up, const float* down, int32_t* ids, float* weights, float* y, int32_t ldy, int32_t groups, int32_t keep,
                  int32_t f32, int32_t path, void* stream);

#ifdef __cplusplus
}
#endif
#endif /* MI355X_VLLM_H */
