/*
 * pegainfer_sopanex.h - C ABI of the Sopanex host runtime in libpegainfer_qwen3.so.
 *
 * Sopanex: a decoder whose layers are listed one by one in config.json ("layers": type, mixer sizes, feed-forward or none) over an
 * fp32 residual stream that starts as the token's embedding row times a constant plus, when "embedding.bigram" is given, the row of a
 * table addressed by the previous and the current token.  Every sublayer has an RMS norm before and after it, with weights kept as
 * offsets from one: x <- x + norm_b(f(norm(x))).  Mixer "parallel": two mixers that read the same input, left_scale * left + right_scale *
 * right.  Left: softmax attention over grouped key/value heads whose values are the unrotated keys, rotation of the first rot.dims values
 * (value i with value i + rot.dims / 2; optional long-context scaling by a ramp over the dimensions), a sink logit per head and a sigmoid
 * gate per head.  Right: gated linear attention, a decay per (head, key channel) and token from a two-step projection, the read-out
 * RMS-normed per head and gated by silu.  Feed-forward: routed experts (softmax over all, a correction that only chooses, renormalised
 * weights times a constant), of which the last `identity` numbers return their input, beside a shared expert with a sigmoid gate per
 * token; experts are W_down gelu(W_up h), the exact gelu.  Logits through a head of their own.
 *
 * Same shape as the other runtimes of this library: one model = one device + one in-order HIP stream; a request is a slot that
 * holds a KvState over the shared PagePool (kv_pool.h) for every layer that caches AND a region of the state arena (seq_state.h:
 * the linear-attention states, fp32); a step's metadata travels as ONE pinned block; every op goes through the kernel library's
 * C ABI.  ONE step function serves prompts, portions of prompts and single decoded tokens of several requests in the same batch.
 * Served in bf16 (matrix products in bf16 with fp32 accumulation; norms, attention scores / weights, angles, the router, the
 * recurrence with its decays, the stream and the logits in fp32) or entirely in fp32.
 * All functions return 0 on success or a negative error (see pegainfer_sopanex_last_error).
 */
#ifndef PEGAINFER_SOPANEX_H
#define PEGAINFER_SOPANEX_H

#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

typedef void* pegainfer_sopanex_t;

/* dtype: 0 = bf16, 1 = fp32 (PEGAINFER_DTYPE_* of pegainfer_duguzen.h).  max_tokens: capacity of the key/value cache in
 * tokens (whole pages of pegainfer_sopanex_page_size() tokens; a live request occupies its length rounded up to pages).
 * max_requests: request slots = state regions = the largest batch of one step. */
pegainfer_sopanex_t pegainfer_sopanex_create(const char* config_json, int32_t device_ordinal, int32_t dtype,
                                             int32_t max_tokens, int32_t max_requests);
pegainfer_sopanex_t pegainfer_sopanex_from_pretrained(const char* model_dir, int32_t device_ordinal, int32_t dtype,
                                                      int32_t max_tokens, int32_t max_requests);
void pegainfer_sopanex_destroy(pegainfer_sopanex_t m);
const char* pegainfer_sopanex_last_error(pegainfer_sopanex_t m);

/* one tensor by its checkpoint name, host bf16 bit patterns (widened exactly when the model is served in fp32) */
int32_t pegainfer_sopanex_load_tensor(pegainfer_sopanex_t m, const char* name, const void* host_bf16, int64_t numel);
/* seeded weights for every tensor the configuration names (benchmarks and tests without a checkpoint) */
int32_t pegainfer_sopanex_fill_synthetic(pegainfer_sopanex_t m, uint64_t seed, float std);
int32_t pegainfer_sopanex_finalize(pegainfer_sopanex_t m);

/* a new request takes a free slot and starts from zero state; a dropped slot, its pages and its state region are handed
 * out again */
int32_t pegainfer_sopanex_new_request(pegainfer_sopanex_t m);
int32_t pegainfer_sopanex_drop_request(pegainfer_sopanex_t m, int32_t request_id);
int32_t pegainfer_sopanex_request_seq_len(pegainfer_sopanex_t m, int32_t request_id);
int32_t pegainfer_sopanex_available_pages(pegainfer_sopanex_t m);
int32_t pegainfer_sopanex_capacity_pages(pegainfer_sopanex_t m);
int32_t pegainfer_sopanex_page_size(pegainfer_sopanex_t m);
int32_t pegainfer_sopanex_max_batch_size(pegainfer_sopanex_t m);
int32_t pegainfer_sopanex_vocab_size(pegainfer_sopanex_t m);
int32_t pegainfer_sopanex_width(pegainfer_sopanex_t m);
int32_t pegainfer_sopanex_num_layer_runs(pegainfer_sopanex_t m);
int32_t pegainfer_sopanex_dtype(pegainfer_sopanex_t m);
/* floats of recurrent state one request holds (the linear-attention states of all layers) */
int64_t pegainfer_sopanex_state_floats(pegainfer_sopanex_t m);

/* THE step: entry i appends lens[i] tokens (tokens_concat, entries back to back) to request request_ids[i], continuing
 * from the cache and state earlier steps left; all entries run as one batch.  want_rows: indices into the concatenated
 * token rows whose logits are computed (n_want = -1: the last row of every entry).  out_logits_host (optional) receives
 * [n_want, vocab] floats; out_tokens (optional) the greedy token of every wanted row.  Nothing is changed when the step
 * is rejected (unknown request, not enough free pages, a request listed twice). */
int32_t pegainfer_sopanex_step(pegainfer_sopanex_t m, int32_t n_entries, const int32_t* request_ids, const int32_t* lens,
                               const uint32_t* tokens_concat, int32_t n_want, const int32_t* want_rows,
                               float* out_logits_host, int32_t* out_tokens);
int32_t pegainfer_sopanex_sample(pegainfer_sopanex_t m, int32_t row, float temperature, int32_t top_k, float top_p,
                                 float random_val, int32_t* out_token);
int32_t pegainfer_sopanex_logprobs(pegainfer_sopanex_t m, int32_t row, uint32_t token, int32_t top_k, float* out_logprob,
                                   uint32_t* out_top_ids, float* out_top_logprobs);

/* the residual stream after every layer, all token rows of the last step: while
 * enabled each step keeps [layer runs, rows, width] floats on the device; debug_hidden copies one run's rows and returns the
 * row count */
int32_t pegainfer_sopanex_debug_hidden_enable(pegainfer_sopanex_t m, int32_t enable);
int32_t pegainfer_sopanex_debug_hidden(pegainfer_sopanex_t m, int32_t layer_run, float* out_host, int32_t max_rows);

float pegainfer_sopanex_last_step_ms(pegainfer_sopanex_t m);
int64_t pegainfer_sopanex_weight_bytes(pegainfer_sopanex_t m);
/* 1: a bf16 model's dense projections run on the plain fp32-arithmetic GEMM instead of the tuned bf16 routes */
int32_t pegainfer_sopanex_set_plain_kernels(pegainfer_sopanex_t m, int32_t on);

#ifdef __cplusplus
}
#endif
#endif /* PEGAINFER_SOPANEX_H */
