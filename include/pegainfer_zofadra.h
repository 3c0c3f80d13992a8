/*
 * pegainfer_zofadra.h - C ABI of the Zofadra host runtime in libpegainfer_qwen3.so.
 *
 * Zofadra: a decoder whose layers are listed one by one in config.json ("layers": type, mixer sizes, feed-forward or none) over
 * several residual streams ("streams") in fp32.  A sublayer reads a learned weighted sum of the streams through a layer norm (a
 * weight, no bias); its output times "residual_mult" joins every stream with a learned weight while the streams are mixed by a
 * learned matrix.  The streams start as the token's embedding row times a constant and are summed at the end.  Mixers:
 * "latent_attention" (queries through a latent with an RMS norm; keys and values from one normed latent per token plus one
 * rotated key part shared by the heads, neighbours rotated together; a layer may read the latents another layer has cached,
 * "kv_from"), "attention" (grouped key/value heads, q and k RMS-normed over the whole projection, a sliding window, a bias that
 * falls linearly with the distance, slope 2^(-8 (h + 1) / heads)) and "lightning" (linear attention with a constant decay per head
 * on silu'd q, k and v; the heads normed together, gated by a sigmoid).  Feed-forward: gelu(W_gate h) * (W_up h), the tanh form.
 * Logits through a head of their own.
 *
 * Same shape as the other runtimes of this library: one model = one device + one in-order HIP stream; a request is a slot that
 * holds a KvState over the shared PagePool (kv_pool.h) for every layer that caches AND a region of the state arena (seq_state.h:
 * the lightning layers' states, fp32); a step's metadata travels as ONE pinned block; every op goes through the kernel library's
 * C ABI.  ONE step function serves prompts, portions of prompts and single decoded tokens of several requests in the same batch.
 * Served in bf16 (matrix products in bf16 with fp32 accumulation; norms, attention scores / weights, angles, the recurrence, the
 * streams and the logits in fp32) or entirely in fp32.
 * All functions return 0 on success or a negative error (see pegainfer_zofadra_last_error).
 */
#ifndef PEGAINFER_ZOFADRA_H
#define PEGAINFER_ZOFADRA_H

#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

typedef void* pegainfer_zofadra_t;

/* dtype: 0 = bf16, 1 = fp32 (PEGAINFER_DTYPE_* of pegainfer_duguzen.h).  max_tokens: capacity of the key/value cache in
 * tokens (whole pages of pegainfer_zofadra_page_size() tokens; a live request occupies its length rounded up to pages).
 * max_requests: request slots = state regions = the largest batch of one step. */
pegainfer_zofadra_t pegainfer_zofadra_create(const char* config_json, int32_t device_ordinal, int32_t dtype,
                                             int32_t max_tokens, int32_t max_requests);
pegainfer_zofadra_t pegainfer_zofadra_from_pretrained(const char* model_dir, int32_t device_ordinal, int32_t dtype,
                                                      int32_t max_tokens, int32_t max_requests);
void pegainfer_zofadra_destroy(pegainfer_zofadra_t m);
const char* pegainfer_zofadra_last_error(pegainfer_zofadra_t m);

/* one tensor by its checkpoint name, host bf16 bit patterns (widened exactly when the model is served in fp32) */
int32_t pegainfer_zofadra_load_tensor(pegainfer_zofadra_t m, const char* name, const void* host_bf16, int64_t numel);
/* seeded weights for every tensor the configuration names (benchmarks and tests without a checkpoint) */
int32_t pegainfer_zofadra_fill_synthetic(pegainfer_zofadra_t m, uint64_t seed, float std);
int32_t pegainfer_zofadra_finalize(pegainfer_zofadra_t m);

/* a new request takes a free slot and starts from zero state; a dropped slot, its pages and its state region are handed
 * out again */
int32_t pegainfer_zofadra_new_request(pegainfer_zofadra_t m);
int32_t pegainfer_zofadra_drop_request(pegainfer_zofadra_t m, int32_t request_id);
int32_t pegainfer_zofadra_request_seq_len(pegainfer_zofadra_t m, int32_t request_id);
int32_t pegainfer_zofadra_available_pages(pegainfer_zofadra_t m);
int32_t pegainfer_zofadra_capacity_pages(pegainfer_zofadra_t m);
int32_t pegainfer_zofadra_page_size(pegainfer_zofadra_t m);
int32_t pegainfer_zofadra_max_batch_size(pegainfer_zofadra_t m);
int32_t pegainfer_zofadra_vocab_size(pegainfer_zofadra_t m);
int32_t pegainfer_zofadra_width(pegainfer_zofadra_t m);
int32_t pegainfer_zofadra_num_layer_runs(pegainfer_zofadra_t m);
int32_t pegainfer_zofadra_dtype(pegainfer_zofadra_t m);
/* floats of recurrent state one request holds (the states of all lightning layers) */
int64_t pegainfer_zofadra_state_floats(pegainfer_zofadra_t m);

/* THE step: entry i appends lens[i] tokens (tokens_concat, entries back to back) to request request_ids[i], continuing
 * from the cache and state earlier steps left; all entries run as one batch.  want_rows: indices into the concatenated
 * token rows whose logits are computed (n_want = -1: the last row of every entry).  out_logits_host (optional) receives
 * [n_want, vocab] floats; out_tokens (optional) the greedy token of every wanted row.  Nothing is changed when the step
 * is rejected (unknown request, not enough free pages, a request listed twice). */
int32_t pegainfer_zofadra_step(pegainfer_zofadra_t m, int32_t n_entries, const int32_t* request_ids, const int32_t* lens,
                               const uint32_t* tokens_concat, int32_t n_want, const int32_t* want_rows,
                               float* out_logits_host, int32_t* out_tokens);
int32_t pegainfer_zofadra_sample(pegainfer_zofadra_t m, int32_t row, float temperature, int32_t top_k, float top_p,
                                 float random_val, int32_t* out_token);
int32_t pegainfer_zofadra_logprobs(pegainfer_zofadra_t m, int32_t row, uint32_t token, int32_t top_k, float* out_logprob,
                                   uint32_t* out_top_ids, float* out_top_logprobs);

/* the sum of the residual streams after every layer, all token rows of the last step: while
 * enabled each step keeps [layer runs, rows, width] floats on the device; debug_hidden copies one run's rows and returns the
 * row count */
int32_t pegainfer_zofadra_debug_hidden_enable(pegainfer_zofadra_t m, int32_t enable);
int32_t pegainfer_zofadra_debug_hidden(pegainfer_zofadra_t m, int32_t layer_run, float* out_host, int32_t max_rows);

float pegainfer_zofadra_last_step_ms(pegainfer_zofadra_t m);
int64_t pegainfer_zofadra_weight_bytes(pegainfer_zofadra_t m);
/* 1: a bf16 model's dense projections run on the plain fp32-arithmetic GEMM instead of the tuned bf16 routes */
int32_t pegainfer_zofadra_set_plain_kernels(pegainfer_zofadra_t m, int32_t on);

#ifdef __cplusplus
}
#endif
#endif /* PEGAINFER_ZOFADRA_H */
