// Log-probabilities of one row of logits on the host (declared in pegainfer_qwen3.h, shared by all runtimes of this library).
#include <algorithm>
#include <cmath>
#include <utility>
#include <vector>

#include "pegainfer_qwen3.h"

extern "C" {
// compute_logprobs_from_cpu (executor.rs:400-434), statement for statement: f32 max fold, f32 sequential sum of
// exp(x - max), log_sum_exp = max + ln(sum); the top list is built by the reference's ordered insertion (strictly-greater
// test against the last entry, insertion at partition_point(v > val): value descending, a later equal value in FRONT of
// an earlier one, none displaced from a full list by an equal value).  Returns the number of top
// entries written (min(top_k, n)), or -1 (empty row / token out of range: the reference returns None)
int32_t pegainfer_logprobs_from_logits(const float* logits_f32, int32_t n, uint32_t token, int32_t top_k,
                                       float* out_logprob, uint32_t* out_top_ids, float* out_top_logprobs) {
  if (!logits_f32 || n <= 0 || token >= (uint32_t)n) return -1;
  float max_val = -INFINITY;
  for (int i = 0; i < n; ++i) max_val = std::fmax(max_val, logits_f32[i]);   // f32::max: NaN-ignoring like fmaxf
  float sum_exp = 0.f;
  for (int i = 0; i < n; ++i) sum_exp += std::exp(logits_f32[i] - max_val);
  const float lse = max_val + std::log(sum_exp);
  if (out_logprob) *out_logprob = logits_f32[token] - lse;
  const int k = std::min(std::max(top_k, 0), n);
  if (k == 0) return 0;
  std::vector<std::pair<uint32_t, float>> best;
  best.reserve((size_t)k + 1);
  for (int i = 0; i < n; ++i) {
    const float val = logits_f32[i];
    if ((int)best.size() < k || val > best.back().second) {
      size_t pos = 0;   // partition_point(|v| v > val)
      size_t lo = 0, hi = best.size();
      while (lo < hi) { const size_t mid = (lo + hi) / 2; if (best[mid].second > val) lo = mid + 1; else hi = mid; }
      pos = lo;
      best.insert(best.begin() + pos, {(uint32_t)i, val});
      if ((int)best.size() > k) best.pop_back();
    }
  }
  for (size_t i = 0; i < best.size(); ++i) {
    if (out_top_ids) out_top_ids[i] = best[i].first;
    if (out_top_logprobs) out_top_logprobs[i] = best[i].second - lse;
  }
  return (int32_t)best.size();
}
}  // extern "C"
