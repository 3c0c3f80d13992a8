// What the token-by-token recurrences share (recurrent.hip, decay_attn.hip, gated_linear.hip): the layout of a workgroup - 16 value columns, a column's
// state over the sixteen lanes of a DPP row - and the staging of 16 tokens' q | k | v through registers into LDS.
#pragma once

#include "common.h"

namespace pk {

constexpr int kRecTokens = 16;   // tokens staged per round
constexpr int kRecCols = 16;     // value columns per workgroup (four per wave)
constexpr int kRecSlices = 16;   // lanes that share one column

// One round's q | k | v values, fetched into registers (issue) and put into LDS later (land).  Thread t serves token t / 16
// of the round: values t % 16, t % 16 + 16, ... of its query and key and column t % 16 of its value, so which register holds
// what is known at compile time and neighbouring lanes read neighbouring addresses.
template <int NS>
struct RoundFetch {
  static constexpr int DP = kRecSlices * NS;
  float q[NS], k[NS], v;
  template <typename LoadQ, typename LoadK, typename LoadV>
  __device__ __forceinline__ void issue(int tc, int tid, int dim, LoadQ&& lq, LoadK&& lk, LoadV&& lv) {
    const int tt = tid >> 4, part = tid & 15;
    const bool live = tt < tc;
#pragma unroll
    for (int j = 0; j < NS; ++j) {
      const int d = part + 16 * j;
      q[j] = live && d < dim ? lq(tt, d) : 0.f;
      k[j] = live && d < dim ? lk(tt, d) : 0.f;
    }
    v = live ? lv(tt, part) : 0.f;
  }
  __device__ __forceinline__ void land(int tid, float (*s_q)[DP], float (*s_k)[DP], float (*s_v)[kRecCols]) {
    land(tid, s_q, s_k, s_v, [](float x) { return x; });
  }
  // act: applied to every value on its way into LDS, when the loads have long arrived (act(0) = 0)
  template <typename Act>
  __device__ __forceinline__ void land(int tid, float (*s_q)[DP], float (*s_k)[DP], float (*s_v)[kRecCols], Act&& act) {
    const int tt = tid >> 4, part = tid & 15;
#pragma unroll
    for (int j = 0; j < NS; ++j) {
      s_q[tt][part + 16 * j] = act(q[j]);
      s_k[tt][part + 16 * j] = act(k[j]);
    }
    s_v[tt][part] = act(v);
  }
};

template <typename F>
inline bool by_slices(int dim, F&& fn) {
  if (dim <= 16) fn(std::integral_constant<int, 1>());
  else if (dim <= 32) fn(std::integral_constant<int, 2>());
  else if (dim <= 64) fn(std::integral_constant<int, 4>());
  else if (dim <= 128) fn(std::integral_constant<int, 8>());
  else if (dim <= 256) fn(std::integral_constant<int, 16>());
  else return false;
  return true;
}

}  // namespace pk
