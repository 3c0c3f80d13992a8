// Routed feed-forward: the router and the bookkeeping around the expert GEMMs (which run on the grouped form of
// pegainfer_gemm_strided).
//   route_kernel    one workgroup per token row: fp32 router logits (a wave per expert, lanes over the width), sigmoid
//                   scores, the correction added for the CHOICE only, group scores = the two largest choices of a group,
//                   the best `keep` groups stay eligible, then the `top` largest eligible choices; weights = the plain
//                   sigmoid scores of the chosen experts.  Selection runs on one wave: a lane per group for the group
//                   scores and ranks, then `top` wave-wide arg-max steps; ties go to the lower index.
//   sort_kernel     (row, choice) pairs bucketed by expert with LDS counters, an exclusive scan, and the table of <= 64-row
//                   tiles the grouped GEMM walks.  The order of pairs inside an expert comes from atomics; every pair owns
//                   its output row, so results do not depend on it.  Tiles hold <= 64 or <= 128 rows, as the GEMM form that walks them wants.
//   combine_kernel  out[row] = sum over the row's choices, in choice order, of weight * expert output (fp32 sum), plus a row
//                   every token gets (a shared expert), optionally times the sigmoid of a per-row gate logit.
// Options of the selection: a group's score = its two largest choices (default) or its largest; the chosen weights as they
// are (default) or divided by their sum, times a factor.  Expert numbers past the experts that have tensors are identity experts:
// they get no position in the sort, and the combine takes the feed-forward's input row for them.
//   route_plan_kernel  selection and sort in one launch for steps of few rows
#include <algorithm>

#include "common.h"
#include "typed.h"
#include "pegainfer_kernels_blocks.h"

namespace pk {

// Selection on one wave from per-expert values in LDS (s: sigmoid scores, or logits when score is softmax; ch: s + correction):
// softmax over ALL experts if asked, group scores, kept groups, then `top` wave-wide arg-max steps.  LDS accesses of one wave
// complete in order, so no barrier is needed between its steps.
template <typename A>
__device__ __forceinline__ void route_select_wave(float* s, float* ch, float* gs, const A* __restrict__ corr,
                                                  int32_t* __restrict__ out_e, float* __restrict__ out_w, int row, int lane, int E,
                                                  int G, int keep, int top, int score, int group_kind = 0, int renorm = 0,
                                                  float factor = 1.0f) {
  if (score == PEGAINFER_SCORE_SOFTMAX) {            // s = exp(z - max) / sum over ALL experts, then the choice scores
    float mx = -INFINITY;
    for (int e = lane; e < E; e += 64) mx = fmaxf(mx, s[e]);
    mx = wave_max(mx);
    float sum = 0.f;
    for (int e = lane; e < E; e += 64) sum += expf(s[e] - mx);
    sum = wave_sum(sum);
    for (int e = lane; e < E; e += 64) {
      const float sc = expf(s[e] - mx) / sum;
      s[e] = sc;
      ch[e] = corr ? sc + ld(corr + e) : sc;
    }
    __builtin_amdgcn_wave_barrier();
  }
  if (G > 1) {
    const int per = E / G;
    for (int g = lane; g < G; g += 64) {             // a lane scores a group: its two largest choices
      float b0 = -INFINITY, b1 = -INFINITY;
      for (int i = 0; i < per; ++i) {
        const float v = ch[g * per + i];
        if (v > b0) { b1 = b0; b0 = v; } else if (v > b1) b1 = v;
      }
      gs[g] = per >= 2 && group_kind == PEGAINFER_GROUP_TOP2_SUM ? b0 + b1 : b0;
    }
    __builtin_amdgcn_wave_barrier();
    for (int g = lane; g < G; g += 64) {             // kept = fewer than `keep` groups rank ahead (ties: the lower index)
      const float mine = gs[g];
      int ahead = 0;
      for (int o = 0; o < G; ++o) {
        const float v = gs[o];
        ahead += (v > mine || (v == mine && o < g)) ? 1 : 0;
      }
      if (ahead >= keep)
        for (int i = 0; i < per; ++i) ch[g * per + i] = -INFINITY;
    }
    __builtin_amdgcn_wave_barrier();
  }
  for (int k = 0; k < top; ++k) {
    float bv = -INFINITY;
    int be = 0x7FFFFFFF;
    for (int e = lane; e < E; e += 64) {             // ascending e per lane: the first maximum is the lowest index
      const float v = ch[e];
      if (v > bv) { bv = v; be = e; }
    }
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) {
      const float ov = __shfl_xor(bv, off, kWave);
      const int oe = __shfl_xor(be, off, kWave);
      if (ov > bv || (ov == bv && oe < be)) { bv = ov; be = oe; }
    }
    const bool found = bv != -INFINITY;
    if (lane == 0) {
      out_e[(size_t)row * top + k] = found ? be : 0;
      out_w[(size_t)row * top + k] = found ? s[be] : 0.f;
      if (found) ch[be] = -INFINITY;
    }
    __builtin_amdgcn_wave_barrier();
  }
  if ((renorm || factor != 1.0f) && lane == 0) {   // the chosen weights divided by their sum (in choice order), times the factor
    float sum = 0.f;
    for (int k = 0; k < top; ++k) sum += out_w[(size_t)row * top + k];
    const float inv = factor * (renorm ? 1.0f / (sum + 1e-20f) : 1.0f);
    for (int k = 0; k < top; ++k) out_w[(size_t)row * top + k] *= inv;
  }
}

template <typename A>
__global__ __launch_bounds__(256) void route_kernel(const A* __restrict__ h, const A* __restrict__ wr,
                                                    const A* __restrict__ corr, int32_t* __restrict__ out_e,
                                                    float* __restrict__ out_w, int d, int E, int G, int keep, int top,
                                                    int score) {
  extern __shared__ float sm[];
  float* s = sm;            // [E] sigmoid scores
  float* ch = sm + E;       // [E] choice scores (eligible) or -inf
  float* gs = sm + 2 * E;   // [G] group scores
  const int row = blockIdx.x, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const A* x = h + (size_t)row * d;
  const bool vec = (d & 7) == 0 && aligned16(x) && aligned16(wr);
  // a wave takes four experts at a time (four independent weight streams in flight), waves interleaved over the groups of four
  constexpr int EB = 4;
  for (int e0 = wave * EB; e0 < E; e0 += 4 * EB) {
    float a[EB] = {0.f, 0.f, 0.f, 0.f};
    if (vec) {
      for (int i = lane * 8; i < d; i += 512) {
        float xv[8];
        Vec8<A>::load(x + i, xv);
#pragma unroll
        for (int q = 0; q < EB; ++q) {
          float wv[8];
          Vec8<A>::load(wr + (size_t)min(e0 + q, E - 1) * d + i, wv);
#pragma unroll
          for (int k = 0; k < 8; ++k) a[q] = fmaf(xv[k], wv[k], a[q]);
        }
      }
    } else {
      for (int i = lane; i < d; i += 64) {
        const float xv = ld(x + i);
#pragma unroll
        for (int q = 0; q < EB; ++q) a[q] = fmaf(xv, ld(wr + (size_t)min(e0 + q, E - 1) * d + i), a[q]);
      }
    }
#pragma unroll
    for (int q = 0; q < EB; ++q) {
      const float z = wave_sum(a[q]);
      const int e = e0 + q;
      if (lane == 0 && e < E) {
        const float sc = score == PEGAINFER_SCORE_SOFTMAX ? z : sigmoid_f(z);   // softmax: the logit for now
        s[e] = sc;
        ch[e] = corr ? sc + ld(corr + e) : sc;
      }
    }
  }
  __syncthreads();
  if (wave != 0) return;
  route_select_wave(s, ch, gs, corr, out_e, out_w, row, lane, E, G, keep, top, score);
}

// The same selection from router logits that a GEMM has left in fp32 ([rows][E] at a stride), by one wave with LDS of its own.
struct RouteForm {
  int E, G, keep, top, score, group_kind, renorm;
  float factor;
  int64_t logits_stride;
};
template <typename A>
__device__ __forceinline__ void route_row_from_logits(const float* __restrict__ logits, const A* __restrict__ corr, int32_t* out_e,
                                                      float* out_w, const RouteForm& f, int row, int lane, float* s) {
  float *ch = s + f.E, *gs = s + 2 * f.E;
  for (int e = lane; e < f.E; e += 64) {
    const float z = logits[(size_t)row * f.logits_stride + e];
    const float sc = f.score == PEGAINFER_SCORE_SOFTMAX ? z : sigmoid_f(z);
    s[e] = sc;
    ch[e] = corr ? sc + ld(corr + e) : sc;
  }
  __builtin_amdgcn_wave_barrier();
  route_select_wave(s, ch, gs, corr, out_e, out_w, row, lane, f.E, f.G, f.keep, f.top, f.score, f.group_kind, f.renorm, f.factor);
}
// a wave per row, four rows per workgroup
template <typename A>
__global__ __launch_bounds__(256) void route_from_logits_kernel(const float* __restrict__ logits, const A* __restrict__ corr,
                                                                int32_t* __restrict__ out_e, float* __restrict__ out_w, int rows,
                                                                RouteForm f) {
  extern __shared__ float sm[];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int row = blockIdx.x * 4 + wave;
  if (row >= rows) return;
  route_row_from_logits(logits, corr, out_e, out_w, f, row, lane, sm + wave * (2 * f.E + f.G));
}

struct SortOut {
  int32_t *pos_pair, *pos_row, *tile_group, *tile_row0, *tile_rows, *n_tiles;
  int max_tiles, per_tile;
};
// Pairs whose expert number is E or more (identity experts) get no position.  One workgroup of N threads; cnt: [2 E] of LDS.
template <int N>
__device__ __forceinline__ void route_sort_block(const int32_t* expert, int n_pairs, int top, int E, const SortOut& o, int* cnt) {
  int* cur = cnt + E;            // [E] counts, then [E] cursors
  for (int e = threadIdx.x; e < E; e += N) cnt[e] = 0;
  __syncthreads();
  constexpr int kKeep = 4;       // a thread's first choices stay in registers between the two walks
  int mine[kKeep];
#pragma unroll
  for (int k = 0; k < kKeep; ++k) {
    const int p = threadIdx.x + N * k;
    mine[k] = p < n_pairs ? expert[p] : E;
  }
#pragma unroll
  for (int k = 0; k < kKeep; ++k)
    if (mine[k] < E) atomicAdd(&cnt[mine[k]], 1);
  for (int p = threadIdx.x + N * kKeep; p < n_pairs; p += N) {
    const int e = expert[p];
    if (e < E) atomicAdd(&cnt[e], 1);
  }
  __syncthreads();
  if (threadIdx.x == 0) {
    int off = 0, nt = 0;
    for (int e = 0; e < E; ++e) {
      const int c = cnt[e];
      cur[e] = off;
      for (int r0 = 0; r0 < c && nt < o.max_tiles; r0 += o.per_tile, ++nt) {
        o.tile_group[nt] = e;
        o.tile_row0[nt] = off + r0;
        o.tile_rows[nt] = min(o.per_tile, c - r0);
      }
      off += c;
    }
    *o.n_tiles = nt;
  }
  __syncthreads();
  auto place = [&](int p, int e) {
    if (e >= E) return;
    const int at = atomicAdd(&cur[e], 1);
    o.pos_pair[at] = p;
    o.pos_row[at] = p / top;
  };
#pragma unroll
  for (int k = 0; k < kKeep; ++k) place(threadIdx.x + N * k, mine[k]);
  for (int p = threadIdx.x + N * kKeep; p < n_pairs; p += N) place(p, expert[p]);
}
constexpr int kSortThreads = 1024;
__global__ __launch_bounds__(kSortThreads) void route_sort_kernel(const int32_t* __restrict__ expert, int n_pairs, int top, int E, SortOut o) {
  extern __shared__ int cnt[];
  route_sort_block<kSortThreads>(expert, n_pairs, top, E, o, cnt);
}
// Few rows (decoding): selection and sort in one launch of one workgroup, which sees its own choices after a barrier.
template <typename A>
__global__ __launch_bounds__(256) void route_plan_kernel(const float* __restrict__ logits, const A* __restrict__ corr, int32_t* out_e,
                                                         float* out_w, int rows, RouteForm f, int sort_experts, SortOut o) {
  extern __shared__ float sm[];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  for (int row = wave; row < rows; row += 4) {
    route_row_from_logits(logits, corr, out_e, out_w, f, row, lane, sm + wave * (2 * f.E + f.G));
    __builtin_amdgcn_wave_barrier();
  }
  __threadfence_block();
  __syncthreads();               // the choices are read by other waves of this workgroup; the selection's LDS is free
  route_sort_block<256>(out_e, rows * f.top, f.top, sort_experts, o, reinterpret_cast<int*>(sm));
}

// expert / same: pairs that chose an expert number of same_from or more take the row of `same` (the feed-forward's own input) instead
// of a y_pairs row
template <typename A>
__global__ __launch_bounds__(256) void route_combine_kernel(const float* __restrict__ y, const float* __restrict__ w,
                                                            const A* __restrict__ add, A* __restrict__ out, int d, int top,
                                                            const float* __restrict__ add_gate, int64_t add_gate_stride,
                                                            const int32_t* __restrict__ expert, int same_from,
                                                            const A* __restrict__ same, int64_t same_stride) {
  const int row = blockIdx.x;
  const float gate = add && add_gate ? sigmoid_f(add_gate[(size_t)row * add_gate_stride]) : 1.0f;
  for (int i = blockIdx.y * 256 + threadIdx.x; i < d; i += gridDim.y * 256) {
    float a = add ? ld(add + (size_t)row * d + i) * gate : 0.f;
    for (int c = 0; c < top; ++c) {
      const bool own = same && expert[(size_t)row * top + c] >= same_from;      // uniform over the workgroup
      const float v = own ? ld(same + (size_t)row * same_stride + i) : y[((size_t)row * top + c) * d + i];
      a = fmaf(w[(size_t)row * top + c], v, a);
    }
    st(out + (size_t)row * d + i, a);
  }
}

}  // namespace pk

extern "C" {
using namespace pk;

pegainfer_status_t pegainfer_route_topk(const void* h, const void* w_router, const void* correction, int32_t* out_expert,
                                        float* out_weight, int32_t d, int32_t experts, int32_t n_groups, int32_t keep_groups,
                                        int32_t top, int32_t rows, int32_t score_kind, int32_t dtype, pegainfer_stream_t stream) {
  if (rows <= 0) return 0;
  if (score_kind != PEGAINFER_SCORE_SIGMOID && score_kind != PEGAINFER_SCORE_SOFTMAX) return (pegainfer_status_t)hipErrorInvalidValue;
  if (n_groups < 1) n_groups = 1;
  if (experts <= 0 || experts % n_groups || top <= 0 || top > experts || keep_groups < 1 || keep_groups > n_groups ||
      (size_t)(2 * experts + n_groups) * 4 > 60000)
    return (pegainfer_status_t)hipErrorInvalidValue;
  const size_t smem = (size_t)(2 * experts + n_groups) * sizeof(float);
  if (!by_dtype(dtype, [&](auto* t) {
        using A = std::remove_pointer_t<decltype(t)>;
        route_kernel<A><<<rows, 256, smem, as_stream(stream)>>>(static_cast<const A*>(h), static_cast<const A*>(w_router),
                                                                static_cast<const A*>(correction), out_expert, out_weight, d,
                                                                experts, n_groups, keep_groups, top, score_kind);
      }))
    return (pegainfer_status_t)hipErrorInvalidValue;
  return (pegainfer_status_t)hipGetLastError();
}

pegainfer_status_t pegainfer_route_plan(const pegainfer_route_plan_desc* q, pegainfer_stream_t stream) {
  constexpr pegainfer_status_t bad = (pegainfer_status_t)hipErrorInvalidValue;
  if (!q) return bad;
  if (q->rows <= 0) return 0;
  const int E = q->experts, groups = std::max(1, q->n_groups), keep = q->n_groups < 1 ? 1 : q->keep_groups, top = q->top;
  if (!q->logits || !q->out_expert || !q->out_weight || E <= 0 || E % groups || top <= 0 || top > E || keep < 1 || keep > groups ||
      q->logits_stride < E || (size_t)(2 * E + groups) * 16 > 60000 ||
      (q->score_kind != PEGAINFER_SCORE_SIGMOID && q->score_kind != PEGAINFER_SCORE_SOFTMAX) ||
      (q->group_kind != PEGAINFER_GROUP_TOP2_SUM && q->group_kind != PEGAINFER_GROUP_MAX))
    return bad;
  const int64_t pairs = (int64_t)q->rows * top;
  const bool sorted = q->sort_experts > 0;
  if (sorted && ((q->rows_per_tile != 64 && q->rows_per_tile != 128) || q->sort_experts > 7000 || pairs > 0x7FFFFFFF || !q->pos_pair ||
                 !q->pos_row || !q->tile_group || !q->tile_row0 || !q->tile_rows || !q->n_tiles ||
                 q->max_tiles < std::min<int64_t>(pairs, (pairs + q->rows_per_tile - 1) / q->rows_per_tile + q->sort_experts)))
    return bad;
  const RouteForm f{E, groups, keep, top, q->score_kind, q->group_kind, q->renorm, q->factor, q->logits_stride};
  const SortOut o{q->pos_pair, q->pos_row, q->tile_group, q->tile_row0, q->tile_rows, q->n_tiles, q->max_tiles, q->rows_per_tile};
  const size_t smem = (size_t)4 * (2 * E + groups) * sizeof(float), sort_smem = (size_t)2 * std::max(0, q->sort_experts) * sizeof(int);
  if (!by_dtype(q->dtype, [&](auto* t) {
        using A = std::remove_pointer_t<decltype(t)>;
        const A* corr = static_cast<const A*>(q->correction);
        if (sorted && q->rows <= 16) {
          route_plan_kernel<A><<<1, 256, std::max(smem, sort_smem), as_stream(stream)>>>(q->logits, corr, q->out_expert, q->out_weight,
                                                                                        q->rows, f, q->sort_experts, o);
          return;
        }
        route_from_logits_kernel<A><<<ceil_div(q->rows, 4), 256, smem, as_stream(stream)>>>(q->logits, corr, q->out_expert, q->out_weight,
                                                                                            q->rows, f);
        if (sorted)
          route_sort_kernel<<<1, kSortThreads, sort_smem, as_stream(stream)>>>(q->out_expert, (int)pairs, top, q->sort_experts, o);
      }))
    return bad;
  return (pegainfer_status_t)hipGetLastError();
}

pegainfer_status_t pegainfer_route_from_logits_ex(const float* logits, int64_t logits_stride, const void* correction,
                                                  int32_t* out_expert, float* out_weight, int32_t experts, int32_t n_groups,
                                                  int32_t keep_groups, int32_t top, int32_t rows, int32_t score_kind,
                                                  int32_t group_kind, int32_t renorm, int32_t dtype, pegainfer_stream_t stream) {
  pegainfer_route_plan_desc q{};
  q.logits = logits; q.logits_stride = logits_stride; q.correction = correction; q.out_expert = out_expert; q.out_weight = out_weight;
  q.experts = experts; q.n_groups = n_groups; q.keep_groups = keep_groups; q.top = top; q.rows = rows; q.score_kind = score_kind;
  q.group_kind = group_kind; q.renorm = renorm; q.factor = 1.0f; q.dtype = dtype;
  return pegainfer_route_plan(&q, stream);
}

pegainfer_status_t pegainfer_route_from_logits(const float* logits, const void* correction, int32_t* out_expert, float* out_weight,
                                               int32_t experts, int32_t n_groups, int32_t keep_groups, int32_t top, int32_t rows,
                                               int32_t score_kind, int32_t dtype, pegainfer_stream_t stream) {
  return pegainfer_route_from_logits_ex(logits, experts, correction, out_expert, out_weight, experts, n_groups, keep_groups, top, rows,
                                        score_kind, PEGAINFER_GROUP_TOP2_SUM, 0, dtype, stream);
}

pegainfer_status_t pegainfer_route_sigmoid_grouped(const void* h, const void* w_router, const void* correction,
                                                   int32_t* out_expert, float* out_weight, int32_t d, int32_t experts,
                                                   int32_t n_groups, int32_t keep_groups, int32_t top, int32_t rows,
                                                   int32_t dtype, pegainfer_stream_t stream) {
  return pegainfer_route_topk(h, w_router, correction, out_expert, out_weight, d, experts, n_groups, keep_groups, top, rows,
                              PEGAINFER_SCORE_SIGMOID, dtype, stream);
}

pegainfer_status_t pegainfer_route_sort(const int32_t* expert, int32_t n_pairs, int32_t top, int32_t experts,
                                        int32_t* pos_pair, int32_t* pos_row, int32_t* tile_group, int32_t* tile_row0,
                                        int32_t* tile_rows, int32_t* n_tiles, int32_t max_tiles, int32_t rows_per_tile,
                                        pegainfer_stream_t stream) {
  if (n_pairs <= 0) return 0;
  if ((rows_per_tile != 64 && rows_per_tile != 128) || experts <= 0 || experts > 7000 ||
      max_tiles < (n_pairs + rows_per_tile - 1) / rows_per_tile + experts)
    return (pegainfer_status_t)hipErrorInvalidValue;
  const SortOut o{pos_pair, pos_row, tile_group, tile_row0, tile_rows, n_tiles, max_tiles, rows_per_tile};
  route_sort_kernel<<<1, kSortThreads, (size_t)2 * experts * sizeof(int), as_stream(stream)>>>(expert, n_pairs, top, experts, o);
  return (pegainfer_status_t)hipGetLastError();
}

pegainfer_status_t pegainfer_route_combine_gated(const float* y_pairs, const float* weight, const void* add,
                                                 const float* add_gate, int64_t add_gate_stride, void* out, int32_t d,
                                                 int32_t top, int32_t rows, int32_t dtype, pegainfer_stream_t stream) {
  return pegainfer_route_combine_same(y_pairs, weight, nullptr, 0, nullptr, 0, add, add_gate, add_gate_stride, out, d, top, rows, dtype, stream);
}

pegainfer_status_t pegainfer_route_combine_same(const float* y_pairs, const float* weight, const int32_t* expert, int32_t same_from,
                                                const void* same, int64_t same_stride, const void* add, const float* add_gate,
                                                int64_t add_gate_stride, void* out, int32_t d, int32_t top, int32_t rows, int32_t dtype,
                                                pegainfer_stream_t stream) {
  if (rows <= 0) return 0;
  if (same && !expert) return (pegainfer_status_t)hipErrorInvalidValue;
  if (!by_dtype(dtype, [&](auto* t) {
        using A = std::remove_pointer_t<decltype(t)>;
        // few rows (decoding): the row is cut over several workgroups
        const dim3 grid(rows, rows >= 256 ? 1 : std::min(16, ceil_div(d, 256)));
        route_combine_kernel<A><<<grid, 256, 0, as_stream(stream)>>>(y_pairs, weight, static_cast<const A*>(add), static_cast<A*>(out), d,
                                                                     top, add_gate, add_gate_stride, expert, same_from,
                                                                     static_cast<const A*>(same), same_stride);
      }))
    return (pegainfer_status_t)hipErrorInvalidValue;
  return (pegainfer_status_t)hipGetLastError();
}

pegainfer_status_t pegainfer_route_combine_add(const float* y_pairs, const float* weight, const void* add, void* out, int32_t d,
                                               int32_t top, int32_t rows, int32_t dtype, pegainfer_stream_t stream) {
  return pegainfer_route_combine_gated(y_pairs, weight, add, nullptr, 0, out, d, top, rows, dtype, stream);
}

pegainfer_status_t pegainfer_route_combine(const float* y_pairs, const float* weight, void* out, int32_t d, int32_t top,
                                           int32_t rows, int32_t dtype, pegainfer_stream_t stream) {
  return pegainfer_route_combine_add(y_pairs, weight, nullptr, out, d, top, rows, dtype, stream);
}

}  // extern "C"
