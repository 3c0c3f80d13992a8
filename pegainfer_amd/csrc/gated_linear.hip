// Gated linear attention: a linear recurrence with one decay per (head, key channel) and token, over ragged batches, fp32 state and
// fp32 arithmetic throughout:
//     S <- diag(a) S + k v^T,   y = S^T q,      a = sigmoid(z + bias)^(1 / tau),   q times a constant
// Two equivalent forms.
//   gated_scan_kernel         token by token, the layout of recurrent.hip (a workgroup owns 16 value columns of one (entry, head), a
//                             column's state lies over the sixteen lanes of a DPP row): decoding and short portions
//   gated_chunk_sum_kernel    long portions, in chunks of <= 64 tokens that run side by side: U_c = sum_i (k_i * w_i) v_i^T with w_i the
//                             product of the decays behind token i, and the product of all the chunk's decays
//   gated_chunk_state_kernel  walks the chunks of an entry, S <- diag(total_c) S + U_c, and leaves the state BEFORE each in U_c's place
//   gated_chunk_out_kernel    every chunk's outputs
// Decays enter the chunk form as products of the decays themselves, taken inside sub-blocks of 16 tokens: p_i = a_1 .. a_i from a
// sub-block's start, s_j = a_(j+1) .. a_16 to its end, t = a_1 .. a_16 for the whole.  A query of sub-block I meets a key of an earlier
// sub-block J through (q_i p_i) (t between J and I) (k_j s_j): every factor is at most 1, so nothing overflows however fast a channel
// forgets, and nothing cancels.  The queries start as q_i p_i and are multiplied by t_(I-1), t_(I-2), .. as they pass to earlier keys;
// after the first sub-block's t they are what reads the state before the chunk.  Inside a sub-block the score of query i and key j is
// sum_d q_i[d] k_j[d] a_(j+1)[d] .. a_i[d]: a lane carries k_j of its channels along the queries, one multiplication by a_i at a time.
// Products run on v_mfma_f32_16x16x4_f32 (see chunk_core.h); scores are computed transposed (keys as rows), which leaves lane l with
// the scores of query l % 16 against keys 4 (l / 16) + r - the A operand of the product with the values.
#include <algorithm>

#include "common.h"
#include "typed.h"
#include "recurrent_core.h"
#include "chunk_core.h"
#include "pegainfer_kernels_blocks.h"

namespace pk {

// sigmoid(z)^p through x = p (min(z, 0) - log(1 + e^-|z|)).  A decay near one multiplies hundreds of tokens, so its error must not lean to
// one side: there the logarithm comes from the series of 2 artanh(t / (2 + t)) and e^x from its own series around 1, whose last step is
// the only rounding that counts; a decay further down is forgotten before the hardware exponential's last bit shows.
__device__ __forceinline__ float sigmoid_power(float z, float p) {
  constexpr float kLog2e = 1.44269504088896341f;
  const float t = __builtin_amdgcn_exp2f(-fabsf(z) * kLog2e);
  const float s = t / (2.0f + t), q = s * s;           // s <= 1/3
  float l = 2.0f / 15.0f;
  l = fmaf(l, q, 2.0f / 13.0f);
  l = fmaf(l, q, 2.0f / 11.0f);
  l = fmaf(l, q, 2.0f / 9.0f);
  l = fmaf(l, q, 2.0f / 7.0f);
  l = fmaf(l, q, 2.0f / 5.0f);
  l = fmaf(l, q, 2.0f / 3.0f);
  l = fmaf(l, q, 2.0f);
  const float x = (fminf(z, 0.f) - l * s) * p;
  float e = 1.0f / 362880.0f;                          // (e^x - 1) / x for -1/2 < x <= 0
  e = fmaf(e, x, 1.0f / 40320.0f);
  e = fmaf(e, x, 1.0f / 5040.0f);
  e = fmaf(e, x, 1.0f / 720.0f);
  e = fmaf(e, x, 1.0f / 120.0f);
  e = fmaf(e, x, 1.0f / 24.0f);
  e = fmaf(e, x, 1.0f / 6.0f);
  e = fmaf(e, x, 0.5f);
  e = fmaf(e, x, 1.0f);
  return x > -0.5f ? fmaf(e, x, 1.0f) : __builtin_amdgcn_exp2f(x * kLog2e);
}

template <typename A>
struct GatedIn {
  const A* proj;
  int64_t stride, q_off, k_off, v_off;
  float q_scale;
  const float* z;              // [rows][heads * dim] decay inputs
  int64_t z_stride;
  const A* z_bias;             // [heads * dim], or NULL
  float inv_tau;
  // with z NULL: the scan makes the decay inputs itself, W_up [heads * dim][rank_stride] times the row's `rank` values at low_off
  const A* w_up;
  int64_t low_off;
  int rank, rank_stride;
  __device__ __forceinline__ float decay(float zb) const { return sigmoid_power(zb, inv_tau); }
};
constexpr int kLowRank = 256;                        // most values of a row's low-rank part that the scan takes

template <int NS, typename A, bool FUSED>
__global__ __launch_bounds__(256) void gated_scan_kernel(GatedIn<A> in, float* __restrict__ state, int64_t slot_stride,
                                                         float* __restrict__ o, int H, int dim, int vdim,
                                                         const int32_t* __restrict__ entry_row0,
                                                         const int32_t* __restrict__ entry_slot, int scan_max) {
  constexpr int DP = kRecSlices * NS;
  __shared__ __attribute__((aligned(16))) float s_k[kRecTokens][DP], s_q[kRecTokens][DP], s_a[kRecTokens][DP];
  __shared__ float s_v[kRecTokens][kRecCols];
  __shared__ __attribute__((aligned(16))) float s_low[FUSED ? kLowRank : 4];
  const int e = blockIdx.z, h = blockIdx.y, col0 = blockIdx.x * kRecCols;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, r = lane & 15, cl = wave * 4 + (lane >> 4);
  const int col = col0 + cl;
  const int row0 = entry_row0[e], len = entry_row0[e + 1] - row0;
  if (scan_max > 0 && len > scan_max) return;      // the chunk form has this entry
  float* S_g = state + (int64_t)entry_slot[e] * slot_stride + (int64_t)h * dim * vdim;
  float S[NS];
#pragma unroll
  for (int i = 0; i < NS; ++i) {
    const int d = r * NS + i;
    S[i] = d < dim && col < vdim ? S_g[(int64_t)d * vdim + col] : 0.f;
  }
  const int tt_l = tid >> 4, part = tid & 15;        // the token and the first value this thread stages
  float bias[NS];
#pragma unroll
  for (int j = 0; j < NS; ++j) {
    const int d = part + 16 * j;
    bias[j] = !FUSED && in.z_bias && d < dim ? ld(in.z_bias + (int64_t)h * dim + d) : 0.f;
  }
  RoundFetch<NS> nxt;
  float znx[NS];
  auto fetch = [&](int t0) {
    const A* base = in.proj + (int64_t)(row0 + t0) * in.stride;
    const A *qb = base + in.q_off + (int64_t)h * dim, *kb = base + in.k_off + (int64_t)h * dim, *vb = base + in.v_off + (int64_t)h * vdim + col0;
    const int tc = min(kRecTokens, len - t0);
    nxt.issue(tc, tid, dim, [=](int tt, int d) { return ld(qb + (int64_t)tt * in.stride + d); },
              [=](int tt, int d) { return ld(kb + (int64_t)tt * in.stride + d); },
              [=](int tt, int c) { return col0 + c < vdim ? ld(vb + (int64_t)tt * in.stride + c) : 0.f; });
    if constexpr (FUSED) return;
#pragma unroll
    for (int j = 0; j < NS; ++j) {
      const int d = part + 16 * j;
      znx[j] = tt_l < tc && d < dim ? in.z[(int64_t)(row0 + t0 + tt_l) * in.z_stride + (int64_t)h * dim + d] : 0.f;
    }
  };
  fetch(0);
  for (int t0 = 0; t0 < len; t0 += kRecTokens) {
    const int tc = min(kRecTokens, len - t0);
    __syncthreads();
    nxt.land(tid, s_q, s_k, s_v);
    // rows past the entry's end: no decay, k = v = 0 - a step that leaves S as it is
    if constexpr (FUSED) {
#pragma unroll
      for (int j = 0; j < NS; ++j) s_a[tt_l][part + 16 * j] = 1.0f;
      for (int tt = 0; tt < tc; ++tt) {              // two threads per channel, eight values of the rank at a time
        const A* low = in.proj + (int64_t)(row0 + t0 + tt) * in.stride + in.low_off;
        __syncthreads();
        if (tid < in.rank_stride) s_low[tid] = tid < in.rank ? ld(low + tid) : 0.f;
        __syncthreads();
        for (int d = tid >> 1; d < dim; d += 128) {
          const A* wr = in.w_up + ((int64_t)h * dim + d) * in.rank_stride;
          float sum = 0.f;
          for (int c = (tid & 1) * 8; c < in.rank_stride; c += 16) {
            float wv[8];
            Vec8<A>::load(wr + c, wv);
#pragma unroll
            for (int u = 0; u < 8; ++u) sum = fmaf(wv[u], s_low[c + u], sum);
          }
          sum += __shfl_xor(sum, 1, kWave);
          if (!(tid & 1)) s_a[tt][d] = in.decay(sum + (in.z_bias ? ld(in.z_bias + (int64_t)h * dim + d) : 0.f));
        }
      }
    } else {
#pragma unroll
      for (int j = 0; j < NS; ++j) s_a[tt_l][part + 16 * j] = tt_l < tc ? in.decay(znx[j] + bias[j]) : 1.0f;
    }
    __syncthreads();
    if (t0 + kRecTokens < len) fetch(t0 + kRecTokens);
    float okeep = 0.f;
    auto token = [&](int tt) {
      const float vv = s_v[tt][cl];
      float y0 = 0.f, y1 = 0.f;
#pragma unroll
      for (int i = 0; i < NS; ++i) {
        const float kk = s_k[tt][r * NS + i], qq = s_q[tt][r * NS + i], aa = s_a[tt][r * NS + i];
        S[i] = fmaf(vv, kk, aa * S[i]);
        if (i & 1) y1 = fmaf(S[i], qq, y1); else y0 = fmaf(S[i], qq, y0);
      }
      const float y = row16_sum(y0 + y1) * in.q_scale;
      okeep = tt == r ? y : okeep;
    };
    if (tc == 1) {
      token(0);
    } else {
      for (int t4 = 0; t4 < tc; t4 += 4) {           // no sum of a token feeds the state: four read-outs are in flight together
#pragma unroll
        for (int uu = 0; uu < 4; ++uu) token(t4 + uu);
      }
    }
    if (r < tc && col < vdim) o[(int64_t)(row0 + t0 + r) * ((int64_t)H * vdim) + (int64_t)h * vdim + col] = okeep;
  }
#pragma unroll
  for (int i = 0; i < NS; ++i) {
    const int d = r * NS + i;
    if (d < dim && col < vdim) S_g[(int64_t)d * vdim + col] = S[i];
  }
}

constexpr int kSub = 16;                             // tokens of a sub-block
constexpr int kSubs = kDecayChunk / kSub;
// key channels of the workspace and of the staged rows
__host__ __device__ constexpr int pad_channels(int dim) { return dim <= 32 ? 32 : dim <= 64 ? 64 : 128; }

// One channel of one sub-block, a thread's share: its 16 tokens' decays (1 past the chunk's end), and NV more rows' values (0 there).
// Loads are always in bounds.
template <typename A, int NV>
__device__ __forceinline__ void load_channel(const GatedIn<A>& in, const int64_t* offs, int64_t chan, bool live, int row0, int i0, int n,
                                             float* a, float (*x)[kSub]) {
  float z[kSub];
#pragma unroll
  for (int i = 0; i < kSub; ++i) {
    const int64_t row = row0 + min(i0 + i, n - 1);
    z[i] = in.z[row * in.z_stride + chan];
#pragma unroll
    for (int v = 0; v < NV; ++v) x[v][i] = ld(in.proj + row * in.stride + offs[v] + chan);
  }
  const float b = in.z_bias ? ld(in.z_bias + chan) : 0.f;
#pragma unroll
  for (int i = 0; i < kSub; ++i) {
    const bool in_chunk = live && i0 + i < n;
    a[i] = in_chunk ? in.decay(z[i] + b) : 1.0f;
#pragma unroll
    for (int v = 0; v < NV; ++v) x[v][i] = in_chunk ? x[v][i] : 0.f;
  }
}

// one workgroup per (chunk, head); thread = (sub-block, channel) for the decays, a wave per block of 16 rows x (16 NB) columns of U
template <typename A, int NB>
__global__ __launch_bounds__(512) void gated_chunk_sum_kernel(GatedIn<A> in, float* __restrict__ ws, float* __restrict__ ws_total, int H,
                                                              int dim, int vdim, const int32_t* __restrict__ chunk_row0,
                                                              const int32_t* __restrict__ chunk_rows) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  __shared__ float s_tot[kSubs][128];
  const int c = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, l15 = lane & 15, lg = lane >> 4;
  const int row0 = chunk_row0[c], n = chunk_rows[c];
  const int dp = pad_channels(dim), vp = pad_values(vdim), sk = stride_rows4(dp), sv = stride_rows4(vp);
  float *s_k = sm, *s_v = sm + kDecayChunk * sk;
  const int sub = tid >> 7, d = tid & 127;
  float a[kSub], k[1][kSub], tot = 1.f;
  {
    const int64_t offs[1] = {in.k_off};
    load_channel<A, 1>(in, offs, (int64_t)h * dim + min(d, dim - 1), d < dim, row0, sub * kSub, n, a, k);
  }
  stage_rows<8>(in.proj, in.stride, in.v_off + (int64_t)h * vdim, row0, n, vdim, vp, s_v, sv, nullptr, tid, [](float x) { return x; });
#pragma unroll
  for (int i = 0; i < kSub; ++i) tot *= a[i];
  s_tot[sub][d] = tot;
  __syncthreads();
  if (d < dp) {
    float w = 1.f;
    for (int s = sub + 1; s < kSubs; ++s) w *= s_tot[s][d];
#pragma unroll
    for (int i = kSub - 1; i >= 0; --i) {
      s_k[(sub * kSub + i) * sk + d] = k[0][i] * w;
      w *= a[i];
    }
    if (sub == 0) ws_total[((int64_t)c * H + h) * dp + d] = w;
  }
  __syncthreads();
  float* U = ws + ((int64_t)c * H + h) * dp * vp;
  const int steps = (n + 3) >> 2, col_blocks = vp / (16 * NB), blocks = (dp >> 4) * col_blocks;
  for (int blk = wave; blk < blocks; blk += 8) {
    const int d0 = (blk / col_blocks) * 16, c0 = (blk % col_blocks) * 16 * NB;
    f32x4 acc[NB];
#pragma unroll
    for (int b = 0; b < NB; ++b) acc[b] = f32x4{0.f, 0.f, 0.f, 0.f};
    const float *ka = s_k + lg * sk + d0 + l15, *vb = s_v + lg * sv + c0 + l15;
#pragma unroll 2
    for (int i = 0; i < steps; ++i) {
      const float av = ka[4 * i * sk];
#pragma unroll
      for (int b = 0; b < NB; ++b) acc[b] = __builtin_amdgcn_mfma_f32_16x16x4f32(av, vb[4 * i * sv + 16 * b], acc[b], 0, 0, 0);
    }
#pragma unroll
    for (int b = 0; b < NB; ++b)
#pragma unroll
      for (int r = 0; r < 4; ++r) U[(int64_t)(d0 + 4 * lg + r) * vp + c0 + 16 * b + l15] = acc[b][r];
  }
}

// One thread per element of the state: through the entry's chunks, the state before each left in U's place.
__global__ __launch_bounds__(256) void gated_chunk_state_kernel(float* ws, const float* __restrict__ ws_total, float* __restrict__ state,
                                                                int64_t slot_stride, int H, int dim, int vdim,
                                                                const int32_t* __restrict__ long_chunk0,
                                                                const int32_t* __restrict__ long_slot) {
  const int e = blockIdx.z, h = blockIdx.y, i = blockIdx.x * 256 + threadIdx.x;
  if (i >= dim * vdim) return;
  const int dp = pad_channels(dim), vp = pad_values(vdim), d = i / vdim;
  float* sp = state + (int64_t)long_slot[e] * slot_stride + (int64_t)h * dim * vdim + i;
  const int64_t cs = (int64_t)H * dp * vp, ts = (int64_t)H * dp;
  float* u = ws + (int64_t)h * dp * vp + (int64_t)d * vp + i % vdim;
  const float* tp = ws_total + (int64_t)h * dp + d;
  const int c_end = long_chunk0[e + 1];
  float S = *sp;
  for (int c0 = long_chunk0[e]; c0 < c_end; c0 += 8) {      // eight chunks' loads in flight before the first store
    float t[8], w[8];
#pragma unroll
    for (int k = 0; k < 8; ++k) {
      t[k] = c0 + k < c_end ? u[(c0 + k) * cs] : 0.f;
      w[k] = c0 + k < c_end ? tp[(c0 + k) * ts] : 0.f;
    }
#pragma unroll
    for (int k = 0; k < 8; ++k)
      if (c0 + k < c_end) {
        u[(c0 + k) * cs] = S;
        S = fmaf(w[k], S, t[k]);
      }
  }
  *sp = S;
}

// Eight waves.  Decays and rows: thread = (sub-block, channel).  Scores inside the sub-blocks: wave = (sub-block, half of the channels).
// Products: wave w takes 16 rows of the chunk and half of the value columns (NB blocks of 16); the two halves take the row blocks in
// opposite order, so that the two waves of a SIMD have the same number of sub-blocks between them.
template <typename A, int NB, int DP>
__global__ __launch_bounds__(512) void gated_chunk_out_kernel(GatedIn<A> in, const float* __restrict__ ws, float* __restrict__ o, int H,
                                                              int dim, int vdim, const int32_t* __restrict__ chunk_row0,
                                                              const int32_t* __restrict__ chunk_rows) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  constexpr int vp = 32 * NB, sv = stride_rows16(vp), sq = stride_rows16(DP), SS = kSub + 4;
  __shared__ __attribute__((aligned(16))) float s_own[2][kDecayChunk][SS];     // scores inside the sub-blocks, one part per half of the channels
  __shared__ float s_t[kSubs][DP];
  const int c = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, l15 = lane & 15, lg = lane >> 4;
  const int row0 = chunk_row0[c], n = chunk_rows[c];
  float *s_q = sm, *s_k = s_q + kDecayChunk * sq, *s_x = s_k + kDecayChunk * sq;   // s_x: the decays first, the values afterwards
  {
    const int sub = tid >> 7, d = tid & 127;
    float a[kSub], x[2][kSub];
    {
      const int64_t offs[2] = {in.q_off, in.k_off};
      load_channel<A, 2>(in, offs, (int64_t)h * dim + min(d, dim - 1), d < dim, row0, sub * kSub, n, a, x);
    }
    if (d < DP) {
#pragma unroll
      for (int i = 0; i < kSub; ++i) {
        const int row = sub * kSub + i;
        x[0][i] *= in.q_scale;
        s_q[row * sq + d] = x[0][i];
        s_k[row * sq + d] = x[1][i];
        s_x[row * sq + d] = a[i];
      }
    }
    __syncthreads();
    {   // lane: channels ch .. ch + NX - 1, keys lg, lg + 4, lg + 8, lg + 12 of the wave's sub-block
      constexpr int NX = DP / 32;
      const int base = (wave >> 1) * kSub, ch = (wave & 1) * (DP / 2) + l15 * NX;
      float kk[4][NX], w[4][NX], keep[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int jj = 0; jj < 4; ++jj)
#pragma unroll
        for (int y = 0; y < NX; ++y) {
          kk[jj][y] = s_k[(base + lg + 4 * jj) * sq + ch + y];
          w[jj][y] = 0.f;
        }
#pragma unroll
      for (int i = 0; i < kSub; ++i) {
        float qi[NX], ai[NX];
#pragma unroll
        for (int y = 0; y < NX; ++y) {
          qi[y] = s_q[(base + i) * sq + ch + y];
          ai[y] = s_x[(base + i) * sq + ch + y];
        }
#pragma unroll
        for (int jj = 0; jj < 4; ++jj) {
          if (4 * jj > i) continue;                  // keys 4 jj .. 4 jj + 3 all come after query i
          const bool first = i == lg + 4 * jj;       // the key's own token: its values join undecayed
          float p = 0.f;
#pragma unroll
          for (int y = 0; y < NX; ++y) {
            w[jj][y] = fmaf(w[jj][y], ai[y], first ? kk[jj][y] : 0.f);
            p = fmaf(w[jj][y], qi[y], p);
          }
          p = row16_sum(p);
          keep[jj] = i == l15 ? p : keep[jj];        // lane l15 of the DPP row keeps query l15
        }
      }
#pragma unroll
      for (int jj = 0; jj < 4; ++jj) s_own[wave & 1][base + l15][lg + 4 * jj] = keep[jj];
    }
    __syncthreads();                                 // the plain rows have been read
    if (d < DP) {
      float p = 1.f;
#pragma unroll
      for (int i = 0; i < kSub; ++i) {
        p *= a[i];
        s_q[(sub * kSub + i) * sq + d] = x[0][i] * p;
      }
      p = 1.f;
#pragma unroll
      for (int i = kSub - 1; i >= 0; --i) {
        s_k[(sub * kSub + i) * sq + d] = x[1][i] * p;
        p *= a[i];
      }
      s_t[sub][d] = p;
    }
    stage_rows<8>(in.proj, in.stride, in.v_off + (int64_t)h * vdim, row0, n, vdim, vp, s_x, sv, nullptr, tid, [](float v) { return v; });
  }
  __syncthreads();
  const int half = wave >> 2, rb = half ? 3 - (wave & 3) : wave & 3, i0 = rb * kSub, c0 = half * 16 * NB;
  if (i0 >= n) return;                               // no barrier follows
  const float* s_v = s_x;
  f32x4 acc[NB];
#pragma unroll
  for (int b = 0; b < NB; ++b) acc[b] = f32x4{0.f, 0.f, 0.f, 0.f};
  auto add_values = [&](float p, int j) {            // p: score of query l15 against key j (of this lane's four)
#pragma unroll
    for (int b = 0; b < NB; ++b) acc[b] = __builtin_amdgcn_mfma_f32_16x16x4f32(p, s_v[j * sv + c0 + 16 * b + l15], acc[b], 0, 0, 0);
  };
  {   // the sub-block's own keys; keys after the query have left zeros
    const f32x4 p0 = *reinterpret_cast<const f32x4*>(&s_own[0][i0 + l15][4 * lg]), p1 = *reinterpret_cast<const f32x4*>(&s_own[1][i0 + l15][4 * lg]);
#pragma unroll
    for (int r = 0; r < 4; ++r) add_values(p0[r] + p1[r], i0 + 4 * lg + r);
  }
  float q[DP / 4];                                   // the lane's part of the queries as A operands: row l15, channels lg, lg + 4, ...
#pragma unroll
  for (int s = 0; s < DP / 4; ++s) q[s] = s_q[(i0 + l15) * sq + lg + 4 * s];
  for (int jb = rb - 1; jb >= 0; --jb) {             // earlier sub-blocks, nearest first
    f32x4 s4[4] = {};
    const float* kr = s_k + (jb * kSub + l15) * sq + lg;
#pragma unroll
    for (int s = 0; s < DP / 4; ++s) s4[s & 3] = __builtin_amdgcn_mfma_f32_16x16x4f32(kr[4 * s], q[s], s4[s & 3], 0, 0, 0);
    const f32x4 p = (s4[0] + s4[1]) + (s4[2] + s4[3]);
#pragma unroll
    for (int r = 0; r < 4; ++r) add_values(p[r], jb * kSub + 4 * lg + r);
#pragma unroll
    for (int s = 0; s < DP / 4; ++s) q[s] *= s_t[jb][lg + 4 * s];
  }
  {   // what the tokens before the chunk left
    const float* S = ws + ((int64_t)c * H + h) * DP * vp + (int64_t)lg * vp + c0 + l15;
    constexpr int U = NB <= 4 ? 4 : 2;               // steps whose state values are fetched together, one group ahead of its use
    float cur[U][NB], nxt[U][NB];
    auto fetch = [&](int s0, float (*t)[NB]) {
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int b = 0; b < NB; ++b) t[u][b] = S[(int64_t)4 * (s0 + u) * vp + 16 * b];
    };
    fetch(0, cur);
#pragma unroll
    for (int s0 = 0; s0 < DP / 4; s0 += U) {
      if (s0 + U < DP / 4) fetch(s0 + U, nxt);
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int b = 0; b < NB; ++b) acc[b] = __builtin_amdgcn_mfma_f32_16x16x4f32(q[s0 + u], cur[u][b], acc[b], 0, 0, 0);
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int b = 0; b < NB; ++b) cur[u][b] = nxt[u][b];
    }
  }
#pragma unroll
  for (int b = 0; b < NB; ++b) {
    const int col = c0 + 16 * b + l15;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = i0 + 4 * lg + r;
      if (i < n && col < vdim) o[(int64_t)(row0 + i) * ((int64_t)H * vdim) + (int64_t)h * vdim + col] = acc[b][r];
    }
  }
}

static size_t gated_sum_lds(int dim, int vdim) {
  return (size_t)kDecayChunk * (stride_rows4(pad_channels(dim)) + stride_rows4(pad_values(vdim))) * sizeof(float);
}
static size_t gated_out_lds(int dim, int vdim) {
  const int sq = stride_rows16(pad_channels(dim)), sv = stride_rows16(pad_values(vdim));
  return (size_t)kDecayChunk * (2 * sq + std::max(sq, sv)) * sizeof(float);
}
constexpr size_t kGatedStatic = (2 * kDecayChunk * (kSub + 4) + kSubs * 128) * sizeof(float);   // the out kernel's static tables

}  // namespace pk

extern "C" {
using namespace pk;

int32_t pegainfer_gated_linear_chunked_ok(int32_t dim, int32_t vdim) {
  return dim > 0 && dim <= 128 && vdim > 0 && vdim <= 256 && gated_sum_lds(dim, vdim) + 4096 <= kLdsMost &&
         gated_out_lds(dim, vdim) + kGatedStatic <= kLdsMost;
}

int32_t pegainfer_gated_linear_fused_ok(int32_t rank, int32_t rank_stride, const void* w_up) {
  return rank > 0 && rank <= rank_stride && rank_stride <= kLowRank && rank_stride % 8 == 0 && host_aligned16(w_up);
}

int64_t pegainfer_gated_linear_workspace(int32_t n_chunks, int32_t heads, int32_t dim, int32_t vdim) {
  return (int64_t)n_chunks * heads * pad_channels(dim) * (pad_values(vdim) + 1);
}

pegainfer_status_t pegainfer_gated_linear(const pegainfer_gated_linear_desc* q, pegainfer_stream_t stream) {
  constexpr pegainfer_status_t bad = (pegainfer_status_t)hipErrorInvalidValue;
  if (!q) return bad;
  if (q->n_entries <= 0) return 0;
  const int H = q->heads, dim = q->dim, vdim = q->vdim;
  if (H <= 0 || H > 65535 || dim <= 0 || dim > 256 || vdim <= 0 || q->n_entries > 65535 || !(q->tau > 0.f) || !q->proj ||
      !q->state || !q->o || !q->entry_row0 || !q->entry_slot)
    return bad;
  const bool chunks = q->n_chunks > 0 && q->n_long > 0, fused = !q->z;
  if (fused && (chunks || !q->w_up || !pegainfer_gated_linear_fused_ok(q->rank, q->rank_stride, q->w_up))) return bad;
  if (chunks && (!pegainfer_gated_linear_chunked_ok(dim, vdim) || !q->workspace || !q->chunk_row0 || !q->chunk_rows || !q->long_chunk0 ||
                 !q->long_slot || q->scan_max <= 0 || q->n_long > 65535))
    return bad;
  hipStream_t st = as_stream(stream);
  bool ok = true;
  const bool known = by_dtype(q->dtype, [&](auto* t) {
    using A = std::remove_pointer_t<decltype(t)>;
    const GatedIn<A> in{static_cast<const A*>(q->proj), q->proj_stride, q->q_off, q->k_off, q->v_off, q->q_scale, q->z, q->z_stride,
                        static_cast<const A*>(q->z_bias), 1.0f / q->tau, static_cast<const A*>(q->w_up), q->low_off, q->rank, q->rank_stride};
    if (q->n_entries > (chunks ? q->n_long : 0))
      ok = by_slices(dim, [&](auto ns) {
        auto scan = [&](auto kern) {
          kern<<<dim3(ceil_div(vdim, kRecCols), H, q->n_entries), 256, 0, st>>>(in, q->state, q->slot_stride, q->o, H, dim, vdim, q->entry_row0,
                                                                                q->entry_slot, chunks ? q->scan_max : 0);
        };
        if (fused) scan(gated_scan_kernel<decltype(ns)::value, A, true>);
        else scan(gated_scan_kernel<decltype(ns)::value, A, false>);
      });
    if (!ok || !chunks) return;
    float* total = q->workspace + (int64_t)q->n_chunks * H * pad_channels(dim) * pad_values(vdim);
    const dim3 grid(q->n_chunks, H);
    auto sums = [&](auto kern) {
      kern<<<grid, 512, with_lds(kern, gated_sum_lds(dim, vdim)), st>>>(in, q->workspace, total, H, dim, vdim, q->chunk_row0, q->chunk_rows);
    };
    if (vdim <= 32) sums(gated_chunk_sum_kernel<A, 2>);
    else sums(gated_chunk_sum_kernel<A, 4>);
    gated_chunk_state_kernel<<<dim3(ceil_div((long)dim * vdim, 256), H, q->n_long), 256, 0, st>>>(
        q->workspace, total, q->state, q->slot_stride, H, dim, vdim, q->long_chunk0, q->long_slot);
    auto out = [&](auto kern) {
      kern<<<grid, 512, with_lds(kern, gated_out_lds(dim, vdim)), st>>>(in, q->workspace, q->o, H, dim, vdim, q->chunk_row0, q->chunk_rows);
    };
    auto by_channels = [&](auto nb) {
      constexpr int NB = decltype(nb)::value;
      if (dim <= 32) out(gated_chunk_out_kernel<A, NB, 32>);
      else if (dim <= 64) out(gated_chunk_out_kernel<A, NB, 64>);
      else out(gated_chunk_out_kernel<A, NB, 128>);
    };
    if (vdim <= 32) by_channels(std::integral_constant<int, 1>());
    else if (vdim <= 64) by_channels(std::integral_constant<int, 2>());
    else if (vdim <= 128) by_channels(std::integral_constant<int, 4>());
    else by_channels(std::integral_constant<int, 8>());
  });
  return known && ok ? (pegainfer_status_t)hipGetLastError() : bad;
}

}  // extern "C"
