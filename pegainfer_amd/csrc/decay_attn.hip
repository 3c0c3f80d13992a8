// Linear attention with a constant decay per head over ragged batches, fp32 state and fp32 arithmetic throughout:
//     S <- g S + k v^T,   y = S^T q          q, k, v optionally through silu as they are read (rows of the projection)
// The decay does not depend on the token, so the recurrence has two equivalent forms.
//   decay_scan_kernel         token by token, the layout of recurrent.hip (a workgroup owns 16 value columns of one (entry, head), a
//                             column's state lies over the sixteen lanes of a DPP row): decoding and short portions
//   decay_chunk_sum_kernel    long portions, in chunks of <= 64 tokens that run side by side: U_c = sum_i g^(n-1-i) k_i v_i^T
//   decay_chunk_state_kernel  walks the chunks of an entry, S <- g^n S + U_c, and leaves the state BEFORE each chunk in U_c's place
//   decay_chunk_out_kernel    y_i = g^(i+1) S^T q_i + sum_{j <= i} g^(i-j) (q_i . k_j) v_j
// Products of the chunk form run on v_mfma_f32_16x16x4_f32 (exact fp32 products and sums).  Its operand layout: lane l holds
// A[l % 16][l / 16] and B[l / 16][l % 16]; the result holds rows 4 (l / 16) + r, column l % 16.  The score block is computed
// transposed (keys as rows), which leaves lane l with the scores of query l % 16 against keys 4 (l / 16) + r - the A operand of the
// second product when its step r takes keys r, 4 + r, 8 + r, 12 + r.
// Powers of the decay come from a table made once at load time in double precision.
#include <algorithm>

#include "common.h"
#include "typed.h"
#include "recurrent_core.h"
#include "chunk_core.h"
#include "pegainfer_kernels_blocks.h"

namespace pk {

template <typename A>
struct DecayIn {
  const A* proj;
  int64_t stride, q_off, k_off, v_off;
  int silu;
  __device__ __forceinline__ float act(float v) const { return silu ? silu_f(v) : v; }
};

template <int NS, typename A>
__global__ __launch_bounds__(256) void decay_scan_kernel(DecayIn<A> in, const float* __restrict__ decay_pow, int pow_n,
                                                         float* __restrict__ state, int64_t slot_stride, float* __restrict__ o, int H,
                                                         int dim, int vdim, const int32_t* __restrict__ entry_row0,
                                                         const int32_t* __restrict__ entry_slot, int scan_max) {
  constexpr int DP = kRecSlices * NS;
  __shared__ __attribute__((aligned(16))) float s_k[kRecTokens][DP], s_q[kRecTokens][DP];
  __shared__ float s_v[kRecTokens][kRecCols];
  const int e = blockIdx.z, h = blockIdx.y, col0 = blockIdx.x * kRecCols;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, r = lane & 15, cl = wave * 4 + (lane >> 4);
  const int col = col0 + cl;
  const int row0 = entry_row0[e], len = entry_row0[e + 1] - row0;
  if (scan_max > 0 && len > scan_max) return;      // the chunk form has this entry
  float* S_g = state + (int64_t)entry_slot[e] * slot_stride + (int64_t)h * dim * vdim;
  const float g = decay_pow[(int64_t)h * pow_n + 1];
  float S[NS];
#pragma unroll
  for (int i = 0; i < NS; ++i) {
    const int d = r * NS + i;
    S[i] = d < dim && col < vdim ? S_g[(int64_t)d * vdim + col] : 0.f;
  }
  RoundFetch<NS> nxt;
  auto fetch = [&](int t0) {
    const A* base = in.proj + (int64_t)(row0 + t0) * in.stride;
    const A *qb = base + in.q_off + (int64_t)h * dim, *kb = base + in.k_off + (int64_t)h * dim, *vb = base + in.v_off + (int64_t)h * vdim + col0;
    nxt.issue(min(kRecTokens, len - t0), tid, dim, [=](int tt, int d) { return ld(qb + (int64_t)tt * in.stride + d); },
              [=](int tt, int d) { return ld(kb + (int64_t)tt * in.stride + d); },
              [=](int tt, int c) { return col0 + c < vdim ? ld(vb + (int64_t)tt * in.stride + c) : 0.f; });
  };
  fetch(0);
  for (int t0 = 0; t0 < len; t0 += kRecTokens) {
    const int tc = min(kRecTokens, len - t0);
    __syncthreads();
    nxt.land(tid, s_q, s_k, s_v, [=](float x) { return in.act(x); });
    __syncthreads();
    if (t0 + kRecTokens < len) fetch(t0 + kRecTokens);
    float okeep = 0.f;
    for (int t4 = 0; t4 < tc; t4 += 4) {           // no sum of a token feeds the state: four read-outs are in flight together
#pragma unroll
      for (int uu = 0; uu < 4; ++uu) {
        const int tt = t4 + uu;
        const float a = tt < tc ? g : 1.0f, vv = s_v[tt][cl];   // rows past the entry's end: v = 0 and no decay leave S as it is
        float y0 = 0.f, y1 = 0.f;
#pragma unroll
        for (int i = 0; i < NS; ++i) {
          const float kk = s_k[tt][r * NS + i], qq = s_q[tt][r * NS + i];
          S[i] = fmaf(vv, kk, a * S[i]);
          if (i & 1) y1 = fmaf(S[i], qq, y1); else y0 = fmaf(S[i], qq, y0);
        }
        const float y = row16_sum(y0 + y1);
        okeep = tt == r ? y : okeep;
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

// U_c[d][col] = sum_i g^(n-1-i) k_i[d] v_i[col]; one workgroup per (chunk, head), a wave per block of 16 rows x (16 NB) columns of U
template <typename A, int NB>
__global__ __launch_bounds__(512) void decay_chunk_sum_kernel(DecayIn<A> in, const float* __restrict__ decay_pow, int pow_n,
                                                              float* __restrict__ ws, int H, int dim, int vdim,
                                                              const int32_t* __restrict__ chunk_row0,
                                                              const int32_t* __restrict__ chunk_rows) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  __shared__ float s_f[kDecayChunk];
  const int c = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, l15 = lane & 15, lg = lane >> 4;
  const int row0 = chunk_row0[c], n = chunk_rows[c];
  const int dp = pad16(dim), vp = pad_values(vdim), sk = stride_rows4(dim), sv = stride_rows4(vp);
  float *s_k = sm, *s_v = sm + kDecayChunk * sk;
  auto act = [=](float x) { return in.act(x); };
  if (tid < kDecayChunk) s_f[tid] = tid < n ? decay_pow[(int64_t)h * pow_n + n - 1 - tid] : 0.f;
  __syncthreads();
  stage_rows<8>(in.proj, in.stride, in.k_off + (int64_t)h * dim, row0, n, dim, dp, s_k, sk, s_f, tid, act);
  stage_rows<8>(in.proj, in.stride, in.v_off + (int64_t)h * vdim, row0, n, vdim, vp, s_v, sv, nullptr, tid, act);
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
      const float a = ka[4 * i * sk];
#pragma unroll
      for (int b = 0; b < NB; ++b) acc[b] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, vb[4 * i * sv + 16 * b], acc[b], 0, 0, 0);
    }
#pragma unroll
    for (int b = 0; b < NB; ++b)
#pragma unroll
      for (int r = 0; r < 4; ++r) U[(int64_t)(d0 + 4 * lg + r) * vp + c0 + 16 * b + l15] = acc[b][r];
  }
}

// One thread per element of the state: through the entry's chunks, the state before each left in U's place.
__global__ __launch_bounds__(256) void decay_chunk_state_kernel(const float* __restrict__ decay_pow, int pow_n, float* ws,
                                                                float* __restrict__ state, int64_t slot_stride, int H, int dim, int vdim,
                                                                const int32_t* __restrict__ chunk_rows,
                                                                const int32_t* __restrict__ long_chunk0,
                                                                const int32_t* __restrict__ long_slot) {
  const int e = blockIdx.z, h = blockIdx.y, i = blockIdx.x * 256 + threadIdx.x;
  if (i >= dim * vdim) return;
  const int dp = pad16(dim), vp = pad_values(vdim);
  float* sp = state + (int64_t)long_slot[e] * slot_stride + (int64_t)h * dim * vdim + i;
  const int64_t cs = (int64_t)H * dp * vp;
  float* u = ws + (int64_t)h * dp * vp + (int64_t)(i / vdim) * vp + i % vdim;
  const int c_end = long_chunk0[e + 1];
  float S = *sp;
  for (int c0 = long_chunk0[e]; c0 < c_end; c0 += 8) {      // eight chunks' loads in flight before the first store
    float t[8];
#pragma unroll
    for (int k = 0; k < 8; ++k) t[k] = c0 + k < c_end ? u[(c0 + k) * cs] : 0.f;
#pragma unroll
    for (int k = 0; k < 8; ++k)
      if (c0 + k < c_end) {
        u[(c0 + k) * cs] = S;
        S = fmaf(decay_pow[(int64_t)h * pow_n + chunk_rows[c0 + k]], S, t[k]);
      }
  }
  *sp = S;
}

// Eight waves: wave w takes 16 rows of the chunk and half of the value columns (NB blocks of 16); the two halves take the row blocks
// in opposite order, so that the two waves of a SIMD have the same number of key blocks between them.
template <typename A, int NB>
__global__ __launch_bounds__(512) void decay_chunk_out_kernel(DecayIn<A> in, const float* __restrict__ decay_pow, int pow_n,
                                                              const float* __restrict__ ws, float* __restrict__ o, int H, int dim,
                                                              int vdim, const int32_t* __restrict__ chunk_row0,
                                                              const int32_t* __restrict__ chunk_rows) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  __shared__ float s_pow[kDecayChunk + 1];
  constexpr int vp = 32 * NB, sv = stride_rows16(vp);
  const int c = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, l15 = lane & 15, lg = lane >> 4;
  const int row0 = chunk_row0[c], n = chunk_rows[c];
  const int dp = pad16(dim), sq = stride_rows16(dim);
  float *s_q = sm, *s_k = s_q + kDecayChunk * sq, *s_v = s_k + kDecayChunk * sq;
  const int half = wave >> 2, rb = half ? 3 - (wave & 3) : wave & 3, i0 = rb * 16, c0 = half * 16 * NB;
  auto act = [=](float x) { return in.act(x); };
  if (tid <= kDecayChunk) s_pow[tid] = tid <= n ? decay_pow[(int64_t)h * pow_n + tid] : 0.f;
  stage_rows<8>(in.proj, in.stride, in.q_off + (int64_t)h * dim, row0, n, dim, dp, s_q, sq, nullptr, tid, act);
  stage_rows<8>(in.proj, in.stride, in.k_off + (int64_t)h * dim, row0, n, dim, dp, s_k, sq, nullptr, tid, act);
  stage_rows<8>(in.proj, in.stride, in.v_off + (int64_t)h * vdim, row0, n, vdim, vp, s_v, sv, nullptr, tid, act);
  __syncthreads();
  if (i0 >= n) return;                               // no barrier follows
  const int my_i = i0 + l15;                         // the query this lane holds scores of
  f32x4 acc[NB];
#pragma unroll
  for (int b = 0; b < NB; ++b) acc[b] = f32x4{0.f, 0.f, 0.f, 0.f};
  const float* qr = s_q + my_i * sq + lg;
  {   // what the tokens before the chunk left; rows dim .. dp - 1 and columns vdim .. vp - 1 of the state before a chunk are zeros
    const float f = s_pow[min(my_i + 1, n)];         // rows past n are not stored
    const float* S = ws + ((int64_t)c * H + h) * dp * vp + (int64_t)lg * vp + c0 + l15;
    constexpr int U = NB <= 4 ? 4 : 2;               // steps whose state values are fetched together, one group ahead of its use
    float cur[U][NB], nxt[U][NB];
    auto fetch = [&](int d0, float (*t)[NB]) {
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int b = 0; b < NB; ++b) t[u][b] = S[(int64_t)(d0 + 4 * u) * vp + 16 * b];
    };
    fetch(0, cur);
    for (int d0 = 0; d0 < dp; d0 += 4 * U) {
      fetch(min(d0 + 4 * U, dp - 4 * U), nxt);
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const float a = qr[d0 + 4 * u] * f;
#pragma unroll
        for (int b = 0; b < NB; ++b) acc[b] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, cur[u][b], acc[b], 0, 0, 0);
      }
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int b = 0; b < NB; ++b) cur[u][b] = nxt[u][b];
    }
  }
  for (int jb = 0; jb <= rb; ++jb) {                 // the chunk's own tokens, 16 keys at a time
    f32x4 s0 = {0.f, 0.f, 0.f, 0.f}, s1 = s0, s2 = s0, s3 = s0;
    const float* kr = s_k + (jb * 16 + l15) * sq + lg;
    for (int d = 0; d < dp; d += 16) {
      s0 = __builtin_amdgcn_mfma_f32_16x16x4f32(kr[d], qr[d], s0, 0, 0, 0);
      s1 = __builtin_amdgcn_mfma_f32_16x16x4f32(kr[d + 4], qr[d + 4], s1, 0, 0, 0);
      s2 = __builtin_amdgcn_mfma_f32_16x16x4f32(kr[d + 8], qr[d + 8], s2, 0, 0, 0);
      s3 = __builtin_amdgcn_mfma_f32_16x16x4f32(kr[d + 12], qr[d + 12], s3, 0, 0, 0);
    }
    s0 = (s0 + s1) + (s2 + s3);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int j = jb * 16 + 4 * lg + r;
      const float p = j <= my_i ? s0[r] * s_pow[min(my_i - j, n)] : 0.f;
#pragma unroll
      for (int b = 0; b < NB; ++b) acc[b] = __builtin_amdgcn_mfma_f32_16x16x4f32(p, s_v[j * sv + c0 + 16 * b + l15], acc[b], 0, 0, 0);
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

static size_t decay_sum_lds(int dim, int vdim) { return (size_t)kDecayChunk * (stride_rows4(dim) + stride_rows4(pad_values(vdim))) * sizeof(float); }
static size_t decay_out_lds(int dim, int vdim) { return (size_t)kDecayChunk * (2 * stride_rows16(dim) + stride_rows16(pad_values(vdim))) * sizeof(float); }

}  // namespace pk

extern "C" {
using namespace pk;

int32_t pegainfer_decay_attention_chunked_ok(int32_t dim, int32_t vdim) {
  return dim > 0 && vdim > 0 && vdim <= 256 && decay_sum_lds(dim, vdim) <= kLdsMost && decay_out_lds(dim, vdim) <= kLdsMost;
}

int64_t pegainfer_decay_attention_workspace(int32_t n_chunks, int32_t heads, int32_t dim, int32_t vdim) {
  return (int64_t)n_chunks * heads * pad16(dim) * pad_values(vdim);
}

pegainfer_status_t pegainfer_decay_attention(const pegainfer_decay_attention_desc* q, pegainfer_stream_t stream) {
  constexpr pegainfer_status_t bad = (pegainfer_status_t)hipErrorInvalidValue;
  if (!q) return bad;
  if (q->n_entries <= 0) return 0;
  const int H = q->heads, dim = q->dim, vdim = q->vdim;
  if (H <= 0 || H > 65535 || dim <= 0 || dim > 256 || vdim <= 0 || q->n_entries > 65535 || q->pow_n < 2 || !q->decay_pow || !q->proj ||
      !q->state || !q->o)
    return bad;
  const bool chunks = q->n_chunks > 0 && q->n_long > 0;
  if (chunks && (!pegainfer_decay_attention_chunked_ok(dim, vdim) || q->pow_n <= kDecayChunk || !q->workspace || !q->chunk_row0 ||
                 !q->chunk_rows || !q->long_chunk0 || !q->long_slot || q->scan_max <= 0 || q->n_long > 65535))
    return bad;
  hipStream_t st = as_stream(stream);
  bool ok = true;
  const bool known = by_dtype(q->dtype, [&](auto* t) {
    using A = std::remove_pointer_t<decltype(t)>;
    const DecayIn<A> in{static_cast<const A*>(q->proj), q->proj_stride, q->q_off, q->k_off, q->v_off, q->silu};
    if (q->n_entries > (chunks ? q->n_long : 0))
      ok = by_slices(dim, [&](auto ns) {
        decay_scan_kernel<decltype(ns)::value, A><<<dim3(ceil_div(vdim, kRecCols), H, q->n_entries), 256, 0, st>>>(
            in, q->decay_pow, q->pow_n, q->state, q->slot_stride, q->o, H, dim, vdim, q->entry_row0, q->entry_slot, chunks ? q->scan_max : 0);
      });
    if (!ok || !chunks) return;
    auto sums = [&](auto kern) {
      kern<<<dim3(q->n_chunks, H), 512, with_lds(kern, decay_sum_lds(dim, vdim)), st>>>(in, q->decay_pow, q->pow_n, q->workspace, H, dim, vdim,
                                                                                  q->chunk_row0, q->chunk_rows);
    };
    if (vdim <= 32) sums(decay_chunk_sum_kernel<A, 2>);
    else sums(decay_chunk_sum_kernel<A, 4>);
    decay_chunk_state_kernel<<<dim3(ceil_div((long)dim * vdim, 256), H, q->n_long), 256, 0, st>>>(
        q->decay_pow, q->pow_n, q->workspace, q->state, q->slot_stride, H, dim, vdim, q->chunk_rows, q->long_chunk0, q->long_slot);
    auto out = [&](auto kern) {
      kern<<<dim3(q->n_chunks, H), 512, with_lds(kern, decay_out_lds(dim, vdim)), st>>>(in, q->decay_pow, q->pow_n, q->workspace, q->o, H, dim, vdim,
                                                                                  q->chunk_row0, q->chunk_rows);
    };
    if (vdim <= 32) out(decay_chunk_out_kernel<A, 1>);
    else if (vdim <= 64) out(decay_chunk_out_kernel<A, 2>);
    else if (vdim <= 128) out(decay_chunk_out_kernel<A, 4>);
    else out(decay_chunk_out_kernel<A, 8>);
  });
  return known && ok ? (pegainfer_status_t)hipGetLastError() : bad;
}

}  // extern "C"
