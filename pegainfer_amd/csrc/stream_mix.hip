// Several residual streams with learned mixing (hyper-connections), fp32 streams in a bf16 and an fp32 storage instance of
// weights and activations.
//
// A token's row holds its S streams back to back, [S][d] fp32.  Between two sublayers ONE launch (one workgroup per row) does
// everything that touches the streams: the sublayer that ends writes its output into all of them, every new stream a mix of the
// old ones, and the sublayer that begins reads its weighted sum of the new streams through its norm:
//     X_t <- sum_s M[s, t] X_s + mult * b[t] * y            (all t from the old streams)
//     u    = sum_s a[s] X_s;   h = norm(u) * gain           (layer norm without bias, or RMS norm)
// The same kernel opens a model (every stream starts as the token's embedding row times a constant) and closes it (a plain sum of
// the streams, normed, on the rows whose logits are wanted).  A thread owns columns, so it holds all S values of a column while it
// mixes them: each stream is read and written once.  The row's u waits in LDS between the sums and the norm.
#include <algorithm>

#include "common.h"
#include "typed.h"
#include "pegainfer_kernels_blocks.h"

namespace pk {

template <typename A>
struct StreamMix {
  const float* x_in;           // [rows][S][d], or NULL: the embedding
  const A* embed; const uint32_t* ids; float embed_scale;
  const int32_t* row_index;    // source row of an output row (NULL: itself)
  const A* y; int64_t y_stride;
  const A *mix, *out_w;        // [S][S] from, to; [S]
  float mult;
  float* x_out;
  float* sum_out;              // the plain sum of the new streams
  const A* read_w;             // [S]; NULL: ones
  const A* gain; A* n_out;
  float eps;
  int layer_norm;              // 0: RMS norm
};

// MS: the streams a thread's registers hold (S <= MS).  VEC: d, strides and pointers allow four values per load.  WAVES: of the
// workgroup - a step of few rows (decoding) spreads a row over more of them.
template <typename A, int MS, bool VEC, int WAVES>
__global__ __launch_bounds__(64 * WAVES) void stream_mix_kernel(StreamMix<A> p, int S, int d) {
  extern __shared__ __attribute__((aligned(16))) float s_u[];   // [d] when a norm follows
  __shared__ float s_mix[MS * MS], s_out[MS], s_read[MS], red[WAVES];
  constexpr int V = VEC ? 4 : 1, N = 64 * WAVES;
  const int row = blockIdx.x, tid = threadIdx.x;
  const int64_t src = p.row_index ? p.row_index[row] : row;
  const float* xr = p.x_in ? p.x_in + src * S * d : nullptr;
  const A* er = p.x_in ? nullptr : p.embed + (int64_t)p.ids[src] * d;
  float x[MS][V], y[V];
  auto load = [&](int i) {
    if (xr) {
#pragma unroll
      for (int s = 0; s < MS; ++s)
        if (s < S) {
          if constexpr (VEC) ld4(xr + (int64_t)s * d + i, x[s]); else x[s][0] = xr[(int64_t)s * d + i];
        }
    } else {
      float e[V];
      if constexpr (VEC) ld4(er + i, e); else e[0] = ld(er + i);
#pragma unroll
      for (int s = 0; s < MS; ++s)
#pragma unroll
        for (int u = 0; u < V; ++u) x[s][u] = e[u] * p.embed_scale;
    }
    if (p.y) {
      const A* yr = p.y + (int64_t)row * p.y_stride;
      if constexpr (VEC) ld4(yr + i, y); else y[0] = ld(yr + i);
    }
  };
  if (tid * V < d) load(tid * V);            // in flight while the coefficients arrive
  if (p.y) {
    for (int i = tid; i < S * S; i += N) s_mix[i] = ld(p.mix + i);
    if (tid < S) s_out[tid] = p.mult * ld(p.out_w + tid);
  }
  if (tid < S) s_read[tid] = p.read_w ? ld(p.read_w + tid) : 1.0f;
  __syncthreads();
  float total = 0.f;
  for (int i = tid * V; i < d; i += N * V) {
    float n[MS][V];
    if (i != tid * V) load(i);
    if (p.y) {
#pragma unroll
      for (int t = 0; t < MS; ++t)
        if (t < S) {
          const float b = s_out[t];
#pragma unroll
          for (int u = 0; u < V; ++u) n[t][u] = b * y[u];
#pragma unroll
          for (int s = 0; s < MS; ++s)
            if (s < S) {
              const float m = s_mix[s * S + t];
#pragma unroll
              for (int u = 0; u < V; ++u) n[t][u] = fmaf(m, x[s][u], n[t][u]);
            }
        }
    } else {
#pragma unroll
      for (int s = 0; s < MS; ++s)
#pragma unroll
        for (int u = 0; u < V; ++u) n[s][u] = x[s][u];
    }
    float uu[V], sum[V];
#pragma unroll
    for (int u = 0; u < V; ++u) { uu[u] = 0.f; sum[u] = 0.f; }
#pragma unroll
    for (int s = 0; s < MS; ++s)
      if (s < S) {
        if (p.x_out) {
          float* o = p.x_out + ((int64_t)row * S + s) * d + i;
          if constexpr (VEC) st4(o, n[s]); else *o = n[s][0];
        }
        const float a = s_read[s];
#pragma unroll
        for (int u = 0; u < V; ++u) { uu[u] = fmaf(a, n[s][u], uu[u]); sum[u] += n[s][u]; }
      }
    if (p.sum_out) {
      if constexpr (VEC) st4(p.sum_out + (int64_t)row * d + i, sum); else p.sum_out[(int64_t)row * d + i] = sum[0];
    }
    if (p.n_out) {
#pragma unroll
      for (int u = 0; u < V; ++u) {
        s_u[i + u] = uu[u];                  // read back by this thread only: no barrier needed
        total += p.layer_norm ? uu[u] : uu[u] * uu[u];
      }
    }
  }
  if (!p.n_out) return;                      // uniform over the grid
  total = block_sum<WAVES>(total, red);
  float mean = 0.f, var = total / (float)d;
  if (p.layer_norm) {
    mean = total / (float)d;
    float sq = 0.f;
    for (int i = tid * V; i < d; i += N * V)
#pragma unroll
      for (int u = 0; u < V; ++u) {
        const float z = s_u[i + u] - mean;
        sq = fmaf(z, z, sq);
      }
    var = block_sum<WAVES>(sq, red) / (float)d;
  }
  const float inv = 1.0f / sqrtf(var + p.eps);
  for (int i = tid * V; i < d; i += N * V) {
    float g[V], o[V];
    if constexpr (VEC) ld4(p.gain + i, g); else g[0] = ld(p.gain + i);
#pragma unroll
    for (int u = 0; u < V; ++u) o[u] = (s_u[i + u] - mean) * inv * g[u];
    if constexpr (VEC) st4(p.n_out + (int64_t)row * d + i, o); else st(p.n_out + (int64_t)row * d + i, o[0]);
  }
}

}  // namespace pk

extern "C" {
using namespace pk;

pegainfer_status_t pegainfer_stream_mix(const pegainfer_stream_mix_desc* q, pegainfer_stream_t stream) {
  constexpr pegainfer_status_t bad = (pegainfer_status_t)hipErrorInvalidValue;
  if (!q) return bad;
  if (q->rows <= 0) return 0;
  const int S = q->streams, d = q->d;
  if (S < 1 || S > 16 || d <= 0 || d > 32768 || (!q->x_in && (!q->embed || !q->token_ids)) || (q->y && (!q->mix || !q->out_w)) ||
      (!q->x_out && !q->sum_out && !q->n_out) || (q->n_out && !q->gain) || (q->row_index && q->x_out && q->x_out == q->x_in) ||
      (q->norm_kind != PEGAINFER_NORM_RMS && q->norm_kind != PEGAINFER_NORM_LAYER))
    return bad;
  if (!by_dtype(q->dtype, [&](auto* t) {
        using A = std::remove_pointer_t<decltype(t)>;
        StreamMix<A> p{q->x_in, static_cast<const A*>(q->embed), q->token_ids, q->embed_scale, q->row_index,
                       static_cast<const A*>(q->y), q->y_row_stride, static_cast<const A*>(q->mix), static_cast<const A*>(q->out_w), q->mult,
                       q->x_out, q->sum_out, static_cast<const A*>(q->read_w), static_cast<const A*>(q->gain), static_cast<A*>(q->n_out),
                       q->eps, q->norm_kind == PEGAINFER_NORM_LAYER};
        const bool vec = d % 4 == 0 && q->y_row_stride % 4 == 0 && host_aligned16(q->x_in) && host_aligned16(q->embed) &&
                         host_aligned16(q->y) && host_aligned16(q->x_out) && host_aligned16(q->sum_out) && host_aligned16(q->gain) &&
                         host_aligned16(q->n_out);
        const size_t lds = q->n_out ? (size_t)d * sizeof(float) : 0;
        auto launch = [&](auto kern, int threads) {
          if (lds > 48 * 1024)
            (void)hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
          kern<<<q->rows, threads, lds, as_stream(stream)>>>(p, S, d);
        };
        auto by_streams = [&](auto v, auto waves) {
          constexpr bool VEC = decltype(v)::value;
          constexpr int W = decltype(waves)::value;
          if (S <= 2) launch(stream_mix_kernel<A, 2, VEC, W>, 64 * W);
          else if (S <= 4) launch(stream_mix_kernel<A, 4, VEC, W>, 64 * W);
          else launch(stream_mix_kernel<A, 16, VEC, 4>, 256);   // its registers fit four waves only
        };
        const bool wide = q->rows < 128 && d > 1024;
        if (vec && wide) by_streams(std::true_type(), std::integral_constant<int, 16>());
        else if (vec) by_streams(std::true_type(), std::integral_constant<int, 4>());
        else by_streams(std::false_type(), std::integral_constant<int, 4>());
      }))
    return bad;
  return (pegainfer_status_t)hipGetLastError();
}

}  // extern "C"
