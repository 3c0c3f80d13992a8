// What the chunk forms of linear recurrences share (decay_attn.hip, gated_linear.hip): an entry's tokens in chunks of <= 64 that run side
// by side - every chunk's own contribution to the state, a walk over the chunks, every chunk's outputs - with fp32 rows in LDS and
// products on v_mfma_f32_16x16x4_f32 (lane l holds A[l % 16][l / 16] and B[l / 16][l % 16]; the result holds rows 4 (l / 16) + r,
// column l % 16).
#pragma once

#include "common.h"
#include "typed.h"
#include "pegainfer_kernels_blocks.h"

namespace pk {

constexpr int kDecayChunk = PEGAINFER_DECAY_CHUNK;
constexpr size_t kLdsMost = 159 * 1024;              // beside the kernels' static tables

// A chunk's rows of one head into LDS (fp32, activated), rows past `n` and columns past `dim` as zeros; TPR threads per row, four
// loads of eight values in flight per thread.
template <int TPR, typename A, typename Act>
__device__ __forceinline__ void stage_rows(const A* __restrict__ rows, int64_t row_stride, int64_t off, int row0, int n, int dim, int padded,
                                           float* dst, int stride, const float* row_factor, int tid, Act&& act) {
  const int j = tid / TPR, sub = tid % TPR;
  const A* src = rows + (int64_t)(row0 + min(j, n - 1)) * row_stride + off;
  const float f = j < n ? (row_factor ? row_factor[j] : 1.0f) : 0.f;
  const bool vec = (dim & 7) == 0 && (off & 7) == 0 && (row_stride & 7) == 0 && aligned16(rows);
  float* d = dst + j * stride;
  for (int c0 = sub * 8; c0 < padded; c0 += 32 * TPR) {
    float t[4][8];
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const int c = c0 + 8 * TPR * k;
      if (vec) {
        Vec8<A>::load(src + (c < dim ? c : 0), t[k]);      // always in bounds; what lies past dim or n becomes zero below
      } else {
#pragma unroll
        for (int u = 0; u < 8; ++u) t[k][u] = ld(src + (c + u < dim ? c + u : 0));
      }
    }
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const int c = c0 + 8 * TPR * k;
      if (c >= padded) break;
#pragma unroll
      for (int u = 0; u < 8; ++u) t[k][u] = j < n && c + u < dim ? act(t[k][u]) * f : 0.f;
      *reinterpret_cast<f32x4*>(d + c) = f32x4{t[k][0], t[k][1], t[k][2], t[k][3]};
      *reinterpret_cast<f32x4*>(d + c + 4) = f32x4{t[k][4], t[k][5], t[k][6], t[k][7]};
    }
  }
}

// LDS row strides (floats, multiples of 4): a fragment read of 4 rows x 16 columns wants rows 16 banks apart, one of 16 rows x 4
// columns (and one of rows 4 apart x 16 columns) wants an odd multiple of 4
__host__ __device__ constexpr int pad16(int n) { return (n + 15) & ~15; }
__host__ __device__ constexpr int stride_rows4(int n) { return pad16(n) % 32 == 0 ? pad16(n) + 16 : pad16(n); }
__host__ __device__ constexpr int stride_rows16(int n) { return pad16(n) + 4; }
// value columns of the workspace and of the staged values: what the kernels' 16-column blocks cover
__host__ __device__ constexpr int pad_values(int vdim) { return vdim <= 32 ? 32 : vdim <= 64 ? 64 : vdim <= 128 ? 128 : 256; }

// opt a kernel into more than the default LDS
template <typename K>
inline size_t with_lds(K kern, size_t bytes) {
  if (bytes > 48 * 1024)
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes);
  return bytes;
}

}  // namespace pk
