// A product of few rows inside a block: 64 columns of R rows, PARTS threads a column.  Each thread
// takes 32 of every PARTS * 32 elements of the sum and asks for all their weights at once, from
// clamped places, so that none waits behind a branch and a step of few rows is not a chain of trips
// to memory; x goes through LDS (element by element of the sum, the R rows of one together), the
// parts add up through LDS.
#pragma once

#include "common.h"

namespace ei {

constexpr int kFewCols = 64;      // columns of a block
constexpr int kFewK = 32;         // elements of the sum a thread takes at a time

template <int R, int PARTS>
struct FewRows {
  static constexpr int kThreads = kFewCols * PARTS;
  static constexpr int kTile = PARTS * kFewK;
  float xs[kTile][R] __attribute__((aligned(16)));
  float sums[PARTS][R][kFewCols];

  // sums over i < K of x(r, i) * w[i * stride + j], j the thread's column (clamped to `last_col`
  // for the loads); x(r, i) is asked for r < R and i < K only.  Every thread of the block calls it;
  // `total(r, column)` may be read afterwards.
  template <typename TW, typename X>
  __device__ __forceinline__ void product(const TW* __restrict__ w, size_t stride, int K, int j,
                                          int last_col, X x) {
    const int col = threadIdx.x % kFewCols, part = threadIdx.x / kFewCols;
    const int at = j < last_col ? j : last_col;
    float acc[R];
#pragma unroll
    for (int r = 0; r < R; ++r) acc[r] = 0.f;
    for (int k0 = 0; k0 < K; k0 += kTile) {
      TW wv[kFewK];
#pragma unroll
      for (int u = 0; u < kFewK; ++u)
        wv[u] = w[static_cast<size_t>(min(k0 + part * kFewK + u, K - 1)) * stride + at];
      if (k0 > 0) __syncthreads();                 // the last tile has been used
      const int kn = min(kTile, K - k0);
      for (int idx = threadIdx.x; idx < R * kTile; idx += kThreads) {
        const int r = idx / kTile, k = idx % kTile;
        xs[k][r] = k < kn ? x(r, k0 + k) : 0.f;    // (beyond the end: zeros for the clamped weights)
      }
      __syncthreads();
#pragma unroll
      for (int u = 0; u < kFewK; ++u) {
        const float wu = to_f32<TW>(wv[u]);
#pragma unroll
        for (int r = 0; r < R; ++r) acc[r] = fmaf(xs[part * kFewK + u][r], wu, acc[r]);
      }
    }
#pragma unroll
    for (int r = 0; r < R; ++r) sums[part][r][col] = acc[r];
    __syncthreads();
  }

  __device__ __forceinline__ float total(int r, int col) const {
    float v = sums[0][r][col];
#pragma unroll
    for (int p = 1; p < PARTS; ++p) v += sums[p][r][col];
    return v;
  }
};

}  // namespace ei
