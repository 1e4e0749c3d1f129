// Short causal convolution over time per channel, with the last taps - 1 inputs of a sequence kept in its state slot
// (fp32 rows [taps - 1][channels], oldest first): y_t[c] = b[c] + sum_i w[i][c] x_(t - taps + 1 + i)[c], zeros before the
// sequence's start. A token reads the rows of its own portion and, for the first taps - 1 tokens of a portion, the slot;
// the slot is rewritten (short_conv_keep) in a later launch than every such read.
#pragma once
#include "common.h"

namespace vgate {

__device__ __forceinline__ float conv_ldx(const void* p, int64_t i, int f32) {
  return f32 ? reinterpret_cast<const float*>(p)[i] : bf2f(reinterpret_cast<const bf16_t*>(p)[i]);
}

// Channel c of token t (a row of x) of a portion that starts at row t0 and position pos0; w [taps][nw], the channel's
// column wc; kept: the slot's rows of nk channels, the channel's column kc.
__device__ __forceinline__ float short_conv_at(const void* x, int64_t ld, int f32, int c, const float* w, int nw, int wc, float b,
                                               const float* kept, int nk, int kc, int t, int t0, int pos0, int taps) {
  float y = b;
  for (int i0 = 0; i0 < taps; i0 += 4) {
    float v[4], ww[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {  // four taps' loads asked for together
      const int i = i0 + u, tt = t - (taps - 1) + i;
      v[u] = 0.f; ww[u] = 0.f;
      if (i < taps) {
        ww[u] = w[(int64_t)i * nw + wc];
        if (tt >= t0) v[u] = conv_ldx(x, (int64_t)tt * ld + c, f32);
        else if (pos0 > 0) v[u] = kept[(int64_t)(tt - t0 + taps - 1) * nk + kc];
      }
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) y = fmaf(ww[u], v[u], y);
  }
  return y;
}

// The slot's rows of one channel after a portion of rows [t0, t1): its last taps - 1 inputs (older ones move down; rows
// are read at a higher index than the one written, so ascending order is in place).
__device__ __forceinline__ void short_conv_keep(const void* x, int64_t ld, int f32, int c, float* kept, int nk, int kc, int t0,
                                                int t1, int pos0, int taps) {
  for (int j0 = 0; j0 < taps - 1; j0 += 4) {
    float v[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {  // four rows' loads asked for together
      const int tt = t1 - (taps - 1) + j0 + u;
      v[u] = 0.f;
      if (j0 + u < taps - 1) {
        if (tt >= t0) v[u] = conv_ldx(x, (int64_t)tt * ld + c, f32);
        else if (pos0 > 0) v[u] = kept[(int64_t)(tt - t0 + taps - 1) * nk + kc];
      }
    }
#pragma unroll
    for (int u = 0; u < 4; ++u)
      if (j0 + u < taps - 1) kept[(int64_t)(j0 + u) * nk + kc] = v[u];
  }
}

// Channel c of the eight tokens from row t on, at most four taps, without activation; the rows between the tokens are
// read once (values of rows at or past t1 mean nothing). F32: the rows' dtype.
template <bool F32>
__device__ __forceinline__ void short_conv_run8(const void* x, int64_t ld, int c, const float* w, int nw, int wc, const float* kept,
                                                int nk, int kc, int t, int t0, int t1, int pos0, int taps, float (&y)[8]) {
  float wl[4], v[11];
#pragma unroll
  for (int m = 0; m < 4; ++m) wl[m] = m >= 4 - taps ? w[(int64_t)max(m - (4 - taps), 0) * nw + wc] : 0.f;
#pragma unroll
  for (int m = 0; m < 11; ++m) v[m] = conv_ldx(x, (int64_t)min(max(t - 3 + m, t0), t1 - 1) * ld + c, F32 ? 1 : 0);
  if (t - 3 < t0) {  // (uniform) the portion's first tokens: from the slot
#pragma unroll
    for (int m = 0; m < 3; ++m) {
      const int r = t - 3 + m - t0 + taps - 1;
      if (t - 3 + m < t0) v[m] = (pos0 > 0 && r >= 0) ? kept[(int64_t)r * nk + kc] : 0.f;
    }
  }
#pragma unroll
  for (int u = 0; u < 8; ++u) {
    y[u] = 0.f;
#pragma unroll
    for (int m = 0; m < 4; ++m) y[u] = fmaf(wl[m], v[u + m], y[u]);
  }
}

__device__ __forceinline__ int seq_of_row(const int32_t* query_start, int S, int t) {
  int lo = 0, hi = S - 1;  // query_start[s] <= t < query_start[s + 1]
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (query_start[mid] <= t) lo = mid; else hi = mid - 1;
  }
  return lo;
}

}  // namespace vgate
