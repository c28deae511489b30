// The state of a short convolution over time behind a step: shared by the convolution on its own and the kernels that take it in.
#pragma once
#include "common.h"

// the state after the step: the last K - 1 rows of the sequence so far.  A thread owns a channel and walks the
// state's rows upwards: what it still reads of the old state lies above what it has written.
static __global__ void __launch_bounds__(256)
short_conv_state_kernel(const float* __restrict__ u, long ld, float* __restrict__ state, const int* __restrict__ entries, int C, int K) {
  const int e = blockIdx.x;
  const int row0 = entries[4 * e], n = entries[4 * e + 1], slot = entries[4 * e + 3];
  float* st_rows = state + (size_t)slot * (K - 1) * C;
  for (int c = blockIdx.y * 256 + threadIdx.x; c < C; c += gridDim.y * 256)
    for (int i = 0; i < K - 1; ++i) {
      const int r = n - (K - 1) + i;      // the step's row that lands here; below zero: a row the state already holds
      st_rows[(size_t)i * C + c] = r >= 0 ? u[(size_t)(row0 + r) * ld + c] : st_rows[(size_t)(i + n) * C + c];
    }
}
