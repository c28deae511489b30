// libti_short_conv: a causal convolution of a few taps over time on every channel of a step's rows, the rows before an entry's
// start taken from its per-request state, which then gets the last rows of the step.  All arithmetic is 32-bit.
//
//   out[m, c] = act(bias[c] + sum_j taps[c][j] u(position of m - (K - 1) + j)[c]),   act: silu or none
//
// u lies in rows of ld floats; state f32 [slots][K - 1][C] holds the K - 1 rows before each entry's start, zeros before a
// sequence's.  Every sum starts at zero and takes the taps in ascending order, then the bias: the same bits in every kernel here.
#include "common.h"
#include "short_conv.h"
#include "tinyinfer_kernels.h"

TI_ERROR_API

__device__ __forceinline__ float sc_finish(float acc, const float* __restrict__ bias, int c, int silu) {
  if (bias) acc += bias[c];
  return silu ? acc * __frcp_rn(1.0f + __expf(-acc)) : acc;
}

// any number of taps: a workgroup per row
__global__ void __launch_bounds__(256)
short_conv_kernel(const float* __restrict__ u, long ld, const float* __restrict__ taps, const float* __restrict__ bias, int silu,
                  const float* __restrict__ state, const int* __restrict__ entries, const int* __restrict__ entry_of,
                  const int* __restrict__ pos, float* __restrict__ out, int C, int K) {
  const int m = blockIdx.x;
  const int e = entry_of[m];
  const int row0 = entries[4 * e], start = entries[4 * e + 2], slot = entries[4 * e + 3];
  const int p = pos[m];
  const float* st_rows = state + (size_t)slot * (K - 1) * C;
  for (int c = threadIdx.x; c < C; c += 256) {
    float acc = 0.f;
    for (int j = 0; j < K; ++j) {
      const int s = p - (K - 1) + j;
      const float v = s >= start ? u[(size_t)(row0 + s - start) * ld + c] : st_rows[(size_t)(s - start + K - 1) * C + c];
      acc = fmaf(taps[(size_t)c * K + j], v, acc);
    }
    out[(size_t)m * C + c] = sc_finish(acc, bias, c, silu);
  }
}

// A few taps: a thread owns a channel and walks SHORT_ROWS rows of the step, the K - 1 rows behind it in registers; where an entry
// starts among them it takes them up anew.  One row an entry (`single`): the same thread moves the state on.
#define SHORT_ROWS 8
template <int K>
__global__ void __launch_bounds__(256)
short_conv_rows_kernel(const float* __restrict__ u, long ld, const float* __restrict__ taps, const float* __restrict__ bias, int silu,
                       float* state, const int* __restrict__ entries, const int* __restrict__ entry_of, const int* __restrict__ pos,
                       float* __restrict__ out, int M, int C, int rows_each, int single) {
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= C) return;
  float w[K], back[K];      // back[j]: the row K - 1 - j steps before the current one
#pragma unroll
  for (int j = 0; j < K; ++j) w[j] = taps[(size_t)c * K + j];
  const int m0 = blockIdx.x * rows_each;
  int e_now = -1;
  for (int m = m0; m < min(M, m0 + rows_each); ++m) {
    const int e = entry_of[m];
    const int row0 = entries[4 * e], start = entries[4 * e + 2], slot = entries[4 * e + 3];
    if (e != e_now) {
      const int p = pos[m];
#pragma unroll
      for (int j = 0; j < K - 1; ++j) {
        const int s = p - (K - 1) + j;
        back[j] = s >= start ? u[(size_t)(row0 + s - start) * ld + c] : state[((size_t)slot * (K - 1) + (s - start + K - 1)) * C + c];
      }
      e_now = e;
    } else {
#pragma unroll
      for (int j = 0; j < K - 1; ++j) back[j] = back[j + 1];
    }
    back[K - 1] = u[(size_t)m * ld + c];
    float acc = 0.f;
#pragma unroll
    for (int j = 0; j < K; ++j) acc = fmaf(w[j], back[j], acc);
    out[(size_t)m * C + c] = sc_finish(acc, bias, c, silu);
    if (single) {
#pragma unroll
      for (int j = 0; j < K - 1; ++j) state[((size_t)slot * (K - 1) + j) * C + c] = back[j + 1];
    }
  }
}

extern "C" int ti_short_conv(const float* u, long ld, const float* taps, const float* bias, int silu, float* state, const int* entries,
                             int n_entries, const int* entry_of, const int* pos, float* out, int M, int C, int K, hipStream_t stream) {
  TI_REQUIRE(M >= 0 && C > 0 && K >= 1 && n_entries >= 0 && ld >= C, "short_conv: bad sizes M=%d C=%d taps=%d rows of %ld", M, C, K, ld);
  TI_REQUIRE(K == 1 || state, "short_conv: %d taps need a state", K);
  if (M == 0) return 0;
  const int single = n_entries == M ? 1 : 0;      // one token an entry
  const int each = single ? 1 : SHORT_ROWS;
  const dim3 grid((M + each - 1) / each, (C + 255) / 256);
  bool moved = false;
  if (K >= 2 && K <= 4 && grid.y <= 65535) {
#define SHORT_CONV(N) short_conv_rows_kernel<N><<<grid, 256, 0, stream>>>(u, ld, taps, bias, silu, state, entries, entry_of, pos, out, M, C, each, single)
    if (K == 2) SHORT_CONV(2);
    else if (K == 3) SHORT_CONV(3);
    else SHORT_CONV(4);
#undef SHORT_CONV
    moved = single != 0;
  } else {
    short_conv_kernel<<<M, 256, 0, stream>>>(u, ld, taps, bias, silu, state, entries, entry_of, pos, out, C, K);
  }
  TI_LAUNCH_CHECK();
  if (K > 1 && n_entries > 0 && !moved) {
    const dim3 each_entry(n_entries, (C + 255) / 256 < 64 ? (C + 255) / 256 : 64);
    short_conv_state_kernel<<<each_entry, 256, 0, stream>>>(u, ld, state, entries, C, K);
    TI_LAUNCH_CHECK();
  }
  return 0;
}
