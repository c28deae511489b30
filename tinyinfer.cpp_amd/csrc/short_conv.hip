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

// A few taps: a thread owns N neighbouring channels (N 4: everything aligned to 16 bytes) of ROWS rows of the step; it asks for all
// the rows its sums read at once, those in front of an entry's start come from the state instead.  One row an entry (`single`):
// the same thread moves the state on.
template <int N> struct ScPiece { float v[N]; };
template <int N> __device__ __forceinline__ ScPiece<N> sc_load(const float* p) {
  ScPiece<N> x;
  if constexpr (N == 4) {
    const float4 a = *reinterpret_cast<const float4*>(p);
    x.v[0] = a.x; x.v[1] = a.y; x.v[2] = a.z; x.v[3] = a.w;
  } else {
    x.v[0] = *p;
  }
  return x;
}
template <int N> __device__ __forceinline__ void sc_store(float* p, const ScPiece<N>& x) {
  if constexpr (N == 4) *reinterpret_cast<float4*>(p) = make_float4(x.v[0], x.v[1], x.v[2], x.v[3]);
  else *p = x.v[0];
}
template <int K, int N, int ROWS>
__global__ void __launch_bounds__(256)
short_conv_rows_kernel(const float* __restrict__ u, long ld, const float* __restrict__ taps, const float* __restrict__ bias, int silu,
                       float* state, const int* __restrict__ entries, const int* __restrict__ entry_of, float* __restrict__ out, int M, int C,
                       int single) {
  const int c = (blockIdx.y * 256 + threadIdx.x) * N;
  if (c >= C) return;
  const int m0 = blockIdx.x * ROWS;
  ScPiece<N> rows[ROWS + K - 1];      // rows[i]: row m0 - (K - 1) + i of the step
#pragma unroll
  for (int i = 0; i < ROWS + K - 1; ++i) rows[i] = sc_load<N>(u + (size_t)min(max(m0 - (K - 1) + i, 0), M - 1) * ld + c);
  float w[N][K];
#pragma unroll
  for (int x = 0; x < N; ++x)
#pragma unroll
    for (int j = 0; j < K; ++j) w[x][j] = taps[(size_t)(c + x) * K + j];
  int first[ROWS], slots[ROWS];      // of the rows' entries: all asked for before the first is needed
#pragma unroll
  for (int i = 0; i < ROWS; ++i) first[i] = entry_of[min(m0 + i, M - 1)];
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
    const int e = first[i];
    first[i] = entries[4 * e];
    slots[i] = entries[4 * e + 3];
  }
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
    const int m = m0 + i, row0 = first[i];
    if (m >= M) break;
    float* st_rows = state + (size_t)slots[i] * (K - 1) * C + c;
    ScPiece<N> back[K];
#pragma unroll
    for (int j = 0; j < K; ++j) {
      const int r = m - (K - 1) + j;      // the step's row; in front of the entry's first one: row r - row0 + K - 1 of the state
      back[j] = rows[i + j];
      if (r < row0) back[j] = sc_load<N>(st_rows + (size_t)(r - row0 + K - 1) * C);
    }
    ScPiece<N> y;
#pragma unroll
    for (int x = 0; x < N; ++x) {
      float acc = 0.f;
#pragma unroll
      for (int j = 0; j < K; ++j) acc = fmaf(w[x][j], back[j].v[x], acc);
      y.v[x] = sc_finish(acc, bias, c + x, silu);
    }
    sc_store<N>(out + (size_t)m * C + c, y);
    if (single) {
#pragma unroll
      for (int j = 0; j < K - 1; ++j) sc_store<N>(st_rows + (size_t)j * C, back[j + 1]);
    }
  }
}

template <int K>
static void launch_rows(bool vec, bool single, const float* u, long ld, const float* taps, const float* bias, int silu, float* state, const int* entries,
                        const int* entry_of, float* out, int M, int C, hipStream_t stream) {
#define SHORT_CONV(N, ROWS)                                                                                                              \
  short_conv_rows_kernel<K, N, ROWS><<<dim3((M + ROWS - 1) / ROWS, (C + 256 * N - 1) / (256 * N)), 256, 0, stream>>>(u, ld, taps, bias, silu,   \
                                                                                                                  state, entries, entry_of, out, M, C, single)
  if (single) {
    SHORT_CONV(1, 1);
  } else if (vec) {
    SHORT_CONV(4, 8);
  } else {
    SHORT_CONV(1, 8);
  }
#undef SHORT_CONV
}

extern "C" int ti_short_conv(const float* u, long ld, const float* taps, const float* bias, int silu, float* state, const int* entries,
                             int n_entries, const int* entry_of, const int* pos, float* out, int M, int C, int K, hipStream_t stream) {
  TI_REQUIRE(M >= 0 && C > 0 && K >= 1 && n_entries >= 0 && ld >= C, "short_conv: bad sizes M=%d C=%d taps=%d rows of %ld", M, C, K, ld);
  TI_REQUIRE(K == 1 || state, "short_conv: %d taps need a state", K);
  if (M == 0) return 0;
  const int single = n_entries == M ? 1 : 0;      // one token an entry
  const bool vec = C % 4 == 0 && ld % 4 == 0 && (((uintptr_t)u | (uintptr_t)state | (uintptr_t)out) & 15) == 0;
  bool moved = false;
  if (K >= 2 && K <= 4 && (C + 255) / 256 <= 65535) {
    if (K == 2) launch_rows<2>(vec, single != 0, u, ld, taps, bias, silu, state, entries, entry_of, out, M, C, stream);
    else if (K == 3) launch_rows<3>(vec, single != 0, u, ld, taps, bias, silu, state, entries, entry_of, out, M, C, stream);
    else launch_rows<4>(vec, single != 0, u, ld, taps, bias, silu, state, entries, entry_of, out, M, C, stream);
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
