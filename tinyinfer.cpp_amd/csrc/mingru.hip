// libti_mingru: an element-wise gated recurrence whose gate and candidate read the current token only (a minimal GRU).
// From the 32-bit sums of one stacked projection with columns [z | x | g] of `width` entries each and biases on z and x:
//   s = sigmoid(z + bz);  u = x + bx;  c = u + 1/2 where u >= 0, sigmoid(u) where u < 0
//   S_t = (1 - s) S_(t-1) + s c;       out_t = S_t g sigmoid(g)
// S (width floats a request) lives in the request's state slot; all arithmetic is 32-bit, the output is rounded once.
//
//   mingru_step     a thread per (entry, channel) walks the entry's tokens, eight tokens' columns in flight at a time
//   mingru_chunks   long portions in chunks side by side: a chunk is the affine map S -> A S + B with A = prod (1 - s);
//                   the first launch leaves every chunk's (A, B), the second folds the maps in front of a chunk into its
//                   start state and walks the chunk with outputs.  In both a workgroup owns 64 channels and its four
//                   wavefronts a quarter of the tokens each, composed through LDS
#include "common.h"
#include "tinyinfer_kernels.h"

TI_ERROR_API

#define MG_SUB 16                    // tokens a wavefront takes of a block
#define MG_BLOCK (4 * MG_SUB)        // tokens a workgroup takes at a time

// sigmoid(a) and 1 - sigmoid(a), neither by a difference of close numbers.  FAST: the hardware's exponential and
// reciprocal (about 1e-7 of the value), for results that are rounded to bfloat16 behind the recurrence
template <bool FAST>
__device__ __forceinline__ void mg_sigmoid(float a, float* s, float* rest) {
  const float e = FAST ? __builtin_amdgcn_exp2f(-fabsf(a) * 1.4426950408889634f) : expf(-fabsf(a));
  const float r = FAST ? __builtin_amdgcn_rcpf(1.0f + e) : 1.0f / (1.0f + e);
  const float small = e * r;
  *s = a >= 0.f ? r : small;
  *rest = a >= 0.f ? small : r;
}

// the step's map: S -> keep S + put
template <bool FAST>
__device__ __forceinline__ void mg_map(float z, float x, float bz, float bx, float* keep, float* put) {
  float s, rest, us, ur;
  mg_sigmoid<FAST>(z + bz, &s, &rest);
  const float u = x + bx;
  mg_sigmoid<FAST>(u, &us, &ur);
  *keep = rest;
  *put = s * (u >= 0.f ? u + 0.5f : us);
}

template <bool FAST>
__device__ __forceinline__ float mg_out(float S, float g) {
  float s, rest;
  mg_sigmoid<FAST>(g, &s, &rest);
  return S * (g * s);
}

template <typename T>
__global__ void __launch_bounds__(256)
mingru_step_kernel(const float* __restrict__ proj, int ldp, int off_z, int off_x, int off_g, const float* __restrict__ bias_z,
                   const float* __restrict__ bias_x, float* __restrict__ state, long slot_stride, const int* __restrict__ entry_meta,
                   T* __restrict__ out, int W) {
  constexpr bool FAST = sizeof(T) == 2;
  constexpr int U = 8;
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= W) return;
  const int row0 = entry_meta[4 * blockIdx.y], n = entry_meta[4 * blockIdx.y + 1], slot = entry_meta[4 * blockIdx.y + 3];
  float* const cell = state + (size_t)slot * slot_stride + c;
  const float bz = bias_z[c], bx = bias_x[c];
  float S = *cell;
  for (int t0 = 0; t0 < n; t0 += U) {
    float z[U], x[U], g[U];
#pragma unroll
    for (int i = 0; i < U; ++i) {
      const float* row = proj + (size_t)(row0 + min(t0 + i, n - 1)) * ldp + c;      // (rows beyond the last: the last one again)
      z[i] = row[off_z];
      x[i] = row[off_x];
      g[i] = row[off_g];
    }
#pragma unroll
    for (int i = 0; i < U; ++i)
      if (t0 + i < n) {
        float keep, put;
        mg_map<FAST>(z[i], x[i], bz, bx, &keep, &put);
        S = fmaf(keep, S, put);
        st<T>(out + (size_t)(row0 + t0 + i) * W + c, mg_out<FAST>(S, g[i]));
      }
  }
  *cell = S;
}

// PASS 1: the chunk's map to maps [chunk][2][W]; an entry's first chunk also leaves the slot's state in start [entry][W].
// PASS 2: the maps of the entry's chunks in front of this one and that state give the chunk's start state; outputs; the entry's
// last chunk writes the slot (which no chunk of this launch reads, but one that is its entry's only one, itself).
template <typename T, int PASS>
__global__ void __launch_bounds__(256)
mingru_chunk_kernel(const float* __restrict__ proj, int ldp, int off_z, int off_x, int off_g, const float* __restrict__ bias_z,
                    const float* __restrict__ bias_x, float* __restrict__ state, long slot_stride,
                    const int* __restrict__ entry_meta, const int* __restrict__ chunks, const int* __restrict__ spans,
                    float* __restrict__ maps, float* __restrict__ start, T* __restrict__ out, int W) {
  constexpr bool FAST = sizeof(T) == 2;
  __shared__ float s_a[4][64], s_b[4][64];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int c = blockIdx.x * 64 + lane;
  const bool live = c < W;
  const int cc = live ? c : W - 1;
  const int chunk = blockIdx.y;
  const int entry = chunks[4 * chunk], row0 = chunks[4 * chunk + 1], n = chunks[4 * chunk + 2], flags = chunks[4 * chunk + 3];
  const float bz = bias_z[cc], bx = bias_x[cc];
  float S = 0.f;       // PASS 2: the state in front of the block at hand
  float* const cell = state + (size_t)entry_meta[4 * entry + 3] * slot_stride + cc;
  if (PASS == 1) {
    if (flags & 2) return;      // nobody folds the map of an entry's last chunk
    if ((flags & 1) && live && wave == 0) start[(size_t)entry * W + c] = *cell;
  }
  if (PASS == 2) {
    // the maps in front of this chunk: a wavefront folds a quarter of them in order, the quarters are joined in order
    const int first = spans[2 * entry], before = chunk - first;
    const int per = (before + 3) / 4, lo = min(wave * per, before), hi = min(lo + per, before);
    float A = 1.f, B = 0.f;
    for (int i0 = lo; i0 < hi; i0 += 8) {
      float a[8], b[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const size_t at = (size_t)(first + min(i0 + i, hi - 1)) * 2 * W + cc;
        a[i] = maps[at];
        b[i] = maps[at + W];
      }
#pragma unroll
      for (int i = 0; i < 8; ++i)
        if (i0 + i < hi) {
          A *= a[i];
          B = fmaf(a[i], B, b[i]);
        }
    }
    s_a[wave][lane] = A;
    s_b[wave][lane] = B;
    __syncthreads();
    S = (flags & 3) == 3 ? *cell : start[(size_t)entry * W + cc];
#pragma unroll
    for (int w = 0; w < 4; ++w) S = fmaf(s_a[w][lane], S, s_b[w][lane]);
    __syncthreads();
  }
  float CA = 1.f, CB = 0.f;      // PASS 1: the map of the blocks so far
  for (int t0 = 0; t0 < n; t0 += MG_BLOCK) {
    const int lo = t0 + wave * MG_SUB, live_n = min(MG_SUB, n - lo);      // this wavefront's tokens (live_n may be below 1)
    float keep[MG_SUB], put[MG_SUB], g[PASS == 2 ? MG_SUB : 1];
#pragma unroll
    for (int i = 0; i < MG_SUB; ++i) {
      const float* row = proj + (size_t)(row0 + min(lo + i, n - 1)) * ldp + cc;
      keep[i] = row[off_z];
      put[i] = row[off_x];
      if (PASS == 2) g[i] = row[off_g];
    }
    float A = 1.f, B = 0.f;
#pragma unroll
    for (int i = 0; i < MG_SUB; ++i)
      if (i < live_n) {
        mg_map<FAST>(keep[i], put[i], bz, bx, &keep[i], &put[i]);
        A *= keep[i];
        B = fmaf(keep[i], B, put[i]);
      }
    s_a[wave][lane] = A;
    s_b[wave][lane] = B;
    __syncthreads();
    if (PASS == 1) {
#pragma unroll
      for (int w = 0; w < 4; ++w) {
        CA *= s_a[w][lane];
        CB = fmaf(s_a[w][lane], CB, s_b[w][lane]);
      }
    } else {
      float mine = S;
#pragma unroll
      for (int w = 0; w < 4; ++w) {
        if (w == wave) mine = S;
        S = fmaf(s_a[w][lane], S, s_b[w][lane]);
      }
#pragma unroll
      for (int i = 0; i < MG_SUB; ++i)
        if (i < live_n) {
          mine = fmaf(keep[i], mine, put[i]);
          if (live) st<T>(out + (size_t)(row0 + lo + i) * W + c, mg_out<FAST>(mine, g[i]));
        }
    }
    __syncthreads();
  }
  if (!live || wave != 0) return;
  if (PASS == 1) {
    maps[(size_t)chunk * 2 * W + c] = CA;
    maps[((size_t)chunk * 2 + 1) * W + c] = CB;
  } else if (flags & 2) {
    *cell = S;
  }
}

static int check_mingru(int ldp, int off_z, int off_x, int off_g, long slot_stride, int n_entries, int W) {
  TI_REQUIRE(W > 0 && off_z >= 0 && off_x >= 0 && off_g >= 0 && off_z + W <= ldp && off_x + W <= ldp && off_g + W <= ldp && slot_stride >= W &&
                 n_entries <= 65535,
             "mingru: width %d, columns %d / %d / %d of %d, slots of %ld, %d entries do not fit", W, off_z, off_x, off_g, ldp, slot_stride,
             n_entries);
  return 0;
}

extern "C" int ti_mingru_scan(int out_dtype, const float* proj, int ldp, int off_z, int off_x, int off_g, const float* bias_z,
                              const float* bias_x, float* state, long slot_stride, const int* entry_meta, int n_entries, void* out, int W,
                              hipStream_t stream) {
  if (check_mingru(ldp, off_z, off_x, off_g, slot_stride, n_entries, W)) return 1;
  if (n_entries == 0) return 0;
  const dim3 grid((W + 255) / 256, n_entries);
  if (out_dtype == TI_F32)
    mingru_step_kernel<float><<<grid, 256, 0, stream>>>(proj, ldp, off_z, off_x, off_g, bias_z, bias_x, state, slot_stride, entry_meta,
                                                        (float*)out, W);
  else if (out_dtype == TI_BF16)
    mingru_step_kernel<bf16_t><<<grid, 256, 0, stream>>>(proj, ldp, off_z, off_x, off_g, bias_z, bias_x, state, slot_stride, entry_meta,
                                                         (bf16_t*)out, W);
  else
    TI_REQUIRE(false, "mingru: unknown dtype %d", out_dtype);
  TI_LAUNCH_CHECK();
  return 0;
}

// scratch: float [n_chunks][2][W] and behind it [n_entries][W]
extern "C" int ti_mingru_scan_chunked(int out_dtype, const float* proj, int ldp, int off_z, int off_x, int off_g, const float* bias_z,
                                      const float* bias_x, float* state, long slot_stride, const int* entry_meta, int n_entries,
                                      const int* chunks, int n_chunks, const int* spans, float* scratch, void* out, int W,
                                      hipStream_t stream) {
  if (check_mingru(ldp, off_z, off_x, off_g, slot_stride, n_entries, W)) return 1;
  TI_REQUIRE(chunks && spans && scratch && n_chunks >= n_entries && n_chunks <= 65535, "mingru: %d chunks need their lists and scratch", n_chunks);
  if (n_entries == 0) return 0;
  TI_REQUIRE(out_dtype == TI_F32 || out_dtype == TI_BF16, "mingru: unknown dtype %d", out_dtype);
  float* start = scratch + (size_t)n_chunks * 2 * W;
  const dim3 grid((W + 63) / 64, n_chunks);
#define MG_PASS(T, P)                                                                                                                 \
  mingru_chunk_kernel<T, P><<<grid, 256, 0, stream>>>(proj, ldp, off_z, off_x, off_g, bias_z, bias_x, state, slot_stride, entry_meta, \
                                                      chunks, spans, scratch, start, (T*)out, W)
  if (out_dtype == TI_F32) {
    if (n_chunks > n_entries) MG_PASS(float, 1);
    MG_PASS(float, 2);
  } else {
    if (n_chunks > n_entries) MG_PASS(bf16_t, 1);
    MG_PASS(bf16_t, 2);
  }
#undef MG_PASS
  TI_LAUNCH_CHECK();
  return 0;
}
