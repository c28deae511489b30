// libti_linear_attention: linear attention as a scan over each request's tokens of the step, and the gated norms behind it.
//
//   per head  S_t = a_t S_(t-1) + d_t k_t v_t^T,   o_t = S_t^T q_t (+ c v_t);   S [dk][dv] is per-request state in 32-bit, from
//   and into the request's slot.  q, k (qk_heads x dk, head h reads head h / (heads / qk_heads)) and v (heads x dv) are columns of
//   32-bit rows, with silu on all three, or q and k rotated, or as they are; k times a number.
//   Fixed decay: a_t = decay_h, d_t = 1.   Selective: d_t = softplus(dt_t + bias_h), a_t = exp(-exp(A_h) d_t), c = skip_h.
// Everything here is 32-bit.
//
// Short runs of tokens: a workgroup per (entry, head) walks them one by one.  The state lives in registers: thread (rg, j) holds
// RPT neighbouring rows of column j (RG = threads / padded dv row groups).  Tokens are staged TB at a time in LDS (activations
// applied on the way); per token a thread updates its rows and leaves its share of o_t[j] in LDS; after the TB tokens the shares
// are added in ascending rg.  The order of every sum depends on the sizes alone, never on how the tokens were cut into steps.
//
// Long runs are cut into chunks of up to 64 tokens.  With L_t the sum of the logarithms of a up to t inside a chunk,
//   what the chunk adds to an empty state:   sum_s e^(L_n - L_s) d_s k_s v_s^T                          (scan_chunk_states)
//   the states the chunks start from:        S <- e^(L_n) S + that, element by element                   (scan_carry)
//   outputs:  e^(L_t) S^T q_t + sum_(s <= t) e^(L_t - L_s) (q_t . k_s) d_s v_s                            (scan_chunk_outputs)
// the sums over tokens and over the state's rows as 32-bit matrix products (v_mfma_f32_16x16x4_f32: exact products, 32-bit
// sums).  No exponent is positive.
#include "common.h"
#include "tinyinfer_kernels.h"

TI_ERROR_API

// z sigmoid(z) with the hardware's exponential and reciprocal (a few units of 32-bit rounding)
__device__ __forceinline__ float la_silu(float z) { return z * __frcp_rn(1.0f + __expf(-z)); }
__device__ __forceinline__ float la_softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

// entry i of a query or key head of row m at position p, as it enters the recurrence (`head`: the head's columns of the row)
__device__ __forceinline__ float scan_entry(const ti_scan_inputs& in, const float* __restrict__ head, int i, int p) {
  const float x = head[i];
  if (in.act) return la_silu(x);
  if (i >= in.rot_dims) return x;
  const int half = in.rot_dims / 2, f = i < half ? i : i - half;
  const float other = head[i < half ? i + half : i - half];
  float c, s;
  if (in.rope_table && p < in.table_len) {
    c = in.rope_table[((size_t)p * half + f) * 2];
    s = in.rope_table[((size_t)p * half + f) * 2 + 1];
  } else {
    const float a = (float)p * in.inv_freq[f];
    c = cosf(a);
    s = sinf(a);
  }
  return i < half ? x * c - other * s : x * c + other * s;
}
__device__ __forceinline__ float scan_value(const ti_scan_inputs& in, float x) { return in.act ? la_silu(x) : x; }
// the step size of row m, head h
__device__ __forceinline__ float scan_dt(const ti_scan_inputs& in, int m, int h) {
  return la_softplus(in.dt[(size_t)m * in.dt_ld + h] + in.dt_bias[h]);
}

template <int NT, int RPT, int TB>
__global__ void __launch_bounds__(NT)
scan_tokens_kernel(const ti_scan_inputs in, float* __restrict__ state, long slot_stride, const int* __restrict__ entry_meta,
                   float* __restrict__ o, int heads, int dk, int dv, int dvs, int dvp) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int h = blockIdx.y, hq = h / (heads / in.qk_heads);
  const int row0 = entry_meta[4 * blockIdx.x], n = entry_meta[4 * blockIdx.x + 1], slot = entry_meta[4 * blockIdx.x + 3];
  const int RG = NT / dvp;
  const int dkp = RPT * RG;
  const int j = threadIdx.x % dvp, rg = threadIdx.x / dvp;
  const int i0 = rg * RPT;
  const int col0 = blockIdx.z * dvs, jg = col0 + j;      // this workgroup's slice of the state's columns: they never meet
  const bool live = j < dvs && jg < dv;
  float* s_q = lds;                               // [TB][dkp]
  float* s_k = s_q + TB * dkp;                    // [TB][dkp]
  float* s_v = s_k + TB * dkp;                    // [TB][dvs]
  float* s_part = s_v + TB * dvs;                 // [TB][RG][dvp] = [TB][NT]
  float* s_a = s_part + TB * NT;                  // [TB] the tokens' decays
  float* s_d = s_a + TB;                          // [TB] ... and step sizes
  float* S = state + (size_t)slot * slot_stride + (size_t)h * dk * dv;
  const float fixed = in.decay ? in.decay[h] : 0.f, rate = in.decay ? 0.f : expf(in.a_log[h]);
  const float skip = in.skip ? in.skip[h] : 0.f;
  float reg[RPT];
#pragma unroll
  for (int r = 0; r < RPT; ++r) reg[r] = (live && i0 + r < dk) ? S[(size_t)(i0 + r) * dv + jg] : 0.f;
  const int width = 2 * dkp + dvs;
  for (int t0 = 0; t0 < n; t0 += TB) {
    const int nt = min(TB, n - t0);
    __syncthreads();
    for (int x = threadIdx.x; x < nt * width; x += NT) {
      const int tt = x / width, c = x % width, m = row0 + t0 + tt;
      const float* row = in.proj + (size_t)m * in.ld;
      const int p = in.rot_dims ? in.pos[m] : 0;
      if (c < dkp) s_q[tt * dkp + c] = c < dk ? scan_entry(in, row + in.off_q + hq * dk, c, p) : 0.f;
      else if (c < 2 * dkp) s_k[tt * dkp + c - dkp] = c - dkp < dk ? scan_entry(in, row + in.off_k + hq * dk, c - dkp, p) * in.k_scale : 0.f;
      else s_v[tt * dvs + c - 2 * dkp] = col0 + c - 2 * dkp < dv ? scan_value(in, row[in.off_v + h * dv + col0 + c - 2 * dkp]) : 0.f;
    }
    if (threadIdx.x < nt) {
      const float d = in.decay ? 1.f : scan_dt(in, row0 + t0 + threadIdx.x, h);
      s_d[threadIdx.x] = d;
      s_a[threadIdx.x] = in.decay ? fixed : expf(-rate * d);
    }
    __syncthreads();
    for (int tt = 0; tt < nt; ++tt) {
      const float a = s_a[tt], vj = live ? s_v[tt * dvs + j] * s_d[tt] : 0.f;
      float part = 0.f;
      if constexpr (RPT % 4 == 0) {
        const float4* k4 = reinterpret_cast<const float4*>(s_k + tt * dkp + i0);
        const float4* q4 = reinterpret_cast<const float4*>(s_q + tt * dkp + i0);
#pragma unroll
        for (int r = 0; r < RPT / 4; ++r) {
          const float4 kk = k4[r];
          reg[4 * r] = fmaf(a, reg[4 * r], kk.x * vj);
          reg[4 * r + 1] = fmaf(a, reg[4 * r + 1], kk.y * vj);
          reg[4 * r + 2] = fmaf(a, reg[4 * r + 2], kk.z * vj);
          reg[4 * r + 3] = fmaf(a, reg[4 * r + 3], kk.w * vj);
          const float4 qq = q4[r];
          part = fmaf(reg[4 * r], qq.x, part);
          part = fmaf(reg[4 * r + 1], qq.y, part);
          part = fmaf(reg[4 * r + 2], qq.z, part);
          part = fmaf(reg[4 * r + 3], qq.w, part);
        }
      } else {
#pragma unroll
        for (int r = 0; r < RPT; ++r) {
          reg[r] = fmaf(a, reg[r], s_k[tt * dkp + i0 + r] * vj);
          part = fmaf(reg[r], s_q[tt * dkp + i0 + r], part);
        }
      }
      s_part[tt * NT + threadIdx.x] = part;
    }
    __syncthreads();
    for (int x = threadIdx.x; x < nt * dvs; x += NT) {
      const int tt = x / dvs, c = x % dvs;
      if (col0 + c >= dv) continue;
      float acc = 0.f;
      for (int g = 0; g < RG; ++g) acc += s_part[tt * NT + g * dvp + c];
      if (in.skip) acc = fmaf(skip, s_v[tt * dvs + c], acc);
      o[(size_t)(row0 + t0 + tt) * heads * dv + (size_t)h * dv + col0 + c] = acc;
    }
  }
#pragma unroll
  for (int r = 0; r < RPT; ++r)
    if (live && i0 + r < dk) S[(size_t)(i0 + r) * dv + jg] = reg[r];
}

// ------------------------------------------------------------ chunks side by side
#define SC_N 64                 // tokens of a chunk, rows and columns of a block of the state
#define SC_ROW 68               // floats between rows that are read four neighbours at a time
#define SC_COL 80               // ... and between rows that are read column by column
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float sc_float4;

// The chunk's weights: with a fixed decay the powers of it, pw[t - s]; else the sums L_t of the logarithms in double precision,
// so that the difference of two large sums keeps its digits, and the step sizes.  Called by all threads; no barrier inside.
struct ChunkWeights {
  float pw[SC_N + 1], d[SC_N];
  double L[SC_N];
};
__device__ __forceinline__ void chunk_weights(const ti_scan_inputs& in, ChunkWeights& w, int row0, int n, int h) {
  if (in.decay) {
    if (threadIdx.x <= SC_N) {
      double p = 1.0;
      const double a = (double)in.decay[h];
      for (int i = 0; i < (int)threadIdx.x; ++i) p *= a;
      w.pw[threadIdx.x] = (float)p;
    }
    return;
  }
  if (threadIdx.x < SC_N) {      // the first wavefront
    const int t = threadIdx.x;
    const float d = t < n ? scan_dt(in, row0 + t, h) : 0.f;
    double l = t < n ? -(double)(expf(in.a_log[h]) * d) : 0.0;
#pragma unroll
    for (int o = 1; o < SC_N; o <<= 1) {
      const double up = __shfl_up(l, o, TI_WAVE);
      if (t >= o) l += up;
    }
    w.L[t] = l;
    w.d[t] = d;
  }
}
// e^(L_t - L_s) for s <= t; e^(L_t) with s = -1
__device__ __forceinline__ float chunk_factor(const ti_scan_inputs& in, const ChunkWeights& w, int t, int s) {
  if (in.decay) return w.pw[t - s];
  return expf((float)(s < 0 ? w.L[t] : w.L[t] - w.L[s]));
}

// scratch [chunk][head][dk][dv] = what the chunk adds to an empty state, chunk_decay [chunk][head] = e^(L_n).  A workgroup per
// (chunk, head, block of 64 x 64 of the state); its four wavefronts two by two, each 32 x 32: the sum over the chunk's tokens as
// matrix products k^T v.
__global__ void __launch_bounds__(256)
scan_chunk_states_kernel(const ti_scan_inputs in, const int* __restrict__ chunks, float* __restrict__ scratch, float* __restrict__ chunk_decay,
                         int heads, int dk, int dv, int col_blocks) {
  __shared__ float s_k[SC_N][SC_COL], s_v[SC_N][SC_COL];
  __shared__ ChunkWeights w;
  const int h = blockIdx.y, hq = h / (heads / in.qk_heads);
  const int row0 = chunks[4 * blockIdx.x + 1], n = chunks[4 * blockIdx.x + 2];
  const int i0 = blockIdx.z / col_blocks * SC_N, j0 = blockIdx.z % col_blocks * SC_N;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r16 = lane & 15, quad = lane >> 4;
  const int c = threadIdx.x & 63;
  chunk_weights(in, w, row0, n, h);
  __syncthreads();
#pragma unroll
  for (int k = 0; k < SC_N / 4; ++k) {
    const int t = wave + 4 * k, m = row0 + t;
    float kv = 0.f, vv = 0.f;
    if (t < n) {
      const float* row = in.proj + (size_t)m * in.ld;
      const float f = in.decay ? chunk_factor(in, w, n - 1, t) : chunk_factor(in, w, n - 1, t) * w.d[t];
      if (i0 + c < dk) kv = scan_entry(in, row + in.off_k + hq * dk, i0 + c, in.rot_dims ? in.pos[m] : 0) * in.k_scale * f;
      if (j0 + c < dv) vv = scan_value(in, row[in.off_v + h * dv + j0 + c]);
    }
    s_k[t][c] = kv;
    s_v[t][c] = vv;
  }
  if (blockIdx.z == 0 && threadIdx.x == 0) chunk_decay[(size_t)blockIdx.x * heads + h] = chunk_factor(in, w, n - 1, -1);
  __syncthreads();
  const int wy = (wave >> 1) * 32, wx = (wave & 1) * 32;
  sc_float4 acc[2][2] = {};
#pragma unroll
  for (int s = 0; s < SC_N; s += 4) {
    float a[2], b[2];
#pragma unroll
    for (int x = 0; x < 2; ++x) {
      a[x] = s_k[s + quad][wy + 16 * x + r16];
      b[x] = s_v[s + quad][wx + 16 * x + r16];
    }
#pragma unroll
    for (int x = 0; x < 2; ++x)
#pragma unroll
      for (int y = 0; y < 2; ++y) acc[x][y] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[x], b[y], acc[x][y], 0, 0, 0);
  }
  float* out = scratch + ((size_t)blockIdx.x * heads + h) * dk * dv;
#pragma unroll
  for (int x = 0; x < 2; ++x)
#pragma unroll
    for (int y = 0; y < 2; ++y)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = i0 + wy + 16 * x + 4 * quad + r, j = j0 + wx + 16 * y + r16;
        if (i < dk && j < dv) out[(size_t)i * dv + j] = acc[x][y][r];
      }
}

// The states the chunks of an entry start from: chunk c starts from S and leaves chunk_decay_c S + A_c.  scratch [chunk][head]
// [dk dv] holds A_c when the kernel starts and the chunk's start state when it ends; the slot gets the state behind the last
// chunk.  A thread per element of the state; spans [entry][2] = (first chunk, chunks).
__global__ void scan_carry_kernel(float* __restrict__ scratch, const float* __restrict__ chunk_decay, const int* __restrict__ spans,
                                  const int* __restrict__ entry_meta, float* __restrict__ state, long slot_stride, int heads, int per_head) {
  const int e = blockIdx.x, h = blockIdx.y;
  const int x = blockIdx.z * blockDim.x + threadIdx.x;
  if (x >= per_head) return;
  const int c0 = spans[2 * e], nc = spans[2 * e + 1];
  float* slot = state + (size_t)entry_meta[4 * e + 3] * slot_stride + (size_t)h * per_head + x;
  float S = *slot;
  // eight chunks' shares are asked for together: the walk waits for memory once per eight chunks, not once per chunk
  for (int c = c0; c < c0 + nc; c += 8) {
    float add[8], f[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int ci = min(c + i, c0 + nc - 1);
      add[i] = scratch[((size_t)ci * heads + h) * per_head + x];
      f[i] = chunk_decay[(size_t)ci * heads + h];
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      if (c + i >= c0 + nc) break;
      scratch[((size_t)(c + i) * heads + h) * per_head + x] = S;
      S = fmaf(f[i], S, add[i]);
    }
  }
  *slot = S;
}

// The outputs of a chunk from the state it starts from: a workgroup per (chunk, head, 64 columns of the state), its four
// wavefronts two by two over 64 tokens x 64 columns.  q . k and q . S over blocks of 64 of the state's rows, then the weighted
// and masked q . k against the values.
__global__ void __launch_bounds__(256)
scan_chunk_outputs_kernel(const ti_scan_inputs in, const int* __restrict__ chunks, const float* __restrict__ scratch, float* __restrict__ o,
                          int heads, int dk, int dv) {
  __shared__ __attribute__((aligned(16))) float s_q[SC_N][SC_ROW], s_k[SC_N][SC_ROW];
  __shared__ float s_s[SC_N][SC_COL];
  __shared__ ChunkWeights w;
  const int h = blockIdx.y, hq = h / (heads / in.qk_heads);
  const int row0 = chunks[4 * blockIdx.x + 1], n = chunks[4 * blockIdx.x + 2];
  const int j0 = blockIdx.z * SC_N;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r16 = lane & 15, quad = lane >> 4;
  const int c = threadIdx.x & 63;
  const int wy = (wave >> 1) * 32, wx = (wave & 1) * 32;
  const float* S = scratch + ((size_t)blockIdx.x * heads + h) * dk * dv;
  const bool masked = wy + 31 < wx;      // none of this wavefront's (token, earlier token) pairs is in order
  chunk_weights(in, w, row0, n, h);
  sc_float4 P[2][2] = {}, O[2][2] = {};
  for (int i0 = 0; i0 < dk; i0 += SC_N) {
    __syncthreads();
#pragma unroll
    for (int k = 0; k < SC_N / 4; ++k) {
      const int t = wave + 4 * k, m = row0 + t;
      float qv = 0.f, kv = 0.f;
      if (t < n && i0 + c < dk) {
        const float* row = in.proj + (size_t)m * in.ld;
        const int p = in.rot_dims ? in.pos[m] : 0;
        qv = scan_entry(in, row + in.off_q + hq * dk, i0 + c, p);
        kv = scan_entry(in, row + in.off_k + hq * dk, i0 + c, p) * in.k_scale;
      }
      s_q[t][c] = qv;
      s_k[t][c] = kv;
      s_s[t][c] = (i0 + t < dk && j0 + c < dv) ? S[(size_t)(i0 + t) * dv + j0 + c] : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < SC_N; i += 16) {
      // lane group g holds the rows i + 4 g .. i + 4 g + 3 of the sum: product e takes entry e of every group
      float4 a[2], b[2];
#pragma unroll
      for (int x = 0; x < 2; ++x) {
        a[x] = *reinterpret_cast<const float4*>(&s_q[wy + 16 * x + r16][i + 4 * quad]);
        if (!masked) b[x] = *reinterpret_cast<const float4*>(&s_k[wx + 16 * x + r16][i + 4 * quad]);
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        float v[2];
#pragma unroll
        for (int y = 0; y < 2; ++y) v[y] = s_s[i + 4 * quad + e][wx + 16 * y + r16];
#pragma unroll
        for (int x = 0; x < 2; ++x) {
          const float ax = e == 0 ? a[x].x : e == 1 ? a[x].y : e == 2 ? a[x].z : a[x].w;
#pragma unroll
          for (int y = 0; y < 2; ++y) {
            O[x][y] = __builtin_amdgcn_mfma_f32_16x16x4f32(ax, v[y], O[x][y], 0, 0, 0);
            if (!masked) {
              const float by = e == 0 ? b[y].x : e == 1 ? b[y].y : e == 2 ? b[y].z : b[y].w;
              P[x][y] = __builtin_amdgcn_mfma_f32_16x16x4f32(ax, by, P[x][y], 0, 0, 0);
            }
          }
        }
      }
    }
  }
  __syncthreads();
  // a lane's four entries of a block: tokens 4 quad .. 4 quad + 3, column r16
#pragma unroll
  for (int x = 0; x < 2; ++x)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = wy + 16 * x + 4 * quad + r;
      const float f = t < n ? chunk_factor(in, w, t, -1) : 0.f;
#pragma unroll
      for (int y = 0; y < 2; ++y) {
        O[x][y][r] *= f;
        const int s = wx + 16 * y + r16;
        float p = 0.f;
        if (s <= t && t < n) p = P[x][y][r] * chunk_factor(in, w, t, s) * (in.decay ? 1.f : w.d[s]);
        s_q[t][s] = p;
      }
    }
#pragma unroll
  for (int k = 0; k < SC_N / 4; ++k) {
    const int t = wave + 4 * k;
    s_s[t][c] = (t < n && j0 + c < dv) ? scan_value(in, in.proj[(size_t)(row0 + t) * in.ld + in.off_v + h * dv + j0 + c]) : 0.f;
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < SC_N; i += 16) {
    if (i > wy + 31) break;      // later tokens than any of this wavefront's
    float4 a[2];
#pragma unroll
    for (int x = 0; x < 2; ++x) a[x] = *reinterpret_cast<const float4*>(&s_q[wy + 16 * x + r16][i + 4 * quad]);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      float v[2];
#pragma unroll
      for (int y = 0; y < 2; ++y) v[y] = s_s[i + 4 * quad + e][wx + 16 * y + r16];
#pragma unroll
      for (int x = 0; x < 2; ++x) {
        const float ax = e == 0 ? a[x].x : e == 1 ? a[x].y : e == 2 ? a[x].z : a[x].w;
#pragma unroll
        for (int y = 0; y < 2; ++y) O[x][y] = __builtin_amdgcn_mfma_f32_16x16x4f32(ax, v[y], O[x][y], 0, 0, 0);
      }
    }
  }
  const float skip = in.skip ? in.skip[h] : 0.f;
#pragma unroll
  for (int x = 0; x < 2; ++x)
#pragma unroll
    for (int y = 0; y < 2; ++y)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = wy + 16 * x + 4 * quad + r, j = wx + 16 * y + r16;
        if (t >= n || j0 + j >= dv) continue;
        float v = O[x][y][r];
        if (in.skip) v = fmaf(skip, s_s[t][j], v);
        o[(size_t)(row0 + t) * heads * dv + (size_t)h * dv + j0 + j] = v;
      }
}

template <int NT, int TB>
static int launch_scan(int rpt, dim3 grid, size_t lds, hipStream_t stream, const ti_scan_inputs& in, float* state, long slot_stride,
                       const int* entry_meta, float* o, int heads, int dk, int dv, int dvs, int dvp) {
#define LA_CASE(R)                                                                                                                  \
  case R:                                                                                                                           \
    scan_tokens_kernel<NT, R, TB><<<grid, NT, lds, stream>>>(in, state, slot_stride, entry_meta, o, heads, dk, dv, dvs, dvp);       \
    return 0;
  switch (rpt) {
    LA_CASE(1) LA_CASE(2) LA_CASE(4) LA_CASE(8) LA_CASE(16) LA_CASE(32) LA_CASE(64)
  }
#undef LA_CASE
  return 1;
}

// wide states are cut into slices of 64 columns, a workgroup each: more workgroups, and fewer rows a thread
struct ScanShape { int dvs, slices, dvp, nt, tb, rpt; size_t lds; bool big; };
static ScanShape scan_shape(int dk, int dv) {
  ScanShape s;
  s.dvs = dv > 64 ? 64 : dv;
  s.slices = (dv + s.dvs - 1) / s.dvs;
  s.dvp = 1;
  while (s.dvp < s.dvs) s.dvp *= 2;
  s.big = (long)dk * s.dvp > 64L * 256;
  s.nt = s.big ? 1024 : 256;
  s.tb = s.big ? 4 : 16;
  const int rgs = s.nt / s.dvp;
  s.rpt = 1;
  while (s.rpt * rgs < dk) s.rpt *= 2;
  s.lds = ((size_t)s.tb * (2 * s.rpt * rgs + s.dvs) + (size_t)s.tb * s.nt + 2 * s.tb) * 4;
  return s;
}

static int check_scan(const char* what, const ti_scan_inputs* in, long slot_stride, int heads, int dk, int dv) {
  TI_REQUIRE(heads > 0 && heads <= 65535 && dk > 0 && dk <= 256 && dv > 0 && dv <= 256, "%s: bad sizes heads=%d dk=%d dv=%d (up to 256)",
             what, heads, dk, dv);
  TI_REQUIRE(in->qk_heads > 0 && heads % in->qk_heads == 0, "%s: %d heads over %d query and key heads", what, heads, in->qk_heads);
  TI_REQUIRE(in->off_q >= 0 && in->off_k >= 0 && in->off_v >= 0 && in->off_q + in->qk_heads * dk <= in->ld && in->off_k + in->qk_heads * dk <= in->ld &&
                 in->off_v + heads * dv <= in->ld,
             "%s: the columns do not lie inside rows of %d", what, in->ld);
  TI_REQUIRE(in->rot_dims >= 0 && in->rot_dims % 2 == 0 && in->rot_dims <= dk && (!in->rot_dims || (in->inv_freq && in->pos && !in->act)),
             "%s: a rotation of %d of %d entries is not served", what, in->rot_dims, dk);
  TI_REQUIRE(in->decay || (in->dt && in->dt_bias && in->a_log && in->dt_ld >= heads), "%s: neither fixed decays nor step sizes", what);
  TI_REQUIRE(slot_stride >= (long)heads * dk * dv, "%s: a slot of %ld floats does not hold the state", what, slot_stride);
  return 0;
}

// state f32 [slots][heads][dk][dv] (slot_stride floats a slot); entry_meta [n_entries][4] = (row0, tokens, start, slot);
// o f32 [M, heads dv]
extern "C" int ti_linear_scan(const ti_scan_inputs* in, float* state, long slot_stride, const int* entry_meta, int n_entries, float* o,
                              int heads, int dk, int dv, hipStream_t stream) {
  if (check_scan("linear_scan", in, slot_stride, heads, dk, dv)) return 1;
  if (n_entries == 0) return 0;
  const ScanShape s = scan_shape(dk, dv);
  TI_REQUIRE(s.rpt <= 64, "linear_scan: a state of %d x %d is not served", dk, dv);
  const dim3 grid(n_entries, heads, s.slices);
  const int rc = s.big ? launch_scan<1024, 4>(s.rpt, grid, s.lds, stream, *in, state, slot_stride, entry_meta, o, heads, dk, dv, s.dvs, s.dvp)
                       : launch_scan<256, 16>(s.rpt, grid, s.lds, stream, *in, state, slot_stride, entry_meta, o, heads, dk, dv, s.dvs, s.dvp);
  TI_REQUIRE(rc == 0, "linear_scan: no kernel for %d rows a thread", s.rpt);
  TI_LAUNCH_CHECK();
  return 0;
}

// The same with every entry's tokens cut into chunks of up to 64 that run side by side.  chunks int [n_chunks][4] = (entry, first
// row, tokens, flags), spans int [n_entries][2] = (first chunk, chunks), both in device memory; scratch float
// [n_chunks][heads][dk dv + 1]
extern "C" int ti_linear_scan_chunked(const ti_scan_inputs* in, float* state, long slot_stride, const int* entry_meta, int n_entries,
                                      const int* chunks, int n_chunks, const int* spans, float* scratch, float* o, int heads, int dk,
                                      int dv, hipStream_t stream) {
  if (check_scan("linear_scan", in, slot_stride, heads, dk, dv)) return 1;
  TI_REQUIRE(chunks && spans && scratch && n_chunks >= n_entries, "linear_scan: chunks need their lists and scratch");
  if (n_entries == 0) return 0;
  const int rb = (dk + SC_N - 1) / SC_N, cb = (dv + SC_N - 1) / SC_N, per_head = dk * dv;
  float* chunk_decay = scratch + (size_t)n_chunks * heads * per_head;
  scan_chunk_states_kernel<<<dim3(n_chunks, heads, rb * cb), 256, 0, stream>>>(*in, chunks, scratch, chunk_decay, heads, dk, dv, cb);
  scan_carry_kernel<<<dim3(n_entries, heads, (per_head + 255) / 256), 256, 0, stream>>>(scratch, chunk_decay, spans, entry_meta, state, slot_stride,
                                                                                      heads, per_head);
  scan_chunk_outputs_kernel<<<dim3(n_chunks, heads, cb), 256, 0, stream>>>(*in, chunks, scratch, o, heads, dk, dv);
  TI_LAUNCH_CHECK();
  return 0;
}

// The norm behind such a mixer and its gate: a row of W entries in `groups` equal runs, each divided by its own root mean square,
// times w (null: none), with the gate's activation of gate columns off_g .. (0: sigmoid, 1: silu) multiplied in behind the
// norm, or in front of it (gate_first); rounded once to T.  WAVES: a wavefront per run (runs of up to 1024 entries, in
// registers), else a workgroup.
template <typename T, bool WAVES>
__global__ void __launch_bounds__(256)
gated_group_norm_kernel(const float* __restrict__ o, const float* __restrict__ gate, int ld, int off_g, const float* __restrict__ w,
                        T* __restrict__ out, int M, int W, int groups, float eps, int silu, int gate_first) {
  __shared__ float red[4];
  const int size = W / groups;
  auto gate_of = [&](float g) { return silu ? la_silu(g) : 1.0f / (1.0f + expf(-g)); };
  if constexpr (WAVES) {
    const long run = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (run >= (long)M * groups) return;
    const int lane = threadIdx.x & 63;
    const size_t m = run / groups;
    const int c0 = (int)(run % groups) * size;
    const float* src = o + m * W + c0;
    const float* g = gate + m * ld + off_g + c0;
    float v[16], f[16];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int c = lane + 64 * i;
      if (64 * i >= size) break;
      v[i] = f[i] = 0.f;
      if (c < size) {
        f[i] = gate_of(g[c]);
        v[i] = src[c];
        if (gate_first) v[i] *= f[i];
      }
      ss = fmaf(v[i], v[i], ss);
    }
    const float inv = 1.0f / sqrtf(group_sum<TI_WAVE>(ss) / (float)size + eps);
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int c = lane + 64 * i;
      if (64 * i >= size) break;
      if (c < size) st<T>(out + m * W + c0 + c, v[i] * inv * (w ? w[c0 + c] : 1.f) * (gate_first ? 1.f : f[i]));
    }
  } else {
    const size_t m = blockIdx.x / groups;
    const int c0 = (int)(blockIdx.x % groups) * size;
    const float* src = o + m * W + c0;
    const float* g = gate + m * ld + off_g + c0;
    float ss = 0.f;
    for (int c = threadIdx.x; c < size; c += 256) {
      const float v = gate_first ? src[c] * gate_of(g[c]) : src[c];
      ss = fmaf(v, v, ss);
    }
    const float inv = 1.0f / sqrtf(block_sum<256>(ss, red) / (float)size + eps);
    for (int c = threadIdx.x; c < size; c += 256) st<T>(out + m * W + c0 + c, src[c] * inv * (w ? w[c0 + c] : 1.f) * gate_of(g[c]));
  }
}

extern "C" int ti_gated_group_norm(int out_dtype, const float* o, const float* gate, int ld, int off_g, const float* w, void* out, int M,
                                   int W, int groups, float eps, int silu, int gate_first, hipStream_t stream) {
  TI_REQUIRE(M >= 0 && W > 0 && groups > 0 && W % groups == 0 && off_g >= 0 && off_g + W <= ld,
             "gated_group_norm: bad sizes M=%d W=%d in %d runs, gate columns %d of %d", M, W, groups, off_g, ld);
  TI_REQUIRE(out_dtype == TI_F32 || out_dtype == TI_BF16, "gated_group_norm: unknown dtype %d", out_dtype);
  if (M == 0) return 0;
  const bool waves = groups > 1 && W / groups <= 1024;
  const long runs = (long)M * groups;
  const unsigned blocks = (unsigned)(waves ? (runs + 3) / 4 : runs);
#define GGN(T, V) gated_group_norm_kernel<T, V><<<blocks, 256, 0, stream>>>(o, gate, ld, off_g, w, (T*)out, M, W, groups, eps, silu, gate_first)
  if (out_dtype == TI_F32) {
    if (waves) GGN(float, true);
    else GGN(float, false);
  } else {
    if (waves) GGN(bf16_t, true);
    else GGN(bf16_t, false);
  }
#undef GGN
  TI_LAUNCH_CHECK();
  return 0;
}
