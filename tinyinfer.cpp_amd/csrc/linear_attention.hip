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

#define SCAN_NT 256         // threads of a workgroup
#define SCAN_TB 16          // tokens staged together
// how q, k, v and the decays come about
#define SCAN_SILU 0         // silu on all three, fixed decays
#define SCAN_ROTATED 1      // q and k rotated, or as they are; fixed decays
#define SCAN_SELECTIVE 2    // as they are; step sizes
__device__ __forceinline__ void scan_angle(const ti_scan_inputs& in, int p, int half, int f, float* c, float* s) {
  if (in.rope_table && p < in.table_len) {
    *c = in.rope_table[((size_t)p * half + f) * 2];
    *s = in.rope_table[((size_t)p * half + f) * 2 + 1];
  } else {
    const float a = (float)p * in.inv_freq[f];
    *c = cosf(a);
    *s = sinf(a);
  }
}
// entry i of a query or key head of row m at position p, as it enters the recurrence (`head`: the head's columns of the row)
template <int FORM> __device__ __forceinline__ float scan_entry(const ti_scan_inputs& in, const float* __restrict__ head, int i, int p) {
  const float x = head[i];
  if (FORM == SCAN_SILU) return la_silu(x);
  if (FORM == SCAN_SELECTIVE || i >= in.rot_dims) return x;
  const int half = in.rot_dims / 2;
  float c, s;
  scan_angle(in, p, half, i < half ? i : i - half, &c, &s);
  return i < half ? x * c - head[i + half] * s : x * c + head[i - half] * s;
}
// the step size of row m, head h
__device__ __forceinline__ float scan_dt(const ti_scan_inputs& in, int m, int h) {
  return la_softplus(in.dt[(size_t)m * in.dt_ld + h] + in.dt_bias[h]);
}

template <int FORM, int NT, int RPT, int TB>
__global__ void __launch_bounds__(NT)
scan_tokens_kernel(const ti_scan_inputs in, float* __restrict__ state, long slot_stride, const int* __restrict__ entry_meta,
                   float* __restrict__ o, int heads, int dk, int dv, int dvs, int dvp) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int h = blockIdx.y, hq = h / (heads / in.qk_heads);
  const int* entry = entry_meta + 4 * blockIdx.x;
  const int row0 = entry[0], n = entry[1], start = entry[2], slot = entry[3];
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
  const float fixed = FORM == SCAN_SELECTIVE ? 0.f : in.decay[h], rate = FORM == SCAN_SELECTIVE ? expf(in.a_log[h]) : 0.f;
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
      if (c < 2 * dkp) {
        const bool is_q = c < dkp;
        const int i = is_q ? c : c - dkp;
        const float e = i < dk ? scan_entry<FORM>(in, row + (is_q ? in.off_q : in.off_k) + hq * dk, i, start + t0 + tt) : 0.f;
        (is_q ? s_q : s_k)[tt * dkp + i] = is_q ? e : e * in.k_scale;
      } else {
        const int i = c - 2 * dkp;
        const float e = col0 + i < dv ? row[in.off_v + h * dv + col0 + i] : 0.f;
        s_v[tt * dvs + i] = FORM == SCAN_SILU ? la_silu(e) : e;
      }
    }
    if (threadIdx.x < nt) {
      const float d = FORM == SCAN_SELECTIVE ? scan_dt(in, row0 + t0 + threadIdx.x, h) : 1.f;
      s_d[threadIdx.x] = d;
      s_a[threadIdx.x] = FORM == SCAN_SELECTIVE ? expf(-rate * d) : fixed;
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
template <bool SELECTIVE> __device__ __forceinline__ void chunk_weights(const ti_scan_inputs& in, ChunkWeights& w, int row0, int n, int h) {
  if (!SELECTIVE) {
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
template <bool SELECTIVE> __device__ __forceinline__ float chunk_factor(const ChunkWeights& w, int t, int s) {
  if (!SELECTIVE) return w.pw[t - s];
  return expf((float)(s < 0 ? w.L[t] : w.L[t] - w.L[s]));
}

// A block of 64 rows x 64 columns of 32-bit numbers on its way into LDS: a thread asks for four pieces of four neighbouring columns
// (rows threadIdx.x / 16 + 16 k), all in flight together, and puts them down later.  Rows from n_rows and columns from n_cols on
// are zeros.  VEC: the pieces are aligned to 16 bytes and n_cols is a multiple of four.
template <bool VEC> struct Block64 {
  float4 v[4];
  __device__ __forceinline__ void load(const float* __restrict__ src, size_t ld, int n_rows, int n_cols) {
    const int c = (threadIdx.x & 15) * 4;
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const int r = (threadIdx.x >> 4) + 16 * k;
      const float* p = src + (size_t)min(r, n_rows - 1) * ld;      // (a row that is not there: the last one's numbers, dropped below)
      float4 x = make_float4(0.f, 0.f, 0.f, 0.f);
      if (VEC) {
        x = *reinterpret_cast<const float4*>(p + min(c, n_cols - 4));
      } else {
        x.x = p[min(c, n_cols - 1)];
        x.y = p[min(c + 1, n_cols - 1)];
        x.z = p[min(c + 2, n_cols - 1)];
        x.w = p[min(c + 3, n_cols - 1)];
      }
      v[k] = x;
    }
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const bool row = (int)(threadIdx.x >> 4) + 16 * k < n_rows;
      v[k].x = row && c < n_cols ? v[k].x : 0.f;
      v[k].y = row && c + 1 < n_cols ? v[k].y : 0.f;
      v[k].z = row && c + 2 < n_cols ? v[k].z : 0.f;
      v[k].w = row && c + 3 < n_cols ? v[k].w : 0.f;
    }
  }
  __device__ __forceinline__ void silu() {      // (of zero: zero)
#pragma unroll
    for (int k = 0; k < 4; ++k) v[k] = make_float4(la_silu(v[k].x), la_silu(v[k].y), la_silu(v[k].z), la_silu(v[k].w));
  }
  template <class F> __device__ __forceinline__ void scale_rows(F f) {
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const float s = f((int)(threadIdx.x >> 4) + 16 * k);
      v[k] = make_float4(v[k].x * s, v[k].y * s, v[k].z * s, v[k].w * s);
    }
  }
  template <int ROW> __device__ __forceinline__ void put(float (*dst)[ROW]) const {
#pragma unroll
    for (int k = 0; k < 4; ++k) *reinterpret_cast<float4*>(&dst[(threadIdx.x >> 4) + 16 * k][(threadIdx.x & 15) * 4]) = v[k];
  }
};

// scratch [chunk][head][dk][dv] = what the chunk adds to an empty state, chunk_decay [chunk][head] = e^(L_n).  A workgroup per
// (chunk, head, block of 64 x 64 of the state); its four wavefronts two by two, each 32 x 32: the sum over the chunk's tokens as
// matrix products k^T v.
template <int FORM, bool VEC>
__global__ void __launch_bounds__(256)
scan_chunk_states_kernel(const ti_scan_inputs in, const int* __restrict__ chunks, float* __restrict__ scratch, float* __restrict__ chunk_decay,
                         int heads, int dk, int dv, int col_blocks) {
  __shared__ __attribute__((aligned(16))) float s_k[SC_N][SC_COL], s_v[SC_N][SC_COL];
  __shared__ ChunkWeights w;
  constexpr bool SEL = FORM == SCAN_SELECTIVE;
  const int h = blockIdx.y, hq = h / (heads / in.qk_heads);
  const int row0 = chunks[4 * blockIdx.x + 1], n = chunks[4 * blockIdx.x + 2];
  const int i0 = blockIdx.z / col_blocks * SC_N, j0 = blockIdx.z % col_blocks * SC_N;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r16 = lane & 15, quad = lane >> 4;
  const float* rows = in.proj + (size_t)row0 * in.ld;
  Block64<VEC> k, v;
  k.load(rows + in.off_k + hq * dk + i0, in.ld, n, dk - i0);
  v.load(rows + in.off_v + h * dv + j0, in.ld, n, dv - j0);
  chunk_weights<SEL>(in, w, row0, n, h);
  __syncthreads();
  if (FORM == SCAN_SILU) {
    k.silu();
    v.silu();
  }
  k.scale_rows([&](int t) {
    if (t >= n) return 0.f;
    const float f = chunk_factor<SEL>(w, n - 1, t) * in.k_scale;
    return SEL ? f * w.d[t] : f;
  });
  k.put(s_k);
  v.put(s_v);
  if (blockIdx.z == 0 && threadIdx.x == 0) chunk_decay[(size_t)blockIdx.x * heads + h] = chunk_factor<SEL>(w, n - 1, -1);
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
// wavefronts two by two over 64 tokens x 64 columns.  q . k and q . S over blocks of 64 of the state's rows (the next block is on
// its way from memory meanwhile), then the weighted and masked q . k against the values.
template <int FORM, bool VEC>
__global__ void __launch_bounds__(256)
scan_chunk_outputs_kernel(const ti_scan_inputs in, const int* __restrict__ chunks, const float* __restrict__ scratch, float* __restrict__ o,
                          int heads, int dk, int dv) {
  __shared__ __attribute__((aligned(16))) float s_q[SC_N][SC_ROW], s_k[SC_N][SC_ROW], s_s[SC_N][SC_COL];
  __shared__ ChunkWeights w;
  constexpr bool SEL = FORM == SCAN_SELECTIVE;
  const int h = blockIdx.y, hq = h / (heads / in.qk_heads);
  const int row0 = chunks[4 * blockIdx.x + 1], n = chunks[4 * blockIdx.x + 2];
  const int j0 = blockIdx.z * SC_N;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r16 = lane & 15, quad = lane >> 4;
  const int wy = (wave >> 1) * 32, wx = (wave & 1) * 32;
  const bool masked = wy + 31 < wx;      // none of this wavefront's (token, earlier token) pairs is in order
  const float* S = scratch + ((size_t)blockIdx.x * heads + h) * dk * dv + j0;
  const float* rows = in.proj + (size_t)row0 * in.ld;
  const float* row_q = rows + in.off_q + hq * dk;
  const float* row_k = rows + in.off_k + hq * dk;
  Block64<VEC> q, k, v;      // v: the state's rows, behind the last block the values
  q.load(row_q, in.ld, n, dk);
  k.load(row_k, in.ld, n, dk);
  v.load(S, dv, dk, dv - j0);
  chunk_weights<SEL>(in, w, row0, n, h);
  sc_float4 P[2][2] = {}, O[2][2] = {};
  for (int i0 = 0; i0 < dk; i0 += SC_N) {
    __syncthreads();
    if (FORM == SCAN_SILU) {
      q.silu();
      k.silu();
    }
    q.put(s_q);
    k.put(s_k);
    v.put(s_s);
    __syncthreads();
    const int next = i0 + SC_N;
    if (next < dk) {
      q.load(row_q + next, in.ld, n, dk - next);
      k.load(row_k + next, in.ld, n, dk - next);
      v.load(S + (size_t)next * dv, dv, dk - next, dv - j0);
    } else {
      v.load(rows + in.off_v + h * dv + j0, in.ld, n, dv - j0);
    }
#pragma unroll
    for (int i = 0; i < SC_N; i += 16) {
      // lane group g holds the rows i + 4 g .. i + 4 g + 3 of the sum: product e takes entry e of every group
      float4 a[2], b[2];
#pragma unroll
      for (int x = 0; x < 2; ++x) {
        a[x] = *reinterpret_cast<const float4*>(&s_q[wy + 16 * x + r16][i + 4 * quad]);
        b[x] = *reinterpret_cast<const float4*>(&s_k[wx + 16 * x + r16][i + 4 * quad]);
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        float sv[2];
#pragma unroll
        for (int y = 0; y < 2; ++y) sv[y] = s_s[i + 4 * quad + e][wx + 16 * y + r16];
#pragma unroll
        for (int x = 0; x < 2; ++x) {
          const float ax = e == 0 ? a[x].x : e == 1 ? a[x].y : e == 2 ? a[x].z : a[x].w;
#pragma unroll
          for (int y = 0; y < 2; ++y) {
            O[x][y] = __builtin_amdgcn_mfma_f32_16x16x4f32(ax, sv[y], O[x][y], 0, 0, 0);
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
      const float f = t < n ? chunk_factor<SEL>(w, t, -1) : 0.f;
#pragma unroll
      for (int y = 0; y < 2; ++y) {
        O[x][y][r] *= f;
        const int s = wx + 16 * y + r16;
        float p = 0.f;
        if (s <= t && t < n) p = P[x][y][r] * chunk_factor<SEL>(w, t, s) * in.k_scale * (SEL ? w.d[s] : 1.f);
        s_q[t][s] = p;
      }
    }
  if (FORM == SCAN_SILU) v.silu();
  v.put(s_s);
  __syncthreads();
#pragma unroll
  for (int i = 0; i < SC_N; i += 16) {
    if (i > wy + 31) break;      // later tokens than any of this wavefront's
    float4 a[2];
#pragma unroll
    for (int x = 0; x < 2; ++x) a[x] = *reinterpret_cast<const float4*>(&s_q[wy + 16 * x + r16][i + 4 * quad]);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      float sv[2];
#pragma unroll
      for (int y = 0; y < 2; ++y) sv[y] = s_s[i + 4 * quad + e][wx + 16 * y + r16];
#pragma unroll
      for (int x = 0; x < 2; ++x) {
        const float ax = e == 0 ? a[x].x : e == 1 ? a[x].y : e == 2 ? a[x].z : a[x].w;
#pragma unroll
        for (int y = 0; y < 2; ++y) O[x][y] = __builtin_amdgcn_mfma_f32_16x16x4f32(ax, sv[y], O[x][y], 0, 0, 0);
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
        float y_t = O[x][y][r];
        if (in.skip) y_t = fmaf(skip, s_s[t][j], y_t);
        o[(size_t)(row0 + t) * heads * dv + (size_t)h * dv + j0 + j] = y_t;
      }
}

// The rotation of the step's queries and keys in place, in front of the chunks (which then take them as they are): a workgroup per
// (row, 1024 pairs of entries), four neighbouring pairs a thread (VEC: aligned to 16 bytes) or one.
template <bool VEC> __global__ void __launch_bounds__(256) scan_rotate_kernel(float* __restrict__ proj, const ti_scan_inputs in, int dk) {
  constexpr int N = VEC ? 4 : 1;
  const int half = in.rot_dims / 2, n_pairs = 2 * in.qk_heads * half;
  float* const row = proj + (size_t)blockIdx.x * in.ld;
  const int p = in.pos[blockIdx.x];
  for (int x = (blockIdx.y * 256 + threadIdx.x) * N; x < n_pairs; x += gridDim.y * 256 * N) {
    const int f = x % half, u = x / half;      // (VEC: half is a multiple of four, the pairs lie in one head)
    float* a = row + (u < in.qk_heads ? in.off_q + u * dk : in.off_k + (u - in.qk_heads) * dk) + f;
    float* b = a + half;
    float c[N], s[N];
#pragma unroll
    for (int i = 0; i < N; ++i) scan_angle(in, p, half, f + i, &c[i], &s[i]);
    if constexpr (VEC) {
      const float4 va = *reinterpret_cast<const float4*>(a), vb = *reinterpret_cast<const float4*>(b);
      *reinterpret_cast<float4*>(a) = make_float4(va.x * c[0] - vb.x * s[0], va.y * c[1] - vb.y * s[1], va.z * c[2] - vb.z * s[2], va.w * c[3] - vb.w * s[3]);
      *reinterpret_cast<float4*>(b) = make_float4(vb.x * c[0] + va.x * s[0], vb.y * c[1] + va.y * s[1], vb.z * c[2] + va.z * s[2], vb.w * c[3] + va.w * s[3]);
    } else {
      const float va = *a, vb = *b;
      *a = va * c[0] - vb * s[0];
      *b = vb * c[0] + va * s[0];
    }
  }
}

template <int FORM>
static int launch_scan(int rpt, dim3 grid, size_t lds, hipStream_t stream, const ti_scan_inputs& in, float* state, long slot_stride,
                       const int* entry_meta, float* o, int heads, int dk, int dv, int dvs, int dvp) {
#define LA_CASE(R)                                                                                                                        \
  case R:                                                                                                                                 \
    scan_tokens_kernel<FORM, SCAN_NT, R, SCAN_TB><<<grid, SCAN_NT, lds, stream>>>(in, state, slot_stride, entry_meta, o, heads, dk, dv,   \
                                                                                  dvs, dvp);                                              \
    return 0;
  switch (rpt) {
    LA_CASE(1) LA_CASE(2) LA_CASE(4) LA_CASE(8) LA_CASE(16) LA_CASE(32) LA_CASE(64)
  }
#undef LA_CASE
  return 1;
}

// wide states are cut into slices of 32 columns, a workgroup each: more workgroups, and fewer rows a thread
struct ScanShape { int dvs, slices, dvp, rpt; size_t lds; };
static ScanShape scan_shape(int dk, int dv) {
  ScanShape s;
  s.dvs = dv > 32 ? 32 : dv;
  s.slices = (dv + s.dvs - 1) / s.dvs;
  s.dvp = 1;
  while (s.dvp < s.dvs) s.dvp *= 2;
  const int rgs = SCAN_NT / s.dvp;
  s.rpt = 1;
  while (s.rpt * rgs < dk) s.rpt *= 2;
  s.lds = ((size_t)SCAN_TB * (2 * s.rpt * rgs + s.dvs) + (size_t)SCAN_TB * SCAN_NT + 2 * SCAN_TB) * 4;
  return s;
}
static int scan_form(const ti_scan_inputs* in) { return in->act ? SCAN_SILU : in->decay ? SCAN_ROTATED : SCAN_SELECTIVE; }

static int check_scan(const char* what, const ti_scan_inputs* in, long slot_stride, int heads, int dk, int dv) {
  TI_REQUIRE(heads > 0 && heads <= 65535 && dk > 0 && dk <= 256 && dv > 0 && dv <= 256, "%s: bad sizes heads=%d dk=%d dv=%d (up to 256)",
             what, heads, dk, dv);
  TI_REQUIRE(in->qk_heads > 0 && heads % in->qk_heads == 0, "%s: %d heads over %d query and key heads", what, heads, in->qk_heads);
  TI_REQUIRE(in->off_q >= 0 && in->off_k >= 0 && in->off_v >= 0 && in->off_q + in->qk_heads * dk <= in->ld && in->off_k + in->qk_heads * dk <= in->ld &&
                 in->off_v + heads * dv <= in->ld,
             "%s: the columns do not lie inside rows of %d", what, in->ld);
  TI_REQUIRE(in->rot_dims >= 0 && in->rot_dims % 2 == 0 && in->rot_dims <= dk && (!in->rot_dims || (in->inv_freq && in->pos && !in->act)),
             "%s: a rotation of %d of %d entries is not served", what, in->rot_dims, dk);
  TI_REQUIRE(in->decay || (in->dt && in->dt_bias && in->a_log && in->dt_ld >= heads && !in->act && !in->rot_dims),
             "%s: neither fixed decays nor step sizes, or step sizes beside an activation or a rotation", what);
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
  int rc;
#define SCAN_CALL(F) rc = launch_scan<F>(s.rpt, grid, s.lds, stream, *in, state, slot_stride, entry_meta, o, heads, dk, dv, s.dvs, s.dvp)
  switch (scan_form(in)) {
    case SCAN_SILU: SCAN_CALL(SCAN_SILU); break;
    case SCAN_ROTATED: SCAN_CALL(SCAN_ROTATED); break;
    default: SCAN_CALL(SCAN_SELECTIVE);
  }
#undef SCAN_CALL
  TI_REQUIRE(rc == 0, "linear_scan: no kernel for %d rows a thread", s.rpt);
  TI_LAUNCH_CHECK();
  return 0;
}

// The same with every entry's tokens cut into chunks of up to 64 that run side by side.  chunks int [n_chunks][4] = (entry, first
// row, tokens, flags), spans int [n_entries][2] = (first chunk, chunks), both in device memory; scratch float
// [n_chunks][heads][dk dv + 1]
template <int FORM, bool VEC>
static void launch_chunks(const ti_scan_inputs& in, float* state, long slot_stride, const int* entry_meta, int n_entries, const int* chunks,
                          int n_chunks, const int* spans, float* scratch, float* o, int heads, int dk, int dv, hipStream_t stream) {
  const int rb = (dk + SC_N - 1) / SC_N, cb = (dv + SC_N - 1) / SC_N, per_head = dk * dv;
  float* chunk_decay = scratch + (size_t)n_chunks * heads * per_head;
  scan_chunk_states_kernel<FORM, VEC><<<dim3(n_chunks, heads, rb * cb), 256, 0, stream>>>(in, chunks, scratch, chunk_decay, heads, dk, dv, cb);
  scan_carry_kernel<<<dim3(n_entries, heads, (per_head + 255) / 256), 256, 0, stream>>>(scratch, chunk_decay, spans, entry_meta, state, slot_stride,
                                                                                      heads, per_head);
  scan_chunk_outputs_kernel<FORM, VEC><<<dim3(n_chunks, heads, cb), 256, 0, stream>>>(in, chunks, scratch, o, heads, dk, dv);
}

// (rotated queries and keys are turned in place: the columns of proj are overwritten)
extern "C" int ti_linear_scan_chunked(const ti_scan_inputs* inputs, int M, float* state, long slot_stride, const int* entry_meta, int n_entries,
                                      const int* chunks, int n_chunks, const int* spans, float* scratch, float* o, int heads, int dk,
                                      int dv, hipStream_t stream) {
  ti_scan_inputs in = *inputs;
  if (check_scan("linear_scan", &in, slot_stride, heads, dk, dv)) return 1;
  TI_REQUIRE(chunks && spans && scratch && n_chunks >= n_entries, "linear_scan: chunks need their lists and scratch");
  if (n_entries == 0 || M == 0) return 0;
  if (in.rot_dims) {
    const int half = in.rot_dims / 2;
    const bool vec = half % 4 == 0 && dk % 4 == 0 && in.ld % 4 == 0 && in.off_q % 4 == 0 && in.off_k % 4 == 0 && ((uintptr_t)in.proj & 15) == 0;
    const int each = vec ? 1024 : 256, pieces = (2 * in.qk_heads * half + each - 1) / each;
    const dim3 grid(M, pieces < 64 ? pieces : 64);
    if (vec) scan_rotate_kernel<true><<<grid, 256, 0, stream>>>((float*)in.proj, in, dk);
    else scan_rotate_kernel<false><<<grid, 256, 0, stream>>>((float*)in.proj, in, dk);
    in.rot_dims = 0;
  }
  const bool vec = dk % 4 == 0 && dv % 4 == 0 && in.ld % 4 == 0 && in.off_q % 4 == 0 && in.off_k % 4 == 0 && in.off_v % 4 == 0 &&
                   (((uintptr_t)in.proj | (uintptr_t)scratch) & 15) == 0;
#define SCAN_CHUNKS(F)                                                                                                                    \
  do {                                                                                                                                    \
    if (vec) launch_chunks<F, true>(in, state, slot_stride, entry_meta, n_entries, chunks, n_chunks, spans, scratch, o, heads, dk, dv, stream); \
    else launch_chunks<F, false>(in, state, slot_stride, entry_meta, n_entries, chunks, n_chunks, spans, scratch, o, heads, dk, dv, stream);    \
  } while (0)
  switch (scan_form(&in)) {
    case SCAN_SILU: SCAN_CHUNKS(SCAN_SILU); break;
    case SCAN_ROTATED: SCAN_CHUNKS(SCAN_ROTATED); break;
    default: SCAN_CHUNKS(SCAN_SELECTIVE);
  }
#undef SCAN_CHUNKS
  TI_LAUNCH_CHECK();
  return 0;
}

// The norm behind such a mixer and its gate: a row of W entries in `groups` equal runs, each divided by its own root mean square,
// times w (null: none), with the gate's activation of gate columns off_g .. (0: sigmoid, 1: silu) multiplied in behind the
// norm, or in front of it (gate_first); rounded once to T.  TPR threads a run (a wavefront or the whole workgroup), each N
// neighbouring entries at a time (N 4: everything aligned to 16 bytes), PIECES of them in registers (0: any length, from memory).
template <typename T, int TPR, int N, int PIECES>
__global__ void __launch_bounds__(256)
gated_group_norm_kernel(const float* __restrict__ o, const float* __restrict__ gate, int ld, int off_g, const float* __restrict__ w,
                        T* __restrict__ out, int M, int W, int groups, float eps, int silu, int gate_first) {
  __shared__ float red[4];
  const int size = W / groups;
  const long run = (long)blockIdx.x * (256 / TPR) + threadIdx.x / TPR;
  if (run >= (long)M * groups) return;      // (whole wavefronts; with a workgroup a run there is none)
  const int lane = threadIdx.x % TPR;
  const size_t m = run / groups;
  const int c0 = (int)(run % groups) * size;
  const float* src = o + m * W + c0;
  const float* g = gate + m * ld + off_g + c0;
  const float* wr = w ? w + c0 : nullptr;
  T* dst = out + m * W + c0;
  auto gate_of = [&](float z) { return silu ? la_silu(z) : 1.0f / (1.0f + expf(-z)); };
  auto total = [&](float ss) {
    if (TPR == 256) return block_sum<256>(ss, red);
    return group_sum<TI_WAVE>(ss);
  };
  if constexpr (PIECES > 0) {
    float v[PIECES][N], f[PIECES][N];
#pragma unroll
    for (int i = 0; i < PIECES; ++i) {
      const int c = (lane + TPR * i) * N;
#pragma unroll
      for (int j = 0; j < N; ++j) v[i][j] = f[i][j] = 0.f;
      if (c < size) {
        if constexpr (N == 4) {
          const float4 a = *reinterpret_cast<const float4*>(src + c), b = *reinterpret_cast<const float4*>(g + c);
          v[i][0] = a.x; v[i][1] = a.y; v[i][2] = a.z; v[i][3] = a.w;
          f[i][0] = b.x; f[i][1] = b.y; f[i][2] = b.z; f[i][3] = b.w;
        } else {
          v[i][0] = src[c];
          f[i][0] = g[c];
        }
      }
    }
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < PIECES; ++i)
#pragma unroll
      for (int j = 0; j < N; ++j) {
        f[i][j] = gate_of(f[i][j]);
        if (gate_first) v[i][j] *= f[i][j];
        ss = fmaf(v[i][j], v[i][j], ss);
      }
    const float inv = 1.0f / sqrtf(total(ss) / (float)size + eps);
#pragma unroll
    for (int i = 0; i < PIECES; ++i) {
      const int c = (lane + TPR * i) * N;
      if (c >= size) continue;
      float y[N];
#pragma unroll
      for (int j = 0; j < N; ++j) y[j] = v[i][j] * inv * (wr ? wr[c + j] : 1.f) * (gate_first ? 1.f : f[i][j]);
      if constexpr (N == 4) {
        if constexpr (sizeof(T) == 2) *reinterpret_cast<uint2*>(dst + c) = make_uint2(pack_bf16x2(y[0], y[1]), pack_bf16x2(y[2], y[3]));
        else *reinterpret_cast<float4*>(dst + c) = make_float4(y[0], y[1], y[2], y[3]);
      } else {
        st<T>(dst + c, y[0]);
      }
    }
  } else {
    float ss = 0.f;
    for (int c = lane; c < size; c += TPR) {
      const float v = gate_first ? src[c] * gate_of(g[c]) : src[c];
      ss = fmaf(v, v, ss);
    }
    const float inv = 1.0f / sqrtf(total(ss) / (float)size + eps);
    for (int c = lane; c < size; c += TPR) st<T>(dst + c, src[c] * inv * (wr ? wr[c] : 1.f) * gate_of(g[c]));
  }
}

template <typename T>
static void launch_group_norm(bool vec, const float* o, const float* gate, int ld, int off_g, const float* w, void* out, int M, int W, int groups,
                              float eps, int silu, int gate_first, hipStream_t stream) {
  const int size = W / groups;
  const long runs = (long)M * groups;
#define GGN(TPR, N, P)                                                                                                              \
  gated_group_norm_kernel<T, TPR, N, P><<<(unsigned)((runs + 256 / TPR - 1) / (256 / TPR)), 256, 0, stream>>>(o, gate, ld, off_g, w, (T*)out, M, W, \
                                                                                                           groups, eps, silu, gate_first)
  if (vec && size <= 256) GGN(64, 4, 1);
  else if (!vec && size <= 64) GGN(64, 1, 1);
  else if (!vec && size <= 256) GGN(64, 1, 4);
  else if (vec && size <= 1024) GGN(256, 4, 1);
  else if (vec && size <= 2048) GGN(256, 4, 2);
  else if (vec && size <= 4096) GGN(256, 4, 4);
  else if (vec && size <= 8192) GGN(256, 4, 8);
  else GGN(256, 1, 0);
#undef GGN
}

extern "C" int ti_gated_group_norm(int out_dtype, const float* o, const float* gate, int ld, int off_g, const float* w, void* out, int M,
                                   int W, int groups, float eps, int silu, int gate_first, hipStream_t stream) {
  TI_REQUIRE(M >= 0 && W > 0 && groups > 0 && W % groups == 0 && off_g >= 0 && off_g + W <= ld,
             "gated_group_norm: bad sizes M=%d W=%d in %d runs, gate columns %d of %d", M, W, groups, off_g, ld);
  TI_REQUIRE(out_dtype == TI_F32 || out_dtype == TI_BF16, "gated_group_norm: unknown dtype %d", out_dtype);
  if (M == 0) return 0;
  const bool vec = (W / groups) % 4 == 0 && ld % 4 == 0 && off_g % 4 == 0 && (((uintptr_t)o | (uintptr_t)gate | (uintptr_t)out) & 15) == 0;
  if (out_dtype == TI_F32) launch_group_norm<float>(vec, o, gate, ld, off_g, w, out, M, W, groups, eps, silu, gate_first, stream);
  else launch_group_norm<bf16_t>(vec, o, gate, ld, off_g, w, out, M, W, groups, eps, silu, gate_first, stream);
  TI_LAUNCH_CHECK();
  return 0;
}
