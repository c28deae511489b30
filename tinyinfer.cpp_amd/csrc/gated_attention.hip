// libti_gated_attention: softmax attention with what sits around it in gated layers, for any sizes up to 256 and both
// storage types (the float32 path of such layers, and the path of sizes the matrix-core kernels do not take).
//
//   preparation   from the 32-bit sums of one stacked projection [q | k | v | ...]: per-head RMS norms of q and k (a weight
//                 of the head's size shared by all heads, before the rotation; or none, behind it), rotation of the first
//                 rot_dims entries of every query and key head (entry i with entry i + rot_dims / 2, or neighbours in pairs),
//                 values that are the keys as projected (no v columns), values mixed with the values another layer left for
//                 the same tokens, q out, k and v into the pages
//   attention     causal softmax over the pages with a learned number a head in the denominator (a sink: no key, no value,
//                 not scaled) and a sigmoid gate on the output, one number an entry or one a head, read from the 32-bit sums
//
// A page is K [n_kv][P][dk] | V [n_kv][dvr][P], as the other attention kernels of keys and values of their own sizes read it;
// dvr >= dv rows a value head: rows beyond dv are written as zeros (values padded to the keys' size, so that kernels that
// hold keys and values of one size can read the pages).
#include "common.h"
#include "tinyinfer_kernels.h"

TI_ERROR_API

__device__ __forceinline__ void ga_rotation(const float* __restrict__ inv_freq, const float* __restrict__ rope_table, int table_len,
                                            float mag, int half, int p, int i, float* c, float* s) {
  if (rope_table && p < table_len) {
    *c = rope_table[((size_t)p * half + i) * 2];
    *s = rope_table[((size_t)p * half + i) * 2 + 1];
  } else {
    const float a = (float)p * inv_freq[i];
    *c = cosf(a) * mag;
    *s = sinf(a) * mag;
  }
}

// A wavefront per token and HPW query or key heads (one after the other in the order q, k), four wavefronts to a workgroup: the
// position, its page and its angles are fetched once for the heads of a wavefront, whose loads are in flight together.  Behind
// them (blockIdx.y = the number of such workgroups a token) workgroups of sixteen tokens and one value head each: the values pass
// through LDS, so that sixteen tokens that lie in a page one after the other are written sixteen to a piece.  Values that are the
// keys as projected are written by the key heads.
// pairs: entries 2i and 2i + 1 turn together (else i and i + rot_dims / 2); unit_norm: the head divided by its root mean square
// behind the rotation.  DPL: entries of a head a lane holds.
#define GA_PREP_WAVES 4
#define GA_V_TOKENS 16
template <typename T>
__device__ __forceinline__ void prep_values(const float* __restrict__ proj, int ld, int off_v, int mix_mode, const float* __restrict__ mix_lambda,
                                            float* __restrict__ v_kept, const int* __restrict__ pos, const int* __restrict__ slot,
                                            const int* __restrict__ table, int table_stride, T* __restrict__ pool, int M, int n_kv, int dk,
                                            int dv, int dvr, int P) {
  __shared__ T s_v[256][GA_V_TOKENS + 2];
  __shared__ int s_page[GA_V_TOKENS], s_row[GA_V_TOKENS];
  const int item = blockIdx.x;
  const int n_groups = (M + GA_V_TOKENS - 1) / GA_V_TOKENS;
  if (item >= n_groups * n_kv) return;
  const int m0 = item / n_kv * GA_V_TOKENS, h = item % n_kv, n = min(GA_V_TOKENS, M - m0);
  if (threadIdx.x < GA_V_TOKENS) {
    const int i = threadIdx.x;
    int page = -1, r = 0;
    if (i < n) {
      const int p = pos[m0 + i];
      page = table[(size_t)slot[m0 + i] * table_stride + p / P];
      r = p % P;
    }
    s_page[i] = page;
    s_row[i] = r;
  }
  const float lam = mix_mode == 2 ? mix_lambda[0] : 0.f;
  for (int e = threadIdx.x; e < n * dvr; e += TI_WAVE * GA_PREP_WAVES) {
    const int i = e / dvr, d = e % dvr, m = m0 + i;
    float x = 0.f;                                                    // rows beyond the value's size: zeros
    if (d < dv) {
      x = proj[(size_t)m * ld + off_v + (size_t)h * dv + d];
      float* kept = v_kept ? v_kept + ((size_t)m * n_kv + h) * dv + d : nullptr;
      if (mix_mode == 1) *kept = x;                                   // the layer whose values the later ones mix in
      else if (mix_mode == 2) x = fmaf(lam, *kept, (1.0f - lam) * x);
    }
    st<T>(&s_v[d][i], x);
  }
  __syncthreads();
  const size_t page_elems = (size_t)n_kv * P * (dk + dvr), v_off = (size_t)n_kv * P * dk + (size_t)h * dvr * P;
  // one run of sixteen rows of one page, on a boundary of sixteen
  bool run = n == GA_V_TOKENS && P % GA_V_TOKENS == 0 && s_page[0] >= 0 && s_row[0] % GA_V_TOKENS == 0 && (((uintptr_t)pool | (page_elems * sizeof(T)) | (v_off * sizeof(T))) & 15) == 0;
#pragma unroll
  for (int i = 1; i < GA_V_TOKENS; ++i) run = run && s_page[i] == s_page[0] && s_row[i] == s_row[0] + i;
  if (run) {
    constexpr int N = 16 / sizeof(T), PIECES = GA_V_TOKENS / N;       // elements of a piece of 16 bytes, pieces of a value's entry
    T* base = pool + (size_t)s_page[0] * page_elems + v_off + s_row[0];
    for (int e = threadIdx.x; e < dvr * PIECES; e += TI_WAVE * GA_PREP_WAVES) {
      const int d = e / PIECES, k = e % PIECES;
      T v[N];
#pragma unroll
      for (int j = 0; j < N; ++j) v[j] = s_v[d][k * N + j];
      uint4 out;
      __builtin_memcpy(&out, v, 16);
      *reinterpret_cast<uint4*>(base + (size_t)d * P + k * N) = out;
    }
    return;
  }
  for (int e = threadIdx.x; e < n * dvr; e += TI_WAVE * GA_PREP_WAVES) {
    const int i = e % n, d = e / n;
    if (s_page[i] >= 0) pool[(size_t)s_page[i] * page_elems + v_off + (size_t)d * P + s_row[i]] = s_v[d][i];
  }
}

template <typename T, int DPL, int HPW>
__global__ void __launch_bounds__(TI_WAVE * GA_PREP_WAVES)
gated_qkv_prep_kernel(const float* __restrict__ proj, int ld, int off_q, int off_k, int off_v, const float* __restrict__ q_w,
                      const float* __restrict__ k_w, float eps, const float* __restrict__ inv_freq,
                      const float* __restrict__ rope_table, int table_len, float mag, int rot_dims, int mix_mode,
                      const float* __restrict__ mix_lambda, float* __restrict__ v_kept, const int* __restrict__ pos,
                      const int* __restrict__ slot, const int* __restrict__ table, int table_stride, T* __restrict__ pool,
                      T* __restrict__ q_out, int M, int n_head, int n_kv, int dk, int dv, int dvr, int P, int pairs, int unit_norm) {
  __shared__ float s_all[GA_PREP_WAVES][DPL * TI_WAVE];
  const int per_group = GA_PREP_WAVES * HPW;
  const int n_units = (n_head + n_kv + per_group - 1) / per_group;
  if ((int)blockIdx.y >= n_units) {
    prep_values<T>(proj, ld, off_v, mix_mode, mix_lambda, v_kept, pos, slot, table, table_stride, pool, M, n_kv, dk, dv, dvr, P);
    return;
  }
  if ((int)blockIdx.x >= M) return;
  const int m = blockIdx.x, wave = threadIdx.x / TI_WAVE, lane = threadIdx.x % TI_WAVE;
  const int first = blockIdx.y * per_group + wave * HPW, n = min(HPW, n_head + n_kv - first);
  if (n <= 0) return;      // (no barrier below: a wavefront keeps to itself)
  float* const s_h = s_all[wave];
  const int p = pos[m];
  const float* row = proj + (size_t)m * ld;
  float v[HPW][DPL];
#pragma unroll
  for (int k = 0; k < HPW; ++k) {
    const int unit = first + min(k, n - 1);      // (heads beyond the last: the last one again, not written)
    const float* src = unit < n_head ? row + off_q + (size_t)unit * dk : row + off_k + (size_t)(unit - n_head) * dk;
#pragma unroll
    for (int i = 0; i < DPL; ++i) {
      const int d = lane + i * TI_WAVE;
      v[k][i] = d < dk ? src[d] : 0.f;
    }
  }
  const int page = table[(size_t)slot[m] * table_stride + p / P];
  const int r = p % P;
  const int half = inv_freq ? rot_dims / 2 : 0;
  float c[DPL], s[DPL];
#pragma unroll
  for (int i = 0; i < DPL; ++i) {
    const int d = lane + i * TI_WAVE;
    c[i] = 1.f;
    s[i] = 0.f;
    if (d < 2 * half) ga_rotation(inv_freq, rope_table, table_len, mag, half, p, pairs ? d >> 1 : d < half ? d : d - half, &c[i], &s[i]);
  }
  T* base = pool + (size_t)max(page, 0) * ((size_t)n_kv * P * (dk + dvr));
#pragma unroll
  for (int k = 0; k < HPW; ++k) {
    const int unit = first + k;
    const bool is_q = unit < n_head;
    const int h = is_q ? unit : unit - n_head;
    if (k < n && !is_q && off_v < 0 && page >= 0) {
      // the values are the keys as projected: before norm and rotation
      T* vbase = base + (size_t)n_kv * P * dk + (size_t)h * dvr * P + r;
#pragma unroll
      for (int i = 0; i < DPL; ++i) {
        const int d = lane + i * TI_WAVE;
        if (d < dv) st<T>(vbase + (size_t)d * P, v[k][i]);
      }
    }
    const float* nw = is_q ? q_w : k_w;
    if (nw) {
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < DPL; ++i) ss = fmaf(v[k][i], v[k][i], ss);      // (entries beyond the head are zero)
      const float inv = 1.0f / sqrtf(group_sum<TI_WAVE>(ss) / (float)dk + eps);
#pragma unroll
      for (int i = 0; i < DPL; ++i) {
        const int d = lane + i * TI_WAVE;
        if (d < dk) v[k][i] = v[k][i] * inv * nw[d];
      }
    }
    if (half > 0 && pairs) {
      // neighbours lie in neighbouring lanes
#pragma unroll
      for (int i = 0; i < DPL; ++i)
        if (i * TI_WAVE < 2 * half) {      // (the same in every lane)
          const float other = __shfl_xor(v[k][i], 1, TI_WAVE);
          if (lane + i * TI_WAVE < 2 * half) v[k][i] = (lane & 1) ? v[k][i] * c[i] + other * s[i] : v[k][i] * c[i] - other * s[i];
        }
    } else if (half > 0) {
#pragma unroll
      for (int i = 0; i < DPL; ++i) s_h[lane + i * TI_WAVE] = v[k][i];
      __threadfence_block();      // (a wavefront's LDS accesses are served in order)
#pragma unroll
      for (int i = 0; i < DPL; ++i) {
        const int d = lane + i * TI_WAVE;
        if (d < 2 * half) v[k][i] = d < half ? s_h[d] * c[i] - s_h[d + half] * s[i] : s_h[d] * c[i] + s_h[d - half] * s[i];
      }
      __threadfence_block();
    }
    if (unit_norm) {
      float sr = 0.f;
#pragma unroll
      for (int i = 0; i < DPL; ++i) sr = fmaf(v[k][i], v[k][i], sr);
      const float inv = 1.0f / sqrtf(group_sum<TI_WAVE>(sr) / (float)dk + eps);
#pragma unroll
      for (int i = 0; i < DPL; ++i) v[k][i] *= inv;
    }
    if (k >= n || (!is_q && page < 0)) continue;      // the host reserves pages first; never write astray
    T* dst = is_q ? q_out + ((size_t)m * n_head + h) * dk : base + ((size_t)h * P + r) * dk;
#pragma unroll
    for (int i = 0; i < DPL; ++i) {
      const int d = lane + i * TI_WAVE;
      if (d < dk) st<T>(dst + d, v[k][i]);
    }
  }
}

extern "C" int ti_gated_qkv_prep(int dtype, const float* proj, int ld, int off_q, int off_k, int off_v, const float* q_w,
                                 const float* k_w, float eps, const float* inv_freq, const float* rope_table, int table_len,
                                 float mag, int rot_dims, int mix_mode, const float* mix_lambda, float* v_kept, const int* pos,
                                 const int* slot, const int* table, int table_stride, void* pool, void* q_out, int M, int n_head,
                                 int n_kv, int dk, int dv, int dv_rows, int page_size, hipStream_t stream) {
  return ti_gated_qkv_prep_form(dtype, proj, ld, off_q, off_k, off_v, q_w, k_w, eps, inv_freq, rope_table, table_len, mag, rot_dims, mix_mode,
                                mix_lambda, v_kept, pos, slot, table, table_stride, pool, q_out, M, n_head, n_kv, dk, dv, dv_rows, page_size,
                                0, 0, stream);
}

extern "C" int ti_gated_qkv_prep_form(int dtype, const float* proj, int ld, int off_q, int off_k, int off_v, const float* q_w,
                                      const float* k_w, float eps, const float* inv_freq, const float* rope_table, int table_len,
                                      float mag, int rot_dims, int mix_mode, const float* mix_lambda, float* v_kept, const int* pos,
                                      const int* slot, const int* table, int table_stride, void* pool, void* q_out, int M, int n_head,
                                      int n_kv, int dk, int dv, int dv_rows, int page_size, int pairs, int unit_norm, hipStream_t stream) {
  const int dvr = dv_rows > 0 ? dv_rows : dv;
  TI_REQUIRE(n_head > 0 && n_kv > 0 && dk > 0 && dk <= 256 && dv > 0 && dv <= 256 && dvr >= dv && dvr <= 256 && page_size > 0 &&
                 table_stride > 0 && n_head + n_kv <= 65535,
             "gated_qkv_prep: bad sizes heads=%d kv_heads=%d dk=%d dv=%d (%d rows) page=%d", n_head, n_kv, dk, dv, dvr, page_size);
  TI_REQUIRE(!inv_freq || (rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= dk),
             "gated_qkv_prep: %d rotated entries do not fit a head of %d (even, at most the head)", rot_dims, dk);
  TI_REQUIRE(off_v >= 0 || dv == dk, "gated_qkv_prep: values that are the keys have the keys' size (%d, not %d)", dk, dv);
  TI_REQUIRE(mix_mode == 0 || (off_v >= 0 && v_kept && (mix_mode == 1 || (mix_mode == 2 && mix_lambda))),
             "gated_qkv_prep: mixing values (mode %d) needs value columns, the kept values and the factor", mix_mode);
  TI_REQUIRE(off_q >= 0 && off_k >= 0 && off_q + n_head * dk <= ld && off_k + n_kv * dk <= ld && (off_v < 0 || off_v + n_kv * dv <= ld),
             "gated_qkv_prep: the columns do not lie inside rows of %d", ld);
  if (M == 0) return 0;
  const int n_groups = off_v < 0 ? 0 : (M + GA_V_TOKENS - 1) / GA_V_TOKENS * n_kv;       // workgroups of the values
  // few tokens: a wavefront a head; many: four heads a wavefront (the same arithmetic)
  const int hpw = (long)M * (n_head + n_kv) > 8192 ? 4 : 1;
  const int per_group = GA_PREP_WAVES * hpw;
  const dim3 grid(M > n_groups ? M : n_groups, (n_head + n_kv + per_group - 1) / per_group + (n_groups ? 1 : 0));
#define GA_PREP(T, D, N)                                                                                                               \
  gated_qkv_prep_kernel<T, D, N><<<grid, TI_WAVE * GA_PREP_WAVES, 0, stream>>>(proj, ld, off_q, off_k, off_v, q_w, k_w, eps, inv_freq, \
                                                                               rope_table, table_len, mag, rot_dims, mix_mode,         \
                                                                               mix_lambda, v_kept, pos, slot, table, table_stride,     \
                                                                               (T*)pool, (T*)q_out, M, n_head, n_kv, dk, dv, dvr,      \
                                                                               page_size, pairs, unit_norm)
#define GA_PREP_SIZE(T)                   \
  do {                                    \
    if (dk <= 64) {                       \
      if (hpw == 4) GA_PREP(T, 1, 4);     \
      else GA_PREP(T, 1, 1);              \
    } else if (dk <= 128) {               \
      if (hpw == 4) GA_PREP(T, 2, 4);     \
      else GA_PREP(T, 2, 1);              \
    } else {                              \
      if (hpw == 4) GA_PREP(T, 4, 4);     \
      else GA_PREP(T, 4, 1);              \
    }                                     \
  } while (0)
  if (dtype == TI_F32) GA_PREP_SIZE(float);
  else if (dtype == TI_BF16) GA_PREP_SIZE(bf16_t);
  else
    TI_REQUIRE(false, "gated_qkv_prep: unknown dtype %d", dtype);
#undef GA_PREP_SIZE
#undef GA_PREP
  TI_LAUNCH_CHECK();
  return 0;
}

// The gate on its own, behind attention kernels that do not take it in: out[m, h dv + d] = src[m, h src_dv + d] times
// sigmoid(gate[m, h dv + d] or gate[m, h]) (gate null: times one).  src_dv > dv: the heads of src are padded and come out packed;
// src may be out where src_dv = dv.
template <typename T>
__global__ void sigmoid_gate_kernel(const T* __restrict__ src, int src_dv, T* __restrict__ out, const float* __restrict__ gate,
                                    int gate_ld, int gate_mode, long n, int n_head, int dv) {
  const int W = n_head * dv;
  for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (long)gridDim.x * blockDim.x) {
    const long m = i / W;
    const int c = (int)(i % W), h = c / dv;
    float y = ld<T>(src + m * ((long)n_head * src_dv) + (long)h * src_dv + (c - h * dv));
    if (gate) y *= 1.0f / (1.0f + expf(-gate[m * gate_ld + (gate_mode == 1 ? c : h)]));
    st<T>(out + i, y);
  }
}

// the same, eight neighbouring entries a thread: dv a multiple of 8, 16-byte aligned rows; the same bits.  Grid (pieces of the
// heads side by side, rows).
__global__ void __launch_bounds__(256)
sigmoid_gate_wide_kernel(const bf16_t* __restrict__ src, int src_dv, bf16_t* __restrict__ out, const float* __restrict__ gate, int gate_ld,
                         int gate_mode, int n_head, int dv) {
  const int m = blockIdx.y, c = (blockIdx.x * 256 + threadIdx.x) * 8;
  const int W = n_head * dv;
  if (c >= W) return;
  const int h = c / dv;
  const uint4 a = *reinterpret_cast<const uint4*>(src + (size_t)m * n_head * src_dv + (size_t)h * src_dv + (c - h * dv));
  const unsigned w[4] = {a.x, a.y, a.z, a.w};
  float y[8];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    y[2 * i] = __uint_as_float(w[i] << 16);
    y[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
  }
  if (gate) {
    const float* g = gate + (size_t)m * gate_ld;
    if (gate_mode == 2) {
      const float s = 1.0f / (1.0f + expf(-g[h]));
#pragma unroll
      for (int i = 0; i < 8; ++i) y[i] *= s;
    } else {
#pragma unroll
      for (int i = 0; i < 8; ++i) y[i] *= 1.0f / (1.0f + expf(-g[c + i]));
    }
  }
  *reinterpret_cast<uint4*>(out + (size_t)m * W + c) = make_uint4(pack_bf16x2(y[0], y[1]), pack_bf16x2(y[2], y[3]), pack_bf16x2(y[4], y[5]),
                                                                  pack_bf16x2(y[6], y[7]));
}

extern "C" int ti_sigmoid_gate(int dtype, const void* src, int src_dv, void* out, const float* gate, int gate_ld, int gate_mode, int M,
                               int n_head, int dv, hipStream_t stream) {
  TI_REQUIRE(M >= 0 && n_head > 0 && dv > 0 && src_dv >= dv && (src != out || src_dv == dv) &&
                 (!gate || (gate_mode == 1 && gate_ld >= n_head * dv) || (gate_mode == 2 && gate_ld >= n_head)),
             "sigmoid_gate: bad sizes M=%d heads=%d dv=%d (from %d) gate mode %d in rows of %d", M, n_head, dv, src_dv, gate_mode, gate_ld);
  if (M == 0) return 0;
  if (dtype == TI_BF16 && dv % 8 == 0 && src_dv % 8 == 0 && M <= 65535 && (((uintptr_t)src | (uintptr_t)out) & 15) == 0) {
    sigmoid_gate_wide_kernel<<<dim3((n_head * dv / 8 + 255) / 256, M), 256, 0, stream>>>((const bf16_t*)src, src_dv, (bf16_t*)out, gate, gate_ld,
                                                                                        gate_mode, n_head, dv);
    TI_LAUNCH_CHECK();
    return 0;
  }
  const long n = (long)M * n_head * dv;
  const unsigned blocks = (unsigned)((n + 255) / 256 < 16384 ? (n + 255) / 256 : 16384);
  if (dtype == TI_F32)
    sigmoid_gate_kernel<float><<<blocks, 256, 0, stream>>>((const float*)src, src_dv, (float*)out, gate, gate_ld, gate_mode, n, n_head, dv);
  else if (dtype == TI_BF16)
    sigmoid_gate_kernel<bf16_t><<<blocks, 256, 0, stream>>>((const bf16_t*)src, src_dv, (bf16_t*)out, gate, gate_ld, gate_mode, n, n_head, dv);
  else
    TI_REQUIRE(false, "sigmoid_gate: unknown dtype %d", dtype);
  TI_LAUNCH_CHECK();
  return 0;
}

// ------------------------------------------------------------------------------------------------
// A workgroup per (row, head): sixteen groups of sixteen lanes, group g the keys at positions g, g + 16, ... with a running
// softmax each, merged in a fixed order (a key's group depends on its position alone, so every cut of the same tokens takes
// the same sums in the same order).  The sink joins the merge as a share of its own with maximum sink[h], weight 1 and no
// values.  gate (null: none): rows of gate_ld floats; gate_mode 1: entry h * dv + d of the row, 2: entry h.
#define GA_LANES 16
#define GA_GROUPS 16

template <typename T, int DPL>
__global__ void __launch_bounds__(256)
gated_attention_kernel(const T* __restrict__ q, const T* __restrict__ pool, const int* __restrict__ table, int table_stride,
                       const int* __restrict__ pos, const int* __restrict__ slot, const float* __restrict__ sink,
                       const float* __restrict__ gate, int gate_ld, int gate_mode, T* __restrict__ out, int n_head, int n_kv,
                       int dk, int dv, int dvr, int P, float scale, int window) {
  constexpr int HD = DPL * GA_LANES;
  __shared__ float s_o[GA_GROUPS][HD];
  __shared__ float s_m[GA_GROUPS], s_l[GA_GROUPS];
  const int m = blockIdx.x, h = blockIdx.y;
  const int g = threadIdx.x / GA_LANES, lane = threadIdx.x % GA_LANES;
  const int kvh = h / (n_head / n_kv);
  const int p_q = pos[m];
  const int lo = (window > 0 && p_q - window + 1 > 0) ? p_q - window + 1 : 0;
  const int* tab = table + (size_t)slot[m] * table_stride;
  const size_t page_elems = (size_t)n_kv * P * (dk + dvr);
  const size_t k_off = (size_t)kvh * P * dk;
  const size_t v_off = (size_t)n_kv * P * dk + (size_t)kvh * dvr * P;

  float qv[DPL], o[DPL];
  const T* qh = q + ((size_t)m * n_head + h) * dk;
#pragma unroll
  for (int i = 0; i < DPL; ++i) {
    const int d = lane + i * GA_LANES;
    qv[i] = d < dk ? ld<T>(qh + d) : 0.f;
    o[i] = 0.f;
  }
  float mx = -INFINITY, l = 0.f;
  for (int p = lo - lo % GA_GROUPS + g; p <= p_q; p += GA_GROUPS) {
    if (p < lo) continue;
    const int page = tab[p / P];
    if (page < 0) continue;
    const T* kp = pool + (size_t)page * page_elems + k_off + (size_t)(p % P) * dk;
    const T* vp = pool + (size_t)page * page_elems + v_off + (p % P);
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < DPL; ++i) {
      const int d = lane + i * GA_LANES;
      if (d < dk) s = fmaf(qv[i], ld<T>(kp + d), s);
    }
    s = group_sum<GA_LANES>(s) * scale;
    const float m_new = fmaxf(mx, s);
    const float alpha = expf(mx - m_new);
    const float w = expf(s - m_new);
    l = l * alpha + w;
#pragma unroll
    for (int i = 0; i < DPL; ++i) {
      const int d = lane + i * GA_LANES;
      if (d < dv) o[i] = o[i] * alpha + w * ld<T>(vp + (size_t)d * P);
    }
    mx = m_new;
  }
#pragma unroll
  for (int i = 0; i < DPL; ++i) s_o[g][lane + i * GA_LANES] = o[i];
  if (lane == 0) {
    s_m[g] = mx;
    s_l[g] = l;
  }
  __syncthreads();
  const float sk = sink ? sink[h] : -INFINITY;
  const float* grow = gate ? gate + (size_t)m * gate_ld : nullptr;
  for (int d = threadIdx.x; d < dv; d += 256) {
    float mm = sk;
#pragma unroll
    for (int j = 0; j < GA_GROUPS; ++j) mm = fmaxf(mm, s_m[j]);
    float lt = sink ? expf(sk - mm) : 0.f, acc = 0.f;
#pragma unroll
    for (int j = 0; j < GA_GROUPS; ++j) {
      const float w = (s_m[j] == -INFINITY) ? 0.f : expf(s_m[j] - mm);
      lt += s_l[j] * w;
      acc += s_o[j][d] * w;
    }
    float y = acc / lt;
    if (grow) {
      const float z = grow[gate_mode == 1 ? h * dv + d : h];
      y *= 1.0f / (1.0f + expf(-z));
    }
    st<T>(out + ((size_t)m * n_head + h) * dv + d, y);
  }
}

template <typename T>
static int launch_gated(int dpl, dim3 grid, const void* q, const void* pool, const int* table, int table_stride, const int* pos,
                        const int* slot, const float* sink, const float* gate, int gate_ld, int gate_mode, void* out, int n_head,
                        int n_kv, int dk, int dv, int dvr, int P, float scale, int window, hipStream_t stream) {
#define GA_CASE(D)                                                                                                       \
  case D:                                                                                                                \
    gated_attention_kernel<T, D><<<grid, 256, 0, stream>>>((const T*)q, (const T*)pool, table, table_stride, pos, slot, sink, \
                                                           gate, gate_ld, gate_mode, (T*)out, n_head, n_kv, dk, dv, dvr, P, scale, \
                                                           window);                                                      \
    break;
  switch (dpl) {
    GA_CASE(1) GA_CASE(2) GA_CASE(3) GA_CASE(4) GA_CASE(5) GA_CASE(6) GA_CASE(7) GA_CASE(8)
    GA_CASE(9) GA_CASE(10) GA_CASE(11) GA_CASE(12) GA_CASE(13) GA_CASE(14) GA_CASE(15) GA_CASE(16)
    default:
      return 1;
  }
#undef GA_CASE
  return 0;
}

// q: [M, n_head, dk], out: [M, n_head, dv] in T
extern "C" int ti_gated_attention_rows(int dtype, const void* q, const void* pool, const int* table, int table_stride,
                                       const int* pos, const int* slot, const float* sink, const float* gate, int gate_ld,
                                       int gate_mode, void* out, int M, int n_head, int n_kv, int dk, int dv, int dv_rows, int page_size,
                                       float scale, int window, hipStream_t stream) {
  const int dvr = dv_rows > 0 ? dv_rows : dv;
  TI_REQUIRE(dvr >= dv && dvr <= 256, "gated attention: %d rows a value head do not hold values of %d", dvr, dv);
  TI_REQUIRE(dk >= 1 && dk <= 256 && dv >= 1 && dv <= 256, "gated attention: key size %d / value size %d are not served (up to 256)",
             dk, dv);
  TI_REQUIRE(n_head > 0 && n_kv > 0 && n_head % n_kv == 0 && n_head <= 65535, "gated attention: heads %d / kv_heads %d", n_head, n_kv);
  TI_REQUIRE(page_size > 0 && table_stride > 0, "gated attention: bad page_size %d / table_stride %d", page_size, table_stride);
  TI_REQUIRE(!gate || ((gate_mode == 1 && gate_ld >= n_head * dv) || (gate_mode == 2 && gate_ld >= n_head)),
             "gated attention: the gate (mode %d) does not fit rows of %d", gate_mode, gate_ld);
  if (M == 0) return 0;
  dim3 grid(M, n_head);
  const int big = dk > dv ? dk : dv;
  const int dpl = (big + GA_LANES - 1) / GA_LANES;
  int rc;
  if (dtype == TI_F32)
    rc = launch_gated<float>(dpl, grid, q, pool, table, table_stride, pos, slot, sink, gate, gate_ld, gate_mode, out, n_head, n_kv, dk,
                             dv, dvr, page_size, scale, window, stream);
  else if (dtype == TI_BF16)
    rc = launch_gated<bf16_t>(dpl, grid, q, pool, table, table_stride, pos, slot, sink, gate, gate_ld, gate_mode, out, n_head, n_kv,
                              dk, dv, dvr, page_size, scale, window, stream);
  else
    TI_REQUIRE(false, "gated attention: unknown dtype %d", dtype);
  TI_REQUIRE(rc == 0, "gated attention: no kernel for sizes %d / %d", dk, dv);
  TI_LAUNCH_CHECK();
  return 0;
}
