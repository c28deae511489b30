// A mixture of experts for any sizes, float32 or bfloat16 storage: the router (logits and scores in
// 32-bit, the `top` largest scores chosen, ties to the lower index) and the experts row by row:
//   y[m] = sum over the chosen experts e, in the order they were chosen, of  W_down[e] act(W_up[e] (s_e h[m]))
// with the score scaling the expert's input (scale_input) or its output, and act = relu(z)^2.
// Products accumulate in 32-bit with fused multiply-adds in a fixed order; what a product reads is rounded
// to the storage type first (the scaled input, the activated rows), as a matrix-core kernel's operands are.
#include "common.h"
#include "tinyinfer_kernels.h"

TI_ERROR_API

#define MOE_MAX_EXPERTS 1024
#define MOE_MAX_TOP 64

// score kinds
#define MOE_SIGMOID 0
#define MOE_SOFTMAX 1
#define MOE_SOFTMAX_CHOSEN 2      // the largest logits are chosen; the weights are the softmax over the chosen logits alone

template <typename T> struct Piece;
template <> struct Piece<float> {
  static constexpr int N = 4;
  static __device__ __forceinline__ void load(const float* p, float* v) {
    const float4 a = *reinterpret_cast<const float4*>(p);
    v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w;
  }
};
template <> struct Piece<bf16_t> {
  static constexpr int N = 8;
  static __device__ __forceinline__ void load(const bf16_t* p, float* v) {
    const uint4 a = *reinterpret_cast<const uint4*>(p);
    const unsigned w[4] = {a.x, a.y, a.z, a.w};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      v[2 * i] = __uint_as_float(w[i] << 16);
      v[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
    }
  }
};

// ------------------------------------------------------------ router
// A workgroup per TM tokens (1, or 4 in long steps: a row of the router is fetched once for four tokens).  Logits: wavefront w takes
// experts w, w + 4, ...; lanes share the tokens' rows in pieces of 16 bytes (lane l the pieces l, l + 64, ... in ascending order,
// then a butterfly).  Choice: wavefront t holds token t's scores (lane l the experts l, l + 64, ...) and takes the largest `top`
// times.  The order of every sum is the same whatever TM.
struct RouteForm {
  int W, E, top, score_kind, renormalize, n_groups, keep;
  float weight_scale, sum_floor;
};
// what lanes of the wavefront left in LDS is there for its other lanes
__device__ __forceinline__ void wave_publish() {
  __builtin_amdgcn_wave_barrier();
  __threadfence_block();
}
template <typename T, bool VEC, int TM>
__global__ void __launch_bounds__(256)
moe_route_kernel(const T* __restrict__ h, const float* __restrict__ router, int* __restrict__ ids, float* __restrict__ wts, int M,
                 const RouteForm a, const float* __restrict__ correction, const float* __restrict__ gate_row, float* __restrict__ gate_out) {
  extern __shared__ float s_route[];      // [TM][E] scores, [TM][E] the scores the weights are taken from, [TM][groups]
  const int E = a.E, W = a.W;
  const bool corrected = correction != nullptr || a.n_groups > 1;
  const int m0 = blockIdx.x * TM;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const T* rows[TM];
#pragma unroll
  for (int t = 0; t < TM; ++t) rows[t] = h + (size_t)min(m0 + t, M - 1) * W;
  auto dots = [&](const float* __restrict__ w, float* z) {      // w . every token's row
#pragma unroll
    for (int t = 0; t < TM; ++t) z[t] = 0.f;
    if (VEC) {
      constexpr int N = Piece<T>::N;
      for (int c = lane * N; c < W; c += 64 * N) {
        float f[N];
#pragma unroll
        for (int i = 0; i < N; ++i) f[i] = w[c + i];
#pragma unroll
        for (int t = 0; t < TM; ++t) {
          float v[N];
          Piece<T>::load(rows[t] + c, v);
#pragma unroll
          for (int i = 0; i < N; ++i) z[t] = fmaf(f[i], v[i], z[t]);
        }
      }
    } else {
      for (int c = lane; c < W; c += 64) {
        const float f = w[c];
#pragma unroll
        for (int t = 0; t < TM; ++t) z[t] = fmaf(f, ld<T>(rows[t] + c), z[t]);
      }
    }
#pragma unroll
    for (int t = 0; t < TM; ++t) z[t] = group_sum<64>(z[t]);
  };
  for (int e = wave; e < E; e += 4) {
    float z[TM];
    dots(router + (size_t)e * W, z);
    if (lane == 0) {
#pragma unroll
      for (int t = 0; t < TM; ++t) s_route[t * E + e] = z[t];
    }
  }
  if (gate_row && wave == E % 4) {      // one more row beside the router's: sigmoid(gate_row . h), a factor for another branch
    float z[TM];
    dots(gate_row, z);
    if (lane == 0) {
#pragma unroll
      for (int t = 0; t < TM; ++t)
        if (m0 + t < M) gate_out[m0 + t] = 1.0f / (1.0f + expf(-z[t]));
    }
  }
  __syncthreads();
  if (wave >= TM || m0 + wave >= M) return;
  const int m = m0 + wave;
  float* const s_score = s_route + wave * E;
  float* const s_plain = s_route + (TM + wave) * E;
  if (a.score_kind == MOE_SOFTMAX) {
    float mx = -INFINITY, sum = 0.f;
    for (int e = lane; e < E; e += 64) mx = fmaxf(mx, s_score[e]);
    mx = group_max<64>(mx);
    for (int e = lane; e < E; e += 64) sum += expf(s_score[e] - mx);
    sum = group_sum<64>(sum);
    for (int e = lane; e < E; e += 64) s_score[e] = expf(s_score[e] - mx) / sum;
  } else if (a.score_kind == MOE_SIGMOID) {
    for (int e = lane; e < E; e += 64) s_score[e] = 1.0f / (1.0f + expf(-s_score[e]));
  }
  if (corrected) {
    // the choice reads score + correction; the weights keep the score itself
    for (int e = lane; e < E; e += 64) {
      s_plain[e] = s_score[e];
      if (correction) s_score[e] += correction[e];
    }
    wave_publish();
    if (a.n_groups > 1) {
      // groups of E / n_groups neighbours: a group's score is the sum of its two largest choice scores; experts outside
      // the `keep` best groups (ties to the lower group) cannot be chosen
      float* const s_group = s_route + 2 * TM * E + wave * a.n_groups;
      const int per = E / a.n_groups;
      for (int g = lane; g < a.n_groups; g += 64) {
        float x = -INFINITY, y = -INFINITY;
        for (int e = g * per; e < (g + 1) * per; ++e) {
          const float s = s_score[e];
          if (s > x) {
            y = x;
            x = s;
          } else if (s > y) {
            y = s;
          }
        }
        s_group[g] = per > 1 ? x + y : x;
      }
      wave_publish();
      for (int g = lane; g < a.n_groups; g += 64) {
        int better = 0;
        for (int o = 0; o < a.n_groups; ++o) better += (s_group[o] > s_group[g] || (s_group[o] == s_group[g] && o < g)) ? 1 : 0;
        if (better >= a.keep)
          for (int e = g * per; e < (g + 1) * per; ++e) s_score[e] = -INFINITY;
      }
    }
  }
  wave_publish();
  const int top = a.top;
  float total = 0.f, first = 0.f;
  for (int k = 0; k < top; ++k) {
    float best = -INFINITY;
    int at = 0x7fffffff;
    for (int e = lane; e < E; e += 64) {
      const float s = s_score[e];
      if (s > best) {      // ascending e: the first of equals stays
        best = s;
        at = e;
      }
    }
    // the largest of all lanes, then the lowest index among those that hold it (indices are exact in 32-bit floats)
    const float largest = group_max<64>(best);
    const float low = -group_max<64>(best == largest && at < E ? -(float)at : -2048.f);
    best = largest;
    at = low < 2048.f ? (int)low : 0x7fffffff;
    if (at >= E) at = k;      // no score compares as larger (not a number): an expert that exists all the same
    if (corrected) best = s_plain[at];
    if (lane == 0) {
      ids[(size_t)m * top + k] = at;
      wts[(size_t)m * top + k] = best;
      s_score[at] = -INFINITY;
    }
    if (a.score_kind == MOE_SOFTMAX_CHOSEN) {
      // the first choice is the largest logit: every weight is exp(z - z_first) over the sum of those, in the order of choice
      if (k == 0) first = best;
      const float w = expf(best - first);
      if (lane == 0) wts[(size_t)m * top + k] = w;
      total += w;
    } else {
      total += best;
    }
    wave_publish();
  }
  if ((a.renormalize || a.score_kind == MOE_SOFTMAX_CHOSEN) && lane < top) wts[(size_t)m * top + lane] /= total + a.sum_floor;
  if (a.weight_scale != 1.f && lane < top) wts[(size_t)m * top + lane] *= a.weight_scale;
}

extern "C" int ti_moe_route(int dtype, const void* h, const float* router, int* ids, float* wts, int M, int W, int E, int top,
                            int score_kind, int renormalize, hipStream_t stream) {
  return ti_moe_route_grouped(dtype, h, router, nullptr, ids, wts, M, W, E, top, score_kind, renormalize, 0, 0, 1.f, 0.f, stream);
}

// the same with what a grouped router adds: `correction` f32 [E] (null: none) joins the scores for the choice only; the experts
// form n_groups groups of neighbours of which the `keep` best may be chosen from (n_groups <= 1: no groups); the weights are
// the chosen experts' uncorrected scores, divided by their sum + sum_floor where `renormalize`, times weight_scale
extern "C" int ti_moe_route_grouped(int dtype, const void* h, const float* router, const float* correction, int* ids, float* wts,
                                    int M, int W, int E, int top, int score_kind, int renormalize, int n_groups, int keep,
                                    float weight_scale, float sum_floor, hipStream_t stream) {
  return ti_moe_route_gate(dtype, h, router, correction, ids, wts, M, W, E, top, score_kind, renormalize, n_groups, keep, weight_scale,
                           sum_floor, nullptr, nullptr, stream);
}

// the same, and gate_out f32 [M] = sigmoid(gate_row . h) with gate_row f32 [W] (null: none), in 32-bit
extern "C" int ti_moe_route_gate(int dtype, const void* h, const float* router, const float* correction, int* ids, float* wts, int M, int W,
                                 int E, int top, int score_kind, int renormalize, int n_groups, int keep, float weight_scale,
                                 float sum_floor, const float* gate_row, float* gate_out, hipStream_t stream) {
  TI_REQUIRE(!gate_row || gate_out, "moe_route: a gate needs room for its numbers");
  TI_REQUIRE(n_groups <= 1 || (E % n_groups == 0 && keep >= 1 && keep <= n_groups && (long)keep * (E / n_groups) >= top),
             "moe_route: %d groups of which %d are kept do not fit %d experts and top %d", n_groups, keep, E, top);
  TI_REQUIRE((!correction && n_groups <= 1) || score_kind != MOE_SOFTMAX_CHOSEN, "moe_route: a correction or groups do not go with weights from the chosen logits");
  TI_REQUIRE(M >= 0 && W > 0 && E > 0 && E <= MOE_MAX_EXPERTS && top > 0 && top <= E && top <= MOE_MAX_TOP,
             "moe_route: bad sizes M=%d W=%d experts=%d top=%d (up to %d experts, top up to %d)", M, W, E, top, MOE_MAX_EXPERTS,
             MOE_MAX_TOP);
  TI_REQUIRE(score_kind == MOE_SIGMOID || score_kind == MOE_SOFTMAX || score_kind == MOE_SOFTMAX_CHOSEN, "moe_route: unknown score kind %d", score_kind);
  if (M == 0) return 0;
  const int piece = dtype == TI_F32 ? 4 : 8;
  const bool vec = W % piece == 0 && ((uintptr_t)h & 15) == 0;
  const RouteForm form = {W, E, top, score_kind, renormalize, n_groups, keep, weight_scale, sum_floor};
  const size_t per_token = ((size_t)2 * E + (n_groups > 1 ? n_groups : 0)) * 4;
  const bool four = M >= 512 && 4 * per_token <= 64 * 1024;
#define MOE_ROUTE(T, V)                                                                                                                          \
  do {                                                                                                                                           \
    if (four) moe_route_kernel<T, V, 4><<<(M + 3) / 4, 256, 4 * per_token, stream>>>((const T*)h, router, ids, wts, M, form, correction, gate_row, gate_out); \
    else moe_route_kernel<T, V, 1><<<M, 256, per_token, stream>>>((const T*)h, router, ids, wts, M, form, correction, gate_row, gate_out);        \
  } while (0)
  if (dtype == TI_F32) {
    if (vec) MOE_ROUTE(float, true);
    else MOE_ROUTE(float, false);
  } else if (dtype == TI_BF16) {
    if (vec) MOE_ROUTE(bf16_t, true);
    else MOE_ROUTE(bf16_t, false);
  } else {
    TI_REQUIRE(false, "moe_route: unknown dtype %d", dtype);
  }
#undef MOE_ROUTE
  TI_LAUNCH_CHECK();
  return 0;
}

// ------------------------------------------------------------ the experts, an output a wavefront
// up [E][F][W], down [E][W][F] in T.  Two kernels, a wavefront per (expert, a few outputs), on its own from beginning to end: it
// finds the pairs (token, choice) of its expert, up to four at a time, and walks its rows of the weight once for all of them: an
// expert's weights are read once a step for every four tokens that chose it.
//   act[pair][f] = relu(up[e][f] . (s h[token]))^2 rounded to T;   part[pair][c] = down[e][c] . act[pair]
// and a token's rows of `part` are added in the order its experts were chosen by whoever reads them (moe_sum_pairs, or the
// norm that follows).  A wavefront owns four rows of the weight; its lanes share a row in pieces of 16 bytes (lane l the
// pieces l, l + 64, ... in ascending order, then a butterfly): the order of every sum is fixed, whatever else the step holds.
#define MOE_ROWS 4      // rows of the weight a wavefront
#define MOE_PAIRS 4     // pairs at a time

// the next pairs of expert e from pair `next` on, at most MOE_PAIRS: lane p gets the p-th one's index; returns how many, `next` goes on
__device__ __forceinline__ int next_pairs(const int* __restrict__ ids, int n_pairs, int e, int lane, int& next, int& mine) {
  int n = 0, i = next;
  while (i < n_pairs && n < MOE_PAIRS) {
    const bool hit = i + lane < n_pairs && ids[i + lane] == e;
    unsigned long long mask = __ballot(hit);
    int consumed = 64;
    while (mask) {
      const int b = __ffsll((long long)mask) - 1;
      if (n == MOE_PAIRS) {       // this one waits for the next round
        consumed = b;
        break;
      }
      if (lane == n) mine = i + b;
      ++n;
      mask &= mask - 1;
    }
    i += consumed;
  }
  next = i;
  return n;
}

// one element of a pair's row as a product reads it: in T, times the score where that scales the input
template <typename T> __device__ __forceinline__ float scaled_input(float v, float s);
template <> __device__ __forceinline__ float scaled_input<float>(float v, float s) { return v * s; }
template <> __device__ __forceinline__ float scaled_input<bf16_t>(float v, float s) { return bf2f(f2bf(v * s)); }

// z[r][p] = row p of the pairs . br[r]: the loads of all the weight's rows and of all the pairs' rows are in flight together.  Every
// sum runs over a lane's pieces in ascending order, then a butterfly.  SCALED: a pair's row is multiplied by s[p] first.
template <typename T, bool VEC, int NP, bool SCALED>
__device__ __forceinline__ void wave_dots(const T* const* rows, const float* s, const T* const* br, int K, int lane, float (*z)[MOE_PAIRS]) {
#pragma unroll
  for (int r = 0; r < MOE_ROWS; ++r)
#pragma unroll
    for (int p = 0; p < NP; ++p) z[r][p] = 0.f;
  constexpr int N = VEC ? Piece<T>::N : 1;
#pragma unroll 2
  for (int c = lane * N; c < K; c += 64 * N) {
    float v[MOE_ROWS][N], a[NP][N];
#pragma unroll
    for (int r = 0; r < MOE_ROWS; ++r) {
      if constexpr (VEC) Piece<T>::load(br[r] + c, v[r]);
      else v[r][0] = ld<T>(br[r] + c);
    }
#pragma unroll
    for (int p = 0; p < NP; ++p) {
      if constexpr (VEC) Piece<T>::load(rows[p] + c, a[p]);
      else a[p][0] = ld<T>(rows[p] + c);
    }
#pragma unroll
    for (int p = 0; p < NP; ++p)
#pragma unroll
      for (int i = 0; i < N; ++i) {
        const float x = SCALED ? scaled_input<T>(a[p][i], s[p]) : a[p][i];
#pragma unroll
        for (int r = 0; r < MOE_ROWS; ++r) z[r][p] = fmaf(x, v[r][i], z[r][p]);
      }
  }
#pragma unroll
  for (int r = 0; r < MOE_ROWS; ++r)
#pragma unroll
    for (int p = 0; p < NP; ++p) z[r][p] = group_sum<64>(z[r][p]);
}

// a gated expert's activation of the two sums.  kind 0: silu(g) u; 1: g = min(g, limit), u = clamp(u, -limit, limit),
// g sigmoid(alpha g) (u + 1)
__device__ __forceinline__ float moe_gate(float g, float u, int kind, float limit, float alpha) {
  if (kind == 0) return g / (1.0f + expf(-g)) * u;
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g / (1.0f + expf(-alpha * g)) * (u + 1.0f);
}

// what a wavefront per (expert, outputs) does
#define MOE_UP 0       // in: the tokens' inputs h (scaled by the score where it scales the input), K = W, N = F outputs: relu^2 to act (T)
#define MOE_GATED 1    // in: h, K = W, N = F: an expert's weight is [2 F][W], gate rows above up rows; the gated activation to act (T)
#define MOE_DOWN 2     // in: act, K = F, N = W: 32-bit to part (times the score where it scales the output)
// ids from E on are identity experts: MOE_DOWN's workgroups of blockIdx.x = E (launched where there are any) write their
// pairs' rows of part, the score times the token's row of `self`.
struct MoeRows { int n_pairs, K, N, top, scale_input, E, kind; float limit, alpha; };
template <typename T, bool VEC, int FORM>
__global__ void __launch_bounds__(256)
moe_expert_rows_kernel(const T* __restrict__ in, const int* __restrict__ ids, const float* __restrict__ wts, const T* __restrict__ w,
                       void* __restrict__ out, const T* __restrict__ self, const MoeRows a) {
  const int e = blockIdx.x, K = a.K, N = a.N;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  if (FORM == MOE_DOWN && e == a.E) {
    for (int pair = blockIdx.y; pair < a.n_pairs; pair += gridDim.y) {
      if (ids[pair] < a.E) continue;
      const float s = wts[pair];
      for (int c = threadIdx.x; c < N; c += 256) ((float*)out)[(size_t)pair * N + c] = ld<T>(self + (size_t)(pair / a.top) * N + c) * s;
    }
    return;
  }
  constexpr int OUT = FORM == MOE_GATED ? MOE_ROWS / 2 : MOE_ROWS;      // outputs a wavefront
  const int n0 = (blockIdx.y * 4 + wave) * OUT;
  if (n0 >= N) return;      // (no barrier below)
  const T* we = w + (size_t)e * (FORM == MOE_GATED ? 2 * N : N) * K;
  const T* br[MOE_ROWS];      // (outputs beyond the last one: the last one's rows)
#pragma unroll
  for (int r = 0; r < MOE_ROWS; ++r) {
    const int n = min(n0 + r % OUT, N - 1);
    br[r] = we + (size_t)(r < OUT ? n : N + n) * K;
  }
  int next = 0;
  while (next < a.n_pairs) {
    int mine = 0;
    const int n_live = next_pairs(ids, a.n_pairs, e, lane, next, mine);
    if (n_live == 0) break;
    int pairs[MOE_PAIRS];
    const T* rows[MOE_PAIRS];
    float s[MOE_PAIRS];
#pragma unroll
    for (int p = 0; p < MOE_PAIRS; ++p) {      // (places beyond the last pair: the first one again, not written)
      pairs[p] = __builtin_amdgcn_readlane(mine, p < n_live ? p : 0);
      rows[p] = in + (size_t)(FORM == MOE_DOWN ? pairs[p] : pairs[p] / a.top) * K;
      s[p] = FORM == MOE_GATED ? 1.f : wts[pairs[p]];
    }
    float z[MOE_ROWS][MOE_PAIRS];
#define MOE_DOTS(NP)                                                                                         \
  do {                                                                                                       \
    if (FORM == MOE_UP && a.scale_input) wave_dots<T, VEC, NP, true>(rows, s, br, K, lane, z);               \
    else wave_dots<T, VEC, NP, false>(rows, s, br, K, lane, z);                                              \
  } while (0)
    if (n_live == 1) MOE_DOTS(1);
    else MOE_DOTS(MOE_PAIRS);
#undef MOE_DOTS
    if (lane == 0) {
#pragma unroll
      for (int r = 0; r < OUT; ++r)
#pragma unroll
        for (int p = 0; p < MOE_PAIRS; ++p)
          if (n0 + r < N && p < n_live) {
            const size_t at = (size_t)pairs[p] * N + n0 + r;
            if (FORM == MOE_DOWN) {
              ((float*)out)[at] = a.scale_input ? z[r][p] : z[r][p] * s[p];
            } else if (FORM == MOE_GATED) {
              st<T>((T*)out + at, moe_gate(z[r][p], z[(r + OUT) % MOE_ROWS][p], a.kind, a.limit, a.alpha));
            } else {
              const float v = fmaxf(z[r][p], 0.f);
              st<T>((T*)out + at, v * v);
            }
          }
    }
  }
}

// y[m] = sum_k part[m top + k], k ascending
__global__ void moe_sum_pairs_kernel(const float* __restrict__ part, float* __restrict__ y, int W, int top) {
  const int m = blockIdx.x;
  for (int c = threadIdx.x; c < W; c += blockDim.x) {
    float v = part[(size_t)m * top * W + c];
    for (int k = 1; k < top; ++k) v += part[((size_t)m * top + k) * W + c];
    y[(size_t)m * W + c] = v;
  }
}

template <typename T, bool VEC, int FORM>
static void expert_rows(const void* in, const int* ids, const float* wts, const void* w, void* out, const void* self, const MoeRows& a,
                        hipStream_t stream) {
  const int each = 4 * (FORM == MOE_GATED ? MOE_ROWS / 2 : MOE_ROWS);
  const dim3 grid(a.E + (FORM == MOE_DOWN && self ? 1 : 0), (a.N + each - 1) / each);
  moe_expert_rows_kernel<T, VEC, FORM><<<grid, 256, 0, stream>>>((const T*)in, ids, wts, (const T*)w, out, (const T*)self, a);
}

// both products of all pairs: act (T) [n_pairs][F], part f32 [n_pairs][W]
template <typename T, bool VEC, int UP>
static void experts_rows(const void* h, const int* ids, const float* wts, const void* up, const void* down, void* act, float* part, int M, int W,
                        int F, int E, int top, int scale_input, int identity, int kind, float limit, float alpha, hipStream_t stream) {
  MoeRows a = {M * top, W, F, top, scale_input, E, kind, limit, alpha};
  expert_rows<T, VEC, UP>(h, ids, wts, up, act, nullptr, a, stream);
  a.K = F;
  a.N = W;
  expert_rows<T, VEC, MOE_DOWN>(act, ids, wts, down, part, identity ? h : nullptr, a, stream);
}

template <int UP>
static int experts_rows_any(int dtype, const void* h, const int* ids, const float* wts, const void* up, const void* down, void* act, float* part,
                            float* y, int M, int W, int F, int E, int top, int scale_input, int identity, int kind, float limit, float alpha,
                            hipStream_t stream) {
  TI_REQUIRE(M >= 0 && W > 0 && F > 0 && top > 0 && E > 0, "moe_experts: bad sizes M=%d W=%d F=%d top=%d", M, W, F, top);
  TI_REQUIRE(dtype == TI_F32 || dtype == TI_BF16, "moe_experts: unknown dtype %d", dtype);
  if (M == 0) return 0;
  TI_REQUIRE((F + 7) / 8 <= 65535 && (W + 15) / 16 <= 65535, "moe_experts: sizes W=%d F=%d are too large", W, F);
  const int piece = 16 / (dtype == TI_F32 ? 4 : 2);
  const bool vec = W % piece == 0 && F % piece == 0 && (((uintptr_t)up | (uintptr_t)down | (uintptr_t)act | (uintptr_t)h) & 15) == 0;
#define MOE_BOTH(T, V) experts_rows<T, V, UP>(h, ids, wts, up, down, act, part, M, W, F, E, top, scale_input, identity, kind, limit, alpha, stream)
  if (dtype == TI_F32) {
    if (vec) MOE_BOTH(float, true);
    else MOE_BOTH(float, false);
  } else {
    if (vec) MOE_BOTH(bf16_t, true);
    else MOE_BOTH(bf16_t, false);
  }
#undef MOE_BOTH
  if (y) moe_sum_pairs_kernel<<<M, 256, 0, stream>>>(part, y, W, top);
  TI_LAUNCH_CHECK();
  return 0;
}

// y[m] = the sum of a token's rows of part f32 [M top][W], in ascending order
extern "C" int ti_moe_sum_pairs(const float* part, float* y, int M, int W, int top, hipStream_t stream) {
  TI_REQUIRE(M >= 0 && W > 0 && top > 0, "moe_sum_pairs: bad sizes M=%d W=%d top=%d", M, W, top);
  if (M == 0) return 0;
  moe_sum_pairs_kernel<<<M, 256, 0, stream>>>(part, y, W, top);
  TI_LAUNCH_CHECK();
  return 0;
}

// act: scratch in the dtype of h, [M top][F]; part: f32 [M top][W], a token's rows to be added in ascending order: into y where
// y is given, else by the caller.  identity: ids from E on are identity experts
extern "C" int ti_moe_experts_rows(int dtype, const void* h, const int* ids, const float* wts, const void* up, const void* down,
                                   void* act, float* part, float* y, int M, int W, int F, int E, int top, int scale_input, int identity,
                                   hipStream_t stream) {
  return experts_rows_any<MOE_UP>(dtype, h, ids, wts, up, down, act, part, y, M, W, F, E, top, scale_input, identity, 0, 0.f, 0.f, stream);
}

// gated experts: y[m] = sum_k s_k W_down[e_k] act(W_gate[e_k] h, W_up[e_k] h): gate_up [E][2F][W] holds an expert's gate rows above
// its up rows; act_kind as moe_gate's
extern "C" int ti_moe_experts_rows_gated(int dtype, const void* h, const int* ids, const float* wts, const void* gate_up, const void* down,
                                         void* act, float* part, float* y, int M, int W, int F, int E, int top, int act_kind, float limit,
                                         float alpha, int identity, hipStream_t stream) {
  TI_REQUIRE(act_kind == 0 || act_kind == 1, "moe_experts: unknown gated activation %d", act_kind);
  return experts_rows_any<MOE_GATED>(dtype, h, ids, wts, gate_up, down, act, part, y, M, W, F, E, top, 0, identity, act_kind, limit, alpha,
                                     stream);
}
