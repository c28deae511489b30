// The experts of a mixture of experts, bfloat16 on the matrix cores of gfx950.  Steps of few tokens: moe_few (at the end of this
// file).  Steps of many tokens:
//
//   1. moe_group: counts the (token, expert) pairs of every expert, lays the experts' runs of rows one after
//      the other and cuts them into tiles of 128 rows: offsets, the list of tiles, cursors at zero.
//   2. moe_place: every pair takes a free row of its expert's run (which row does not matter: a row of a
//      product depends on no other row) and writes its scaled input there, rounded to bfloat16; where the weights are
//      on the outputs it leaves its token's number, and the first product gathers its rows from the step's own.  Pairs of
//      identity experts (ids from E on) have a run of their own behind the others' and no tile: their rows of the result, the
//      score times the token's input, are written here.
//   3. two grouped products over the tiles: act = relu(A up_e^T)^2, or act(A gate_e^T, A up_e^T) of gated experts (bfloat16), out =
//      act down_e^T (32-bit).
//      Weights are the A operand of v_mfma_f32_16x16x32_bf16 and tokens the 16 columns, both in their own
//      layouts through LDS; a lane ends with four consecutive outputs of one token.
//   4. a token's rows are added in the order its experts were chosen: by the norm that reads them next
//      (it is handed the list `where`), or by moe_combine.
#include "common.h"
#include "tinyinfer_kernels.h"

TI_ERROR_API

typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 bf16x8;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float floatx4;
union Frag8 {
  uint4 u;
  bf16x8 v;
};

#define MOE_TILE 128         // rows (pairs) of a tile
#define MOE_MAX_E 1024

// meta int32: [0] number of tiles, [1 .. R + 1] offsets of the experts' runs, then R cursors, then tiles [max][3] =
// (expert, first row, rows).  R runs: the E experts', and one more for the identity experts (ids from E on) where R = E + 1.
// One workgroup.
__global__ void __launch_bounds__(1024)
moe_group_kernel(const int* __restrict__ ids, int n_pairs, int E, int R, int* __restrict__ meta) {
  __shared__ int count[MOE_MAX_E + 1];
  __shared__ int first_tile[MOE_MAX_E + 2];
  for (int e = threadIdx.x; e < R; e += 1024) count[e] = 0;
  __syncthreads();
  for (int i = threadIdx.x; i < n_pairs; i += 1024) atomicAdd(&count[min(ids[i], R - 1)], 1);
  __syncthreads();
  int* offsets = meta + 1;
  int* cursors = meta + 1 + R + 1;
  int* tiles = cursors + R;
  if (threadIdx.x == 0) {
    int at = 0, t = 0;
    for (int e = 0; e < R; ++e) {
      offsets[e] = at;
      first_tile[e] = t;
      at += count[e];
      if (e < E) t += (count[e] + MOE_TILE - 1) / MOE_TILE;
    }
    offsets[R] = at;
    meta[0] = t;
  }
  __syncthreads();
  for (int e = threadIdx.x; e < R; e += 1024) {
    cursors[e] = 0;
    const int n = e < E ? count[e] : 0, t0 = first_tile[e];
    for (int k = 0; k * MOE_TILE < n; ++k) {
      tiles[3 * (t0 + k)] = e;
      tiles[3 * (t0 + k) + 1] = offsets[e] + k * MOE_TILE;
      tiles[3 * (t0 + k) + 2] = min(MOE_TILE, n - k * MOE_TILE);
    }
  }
}

// A workgroup per 64 pairs: where[pair] = its row; rows[row] = bf16(s h[token]), or, with `tokens` in the place of `rows` (inputs
// without a factor), tokens[row] = its token, for a product that gathers its rows from h.  The workgroup counts its pairs per
// expert in LDS and takes a run of rows from every expert's cursor at once (one atomic per expert it met, not one per pair);
// inside the run a pair's place is its count in LDS.
__global__ void __launch_bounds__(256)
moe_place_kernel(const bf16_t* __restrict__ h, const int* __restrict__ ids, const float* __restrict__ wts, int* __restrict__ meta,
                 int E, int R, int top, int W, int n_pairs, int* __restrict__ where, bf16_t* __restrict__ rows,
                 float* __restrict__ row_w, int* __restrict__ tokens, float* __restrict__ out) {
  __shared__ int count[MOE_MAX_E + 1];      // pairs of this workgroup per expert, then the first row of their run
  __shared__ int s_row[64], s_self[64], s_n_self;
  const int pair0 = blockIdx.x * 64;
  for (int e = threadIdx.x; e < R; e += 256) count[e] = 0;
  if (threadIdx.x == 0) s_n_self = 0;
  __syncthreads();
  int e_mine = -1, local = 0;
  if (threadIdx.x < 64 && pair0 + threadIdx.x < n_pairs) {
    e_mine = min(ids[pair0 + threadIdx.x], R - 1);
    local = atomicAdd(&count[e_mine], 1);
  }
  __syncthreads();
  for (int e = threadIdx.x; e < R; e += 256)
    if (count[e] > 0) count[e] = meta[1 + e] + atomicAdd(&meta[1 + R + 1 + e], count[e]);
  __syncthreads();
  if (e_mine >= 0) {
    const int r = count[e_mine] + local;
    where[pair0 + threadIdx.x] = r;
    if (row_w) row_w[r] = wts[pair0 + threadIdx.x];      // weights on the experts' outputs: with the row
    s_row[threadIdx.x] = r;
    if (e_mine >= E) s_self[atomicAdd(&s_n_self, 1)] = threadIdx.x;      // an identity expert's pair (in any order: a pair is a row of its own)
    if (tokens) tokens[r] = (pair0 + threadIdx.x) / top;
  }
  if (tokens && R == E) return;
  __syncthreads();
  // 16 bytes of a row at a time (W is a multiple of 32)
  auto piece = [&](int local_pair, int c, float* f) {
    const float s = wts[pair0 + local_pair];
    const uint4 a = *reinterpret_cast<const uint4*>(h + (size_t)((pair0 + local_pair) / top) * W + c);
    const unsigned w[4] = {a.x, a.y, a.z, a.w};
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      f[2 * k] = __uint_as_float(w[k] << 16) * s;
      f[2 * k + 1] = __uint_as_float(w[k] & 0xffff0000u) * s;
    }
  };
  const int pieces = W / 8;
  if (!tokens) {      // scaled inputs, laid out expert by expert: a wavefront copies 16 of the rows
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    for (int i = 0; i < 16; ++i) {
      const int p = wave * 16 + i;
      if (pair0 + p >= n_pairs) break;
      for (int c = lane * 8; c < W; c += 64 * 8) {
        float f[8];
        piece(p, c, f);
        *reinterpret_cast<uint4*>(rows + (size_t)s_row[p] * W + c) =
            make_uint4(pack_bf16x2(f[0], f[1]), pack_bf16x2(f[2], f[3]), pack_bf16x2(f[4], f[5]), pack_bf16x2(f[6], f[7]));
      }
    }
  }
  for (int x = threadIdx.x; x < s_n_self * pieces; x += 256) {
    const int p = s_self[x / pieces], c = x % pieces * 8;
    float f[8];
    piece(p, c, f);
    float4* dst = reinterpret_cast<float4*>(out + (size_t)s_row[p] * W + c);
    dst[0] = make_float4(f[0], f[1], f[2], f[3]);
    dst[1] = make_float4(f[4], f[5], f[6], f[7]);
  }
}

// out[row][n] (op)= sum_k rows[row][k] w[e][n][k] over the tiles.  A workgroup: one tile of 128 rows x 128 outputs, its four
// wavefronts two by two, each 64 outputs (four blocks of 16) against 64 rows (four blocks of 16).  A step of 32 along k of both
// operands is fetched once by the workgroup (thread t the 16-byte pieces t, t + 256) into one of two LDS stages while the step
// before it is multiplied from the other; one barrier a step.  Rows of a stage are 80 bytes apart, so that the fragments'
// reads spread over the banks.  tokens (null: none): row r of the operand is row tokens[r] of `rows`.  EPI 0: relu^2, bfloat16;
// 1: 32-bit; 2: 32-bit, times the row's weight row_w[row]; 3: a gated expert, w [E][2 N][K] with gate rows above up rows: 64
// outputs a workgroup, every wavefront the gate and the up rows of its own 32 outputs, the activation of the two sums in bfloat16.
// R: the runs of `meta`.
#define MOE_LDS_ROW 40       // bfloat16 elements between rows of a stage (32 + 8)
template <int EPI>
__global__ void __launch_bounds__(256)
moe_grouped_kernel(const bf16_t* __restrict__ rows, const bf16_t* __restrict__ w, const int* __restrict__ meta, int R, void* __restrict__ out,
                   int N, int K, const float* __restrict__ row_w = nullptr, const int* __restrict__ tokens = nullptr, int kind = 0,
                   float limit = 0.f, float alpha = 0.f) {
  __shared__ __attribute__((aligned(16))) bf16_t lds[2][2][128 * MOE_LDS_ROW];      // [stage][weights | rows]
  const int n_tiles = meta[0];
  if ((int)blockIdx.x >= n_tiles) return;
  const int* tile = meta + 1 + R + 1 + R + 3 * blockIdx.x;
  const int e = tile[0], row0 = tile[1], n_rows = tile[2];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int r16 = lane & 15, quad = lane >> 4;
  const int wy = wave >> 1, wx = wave & 1;
  const int n_blk = blockIdx.y * (EPI == 3 ? 64 : 128);
  // row r of the weights' stage
  auto weight_row = [&](int r) {
    if (EPI != 3) return (size_t)e * N + min(n_blk + r, N - 1);
    const int f = n_blk + (r >> 6) * 32 + (r & 31);
    return (size_t)e * 2 * N + ((r & 32) ? N : 0) + min(f, N - 1);
  };
  // what this thread fetches: rows u / 4 of both operands, 16 bytes from element 8 (u % 4) on
  const int u0 = threadIdx.x, u1 = threadIdx.x + 256;
  const bf16_t* const src_w0 = w + weight_row(u0 >> 2) * K + (u0 & 3) * 8;
  const bf16_t* const src_w1 = w + weight_row(u1 >> 2) * K + (u1 & 3) * 8;
  const int at0 = row0 + min(u0 >> 2, n_rows - 1), at1 = row0 + min(u1 >> 2, n_rows - 1);
  const bf16_t* const src_r0 = rows + (size_t)(tokens ? tokens[at0] : at0) * K + (u0 & 3) * 8;
  const bf16_t* const src_r1 = rows + (size_t)(tokens ? tokens[at1] : at1) * K + (u1 & 3) * 8;
  const int park0 = (u0 >> 2) * MOE_LDS_ROW + (u0 & 3) * 8, park1 = (u1 >> 2) * MOE_LDS_ROW + (u1 & 3) * 8;
  floatx4 acc[4][4];
#pragma unroll
  for (int a = 0; a < 4; ++a)
#pragma unroll
    for (int b = 0; b < 4; ++b) acc[a][b] = floatx4{0.f, 0.f, 0.f, 0.f};
  uint4 w0 = *reinterpret_cast<const uint4*>(src_w0), w1 = *reinterpret_cast<const uint4*>(src_w1);
  uint4 t0 = *reinterpret_cast<const uint4*>(src_r0), t1 = *reinterpret_cast<const uint4*>(src_r1);
  *reinterpret_cast<uint4*>(&lds[0][0][park0]) = w0;
  *reinterpret_cast<uint4*>(&lds[0][0][park1]) = w1;
  *reinterpret_cast<uint4*>(&lds[0][1][park0]) = t0;
  *reinterpret_cast<uint4*>(&lds[0][1][park1]) = t1;
  __syncthreads();
  int cur = 0;
  for (int k = 0; k < K; k += 32, cur ^= 1) {       // K is a multiple of 32
    const bool more = k + 32 < K;
    if (more) {
      w0 = *reinterpret_cast<const uint4*>(src_w0 + k + 32);
      w1 = *reinterpret_cast<const uint4*>(src_w1 + k + 32);
      t0 = *reinterpret_cast<const uint4*>(src_r0 + k + 32);
      t1 = *reinterpret_cast<const uint4*>(src_r1 + k + 32);
    }
    Frag8 fa[4], fb[4];
#pragma unroll
    for (int a = 0; a < 4; ++a) fa[a].u = *reinterpret_cast<const uint4*>(&lds[cur][0][(64 * wy + 16 * a + r16) * MOE_LDS_ROW + quad * 8]);
#pragma unroll
    for (int b = 0; b < 4; ++b) fb[b].u = *reinterpret_cast<const uint4*>(&lds[cur][1][(64 * wx + 16 * b + r16) * MOE_LDS_ROW + quad * 8]);
#pragma unroll
    for (int a = 0; a < 4; ++a)
#pragma unroll
      for (int b = 0; b < 4; ++b) acc[a][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fa[a].v, fb[b].v, acc[a][b], 0, 0, 0);
    if (more) {
      *reinterpret_cast<uint4*>(&lds[cur ^ 1][0][park0]) = w0;
      *reinterpret_cast<uint4*>(&lds[cur ^ 1][0][park1]) = w1;
      *reinterpret_cast<uint4*>(&lds[cur ^ 1][1][park0]) = t0;
      *reinterpret_cast<uint4*>(&lds[cur ^ 1][1][park1]) = t1;
    }
    __syncthreads();
  }
  // lane: outputs n0 + 16 a + 4 quad + i of row 64 wx + 16 b + r16
  const int n0 = n_blk + (EPI == 3 ? 32 : 64) * wy;
#pragma unroll
  for (int b = 0; b < 4; ++b) {
    const int r = 64 * wx + 16 * b + r16;
    if (r >= n_rows) continue;
    if constexpr (EPI == 3) {
#pragma unroll
      for (int a = 0; a < 2; ++a) {
        const int n = n0 + 16 * a + 4 * quad;
        if (n >= N) continue;
        float z[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          float g = acc[a][b][i], u = acc[a + 2][b][i];
          if (kind == 0) {
            z[i] = g * __frcp_rn(1.0f + __expf(-g)) * u;
          } else {
            g = fminf(g, limit);
            u = fminf(fmaxf(u, -limit), limit);
            z[i] = g * __frcp_rn(1.0f + __expf(-alpha * g)) * (u + 1.0f);
          }
        }
        *reinterpret_cast<uint2*>((bf16_t*)out + (size_t)(row0 + r) * N + n) = make_uint2(pack_bf16x2(z[0], z[1]), pack_bf16x2(z[2], z[3]));
      }
      continue;
    }
    const float s = EPI == 2 ? row_w[row0 + r] : 1.f;
#pragma unroll
    for (int a = 0; a < 4; ++a) {
      const int n = n0 + 16 * a + 4 * quad;
      if (n >= N) continue;                 // N is a multiple of 4
      const floatx4 v = acc[a][b];
      if (EPI == 0) {
        float z[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          z[i] = fmaxf(v[i], 0.f);
          z[i] *= z[i];
        }
        *reinterpret_cast<uint2*>((bf16_t*)out + (size_t)(row0 + r) * N + n) = make_uint2(pack_bf16x2(z[0], z[1]), pack_bf16x2(z[2], z[3]));
      } else if (EPI == 2) {
        *reinterpret_cast<float4*>((float*)out + (size_t)(row0 + r) * N + n) = make_float4(v[0] * s, v[1] * s, v[2] * s, v[3] * s);
      } else {
        *reinterpret_cast<float4*>((float*)out + (size_t)(row0 + r) * N + n) = make_float4(v[0], v[1], v[2], v[3]);
      }
    }
  }
}

// y[m] = sum_k out[where[m top + k]], k ascending
__global__ void moe_combine_kernel(const float* __restrict__ out, const int* __restrict__ where, float* __restrict__ y, int W, int top) {
  const int m = blockIdx.x;
  for (int c = threadIdx.x; c < W; c += blockDim.x) {
    float v = 0.f;
    for (int k = 0; k < top; ++k) v += out[(size_t)where[m * top + k] * W + c];
    y[(size_t)m * W + c] = v;
  }
}

extern "C" long ti_moe_grouped_meta_ints(int n_pairs, int E) { return 1 + (E + 2) + (E + 1) + 3L * ((n_pairs + MOE_TILE - 1) / MOE_TILE + E); }

// h bf16 [M, W]; ids, wts [M top]; up [E][F][W] (gated: [E][2F][W], gate rows above up rows), down [E][W][F] bf16.  Scratch: meta
// int32 [ti_moe_grouped_meta_ints], where int32 [M top], rows bf16 [M top][W] (weights on the outputs: int32 [M top], the rows'
// tokens), act bf16 [M top][F], out f32 [M top][W].  y (may be null): the tokens' sums; without it the caller adds the rows
// out[where[m top + k]] itself.  The weights multiply the experts' inputs (scale_input) or their outputs (row_w: f32 scratch
// [M top]).  act_kind < 0: relu^2; else gated.  identity: ids from E on are identity experts.
// 3: sizes not served (W, F multiples of 32, E <= 1024).
extern "C" int ti_moe_experts_grouped_bf16(const void* h, const int* ids, const float* wts, const void* up, const void* down,
                                           int* meta, int* where, void* rows, void* act, float* out, float* y, int M, int W, int F,
                                           int E, int top, int scale_input, float* row_w, int act_kind, float limit, float alpha,
                                           int identity, hipStream_t stream) {
  if (W % 32 || F % 32 || E > MOE_MAX_E) {
    ti_set_error("moe_experts (grouped): W=%d, F=%d, %d experts are not served", W, F, E);
    return 3;
  }
  TI_REQUIRE(M >= 0 && top > 0 && E > 0 && (scale_input || row_w) && act_kind <= 1 && !(act_kind >= 0 && scale_input), "moe_experts (grouped): bad arguments");
  if (M == 0) return 0;
  const int n_pairs = M * top, R = E + (identity ? 1 : 0);
  const int max_tiles = (n_pairs + MOE_TILE - 1) / MOE_TILE + E;
  moe_group_kernel<<<1, 1024, 0, stream>>>(ids, n_pairs, E, R, meta);
  int* tokens = scale_input ? nullptr : (int*)rows;
  moe_place_kernel<<<(n_pairs + 63) / 64, 256, 0, stream>>>((const bf16_t*)h, ids, wts, meta, E, R, top, W, n_pairs, where, (bf16_t*)rows,
                                                            scale_input ? nullptr : row_w, tokens, out);
  const bf16_t* in = (const bf16_t*)(tokens ? h : rows);
  if (act_kind >= 0)
    moe_grouped_kernel<3><<<dim3(max_tiles, (F + 63) / 64), 256, 0, stream>>>(in, (const bf16_t*)up, meta, R, act, F, W, nullptr, tokens, act_kind,
                                                                              limit, alpha);
  else
    moe_grouped_kernel<0><<<dim3(max_tiles, (F + 127) / 128), 256, 0, stream>>>(in, (const bf16_t*)up, meta, R, act, F, W, nullptr, tokens);
  const dim3 grid_down(max_tiles, (W + 127) / 128);
  if (scale_input) moe_grouped_kernel<1><<<grid_down, 256, 0, stream>>>((const bf16_t*)act, (const bf16_t*)down, meta, R, out, W, F);
  else moe_grouped_kernel<2><<<grid_down, 256, 0, stream>>>((const bf16_t*)act, (const bf16_t*)down, meta, R, out, W, F, row_w);
  if (y) moe_combine_kernel<<<M, 256, 0, stream>>>(out, where, y, W, top);
  TI_LAUNCH_CHECK();
  return 0;
}

// ------------------------------------------------------------ steps of few tokens
// A workgroup per (expert, 16 outputs): the expert's rows of the weight are the A operand of v_mfma_f32_16x16x32_bf16, up to sixteen
// of the pairs that chose it the columns; both come straight from memory in their own layouts.  The four wavefronts take the steps
// of 32 along k in turn, eight of a wavefront's in flight together; their sums are added in LDS in a fixed order.  A workgroup
// whose expert nobody chose ends at once; more than sixteen pairs take another round.
//   FORM 0: act = relu(up (s h))^2 (s 1 unless the score scales the input), 1: act = the gated activation of (gate h, up h) (w
// [E][2 N][K], gate rows above up rows), 2: part = s down act, or down act where the score was in the input.
// ids from E on are identity experts: FORM 2's workgroups of blockIdx.x = E write their pairs' rows, s self[token].
#define FEW_AHEAD 8
struct MoeFew { int n_pairs, K, N, top, scale_input, E, kind; float limit, alpha; };
template <int FORM, bool SCALED>
__global__ void __launch_bounds__(256)
moe_few_kernel(const bf16_t* __restrict__ in, const int* __restrict__ ids, const float* __restrict__ wts, const bf16_t* __restrict__ w,
               void* __restrict__ out, const bf16_t* __restrict__ self, const MoeFew a) {
  constexpr int SETS = FORM == 1 ? 2 : 1;      // runs of 16 rows of the weight
  __shared__ int s_pairs[4][16];
  __shared__ float s_sum[4][SETS][256];
  const int e = blockIdx.x, K = a.K, N = a.N;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r16 = lane & 15, quad = lane >> 4;
  if (FORM == 2 && e == a.E) {
    for (int pair = blockIdx.y; pair < a.n_pairs; pair += gridDim.y) {
      if (ids[pair] < a.E) continue;
      const float s = wts[pair];
      for (int c = threadIdx.x; c < N; c += 256) ((float*)out)[(size_t)pair * N + c] = bf2f(self[(size_t)(pair / a.top) * N + c]) * s;
    }
    return;
  }
  const int n0 = blockIdx.y * 16, steps = K / 32;
  const bf16_t* src_w[SETS];
#pragma unroll
  for (int x = 0; x < SETS; ++x) src_w[x] = w + ((size_t)e * SETS * N + (size_t)x * N + min(n0 + r16, N - 1)) * K + quad * 8;
  for (int base = 0;; base += 16) {
    // the expert's pairs base .. base + 15, every wavefront for itself
    int n_live = 0;
    for (int i = 0; i < a.n_pairs; i += 64) {
      const bool hit = i + lane < a.n_pairs && ids[i + lane] == e;
      const unsigned long long mask = __ballot(hit);
      const int rank = n_live + __popcll(mask & ((1ull << lane) - 1ull)) - base;
      if (hit && rank >= 0 && rank < 16) s_pairs[wave][rank] = i + lane;
      n_live += __popcll(mask);
    }
    n_live = min(16, n_live - base);
    if (n_live <= 0) return;      // (the same in all four)
    __builtin_amdgcn_wave_barrier();
    __threadfence_block();
    const int mine = s_pairs[wave][r16 < n_live ? r16 : 0];      // (columns beyond the last pair: the first one again, not written)
    const bf16_t* src_p = in + (size_t)(FORM == 2 ? mine : mine / a.top) * K + quad * 8;
    const float s = SCALED ? wts[mine] : 1.f;
    floatx4 acc[SETS];
#pragma unroll
    for (int x = 0; x < SETS; ++x) acc[x] = floatx4{0.f, 0.f, 0.f, 0.f};
    for (int step = wave; step < steps; step += 4 * FEW_AHEAD) {
      Frag8 fw[FEW_AHEAD][SETS], fp[FEW_AHEAD];
#pragma unroll
      for (int j = 0; j < FEW_AHEAD; ++j) {
        const int k = min(step + 4 * j, steps - 1) * 32;      // (a step that is not there: the last one's operands, not multiplied)
#pragma unroll
        for (int x = 0; x < SETS; ++x) fw[j][x].u = *reinterpret_cast<const uint4*>(src_w[x] + k);
        fp[j].u = *reinterpret_cast<const uint4*>(src_p + k);
      }
#pragma unroll
      for (int j = 0; j < FEW_AHEAD; ++j) {
        if (step + 4 * j >= steps) break;
        if (SCALED) {
          const unsigned v[4] = {fp[j].u.x, fp[j].u.y, fp[j].u.z, fp[j].u.w};
          unsigned o[4];
#pragma unroll
          for (int i = 0; i < 4; ++i) o[i] = pack_bf16x2(__uint_as_float(v[i] << 16) * s, __uint_as_float(v[i] & 0xffff0000u) * s);
          fp[j].u = make_uint4(o[0], o[1], o[2], o[3]);
        }
#pragma unroll
        for (int x = 0; x < SETS; ++x) acc[x] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fw[j][x].v, fp[j].v, acc[x], 0, 0, 0);
      }
    }
    // lane: outputs 4 quad + i of column r16
#pragma unroll
    for (int x = 0; x < SETS; ++x) *reinterpret_cast<floatx4*>(&s_sum[wave][x][lane * 4]) = acc[x];
    __syncthreads();
    const int row = threadIdx.x & 15, col = threadIdx.x >> 4;
    const int at = ((row >> 2) * 16 + col) * 4 + (row & 3);
    float z[SETS];
#pragma unroll
    for (int x = 0; x < SETS; ++x) z[x] = ((s_sum[0][x][at] + s_sum[1][x][at]) + s_sum[2][x][at]) + s_sum[3][x][at];
    if (col < n_live && n0 + row < N) {
      const int pair = s_pairs[wave][col];
      const size_t to = (size_t)pair * N + n0 + row;
      if (FORM == 0) {
        const float v = fmaxf(z[0], 0.f);
        ((bf16_t*)out)[to] = f2bf(v * v);
      } else if (FORM == 1) {
        float g = z[0], u = z[SETS - 1];
        if (a.kind == 0) {
          g = g / (1.0f + expf(-g)) * u;
        } else {
          g = fminf(g, a.limit);
          u = fminf(fmaxf(u, -a.limit), a.limit);
          g = g / (1.0f + expf(-a.alpha * g)) * (u + 1.0f);
        }
        ((bf16_t*)out)[to] = f2bf(g);
      } else {
        ((float*)out)[to] = a.scale_input ? z[0] : z[0] * wts[pair];
      }
    }
    __syncthreads();      // sums and pairs are read to the end before the next round writes them
  }
}

// what ti_moe_experts_rows (act_kind < 0: relu^2) / ti_moe_experts_rows_gated do, for bfloat16 and W, F multiples of 32
// (3: sizes not served); part f32 [M top][W], a token's rows to be added by the caller
extern "C" int ti_moe_experts_few_bf16(const void* h, const int* ids, const float* wts, const void* up, const void* down, void* act, float* part,
                                       int M, int W, int F, int E, int top, int scale_input, int act_kind, float limit, float alpha, int identity,
                                       hipStream_t stream) {
  if (W % 32 || F % 32 || (((uintptr_t)h | (uintptr_t)up | (uintptr_t)down | (uintptr_t)act) & 15) != 0 || (W + 15) / 16 > 65535 || (F + 15) / 16 > 65535) {
    ti_set_error("moe_experts (few): W=%d, F=%d are not served", W, F);
    return 3;
  }
  TI_REQUIRE(M >= 0 && top > 0 && E > 0 && act_kind <= 1 && !(act_kind >= 0 && scale_input), "moe_experts (few): bad arguments");
  if (M == 0) return 0;
  MoeFew a = {M * top, W, F, top, scale_input, E, act_kind, limit, alpha};
  const dim3 grid_up(E, (F + 15) / 16);
  if (act_kind >= 0)
    moe_few_kernel<1, false><<<grid_up, 256, 0, stream>>>((const bf16_t*)h, ids, wts, (const bf16_t*)up, act, nullptr, a);
  else if (scale_input)
    moe_few_kernel<0, true><<<grid_up, 256, 0, stream>>>((const bf16_t*)h, ids, wts, (const bf16_t*)up, act, nullptr, a);
  else
    moe_few_kernel<0, false><<<grid_up, 256, 0, stream>>>((const bf16_t*)h, ids, wts, (const bf16_t*)up, act, nullptr, a);
  a.K = F;
  a.N = W;
  moe_few_kernel<2, false><<<dim3(E + (identity ? 1 : 0), (W + 15) / 16), 256, 0, stream>>>((const bf16_t*)act, ids, wts, (const bf16_t*)down, part,
                                                                                          (const bf16_t*)h, a);
  TI_LAUNCH_CHECK();
  return 0;
}
