// Kernels of layers that norm what a sublayer returns instead of what it reads: the RMS norm of a
// 32-bit row written (or added) into the 32-bit residual, and the rounding of the residual to the
// compute dtype for the products that read it directly.  All arithmetic is 32-bit.
#include "common.h"
#include "tinyinfer_kernels.h"

TI_ERROR_API

// x[m] (+)= y'[m] / sqrt(mean(y'[m]^2) + eps) * g, with y'[m] = y[m], or, with `gather`, the sum of the
// n_gather rows y[gather[m n_gather + k]] in ascending k (the rows a token's experts left; without a list: the rows
// y[m n_gather + k]).
// A workgroup per row; each thread owns the elements t, t + 256, ... in both passes, so y and x may be
// the same memory.  The sum of squares: per thread in ascending order, then block_sum (fixed order).
// RT: also `rounded` (RT) [M][H] = the new x rounded, for the product that reads the residual next.
// V4: four elements a thread at a time (H a multiple of 4, 16-byte aligned operands): fewer, wider loads in flight.
template <typename RT, bool V4>
__global__ void __launch_bounds__(256)
norm_residual_kernel(float* x, const float* y, const float* __restrict__ g,      // (y may be x)
                     const int* __restrict__ gather, int n_gather, int H, float eps, int accumulate, RT* __restrict__ rounded) {
  __shared__ float red[4];
  const int m = blockIdx.x;
  constexpr int N = V4 ? 4 : 1;
  // elements i .. i + N - 1 of the row to be normed
  auto value = [&](int i, float* v) {
    const int terms = (gather || n_gather > 1) ? n_gather : 1;
    for (int k = 0; k < terms; ++k) {
      const size_t r = gather ? (size_t)gather[(size_t)m * n_gather + k] : (size_t)m * terms + k;
      float t[N];
      if (V4) {
        const float4 a = *reinterpret_cast<const float4*>(y + r * H + i);
        t[0] = a.x;
        if (N > 1) { t[1] = a.y; t[2] = a.z; t[3] = a.w; }
      } else {
        t[0] = y[r * H + i];
      }
#pragma unroll
      for (int j = 0; j < N; ++j) v[j] = k == 0 ? t[j] : v[j] + t[j];
    }
  };
  float ss = 0.f;
  for (int i = threadIdx.x * N; i < H; i += 256 * N) {
    float v[N];
    value(i, v);
#pragma unroll
    for (int j = 0; j < N; ++j) ss = fmaf(v[j], v[j], ss);
  }
  ss = block_sum<256>(ss, red);
  const float scale = 1.0f / sqrtf(ss / (float)H + eps);
  float* row = x + (size_t)m * H;
  for (int i = threadIdx.x * N; i < H; i += 256 * N) {
    float v[N];
    value(i, v);
#pragma unroll
    for (int j = 0; j < N; ++j) {
      const float add = v[j] * scale * g[i + j];
      const float now = accumulate ? row[i + j] + add : add;
      row[i + j] = now;
      if (rounded) st<RT>(rounded + (size_t)m * H + i + j, now);
    }
  }
}

extern "C" int ti_norm_residual(float* x, const float* y, const float* g, const int* gather, int n_gather, int M, int H,
                                float eps, int accumulate, void* rounded, int rounded_dtype, hipStream_t stream) {
  TI_REQUIRE(M >= 0 && H > 0 && (!gather || n_gather > 0), "norm_residual: bad sizes M=%d H=%d gather=%d", M, H, n_gather);
  TI_REQUIRE(!rounded || rounded_dtype == TI_F32 || rounded_dtype == TI_BF16, "norm_residual: unknown dtype %d", rounded_dtype);
  if (M == 0) return 0;
  const bool v4 = H % 4 == 0 && (((uintptr_t)x | (uintptr_t)y | (uintptr_t)g) & 15) == 0;
  if (rounded && rounded_dtype == TI_BF16) {
    if (v4) norm_residual_kernel<bf16_t, true><<<M, 256, 0, stream>>>(x, y, g, gather, n_gather, H, eps, accumulate, (bf16_t*)rounded);
    else norm_residual_kernel<bf16_t, false><<<M, 256, 0, stream>>>(x, y, g, gather, n_gather, H, eps, accumulate, (bf16_t*)rounded);
  } else {
    if (v4) norm_residual_kernel<float, true><<<M, 256, 0, stream>>>(x, y, g, gather, n_gather, H, eps, accumulate, (float*)rounded);
    else norm_residual_kernel<float, false><<<M, 256, 0, stream>>>(x, y, g, gather, n_gather, H, eps, accumulate, (float*)rounded);
  }
  TI_LAUNCH_CHECK();
  return 0;
}

// Layers with a norm on either side of a sublayer, both in one pass over the row:
//   x[m] += factor N(y'[m]) g,   then   out[m] = N(x[m]) next_g  (RT)
// with N(z) = z / sqrt(mean(z^2) + eps), or, centered, (z - mean z) / sqrt(mean((z - mean z)^2) + eps).
// y'[m]: y_scale times the rows of y as above, in ascending order, and behind them plus_scale plus_gate[m] plus[m] (plus null:
// none; plus_gate null: one).  out null: the first line alone.  A workgroup per row; x, y' and both gains are asked for before
// the first sum is known and stay in registers: NV pieces of four elements a thread (NV 0: any width, element by element from
// memory).
template <typename RT, int NV>
__global__ void __launch_bounds__(256)
norm_residual_next_kernel(float* __restrict__ x, const float* __restrict__ y, const int* __restrict__ gather, int n_gather,
                          const float* __restrict__ plus, const float* __restrict__ plus_gate, const ti_norm_pair p, RT* __restrict__ out,
                          int H) {
  __shared__ float red[4];
  const int m = blockIdx.x;
  const int terms = (gather || n_gather > 1) ? n_gather : 1;
  const float pg = p.plus_scale * (plus_gate ? plus_gate[m] : 1.f);
  float* const row = x + (size_t)m * H;
  auto source = [&](int k) { return y + (gather ? (size_t)gather[(size_t)m * n_gather + k] : (size_t)m * terms + k) * H; };
  if constexpr (NV > 0) {
    float4 v[NV], xv[NV], gv[NV], nv[NV];
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int i = (j * 256 + threadIdx.x) * 4;
      const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
      v[j] = xv[j] = gv[j] = nv[j] = zero;
      if (i < H) {
        xv[j] = *reinterpret_cast<const float4*>(row + i);
        gv[j] = *reinterpret_cast<const float4*>(p.g + i);
        if (out) nv[j] = *reinterpret_cast<const float4*>(p.next_g + i);
      }
    }
    for (int k = 0; k < terms; ++k) {
      const float* src = source(k);
#pragma unroll
      for (int j = 0; j < NV; ++j) {
        const int i = (j * 256 + threadIdx.x) * 4;
        if (i < H) {
          const float4 a = *reinterpret_cast<const float4*>(src + i);
          v[j] = k == 0 ? a : make_float4(v[j].x + a.x, v[j].y + a.y, v[j].z + a.z, v[j].w + a.w);
        }
      }
    }
    if (p.y_scale != 1.f) {
#pragma unroll
      for (int j = 0; j < NV; ++j) v[j] = make_float4(v[j].x * p.y_scale, v[j].y * p.y_scale, v[j].z * p.y_scale, v[j].w * p.y_scale);
    }
    if (plus) {
#pragma unroll
      for (int j = 0; j < NV; ++j) {
        const int i = (j * 256 + threadIdx.x) * 4;
        if (i < H) {
          const float4 a = *reinterpret_cast<const float4*>(plus + (size_t)m * H + i);
          v[j] = make_float4(fmaf(pg, a.x, v[j].x), fmaf(pg, a.y, v[j].y), fmaf(pg, a.z, v[j].z), fmaf(pg, a.w, v[j].w));
        }
      }
    }
    // the row in the threads' registers becomes what N divides (its mean off where centered), the result is the divisor's inverse
    auto inverse = [&](float4* z, int centered, float eps) {
      if (centered) {
        float sum = 0.f;
#pragma unroll
        for (int j = 0; j < NV; ++j) sum += (z[j].x + z[j].y) + (z[j].z + z[j].w);      // (zeros beyond the row)
        const float mean = block_sum<256>(sum, red) / (float)H;
#pragma unroll
        for (int j = 0; j < NV; ++j)
          if ((j * 256 + (int)threadIdx.x) * 4 < H) z[j] = make_float4(z[j].x - mean, z[j].y - mean, z[j].z - mean, z[j].w - mean);
      }
      float ss = 0.f;
#pragma unroll
      for (int j = 0; j < NV; ++j) ss = rms_accumulate(ss, z[j]);
      return 1.0f / sqrtf(block_sum<256>(ss, red) / (float)H + eps);
    };
    const float scale = p.factor * inverse(v, p.centered, p.eps);
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int i = (j * 256 + threadIdx.x) * 4;
      xv[j] = make_float4(xv[j].x + v[j].x * scale * gv[j].x, xv[j].y + v[j].y * scale * gv[j].y, xv[j].z + v[j].z * scale * gv[j].z,
                          xv[j].w + v[j].w * scale * gv[j].w);
      if (i < H) *reinterpret_cast<float4*>(row + i) = xv[j];
    }
    if (!out) return;
    const float next = inverse(xv, p.next_centered, p.next_eps);
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int i = (j * 256 + threadIdx.x) * 4;
      if (i >= H) continue;
      const float4 o = make_float4(xv[j].x * next * nv[j].x, xv[j].y * next * nv[j].y, xv[j].z * next * nv[j].z, xv[j].w * next * nv[j].w);
      RT* dst = out + (size_t)m * H + i;
      if constexpr (sizeof(RT) == 2) {
        *reinterpret_cast<uint2*>(dst) = make_uint2(pack_bf16x2(o.x, o.y), pack_bf16x2(o.z, o.w));
      } else {
        *reinterpret_cast<float4*>(dst) = o;
      }
    }
  } else {
    auto value = [&](int i) {
      float v = 0.f;
      for (int k = 0; k < terms; ++k) {
        const float a = source(k)[i];
        v = k == 0 ? a : v + a;
      }
      v *= p.y_scale;
      return plus ? fmaf(pg, plus[(size_t)m * H + i], v) : v;
    };
    auto inverse = [&](auto z, int centered, float eps, float* mean) {
      *mean = 0.f;
      if (centered) {
        float sum = 0.f;
        for (int i = threadIdx.x; i < H; i += 256) sum += z(i);
        *mean = block_sum<256>(sum, red) / (float)H;
      }
      float ss = 0.f;
      for (int i = threadIdx.x; i < H; i += 256) {
        const float v = z(i) - *mean;
        ss = fmaf(v, v, ss);
      }
      return 1.0f / sqrtf(block_sum<256>(ss, red) / (float)H + eps);
    };
    float mean;
    const float scale = p.factor * inverse(value, p.centered, p.eps, &mean);
    for (int i = threadIdx.x; i < H; i += 256) row[i] = row[i] + (value(i) - mean) * scale * p.g[i];
    if (!out) return;
    const float next = inverse([&](int i) { return row[i]; }, p.next_centered, p.next_eps, &mean);      // (its own elements)
    for (int i = threadIdx.x; i < H; i += 256) st<RT>(out + (size_t)m * H + i, (row[i] - mean) * next * p.next_g[i]);
  }
}

extern "C" int ti_norm_residual_next(float* x, const float* y, const int* gather, int n_gather, const float* plus, const float* plus_gate,
                                     const ti_norm_pair* norms, void* out, int out_dtype, int M, int H, hipStream_t stream) {
  TI_REQUIRE(M >= 0 && H > 0 && (!gather || n_gather > 0) && norms && norms->g && (!out || norms->next_g),
             "norm_residual_next: bad sizes M=%d H=%d gather=%d", M, H, n_gather);
  TI_REQUIRE(!out || out_dtype == TI_F32 || out_dtype == TI_BF16, "norm_residual_next: unknown dtype %d", out_dtype);
  if (M == 0) return 0;
  const bool v4 = H % 4 == 0 && H <= 8192 &&
                  (((uintptr_t)x | (uintptr_t)y | (uintptr_t)norms->g | (uintptr_t)plus | (uintptr_t)(out ? norms->next_g : nullptr) | (uintptr_t)out) & 15) == 0;
#define TI_NRN(RT, NV) norm_residual_next_kernel<RT, NV><<<M, 256, 0, stream>>>(x, y, gather, n_gather, plus, plus_gate, *norms, (RT*)out, H)
#define TI_NRN_WIDTH(RT)               \
  do {                                 \
    if (!v4) TI_NRN(RT, 0);            \
    else if (H <= 1024) TI_NRN(RT, 1); \
    else if (H <= 2048) TI_NRN(RT, 2); \
    else if (H <= 4096) TI_NRN(RT, 4); \
    else TI_NRN(RT, 8);                \
  } while (0)
  if (out && out_dtype == TI_BF16) TI_NRN_WIDTH(bf16_t);
  else TI_NRN_WIDTH(float);
#undef TI_NRN_WIDTH
#undef TI_NRN
  TI_LAUNCH_CHECK();
  return 0;
}

// y[m] += gate[m] plus[m]  (gate null: times one)
__global__ void add_gated_rows_kernel(float* __restrict__ y, const float* __restrict__ plus, const float* __restrict__ gate, long n, int H) {
  for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (long)gridDim.x * blockDim.x)
    y[i] = fmaf(gate ? gate[i / H] : 1.f, plus[i], y[i]);
}

extern "C" int ti_add_gated_rows(float* y, const float* plus, const float* gate, int M, int H, hipStream_t stream) {
  TI_REQUIRE(M >= 0 && H > 0, "add_gated_rows: bad sizes M=%d H=%d", M, H);
  if (M == 0) return 0;
  const long n = (long)M * H;
  const unsigned blocks = (unsigned)((n + 255) / 256 < 8192 ? (n + 255) / 256 : 8192);
  add_gated_rows_kernel<<<blocks, 256, 0, stream>>>(y, plus, gate, n, H);
  TI_LAUNCH_CHECK();
  return 0;
}

// out = x rounded to the compute dtype
template <typename T>
__global__ void round_rows_kernel(const float* __restrict__ x, T* __restrict__ out, long n) {
  for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (long)gridDim.x * blockDim.x) st<T>(out + i, x[i]);
}
// eight elements a thread (n a multiple of 8, 16-byte aligned operands): the same bits
__global__ void __launch_bounds__(256) round_rows_wide_kernel(const float* __restrict__ x, bf16_t* __restrict__ out, long n8) {
  for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < n8; i += (long)gridDim.x * blockDim.x) {
    const float4 a = reinterpret_cast<const float4*>(x)[2 * i], b = reinterpret_cast<const float4*>(x)[2 * i + 1];
    reinterpret_cast<uint4*>(out)[i] = make_uint4(pack_bf16x2(a.x, a.y), pack_bf16x2(a.z, a.w), pack_bf16x2(b.x, b.y),
                                                  pack_bf16x2(b.z, b.w));
  }
}

extern "C" int ti_round_rows(int out_dtype, const float* x, void* out, long n, hipStream_t stream) {
  TI_REQUIRE(n >= 0, "round_rows: bad count %ld", n);
  if (n == 0) return 0;
  if (out_dtype == TI_BF16 && n % 8 == 0 && (((uintptr_t)x | (uintptr_t)out) & 15) == 0) {
    const long n8 = n / 8;
    const unsigned blocks = (unsigned)((n8 + 255) / 256 < 8192 ? (n8 + 255) / 256 : 8192);
    round_rows_wide_kernel<<<blocks, 256, 0, stream>>>(x, (bf16_t*)out, n8);
    TI_LAUNCH_CHECK();
    return 0;
  }
  const unsigned blocks = (unsigned)((n + 255) / 256 < 16384 ? (n + 255) / 256 : 16384);
  if (out_dtype == TI_F32) round_rows_kernel<float><<<blocks, 256, 0, stream>>>(x, (float*)out, n);
  else if (out_dtype == TI_BF16) round_rows_kernel<bf16_t><<<blocks, 256, 0, stream>>>(x, (bf16_t*)out, n);
  else TI_REQUIRE(false, "round_rows: unknown dtype %d", out_dtype);
  TI_LAUNCH_CHECK();
  return 0;
}

// x *= s
__global__ void scale_kernel(float* __restrict__ x, float s, long n) {
  for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (long)gridDim.x * blockDim.x) x[i] *= s;
}

extern "C" int ti_scale(float* x, float s, long n, hipStream_t stream) {
  TI_REQUIRE(n >= 0, "scale: bad count %ld", n);
  if (n == 0) return 0;
  const unsigned blocks = (unsigned)((n + 255) / 256 < 16384 ? (n + 255) / 256 : 16384);
  scale_kernel<<<blocks, 256, 0, stream>>>(x, s, n);
  TI_LAUNCH_CHECK();
  return 0;
}
