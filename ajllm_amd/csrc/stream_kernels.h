// Hyper-connected residual streams: a row of the residual is S streams of Dp columns, x [M, S, Dp] fp32.  A sublayer reads
// u = sum_s in[s] x_s and its result y (scaled per column) goes back as x_t <- sum_s mix[s][t] x_s + out[t] y.
//
// Both halves are local to a column, so the update of one sublayer and the input of the next are one pass over the streams:
//   streams_norm_kernel    prompts: the pending update, the next input, its RMS norm
//   dense_out_streams      (dense_gemv_kernels.h) one token: the same as the epilogue of the product that makes y
//
// Coefficients of a sublayer, fp32: in[S], out[S], mix[S * S] ([from][to]).
#pragma once
#include "dense_kernels.h"

namespace ajq {

constexpr int kMaxStreams = 16;

// x[m, s, :] = table[token[m], :] for every stream, u[m, :] = (sum of `in`) * that row (optional).  One workgroup per row.
template <typename T>
__global__ __launch_bounds__(256) void embed_streams_kernel(const long long* __restrict__ tokens, const T* __restrict__ table, int V,
                                                            const float* __restrict__ in, float* __restrict__ x,
                                                            float* __restrict__ u, int S, int Dp) {
  const int m = blockIdx.x;
  const long long token = min(max(tokens[m], 0ll), (long long)V - 1);
  const T* row = table + (size_t)token * Dp;
  float* dst = x + (size_t)m * S * Dp;
  for (int i = 4 * threadIdx.x; i < Dp; i += 1024) {
    const float4 v = load4(row + i);
    float4 w = float4{0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < S; ++s) {
      store4(dst + (size_t)s * Dp + i, v);
      if (u) {
        const float f = in[s];
        w.x = fmaf(f, v.x, w.x); w.y = fmaf(f, v.y, w.y); w.z = fmaf(f, v.z, w.z); w.w = fmaf(f, v.w, w.w);
      }
    }
    if (u) store4(u + (size_t)m * Dp + i, w);
  }
}

// Four columns of every stream: update by `y` (already scaled), weighted sum for the next reader.
// `in` null: the plain sum.  Coefficients are uniform over the launch.
template <int MAXS>
__device__ __forceinline__ void mix_streams(float4 (&v)[MAXS], int S, const float* __restrict__ out, const float* __restrict__ mix, float4 y) {
  float4 w[MAXS];
#pragma unroll
  for (int t = 0; t < MAXS; ++t) {
    if (t >= S) continue;
    const float o = out[t];
    w[t] = float4{o * y.x, o * y.y, o * y.z, o * y.w};
#pragma unroll
    for (int s = 0; s < MAXS; ++s) {
      if (s >= S) continue;
      const float f = mix[s * S + t];
      w[t].x = fmaf(f, v[s].x, w[t].x); w[t].y = fmaf(f, v[s].y, w[t].y);
      w[t].z = fmaf(f, v[s].z, w[t].z); w[t].w = fmaf(f, v[s].w, w[t].w);
    }
  }
#pragma unroll
  for (int t = 0; t < MAXS; ++t)
    if (t < S) v[t] = w[t];
}
template <int MAXS>
__device__ __forceinline__ float4 read_streams(const float4 (&v)[MAXS], int S, const float* __restrict__ in) {
  float4 u = float4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int s = 0; s < MAXS; ++s) {
    if (s >= S) continue;
    const float f = in ? in[s] : 1.f;
    u.x = fmaf(f, v[s].x, u.x); u.y = fmaf(f, v[s].y, u.y); u.z = fmaf(f, v[s].z, u.z); u.w = fmaf(f, v[s].w, u.w);
  }
  return u;
}

// With delta: x <- mixed streams + out * (scale * delta), written back.  Then u = sum in[s] x_s (kept if `u` is given) and
// normed = u / sqrt(mean(u^2) + eps) * gain (if given).  One workgroup per row; the first 8192 columns of u stay in registers.
template <typename T, int MAXS>
__global__ __launch_bounds__(256) void streams_norm_kernel(float* __restrict__ x, const float* __restrict__ delta,
                                                           const float* __restrict__ scale, const float* __restrict__ out,
                                                           const float* __restrict__ mix, const float* __restrict__ in,
                                                           const float* __restrict__ gain, float eps, T* __restrict__ normed,
                                                           float* __restrict__ u, int S, int D, int Dp) {
  constexpr int kKeep = 8;
  __shared__ float part[4];
  const size_t base = (size_t)blockIdx.x * Dp;
  float* xr = x + base * S;
  auto take = [&](int i) {
    float4 v[MAXS];
#pragma unroll
    for (int s = 0; s < MAXS; ++s)
      if (s < S) v[s] = load4(xr + (size_t)s * Dp + i);
    if (delta) {
      const float4 d = load4(delta + base + i), f = load4(scale + i);
      mix_streams<MAXS>(v, S, out, mix, float4{d.x * f.x, d.y * f.y, d.z * f.z, d.w * f.w});
#pragma unroll
      for (int s = 0; s < MAXS; ++s)
        if (s < S) store4(xr + (size_t)s * Dp + i, v[s]);
    }
    const float4 r = read_streams<MAXS>(v, S, in);
    if (u) store4(u + base + i, r);
    return r;
  };
  float4 keep[kKeep];
  float ss = 0.f;
  auto square = [&](const float4& v) { ss += (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w); };  // padding columns are zero
#pragma unroll
  for (int j = 0; j < kKeep; ++j) {
    const int i = 4 * (threadIdx.x + 256 * j);
    if (i < Dp) {
      keep[j] = take(i);
      square(keep[j]);
    }
  }
  for (int i = 4 * (threadIdx.x + 256 * kKeep); i < Dp; i += 1024) square(take(i));
  if (!normed) return;
  const Divisor by(sqrtf(block_sum256(ss, part) / (float)D + eps));
  auto put = [&](int i, const float4& v) {
    const float4 g = load4(gain + i);
    store4(normed + base + i, float4{by.divide(v.x) * g.x, by.divide(v.y) * g.y, by.divide(v.z) * g.z, by.divide(v.w) * g.w});
  };
#pragma unroll
  for (int j = 0; j < kKeep; ++j) {
    const int i = 4 * (threadIdx.x + 256 * j);
    if (i < Dp) put(i, keep[j]);
  }
  for (int i = 4 * (threadIdx.x + 256 * kKeep); i < Dp; i += 1024) {  // (this thread's own columns, written above where they changed)
    float4 v[MAXS];
#pragma unroll
    for (int s = 0; s < MAXS; ++s)
      if (s < S) v[s] = load4(xr + (size_t)s * Dp + i);
    put(i, read_streams<MAXS>(v, S, in));
  }
}

}  // namespace ajq
