// Row operators of the dense (unquantized) models, for activations in bf16 or fp32: embedding lookup,
// residual add + normalisation, the split of a latent-attention projection into queries, latents and
// gates, the ring cache's copies, the gated activation, and a plain matrix-vector product.
//
// T is the element type of weights and activations: uint16_t (bf16 bits) or float.  The residual
// stream, norm statistics, angles and gates are fp32 whatever T is.
//
// Padding: every width a kernel sees is a multiple of 8; columns past the model's own width hold
// zeros (the packed weights have zero rows and columns there), and statistics divide by the true width.
#pragma once
#include <type_traits>

#include "ajq_common.h"

namespace ajq {

__device__ __forceinline__ float to_f32(float v) { return v; }
__device__ __forceinline__ float to_f32(uint16_t v) { return __uint_as_float((uint32_t)v << 16); }
template <typename T> __device__ __forceinline__ T from_f32(float v);
template <> __device__ __forceinline__ float from_f32<float>(float v) { return v; }
template <> __device__ __forceinline__ uint16_t from_f32<uint16_t>(float v) { return f32_to_bf16_rne(v); }

__device__ __forceinline__ float4 load4(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ float4 load4(const uint16_t* p) {
  const u32x2_t v = *reinterpret_cast<const u32x2_t*>(p);
  return float4{__uint_as_float(v.x << 16), __uint_as_float(v.x & 0xFFFF0000u), __uint_as_float(v.y << 16),
                __uint_as_float(v.y & 0xFFFF0000u)};
}
__device__ __forceinline__ void store4(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }
__device__ __forceinline__ void store4(uint16_t* p, float4 v) {
  *reinterpret_cast<u32x2_t*>(p) = u32x2_t{pack2_bf16(v.x, v.y), pack2_bf16(v.z, v.w)};
}

struct Float8 {
  float v[8];
};
__device__ __forceinline__ Float8 load8(const float* p) {
  const float4 a = load4(p), b = load4(p + 4);
  return Float8{{a.x, a.y, a.z, a.w, b.x, b.y, b.z, b.w}};
}
__device__ __forceinline__ Float8 load8(const uint16_t* p) {
  const u32x4_t q = *reinterpret_cast<const u32x4_t*>(p);
  Float8 f;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    f.v[2 * i] = __uint_as_float(q[i] << 16);
    f.v[2 * i + 1] = __uint_as_float(q[i] & 0xFFFF0000u);
  }
  return f;
}
__device__ __forceinline__ void store8(float* p, const Float8& f) {
  store4(p, float4{f.v[0], f.v[1], f.v[2], f.v[3]});
  store4(p + 4, float4{f.v[4], f.v[5], f.v[6], f.v[7]});
}
__device__ __forceinline__ void store8(uint16_t* p, const Float8& f) {
  *reinterpret_cast<u32x4_t*>(p) = u32x4_t{pack2_bf16(f.v[0], f.v[1]), pack2_bf16(f.v[2], f.v[3]), pack2_bf16(f.v[4], f.v[5]),
                                           pack2_bf16(f.v[6], f.v[7])};
}

__device__ __forceinline__ float wave_sum64(float v) {
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) v += __shfl_xor(v, off);
  return v;
}
__device__ __forceinline__ float wave_max64(float v) {
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) v = fmaxf(v, __shfl_xor(v, off));
  return v;
}
// sum over a 256-thread workgroup, the result in every thread (`part`: four floats of LDS)
__device__ __forceinline__ float block_sum256(float v, float* part) {
  v = wave_sum64(v);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) part[threadIdx.x >> 6] = v;
  __syncthreads();
  return (part[0] + part[1]) + (part[2] + part[3]);
}

// A position read from device memory cannot be checked by the host: it is held inside the tables.
__device__ __forceinline__ int clamped_position(const long long* pos, int offset, int limit) {
  const long long p = (pos ? *pos : 0ll) + offset;
  return (int)min(max(p, 0ll), (long long)limit - 1);
}

// x[m, :] = table[token[m], :] + positions[p, :] (+ extra); `embedded` (optional) keeps the sum without `extra`.
// p = start + m % T, or *pos + m % T with a device-side position.  One workgroup per row; Dp % 8 == 0.
template <typename T>
__global__ __launch_bounds__(256) void embed_kernel(const long long* __restrict__ tokens, const T* __restrict__ table, int V,
                                                    const T* __restrict__ positions, int P, int start,
                                                    const long long* __restrict__ pos, int seq,
                                                    const float* __restrict__ extra, float* __restrict__ x,
                                                    float* __restrict__ embedded, int Dp) {
  const int m = blockIdx.x;
  const long long token = min(max(tokens[m], 0ll), (long long)V - 1);
  const T* row = table + (size_t)token * Dp;
  const T* prow = positions ? positions + (size_t)clamped_position(pos, start + m % seq, P) * Dp : nullptr;
  for (int i = 4 * threadIdx.x; i < Dp; i += 1024) {
    float4 v = load4(row + i);
    if (prow) {
      const float4 p = load4(prow + i);
      v.x += p.x; v.y += p.y; v.z += p.z; v.w += p.w;
    }
    if (embedded) store4(embedded + (size_t)m * Dp + i, v);
    if (extra) {
      const float4 e = load4(extra + i);
      v.x += e.x; v.y += e.y; v.z += e.z; v.w += e.w;
    }
    store4(x + (size_t)m * Dp + i, v);
  }
}

// x[m, :] += delta[m, :] + again[m, :] + step[:] (each optional; written back when any is given), then for j = 1, 2
// (each optional) out_j[m, :] = (x - mean) / sqrt(variance + eps) * gain_j.  `center` = 0 leaves the mean in: an RMS
// norm.  Statistics over the first D of Dp columns, fp32, deviations squared after the mean is known.
// One workgroup per row; the first 8192 columns stay in registers between the passes.
template <typename T, typename DeltaT>
__global__ __launch_bounds__(256) void add_norms_kernel(float* __restrict__ x, const DeltaT* __restrict__ delta,
                                                        const float* __restrict__ again, const float* __restrict__ step,
                                                        const float* __restrict__ gain1, const float* __restrict__ gain2,
                                                        float eps, int center, T* __restrict__ out1, T* __restrict__ out2,
                                                        int D, int Dp) {
  constexpr int kKeep = 8;
  __shared__ float part[4];
  const size_t base = (size_t)blockIdx.x * Dp;
  const bool changed = delta || again || step;
  auto take = [&](int i) {
    float4 v = load4(x + base + i);
    if (delta) {
      const float4 d = load4(delta + base + i);
      v.x += d.x; v.y += d.y; v.z += d.z; v.w += d.w;
    }
    if (again) {
      const float4 d = load4(again + base + i);
      v.x += d.x; v.y += d.y; v.z += d.z; v.w += d.w;
    }
    if (step) {
      const float4 d = load4(step + i);
      v.x += d.x; v.y += d.y; v.z += d.z; v.w += d.w;
    }
    if (changed) store4(x + base + i, v);
    return v;
  };
  float4 keep[kKeep];
  float sum = 0.f;
#pragma unroll
  for (int j = 0; j < kKeep; ++j) {
    const int i = 4 * (threadIdx.x + 256 * j);
    keep[j] = float4{0.f, 0.f, 0.f, 0.f};
    if (i < Dp) {
      keep[j] = take(i);
      sum += (keep[j].x + keep[j].y) + (keep[j].z + keep[j].w);  // padding columns are zero
    }
  }
  for (int i = 4 * (threadIdx.x + 256 * kKeep); i < Dp; i += 1024) {
    const float4 v = take(i);
    sum += (v.x + v.y) + (v.z + v.w);
  }
  if (!out1 && !out2) return;
  const float mean = center ? block_sum256(sum, part) / (float)D : 0.f;
  float ss = 0.f;
  auto square = [&](int i, const float4& v) {
    const float a = v.x - mean, b = v.y - mean, c = v.z - mean, d = v.w - mean;
    if (i + 3 < D) {
      ss += (a * a + b * b) + (c * c + d * d);
    } else {  // the row's true end lies inside these four columns or before them
      if (i < D) ss += a * a;
      if (i + 1 < D) ss += b * b;
      if (i + 2 < D) ss += c * c;
    }
  };
#pragma unroll
  for (int j = 0; j < kKeep; ++j) {
    const int i = 4 * (threadIdx.x + 256 * j);
    if (i < Dp) square(i, keep[j]);
  }
  for (int i = 4 * (threadIdx.x + 256 * kKeep); i < Dp; i += 1024) square(i, load4(x + base + i));
  const Divisor by(sqrtf(block_sum256(ss, part) / (float)D + eps));
  auto put = [&](int i, const float4& v, const float* gain, T* out) {
    const float4 g = load4(gain + i);
    store4(out + base + i, float4{by.divide(v.x - mean) * g.x, by.divide(v.y - mean) * g.y, by.divide(v.z - mean) * g.z,
                                  by.divide(v.w - mean) * g.w});  // gains are zero in the padding columns
  };
#pragma unroll
  for (int j = 0; j < kKeep; ++j) {
    const int i = 4 * (threadIdx.x + 256 * j);
    if (i < Dp) {
      if (out1) put(i, keep[j], gain1, out1);
      if (out2) put(i, keep[j], gain2, out2);
    }
  }
  for (int i = 4 * (threadIdx.x + 256 * kKeep); i < Dp; i += 1024) {
    const float4 v = load4(x + base + i);
    if (out1) put(i, v, gain1, out1);
    if (out2) put(i, v, gain2, out2);
  }
}

// Sizes of one latent-attention layer as the kernels see them (padded: dimp, rotp, rankp; true: rot, rank).
struct LatentShape {
  int heads, dimp, rot, rotp, rank, rankp;
  float eps;
};
__device__ __forceinline__ float sigmoid_f32(float z) { return 1.0f / (1.0f + expf(-z)); }

// Component i of the rotated vector (halves layout: i pairs with i + rot / 2; slots past rot are padding).
template <typename Y>
__device__ __forceinline__ float rotated(const Y* v, int i, int rot, const float* cosine, const float* sine) {
  const int half = rot >> 1;
  if (i >= rot) return 0.f;
  if (i < half) return to_f32(v[i]) * cosine[i] - to_f32(v[i + half]) * sine[i];
  return to_f32(v[i]) * cosine[i - half] + to_f32(v[i - half]) * sine[i - half];
}
// `count` vectors rotated by the threads of a workgroup, vector n from src(n) to dst(n) (rotp slots): four pairs per
// thread where the halves allow it, one component otherwise.
template <typename Src, typename Dst>
__device__ __forceinline__ void rotate_all(int count, int rot, int rotp, const float* cosine, const float* sine, int tid,
                                           int threads, Src&& src, Dst&& dst) {
  const int half = rot >> 1;
  if ((half & 3) == 0 && rot == rotp) {
    const int quads = half >> 2;
    for (int i = tid; i < count * quads; i += threads) {
      const int n = i / quads, e = 4 * (i % quads);
      const float4 a = load4(src(n) + e), b = load4(src(n) + half + e), c = load4(cosine + e), s = load4(sine + e);
      store4(dst(n) + e, float4{a.x * c.x - b.x * s.x, a.y * c.y - b.y * s.y, a.z * c.z - b.z * s.z, a.w * c.w - b.w * s.w});
      store4(dst(n) + half + e, float4{b.x * c.x + a.x * s.x, b.y * c.y + a.y * s.y, b.z * c.z + a.z * s.z, b.w * c.w + a.w * s.w});
    }
  } else {
    for (int i = tid; i < count * rotp; i += threads) {
      const int n = i / rotp, e = i % rotp;
      const float v = rotated(src(n), e, rot, cosine, sine);
      auto* to = dst(n) + e;
      *to = from_f32<typename std::remove_reference<decltype(*to)>::type>(v);
    }
  }
}

// Projection row y[m] = (q: heads x (dimp | rotp), latent: rankp | rotp, gates: heads) of token m = (b, t):
//   qu[m, h, 0..dimp)  = unrotated query part             (row stride qu_ld per head)
//   qr[m, h, 0..rotp)  = rotated query part               (row stride qr_ld per head)
//   rows[b, slot, :]   = (RMS-normed latent | rotated key part), slot = prior + t, or position % cap when the position
//                        is device data (`pos`, one token per call: the ring cache's slot)
//   gates[m, h]        = sigmoid
// One workgroup per token.
template <typename Y, typename T>
__global__ __launch_bounds__(256) void latent_split_kernel(const Y* __restrict__ y, int ldy, LatentShape s,
                                                           const float* __restrict__ latent_gain,
                                                           const float* __restrict__ cosine, const float* __restrict__ sine,
                                                           int table_rows, int start, const long long* __restrict__ pos, int seq,
                                                           int prior, int cap, T* __restrict__ qu, int qu_ld,
                                                           T* __restrict__ qr, int qr_ld, T* __restrict__ rows,
                                                           long long rows_batch, float* __restrict__ gates) {
  __shared__ float part[4];
  const int m = blockIdx.x, b = m / seq, t = m % seq, tid = threadIdx.x;
  const int p = clamped_position(pos, start + t, table_rows);
  const int slot = pos ? p % cap : prior + t;
  const Y* row = y + (size_t)m * ldy;
  const int dq = s.dimp + s.rotp, rot_pairs = s.rot >> 1;
  const float* cs = cosine + (size_t)p * rot_pairs;
  const float* sn = sine + (size_t)p * rot_pairs;
  const int quads = s.dimp >> 2;
  for (int i = tid; i < s.heads * quads; i += 256) {
    const int h = i / quads, d = 4 * (i % quads);
    store4(qu + ((size_t)m * s.heads + h) * qu_ld + d, load4(row + h * dq + d));
  }
  rotate_all(s.heads, s.rot, s.rotp, cs, sn, tid, 256, [&](int h) { return row + h * dq + s.dimp; },
             [&](int h) { return qr + ((size_t)m * s.heads + h) * qr_ld; });
  const Y* lat = row + s.heads * dq;
  float ss = 0.f;
  for (int i = 4 * tid; i < s.rankp; i += 1024) {  // padding columns are zero
    const float4 v = load4(lat + i);
    ss += (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w);
  }
  const Divisor by(sqrtf(block_sum256(ss, part) / (float)s.rank + s.eps));
  T* dst = rows + (size_t)b * rows_batch + (size_t)slot * (s.rankp + s.rotp);
  for (int i = 4 * tid; i < s.rankp; i += 1024) {
    const float4 v = load4(lat + i), w = load4(latent_gain + i);
    store4(dst + i, float4{by.divide(v.x) * w.x, by.divide(v.y) * w.y, by.divide(v.z) * w.z, by.divide(v.w) * w.w});
  }
  rotate_all(1, s.rot, s.rotp, cs, sn, tid, 256, [&](int) { return lat + s.rankp; }, [&](int) { return dst + s.rankp; });
  for (int h = tid; h < s.heads; h += 256) gates[(size_t)m * s.heads + h] = sigmoid_f32(to_f32(lat[s.rankp + s.rotp + h]));
}

// Slot of a position in a ring of cap rows whose first `kept` positions stay where they are.
__host__ __device__ __forceinline__ int ring_slot(int position, int cap, int kept) {
  return position < kept ? position : kept + (position - kept) % (cap - kept);
}
// Rows of a ring cache [B, cap, width] from / to rows first_row .. of a linear buffer [B, lines, line], starting at position
// `position`.  One thread per 16 bytes; chunks = bytes of a row / 16, line likewise.
__global__ __launch_bounds__(256) void ring_copy_kernel(u32x4_t* __restrict__ ring, int cap, int kept, u32x4_t* __restrict__ linear,
                                                        int lines, int line, int first_row, int position, int count, int chunks,
                                                        int batch, int to_ring) {
  const long long idx = (long long)blockIdx.x * 256 + threadIdx.x;
  if (idx >= (long long)batch * count * chunks) return;
  const int c = (int)(idx % chunks);
  const int i = (int)((idx / chunks) % count);
  const int b = (int)(idx / ((long long)chunks * count));
  u32x4_t* r = ring + ((size_t)b * cap + ring_slot(position + i, cap, kept)) * chunks + c;
  u32x4_t* l = linear + ((size_t)b * lines + first_row + i) * line + c;
  if (to_ring) *r = *l; else *l = *r;
}

enum Activation { kActRelu = 0, kActSilu = 1, kActGeluTanh = 2, kActSquaredRelu = 3 };
__device__ __forceinline__ float activate(int kind, float z) {
  if (kind == kActRelu) return fmaxf(z, 0.f);
  if (kind == kActSilu) return z * sigmoid_f32(z);
  if (kind == kActSquaredRelu) {
    const float r = fmaxf(z, 0.f);
    return r * r;
  }
  const float u = 0.7978845608028654f * (z + 0.044715f * z * z * z);  // sqrt(2 / pi)
  return 0.5f * z * (1.0f + tanhf(u));
}

// y [M, 2 F]: blocks of 8 gate columns and the 8 matching up columns -> out[m, f] = act(gate) * up (row stride ldo).
template <typename Y, typename T>
__global__ __launch_bounds__(256) void gated_activation_kernel(const Y* __restrict__ y, T* __restrict__ out, int ldo, int M, int F,
                                                               int kind) {
  const int quads = F >> 2;
  const long long idx = (long long)blockIdx.x * 256 + threadIdx.x;
  if (idx >= (long long)M * quads) return;
  const int m = (int)(idx / quads), f = 4 * (int)(idx % quads);
  const Y* src = y + (size_t)m * 2 * F + 16 * (f >> 3) + (f & 7);
  const float4 a = load4(src), u = load4(src + 8);
  store4(out + (size_t)m * ldo + f, float4{activate(kind, a.x) * u.x, activate(kind, a.y) * u.y, activate(kind, a.z) * u.z,
                                           activate(kind, a.w) * u.w});
}

// out = act(y) over dense rows of eight-column multiples: one thread per 8 values.
template <typename T>
__global__ __launch_bounds__(256) void activation_kernel(const T* __restrict__ y, T* __restrict__ out, long long eighths, int kind) {
  const long long idx = (long long)blockIdx.x * 256 + threadIdx.x;
  if (idx >= eighths) return;
  Float8 v = load8(y + 8 * idx);
#pragma unroll
  for (int e = 0; e < 8; ++e) v.v[e] = activate(kind, v.v[e]);
  store8(out + 8 * idx, v);
}

// Plain product for any type: y[b, g, n] = sum_k w[g, n, k] x[b, g, k], fp32 sums, one wave per output.
// Grid (ceil(N / 4), G, B); K % 8 == 0.
template <typename T, typename O>
__global__ __launch_bounds__(256) void matvec_kernel(const T* __restrict__ w, const T* __restrict__ x, int x_batch, int x_group,
                                                     O* __restrict__ y, int y_batch, int y_group, int N, int K) {
  const int n = 4 * blockIdx.x + (threadIdx.x >> 6), g = blockIdx.y, b = blockIdx.z, lane = threadIdx.x & 63;
  if (n >= N) return;
  const T* wr = w + ((size_t)g * N + n) * K;
  const T* xr = x + (size_t)b * x_batch + (size_t)g * x_group;
  float acc = 0.f;
  for (int k = 4 * lane; k < K; k += 256) {
    const float4 a = load4(wr + k), v = load4(xr + k);
    acc = fmaf(a.x, v.x, acc);
    acc = fmaf(a.y, v.y, acc);
    acc = fmaf(a.z, v.z, acc);
    acc = fmaf(a.w, v.w, acc);
  }
  acc = wave_sum64(acc);
  if (lane == 0) y[(size_t)b * y_batch + (size_t)g * y_group + n] = from_f32<O>(acc);
}

}  // namespace ajq
