// Matrix-vector products of one decode step for dense bf16 weights [N, K] (row-major, N % 16 == 0, K % 8 == 0) on
// MFMA, up to 16 sequences per workgroup (grid.y deals larger batches), with what surrounds them folded in:
//
//   dense_in_kernel      two weight matrices that read the same fp32 residual row through norms of their own: the layer
//                        norm is the prologue (or bf16 rows a norm launch left); the first matrix's outputs are stored
//                        in fp32, the second's are gated pairs (8 gate rows and their 8 up rows per 16-row tile)
//   latent_absorb_kernel per-head products of the unrotated query with the transposed key expansion, so that attention
//                        can run on the latents; beside them the rotation of the query, and the new cache row (RMS norm of
//                        the latent, rotation of the shared key part)
//   latent_expand_kernel merge of the attention's row chunks (with the sink), per-head value expansion, output gate
//   dense_out_kernel     product with the residual add (and whatever the next layer run adds first) as epilogue
//
// A 16 x 16 output tile (16 weight rows, 16 batch columns) belongs to a wave, or to kWaves waves that split K and meet in
// LDS.  Lane l = 16 g + r loads 16 bytes of weight row r at k = 32 step + 8 g: four lanes cover 64 contiguous bytes of a
// row, two steps a cache line.
#pragma once
#include "dense_kernels.h"
#include "prefill_attention.h"

namespace ajq {

constexpr int kGemvBatch = 16;

// acc += W[rows of the tile, steps begin .. end) x; `wrow` points at this lane's row, `x(step)` gives its B fragment
// (batch column r, k = 32 step + 8 g ..), both zero past K.
template <typename XFn>
__device__ __forceinline__ f32x4_t tile_steps(const uint16_t* __restrict__ wrow, int K, int begin, int end, int g, f32x4_t acc,
                                              XFn&& x) {
  constexpr int kUnroll = 8;
  const u32x4_t zero = {0u, 0u, 0u, 0u};
  for (int s0 = begin; s0 < end; s0 += kUnroll) {
    u32x4_t w[kUnroll], v[kUnroll];
#pragma unroll
    for (int i = 0; i < kUnroll; ++i) {
      const int k = 32 * (s0 + i) + 8 * g;
      w[i] = zero;
      if (s0 + i < end && k < K) w[i] = *reinterpret_cast<const u32x4_t*>(wrow + k);
    }
#pragma unroll
    for (int i = 0; i < kUnroll; ++i) {
      v[i] = zero;
      if (s0 + i < end && 32 * (s0 + i) + 8 * g < K) v[i] = x(s0 + i);
    }
#pragma unroll
    for (int i = 0; i < kUnroll; ++i) acc = mfma16(w[i], v[i], acc);
  }
  return acc;
}

// the K range of one of kWaves waves, in pairs of steps (a cache line of a weight row stays with one wave)
__device__ __forceinline__ void wave_steps(int K, int wave, int waves, int& begin, int& end) {
  const int steps = (K + 31) >> 5;
  const int per = ((steps + waves - 1) / waves + 1) & ~1;
  begin = min(steps, wave * per);
  end = min(steps, begin + per);
}

// sum of the waves' tiles; valid in wave 0
template <int kWaves>
__device__ __forceinline__ f32x4_t meet(f32x4_t acc, float* red, int wave, int lane) {
  if (kWaves == 1) return acc;
  float4* slot = reinterpret_cast<float4*>(red);
  if (wave > 0) slot[(wave - 1) * 64 + lane] = float4{acc[0], acc[1], acc[2], acc[3]};
  __syncthreads();
  if (wave == 0) {
#pragma unroll
    for (int w = 0; w < kWaves - 1; ++w) {
      const float4 o = slot[w * 64 + lane];
      acc[0] += o.x; acc[1] += o.y; acc[2] += o.z; acc[3] += o.w;
    }
  }
  return acc;
}

struct DenseIn {
  const float* x;           // [B, Dp] residual rows (norm prologue)
  const uint16_t* n1;       // or [B, Dp] bf16 rows already normed by gain 1 / gain 2
  const uint16_t* n2;
  const float* gain1;
  const float* gain2;
  const uint16_t* w1;       // [16 tiles1, Dp]
  const uint16_t* w2;       // [16 tiles2, Dp], gate / up rows interleaved in blocks of 8
  float* y1;                // [B, 16 tiles1]
  uint16_t* gated;          // [B, gated_ld], column 8 * tile + j
  int batch, D, Dp, tiles1, tiles2, gated_ld, act, center;
  float eps;
};

// kNorm: the norm is formed here, for the rows of one batch block (dynamic LDS: rows x (Dp + 8) bf16).
template <int kWaves, bool kNorm>
__global__ __launch_bounds__(64 * kWaves) void dense_in_kernel(DenseIn a) {
  extern __shared__ __attribute__((aligned(16))) uint16_t normed[];
  __shared__ float red[kWaves > 1 ? (kWaves - 1) * 256 : 4];
  __shared__ float stat[kWaves];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
  const int b0 = blockIdx.y * kGemvBatch, nb = min(kGemvBatch, a.batch - b0);
  const bool second = (int)blockIdx.x >= a.tiles1;
  const int tile = second ? (int)blockIdx.x - a.tiles1 : (int)blockIdx.x;
  const uint16_t* wrow = (second ? a.w2 : a.w1) + (size_t)(16 * tile + r) * a.Dp;
  int begin, end;
  wave_steps(a.Dp, wave, kWaves, begin, end);
  f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
  if constexpr (kNorm) {
    const float* gain = second ? a.gain2 : a.gain1;
    constexpr int kThreads = 64 * kWaves, kKeep = 4;
    const int stride = a.Dp + 8;
    auto block_sum = [&](float v) {
      v = wave_sum64(v);
      __syncthreads();
      if (lane == 0) stat[wave] = v;
      __syncthreads();
      float s = stat[0];
#pragma unroll
      for (int w = 1; w < kWaves; ++w) s += stat[w];
      return s;
    };
    for (int b = 0; b < nb; ++b) {
      const float* x = a.x + (size_t)(b0 + b) * a.Dp;
      float4 keep[kKeep];
      float sum = 0.f;
#pragma unroll
      for (int j = 0; j < kKeep; ++j) {
        const int i = 4 * (threadIdx.x + kThreads * j);
        keep[j] = i < a.Dp ? load4(x + i) : float4{0.f, 0.f, 0.f, 0.f};
        sum += (keep[j].x + keep[j].y) + (keep[j].z + keep[j].w);
      }
      for (int i = 4 * (threadIdx.x + kThreads * kKeep); i < a.Dp; i += 4 * kThreads) {
        const float4 v = load4(x + i);
        sum += (v.x + v.y) + (v.z + v.w);
      }
      const float mean = a.center ? block_sum(sum) / (float)a.D : 0.f;
      float ss = 0.f;
      auto square = [&](int i, const float4& v) {
        const float p = v.x - mean, q = v.y - mean, s = v.z - mean, t = v.w - mean;
        if (i + 3 < a.D) {
          ss += (p * p + q * q) + (s * s + t * t);
        } else {
          if (i < a.D) ss += p * p;
          if (i + 1 < a.D) ss += q * q;
          if (i + 2 < a.D) ss += s * s;
        }
      };
#pragma unroll
      for (int j = 0; j < kKeep; ++j) square(4 * (threadIdx.x + kThreads * j), keep[j]);
      for (int i = 4 * (threadIdx.x + kThreads * kKeep); i < a.Dp; i += 4 * kThreads) square(i, load4(x + i));
      const Divisor by(sqrtf(block_sum(ss) / (float)a.D + a.eps));
      auto put = [&](int i, const float4& v) {
        const float4 w = load4(gain + i);
        store4(normed + b * stride + i, float4{by.divide(v.x - mean) * w.x, by.divide(v.y - mean) * w.y,
                                               by.divide(v.z - mean) * w.z, by.divide(v.w - mean) * w.w});
      };
#pragma unroll
      for (int j = 0; j < kKeep; ++j) {
        const int i = 4 * (threadIdx.x + kThreads * j);
        if (i < a.Dp) put(i, keep[j]);
      }
      for (int i = 4 * (threadIdx.x + kThreads * kKeep); i < a.Dp; i += 4 * kThreads) put(i, load4(x + i));
    }
    __syncthreads();
    const uint16_t* xr = normed + min(r, nb - 1) * stride + 8 * g;
    acc = tile_steps(wrow, a.Dp, begin, end, g, acc, [&](int s) {
      return r < nb ? *reinterpret_cast<const u32x4_t*>(xr + 32 * s) : u32x4_t{0u, 0u, 0u, 0u};
    });
  } else {
    const uint16_t* xr = (second ? a.n2 : a.n1) + (size_t)(b0 + min(r, nb - 1)) * a.Dp + 8 * g;
    acc = tile_steps(wrow, a.Dp, begin, end, g, acc, [&](int s) {
      return r < nb ? *reinterpret_cast<const u32x4_t*>(xr + 32 * s) : u32x4_t{0u, 0u, 0u, 0u};
    });
  }
  acc = meet<kWaves>(acc, red, wave, lane);
  if (wave != 0) return;
  if (!second) {
    if (r < nb) *reinterpret_cast<float4*>(a.y1 + (size_t)(b0 + r) * (16 * a.tiles1) + 16 * tile + 4 * g) =
        float4{acc[0], acc[1], acc[2], acc[3]};
    return;
  }
  // rows 0 .. 7 of the tile (lanes g < 2) are gates, rows 8 .. 15 (lanes g >= 2, 32 lanes on) the matching up rows
  float v[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) v[i] = activate(a.act, acc[i]) * __shfl_xor(acc[i], 32);
  if (g < 2 && r < nb)
    *reinterpret_cast<u32x2_t*>(a.gated + (size_t)(b0 + r) * a.gated_ld + 8 * tile + 4 * g) =
        u32x2_t{pack2_bf16(v[0], v[1]), pack2_bf16(v[2], v[3])};
}

struct DenseOut {
  const uint16_t* in;       // [B, K]
  const uint16_t* w;        // [Dp, K]
  float* x;                 // [B, Dp], updated in place
  const float* again;       // [B, Dp] or null, added too
  const float* step;        // [Dp] or null, added too
  int batch, K, Dp;
};
template <int kWaves>
__global__ __launch_bounds__(64 * kWaves) void dense_out_kernel(DenseOut a) {
  __shared__ float red[kWaves > 1 ? (kWaves - 1) * 256 : 4];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
  const int b0 = blockIdx.y * kGemvBatch, nb = min(kGemvBatch, a.batch - b0);
  const uint16_t* wrow = a.w + (size_t)(16 * blockIdx.x + r) * a.K;
  const uint16_t* xr = a.in + (size_t)(b0 + min(r, nb - 1)) * a.K + 8 * g;
  int begin, end;
  wave_steps(a.K, wave, kWaves, begin, end);
  const size_t at = (size_t)(b0 + min(r, nb - 1)) * a.Dp + 16 * blockIdx.x + 4 * g;
  float4 v = float4{0.f, 0.f, 0.f, 0.f};
  if (wave == 0) {  // what the product is added to, requested ahead of it
    v = load4(a.x + at);
    if (a.again) {
      const float4 e = load4(a.again + at);
      v.x += e.x; v.y += e.y; v.z += e.z; v.w += e.w;
    }
    if (a.step) {
      const float4 e = load4(a.step + 16 * blockIdx.x + 4 * g);
      v.x += e.x; v.y += e.y; v.z += e.z; v.w += e.w;
    }
  }
  f32x4_t acc = tile_steps(wrow, a.K, begin, end, g, f32x4_t{0.f, 0.f, 0.f, 0.f}, [&](int s) {
    return r < nb ? *reinterpret_cast<const u32x4_t*>(xr + 32 * s) : u32x4_t{0u, 0u, 0u, 0u};
  });
  acc = meet<kWaves>(acc, red, wave, lane);
  if (wave != 0 || r >= nb) return;
  store4(a.x + at, float4{v.x + acc[0], v.y + acc[1], v.z + acc[2], v.w + acc[3]});
}

struct LatentAbsorb {
  const float* y;           // [B, ldy] projection rows (see latent_split_kernel)
  const uint16_t* ukt;      // [H, rankp, dimp] transposed key expansion
  const float* latent_gain; // [rankp]
  const float* cosine;      // [table_rows, rot / 2]
  const float* sine;
  const long long* pos;
  uint16_t* q;              // [B, H, rankp + rotp]
  uint16_t* ring;           // [B, cap, rankp + rotp]
  int batch, ldy, table_rows, cap, groups;  // groups: workgroups per head (4 tiles of 16 latent columns each)
  LatentShape s;
};
// Grid (H * groups + 1, batch blocks); the last workgroup of a batch block makes the cache rows.
__global__ __launch_bounds__(256) void latent_absorb_kernel(LatentAbsorb a) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
  const int b0 = blockIdx.y * kGemvBatch, nb = min(kGemvBatch, a.batch - b0);
  const LatentShape s = a.s;
  const int dq = s.dimp + s.rotp, width = s.rankp + s.rotp;
  const int p = clamped_position(a.pos, 0, a.table_rows);
  const float* cs = a.cosine + (size_t)p * (s.rot >> 1);
  const float* sn = a.sine + (size_t)p * (s.rot >> 1);
  if ((int)blockIdx.x == s.heads * a.groups) {
    for (int b = wave; b < nb; b += 4) {  // a wave per sequence
      const float* lat = a.y + (size_t)(b0 + b) * a.ldy + s.heads * dq;
      float ss = 0.f;
      for (int i = 4 * lane; i < s.rankp; i += 256) {  // padding columns are zero
        const float4 v = load4(lat + i);
        ss += (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w);
      }
      const Divisor by(sqrtf(wave_sum64(ss) / (float)s.rank + s.eps));
      uint16_t* dst = a.ring + ((size_t)(b0 + b) * a.cap + p % a.cap) * width;
      for (int i = 4 * lane; i < s.rankp; i += 256) {
        const float4 v = load4(lat + i), w = load4(a.latent_gain + i);
        store4(dst + i, float4{by.divide(v.x) * w.x, by.divide(v.y) * w.y, by.divide(v.z) * w.z, by.divide(v.w) * w.w});
      }
      for (int i = lane; i < s.rotp; i += 64) dst[s.rankp + i] = f32_to_bf16_rne(rotated(lat + s.rankp, i, s.rot, cs, sn));
    }
    return;
  }
  const int h = blockIdx.x / a.groups, grp = blockIdx.x % a.groups;
  if (grp == 0) {
    for (int i = threadIdx.x; i < nb * s.rotp; i += 256) {
      const int b = b0 + i / s.rotp, d = i % s.rotp;
      a.q[((size_t)b * s.heads + h) * width + s.rankp + d] =
          f32_to_bf16_rne(rotated(a.y + (size_t)b * a.ldy + h * dq + s.dimp, d, s.rot, cs, sn));
    }
  }
  const int tile = 4 * grp + wave;
  if (16 * tile >= s.rankp) return;
  const uint16_t* wrow = a.ukt + ((size_t)h * s.rankp + 16 * tile + r) * s.dimp;
  const float* xr = a.y + (size_t)(b0 + min(r, nb - 1)) * a.ldy + h * dq + 8 * g;
  const f32x4_t acc = tile_steps(wrow, s.dimp, 0, (s.dimp + 31) >> 5, g, f32x4_t{0.f, 0.f, 0.f, 0.f}, [&](int st) {
    if (r >= nb) return u32x4_t{0u, 0u, 0u, 0u};
    const float4 u = load4(xr + 32 * st), v = load4(xr + 32 * st + 4);
    return u32x4_t{pack2_bf16(u.x, u.y), pack2_bf16(u.z, u.w), pack2_bf16(v.x, v.y), pack2_bf16(v.z, v.w)};
  });
  if (r < nb)
    *reinterpret_cast<u32x2_t*>(a.q + ((size_t)(b0 + r) * s.heads + h) * width + 16 * tile + 4 * g) =
        u32x2_t{pack2_bf16(acc[0], acc[1]), pack2_bf16(acc[2], acc[3])};
}

// One chunk of cache rows against 16 heads of one sequence, in the latent space: row j of the ring
// (latent rankp | rotated rotp) is the key, its latent part the value, for every head.  Blocks of 64 rows are staged in LDS
// once for both products: S^T = K Q^T (a wave takes 16 keys), then U^T += C^T P^T with the latents read by transposing
// LDS reads (a wave takes every fourth 16-column tile of the latent).  Grid (head tiles, chunks S, B).
// Partial result of (b, h, chunk): (maximum, denominator, 0, 0, rankp sums), base-2 exponents.
struct LatentDecode {
  const uint16_t* q;        // [B, H, width]
  const uint16_t* ring;     // [B, cap, width]
  const long long* pos;
  float* partial;           // [B, H, S, rankp + 4]
  int heads, rankp, width, cap, chunks;
  float scale2;
};
__host__ __device__ constexpr int latent_row_bytes(int width) { return ((width + 31) / 32) * 64 + 16; }
constexpr int kLatentRows = 64;
constexpr int kLatentPBytes = (kLatentRows + 8) * 2;
__host__ __device__ constexpr int latent_decode_lds(int width) {
  return (kLatentRows + 16) * latent_row_bytes(width) + 16 * kLatentPBytes;
}
template <int RT>
__global__ __launch_bounds__(256) void latent_decode_kernel(LatentDecode a) {
  extern __shared__ __attribute__((aligned(1024))) unsigned char lds[];
  __shared__ float smax[4][16], ssum[4][16];
  const uint32_t lds0 = (uint32_t)(uintptr_t)(pf_lds_char_t*)lds;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), r = lane & 15, g = lane >> 4;
  const int b = blockIdx.z, h0 = 16 * blockIdx.x, chunk = blockIdx.y;
  const int rb = latent_row_bytes(a.width), steps = (a.width + 31) >> 5, kc = 4 * steps, cw = a.width >> 3;
  const int valid = (int)min(max(*a.pos, 0ll), (long long)a.cap - 1) + 1;  // rows the ring holds
  const int per = (((valid + a.chunks - 1) / a.chunks) + kLatentRows - 1) & ~(kLatentRows - 1);
  const int begin = chunk * per, end = min(valid, begin + per);
  float* head_out = a.partial + (((size_t)b * a.heads + min(h0 + r, a.heads - 1)) * a.chunks + chunk) * (a.rankp + 4);
  if (begin >= end) {
    if (wave == 0 && g == 0 && h0 + r < a.heads) *reinterpret_cast<float4*>(head_out) = float4{-INFINITY, 0.f, 0.f, 0.f};
    return;
  }
  const u32x4_t zero = {0u, 0u, 0u, 0u};
  const uint32_t q_at = (uint32_t)(kLatentRows * rb), p_at = q_at + (uint32_t)(16 * rb);
  for (int ci = threadIdx.x; ci < 16 * kc; ci += 256) {
    const int row = ci / kc, c = ci % kc;
    u32x4_t v = zero;
    if (h0 + row < a.heads && c < cw)
      v = *reinterpret_cast<const u32x4_t*>(a.q + ((size_t)b * a.heads + h0 + row) * a.width + 8 * c);
    *reinterpret_cast<u32x4_t*>(lds + q_at + row * rb + 16 * c) = v;
  }
  const uint16_t* ring = a.ring + (size_t)b * a.cap * a.width;
  float m = -INFINITY, l = 0.f;
  f32x4_t u[RT];
#pragma unroll
  for (int t = 0; t < RT; ++t) u[t] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  for (int j0 = begin; j0 < end; j0 += kLatentRows) {
    constexpr int kFly = 6;
    for (int c0 = 0; c0 < kLatentRows * kc; c0 += 256 * kFly) {
      u32x4_t v[kFly];
#pragma unroll
      for (int i = 0; i < kFly; ++i) {
        const int ci = c0 + 256 * i + threadIdx.x, row = ci / kc, c = ci % kc;
        v[i] = zero;
        if (row < kLatentRows && j0 + row < end && c < cw)
          v[i] = *reinterpret_cast<const u32x4_t*>(ring + (size_t)(j0 + row) * a.width + 8 * c);
      }
#pragma unroll
      for (int i = 0; i < kFly; ++i) {
        const int ci = c0 + 256 * i + threadIdx.x, row = ci / kc, c = ci % kc;
        if (row < kLatentRows) *reinterpret_cast<u32x4_t*>(lds + row * rb + 16 * c) = v[i];
      }
    }
    __syncthreads();
    f32x4_t sc = {0.f, 0.f, 0.f, 0.f};
    const uint32_t k_rd = lds0 + (uint32_t)((16 * wave + r) * rb + 16 * g), q_rd = lds0 + q_at + (uint32_t)(r * rb + 16 * g);

    for (int s = 0; s < steps; ++s) sc = mfma16(pf_read128(k_rd + 64u * s), pf_read128(q_rd + 64u * s), sc);
    // sc[i]: key j0 + 16 wave + 4 g + i, head h0 + r
    float mx = -INFINITY;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      sc[i] = j0 + 16 * wave + 4 * g + i < end ? sc[i] * a.scale2 : -INFINITY;
      mx = fmaxf(mx, sc[i]);
    }
    mx = quad_max(mx);
    if (g == 0) smax[wave][r] = mx;
    __syncthreads();
    // (finite: the block's first row is valid)
    const float m_new = fmaxf(fmaxf(fmaxf(smax[0][r], smax[1][r]), fmaxf(smax[2][r], smax[3][r])), m);
    const float corr = exp2f(m - m_new);
    m = m_new;
    float p[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) p[i] = exp2f(sc[i] - m);
    l = l * corr + ((p[0] + p[1]) + (p[2] + p[3]));
    *reinterpret_cast<u32x2_t*>(lds + p_at + r * kLatentPBytes + 2 * (16 * wave + 4 * g)) =
        u32x2_t{pack2_bf16(p[0], p[1]), pack2_bf16(p[2], p[3])};
#pragma unroll
    for (int t = 0; t < RT; ++t) u[t] *= corr;
    __syncthreads();
#pragma unroll
    for (int hf = 0; hf < 2; ++hf) {
      const unsigned char* pr = lds + p_at + r * kLatentPBytes + 2 * (32 * hf + 4 * g);
      const u32x2_t plo = *reinterpret_cast<const u32x2_t*>(pr), phi = *reinterpret_cast<const u32x2_t*>(pr + 32);
      const u32x4_t pf = {plo.x, plo.y, phi.x, phi.y};
#pragma unroll
      for (int t = 0; t < RT; ++t) {
        const int tile = wave + 4 * t;
        if (16 * tile < a.rankp) {
          const uint32_t at = lds0 + (uint32_t)((32 * hf + 4 * g + (r >> 2)) * rb + 32 * tile + 8 * (r & 3));
          const u32x2_t lo = pf_read_tr(at), hi = pf_read_tr(at + (uint32_t)(16 * rb));
          u[t] = mfma16(u32x4_t{lo.x, lo.y, hi.x, hi.y}, pf, u[t]);
        }
      }
    }
    __syncthreads();
  }
  l = quad_sum(l);
  if (g == 0) ssum[wave][r] = l;
  __syncthreads();
  if (h0 + r >= a.heads) return;
  if (wave == 0 && g == 0)
    *reinterpret_cast<float4*>(head_out) = float4{m, (ssum[0][r] + ssum[1][r]) + (ssum[2][r] + ssum[3][r]), 0.f, 0.f};
#pragma unroll
  for (int t = 0; t < RT; ++t) {
    const int tile = wave + 4 * t;
    if (16 * tile < a.rankp) store4(head_out + 4 + 16 * tile + 4 * g, float4{u[t][0], u[t][1], u[t][2], u[t][3]});
  }
}

struct LatentExpand {
  const float* partial;     // [B, H, S, rankp + 4]
  const float* sink;        // [H] or null
  const float* gate;        // gate projections, [b * gate_ld + h], or null
  const uint16_t* uv;       // [H, vdimp, rankp]
  uint16_t* out;            // [B, out_ld], head h at column h * vdimp
  int batch, heads, chunks, rankp, vdimp, gate_ld, out_ld, groups;  // groups: workgroups per head (4 tiles each)
};
constexpr int kLatentMaxChunks = 32;
// Grid (H * groups, batch blocks).  Dynamic LDS: 16 x (rankp + 8) bf16 of merged sums.
__global__ __launch_bounds__(256) void latent_expand_kernel(LatentExpand a) {
  extern __shared__ __attribute__((aligned(16))) uint16_t merged[];
  __shared__ float weight[kGemvBatch][kLatentMaxChunks];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
  const int b0 = blockIdx.y * kGemvBatch, nb = min(kGemvBatch, a.batch - b0);
  const int h = blockIdx.x / a.groups, grp = blockIdx.x % a.groups;
  const int stride = a.rankp + 4, ld = a.rankp + 8;
  for (int b = wave; b < nb; b += 4) {  // a wave per sequence, a lane per chunk
    const float* src = a.partial + ((size_t)(b0 + b) * a.heads + h) * a.chunks * stride;
    const bool mine = lane < a.chunks;
    const float mx = mine ? src[lane * stride] : -INFINITY, sum = mine ? src[lane * stride + 1] : 0.f;
    const float sink2 = a.sink ? a.sink[h] * 1.4426950408889634f : -INFINITY;
    const float top = fmaxf(wave_max64(mx), sink2);
    const float w = mx == -INFINITY ? 0.f : exp2f(mx - top);
    const float total = wave_sum64(sum * w) + (a.sink ? exp2f(sink2 - top) : 0.f);
    if (mine) weight[b][lane] = w / total;
  }
  __syncthreads();
  const int quads = a.rankp >> 2;
  for (int i = threadIdx.x; i < nb * quads; i += 256) {
    const int b = i / quads, c = 4 * (i % quads);
    const float* src = a.partial + ((size_t)(b0 + b) * a.heads + h) * a.chunks * stride + 4 + c;
    float4 sum = float4{0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < a.chunks; ++s) {
      const float w = weight[b][s];
      if (w == 0.f) continue;  // an empty chunk left no sums
      const float4 v = load4(src + (size_t)s * stride);
      sum.x = fmaf(v.x, w, sum.x); sum.y = fmaf(v.y, w, sum.y); sum.z = fmaf(v.z, w, sum.z); sum.w = fmaf(v.w, w, sum.w);
    }
    store4(merged + b * ld + c, sum);
  }
  __syncthreads();
  const int tile = 4 * grp + wave;
  if (16 * tile >= a.vdimp) return;
  const uint16_t* wrow = a.uv + ((size_t)h * a.vdimp + 16 * tile + r) * a.rankp;
  const uint16_t* xr = merged + min(r, nb - 1) * ld + 8 * g;
  const f32x4_t acc = tile_steps(wrow, a.rankp, 0, (a.rankp + 31) >> 5, g, f32x4_t{0.f, 0.f, 0.f, 0.f}, [&](int s) {
    return r < nb ? *reinterpret_cast<const u32x4_t*>(xr + 32 * s) : u32x4_t{0u, 0u, 0u, 0u};
  });
  if (r >= nb) return;
  const float f = a.gate ? sigmoid_f32(a.gate[(size_t)(b0 + r) * a.gate_ld + h]) : 1.f;
  *reinterpret_cast<u32x2_t*>(a.out + (size_t)(b0 + r) * a.out_ld + (size_t)h * a.vdimp + 16 * tile + 4 * g) =
      u32x2_t{pack2_bf16(acc[0] * f, acc[1] * f), pack2_bf16(acc[2] * f, acc[3] * f)};
}

}  // namespace ajq
