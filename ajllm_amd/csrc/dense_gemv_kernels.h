// Matrix-vector products of one decode step for dense bf16 weights [N, K] (row-major, N % 16 == 0, K % 8 == 0) on
// MFMA, up to 16 sequences per workgroup (grid.y deals larger batches), with what surrounds them folded in:
//
//   dense_in_kernel      two weight matrices that read the same fp32 residual row through norms of their own: the layer
//                        norm is the prologue (or bf16 rows a norm launch left); the first matrix's outputs are stored
//                        in fp32, the second's go through an activation: gated pairs (8 gate rows and their 8 up rows per
//                        16-row tile), or every row by itself
//   latent_absorb_kernel per-head products of the unrotated query with the transposed key expansion, so that attention
//                        can run on the latents; beside them the rotation of the query, and the new cache row (RMS norm of
//                        the latent, rotation of the shared key part)
//   latent_expand_kernel merge of the attention's row chunks (with the sink), per-head value expansion, output gate
//   dense_out_kernel     product with the residual add (and whatever the next layer run adds first) as epilogue
//   dense_out_streams_kernel  product whose epilogue mixes it into several residual streams and forms what the next sublayer reads
//
// A 16 x 16 output tile (16 weight rows, 16 batch columns) belongs to a wave, or to kWaves waves that split K and meet in
// LDS.  Lane l = 16 g + r loads 16 bytes of weight row r at k = 32 step + 8 g: four lanes cover 64 contiguous bytes of a
// row, two steps a cache line.
#pragma once
#include "dense_kernels.h"
#include "latent_attention.h"
#include "stream_kernels.h"

namespace ajq {

constexpr int kGemvBatch = 16;

// acc[n][t] += W[rows of row tile n, steps begin .. end) x_t; `wrow` points at this lane's row of the first tile (a tile is
// 16 K elements further), `x(t, step)` gives the B fragment of batch tile t (batch column r, k = 32 step + 8 g ..), both
// zero past K.  A weight fragment meets BT batch tiles, an activation fragment RT row tiles.
template <int RT, int BT, typename XFn>
__device__ __forceinline__ void tile_steps(const uint16_t* __restrict__ wrow, int K, int begin, int end, int g,
                                           f32x4_t (&acc)[RT][BT], XFn&& x) {
  constexpr int kUnroll = 8 / RT;
  const u32x4_t zero = {0u, 0u, 0u, 0u};
  for (int s0 = begin; s0 < end; s0 += kUnroll) {
    u32x4_t w[kUnroll][RT], v[kUnroll][BT];
#pragma unroll
    for (int i = 0; i < kUnroll; ++i) {
      const int k = 32 * (s0 + i) + 8 * g;
#pragma unroll
      for (int n = 0; n < RT; ++n) {
        w[i][n] = zero;
        if (s0 + i < end && k < K) w[i][n] = *reinterpret_cast<const u32x4_t*>(wrow + (size_t)n * 16 * K + k);
      }
    }
#pragma unroll
    for (int i = 0; i < kUnroll; ++i)
#pragma unroll
      for (int t = 0; t < BT; ++t) {
        v[i][t] = zero;
        if (s0 + i < end && 32 * (s0 + i) + 8 * g < K) v[i][t] = x(t, s0 + i);
      }
#pragma unroll
    for (int i = 0; i < kUnroll; ++i)
#pragma unroll
      for (int n = 0; n < RT; ++n)
#pragma unroll
        for (int t = 0; t < BT; ++t) acc[n][t] = mfma16(w[i][n], v[i][t], acc[n][t]);
  }
}

// the K range of one of kWaves waves, in pairs of steps (a cache line of a weight row stays with one wave)
__device__ __forceinline__ void wave_steps(int K, int wave, int waves, int& begin, int& end) {
  const int steps = (K + 31) >> 5;
  const int per = ((steps + waves - 1) / waves + 1) & ~1;
  begin = min(steps, wave * per);
  end = min(steps, begin + per);
}

// sum of the waves' tiles; tile (n, t) is valid in wave n BT + t
template <int kWaves, int RT, int BT>
__device__ __forceinline__ void meet(f32x4_t (&acc)[RT][BT], float* red, int wave, int lane) {
  if (kWaves == 1) return;
  static_assert(kWaves == 1 || RT * BT <= kWaves, "a wave per tile");
  float4* slot = reinterpret_cast<float4*>(red);
#pragma unroll
  for (int i = 0; i < RT * BT; ++i) {
    const f32x4_t& v = acc[i / BT][i % BT];
    if (wave != i) slot[(i * kWaves + wave) * 64 + lane] = float4{v[0], v[1], v[2], v[3]};
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < RT * BT; ++i) {
    if (wave != i) continue;
    f32x4_t& v = acc[i / BT][i % BT];
#pragma unroll
    for (int w = 0; w < kWaves; ++w) {
      if (w == i) continue;
      const float4 o = slot[(i * kWaves + w) * 64 + lane];
      v[0] += o.x; v[1] += o.y; v[2] += o.z; v[3] += o.w;
    }
  }
}

struct DenseIn {
  const float* x;           // [B, Dp] residual rows (norm prologue)
  const uint16_t* n1;       // or [B, Dp] bf16 rows already normed by gain 1 / gain 2
  const uint16_t* n2;
  const float* gain1;
  const float* gain2;
  const uint16_t* w1;       // [16 tiles1, Dp]
  const uint16_t* w2;       // [16 tiles2, Dp]; pairs: gate / up rows interleaved in blocks of 8
  float* y1;                // [B, 16 tiles1]
  uint16_t* gated;          // [B, gated_ld], column 8 * tile + j (pairs) or 16 * tile + j
  int batch, D, Dp, tiles1, tiles2, gated_ld, act, center, pairs;
  float eps;
};

// kNorm: the norm is formed here, for the rows of one batch block (dynamic LDS: rows x (Dp + 8) bf16).
// RT: row tiles per workgroup (grid.x counts workgroups of the first matrix, then of the second), BT: batch tiles.
template <int kWaves, bool kNorm, int RT, int BT>
__global__ __launch_bounds__(64 * kWaves) void dense_in_kernel(DenseIn a) {
  extern __shared__ __attribute__((aligned(16))) uint16_t normed[];
  __shared__ __attribute__((aligned(16))) float red[kWaves > 1 ? RT * BT * kWaves * 256 : 4];
  __shared__ float stat[kWaves];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
  const int b0 = blockIdx.y * kGemvBatch * BT, nb = min(kGemvBatch * BT, a.batch - b0);
  const int groups1 = (a.tiles1 + RT - 1) / RT;
  const bool second = (int)blockIdx.x >= groups1;
  const int tiles = second ? a.tiles2 : a.tiles1;
  // the last workgroup of an odd matrix overlaps its neighbour: the same rows give the same values twice
  const int tile0 = max(0, min(RT * (second ? (int)blockIdx.x - groups1 : (int)blockIdx.x), tiles - RT));
  const uint16_t* wrow = (second ? a.w2 : a.w1) + (size_t)(16 * tile0 + r) * a.Dp;
  int begin, end;
  wave_steps(a.Dp, wave, kWaves, begin, end);
  f32x4_t acc[RT][BT] = {};
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
    tile_steps<RT, BT>(wrow, a.Dp, begin, end, g, acc, [&](int t, int s) {
      const int row = 16 * t + r;
      return row < nb ? *reinterpret_cast<const u32x4_t*>(normed + row * stride + 8 * g + 32 * s) : u32x4_t{0u, 0u, 0u, 0u};
    });
  } else {
    const uint16_t* xr = (second ? a.n2 : a.n1) + (size_t)b0 * a.Dp + 8 * g;
    tile_steps<RT, BT>(wrow, a.Dp, begin, end, g, acc, [&](int t, int s) {
      const int row = 16 * t + r;
      return row < nb ? *reinterpret_cast<const u32x4_t*>(xr + (size_t)row * a.Dp + 32 * s) : u32x4_t{0u, 0u, 0u, 0u};
    });
  }
  meet<kWaves, RT, BT>(acc, red, wave, lane);
#pragma unroll
  for (int i = 0; i < RT * BT; ++i) {
    if (kWaves > 1 && wave != i) continue;
    const f32x4_t& sum = acc[i / BT][i % BT];
    const int row = 16 * (i % BT) + r, tile = tile0 + i / BT;
    if (!second) {
      if (row < nb) store4(a.y1 + (size_t)(b0 + row) * (16 * a.tiles1) + 16 * tile + 4 * g, float4{sum[0], sum[1], sum[2], sum[3]});
      continue;
    }
    if (!a.pairs) {
      if (row < nb)
        store4(a.gated + (size_t)(b0 + row) * a.gated_ld + 16 * tile + 4 * g,
               float4{activate(a.act, sum[0]), activate(a.act, sum[1]), activate(a.act, sum[2]), activate(a.act, sum[3])});
      continue;
    }
    // rows 0 .. 7 of the tile (lanes g < 2) are gates, rows 8 .. 15 (lanes g >= 2, 32 lanes on) the matching up rows
    float v[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = activate(a.act, sum[e]) * __shfl_xor(sum[e], 32);
    if (g < 2 && row < nb) store4(a.gated + (size_t)(b0 + row) * a.gated_ld + 8 * tile + 4 * g, float4{v[0], v[1], v[2], v[3]});
  }
}

struct DenseOut {
  const uint16_t* in;       // [B, K]
  const uint16_t* w;        // [Dp, K]
  float* x;                 // [B, Dp], updated in place
  const float* again;       // [B, Dp] or null, added too
  const float* step;        // [Dp] or null, added too
  int batch, K, Dp;
};
template <int kWaves, int RT, int BT>
__global__ __launch_bounds__(64 * kWaves) void dense_out_kernel(DenseOut a) {
  __shared__ __attribute__((aligned(16))) float red[kWaves > 1 ? RT * BT * kWaves * 256 : 4];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
  const int b0 = blockIdx.y * kGemvBatch * BT, nb = min(kGemvBatch * BT, a.batch - b0);
  const int first = blockIdx.x * RT * 16;  // (RT divides the row tiles: x is updated in place)
  const uint16_t* wrow = a.w + (size_t)(first + r) * a.K;
  const uint16_t* xr = a.in + (size_t)b0 * a.K + 8 * g;
  int begin, end;
  wave_steps(a.K, wave, kWaves, begin, end);
  // what the product of tile i = (row tile, batch tile) is added to, requested ahead of it by the wave that will write it
  auto place = [&](int i) { return (size_t)(b0 + min(16 * (i % BT) + r, nb - 1)) * a.Dp + first + 16 * (i / BT) + 4 * g; };
  float4 old[kWaves > 1 ? 1 : RT * BT];
#pragma unroll
  for (int i = 0; i < RT * BT; ++i) {
    if (kWaves > 1 && wave != i) continue;
    float4 v = load4(a.x + place(i));
    if (a.again) {
      const float4 e = load4(a.again + place(i));
      v.x += e.x; v.y += e.y; v.z += e.z; v.w += e.w;
    }
    if (a.step) {
      const float4 e = load4(a.step + first + 16 * (i / BT) + 4 * g);
      v.x += e.x; v.y += e.y; v.z += e.z; v.w += e.w;
    }
    old[kWaves > 1 ? 0 : i] = v;
  }
  f32x4_t acc[RT][BT] = {};
  tile_steps<RT, BT>(wrow, a.K, begin, end, g, acc, [&](int t, int s) {
    const int row = 16 * t + r;
    return row < nb ? *reinterpret_cast<const u32x4_t*>(xr + (size_t)row * a.K + 32 * s) : u32x4_t{0u, 0u, 0u, 0u};
  });
  meet<kWaves, RT, BT>(acc, red, wave, lane);
#pragma unroll
  for (int i = 0; i < RT * BT; ++i) {
    if ((kWaves > 1 && wave != i) || 16 * (i % BT) + r >= nb) continue;
    const float4 v = old[kWaves > 1 ? 0 : i];
    const f32x4_t& sum = acc[i / BT][i % BT];
    store4(a.x + place(i), float4{v.x + sum[0], v.y + sum[1], v.z + sum[2], v.w + sum[3]});
  }
}

struct DenseOutStreams {
  const uint16_t* in;       // [B, K]
  const uint16_t* w;        // [Dp, K]
  float* x;                 // [B, S, Dp], updated in place
  const float* scale;       // [Dp], a factor per column of the product
  const float* out;         // [S]
  const float* mix;         // [S, S]
  const float* next;        // [S], weights of the next reader; null: the plain sum
  float* u;                 // [B, Dp], what the next reader gets
  int batch, K, Dp, streams;
};
template <int kWaves, int RT, int BT, int MAXS>
__global__ __launch_bounds__(64 * kWaves) void dense_out_streams_kernel(DenseOutStreams a) {
  __shared__ __attribute__((aligned(16))) float red[kWaves > 1 ? RT * BT * kWaves * 256 : 4];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
  const int b0 = blockIdx.y * kGemvBatch * BT, nb = min(kGemvBatch * BT, a.batch - b0);
  const int first = blockIdx.x * RT * 16;
  const uint16_t* wrow = a.w + (size_t)(first + r) * a.K;
  const uint16_t* xr = a.in + (size_t)b0 * a.K + 8 * g;
  int begin, end;
  wave_steps(a.K, wave, kWaves, begin, end);
  // the streams at this lane's place of tile i = (row tile, batch tile); with several waves each writes one tile and
  // requests its streams ahead of the product
  auto fetch = [&](int i, float4 (&v)[MAXS]) {
    const float* x = a.x + (size_t)(b0 + min(16 * (i % BT) + r, nb - 1)) * a.streams * a.Dp + first + 16 * (i / BT) + 4 * g;
#pragma unroll
    for (int s = 0; s < MAXS; ++s)
      if (s < a.streams) v[s] = load4(x + (size_t)s * a.Dp);
  };
  float4 v[MAXS];
  if (kWaves > 1 && wave < RT * BT) fetch(wave, v);
  f32x4_t acc[RT][BT] = {};
  tile_steps<RT, BT>(wrow, a.K, begin, end, g, acc, [&](int t, int s) {
    const int row = 16 * t + r;
    return row < nb ? *reinterpret_cast<const u32x4_t*>(xr + (size_t)row * a.K + 32 * s) : u32x4_t{0u, 0u, 0u, 0u};
  });
  meet<kWaves, RT, BT>(acc, red, wave, lane);
#pragma unroll
  for (int i = 0; i < RT * BT; ++i) {
    const int row = 16 * (i % BT) + r, column = first + 16 * (i / BT) + 4 * g;
    if ((kWaves > 1 && wave != i) || row >= nb) continue;
    if (kWaves == 1) fetch(i, v);
    const f32x4_t& sum = acc[i / BT][i % BT];
    const float4 f = load4(a.scale + column);
    mix_streams<MAXS>(v, a.streams, a.out, a.mix, float4{sum[0] * f.x, sum[1] * f.y, sum[2] * f.z, sum[3] * f.w});
    float* x = a.x + (size_t)(b0 + row) * a.streams * a.Dp + column;
#pragma unroll
    for (int s = 0; s < MAXS; ++s)
      if (s < a.streams) store4(x + (size_t)s * a.Dp, v[s]);
    store4(a.u + (size_t)(b0 + row) * a.Dp + column, read_streams<MAXS>(v, a.streams, a.next));
  }
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
// Grid (H * groups + 4, batch blocks); the last four workgroups of a batch block make the cache rows, a wave each.
__global__ __launch_bounds__(256) void latent_absorb_kernel(LatentAbsorb a) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
  const int b0 = blockIdx.y * kGemvBatch, nb = min(kGemvBatch, a.batch - b0);
  const LatentShape s = a.s;
  const int dq = s.dimp + s.rotp, width = s.rankp + s.rotp;
  const int p = clamped_position(a.pos, 0, a.table_rows);
  const float* cs = a.cosine + (size_t)p * (s.rot >> 1);
  const float* sn = a.sine + (size_t)p * (s.rot >> 1);
  if ((int)blockIdx.x >= s.heads * a.groups) {
    const int b = 4 * ((int)blockIdx.x - s.heads * a.groups) + wave;
    if (b < nb) {
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
  f32x4_t acc[1][1] = {};
  tile_steps<1, 1>(wrow, s.dimp, 0, (s.dimp + 31) >> 5, g, acc, [&](int, int st) {
    if (r >= nb) return u32x4_t{0u, 0u, 0u, 0u};
    const float4 u = load4(xr + 32 * st), v = load4(xr + 32 * st + 4);
    return u32x4_t{pack2_bf16(u.x, u.y), pack2_bf16(u.z, u.w), pack2_bf16(v.x, v.y), pack2_bf16(v.z, v.w)};
  });
  if (r < nb)
    store4(a.q + ((size_t)(b0 + r) * s.heads + h) * width + 16 * tile + 4 * g,
           float4{acc[0][0][0], acc[0][0][1], acc[0][0][2], acc[0][0][3]});
}

// One chunk of cache rows against 16 HT heads of one sequence, in the latent space: row j of the ring
// (latent rankp | rotated rotp) is the key, its latent part the value, for every head, so a row is fetched once for all of
// the workgroup's heads and both products.  Four waves per head tile; blocks of 64 rows go into LDS by DMA, one block ahead.
//   S^T = K Q^T:    wave w takes keys 16 (w & 3) .. of the block; KS column steps, its head tile's queries in registers
//   U^T += C^T P^T: wave w takes every fourth 16-column tile of the latent (RT of them), latents by transposing LDS reads
// LDS holds the rows in panels of 128 bytes (64 rows x 8 chunks): chunk c of row k in slot c ^ (k & 6 | k >> 3 & 1), so that
// sixteen rows of one chunk and eight rows of one 32-byte segment (whose two chunks stay neighbours) meet every bank once.
// Partial result of (b, h, chunk): maximum and denominator (base-2 exponents) in `heads_out`, and rankp sums in `sums`, which
// holds [b][head tile][chunk][16-column tile][16 heads][16 columns] so that a wave stores whole lines; zeros for an empty chunk.
// Grid: chunks of sequences x head groups; the groups of a chunk are 8 workgroups apart, on one XCD and its L2.
struct LatentDecode {
  const uint16_t* q;        // [B, H, width]
  const uint16_t* ring;     // [B, cap, width]
  const long long* pos;
  float* sums;
  float2* heads_out;        // [B, H, S]
  int batch, heads, rankp, width, cap, chunks;
  int key_step;             // 32-column steps ahead of it meet zero query columns and are left out of the scores
  float scale2;
};
__host__ __device__ constexpr long long latent_sums_at(int b, int tile, int chunk, int heads, int chunks, int rankp) {
  return (((long long)b * ((heads + 15) / 16) + tile) * chunks + chunk) * 16 * rankp;
}
constexpr int kLatentRows = 64;
constexpr int kLatentPBytes = (kLatentRows + 8) * 2;
constexpr int latent_decode_lds(int ks, int ht) { return ks * 8192 + ht * 16 * kLatentPBytes; }  // two stages of ks / 2 panels
template <int KS, int RT, int HT>
__global__ __launch_bounds__(256 * HT) void latent_decode_kernel(LatentDecode a) {
  constexpr int NP = KS / 2, kPanel = kLatentRows * 128, kStage = NP * kPanel, kWaves = 4 * HT;
  static_assert(KS % 2 == 0, "whole panels");
  extern __shared__ __attribute__((aligned(1024))) unsigned char lds[];
  __shared__ float smax[HT][4][16], ssum[HT][4][16];
  const uint32_t lds0 = (uint32_t)(uintptr_t)(pf_lds_char_t*)lds;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), r = lane & 15, g = lane >> 4;
  const int part = wave & 3, ht = wave >> 2;
  const int groups = (a.heads + 16 * HT - 1) / (16 * HT), units = a.batch * a.chunks;
  int unit, group;
  if ((units & 7) == 0) {
    const int m = (int)(blockIdx.x >> 3);
    group = m % groups;
    unit = 8 * (m / groups) + (int)(blockIdx.x & 7);
  } else {
    group = (int)blockIdx.x % groups;
    unit = (int)blockIdx.x / groups;
  }
  const int b = unit / a.chunks, chunk = unit % a.chunks, h0 = 16 * (HT * group + ht);
  const int cw = a.width >> 3;
  u32x4_t qf[KS];  // requested before the position is known
  const uint16_t* qsrc = a.q + ((size_t)b * a.heads + min(h0 + r, a.heads - 1)) * a.width + 8 * g;
#pragma unroll
  for (int s = 0; s < KS; ++s) {
    qf[s] = u32x4_t{0u, 0u, 0u, 0u};
    if (4 * s + g < cw) qf[s] = *reinterpret_cast<const u32x4_t*>(qsrc + 32 * s);
  }
  const int valid = (int)min(max(*a.pos, 0ll), (long long)a.cap - 1) + 1;  // rows the ring holds
  const int per = (((valid + a.chunks - 1) / a.chunks) + kLatentRows - 1) & ~(kLatentRows - 1);
  const int begin = chunk * per, end = min(valid, begin + per);
  float m = -INFINITY, l = 0.f;
  f32x4_t u[RT] = {};
  if (begin < end) {
    const char* ring = reinterpret_cast<const char*>(a.ring + (size_t)b * a.cap * a.width);
    // a request fills 8 rows of a panel: this lane row lane / 8, slot lane % 8.  Rows past the end repeat the last one (those
    // keys are masked), chunks past the width the last one (they meet zero query columns).
    const int chunk_of = (lane & 7) ^ (((lane >> 3) & 6) | (wave & 1));  // (a wave's requests all start at rows of one parity of 8)
    auto fetch = [&](int j0) {
      const uint32_t to = lds0 + (uint32_t)((((j0 - begin) / kLatentRows) & 1) * kStage);
#pragma unroll
      for (int i = 0; i < (8 * NP + kWaves - 1) / kWaves; ++i) {
        const int req = wave + kWaves * i;  // panel req / 8, rows 8 (req % 8) ..
        if ((8 * NP) % kWaves != 0 && req >= 8 * NP) continue;
        const uint32_t row = (uint32_t)min(j0 + 8 * (req & 7) + (lane >> 3), end - 1);
        const uint32_t c = (uint32_t)min(8 * (req >> 3) + chunk_of, cw - 1);
        dma16_gather(ring + (size_t)row * (uint32_t)(2 * a.width) + 16u * c, to + (uint32_t)(req * 1024));
      }
    };
    fetch(begin);
    // keys: row 16 part + r, chunk 4 (s & 1) + g of panel s / 2
    const uint32_t k_rd[2] = {lds0 + (uint32_t)((16 * part + r) * 128 + 16 * (g ^ (r & 6 | r >> 3))),
                              lds0 + (uint32_t)((16 * part + r) * 128 + 16 * ((4 + g) ^ (r & 6 | r >> 3)))};
    // latents: this lane addresses 8 bytes (piece r & 3) of row 4 g + (r >> 2); tile part + 4 t is segment part of panel t
    const int vrow = 4 * g + (r >> 2);
    const uint32_t v_rd = lds0 + (uint32_t)(vrow * 128 + 16 * ((2 * part | (r & 3) >> 1) ^ (vrow & 6 | vrow >> 3)) + 8 * (r & 1));
    unsigned char* p_lds = lds + 2 * kStage + ht * 16 * kLatentPBytes + r * kLatentPBytes;
    for (int j0 = begin; j0 < end; j0 += kLatentRows) {
      // this block has landed; every wave is done with the one before, whose stage the next block goes to
      asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
      __syncthreads();
      if (j0 + kLatentRows < end) fetch(j0 + kLatentRows);
      const uint32_t stage = (uint32_t)((((j0 - begin) / kLatentRows) & 1) * kStage);
      f32x4_t sc[2] = {};
#pragma unroll
      for (int s = 0; s < KS; ++s)
        if (s >= a.key_step) sc[s & 1] = mfma16(pf_read128(k_rd[s & 1] + stage + (uint32_t)((s >> 1) * kPanel)), qf[s], sc[s & 1]);
      // score i: key j0 + 16 part + 4 g + i, head h0 + r
      float p[4], mx = -INFINITY;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        p[i] = j0 + 16 * part + 4 * g + i < end ? (sc[0][i] + sc[1][i]) * a.scale2 : -INFINITY;
        mx = fmaxf(mx, p[i]);
      }
      mx = quad_max(mx);
      if (g == 0) smax[ht][part][r] = mx;
      __syncthreads();
      // (finite: the block's first row is valid)
      const float m_new = fmaxf(fmaxf(fmaxf(smax[ht][0][r], smax[ht][1][r]), fmaxf(smax[ht][2][r], smax[ht][3][r])), m);
      const float corr = __builtin_amdgcn_exp2f(m - m_new);
      m = m_new;
#pragma unroll
      for (int i = 0; i < 4; ++i) p[i] = __builtin_amdgcn_exp2f(p[i] - m);
      l = l * corr + ((p[0] + p[1]) + (p[2] + p[3]));
      store4(reinterpret_cast<uint16_t*>(p_lds) + 16 * part + 4 * g, float4{p[0], p[1], p[2], p[3]});
#pragma unroll
      for (int t = 0; t < RT; ++t) u[t] *= corr;
      __syncthreads();
#pragma unroll
      for (int hf = 0; hf < 2; ++hf) {
        const unsigned char* pr = p_lds + 2 * (32 * hf + 4 * g);
        const u32x2_t plo = *reinterpret_cast<const u32x2_t*>(pr), phi = *reinterpret_cast<const u32x2_t*>(pr + 32);
        const u32x4_t pf = {plo.x, plo.y, phi.x, phi.y};
        const uint32_t at = v_rd + stage + (uint32_t)(hf * 4096);
        // (panels past the latent hold the rotated part, or nothing of this block: their sums are not written)
        u32x2_t lo[RT], hi[RT];
#pragma unroll
        for (int t = 0; t < RT; ++t) {
          lo[t] = pf_read_tr(at + (uint32_t)(t * kPanel));
          hi[t] = pf_read_tr(at + (uint32_t)(t * kPanel + 2048));
        }
#pragma unroll
        for (int t = 0; t < RT; ++t) u[t] = mfma16(u32x4_t{lo[t].x, lo[t].y, hi[t].x, hi[t].y}, pf, u[t]);
      }
    }
    l = quad_sum(l);
    if (g == 0) ssum[ht][part][r] = l;
    __syncthreads();
    l = (ssum[ht][0][r] + ssum[ht][1][r]) + (ssum[ht][2][r] + ssum[ht][3][r]);
  }
  if (h0 >= a.heads) return;
  if (part == 0 && g == 0 && h0 + r < a.heads) a.heads_out[((size_t)b * a.heads + h0 + r) * a.chunks + chunk] = float2{m, l};
  float* out = a.sums + latent_sums_at(b, h0 >> 4, chunk, a.heads, a.chunks, a.rankp) + 16 * r + 4 * g;
#pragma unroll
  for (int t = 0; t < RT; ++t) {
    const int tile = part + 4 * t;
    if (16 * tile < a.rankp) store4(out + 256 * tile, float4{u[t][0], u[t][1], u[t][2], u[t][3]});
  }
}

struct LatentExpand {
  const float* sums;        // as latent_decode_kernel leaves them
  const float2* heads_in;   // [B, H, S]
  const float* sink;        // [H] or null
  const float* gate;        // gate projections, [b * gate_ld + h], or null
  const uint16_t* uv;       // [H, vdimp, rankp]
  uint16_t* out;            // [B, out_ld], head h at column h * vdimp
  int batch, heads, chunks, rankp, vdimp, gate_ld, out_ld, groups;  // groups: workgroups per head
};
constexpr int kLatentMaxChunks = 32, kExpandBatch = 4, kExpandRank = 512;
// A workgroup of 8 waves per (head, TW 16-column tiles of values, 4 sequences): the chunks are merged by all threads, then
// 8 / TW waves per tile expand the merged latents, a part of them each; their weights are requested first.  One CU takes in
// some 40 KB per microsecond: for few sequences a head's weights (128 KB at 512 x 128) want several workgroups (TW = 2),
// for more the merge, which every workgroup of a head repeats, wants few (TW = 8).  Grid (H * groups, batch blocks).
template <int TW>
__global__ __launch_bounds__(512) void latent_expand_kernel(LatentExpand a) {
  constexpr int kParts = 8 / TW, kSteps = kExpandRank / 32 / kParts;
  extern __shared__ __attribute__((aligned(16))) uint16_t merged[];   // [kExpandBatch][rankp + 8] bf16
  __shared__ float weight[kExpandBatch][kLatentMaxChunks];
  __shared__ float4 part[512];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 15, g = lane >> 4;
  const int b0 = blockIdx.y * kExpandBatch, nb = min(kExpandBatch, a.batch - b0);
  const int h = blockIdx.x / a.groups, tile = TW * (blockIdx.x % a.groups) + wave / kParts;
  const int ld = a.rankp + 8;
  const u32x4_t zero = {0u, 0u, 0u, 0u};
  const bool active = 16 * tile < a.vdimp;
  const int k0 = 32 * kSteps * (wave % kParts) + 8 * g;
  u32x4_t w[kSteps];
  const uint16_t* wrow = a.uv + ((size_t)h * a.vdimp + (active ? 16 * tile : 0) + r) * a.rankp;
#pragma unroll
  for (int s = 0; s < kSteps; ++s) {
    w[s] = zero;
    if (active && k0 + 32 * s < a.rankp) w[s] = *reinterpret_cast<const u32x4_t*>(wrow + k0 + 32 * s);
  }
  // merged[b] = sum over chunks; the threads of a column quad split the chunks where there are more threads than quads.
  // The first chunks' sums are requested before the chunks' weights are known.
  const int quads = a.rankp >> 2, items = nb * quads;
  const int split = items <= 128 ? 4 : items <= 256 ? 2 : 1, span = 512 / split;
  const int which = tid / span;
  constexpr int kAhead = 8;
  float4 ahead[kAhead];
  auto request = [&](int i, int s0) {
    const int b = min(i / quads, nb - 1), c = 4 * (i % quads);
    const float* src = a.sums + latent_sums_at(b0 + b, h >> 4, 0, a.heads, a.chunks, a.rankp) + 256 * (c >> 4) + 16 * (h & 15) + (c & 15);
#pragma unroll
    for (int k = 0; k < kAhead; ++k) ahead[k] = load4(src + (size_t)min(s0 + k * split, a.chunks - 1) * (16 * a.rankp));
  };
  request(tid % span, which);
  if (wave < nb) {  // a wave per sequence, a lane per chunk
    const bool mine = lane < a.chunks;
    const float2 ml = mine ? a.heads_in[((size_t)(b0 + wave) * a.heads + h) * a.chunks + lane] : float2{-INFINITY, 0.f};
    const float mx = ml.x, sum = ml.y;
    const float sink2 = a.sink ? a.sink[h] * kLog2eF : -INFINITY;
    const float top = fmaxf(wave_max64(mx), sink2);
    const float e = mx == -INFINITY ? 0.f : exp2f(mx - top);
    const float total = wave_sum64(sum * e) + (a.sink ? exp2f(sink2 - top) : 0.f);
    if (lane < kLatentMaxChunks) weight[wave][lane] = mine ? e / total : 0.f;
  }
  __syncthreads();
  for (int i0 = 0; i0 < items; i0 += span) {
    const int i = i0 + tid % span, b = min(i / quads, nb - 1);
    float4 sum = float4{0.f, 0.f, 0.f, 0.f};
    for (int s0 = which; s0 < a.chunks; s0 += kAhead * split) {
      if (i0 > 0 || s0 > which) request(i, s0);
#pragma unroll
      for (int k = 0; k < kAhead; ++k) {
        const int s = s0 + k * split;
        const float f = s < a.chunks ? weight[b][s] : 0.f;
        const float4 v = ahead[k];
        sum.x = fmaf(v.x, f, sum.x); sum.y = fmaf(v.y, f, sum.y); sum.z = fmaf(v.z, f, sum.z); sum.w = fmaf(v.w, f, sum.w);
      }
    }
    if (split > 1) {  // (one round: items <= span)
      part[tid] = sum;
      __syncthreads();
      for (int o = 1; o < split; ++o) {
        const float4 v = part[(tid + o * span) & 511];
        sum.x += v.x; sum.y += v.y; sum.z += v.z; sum.w += v.w;
      }
    }
    if (which == 0 && i < items) store4(merged + b * ld + 4 * (i % quads), sum);
  }
  __syncthreads();
  f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int s = 0; s < kSteps; ++s) {
    u32x4_t v = zero;
    if (r < nb && k0 + 32 * s < a.rankp) v = *reinterpret_cast<const u32x4_t*>(merged + r * ld + k0 + 32 * s);
    acc = mfma16(w[s], v, acc);
  }
  if (kParts > 1) {
    part[tid] = float4{acc[0], acc[1], acc[2], acc[3]};  // (last read before the barrier above)
    __syncthreads();
  }
  if (wave % kParts != 0 || !active) return;
#pragma unroll
  for (int q = 1; q < kParts; ++q) {
    const float4 v = part[tid + 64 * q];
    acc[0] += v.x; acc[1] += v.y; acc[2] += v.z; acc[3] += v.w;
  }
  if (r >= nb) return;
  const float f = a.gate ? sigmoid_f32(a.gate[(size_t)(b0 + r) * a.gate_ld + h]) : 1.f;
  store4(a.out + (size_t)(b0 + r) * a.out_ld + (size_t)h * a.vdimp + 16 * tile + 4 * g,
         float4{acc[0] * f, acc[1] * f, acc[2] * f, acc[3] * f});
}

}  // namespace ajq
