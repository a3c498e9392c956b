// Grouped-query attention whose values are the projected keys: the row operators around it.  (The attention itself is
// latent_attention.h's: windowed_prefill_kernel / windowed_attention_kernel for prompts and any width, latent_decode_kernel
// for one token, to which a key/value head is a "sequence" and its query heads are the heads.)
//
// A cache row of one key/value head is (value | key), dimp columns each: the key as projected, and the same key normed and
// rotated.
#pragma once
#include "dense_gemv_kernels.h"

namespace ajq {

// cos and sin of position * half_turns[i] * pi for i < pairs, by the threads of a workgroup.  The product and its reduction
// to (-1, 1] half turns are double, so that any position has an angle that is exact to fp32.
__device__ __forceinline__ void angles(const double* __restrict__ half_turns, int pairs, int position, float* cosine, float* sine) {
  for (int i = threadIdx.x; i < pairs; i += blockDim.x) {
    const double a = (double)position * half_turns[i];
    sincospif((float)(a - 2.0 * rint(0.5 * a)), sine + i, cosine + i);
  }
}

struct KeyValueShape {
  int heads, groups, dim, dimp, rot;  // rot <= dim, the first dimensions of a head; component i pairs with i + rot / 2
  float eps;
};

// One head of a projection row, normed over dim and rotated, of any width and with any pairs, by a team of LPH lanes: four columns
// per lane and turn, through put(column, values); columns dim .. dimp are zero and stay so (the gain is zero there).
template <int LPH, typename Y, typename Put>
__device__ __forceinline__ void norm_rotate(const Y* __restrict__ src, const KeyValueShape& s, const float* __restrict__ gain,
                                            const float* cosine, const float* sine, int lane, Put&& put) {
  float ss = 0.f;
  for (int i = 4 * lane; i < s.dimp; i += 4 * LPH) {
    const float4 v = load4(src + i);
    ss += (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w);
  }
#pragma unroll
  for (int off = LPH / 2; off > 0; off >>= 1) ss += __shfl_xor(ss, off);
  const Divisor by(sqrtf(ss / (float)s.dim + s.eps));
  const int half = s.rot >> 1;
  auto one = [&](int i) { return by.divide(to_f32(src[i])) * gain[i]; };
  auto turned = [&](int i) {
    if (i >= s.rot) return one(i);
    if (i < half) return one(i) * cosine[i] - one(i + half) * sine[i];
    return one(i) * cosine[i - half] + one(i - half) * sine[i - half];
  };
  for (int i = 4 * lane; i < s.dimp; i += 4 * LPH) put(i, float4{turned(i), turned(i + 1), turned(i + 2), turned(i + 3)});
}

struct KeyValueSplit {
  const void* y;            // [M, ldy]: queries (heads x dimp), keys (groups x dimp), then whatever else
  int ldy;
  KeyValueShape s;
  const float *q_gain, *k_gain;  // [dimp]
  const double* half_turns; // [rot / 2]
  int start;                // position of the first token, or
  const long long* pos;     // device-side position (seq = 1): the row goes to its slot of a ring
  int seq, prior, cap, kept;
  void* q;                  // [M, heads, q_ld], the query from column q_at on, zeros ahead of it
  int q_ld, q_at;
  void* rows;               // row slot of (b, group) at b * rows_batch + group * rows_head + slot * 2 dimp
  long long rows_batch, rows_head;
};
// Grid (tokens, slices): the heads of a token are dealt to the teams of LPH lanes of its workgroups.  QUADS: four columns per lane
// hold a head, and its pairs too (dimp <= 4 LPH, half the rotated width a multiple of 4): a head is read once, the first one
// before the angles are known, every other one ahead of the arithmetic of the one before; gains and angles stay in registers.
template <typename Y, typename T, int LPH, bool QUADS>
__global__ __launch_bounds__(256) void key_value_split_kernel(KeyValueSplit a) {
  extern __shared__ __attribute__((aligned(16))) float trig[];
  constexpr int kTeams = 256 / LPH;
  const KeyValueShape s = a.s;
  const int m = blockIdx.x, b = m / a.seq, t = m % a.seq;
  const int half = s.rot >> 1, pitch = (half + 3) & ~3, all = s.heads + s.groups, stride = kTeams * gridDim.y;
  const int p = clamped_position(a.pos, a.start + t, 0x7FFFFFFF);
  const int slot = a.pos ? ring_slot(p, a.cap, a.kept) : a.prior + t;
  const int lane = threadIdx.x % LPH, first = kTeams * blockIdx.y + threadIdx.x / LPH;
  const Y* row = reinterpret_cast<const Y*>(a.y) + (size_t)m * a.ldy;
  auto query = [&](int n) { return reinterpret_cast<T*>(a.q) + ((size_t)m * s.heads + n) * a.q_ld; };
  auto key = [&](int n) {
    return reinterpret_cast<T*>(a.rows) + (size_t)b * a.rows_batch + (size_t)(n - s.heads) * a.rows_head + (size_t)slot * (2 * s.dimp);
  };
  if constexpr (QUADS) {
    const float4 zero = float4{0.f, 0.f, 0.f, 0.f};
    const int i = 4 * lane, o = i < half ? i + half : i - half, e = i < half ? i : o;
    const bool mine = i < s.dimp, pairs = mine && i < s.rot;
    auto read = [&](int n, float4& v, float4& w) {
      v = w = zero;
      if (n < all && mine) v = load4(row + n * s.dimp + i);
      if (n < all && pairs) w = load4(row + n * s.dimp + o);
    };
    float4 v, w, gq = zero, hq = zero, gk = zero, hk = zero, c = float4{1.f, 1.f, 1.f, 1.f}, d = zero;
    read(first, v, w);
    if (mine) { gq = load4(a.q_gain + i); gk = load4(a.k_gain + i); }
    if (pairs) { hq = load4(a.q_gain + o); hk = load4(a.k_gain + o); }
    angles(a.half_turns, half, p, trig, trig + pitch);
    __syncthreads();
    if (pairs) {
      c = load4(trig + e);
      d = load4(trig + pitch + e);
      if (i < half) d = float4{-d.x, -d.y, -d.z, -d.w};
    }
    for (int n = first; n < all; n += stride) {
      float4 nv, nw;
      read(n + stride, nv, nw);
      float ss = (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w);
#pragma unroll
      for (int off = LPH / 2; off > 0; off >>= 1) ss += __shfl_xor(ss, off);
      const Divisor by(sqrtf(ss / (float)s.dim + s.eps));
      const bool is_query = n < s.heads;
      const float4 g = is_query ? gq : gk, h = is_query ? hq : hk;
      const float4 out = float4{by.divide(v.x) * g.x * c.x + by.divide(w.x) * h.x * d.x, by.divide(v.y) * g.y * c.y + by.divide(w.y) * h.y * d.y,
                                by.divide(v.z) * g.z * c.z + by.divide(w.z) * h.z * d.z, by.divide(v.w) * g.w * c.w + by.divide(w.w) * h.w * d.w};
      if (is_query) {
        T* dst = query(n);
        for (int k = i; k < a.q_at; k += 4 * LPH) store4(dst + k, zero);
        if (mine) store4(dst + a.q_at + i, out);
      } else if (mine) {
        T* dst = key(n);
        store4(dst + i, v);
        store4(dst + s.dimp + i, out);
      }
      v = nv;
      w = nw;
    }
  } else {
    angles(a.half_turns, half, p, trig, trig + pitch);
    __syncthreads();
    for (int n = first; n < all; n += stride) {
      const Y* src = row + n * s.dimp;
      if (n < s.heads) {
        T* dst = query(n);
        for (int i = 4 * lane; i < a.q_at; i += 4 * LPH) store4(dst + i, float4{0.f, 0.f, 0.f, 0.f});
        norm_rotate<LPH>(src, s, a.q_gain, trig, trig + pitch, lane, [&](int i, float4 v) { store4(dst + a.q_at + i, v); });
      } else {
        T* dst = key(n);
        for (int i = 4 * lane; i < s.dimp; i += 4 * LPH) store4(dst + i, load4(src + i));
        norm_rotate<LPH>(src, s, a.k_gain, trig, trig + pitch, lane, [&](int i, float4 v) { store4(dst + s.dimp + i, v); });
      }
    }
  }
}

// Merge of latent_decode_kernel's row chunks (a sequence there is a (b, key/value head) here) and the output gate:
// out[b, head, c] = sigmoid(gate) * sum over chunks.  One workgroup per (b, head).
struct GroupMerge {
  const float* sums;        // as latent_decode_kernel leaves them, for batch * groups sequences of `share` heads
  const float2* heads_in;   // [B * groups, share, chunks]
  const float* gate;        // [b * gate_ld + head * dimp + c] before the sigmoid, or null
  uint16_t* out;            // [B, out_ld], head h at column h * dimp
  int groups, share, chunks, dimp, gate_ld, out_ld;
};
__global__ __launch_bounds__(256) void group_merge_kernel(GroupMerge a) {
  __shared__ float weight[kLatentMaxChunks];
  __shared__ float4 part[256];
  const int tid = threadIdx.x, lane = tid & 63, heads = a.groups * a.share;
  const int b = blockIdx.x / heads, head = blockIdx.x % heads, h = head % a.share;
  const int unit = b * a.groups + head / a.share;
  const int quads = a.dimp >> 2, split = max(1, min(256 / quads, a.chunks)), which = tid / quads;
  if (tid < 64) {  // a lane per chunk
    const bool mine = lane < a.chunks;
    const float2 ml = mine ? a.heads_in[((size_t)unit * a.share + h) * a.chunks + lane] : float2{-INFINITY, 0.f};
    const float top = wave_max64(ml.x);
    const float e = ml.x == -INFINITY ? 0.f : exp2f(ml.x - top);
    const float total = wave_sum64(ml.y * e);
    if (mine) weight[lane] = e / total;
  }
  __syncthreads();
  const int c = 4 * (tid % quads);
  float4 sum = float4{0.f, 0.f, 0.f, 0.f};
  if (which < split) {
    const float* src = a.sums + latent_sums_at(unit, h >> 4, 0, a.share, a.chunks, a.dimp) + 256 * (c >> 4) + 16 * (h & 15) + (c & 15);
    for (int s = which; s < a.chunks; s += split) {
      const float4 v = load4(src + (size_t)s * (16 * a.dimp));
      const float f = weight[s];
      sum.x = fmaf(v.x, f, sum.x); sum.y = fmaf(v.y, f, sum.y); sum.z = fmaf(v.z, f, sum.z); sum.w = fmaf(v.w, f, sum.w);
    }
  }
  part[tid] = sum;
  __syncthreads();
  if (which > 0) return;
  for (int o = 1; o < split; ++o) {
    const float4 v = part[tid + o * quads];
    sum.x += v.x; sum.y += v.y; sum.z += v.z; sum.w += v.w;
  }
  if (a.gate) {
    const float4 z = load4(a.gate + (size_t)b * a.gate_ld + (size_t)head * a.dimp + c);
    sum.x *= sigmoid_f32(z.x); sum.y *= sigmoid_f32(z.y); sum.z *= sigmoid_f32(z.z); sum.w *= sigmoid_f32(z.w);
  }
  store4(a.out + (size_t)b * a.out_ld + (size_t)head * a.dimp + c, sum);
}

}  // namespace ajq
