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

// One head of a projection row, normed over dim and rotated, by a team of LPH lanes: four columns per lane and turn, through
// put(column, values); columns dim .. dimp are zero and stay so (the gain is zero there).
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
  const bool quads = (half & 3) == 0;
  auto one = [&](int i) { return by.divide(to_f32(src[i])) * gain[i]; };
  auto turned = [&](int i) {
    if (i >= s.rot) return one(i);
    if (i < half) return one(i) * cosine[i] - one(i + half) * sine[i];
    return one(i) * cosine[i - half] + one(i - half) * sine[i - half];
  };
  for (int i = 4 * lane; i < s.dimp; i += 4 * LPH) {
    if (i < s.rot && !quads) {  // a pair may straddle four columns
      put(i, float4{turned(i), turned(i + 1), turned(i + 2), turned(i + 3)});
      continue;
    }
    const float4 v = load4(src + i), g = load4(gain + i);
    float4 a = float4{by.divide(v.x) * g.x, by.divide(v.y) * g.y, by.divide(v.z) * g.z, by.divide(v.w) * g.w};
    if (i < s.rot) {
      const bool first = i < half;
      const int o = first ? i + half : i - half, e = first ? i : o;
      const float4 w = load4(src + o), h = load4(gain + o), c = load4(cosine + e);
      float4 n = load4(sine + e);
      if (first) n = float4{-n.x, -n.y, -n.z, -n.w};
      a = float4{a.x * c.x + by.divide(w.x) * h.x * n.x, a.y * c.y + by.divide(w.y) * h.y * n.y,
                 a.z * c.z + by.divide(w.z) * h.z * n.z, a.w * c.w + by.divide(w.w) * h.w * n.w};
    }
    put(i, a);
  }
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
// One workgroup per token; a team of LPH lanes per head.
template <typename Y, typename T, int LPH>
__global__ __launch_bounds__(256) void key_value_split_kernel(KeyValueSplit a) {
  extern __shared__ __attribute__((aligned(16))) float trig[];
  const KeyValueShape s = a.s;
  const int m = blockIdx.x, b = m / a.seq, t = m % a.seq;
  const int half = s.rot >> 1, pitch = (half + 3) & ~3;
  const int p = clamped_position(a.pos, a.start + t, 0x7FFFFFFF);
  const int slot = a.pos ? ring_slot(p, a.cap, a.kept) : a.prior + t;
  angles(a.half_turns, half, p, trig, trig + pitch);
  __syncthreads();
  const int lane = threadIdx.x % LPH;
  const Y* row = reinterpret_cast<const Y*>(a.y) + (size_t)m * a.ldy;
  for (int n = threadIdx.x / LPH; n < s.heads + s.groups; n += 256 / LPH) {
    const Y* src = row + n * s.dimp;
    if (n < s.heads) {
      T* dst = reinterpret_cast<T*>(a.q) + ((size_t)m * s.heads + n) * a.q_ld;
      for (int i = 4 * lane; i < a.q_at; i += 4 * LPH) store4(dst + i, float4{0.f, 0.f, 0.f, 0.f});
      norm_rotate<LPH>(src, s, a.q_gain, trig, trig + pitch, lane, [&](int i, float4 v) { store4(dst + a.q_at + i, v); });
    } else {
      T* dst = reinterpret_cast<T*>(a.rows) + (size_t)b * a.rows_batch + (size_t)(n - s.heads) * a.rows_head + (size_t)slot * (2 * s.dimp);
      for (int i = 4 * lane; i < s.dimp; i += 4 * LPH) store4(dst + i, load4(src + i));
      norm_rotate<LPH>(src, s, a.k_gain, trig, trig + pitch, lane, [&](int i, float4 v) { store4(dst + s.dimp + i, v); });
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
