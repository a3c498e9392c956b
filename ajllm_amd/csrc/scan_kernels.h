// Selective scan (a diagonal linear recurrence per channel whose decay, input and output weights depend on the token):
//
//   x   = silu(conv(x))                               causal, per channel, `taps` wide
//   S  <- exp(dt A) S + (dt x) B,   y = S C + D x     S [channels, states] fp32, dt = softplus(raw + bias) per channel
//   out = y silu(z)
//
// Prompts (any number of tokens, from any position; also one token on any operand type):
//   conv_silu_kernel, conv_silu_run_kernel (prompts with usual widths), scan_kernel
// One token in bf16:
//   scan_project_kernel, scan_step_kernel
//
// States and a2 = A log2(e) (decays are taken in base 2) are stored in planes of four: [states / 4][channels][4], so that threads
// of neighbouring channels load whole lines; `states` is a multiple of 4 (states past a model's own are zero).
//
// Whatever the operand type: convolution sums, dt and its softplus, decays, states and y are fp32.  A
// sequence's first token (position 0) starts from zeros whatever the buffers hold.
#pragma once
#include "dense_gemv_kernels.h"

namespace ajq {

__device__ __forceinline__ float silu_f32(float z) { return z * sigmoid_f32(z); }
// For operands in bf16: the hardware's exponential and reciprocal (one ulp each; the argument's rounding makes it |z| ulps).
template <typename T>
__device__ __forceinline__ float silu_for(float z) {
  if (sizeof(T) == 4) return silu_f32(z);
  return z * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z));
}
// max(z, 0) + log(1 + e) with e = exp(-|z|), the exponential in base 2 with the part of its exponent that the product rounded
// away.  1 + e is rounded to u, which log(u) e / (u - 1) makes good (u - 1 is exact).  No branch.
__device__ __forceinline__ float softplus_f32(float z) {
  constexpr float kLog2e = 1.4426950408889634f, kLn2 = 0.6931471805599453f;
  const float x = -fminf(fabsf(z), 100.f), h = x * kLog2e, rest = fmaf(x, kLog2e, -h);
  const float e0 = __builtin_amdgcn_exp2f(h), e = fmaf(e0, rest * kLn2, e0), u = 1.0f + e, d = u - 1.0f;
  const float l = kLn2 * __builtin_amdgcn_logf(u) * (e * __builtin_amdgcn_rcpf(d == 0.f ? 1.f : d));
  return fmaxf(z, 0.f) + (d == 0.f ? e : l);
}

struct ConvSilu {
  const void* y;            // [B * seq, ldy], the convolved columns first
  int ldy;
  void* ring;               // [B, taps - 1, inner]: position p in slot p % (taps - 1); null: the sequence starts here
  const float* weight;      // [taps, inner], the last row meets the token itself
  const float* bias;        // [inner]
  int start;
  const long long* pos;     // device-side position (seq = 1): the token's own column goes into the ring as well
  int rows, seq, inner, taps;
  void* out;                // [B * seq, inner]
};
// A thread makes 8 channels of one token.
template <typename T>
__global__ __launch_bounds__(256) void conv_silu_kernel(ConvSilu a) {
  const int vectors = a.inner >> 3;
  const long long idx = (long long)blockIdx.x * 256 + threadIdx.x;
  if (idx >= (long long)a.rows * vectors) return;
  const int m = (int)(idx / vectors), c = 8 * (int)(idx % vectors), b = m / a.seq, t = m % a.seq, reach = a.taps - 1;
  const int p = clamped_position(a.pos, a.start + t, 0x7FFFFFFF);
  const T* y = reinterpret_cast<const T*>(a.y) + (size_t)m * a.ldy + c;
  T* ring = reinterpret_cast<T*>(a.ring) + (size_t)b * reach * a.inner + c;
  Float8 sum = load8(a.bias + c);
  const Float8 own = load8(y);
  for (int j = min(reach, p); j >= 0; --j) {
    const Float8 w = load8(a.weight + (size_t)(reach - j) * a.inner + c);
    Float8 v = own;
    if (j > t) v = load8(ring + (size_t)((p - j) % reach) * a.inner);
    else if (j > 0) v = load8(y - (size_t)j * a.ldy);
#pragma unroll
    for (int e = 0; e < 8; ++e) sum.v[e] = fmaf(w.v[e], v.v[e], sum.v[e]);
  }
  if (a.pos && reach > 0) store8(ring + (size_t)(p % reach) * a.inner, own);
#pragma unroll
  for (int e = 0; e < 8; ++e) sum.v[e] = silu_for<T>(sum.v[e]);
  store8(reinterpret_cast<T*>(a.out) + (size_t)m * a.inner + c, sum);
}

// The same for prompts (no device-side position): a thread makes 8 channels of kConvTokens tokens, its weights and the last
// TAPS - 1 rows in registers.
constexpr int kConvTokens = 8;
template <typename T, int TAPS>
__global__ __launch_bounds__(256) void conv_silu_run_kernel(ConvSilu a) {
  constexpr int kReach = TAPS - 1;
  const int vectors = a.inner >> 3, runs = (a.seq + kConvTokens - 1) / kConvTokens;
  const long long idx = (long long)blockIdx.x * 256 + threadIdx.x;
  if (idx >= (long long)(a.rows / a.seq) * runs * vectors) return;
  const int c = 8 * (int)(idx % vectors), run = (int)((idx / vectors) % runs), b = (int)(idx / ((long long)vectors * runs));
  const int t0 = run * kConvTokens, count = min(kConvTokens, a.seq - t0);
  const T* y = reinterpret_cast<const T*>(a.y) + ((size_t)b * a.seq + t0) * a.ldy + c;
  const T* ring = reinterpret_cast<const T*>(a.ring) + (size_t)b * kReach * a.inner + c;
  T* out = reinterpret_cast<T*>(a.out) + ((size_t)b * a.seq + t0) * a.inner + c;
  Float8 now[kConvTokens], last[kReach], w[TAPS];  // last[j]: j + 1 tokens back
#pragma unroll
  for (int k = 0; k < kConvTokens; ++k)
    if (k < count) now[k] = load8(y + (size_t)k * a.ldy);
#pragma unroll
  for (int j = 0; j < kReach; ++j) {
    const int t = t0 - 1 - j, p = a.start + t;
    last[j] = Float8{};
    if (t >= 0) last[j] = load8(y - (size_t)(j + 1) * a.ldy);
    else if (p >= 0) last[j] = load8(ring + (size_t)(p % kReach) * a.inner);
  }
#pragma unroll
  for (int j = 0; j < TAPS; ++j) w[j] = load8(a.weight + (size_t)(kReach - j) * a.inner + c);
  const Float8 bias = load8(a.bias + c);
#pragma unroll
  for (int k = 0; k < kConvTokens; ++k) {
    if (k >= count) break;
    Float8 sum = bias;
#pragma unroll
    for (int j = kReach; j >= 0; --j) {
      const Float8& v = j <= k ? now[j <= k ? k - j : 0] : last[j > k ? j - k - 1 : 0];
#pragma unroll
      for (int e = 0; e < 8; ++e) sum.v[e] = fmaf(w[j].v[e], v.v[e], sum.v[e]);
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) sum.v[e] = silu_for<T>(sum.v[e]);
    store8(out + (size_t)k * a.inner, sum);
  }
}

template <int kCtrl>
__device__ __forceinline__ float dpp_add(float v) {
  return v + __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), kCtrl, 0xF, 0xF, true));
}
// sum over L neighbouring lanes (L a power of two), in every one of them
template <int L>
__device__ __forceinline__ float team_sum(float v) {
  if (L > 1) v = dpp_add<0xB1>(v);    // quad_perm [1, 0, 3, 2]
  if (L > 2) v = dpp_add<0x4E>(v);    // quad_perm [2, 3, 0, 1]
  if (L > 4) v = dpp_add<0x141>(v);   // row_half_mirror: quads are uniform by now
  if (L > 8) v = dpp_add<0x140>(v);   // row_mirror
  if (L > 16) v += __shfl_xor(v, 16);
  if (L > 32) v += __shfl_xor(v, 32);
  return v;
}

struct Scan {
  const void* x;            // [B * seq, inner] behind the convolution
  const void* dt;           // [B * seq, dt_ld] raw
  const void* low;          // [B * seq, low_ld]: B at column b_col, C at c_col, `states` each
  const void* z;            // [B * seq, z_ld]
  const float *a2, *d, *dt_bias;  // [states / 4, inner, 4], [inner], [inner]
  float* state;             // [B, states / 4, inner, 4] or null
  int start;
  const long long* pos;
  int seq, inner, states, dt_ld, low_ld, b_col, c_col, z_ld, out_ld;
  void* out;                // [B * seq, out_ld]
};
// L lanes share a channel, NS states each (states <= L NS; the ones past the end stay zero), so that a small model or batch
// still fills the chip: the time loop is sequential, and its length is what a wave costs.  256 / L channels per workgroup.
// A tile of kT tokens is staged in LDS: dt and dt x (the softplus is taken once per channel and token there), B and C; y takes
// dt x's place.  The next tile's operands are requested ahead of the current one's time loop.
template <int K, int NS>
struct Operands {
  float dt[K], dx[K], b[K][NS], c[K][NS];
};
template <int L, int NS>
constexpr int scan_tile() {
  int t = 8 * L;
  while (t * L * NS > 4096) t /= 2;
  return t;
}
template <typename T, int L, int NS>
__global__ __launch_bounds__(256) void scan_kernel(Scan a) {
  constexpr int CH = 256 / L, kT = scan_tile<L, NS>(), kN = L * NS, kVec = kT * CH / 8, kPitch = CH + 4, kTogether = 4;
  static_assert(kT % kTogether == 0, "whole groups of tokens");
  static_assert(kVec >= 1 && kVec <= 256, "at most one vector of 8 channels per thread");
  __shared__ __attribute__((aligned(16))) float dt_s[kT * kPitch], dx_s[kT * kPitch], b_s[kT * kN], c_s[kT * kN];
  const int tid = threadIdx.x, ch = tid / L, part = tid % L;
  const int b = blockIdx.y, c0 = blockIdx.x * CH, c = c0 + ch;
  const bool mine = c < a.inner;
  float s[NS], a2[NS];
  const bool carried = a.state && (a.start > 0 || (a.pos && *a.pos > 0));
  float* state = a.state + (size_t)b * a.inner * a.states;
  auto place = [&](int n) { return ((size_t)(n >> 2) * a.inner + c) * 4 + (n & 3); };
#pragma unroll
  for (int i = 0; i < NS; ++i) {
    const int n = part * NS + i;
    const bool real = mine && n < a.states;
    a2[i] = real ? a.a2[place(n)] : 0.f;
    s[i] = real && carried ? state[place(n)] : 0.f;
  }
  // this thread's vector of a tile: token vt, channels vc ..
  const int vt = tid / (CH / 8), vl = 8 * (tid % (CH / 8)), vc = c0 + vl;
  const bool stages = tid < kVec && vc < a.inner;
  const T* xp = reinterpret_cast<const T*>(a.x) + (size_t)b * a.seq * a.inner + vc;
  const T* dp = reinterpret_cast<const T*>(a.dt) + (size_t)b * a.seq * a.dt_ld + vc;
  const T* zp = reinterpret_cast<const T*>(a.z) + (size_t)b * a.seq * a.z_ld + vc;
  const T* lp = reinterpret_cast<const T*>(a.low) + (size_t)b * a.seq * a.low_ld;
  T* op = reinterpret_cast<T*>(a.out) + (size_t)b * a.seq * a.out_ld + vc;
  constexpr int kLow = (kT * kN + 255) / 256;
  Float8 nx{}, nd{}, nz{}, bias{}, skip{};
  float nb[kLow], nc[kLow];
  if (stages) {
    bias = load8(a.dt_bias + vc);
    skip = load8(a.d + vc);
  }
  auto request = [&](int t0) {
    const int t = t0 + vt;
    if (stages && t < a.seq) {
      nx = load8(xp + (size_t)t * a.inner);
      nd = load8(dp + (size_t)t * a.dt_ld);
      nz = load8(zp + (size_t)t * a.z_ld);
    }
#pragma unroll
    for (int k = 0; k < kLow; ++k) {
      const int i = tid + 256 * k, u = t0 + i / kN, n = i % kN;
      nb[k] = nc[k] = 0.f;
      if (i < kT * kN && u < a.seq && n < a.states) {
        nb[k] = to_f32(lp[(size_t)u * a.low_ld + a.b_col + n]);
        nc[k] = to_f32(lp[(size_t)u * a.low_ld + a.c_col + n]);
      }
    }
  };
  request(0);
  for (int t0 = 0; t0 < a.seq; t0 += kT) {
    const int count = min(kT, a.seq - t0);
    const Float8 x = nx, z = nz;
    if (tid < kVec) {
      float* dts = dt_s + vt * kPitch + vl;
      float* dxs = dx_s + vt * kPitch + vl;
      Float8 d, dx;
      const bool real = stages && vt < count;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float step = softplus_f32(nd.v[e] + bias.v[e]);
        d.v[e] = real ? step : 0.f;
        dx.v[e] = real ? step * x.v[e] : 0.f;
      }
      store8(dts, d);
      store8(dxs, dx);
    }
#pragma unroll
    for (int k = 0; k < kLow; ++k) {
      const int i = tid + 256 * k;
      if (i < kT * kN) {
        b_s[i] = nb[k];
        c_s[i] = nc[k];
      }
    }
    __syncthreads();
    if (t0 + kT < a.seq) request(t0 + kT);
    // (tokens past the end: dt = 0 leaves the states alone)  A group's operands are read ahead of the arithmetic of the one before.
    Operands<kTogether, NS> next;
    auto read = [&](int u) {
#pragma unroll
      for (int k = 0; k < kTogether; ++k) {
        next.dt[k] = dt_s[(u + k) * kPitch + ch];
        next.dx[k] = dx_s[(u + k) * kPitch + ch];
#pragma unroll
        for (int i = 0; i < NS; ++i) {
          next.b[k][i] = b_s[(u + k) * kN + part * NS + i];
          next.c[k][i] = c_s[(u + k) * kN + part * NS + i];
        }
      }
    };
    read(0);
    for (int u = 0; u < count; u += kTogether) {
      const Operands<kTogether, NS> now = next;
      read(min(u + kTogether, kT - kTogether));
      float y[kTogether], f[kTogether][NS];
#pragma unroll
      for (int k = 0; k < kTogether; ++k)
#pragma unroll
        for (int i = 0; i < NS; ++i) f[k][i] = __builtin_amdgcn_exp2f(now.dt[k] * a2[i]);
#pragma unroll
      for (int k = 0; k < kTogether; ++k) {
        y[k] = 0.f;
#pragma unroll
        for (int i = 0; i < NS; ++i) {
          s[i] = fmaf(f[k][i], s[i], now.dx[k] * now.b[k][i]);
          y[k] = fmaf(s[i], now.c[k][i], y[k]);
        }
      }
#pragma unroll
      for (int k = 0; k < kTogether; ++k) y[k] = team_sum<L>(y[k]);
      if (part == 0)
#pragma unroll
        for (int k = 0; k < kTogether; ++k) dx_s[(u + k) * kPitch + ch] = y[k];
    }
    __syncthreads();
    if (stages && vt < count) {
      const float* ys = dx_s + vt * kPitch + vl;
      Float8 o;
#pragma unroll
      for (int e = 0; e < 8; ++e) o.v[e] = fmaf(skip.v[e], x.v[e], ys[e]) * silu_for<T>(z.v[e]);
      store8(op + (size_t)(t0 + vt) * a.out_ld, o);
    }
    __syncthreads();
  }
  if (a.state && mine)
#pragma unroll
    for (int i = 0; i < NS; ++i)
      if (part * NS + i < a.states) state[place(part * NS + i)] = s[i];
}

// ---- one token per sequence, bf16
// Slot of the column `back` tokens (1 .. reach) ahead of the one whose own slot is `slot`.
__device__ __forceinline__ int column_slot(int slot, int back, int reach) {
  const int s = slot - back;
  return s < 0 ? s + reach : s;
}

// The projection of the convolved columns to (dt rank | B | C): `rows` weight rows (a multiple of 16), K = inner cut into
// `splits` parts whose sums scan_step_kernel adds.  A workgroup takes RT row tiles and a part of K in blocks of kScanBlock
// channels: a wave requests its weights, all threads convolve the block's channels into LDS (a thread 8 channels of every
// second sequence, its weights in registers), then the product.  Grid (row groups, splits, batch blocks).
struct ScanProject {
  const float* y;           // [B, ldy]: convolved columns, then z
  const uint16_t* ring;     // [B, taps - 1, inner]
  const float* weight;      // [taps, inner]
  const float* bias;
  const long long* pos;
  const uint16_t* w;        // [rows, inner]
  float* partial;           // [splits, B, rows]
  int batch, ldy, inner, taps, rows, splits;
};
constexpr int kScanBlock = 1024;
// TAPS: the convolution's width, or 0 for any
template <int RT, int TAPS>
__global__ __launch_bounds__(256) void scan_project_kernel(ScanProject a) {
  constexpr int kSteps = kScanBlock / 32 / 4, kLd = kScanBlock + 8;
  __shared__ __attribute__((aligned(16))) uint16_t conv[kGemvBatch * kLd];
  __shared__ __attribute__((aligned(16))) float red[RT * 4 * 256];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 15, g = lane >> 4;
  const int b0 = blockIdx.z * kGemvBatch, nb = min(kGemvBatch, a.batch - b0);
  const int tile0 = max(0, min(RT * (int)blockIdx.x, a.rows / 16 - RT));  // (the last group may repeat its neighbour's rows)
  const int reach = (TAPS ? TAPS : a.taps) - 1, p = clamped_position(a.pos, 0, 0x7FFFFFFF), slot = reach > 0 ? p % reach : 0;
  const int steps = (a.inner + 31) >> 5, per = (steps + a.splits - 1) / a.splits;
  const int lo = min(steps, (int)blockIdx.y * per), hi = min(steps, lo + per);
  const uint16_t* wrow = a.w + (size_t)(16 * tile0 + r) * a.inner;
  const int vl = 8 * (tid & 127);
  f32x4_t acc[RT][1] = {};
  for (int s0 = lo; s0 < hi; s0 += kScanBlock / 32) {
    const int mine = s0 + kSteps * wave;
    u32x4_t w[kSteps][RT];
#pragma unroll
    for (int i = 0; i < kSteps; ++i)
#pragma unroll
      for (int n = 0; n < RT; ++n) {
        const int k = 32 * (mine + i) + 8 * g;
        w[i][n] = u32x4_t{0u, 0u, 0u, 0u};
        if (mine + i < hi && k < a.inner) w[i][n] = *reinterpret_cast<const u32x4_t*>(wrow + (size_t)n * 16 * a.inner + k);
      }
    const int c = 32 * s0 + vl;
    if (c < min(32 * hi, a.inner)) {
      const Float8 bias = load8(a.bias + c);
      Float8 f[TAPS ? TAPS : 1];
#pragma unroll
      for (int j = 0; j < TAPS; ++j) f[j] = load8(a.weight + (size_t)(reach - j) * a.inner + c);
      for (int b = tid >> 7; b < nb; b += 2) {
        const uint16_t* ring = a.ring + (size_t)(b0 + b) * reach * a.inner + c;
        Float8 sum = bias, own = load8(a.y + (size_t)(b0 + b) * a.ldy + c);
        auto tap = [&](const Float8& weight, const Float8& v) {
#pragma unroll
          for (int e = 0; e < 8; ++e) sum.v[e] = fmaf(weight.v[e], v.v[e], sum.v[e]);
        };
        if (TAPS > 0) {
          Float8 held[TAPS > 1 ? TAPS : 1];
#pragma unroll
          for (int j = TAPS - 1; j > 0; --j)
            if (j <= p) held[j] = load8(ring + (size_t)column_slot(slot, j, reach) * a.inner);
#pragma unroll
          for (int j = TAPS - 1; j > 0; --j)
            if (j <= p) tap(f[j], held[j]);
        } else {
          for (int j = min(reach, p); j > 0; --j)
            tap(load8(a.weight + (size_t)(reach - j) * a.inner + c), load8(ring + (size_t)column_slot(slot, j, reach) * a.inner));
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) own.v[e] = to_f32(f32_to_bf16_rne(own.v[e]));  // (as the ring will hold it)
        tap(TAPS ? f[0] : load8(a.weight + (size_t)reach * a.inner + c), own);
#pragma unroll
        for (int e = 0; e < 8; ++e) sum.v[e] = silu_for<uint16_t>(sum.v[e]);
        store8(conv + b * kLd + vl, sum);
      }
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < kSteps; ++i) {
      const int local = 32 * (kSteps * wave + i) + 8 * g;
      u32x4_t v = {0u, 0u, 0u, 0u};
      if (r < nb && mine + i < hi && 32 * s0 + local < a.inner) v = *reinterpret_cast<const u32x4_t*>(conv + r * kLd + local);
#pragma unroll
      for (int n = 0; n < RT; ++n) acc[n][0] = mfma16(w[i][n], v, acc[n][0]);
    }
    __syncthreads();
  }
  meet<4, RT, 1>(acc, red, wave, lane);
#pragma unroll
  for (int i = 0; i < RT; ++i)
    if (wave == i && r < nb)
      store4(a.partial + ((size_t)blockIdx.y * a.batch + b0 + r) * a.rows + 16 * (tile0 + i) + 4 * g,
             float4{acc[i][0][0], acc[i][0][1], acc[i][0][2], acc[i][0][3]});
}

// The rest of the step for 64 channels of BB sequences: the parts of (dt rank | B | C) are added, dt comes from a product on
// MFMA (a wave per 16 channels), then a lane per channel, a wave per sequence and turn: it convolves the channel, moves the
// channel's states on and writes the gated output and the ring's new row.  Everything that does not hang on the parts is
// requested behind them, ahead of the first barrier.  Grid (channel blocks, batch blocks).
struct ScanStep {
  const float* y;           // [B, ldy]: convolved columns, z from column inner on
  uint16_t* ring;
  const float *weight, *bias;
  const long long* pos;
  const float* partial;     // [splits, B, rows]: dt rank from 0, B from rank, C from rank + states
  const uint16_t* w_dt;     // [inner, rank]
  const float *dt_bias, *a2, *d;
  float* state;             // [B, states / 4, inner, 4]
  uint16_t* out;            // [B, out_ld]
  int batch, ldy, inner, taps, rows, splits, rank, states, out_ld;
};
__host__ __device__ constexpr int scan_step_lds(int rank, int states, int bb) {
  return bb * (2 * (rank + 8) + 4 * 2 * states + 4 * 64);
}
template <int BB>
__global__ __launch_bounds__(256) void scan_step_kernel(ScanStep a) {
  constexpr int kTurns = BB / 4, kPlanes = 4, kSteps = 8, kAhead = 8;
  extern __shared__ __attribute__((aligned(16))) unsigned char scan_lds[];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 15, g = lane >> 4;
  const int b0 = blockIdx.y * BB, nb = min(BB, a.batch - b0), c0 = blockIdx.x * 64, c = c0 + lane;
  const int ld = a.rank + 8, used = a.rank + 2 * a.states, quads = used >> 2;
  float* bc = reinterpret_cast<float*>(scan_lds);                  // [BB][2 states]
  float* dt_s = bc + BB * 2 * a.states;                            // [BB][64]
  uint16_t* low = reinterpret_cast<uint16_t*>(dt_s + BB * 64);     // [BB][rank + 8]
  const int reach = a.taps - 1, p = clamped_position(a.pos, 0, 0x7FFFFFFF), slot = reach > 0 ? p % reach : 0;
  float4 ahead[kAhead];
  auto request = [&](int i, int s0) {
    const float* src = a.partial + (size_t)(b0 + i / quads) * a.rows + 4 * (i % quads);
#pragma unroll
    for (int k = 0; k < kAhead; ++k)
      if (s0 + k < a.splits) ahead[k] = load4(src + (size_t)(s0 + k) * a.batch * a.rows);
  };
  if (tid < nb * quads) request(tid, 0);
  // this wave's 16 channels of the step size product
  const bool tile = c0 + 16 * wave < a.inner;
  const uint16_t* wrow = a.w_dt + (size_t)(c0 + 16 * wave + r) * a.rank;
  u32x4_t w[kSteps];
#pragma unroll
  for (int s = 0; s < kSteps; ++s) {
    w[s] = u32x4_t{0u, 0u, 0u, 0u};
    if (tile && 32 * s + 8 * g < a.rank) w[s] = *reinterpret_cast<const u32x4_t*>(wrow + 32 * s + 8 * g);
  }
  // this lane's channel: the convolution, the gate, the first planes of its decays and states
  float x[kTurns], z[kTurns], skip = 0.f;
  uint16_t own[kTurns];
  float4 f[kPlanes], st[kTurns][kPlanes];
  if (c < a.inner) {
    skip = a.d[c];
#pragma unroll
    for (int n = 0; n < kPlanes; ++n)
      if (4 * n < a.states) f[n] = load4(a.a2 + ((size_t)n * a.inner + c) * 4);
  }
#pragma unroll
  for (int t = 0; t < kTurns; ++t) {
    const int b = wave + 4 * t;
    if (c >= a.inner || b >= nb) continue;
    const float* y = a.y + (size_t)(b0 + b) * a.ldy + c;
    const uint16_t* ring = a.ring + (size_t)(b0 + b) * reach * a.inner + c;
    const float* state = a.state + (size_t)(b0 + b) * a.states * a.inner + 4 * c;
#pragma unroll
    for (int n = 0; n < kPlanes; ++n)
      if (4 * n < a.states) st[t][n] = p > 0 ? load4(state + (size_t)n * a.inner * 4) : float4{0.f, 0.f, 0.f, 0.f};
    own[t] = f32_to_bf16_rne(y[0]);
    z[t] = y[a.inner];
    x[t] = a.bias[c];
#pragma unroll 4
    for (int j = min(reach, p); j > 0; --j)
      x[t] = fmaf(a.weight[(size_t)(reach - j) * a.inner + c], to_f32(ring[(size_t)column_slot(slot, j, reach) * a.inner]), x[t]);
    x[t] = fmaf(a.weight[(size_t)reach * a.inner + c], to_f32(own[t]), x[t]);
  }
  for (int i = tid; i < nb * quads; i += 256) {
    float4 v = float4{0.f, 0.f, 0.f, 0.f};
    for (int s0 = 0; s0 < a.splits; s0 += kAhead) {
      if (i != tid || s0 > 0) request(i, s0);
#pragma unroll
      for (int k = 0; k < kAhead; ++k)
        if (s0 + k < a.splits) {
          v.x += ahead[k].x; v.y += ahead[k].y; v.z += ahead[k].z; v.w += ahead[k].w;
        }
    }
    const int b = i / quads, n = 4 * (i % quads);
    if (n < a.rank) store4(low + b * ld + n, v);
    else store4(bc + b * 2 * a.states + n - a.rank, v);
  }
  __syncthreads();
  if (tile) {
    f32x4_t acc[1][1] = {};
    auto operand = [&](int, int s) {
      return r < nb ? *reinterpret_cast<const u32x4_t*>(low + r * ld + 32 * s + 8 * g) : u32x4_t{0u, 0u, 0u, 0u};
    };
#pragma unroll
    for (int s = 0; s < kSteps; ++s)
      if (32 * s < a.rank) acc[0][0] = mfma16(w[s], 32 * s + 8 * g < a.rank ? operand(0, s) : u32x4_t{0u, 0u, 0u, 0u}, acc[0][0]);
    tile_steps<1, 1>(wrow, a.rank, kSteps, (a.rank + 31) >> 5, g, acc, operand);
    if (r < nb) {
      const float4 bias = load4(a.dt_bias + c0 + 16 * wave + 4 * g);
      store4(dt_s + r * 64 + 16 * wave + 4 * g, float4{softplus_f32(acc[0][0][0] + bias.x), softplus_f32(acc[0][0][1] + bias.y),
                                                       softplus_f32(acc[0][0][2] + bias.z), softplus_f32(acc[0][0][3] + bias.w)});
    }
  }
  __syncthreads();
#pragma unroll
  for (int t = 0; t < kTurns; ++t) {
    const int b = wave + 4 * t;
    if (c >= a.inner || b >= nb) continue;
    if (reach > 0) a.ring[((size_t)(b0 + b) * reach + slot) * a.inner + c] = own[t];
    const float v = silu_for<uint16_t>(x[t]), dt = dt_s[b * 64 + lane], dx = dt * v;
    float* state = a.state + (size_t)(b0 + b) * a.states * a.inner + 4 * c;
    const float* bs = bc + b * 2 * a.states;
    float out = skip * v;
    auto move = [&](int n, float4 s, const float4& k) {
      const float4 bn = load4(bs + 4 * n), cn = load4(bs + a.states + 4 * n);
      s.x = fmaf(__builtin_amdgcn_exp2f(dt * k.x), s.x, dx * bn.x);
      s.y = fmaf(__builtin_amdgcn_exp2f(dt * k.y), s.y, dx * bn.y);
      s.z = fmaf(__builtin_amdgcn_exp2f(dt * k.z), s.z, dx * bn.z);
      s.w = fmaf(__builtin_amdgcn_exp2f(dt * k.w), s.w, dx * bn.w);
      store4(state + (size_t)n * a.inner * 4, s);
      out = fmaf(s.x, cn.x, fmaf(s.y, cn.y, fmaf(s.z, cn.z, fmaf(s.w, cn.w, out))));
    };
#pragma unroll
    for (int n = 0; n < kPlanes; ++n)
      if (4 * n < a.states) move(n, st[t][n], f[n]);
#pragma unroll 4
    for (int n = kPlanes; n < a.states / 4; ++n)
      move(n, p > 0 ? load4(state + (size_t)n * a.inner * 4) : float4{0.f, 0.f, 0.f, 0.f}, load4(a.a2 + ((size_t)n * a.inner + c) * 4));
    a.out[(size_t)(b0 + b) * a.out_ld + c] = f32_to_bf16_rne(out * silu_for<uint16_t>(z[t]));
  }
}

}  // namespace ajq
