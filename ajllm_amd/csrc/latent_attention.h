// Attention over keys that are made of a per-head part and (optionally) a part all heads share, with a sliding window, first
// rows that stay visible, an attention sink and an output gate (a factor per head, or a sigmoid per column):
//
//   s_j     = (qu . ku_j + qr . kr_j) * scale            over the visible rows j
//   out     = gate * sum_j exp(s_j) v_j / (exp(sink) + sum_j exp(s_j))
//
// Heads may share key / value heads in groups of `share`.
//
// Three kernels:
//   windowed_attention_kernel   any sizes, bf16 or fp32, one wave per (token, head): fp32 prompts and decoding
//   windowed_prefill_kernel     prompts in bf16 on MFMA, keys and values expanded per head
//   latent_decode_kernel        one token per sequence in bf16 on MFMA, in the latent space: the rows of the cache are
//                               keys and values at once, all heads share them (see below)
//
// Scores, weights and sums are fp32; exponents are taken in base 2, scores multiplied by scale * log2(e).
#pragma once
#include "dense_kernels.h"
#include "prefill_attention.h"  // also dma16, the fragment reads and quad_max / quad_sum

namespace ajq {

struct WindowedAttention {
  const void* q;            // [B * T, H, d1 + d2]: unrotated part, rotated part
  const void* k1;           // per-head key part: batch, row and head strides (elements); d1 wide
  const void* k2;           // shared key part: batch and row strides; d2 wide
  const void* v;            // batch, row and head strides; dv wide
  const float* sink;        // [H] or null
  const float* gates;       // [B * T, H] or null
  const long long* pos;     // device-side position: the first min(*pos + 1, rows) rows are visible (a ring of cap rows)
  void* out;                // [B * T, out_ld], head h at column h * dv
  long long k1_batch, k2_batch, v_batch;
  long long k1_head, v_head;
  int k1_row, k2_row, v_row;
  int d1, d2, dv;           // multiples of 8; d2 may be 0
  int batch, heads, seq;    // T new tokens per sequence
  int rows, prior;          // rows a buffer holds per sequence; query t sits at row prior + t
  int window;               // <= 0: none
  int keep;                 // rows 0 .. keep - 1 are visible whatever the window
  int share;                // heads per key / value head
  int gate_ld;
  const void* column_gates; // [B * T, gate_ld], head h at column h * dv: the output's sigmoid gate before the sigmoid, or null
  int out_ld;
  float scale;
};

constexpr float kLog2eF = 1.4426950408889634f;

// One wave per (b, t, h).  Lanes take one key each for the scores of 64 keys and dv / 64 value columns each for the
// sums.  LDS: q (d1 + d2), output sums (dv), 64 weights.
template <typename T, typename O>
__global__ __launch_bounds__(64) void windowed_attention_kernel(WindowedAttention a) {
  extern __shared__ float sh[];
  const int lane = threadIdx.x, h = blockIdx.y, m = blockIdx.x, b = m / a.seq, t = m % a.seq;
  const int dq = a.d1 + a.d2;
  float* q = sh;
  float* acc = q + dq;
  float* weight = acc + a.dv;
  const T* qsrc = reinterpret_cast<const T*>(a.q) + ((size_t)m * a.heads + h) * dq;
  for (int i = lane; i < dq; i += 64) q[i] = to_f32(qsrc[i]);
  for (int i = lane; i < a.dv; i += 64) acc[i] = 0.f;
  int lo = 0, hi;  // visible rows lo .. hi
  if (a.pos) {
    hi = (int)min(max(*a.pos, 0ll), (long long)a.rows - 1);
  } else {
    hi = a.prior + t;
    if (a.window > 0) lo = max(0, hi - a.window + 1);
  }
  const int kept = min(a.keep, lo), n_rows = kept + hi - lo + 1;  // rows 0 .. kept - 1, then lo .. hi
  auto row_of = [&](int j) { return j < kept ? j : lo + j - kept; };
  const T* k1 = reinterpret_cast<const T*>(a.k1) + (size_t)b * a.k1_batch + (size_t)(h / a.share) * a.k1_head;
  const T* k2 = reinterpret_cast<const T*>(a.k2) + (size_t)b * a.k2_batch;
  const T* v = reinterpret_cast<const T*>(a.v) + (size_t)b * a.v_batch + (size_t)(h / a.share) * a.v_head;
  const float scale2 = a.scale * kLog2eF;
  float mx = a.sink ? a.sink[h] * kLog2eF : -INFINITY, total = a.sink ? 1.f : 0.f;
  __syncthreads();
  for (int j0 = 0; j0 < n_rows; j0 += 64) {
    const int j = row_of(j0 + lane);
    float s = -INFINITY;
    if (j0 + lane < n_rows) {
      float d = 0.f;
      const T* kr = k1 + (size_t)j * a.k1_row;
      for (int i = 0; i < a.d1; i += 4) {
        const float4 k4 = load4(kr + i);
        d = fmaf(q[i], k4.x, d); d = fmaf(q[i + 1], k4.y, d); d = fmaf(q[i + 2], k4.z, d); d = fmaf(q[i + 3], k4.w, d);
      }
      kr = k2 + (size_t)j * a.k2_row;
      for (int i = 0; i < a.d2; i += 4) {
        const float4 k4 = load4(kr + i);
        const float* q2 = q + a.d1 + i;
        d = fmaf(q2[0], k4.x, d); d = fmaf(q2[1], k4.y, d); d = fmaf(q2[2], k4.z, d); d = fmaf(q2[3], k4.w, d);
      }
      s = d * scale2;
    }
    const float m_new = fmaxf(mx, wave_max64(s));
    const float corr = mx == -INFINITY ? 0.f : exp2f(mx - m_new);
    const float w = s == -INFINITY ? 0.f : exp2f(s - m_new);
    total = total * corr + wave_sum64(w);
    mx = m_new;
    weight[lane] = w;
    __syncthreads();
    const int n = min(64, n_rows - j0);
    for (int i = lane; i < a.dv; i += 64) {
      float o = acc[i] * corr;
      for (int jj = 0; jj < n; ++jj) o = fmaf(weight[jj], to_f32(v[(size_t)row_of(j0 + jj) * a.v_row + i]), o);
      acc[i] = o;
    }
    __syncthreads();
  }
  const float factor = a.gates ? a.gates[(size_t)m * a.heads + h] : 1.f;
  O* out = reinterpret_cast<O*>(a.out) + (size_t)m * a.out_ld + (size_t)h * a.dv;
  const T* gate = a.column_gates ? reinterpret_cast<const T*>(a.column_gates) + (size_t)m * a.gate_ld + (size_t)h * a.dv : nullptr;
  for (int i = lane; i < a.dv; i += 64) out[i] = from_f32<O>(acc[i] / total * factor * (gate ? sigmoid_f32(to_f32(gate[i])) : 1.f));
}

// global -> LDS without registers (16 bytes per lane, a wave's 1 KiB contiguous in LDS), every lane with an address of
// its own; the caller orders its completion with an explicit s_waitcnt vmcnt before a barrier (see dma16)
#pragma clang diagnostic push
#pragma clang diagnostic ignored "-Winline-asm"  // m0 is named as clobbered on purpose
__device__ __forceinline__ void dma16_gather(const void* src, uint32_t lds_addr) {
  asm volatile("s_mov_b32 m0, %0\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, off"
               :
               : "s"(lds_addr), "v"(src)
               : "memory", "m0");
}
#pragma clang diagnostic pop

// Prompts, bf16.  The structure of attn_prefill_kernel (both products transposed so that no operand changes layout;
// values read with transposing LDS reads; a row's reference exponent moves only when an exponent outgrows it), with
//   * a workgroup of 4 waves on 64 U query rows of one (b, h), a wave U groups of 16;
//   * keys of KS 32-column steps gathered from two places (the head's own columns, then the shared ones; columns past
//     both meet zero query columns) and values of VT 16-column tiles, one block of 64 rows ahead by DMA;
//   * blocks of the first rows that stay visible, then from the first key in the window of the workgroup's first query to
//     its last query's own;
//   * the sink as the initial state of the running softmax: reference exponent sink, denominator 1.  Every row then
//     has a finite reference from the start, also when a whole block lies outside its window.
// LDS holds key and value rows in panels of 128 bytes (64 rows x 8 chunks of 16 bytes = 8 KiB, keys first):
//   key panel:   chunk c of row k in slot c ^ ((k >> 1) & 7)
//   value panel: the two chunks of 32-byte segment v of row k in segment slot v ^ ((k >> 1) & 3)
// so that a fragment read (16 rows of one chunk, or 8 rows of one segment) meets every bank once.  A DMA request fills 8
// rows of a panel; wave w takes requests w and w + 4, which makes the chunk a lane fetches the same in every request.
constexpr int prefill_panels(int ks, int vt) { return (ks + 1) / 2 + (vt + 3) / 4; }
template <int KS, int VT, int U>
__global__ __launch_bounds__(256, prefill_panels(KS, VT) > 5 ? 1 : 2) void windowed_prefill_kernel(WindowedAttention a) {
  constexpr int KP = (KS + 1) / 2, VP = (VT + 3) / 4;      // key / value panels
  constexpr int kPanel = kPfBK * 128, kStage = (KP + VP) * kPanel;
  extern __shared__ __attribute__((aligned(1024))) unsigned char lds[];
  const uint32_t lds0 = (uint32_t)(uintptr_t)(pf_lds_char_t*)lds;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int r = lane & 15, g = lane >> 4;
  constexpr int kBQ = 64 * U;
  // an XCD takes a contiguous eighth of the (b, h) pairs, neighbouring query blocks of a pair (which share keys) together
  const int qblocks = (a.seq + kBQ - 1) / kBQ, BH = a.batch * a.heads;
  int qb, bh;
  if ((BH & 7) == 0) {
    const int m = (int)(blockIdx.x >> 3);
    qb = m % qblocks;
    bh = (int)(blockIdx.x & 7) * (BH >> 3) + m / qblocks;
  } else {
    qb = (int)blockIdx.x % qblocks;
    bh = (int)blockIdx.x / qblocks;
  }
  const int b = bh / a.heads, h = bh % a.heads;
  const int q0 = qb * kBQ;
  const int total = a.prior + a.seq;
  const int first_q = a.prior + q0, last_q = min(total, first_q + kBQ) - 1;  // rows of the workgroup's first / last query
  const int window = a.window > 0 ? a.window : 0x3FFFFFFF;
  int kept_blocks = (a.keep + kPfBK - 1) / kPfBK;
  int lo = max(0, first_q - window + 1) & ~(kPfBK - 1);
  if (lo <= kept_blocks * kPfBK) {  // one run of blocks
    lo = kept_blocks > 0 ? 0 : lo;
    kept_blocks = 0;
  }
  const int nblk = kept_blocks + (last_q - lo) / kPfBK + 1;
  auto block_row = [&](int j) { return j < kept_blocks ? j * kPfBK : lo + (j - kept_blocks) * kPfBK; };
  const int wave_first = first_q + 16 * U * wave, wave_last = wave_first + 16 * U - 1;

  const uint16_t* k1 = reinterpret_cast<const uint16_t*>(a.k1) + (size_t)b * a.k1_batch + (size_t)(h / a.share) * a.k1_head;
  const uint16_t* k2 = reinterpret_cast<const uint16_t*>(a.k2) + (size_t)b * a.k2_batch;
  const uint16_t* vv = reinterpret_cast<const uint16_t*>(a.v) + (size_t)b * a.v_batch + (size_t)(h / a.share) * a.v_head;
  const int c1 = a.d1 >> 3, c2 = c1 + (a.d2 >> 3), cv = a.dv >> 3;

  // ---- what this lane fetches: row 8 q + lane / 8 of a request, slot lane % 8 of its panel.  Chunks past the widths
  // repeat the last one (finite values that meet zeros, or columns that are not written).
  const int req_row = 8 * wave + (lane >> 3);
  const int kslot = (lane & 7) ^ ((4 * wave + (lane >> 4)) & 7);
  const int vslot = ((((lane & 7) >> 1) ^ ((lane >> 4) & 3)) << 1) | (lane & 1);
  const char* kbase[KP];
  uint32_t kstride[KP];  // bytes
#pragma unroll
  for (int p = 0; p < KP; ++p) {
    const int c = min(8 * p + kslot, c2 - 1);
    kbase[p] = reinterpret_cast<const char*>(c < c1 ? k1 + 8 * c : k2 + 8 * (c - c1));
    kstride[p] = 2u * (uint32_t)(c < c1 ? a.k1_row : a.k2_row);
  }
  const char* vbase[VP];
#pragma unroll
  for (int p = 0; p < VP; ++p) vbase[p] = reinterpret_cast<const char*>(vv + 8 * min(8 * p + vslot, cv - 1));
  const uint32_t vstride = 2u * (uint32_t)a.v_row;
  auto fetch = [&](int j) {
    const uint32_t to = lds0 + (uint32_t)((j & 1) * kStage + wave * 1024);
#pragma unroll
    for (int half = 0; half < 2; ++half) {
      // rows past the end repeat the last one; those keys are masked
      const uint32_t row = (uint32_t)min(block_row(j) + 32 * half + req_row, total - 1);
#pragma unroll
      for (int p = 0; p < KP; ++p) dma16_gather(kbase[p] + (size_t)row * kstride[p], to + (uint32_t)(p * kPanel + half * 4096));
#pragma unroll
      for (int p = 0; p < VP; ++p) dma16_gather(vbase[p] + (size_t)row * vstride, to + (uint32_t)((KP + p) * kPanel + half * 4096));
    }
  };
  // ---- fragment addresses inside a stage
  // keys (16-key tile jb, step s): row 16 jb + r, chunk 4 (s & 1) + g of panel s >> 1
  const uint32_t k_rd[2] = {lds0 + (uint32_t)(r * 128 + 16 * (g ^ ((r >> 1) & 7))),
                            lds0 + (uint32_t)(r * 128 + 16 * ((4 + g) ^ ((r >> 1) & 7)))};
  // values (tile t): this lane addresses 8 bytes (piece r & 3) of key 4 g + (r >> 2), segment t & 3 of panel t >> 2
  uint32_t v_rd[4];
#pragma unroll
  for (int v = 0; v < 4; ++v)
    v_rd[v] = lds0 + (uint32_t)(KP * kPanel + (4 * g + (r >> 2)) * 128 + 32 * (v ^ ((2 * g + (r >> 3)) & 3)) + 8 * (r & 3));

  fetch(0);
  const float scale2 = a.scale * kLog2eF;
  const float sink2 = a.sink ? a.sink[h] * kLog2eF : -1e30f;
  float m_run[U], l_run[U];
  f32x4_t o[U][VT];
  int qrow[U];
  u32x4_t qf[U][KS];
#pragma unroll
  for (int u = 0; u < U; ++u) {
    m_run[u] = sink2;
    l_run[u] = (a.sink && g == 0) ? 1.f : 0.f;  // (lane sums of a row's four lanes meet at the end)
#pragma unroll
    for (int t = 0; t < VT; ++t) o[u][t] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    const int t0 = q0 + 16 * U * wave + 16 * u + r;
    qrow[u] = a.prior + t0;
    const uint16_t* qp = reinterpret_cast<const uint16_t*>(a.q) +
                         (((size_t)b * a.seq + min(t0, a.seq - 1)) * a.heads + h) * (a.d1 + a.d2);
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      const int c = 4 * s + g;
      qf[u][s] = u32x4_t{0u, 0u, 0u, 0u};
      if (c < c2) qf[u][s] = *reinterpret_cast<const u32x4_t*>(qp + 8 * c);
    }
  }
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  __syncthreads();
  for (int j = 0; j < nblk; ++j) {
    // block j is complete in stage j & 1; block j + 1 goes into the other stage, last read before the previous barrier
    const int kb0 = block_row(j);
    if (j + 1 < nblk) fetch(j + 1);
    const uint32_t stage = (uint32_t)((j & 1) * kStage);
    if (kb0 <= wave_last && (kb0 + kPfBK - 1 > wave_first - window || kb0 < a.keep)) {
      f32x4_t sc[U][4];
#pragma unroll
      for (int s = 0; s < KS; ++s) {
        u32x4_t ka[4];
#pragma unroll
        for (int jb = 0; jb < 4; ++jb) ka[jb] = pf_read128(k_rd[s & 1] + stage + (uint32_t)((s >> 1) * kPanel + jb * 2048));
#pragma unroll
        for (int jb = 0; jb < 4; ++jb)
#pragma unroll
          for (int u = 0; u < U; ++u)
            sc[u][jb] = mfma16(ka[jb], qf[u][s], s == 0 ? f32x4_t{0.f, 0.f, 0.f, 0.f} : sc[u][jb]);
      }
      // masks only where the block reaches past the wave's first query or before its last query's window
      if (kb0 + kPfBK - 1 > wave_first || kb0 <= wave_last - window) {
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
          for (int jb = 0; jb < 4; ++jb)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
              const int key = kb0 + 16 * jb + 4 * g + i;
              if (key > qrow[u] || (key <= qrow[u] - window && key >= a.keep)) sc[u][jb][i] = -INFINITY;
            }
      }
      u32x4_t pf[U][2];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        float p[16], psum = 0.f;
#pragma unroll
        for (int e = 0; e < 16; ++e) {
          p[e] = __builtin_amdgcn_exp2f(__builtin_fmaf(sc[u][e >> 2][e & 3], scale2, -m_run[u]));
          psum += p[e];
        }
        if (__builtin_amdgcn_ballot_w64(psum > kPfTrigger) != 0) {
          float mx = -INFINITY;
#pragma unroll
          for (int e = 0; e < 16; ++e) mx = fmaxf(mx, sc[u][e >> 2][e & 3] * scale2);
          mx = quad_max(mx);
          const float m_new = mx > m_run[u] + kPfSlack ? mx : m_run[u];
          const float corr = __builtin_amdgcn_exp2f(m_run[u] - m_new);
          psum = 0.f;
#pragma unroll
          for (int e = 0; e < 16; ++e) {
            p[e] = __builtin_amdgcn_exp2f(__builtin_fmaf(sc[u][e >> 2][e & 3], scale2, -m_new));
            psum += p[e];
          }
          m_run[u] = m_new;
          l_run[u] *= corr;
#pragma unroll
          for (int t = 0; t < VT; ++t) o[u][t] *= corr;
        }
        l_run[u] += psum;
        pf[u][0] = pack8_bf16(&p[0]);
        pf[u][1] = pack8_bf16(&p[8]);
      }
      // value fragments (two transposing reads: a half's first and second 16-key tile), kRing of them in flight
      constexpr int kRing = VT < 4 ? VT : 4;
      auto v_at = [&](int i) { return v_rd[(i % VT) & 3] + stage + (uint32_t)((i / VT) * 4096 + ((i % VT) >> 2) * kPanel); };
      u32x2_t vlo[kRing], vhi[kRing];
#pragma unroll
      for (int i = 0; i < kRing; ++i) {
        vlo[i] = pf_read_tr(v_at(i));
        vhi[i] = pf_read_tr(v_at(i) + 2048u);
      }
#pragma unroll
      for (int i = 0; i < 2 * VT; ++i) {  // i = VT half + tile
        const u32x4_t vf = {vlo[i % kRing].x, vlo[i % kRing].y, vhi[i % kRing].x, vhi[i % kRing].y};
#pragma unroll
        for (int u = 0; u < U; ++u) o[u][i % VT] = mfma16(vf, pf[u][i / VT], o[u][i % VT]);
        if (i + kRing < 2 * VT) {
          vlo[i % kRing] = pf_read_tr(v_at(i + kRing));
          vhi[i % kRing] = pf_read_tr(v_at(i + kRing) + 2048u);
        }
      }
    }
    // the next block must have landed and every wave must be done with this one
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
  }
#pragma unroll
  for (int u = 0; u < U; ++u) {
    const float l = quad_sum(l_run[u]);
    const int t0 = qrow[u] - a.prior;
    if (t0 >= a.seq) continue;
    const size_t m = (size_t)b * a.seq + t0;
    const float factor = (a.gates ? a.gates[m * a.heads + h] : 1.f) / l;
    uint16_t* dst = reinterpret_cast<uint16_t*>(a.out) + m * a.out_ld + (size_t)h * a.dv + 4 * g;
    const uint16_t* gate = a.column_gates ? reinterpret_cast<const uint16_t*>(a.column_gates) + m * a.gate_ld + (size_t)h * a.dv + 4 * g : nullptr;
#pragma unroll
    for (int t = 0; t < VT; ++t)
      if (16 * t < a.dv) {
        float4 v = float4{o[u][t][0] * factor, o[u][t][1] * factor, o[u][t][2] * factor, o[u][t][3] * factor};
        if (gate) {
          const float4 z = load4(gate + 16 * t);
          v.x *= sigmoid_f32(z.x); v.y *= sigmoid_f32(z.y); v.z *= sigmoid_f32(z.z); v.w *= sigmoid_f32(z.w);
        }
        store4(dst + 16 * t, v);
      }
  }
}

}  // namespace ajq
