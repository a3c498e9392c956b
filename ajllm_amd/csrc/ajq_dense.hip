// C ABI of libajq_dense.so (include/ajq_dense.h): argument validation, launch geometry, error reporting.
#include <stdarg.h>
#include <stdio.h>

#include "../../include/ajq_dense.h"
#include "ajq_common.h"
#include "dense_kernels.h"
#include "latent_attention.h"
#include "dense_gemv_kernels.h"

using namespace ajq;

namespace {

thread_local char g_error[512] = "";

int fail(int status, const char* fmt, ...) {
  va_list ap;
  va_start(ap, fmt);
  vsnprintf(g_error, sizeof(g_error), fmt, ap);
  va_end(ap);
  return status;
}
bool aligned16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15u) == 0; }
bool known(int dtype) { return dtype == AJQD_BF16 || dtype == AJQD_F32; }
int check_launch(const char* what) {
  hipError_t e = hipGetLastError();
  if (e != hipSuccess) return fail(AJQ_ERR_HIP, "%s: %s", what, hipGetErrorString(e));
  return AJQ_OK;
}
const long long* positions64(const int64_t* p) { return reinterpret_cast<const long long*>(p); }

// Calls fn(T{}, U{}) for the element types of two dtype flags.
template <typename F>
void with_types(int a, int b, F&& fn) {
  if (a == AJQD_BF16 && b == AJQD_BF16) fn(uint16_t{}, uint16_t{});
  else if (a == AJQD_BF16) fn(uint16_t{}, float{});
  else if (b == AJQD_BF16) fn(float{}, uint16_t{});
  else fn(float{}, float{});
}

constexpr int kLdsLimit = 160 * 1024;
template <typename K>
int allow_lds(K kernel, int bytes, const char* what) {
  if (bytes > kLdsLimit) return fail(AJQ_ERR_UNSUPPORTED, "%s: %d bytes of LDS needed", what, bytes);
  if (bytes > 64 * 1024) {
    hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, bytes);
    if (e != hipSuccess) return fail(AJQ_ERR_HIP, "%s: %s", what, hipGetErrorString(e));
  }
  return AJQ_OK;
}

int check_shape(const ajqd_latent_shape* s, const char* what) {
  if (!s) return fail(AJQ_ERR_NULL, "%s: null shape", what);
  if (s->heads < 1 || s->dimp < 8 || s->dimp % 8 || s->rot < 2 || s->rot % 2 || s->rotp < s->rot || s->rotp % 8 || s->rank < 1 ||
      s->rankp < s->rank || s->rankp % 16)
    return fail(AJQ_ERR_SHAPE, "%s: unsupported latent shape (heads=%d dimp=%d rot=%d/%d rank=%d/%d)", what, s->heads, s->dimp,
                s->rot, s->rotp, s->rank, s->rankp);
  return AJQ_OK;
}
LatentShape device_shape(const ajqd_latent_shape* s) {
  return LatentShape{s->heads, s->dimp, s->rot, s->rotp, s->rank, s->rankp, s->eps};
}

int check_attention(const ajqd_windowed_attention_args* a, const char* what) {
  if (!a || !a->q || !a->k1 || !a->k2 || !a->v || !a->out) return fail(AJQ_ERR_NULL, "%s: null pointer argument", what);
  if (a->batch < 1 || a->heads < 1 || a->seq < 1 || a->rows < 1 || a->prior < 0 || a->d1 < 8 || a->d2 < 8 || a->dv < 16 ||
      a->d1 % 8 || a->d2 % 8 || a->dv % 16 || a->out_ld < a->heads * a->dv || a->out_ld % 4)
    return fail(AJQ_ERR_SHAPE, "%s: unsupported shape (B=%d H=%d T=%d rows=%d prior=%d d=%d+%d dv=%d)", what, a->batch, a->heads,
                a->seq, a->rows, a->prior, a->d1, a->d2, a->dv);
  if (a->pos ? a->seq != 1 : (long long)a->prior + a->seq > a->rows)
    return fail(AJQ_ERR_SHAPE, "%s: %d + %d queries do not fit %d rows", what, a->prior, a->seq, a->rows);
  if (!(a->scale > 0.f)) return fail(AJQ_ERR_SHAPE, "%s: the score scale must be positive", what);
  if (a->k1_row % 8 || a->k1_head % 8 || a->k2_row % 8 || a->v_row % 8 || a->v_head % 8 || a->k1_batch % 8 || a->k2_batch % 8 ||
      a->v_batch % 8 || !aligned16(a->q) || !aligned16(a->k1) || !aligned16(a->k2) || !aligned16(a->v) || !aligned16(a->out))
    return fail(AJQ_ERR_ALIGN, "%s: rows must start on 16-byte boundaries", what);
  return AJQ_OK;
}
WindowedAttention device_attention(const ajqd_windowed_attention_args* a) {
  WindowedAttention w;
  w.q = a->q; w.k1 = a->k1; w.k2 = a->k2; w.v = a->v; w.sink = a->sink; w.gates = a->gates;
  w.pos = positions64(a->pos); w.out = a->out;
  w.k1_batch = a->k1_batch; w.k2_batch = a->k2_batch; w.v_batch = a->v_batch;
  w.k1_row = a->k1_row; w.k1_head = a->k1_head; w.k2_row = a->k2_row; w.v_row = a->v_row; w.v_head = a->v_head;
  w.d1 = a->d1; w.d2 = a->d2; w.dv = a->dv;
  w.batch = a->batch; w.heads = a->heads; w.seq = a->seq;
  w.rows = a->rows; w.prior = a->prior; w.window = a->window; w.out_ld = a->out_ld; w.scale = a->scale;
  return w;
}

// ---- prompt attention: the smallest built (key steps, value tiles) that hold the widths
int prefill_ks(int d) { const int s = (d + 31) / 32; return s <= 4 ? s : s <= 6 ? 6 : s <= 8 ? 8 : 0; }
int prefill_vt(int dv) { const int t = (dv + 15) / 16; return t <= 2 ? 2 : t <= 4 ? 4 : t <= 6 ? 6 : t <= 8 ? 8 : t <= 16 ? 16 : 0; }
template <int KS, int VT>
int launch_prefill(const WindowedAttention& w, hipStream_t stream) {
  constexpr int U = KS + VT > 16 ? 1 : 2;
  constexpr int bytes = 2 * kPfBK * 128 * prefill_panels(KS, VT);
  auto kernel = windowed_prefill_kernel<KS, VT, U>;
  if (int e = allow_lds(kernel, bytes, "ajqd_windowed_prefill")) return e;
  const long long blocks = (long long)((w.seq + 64 * U - 1) / (64 * U)) * w.batch * w.heads;
  if (blocks > 0x7FFFFFFFll) return fail(AJQ_ERR_SHAPE, "ajqd_windowed_prefill: too many workgroups");
  hipLaunchKernelGGL(kernel, dim3((unsigned)blocks), dim3(256), bytes, stream, w);
  return check_launch("ajqd_windowed_prefill");
}
template <int KS>
int launch_prefill_vt(int vt, const WindowedAttention& w, hipStream_t stream) {
  switch (vt) {
    case 2: return launch_prefill<KS, 2>(w, stream);
    case 4: return launch_prefill<KS, 4>(w, stream);
    case 6: return launch_prefill<KS, 6>(w, stream);
    case 8: return launch_prefill<KS, 8>(w, stream);
    default: return launch_prefill<KS, 16>(w, stream);
  }
}

// ---- decode attention: (column steps, latent tiles per wave) that hold the widths
int latent_tiles(int rankp) { const int t = (rankp + 63) / 64; return t <= 2 ? 2 : t <= 4 ? 4 : t <= 8 ? 8 : 0; }
int latent_steps(int width) { const int s = (width + 31) / 32; return s <= 4 ? 4 : s <= 6 ? 6 : s <= 10 ? 10 : s <= 18 ? 18 : 0; }
// the chunks' sums, then (maximum, denominator) per head and chunk
float2* heads_at(const float* partial, int batch, int heads, int chunks, int rankp) {
  return reinterpret_cast<float2*>(const_cast<float*>(partial) + latent_sums_at(batch, 0, 0, heads, chunks, rankp));
}
constexpr int kDecodeWorkgroups = 256;  // one per CU (its LDS holds two blocks of rows)
int latent_head_groups(int heads) { return heads <= 16 ? 1 : (heads + 31) / 32; }  // one or two head tiles per workgroup
int gemv_waves(int k) { return k >= 2048 ? 8 : k >= 256 ? 4 : 1; }

}  // namespace

extern "C" {

const char* ajqd_last_error(void) { return g_error; }

int ajqd_embed(const int64_t* tokens, int rows, int seq, const void* table, int vocab, const void* positions,
               int table_rows, int start, const int64_t* pos, const float* extra, float* x, float* embedded, int width,
               int dtype, void* stream) {
  if (!tokens || !table || !x) return fail(AJQ_ERR_NULL, "ajqd_embed: null pointer argument");
  if (rows < 1 || seq < 1 || rows % seq || vocab < 1 || width < 8 || width % 8 || (pos && seq != 1) ||
      (positions && (table_rows < 1 || start < 0 || (!pos && (long long)start + seq > table_rows))))
    return fail(AJQ_ERR_SHAPE, "ajqd_embed: unsupported shape (rows=%d seq=%d vocab=%d positions=%d start=%d width=%d)", rows, seq,
                vocab, table_rows, start, width);
  if (!known(dtype)) return fail(AJQ_ERR_UNSUPPORTED, "ajqd_embed: unknown dtype %d", dtype);
  with_types(dtype, dtype, [&](auto t, auto) {
    using T = decltype(t);
    hipLaunchKernelGGL(embed_kernel<T>, dim3(rows), dim3(256), 0, (hipStream_t)stream, (const long long*)tokens, (const T*)table,
                       vocab, (const T*)positions, table_rows, start, positions64(pos), seq, extra, x, embedded, width);
  });
  return check_launch("ajqd_embed");
}

int ajqd_add_norms(float* x, const void* delta, int delta_dtype, const float* again, const float* step,
                   const float* gain1, const float* gain2, float eps, int center, void* out1, void* out2, int rows,
                   int true_width, int width, int dtype, void* stream) {
  if (!x || (out1 && !gain1) || (out2 && !gain2)) return fail(AJQ_ERR_NULL, "ajqd_add_norms: null pointer argument");
  if (rows < 1 || true_width < 1 || width < true_width || width % 8)
    return fail(AJQ_ERR_SHAPE, "ajqd_add_norms: unsupported shape (rows=%d width=%d of %d)", rows, true_width, width);
  if (!known(dtype) || !known(delta_dtype)) return fail(AJQ_ERR_UNSUPPORTED, "ajqd_add_norms: unknown dtype");
  with_types(dtype, delta_dtype, [&](auto t, auto d) {
    using T = decltype(t);
    using DT = decltype(d);
    hipLaunchKernelGGL((add_norms_kernel<T, DT>), dim3(rows), dim3(256), 0, (hipStream_t)stream, x, (const DT*)delta, again, step,
                       gain1, gain2, eps, center, (T*)out1, (T*)out2, true_width, width);
  });
  return check_launch("ajqd_add_norms");
}

int ajqd_latent_split(const void* y, int y_dtype, int ldy, const ajqd_latent_shape* shape, const float* latent_gain,
                      const float* cosine, const float* sine, int table_rows, int rows, int seq, int start, const int64_t* pos,
                      int prior, int cap, void* qu, int qu_ld, void* qr, int qr_ld, void* cache_rows, int64_t rows_batch,
                      float* gates, int dtype, void* stream) {
  if (int e = check_shape(shape, "ajqd_latent_split")) return e;
  if (!y || !latent_gain || !cosine || !sine || !qu || !qr || !cache_rows || !gates)
    return fail(AJQ_ERR_NULL, "ajqd_latent_split: null pointer argument");
  const int width = shape->rankp + shape->rotp;
  if (rows < 1 || seq < 1 || rows % seq || start < 0 || prior < 0 || table_rows < 1 || qu_ld < shape->dimp || qr_ld < shape->rotp ||
      ldy < shape->heads * (shape->dimp + shape->rotp) + width + shape->heads || (pos ? (seq != 1 || cap < 1) : (long long)start + seq > table_rows) ||
      rows_batch < (int64_t)(pos ? cap : prior + seq) * width)
    return fail(AJQ_ERR_SHAPE, "ajqd_latent_split: unsupported shape (rows=%d seq=%d start=%d prior=%d cap=%d ldy=%d)", rows, seq,
                start, prior, cap, ldy);
  if (!known(dtype) || !known(y_dtype)) return fail(AJQ_ERR_UNSUPPORTED, "ajqd_latent_split: unknown dtype");
  const LatentShape s = device_shape(shape);
  with_types(y_dtype, dtype, [&](auto yt, auto t) {
    using Y = decltype(yt);
    using T = decltype(t);
    hipLaunchKernelGGL((latent_split_kernel<Y, T>), dim3(rows), dim3(256), 0, (hipStream_t)stream, (const Y*)y, ldy, s, latent_gain,
                       cosine, sine, table_rows, start, positions64(pos), seq, prior, cap, (T*)qu, qu_ld, (T*)qr, qr_ld,
                       (T*)cache_rows, (long long)rows_batch, gates);
  });
  return check_launch("ajqd_latent_split");
}

int ajqd_ring_copy(void* ring, int cap, void* linear, int lines, int first_row, int position, int count, int row_bytes,
                   int batch, int to_ring, void* stream) {
  if (!ring || !linear) return fail(AJQ_ERR_NULL, "ajqd_ring_copy: null pointer argument");
  if (cap < 1 || count < 1 || count > cap || first_row < 0 || (long long)first_row + count > lines || position < 0 || batch < 1 ||
      row_bytes < 16 || row_bytes % 16)
    return fail(AJQ_ERR_SHAPE, "ajqd_ring_copy: unsupported shape (cap=%d lines=%d first=%d position=%d count=%d)", cap, lines,
                first_row, position, count);
  if (!aligned16(ring) || !aligned16(linear)) return fail(AJQ_ERR_ALIGN, "ajqd_ring_copy: buffers must be 16-byte aligned");
  const long long blocks = ((long long)batch * count * (row_bytes / 16) + 255) / 256;
  if (blocks > 0x7FFFFFFFll) return fail(AJQ_ERR_SHAPE, "ajqd_ring_copy: too many elements");
  hipLaunchKernelGGL(ring_copy_kernel, dim3((unsigned)blocks), dim3(256), 0, (hipStream_t)stream, (u32x4_t*)ring, cap,
                     (u32x4_t*)linear, lines, first_row, position, count, row_bytes / 16, batch, to_ring);
  return check_launch("ajqd_ring_copy");
}

int ajqd_gated_activation(const void* y, int y_dtype, void* out, int out_ld, int rows, int width, int act, int dtype,
                          void* stream) {
  if (!y || !out) return fail(AJQ_ERR_NULL, "ajqd_gated_activation: null pointer argument");
  if (rows < 1 || width < 8 || width % 8 || out_ld < width || out_ld % 4)
    return fail(AJQ_ERR_SHAPE, "ajqd_gated_activation: unsupported shape (rows=%d width=%d out_ld=%d)", rows, width, out_ld);
  if (!known(dtype) || !known(y_dtype) || act < 0 || act > AJQD_ACT_GELU_TANH)
    return fail(AJQ_ERR_UNSUPPORTED, "ajqd_gated_activation: unknown dtype or activation");
  const long long blocks = ((long long)rows * (width / 4) + 255) / 256;
  if (blocks > 0x7FFFFFFFll) return fail(AJQ_ERR_SHAPE, "ajqd_gated_activation: too many elements");
  with_types(y_dtype, dtype, [&](auto yt, auto t) {
    using Y = decltype(yt);
    using T = decltype(t);
    hipLaunchKernelGGL((gated_activation_kernel<Y, T>), dim3((unsigned)blocks), dim3(256), 0, (hipStream_t)stream, (const Y*)y, (T*)out,
                       out_ld, rows, width, act);
  });
  return check_launch("ajqd_gated_activation");
}

int ajqd_matvec(const void* w, const void* x, int x_batch, int x_group, void* y, int y_batch, int y_group, int groups,
                int n, int k, int batch, int dtype, int out_dtype, void* stream) {
  if (!w || !x || !y) return fail(AJQ_ERR_NULL, "ajqd_matvec: null pointer argument");
  if (n < 1 || k < 8 || k % 8 || groups < 1 || groups > 65535 || batch < 1 || batch > 65535 || x_batch % 4 || x_group % 4)
    return fail(AJQ_ERR_SHAPE, "ajqd_matvec: unsupported shape (groups=%d n=%d k=%d batch=%d)", groups, n, k, batch);
  if (!known(dtype) || !known(out_dtype)) return fail(AJQ_ERR_UNSUPPORTED, "ajqd_matvec: unknown dtype");
  with_types(dtype, out_dtype, [&](auto t, auto o) {
    using T = decltype(t);
    using O = decltype(o);
    hipLaunchKernelGGL((matvec_kernel<T, O>), dim3((n + 3) / 4, groups, batch), dim3(256), 0, (hipStream_t)stream, (const T*)w,
                       (const T*)x, x_batch, x_group, (O*)y, y_batch, y_group, n, k);
  });
  return check_launch("ajqd_matvec");
}

int ajqd_windowed_attention(const ajqd_windowed_attention_args* args, int dtype, int out_dtype, void* stream) {
  if (int e = check_attention(args, "ajqd_windowed_attention")) return e;
  if (!known(dtype) || !known(out_dtype)) return fail(AJQ_ERR_UNSUPPORTED, "ajqd_windowed_attention: unknown dtype");
  if (args->heads > 65535) return fail(AJQ_ERR_SHAPE, "ajqd_windowed_attention: too many heads");
  const int bytes = 4 * (args->d1 + args->d2 + args->dv + 64);
  const WindowedAttention w = device_attention(args);
  int status = AJQ_OK;
  with_types(dtype, out_dtype, [&](auto t, auto o) {
    auto kernel = windowed_attention_kernel<decltype(t), decltype(o)>;
    status = allow_lds(kernel, bytes, "ajqd_windowed_attention");
    if (status == AJQ_OK)
      hipLaunchKernelGGL(kernel, dim3(w.batch * w.seq, w.heads), dim3(64), bytes, (hipStream_t)stream, w);
  });
  return status != AJQ_OK ? status : check_launch("ajqd_windowed_attention");
}

int ajqd_windowed_prefill_supported(int d1, int d2, int dv) {
  return d1 >= 8 && d2 >= 8 && d1 % 8 == 0 && d2 % 8 == 0 && dv >= 16 && dv % 16 == 0 && prefill_ks(d1 + d2) && prefill_vt(dv);
}

int ajqd_windowed_prefill(const ajqd_windowed_attention_args* args, void* stream) {
  if (int e = check_attention(args, "ajqd_windowed_prefill")) return e;
  if (args->pos) return fail(AJQ_ERR_UNSUPPORTED, "ajqd_windowed_prefill: takes no device-side position");
  if (!ajqd_windowed_prefill_supported(args->d1, args->d2, args->dv))
    return fail(AJQ_ERR_UNSUPPORTED, "ajqd_windowed_prefill: widths %d + %d / %d are not built", args->d1, args->d2, args->dv);
  const WindowedAttention w = device_attention(args);
  const int vt = prefill_vt(args->dv);
  switch (prefill_ks(args->d1 + args->d2)) {
    case 1: return launch_prefill_vt<1>(vt, w, (hipStream_t)stream);
    case 2: return launch_prefill_vt<2>(vt, w, (hipStream_t)stream);
    case 3: return launch_prefill_vt<3>(vt, w, (hipStream_t)stream);
    case 4: return launch_prefill_vt<4>(vt, w, (hipStream_t)stream);
    case 6: return launch_prefill_vt<6>(vt, w, (hipStream_t)stream);
    default: return launch_prefill_vt<8>(vt, w, (hipStream_t)stream);
  }
}

int ajqd_dense_in(const ajqd_dense_in_args* a, void* stream) {
  if (!a || (a->x ? (a->tiles1 && !a->gain1) || (a->tiles2 && !a->gain2) : (a->tiles1 && !a->n1) || (a->tiles2 && !a->n2)) ||
      (a->tiles1 && (!a->w1 || !a->y1)) || (a->tiles2 && (!a->w2 || !a->gated)))
    return fail(AJQ_ERR_NULL, "ajqd_dense_in: null pointer argument");
  if (a->batch < 1 || a->true_width < 1 || a->width < a->true_width || a->width % 8 || a->tiles1 < 0 || a->tiles2 < 0 ||
      a->tiles1 + a->tiles2 < 1 || (a->tiles2 && (a->gated_ld < 8 * a->tiles2 || a->gated_ld % 4)))
    return fail(AJQ_ERR_SHAPE, "ajqd_dense_in: unsupported shape (batch=%d width=%d/%d tiles=%d+%d)", a->batch, a->true_width,
                a->width, a->tiles1, a->tiles2);
  if (a->act < 0 || a->act > AJQD_ACT_GELU_TANH) return fail(AJQ_ERR_UNSUPPORTED, "ajqd_dense_in: unknown activation");
  if (a->x && a->batch > 4) return fail(AJQ_ERR_UNSUPPORTED, "ajqd_dense_in: the norm prologue takes at most 4 rows");
  DenseIn d;
  d.x = a->x; d.n1 = (const uint16_t*)a->n1; d.n2 = (const uint16_t*)a->n2; d.gain1 = a->gain1; d.gain2 = a->gain2;
  d.w1 = (const uint16_t*)a->w1; d.w2 = (const uint16_t*)a->w2; d.y1 = a->y1; d.gated = (uint16_t*)a->gated;
  d.batch = a->batch; d.D = a->true_width; d.Dp = a->width; d.tiles1 = a->tiles1; d.tiles2 = a->tiles2;
  d.gated_ld = a->gated_ld; d.act = a->act; d.center = a->center; d.eps = a->eps;
  // more than 16 sequences: two batch tiles and (from two tiles of rows on) two row tiles per workgroup
  const bool wide = a->batch > kGemvBatch;
  const int block = wide ? 2 * kGemvBatch : kGemvBatch;
  const int rt = wide && a->tiles1 != 1 && a->tiles2 != 1 ? 2 : 1;
  const dim3 grid((a->tiles1 + rt - 1) / rt + (a->tiles2 + rt - 1) / rt, (a->batch + block - 1) / block);
  const int bytes = a->x ? 2 * a->batch * (a->width + 8) : 0;
  auto go = [&](auto kernel, int threads) {
    if (int e = allow_lds(kernel, bytes, "ajqd_dense_in")) return e;
    hipLaunchKernelGGL(kernel, grid, dim3(threads), bytes, (hipStream_t)stream, d);
    return check_launch("ajqd_dense_in");
  };
  const int waves = gemv_waves(a->width);
  if (a->x) return waves == 8 ? go(dense_in_kernel<8, true, 1, 1>, 512) : waves == 4 ? go(dense_in_kernel<4, true, 1, 1>, 256)
                                                                                     : go(dense_in_kernel<1, true, 1, 1>, 64);
  if (rt == 2) return waves == 8 ? go(dense_in_kernel<8, false, 2, 2>, 512) : waves == 4 ? go(dense_in_kernel<4, false, 2, 2>, 256)
                                                                                         : go(dense_in_kernel<1, false, 2, 2>, 64);
  if (wide) return waves == 8 ? go(dense_in_kernel<8, false, 1, 2>, 512) : waves == 4 ? go(dense_in_kernel<4, false, 1, 2>, 256)
                                                                                      : go(dense_in_kernel<1, false, 1, 2>, 64);
  return waves == 8 ? go(dense_in_kernel<8, false, 1, 1>, 512) : waves == 4 ? go(dense_in_kernel<4, false, 1, 1>, 256)
                                                                            : go(dense_in_kernel<1, false, 1, 1>, 64);
}

int ajqd_dense_out(const void* in, const void* w, float* x, const float* again, const float* step, int batch, int k,
                   int width, void* stream) {
  if (!in || !w || !x) return fail(AJQ_ERR_NULL, "ajqd_dense_out: null pointer argument");
  if (batch < 1 || k < 8 || k % 8 || width < 16 || width % 16)
    return fail(AJQ_ERR_SHAPE, "ajqd_dense_out: unsupported shape (batch=%d k=%d width=%d)", batch, k, width);
  DenseOut d{(const uint16_t*)in, (const uint16_t*)w, x, again, step, batch, k, width};
  const bool wide = batch > kGemvBatch;
  const int block = wide ? 2 * kGemvBatch : kGemvBatch;
  const int rt = wide && width % 32 == 0 && width >= 8192 ? 2 : 1;
  const dim3 grid(width / (16 * rt), (batch + block - 1) / block);
  auto go = [&](auto kernel, int threads) {
    hipLaunchKernelGGL(kernel, grid, dim3(threads), 0, (hipStream_t)stream, d);
    return check_launch("ajqd_dense_out");
  };
  const int waves = gemv_waves(k);
  if (rt == 2) return waves == 8 ? go(dense_out_kernel<8, 2, 2>, 512) : waves == 4 ? go(dense_out_kernel<4, 2, 2>, 256)
                                                                                   : go(dense_out_kernel<1, 2, 2>, 64);
  if (wide) return waves == 8 ? go(dense_out_kernel<8, 1, 2>, 512) : waves == 4 ? go(dense_out_kernel<4, 1, 2>, 256)
                                                                                : go(dense_out_kernel<1, 1, 2>, 64);
  return waves == 8 ? go(dense_out_kernel<8, 1, 1>, 512) : waves == 4 ? go(dense_out_kernel<4, 1, 1>, 256)
                                                                      : go(dense_out_kernel<1, 1, 1>, 64);
}

int ajqd_latent_absorb(const float* y, int ldy, const ajqd_latent_shape* shape, const void* ukt, const float* latent_gain,
                       const float* cosine, const float* sine, int table_rows, const int64_t* pos, void* q, void* ring, int cap,
                       int batch, void* stream) {
  if (int e = check_shape(shape, "ajqd_latent_absorb")) return e;
  if (!y || !ukt || !latent_gain || !cosine || !sine || !pos || !q || !ring)
    return fail(AJQ_ERR_NULL, "ajqd_latent_absorb: null pointer argument");
  if (batch < 1 || cap < 1 || table_rows < 1 || ldy % 4 ||
      ldy < shape->heads * (shape->dimp + shape->rotp) + shape->rankp + shape->rotp + shape->heads)
    return fail(AJQ_ERR_SHAPE, "ajqd_latent_absorb: unsupported shape (batch=%d cap=%d ldy=%d)", batch, cap, ldy);
  const int groups = (shape->rankp / 16 + 3) / 4;
  LatentAbsorb d{y, (const uint16_t*)ukt, latent_gain, cosine, sine, positions64(pos), (uint16_t*)q, (uint16_t*)ring,
                 batch, ldy, table_rows, cap, groups, device_shape(shape)};
  hipLaunchKernelGGL(latent_absorb_kernel, dim3(shape->heads * groups + 4, (batch + kGemvBatch - 1) / kGemvBatch), dim3(256), 0,
                     (hipStream_t)stream, d);
  return check_launch("ajqd_latent_absorb");
}

int ajqd_latent_decode_chunks(int batch, int heads, int rankp, int rotp, int cap) {
  if (batch < 1 || heads < 1 || cap < 1 || rankp < 16 || rankp % 16 || rotp < 8 || rotp % 8 || !latent_tiles(rankp) ||
      !latent_steps(rankp + rotp))
    return 0;
  const int groups = batch * latent_head_groups(heads);
  int s = (kDecodeWorkgroups + groups - 1) / groups;
  const int by_rows = (cap + kLatentRows - 1) / kLatentRows;
  if (s > by_rows) s = by_rows;
  return s < 1 ? 1 : s > kLatentMaxChunks ? kLatentMaxChunks : s;
}

size_t ajqd_latent_decode_workspace(int batch, int heads, int rankp, int chunks) {
  if (batch < 1 || heads < 1 || rankp < 1 || chunks < 1) return 0;
  return 4 * (size_t)latent_sums_at(batch, 0, 0, heads, chunks, rankp) + 8 * (size_t)batch * heads * chunks;
}

int ajqd_latent_decode(const void* q, const void* ring, const int64_t* pos, float* partial, int batch, int heads, int rankp,
                       int rotp, int cap, int chunks, float scale, void* stream) {
  if (!q || !ring || !pos || !partial) return fail(AJQ_ERR_NULL, "ajqd_latent_decode: null pointer argument");
  if (ajqd_latent_decode_chunks(batch, heads, rankp, rotp, cap) == 0)
    return fail(AJQ_ERR_UNSUPPORTED, "ajqd_latent_decode: widths %d + %d are not built", rankp, rotp);
  if (chunks < 1 || chunks > kLatentMaxChunks || !(scale > 0.f))
    return fail(AJQ_ERR_SHAPE, "ajqd_latent_decode: unsupported shape (batch=%d chunks=%d)", batch, chunks);
  LatentDecode d{(const uint16_t*)q, (const uint16_t*)ring, positions64(pos), partial,
                 heads_at(partial, batch, heads, chunks, rankp), batch, heads, rankp, rankp + rotp, cap, chunks, scale * kLog2eF};
  const long long blocks = (long long)latent_head_groups(heads) * chunks * batch;
  if (blocks > 0x7FFFFFFFll) return fail(AJQ_ERR_SHAPE, "ajqd_latent_decode: too many workgroups");
  const bool two = heads > 16;
  auto go = [&](auto kernel, int ks) {
    const int bytes = latent_decode_lds(ks, two ? 2 : 1);
    if (int e = allow_lds(kernel, bytes, "ajqd_latent_decode")) return e;
    hipLaunchKernelGGL(kernel, dim3((unsigned)blocks), dim3(two ? 512 : 256), bytes, (hipStream_t)stream, d);
    return check_launch("ajqd_latent_decode");
  };
  auto pick = [&](auto one, auto both, int ks) { return two ? go(both, ks) : go(one, ks); };
  const int tiles = latent_tiles(rankp);
#define AJQD_DECODE(KS, RT) pick(latent_decode_kernel<KS, RT, 1>, latent_decode_kernel<KS, RT, 2>, KS)
  switch (latent_steps(rankp + rotp)) {
    case 4: return AJQD_DECODE(4, 2);  // (at most 128 columns: two tiles per wave)
    case 6: return tiles == 2 ? AJQD_DECODE(6, 2) : AJQD_DECODE(6, 3);
    case 10: return tiles == 2 ? AJQD_DECODE(10, 2) : tiles == 4 ? AJQD_DECODE(10, 4) : AJQD_DECODE(10, 5);
    default: return tiles == 2 ? AJQD_DECODE(18, 2) : tiles == 4 ? AJQD_DECODE(18, 4) : AJQD_DECODE(18, 8);
  }
#undef AJQD_DECODE
}

int ajqd_latent_expand(const float* partial, const float* sink, const float* gate, int gate_ld, const void* uv, void* out,
                       int out_ld, int batch, int heads, int chunks, int rankp, int vdimp, void* stream) {
  if (!partial || !uv || !out) return fail(AJQ_ERR_NULL, "ajqd_latent_expand: null pointer argument");
  if (batch < 1 || heads < 1 || chunks < 1 || chunks > kLatentMaxChunks || rankp < 16 || rankp % 16 || vdimp < 16 || vdimp % 16 ||
      out_ld < heads * vdimp || out_ld % 4)
    return fail(AJQ_ERR_SHAPE, "ajqd_latent_expand: unsupported shape (batch=%d heads=%d chunks=%d rankp=%d vdimp=%d)", batch,
                heads, chunks, rankp, vdimp);
  if (rankp > kExpandRank) return fail(AJQ_ERR_UNSUPPORTED, "ajqd_latent_expand: latents of %d are not built", rankp);
  const bool few = batch <= kExpandBatch;
  const int tw = few ? 2 : 8, groups = (vdimp / 16 + tw - 1) / tw, bytes = 2 * kExpandBatch * (rankp + 8);
  LatentExpand d{partial, heads_at(partial, batch, heads, chunks, rankp), sink, gate, (const uint16_t*)uv, (uint16_t*)out, batch, heads, chunks, rankp, vdimp, gate_ld, out_ld, groups};
  hipLaunchKernelGGL(few ? latent_expand_kernel<2> : latent_expand_kernel<8>, dim3(heads * groups, (batch + kExpandBatch - 1) / kExpandBatch), dim3(512), bytes,
                     (hipStream_t)stream, d);
  return check_launch("ajqd_latent_expand");
}

}  // extern "C"
