// C ABI of libajq_dense.so (include/ajq_dense.h): argument validation, launch geometry, error reporting.
#include <stdarg.h>
#include <stdio.h>

#include "../../include/ajq_dense.h"
#include "ajq_common.h"
#include "dense_kernels.h"
#include "latent_attention.h"
#include "dense_gemv_kernels.h"
#include "grouped_attention.h"
#include "scan_kernels.h"
#include "stream_kernels.h"

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
  if (!a || !a->q || !a->k1 || (a->d2 && !a->k2) || !a->v || !a->out) return fail(AJQ_ERR_NULL, "%s: null pointer argument", what);
  if (a->batch < 1 || a->heads < 1 || a->seq < 1 || a->rows < 1 || a->prior < 0 || a->d1 < 8 || a->d2 < 0 || a->dv < 16 ||
      a->d1 % 8 || a->d2 % 8 || a->dv % 16 || a->out_ld < a->heads * a->dv || a->out_ld % 4 || a->keep < 0 || a->share < 0 ||
      (a->share > 1 && a->heads % a->share) || (a->column_gates && (a->gate_ld < a->heads * a->dv || a->gate_ld % 4)))
    return fail(AJQ_ERR_SHAPE, "%s: unsupported shape (B=%d H=%d T=%d rows=%d prior=%d d=%d+%d dv=%d)", what, a->batch, a->heads,
                a->seq, a->rows, a->prior, a->d1, a->d2, a->dv);
  if (a->pos ? a->seq != 1 : (long long)a->prior + a->seq > a->rows)
    return fail(AJQ_ERR_SHAPE, "%s: %d + %d queries do not fit %d rows", what, a->prior, a->seq, a->rows);
  if (!(a->scale > 0.f)) return fail(AJQ_ERR_SHAPE, "%s: the score scale must be positive", what);
  if (a->k1_row % 8 || a->k1_head % 8 || a->k2_row % 8 || a->v_row % 8 || a->v_head % 8 || a->k1_batch % 8 || a->k2_batch % 8 ||
      a->v_batch % 8 || !aligned16(a->q) || !aligned16(a->k1) || !aligned16(a->k2) || !aligned16(a->v) || !aligned16(a->out) || !aligned16(a->column_gates))
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
  w.keep = a->keep; w.share = a->share > 1 ? a->share : 1; w.gate_ld = a->gate_ld; w.column_gates = a->column_gates;
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
int latent_steps(int width) { const int s = (width + 31) / 32; return s <= 4 ? 4 : s <= 6 ? 6 : s <= 8 ? 8 : s <= 10 ? 10 : s <= 18 ? 18 : 0; }
// the chunks' sums, then (maximum, denominator) per head and chunk
float2* heads_at(const float* partial, int batch, int heads, int chunks, int rankp) {
  return reinterpret_cast<float2*>(const_cast<float*>(partial) + latent_sums_at(batch, 0, 0, heads, chunks, rankp));
}
constexpr int kDecodeWorkgroups = 256;  // one per CU (its LDS holds two blocks of rows)
int latent_head_groups(int heads) { return heads <= 16 ? 1 : (heads + 31) / 32; }  // one or two head tiles per workgroup
// ---- several residual streams
int stream_room(int s) { return s <= 2 ? 2 : s <= 4 ? 4 : kMaxStreams; }
int check_streams(int streams, const char* what) {
  if (streams < 1 || streams > kMaxStreams) return fail(AJQ_ERR_UNSUPPORTED, "%s: %d streams (1 .. %d are built)", what, streams, kMaxStreams);
  return AJQ_OK;
}

// ---- selective scan: lanes per channel and states per lane.  More lanes than the states ask for where there are few channels:
// the time loop is sequential, so what counts then is its length per step and not the work.
template <typename T>
int launch_scan(const Scan& a, int batch, hipStream_t stream) {
  const long long lanes = (long long)batch * a.inner;
  auto go = [&](auto kernel, int per_channel) {
    const int channels = 256 / per_channel;
    hipLaunchKernelGGL(kernel, dim3((a.inner + channels - 1) / channels, batch), dim3(256), 0, stream, a);
    return check_launch("ajqd_scan");
  };
  const bool few = lanes * 4 < 2 * 65536, fewer = lanes * 8 < 2 * 65536;  // (65536 lanes: a wave on every SIMD)
  const int n = a.states;
  if (n <= 16 && fewer) return go(scan_kernel<T, 16, 1>, 16);
  if (n <= 16 && few) return go(scan_kernel<T, 8, 2>, 8);
  if (n <= 16) return go(scan_kernel<T, 4, 4>, 4);
  if (n <= 32 && fewer) return go(scan_kernel<T, 16, 2>, 16);
  if (n <= 32 && few) return go(scan_kernel<T, 8, 4>, 8);
  if (n <= 24) return go(scan_kernel<T, 4, 6>, 4);
  if (n <= 32) return go(scan_kernel<T, 4, 8>, 4);
  if (n <= 64) return few ? go(scan_kernel<T, 16, 4>, 16) : go(scan_kernel<T, 8, 8>, 8);
  if (n <= 128) return go(scan_kernel<T, 16, 8>, 16);
  if (n <= 256) return go(scan_kernel<T, 32, 8>, 32);
  return fail(AJQ_ERR_UNSUPPORTED, "ajqd_scan: %d states per channel (up to 256 are built)", n);
}

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

int ajqd_ring_copy(void* ring, int cap, int kept, void* linear, int lines, int line_bytes, int first_row, int position, int count,
                   int row_bytes, int batch, int to_ring, void* stream) {
  if (!ring || !linear) return fail(AJQ_ERR_NULL, "ajqd_ring_copy: null pointer argument");
  if (cap < 1 || kept < 0 || kept > cap || count < 1 || first_row < 0 || (long long)first_row + count > lines || position < 0 ||
      batch < 1 || row_bytes < 16 || row_bytes % 16 || line_bytes < row_bytes || line_bytes % 16 ||
      (long long)position + count - (position > kept ? position : kept) > cap - kept)
    return fail(AJQ_ERR_SHAPE, "ajqd_ring_copy: unsupported shape (cap=%d lines=%d first=%d position=%d count=%d)", cap, lines,
                first_row, position, count);
  if (!aligned16(ring) || !aligned16(linear)) return fail(AJQ_ERR_ALIGN, "ajqd_ring_copy: buffers must be 16-byte aligned");
  const long long blocks = ((long long)batch * count * (row_bytes / 16) + 255) / 256;
  if (blocks > 0x7FFFFFFFll) return fail(AJQ_ERR_SHAPE, "ajqd_ring_copy: too many elements");
  hipLaunchKernelGGL(ring_copy_kernel, dim3((unsigned)blocks), dim3(256), 0, (hipStream_t)stream, (u32x4_t*)ring, cap, kept,
                     (u32x4_t*)linear, lines, line_bytes / 16, first_row, position, count, row_bytes / 16, batch, to_ring);
  return check_launch("ajqd_ring_copy");
}

int ajqd_gated_activation(const void* y, int y_dtype, void* out, int out_ld, int rows, int width, int act, int dtype,
                          void* stream) {
  if (!y || !out) return fail(AJQ_ERR_NULL, "ajqd_gated_activation: null pointer argument");
  if (rows < 1 || width < 8 || width % 8 || out_ld < width || out_ld % 4)
    return fail(AJQ_ERR_SHAPE, "ajqd_gated_activation: unsupported shape (rows=%d width=%d out_ld=%d)", rows, width, out_ld);
  if (!known(dtype) || !known(y_dtype) || act < 0 || act > AJQD_ACT_SQUARED_RELU)
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
  return d1 >= 8 && d2 >= 0 && d1 % 8 == 0 && d2 % 8 == 0 && dv >= 16 && dv % 16 == 0 && prefill_ks(d1 + d2) && prefill_vt(dv);
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
      a->tiles1 + a->tiles2 < 1 || (a->tiles2 && (a->gated_ld < (a->pairs ? 8 : 16) * a->tiles2 || a->gated_ld % 4)))
    return fail(AJQ_ERR_SHAPE, "ajqd_dense_in: unsupported shape (batch=%d width=%d/%d tiles=%d+%d)", a->batch, a->true_width,
                a->width, a->tiles1, a->tiles2);
  if (a->act < 0 || a->act > AJQD_ACT_SQUARED_RELU) return fail(AJQ_ERR_UNSUPPORTED, "ajqd_dense_in: unknown activation");
  if (a->x && a->batch > 4) return fail(AJQ_ERR_UNSUPPORTED, "ajqd_dense_in: the norm prologue takes at most 4 rows");
  DenseIn d;
  d.x = a->x; d.n1 = (const uint16_t*)a->n1; d.n2 = (const uint16_t*)a->n2; d.gain1 = a->gain1; d.gain2 = a->gain2;
  d.w1 = (const uint16_t*)a->w1; d.w2 = (const uint16_t*)a->w2; d.y1 = a->y1; d.gated = (uint16_t*)a->gated;
  d.batch = a->batch; d.D = a->true_width; d.Dp = a->width; d.tiles1 = a->tiles1; d.tiles2 = a->tiles2;
  d.gated_ld = a->gated_ld; d.act = a->act; d.center = a->center; d.pairs = a->pairs; d.eps = a->eps;
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
                       int rotp, int cap, int chunks, int first_column, float scale, void* stream) {
  if (!q || !ring || !pos || !partial) return fail(AJQ_ERR_NULL, "ajqd_latent_decode: null pointer argument");
  if (ajqd_latent_decode_chunks(batch, heads, rankp, rotp, cap) == 0)
    return fail(AJQ_ERR_UNSUPPORTED, "ajqd_latent_decode: widths %d + %d are not built", rankp, rotp);
  if (chunks < 1 || chunks > kLatentMaxChunks || first_column < 0 || first_column >= rankp + rotp || !(scale > 0.f))
    return fail(AJQ_ERR_SHAPE, "ajqd_latent_decode: unsupported shape (batch=%d chunks=%d)", batch, chunks);
  LatentDecode d{(const uint16_t*)q, (const uint16_t*)ring, positions64(pos), partial,
                 heads_at(partial, batch, heads, chunks, rankp), batch, heads, rankp, rankp + rotp, cap, chunks, first_column / 32, scale * kLog2eF};
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
    case 8: return tiles == 2 ? AJQD_DECODE(8, 2) : AJQD_DECODE(8, 4);
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

// ---- several residual streams
int ajqd_embed_streams(const int64_t* tokens, int rows, const void* table, int vocab, const float* in, float* x, float* u, int streams,
                       int width, int dtype, void* stream) {
  if (!tokens || !table || !x || (u && !in)) return fail(AJQ_ERR_NULL, "ajqd_embed_streams: null pointer argument");
  if (int e = check_streams(streams, "ajqd_embed_streams")) return e;
  if (rows < 1 || vocab < 1 || width < 8 || width % 8)
    return fail(AJQ_ERR_SHAPE, "ajqd_embed_streams: unsupported shape (rows=%d vocab=%d width=%d)", rows, vocab, width);
  if (!known(dtype)) return fail(AJQ_ERR_UNSUPPORTED, "ajqd_embed_streams: unknown dtype %d", dtype);
  with_types(dtype, dtype, [&](auto t, auto) {
    using T = decltype(t);
    hipLaunchKernelGGL(embed_streams_kernel<T>, dim3(rows), dim3(256), 0, (hipStream_t)stream, (const long long*)tokens, (const T*)table,
                       vocab, in, x, u, streams, width);
  });
  return check_launch("ajqd_embed_streams");
}

int ajqd_streams_norm(float* x, const float* delta, const float* scale, const float* out, const float* mix, const float* in,
                      const float* gain, float eps, void* normed, float* u, int streams, int rows, int true_width, int width, int dtype,
                      void* stream) {
  if (!x || (delta && (!scale || !out || !mix)) || (normed && !gain)) return fail(AJQ_ERR_NULL, "ajqd_streams_norm: null pointer argument");
  if (int e = check_streams(streams, "ajqd_streams_norm")) return e;
  if (rows < 1 || true_width < 1 || width < true_width || width % 8)
    return fail(AJQ_ERR_SHAPE, "ajqd_streams_norm: unsupported shape (rows=%d width=%d of %d)", rows, true_width, width);
  if (!known(dtype)) return fail(AJQ_ERR_UNSUPPORTED, "ajqd_streams_norm: unknown dtype %d", dtype);
  with_types(dtype, dtype, [&](auto t, auto) {
    using T = decltype(t);
    auto go = [&](auto kernel) {
      hipLaunchKernelGGL(kernel, dim3(rows), dim3(256), 0, (hipStream_t)stream, x, delta, scale, out, mix, in, gain, eps, (T*)normed, u,
                         streams, true_width, width);
    };
    switch (stream_room(streams)) {
      case 2: go(streams_norm_kernel<T, 2>); break;
      case 4: go(streams_norm_kernel<T, 4>); break;
      default: go(streams_norm_kernel<T, kMaxStreams>); break;
    }
  });
  return check_launch("ajqd_streams_norm");
}

int ajqd_dense_out_streams(const void* in, const void* w, float* x, const float* scale, const float* out, const float* mix,
                           const float* next, float* u, int streams, int batch, int k, int width, void* stream) {
  if (!in || !w || !x || !scale || !out || !mix || !u) return fail(AJQ_ERR_NULL, "ajqd_dense_out_streams: null pointer argument");
  if (int e = check_streams(streams, "ajqd_dense_out_streams")) return e;
  if (batch < 1 || k < 8 || k % 8 || width < 16 || width % 16)
    return fail(AJQ_ERR_SHAPE, "ajqd_dense_out_streams: unsupported shape (batch=%d k=%d width=%d)", batch, k, width);
  DenseOutStreams d{(const uint16_t*)in, (const uint16_t*)w, x, scale, out, mix, next, u, batch, k, width, streams};
  const bool wide = batch > kGemvBatch;
  const int block = wide ? 2 * kGemvBatch : kGemvBatch;
  const int rt = wide && width % 32 == 0 && width >= 8192 ? 2 : 1;
  const dim3 grid(width / (16 * rt), (batch + block - 1) / block);
  auto go = [&](auto kernel, int threads) {
    hipLaunchKernelGGL(kernel, grid, dim3(threads), 0, (hipStream_t)stream, d);
    return check_launch("ajqd_dense_out_streams");
  };
  auto pick = [&](auto room) {
    constexpr int M = decltype(room)::value;
    const int waves = gemv_waves(k);
    if (rt == 2) return waves == 8 ? go(dense_out_streams_kernel<8, 2, 2, M>, 512) : waves == 4 ? go(dense_out_streams_kernel<4, 2, 2, M>, 256)
                                                                                               : go(dense_out_streams_kernel<1, 2, 2, M>, 64);
    if (wide) return waves == 8 ? go(dense_out_streams_kernel<8, 1, 2, M>, 512) : waves == 4 ? go(dense_out_streams_kernel<4, 1, 2, M>, 256)
                                                                                            : go(dense_out_streams_kernel<1, 1, 2, M>, 64);
    return waves == 8 ? go(dense_out_streams_kernel<8, 1, 1, M>, 512) : waves == 4 ? go(dense_out_streams_kernel<4, 1, 1, M>, 256)
                                                                                  : go(dense_out_streams_kernel<1, 1, 1, M>, 64);
  };
  switch (stream_room(streams)) {
    case 2: return pick(std::integral_constant<int, 2>{});
    case 4: return pick(std::integral_constant<int, 4>{});
    default: return pick(std::integral_constant<int, kMaxStreams>{});
  }
}

int ajqd_activation(const void* y, void* out, int64_t count, int act, int dtype, void* stream) {
  if (!y || !out) return fail(AJQ_ERR_NULL, "ajqd_activation: null pointer argument");
  if (count < 8 || count % 8 || count / 8 / 256 > 0x7FFFFFFFll) return fail(AJQ_ERR_SHAPE, "ajqd_activation: unsupported count %lld", (long long)count);
  if (!aligned16(y) || !aligned16(out)) return fail(AJQ_ERR_ALIGN, "ajqd_activation: buffers must be 16-byte aligned");
  if (!known(dtype) || act < 0 || act > AJQD_ACT_SQUARED_RELU) return fail(AJQ_ERR_UNSUPPORTED, "ajqd_activation: unknown dtype or activation");
  with_types(dtype, dtype, [&](auto t, auto) {
    using T = decltype(t);
    hipLaunchKernelGGL(activation_kernel<T>, dim3((unsigned)((count / 8 + 255) / 256)), dim3(256), 0, (hipStream_t)stream, (const T*)y, (T*)out,
                       (long long)count / 8, act);
  });
  return check_launch("ajqd_activation");
}

// ---- grouped-query attention
int ajqd_key_value_split(const ajqd_key_value_split_args* a, int y_dtype, int dtype, void* stream) {
  if (!a || !a->y || !a->q_gain || !a->k_gain || (a->rot && !a->half_turns) || !a->q || !a->rows)
    return fail(AJQ_ERR_NULL, "ajqd_key_value_split: null pointer argument");
  if (a->tokens < 1 || a->seq < 1 || a->tokens % a->seq || a->heads < 1 || a->groups < 1 || a->dim < 1 || a->dimp < a->dim || a->dimp % 16 ||
      a->rot < 0 || a->rot % 2 || a->rot > a->dim || a->start < 0 || a->ldy < (a->heads + a->groups) * a->dimp || a->ldy % 4 || a->q_at < 0 ||
      a->q_at % 4 || a->q_ld < a->q_at + a->dimp || a->q_ld % 4 || a->prior < 0 || a->rows_batch < 0 || a->rows_head < 0 || a->rows_batch % 8 ||
      a->rows_head % 8 || (a->pos ? (a->seq != 1 || a->cap < 1 || a->kept < 0 || a->kept >= a->cap) : (int64_t)a->start + a->seq > 0x7FFFFFFF))
    return fail(AJQ_ERR_SHAPE, "ajqd_key_value_split: unsupported shape (tokens=%d seq=%d heads=%d groups=%d dim=%d/%d rot=%d cap=%d kept=%d)",
                a->tokens, a->seq, a->heads, a->groups, a->dim, a->dimp, a->rot, a->cap, a->kept);
  const int64_t need = (int64_t)(a->pos ? a->cap : a->prior + a->seq) * 2 * a->dimp;
  if ((a->groups > 1 && a->rows_head < need) || (a->tokens > a->seq && a->rows_batch < need))
    return fail(AJQ_ERR_SHAPE, "ajqd_key_value_split: rows of neighbouring heads or sequences overlap");
  if (!known(dtype) || !known(y_dtype)) return fail(AJQ_ERR_UNSUPPORTED, "ajqd_key_value_split: unknown dtype");
  if (!aligned16(a->y) || !aligned16(a->q) || !aligned16(a->rows)) return fail(AJQ_ERR_ALIGN, "ajqd_key_value_split: rows must be 16-byte aligned");
  KeyValueSplit k;
  k.y = a->y; k.ldy = a->ldy; k.s = KeyValueShape{a->heads, a->groups, a->dim, a->dimp, a->rot, a->eps};
  k.q_gain = a->q_gain; k.k_gain = a->k_gain; k.half_turns = a->half_turns; k.start = a->start; k.pos = positions64(a->pos);
  k.seq = a->seq; k.prior = a->prior; k.cap = a->cap; k.kept = a->kept; k.q = a->q; k.q_ld = a->q_ld; k.q_at = a->q_at;
  k.rows = a->rows; k.rows_batch = a->rows_batch; k.rows_head = a->rows_head;
  const int bytes = 4 * 2 * ((a->rot / 2 + 3) & ~3);
  int status = AJQ_OK;
  with_types(y_dtype, dtype, [&](auto yt, auto t) {
    using Y = decltype(yt);
    using T = decltype(t);
    const bool quads = (a->rot / 2) % 4 == 0 && a->dimp <= 256;
    auto go = [&](auto lanes, auto whole) {
      constexpr int L = decltype(lanes)::value;
      auto kernel = key_value_split_kernel<Y, T, L, decltype(whole)::value>;
      // few tokens: a head per team, so that the heads of a token go side by side
      const int teams = 256 / L, slices = a->tokens < 256 ? (a->heads + a->groups + teams - 1) / teams : 1;
      status = allow_lds(kernel, bytes, "ajqd_key_value_split");
      if (status == AJQ_OK) hipLaunchKernelGGL(kernel, dim3(a->tokens, slices), dim3(256), bytes, (hipStream_t)stream, k);
    };
    auto pick = [&](auto whole) {
      if (a->dimp <= 64) go(std::integral_constant<int, 16>{}, whole);
      else if (a->dimp <= 128) go(std::integral_constant<int, 32>{}, whole);
      else go(std::integral_constant<int, 64>{}, whole);
    };
    if (quads) pick(std::true_type{});
    else pick(std::false_type{});
  });
  return status != AJQ_OK ? status : check_launch("ajqd_key_value_split");
}

int ajqd_group_merge(const float* partial, const float* gate, int gate_ld, void* out, int out_ld, int batch, int groups, int share,
                     int chunks, int dimp, void* stream) {
  if (!partial || !out) return fail(AJQ_ERR_NULL, "ajqd_group_merge: null pointer argument");
  if (batch < 1 || groups < 1 || share < 1 || chunks < 1 || chunks > kLatentMaxChunks || dimp < 16 || dimp % 16 || dimp > 1024 ||
      out_ld < groups * share * dimp || out_ld % 4 || (gate && (gate_ld < groups * share * dimp || gate_ld % 4)) ||
      (long long)batch * groups * share > 0x7FFFFFFFll)
    return fail(AJQ_ERR_SHAPE, "ajqd_group_merge: unsupported shape (batch=%d groups=%d share=%d chunks=%d dimp=%d)", batch, groups, share,
                chunks, dimp);
  GroupMerge m{partial, heads_at(partial, batch * groups, share, chunks, dimp), gate, (uint16_t*)out, groups, share, chunks, dimp, gate_ld, out_ld};
  hipLaunchKernelGGL(group_merge_kernel, dim3(batch * groups * share), dim3(256), 0, (hipStream_t)stream, m);
  return check_launch("ajqd_group_merge");
}

// ---- selective scan
int ajqd_conv_silu(const void* y, int ldy, void* ring, const float* weight, const float* bias, int start, const int64_t* pos, int rows,
                   int seq, int inner, int taps, void* out, int dtype, void* stream) {
  if (!y || !weight || !bias || !out || (!ring && taps > 1 && (start > 0 || pos))) return fail(AJQ_ERR_NULL, "ajqd_conv_silu: null pointer argument");
  if (rows < 1 || seq < 1 || rows % seq || inner < 8 || inner % 8 || taps < 1 || ldy < inner || ldy % 8 || start < 0 || (pos && seq != 1))
    return fail(AJQ_ERR_SHAPE, "ajqd_conv_silu: unsupported shape (rows=%d seq=%d inner=%d taps=%d ldy=%d)", rows, seq, inner, taps, ldy);
  if (!known(dtype)) return fail(AJQ_ERR_UNSUPPORTED, "ajqd_conv_silu: unknown dtype %d", dtype);
  if (!aligned16(y) || !aligned16(ring) || !aligned16(out)) return fail(AJQ_ERR_ALIGN, "ajqd_conv_silu: rows must be 16-byte aligned");
  const long long blocks = ((long long)rows * (inner / 8) + 255) / 256;
  if (blocks > 0x7FFFFFFFll) return fail(AJQ_ERR_SHAPE, "ajqd_conv_silu: too many elements");
  ConvSilu c{y, ldy, ring, weight, bias, start, positions64(pos), rows, seq, inner, taps, out};
  const long long run_blocks = ((long long)(rows / seq) * ((seq + kConvTokens - 1) / kConvTokens) * (inner / 8) + 255) / 256;
  with_types(dtype, dtype, [&](auto t, auto) {
    using T = decltype(t);
    auto run = [&](auto kernel) { hipLaunchKernelGGL(kernel, dim3((unsigned)run_blocks), dim3(256), 0, (hipStream_t)stream, c); };
    if (!pos && taps == 2) return run(conv_silu_run_kernel<T, 2>);
    if (!pos && taps == 3) return run(conv_silu_run_kernel<T, 3>);
    if (!pos && taps == 4) return run(conv_silu_run_kernel<T, 4>);
    hipLaunchKernelGGL(conv_silu_kernel<T>, dim3((unsigned)blocks), dim3(256), 0, (hipStream_t)stream, c);
  });
  return check_launch("ajqd_conv_silu");
}

int ajqd_scan(const ajqd_scan_args* a, int dtype, void* stream) {
  if (!a || !a->x || !a->dt || !a->low || !a->z || !a->a2 || !a->d || !a->dt_bias || !a->out || (!a->state && (a->start > 0 || a->pos)))
    return fail(AJQ_ERR_NULL, "ajqd_scan: null pointer argument");
  if (a->batch < 1 || a->batch > 65535 || a->seq < 1 || a->inner < 8 || a->inner % 8 || a->states < 4 || a->states % 4 || a->start < 0 ||
      a->dt_ld < a->inner || a->dt_ld % 8 || a->z_ld < a->inner || a->z_ld % 8 || a->out_ld < a->inner || a->out_ld % 8 || a->b_col < 0 ||
      a->c_col < 0 || a->low_ld < a->b_col + a->states || a->low_ld < a->c_col + a->states || (a->pos && a->seq != 1))
    return fail(AJQ_ERR_SHAPE, "ajqd_scan: unsupported shape (batch=%d seq=%d inner=%d states=%d)", a->batch, a->seq, a->inner, a->states);
  if (!known(dtype)) return fail(AJQ_ERR_UNSUPPORTED, "ajqd_scan: unknown dtype %d", dtype);
  if (!aligned16(a->x) || !aligned16(a->dt) || !aligned16(a->z) || !aligned16(a->out) || !aligned16(a->d) || !aligned16(a->dt_bias))
    return fail(AJQ_ERR_ALIGN, "ajqd_scan: rows must be 16-byte aligned");
  Scan s{a->x, a->dt, a->low, a->z, a->a2, a->d, a->dt_bias, a->state, a->start, positions64(a->pos), a->seq, a->inner, a->states,
         a->dt_ld, a->low_ld, a->b_col, a->c_col, a->z_ld, a->out_ld, a->out};
  return dtype == AJQD_BF16 ? launch_scan<uint16_t>(s, a->batch, (hipStream_t)stream) : launch_scan<float>(s, a->batch, (hipStream_t)stream);
}

int ajqd_scan_splits(int batch, int inner) {
  (void)batch;
  const int s = (inner + kScanBlock - 1) / kScanBlock;
  return s < 1 ? 1 : s > 8 ? 8 : s;
}

int ajqd_scan_project(const float* y, int ldy, const void* ring, const float* weight, const float* bias, const int64_t* pos, const void* w,
                      float* partial, int batch, int inner, int taps, int rows, int splits, void* stream) {
  if (!y || !weight || !bias || !pos || !w || !partial || (!ring && taps > 1)) return fail(AJQ_ERR_NULL, "ajqd_scan_project: null pointer argument");
  if (batch < 1 || inner < 8 || inner % 8 || taps < 1 || rows < 16 || rows % 16 || splits < 1 || splits > 65535 || ldy < 2 * inner || ldy % 4)
    return fail(AJQ_ERR_SHAPE, "ajqd_scan_project: unsupported shape (batch=%d inner=%d taps=%d rows=%d splits=%d)", batch, inner, taps, rows, splits);
  ScanProject p{y, (const uint16_t*)ring, weight, bias, positions64(pos), (const uint16_t*)w, partial, batch, ldy, inner, taps, rows, splits};
  const int rt = batch > 4 && rows >= 32 ? 2 : 1;
  const dim3 grid((rows / 16 + rt - 1) / rt, splits, (batch + kGemvBatch - 1) / kGemvBatch);
  auto go = [&](auto kernel) { hipLaunchKernelGGL(kernel, grid, dim3(256), 0, (hipStream_t)stream, p); };
  if (taps == 4) rt == 2 ? go(scan_project_kernel<2, 4>) : go(scan_project_kernel<1, 4>);
  else rt == 2 ? go(scan_project_kernel<2, 0>) : go(scan_project_kernel<1, 0>);
  return check_launch("ajqd_scan_project");
}

int ajqd_scan_step(const ajqd_scan_step_args* a, void* stream) {
  if (!a || !a->y || !a->weight || !a->bias || !a->pos || !a->partial || !a->w_dt || !a->dt_bias || !a->a2 || !a->d || !a->state || !a->out ||
      (!a->ring && a->taps > 1))
    return fail(AJQ_ERR_NULL, "ajqd_scan_step: null pointer argument");
  if (a->batch < 1 || a->inner < 16 || a->inner % 16 || a->taps < 1 || a->rank < 8 || a->rank % 8 || a->states < 4 || a->states % 4 ||
      a->rows < a->rank + 2 * a->states || a->splits < 1 || a->ldy < 2 * a->inner || a->out_ld < a->inner)
    return fail(AJQ_ERR_SHAPE, "ajqd_scan_step: unsupported shape (batch=%d inner=%d rank=%d states=%d rows=%d)", a->batch, a->inner, a->rank,
                a->states, a->rows);
  ScanStep s{a->y, (uint16_t*)a->ring, a->weight, a->bias, positions64(a->pos), a->partial, (const uint16_t*)a->w_dt, a->dt_bias, a->a2, a->d,
             a->state, (uint16_t*)a->out, a->batch, a->ldy, a->inner, a->taps, a->rows, a->splits, a->rank, a->states, a->out_ld};
  auto go = [&](auto kernel, int bb) {
    const int bytes = scan_step_lds(a->rank, a->states, bb);
    if (int e = allow_lds(kernel, bytes, "ajqd_scan_step")) return e;
    hipLaunchKernelGGL(kernel, dim3((a->inner + 63) / 64, (a->batch + bb - 1) / bb), dim3(256), bytes, (hipStream_t)stream, s);
    return check_launch("ajqd_scan_step");
  };
  return a->batch > 16 ? go(scan_step_kernel<8>, 8) : go(scan_step_kernel<4>, 4);
}

}  // extern "C"
