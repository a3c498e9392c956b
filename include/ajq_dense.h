/*
 * ajq_dense -- operators of the dense (unquantized) model family, libajq_dense.so.
 *
 * Weights and activations are bf16 or fp32 (`dtype`); the residual stream, norm statistics, rotary tables, attention
 * scores and sums, gates and logits are fp32 in both.  All pointers are device pointers unless said otherwise; calls are
 * asynchronous on `stream`, allocate nothing and keep no pointer.  Return value: 0 or a negative status as in ajq.h
 * (ajqd_last_error() gives the calling thread's message).
 *
 * Widths: every row width is a multiple of 8, projection outputs of 16; columns past a model's own width are zero.
 * `pos` (int64, device) where a call takes one: the position of the step's one token per sequence, read by the kernel, so
 * that a recorded graph can be replayed; the ring cache's slot is position % cap.
 */
#ifndef AJQ_DENSE_H
#define AJQ_DENSE_H

#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

#define AJQD_BF16 0
#define AJQD_F32 1

#define AJQD_ACT_RELU 0
#define AJQD_ACT_SILU 1
#define AJQD_ACT_GELU_TANH 2
#define AJQD_ACT_SQUARED_RELU 3

const char* ajqd_last_error(void);

/* x[m] = table[tokens[m]] + positions[start + m % seq] (+ extra); `embedded` (optional) keeps the sum without extra.
 * With pos the position is *pos (seq = 1).  table [vocab, width], positions [table_rows, width] in dtype; rest fp32. */
int ajqd_embed(const int64_t* tokens, int rows, int seq, const void* table, int vocab, const void* positions,
               int table_rows, int start, const int64_t* pos, const float* extra, float* x, float* embedded, int width,
               int dtype, void* stream);

/* x += delta + again + step (each optional, written back), then out_j = norm(x) * gain_j for j = 1, 2 (each optional):
 * layer norm without bias (center = 1) or RMS norm (center = 0), statistics over the first `true_width` columns.
 * delta [rows, width] in delta_dtype; again [rows, width], step [width] fp32; out in dtype. */
int ajqd_add_norms(float* x, const void* delta, int delta_dtype, const float* again, const float* step,
                   const float* gain1, const float* gain2, float eps, int center, void* out1, void* out2, int rows,
                   int true_width, int width, int dtype, void* stream);

typedef struct {
  int32_t heads, dimp, rot, rotp, rank, rankp;  /* dim, rot_dim, kv_rank; the p ones padded */
  float eps;
} ajqd_latent_shape;

/* Splits projection rows y [rows, ldy] = (q: heads x (dimp | rotp), latent: rankp | rotp, gates: heads) into unrotated
 * queries qu (qu_ld elements per head), rotated queries qr (qr_ld per head), cache rows (RMS-normed latent | rotated key
 * part) at cache_rows[b * rows_batch + slot * (rankp + rotp)] and gates = sigmoid.  y in y_dtype, qu / qr / cache rows in
 * dtype.  slot = prior + t at position start + t, or (pos) slot *pos % cap.  Rotation pairs i with i + rot / 2. */
int ajqd_latent_split(const void* y, int y_dtype, int ldy, const ajqd_latent_shape* shape, const float* latent_gain,
                      const float* cosine, const float* sine, int table_rows, int rows, int seq, int start, const int64_t* pos,
                      int prior, int cap, void* qu, int qu_ld, void* qr, int qr_ld, void* cache_rows, int64_t rows_batch,
                      float* gates, int dtype, void* stream);

/* Copies `count` rows of `row_bytes` (a multiple of 16) per sequence between a ring [batch, cap, row] and rows first_row ..
 * of a linear buffer [batch, lines, line], from `position` on.  The ring's first `kept` positions stay: p < kept is in slot p,
 * the others in kept + (p - kept) % (cap - kept); no slot may be met twice. */
int ajqd_ring_copy(void* ring, int cap, int kept, void* linear, int lines, int line_bytes, int first_row, int position, int count,
                   int row_bytes, int batch, int to_ring, void* stream);

/* out[m, f] = act(gate) * up; y [rows, 2 * width] in blocks of 8 gate columns and their 8 up columns. */
int ajqd_gated_activation(const void* y, int y_dtype, void* out, int out_ld, int rows, int width, int act, int dtype,
                          void* stream);

/* y[b, g, n] = sum_k w[g, n, k] x[b, g, k]; w [groups, n, k]; strides in elements. */
int ajqd_matvec(const void* w, const void* x, int x_batch, int x_group, void* y, int y_batch, int y_group, int groups,
                int n, int k, int batch, int dtype, int out_dtype, void* stream);

typedef struct {
  const void *q, *k1, *k2, *v;
  const float *sink, *gates;
  const void* column_gates;
  const int64_t* pos;
  void* out;
  int64_t k1_batch, k2_batch, v_batch, k1_head, v_head;
  int32_t k1_row, k2_row, v_row;
  int32_t d1, d2, dv;
  int32_t batch, heads, share, seq;
  int32_t rows, prior, window, keep, gate_ld, out_ld;
  float scale;
} ajqd_windowed_attention_args;

/* out[b, t, h] = gate * sum_j exp(s_j) v_j / (exp(sink_h) + sum_j exp(s_j)), s_j = (q1 . k1_j + q2 . k2_j) * scale.
 * q [batch * seq, heads, d1 + d2].  Query t sits at row prior + t of the key / value buffers (`rows` rows per sequence)
 * and sees rows max(0, prior + t - window + 1) .. prior + t (window <= 0: all before it) and rows 0 .. keep - 1 up to its own;
 * with pos it sees the first min(*pos + 1, rows) rows.  gate: gates[m, h] and / or sigmoid(column_gates[m, h * dv + c]) (row
 * stride gate_ld, in dtype).  `share` heads use one key / value head (0: as 1).  d1, d2 multiples of 8 (d2 = 0: no shared
 * part), dv of 16.  q, k1, k2, v in dtype, out in out_dtype. */
int ajqd_windowed_attention(const ajqd_windowed_attention_args* args, int dtype, int out_dtype, void* stream);

/* The same for bf16 prompts (no pos) on MFMA; ajqd_windowed_prefill_supported says for which widths. */
int ajqd_windowed_prefill_supported(int d1, int d2, int dv);
int ajqd_windowed_prefill(const ajqd_windowed_attention_args* args, void* stream);

/* ---- one decode step in bf16 (see the kernels for the layouts) ---- */
typedef struct {
  const float* x;
  const void *n1, *n2;
  const float *gain1, *gain2;
  const void *w1, *w2;
  float* y1;
  void* gated;
  int32_t batch, true_width, width, tiles1, tiles2, gated_ld, act, center, pairs;
  float eps;
} ajqd_dense_in_args;
/* y1 = norm1(x) w1^T (fp32), gated = act(norm2(x) w_gate^T) * (norm2(x) w_up^T) (bf16; w2 holds both in blocks of 8 rows), or
 * act(norm2(x) w2^T) with pairs = 0.  With x the norms are formed by the
 * product's own workgroups (batch <= 4); with n1 / n2 the normed bf16 rows are read.  tiles: output rows / 16. */
int ajqd_dense_in(const ajqd_dense_in_args* args, void* stream);

/* x += in w^T (+ again) (+ step); in [batch, k] bf16, w [width, k] bf16, x / again [batch, width], step [width] fp32 */
int ajqd_dense_out(const void* in, const void* w, float* x, const float* again, const float* step, int batch, int k,
                   int width, void* stream);

/* queries into the latent space, and the step's row into the ring cache: y fp32 [batch, ldy] as in ajqd_latent_split,
 * ukt [heads, rankp, dimp] bf16 -> q [batch, heads, rankp + rotp], ring [batch, cap, rankp + rotp] bf16 */
int ajqd_latent_absorb(const float* y, int ldy, const ajqd_latent_shape* shape, const void* ukt, const float* latent_gain,
                       const float* cosine, const float* sine, int table_rows, const int64_t* pos, void* q, void* ring, int cap,
                       int batch, void* stream);

/* row chunks ajqd_latent_decode uses, 0 where these widths are not built; bytes of the partial results it leaves */
int ajqd_latent_decode_chunks(int batch, int heads, int rankp, int rotp, int cap);
size_t ajqd_latent_decode_workspace(int batch, int heads, int rankp, int chunks);
/* (query columns ahead of first_column are zero) */
int ajqd_latent_decode(const void* q, const void* ring, const int64_t* pos, float* partial, int batch, int heads, int rankp,
                       int rotp, int cap, int chunks, int first_column, float scale, void* stream);

/* merge of the chunks with the sink (fp32 [heads] or NULL), value expansion uv [heads, vdimp, rankp] bf16, output gate
 * sigmoid(gate[b * gate_ld + h]) (or NULL) -> out bf16 [batch, out_ld], head h at column h * vdimp */
int ajqd_latent_expand(const float* partial, const float* sink, const float* gate, int gate_ld, const void* uv, void* out,
                       int out_ld, int batch, int heads, int chunks, int rankp, int vdimp, void* stream);

/* ---- several residual streams: x [rows, streams, width] fp32; coefficients in, out [streams], mix [streams (from), streams
 * (to)] fp32 */
/* every stream = table[tokens[m]]; u (optional) = sum of `in` times it */
int ajqd_embed_streams(const int64_t* tokens, int rows, const void* table, int vocab, const float* in, float* x, float* u, int streams,
                       int width, int dtype, void* stream);
/* with delta [rows, width] fp32: x_t = sum_s mix[s, t] x_s + out[t] * scale * delta (scale [width]); then the weighted sum
 * sum_s in[s] x_s (in NULL: plain) -> u (optional) and, RMS-normed times gain, -> normed (optional, dtype) */
int ajqd_streams_norm(float* x, const float* delta, const float* scale, const float* out, const float* mix, const float* in,
                      const float* gain, float eps, void* normed, float* u, int streams, int rows, int true_width, int width, int dtype,
                      void* stream);
/* one decode step in bf16: the same update with delta = in w^T as its epilogue, u = sum_s next[s] x_s (next NULL: plain) */
int ajqd_dense_out_streams(const void* in, const void* w, float* x, const float* scale, const float* out, const float* mix,
                           const float* next, float* u, int streams, int batch, int k, int width, void* stream);

/* out = act(y), `count` (a multiple of 8) elements of dtype; may be in place */
int ajqd_activation(const void* y, void* out, int64_t count, int act, int dtype, void* stream);

/* ---- grouped-query attention whose values are the projected keys */
typedef struct {
  const void* y;
  const float *q_gain, *k_gain;
  const double* half_turns;
  const int64_t* pos;
  void *q, *rows;
  int64_t rows_batch, rows_head;
  int32_t tokens, seq, start, ldy, heads, groups, dim, dimp, rot, q_ld, q_at, prior, cap, kept;
  float eps;
} ajqd_key_value_split_args;
/* Splits projection rows y [tokens, ldy] = (queries: heads x dimp, keys: groups x dimp, ..): every query and key head is
 * RMS-normed over dim (gains [dimp], zero past dim) and its first `rot` components rotated, i against i + rot / 2, by
 * position * half_turns[i] * pi.  Queries go to q [tokens, heads, q_ld] from column q_at (zeros ahead of it); a key
 * makes a row (key as projected | normed and rotated key) of 2 dimp elements at rows[b * rows_batch + group * rows_head + slot *
 * 2 dimp].  slot = prior + t at position start + t, or (pos) the position's slot in a ring of cap rows, `kept` of which stay. */
int ajqd_key_value_split(const ajqd_key_value_split_args* args, int y_dtype, int dtype, void* stream);
/* merge of ajqd_latent_decode's chunks where a (sequence, key / value head) was a sequence of `share` heads and dimp the
 * latent's width; output gate sigmoid(gate[b * gate_ld + head * dimp + c]) (or NULL) -> out bf16 [batch, out_ld] */
int ajqd_group_merge(const float* partial, const float* gate, int gate_ld, void* out, int out_ld, int batch, int groups, int share,
                     int chunks, int dimp, void* stream);

/* ---- selective scan.  inner: channels, states per channel a multiple of 4; a state tensor and a2 = A log2(e) are stored
 * [states / 4, inner, 4] */
/* out [rows, inner] = silu(bias + sum_j weight[taps - 1 - j] y[t - j]) over y [rows, ldy]; positions ahead of start come from ring
 * [batch, taps - 1, inner] (slot = position % (taps - 1)); with pos the step's own row goes there too */
int ajqd_conv_silu(const void* y, int ldy, void* ring, const float* weight, const float* bias, int start, const int64_t* pos, int rows,
                   int seq, int inner, int taps, void* out, int dtype, void* stream);
typedef struct {
  const void *x, *dt, *low, *z;
  const float *a2, *d, *dt_bias;
  float* state;
  const int64_t* pos;
  void* out;
  int32_t batch, seq, start, inner, states, dt_ld, low_ld, b_col, c_col, z_ld, out_ld;
} ajqd_scan_args;
/* dt = softplus(dt + dt_bias); S = 2^(dt a2) S + dt x B; out = (S C + d x) silu(z), token by token; state (optional) is read
 * unless the first token's position is 0, and written.  x, dt, low (B | C), z, out in dtype, one row per token. */
int ajqd_scan(const ajqd_scan_args* args, int dtype, void* stream);
/* one decode step in bf16: y fp32 [batch, ldy] = (columns to convolve: inner | z: inner).  ajqd_scan_project convolves and
 * multiplies by w [rows, inner] = (dt rank | B | C | padding), leaving `splits` parts [splits, batch, rows];
 * ajqd_scan_step adds them and does the rest (w_dt [inner, rank]) -> out bf16 [batch, out_ld] */
int ajqd_scan_splits(int batch, int inner);
int ajqd_scan_project(const float* y, int ldy, const void* ring, const float* weight, const float* bias, const int64_t* pos, const void* w,
                      float* partial, int batch, int inner, int taps, int rows, int splits, void* stream);
typedef struct {
  const float* y;
  void* ring;
  const float *weight, *bias;
  const int64_t* pos;
  const float* partial;
  const void* w_dt;
  const float *dt_bias, *a2, *d;
  float* state;
  void* out;
  int32_t batch, ldy, inner, taps, rows, splits, rank, states, out_ld;
} ajqd_scan_step_args;
int ajqd_scan_step(const ajqd_scan_step_args* args, void* stream);

#ifdef __cplusplus
}
#endif
#endif /* AJQ_DENSE_H */
