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

/* Copies `count` rows of `row_bytes` (a multiple of 16) per sequence between a ring [batch, cap, row] (slot = position %
 * cap, from `position` on) and rows first_row .. of a linear buffer [batch, lines, row]; count <= cap. */
int ajqd_ring_copy(void* ring, int cap, void* linear, int lines, int first_row, int position, int count, int row_bytes,
                   int batch, int to_ring, void* stream);

/* out[m, f] = act(gate) * up; y [rows, 2 * width] in blocks of 8 gate columns and their 8 up columns. */
int ajqd_gated_activation(const void* y, int y_dtype, void* out, int out_ld, int rows, int width, int act, int dtype,
                          void* stream);

/* y[b, g, n] = sum_k w[g, n, k] x[b, g, k]; w [groups, n, k]; strides in elements. */
int ajqd_matvec(const void* w, const void* x, int x_batch, int x_group, void* y, int y_batch, int y_group, int groups,
                int n, int k, int batch, int dtype, int out_dtype, void* stream);

typedef struct {
  const void *q, *k1, *k2, *v;
  const float *sink, *gates;
  const int64_t* pos;
  void* out;
  int64_t k1_batch, k2_batch, v_batch;
  int32_t k1_row, k1_head, k2_row, v_row, v_head;
  int32_t d1, d2, dv;
  int32_t batch, heads, seq;
  int32_t rows, prior, window, out_ld;
  float scale;
} ajqd_windowed_attention_args;

/* out[b, t, h] = gate * sum_j exp(s_j) v_j / (exp(sink_h) + sum_j exp(s_j)), s_j = (q1 . k1_j + q2 . k2_j) * scale.
 * q [batch * seq, heads, d1 + d2].  Query t sits at row prior + t of the key / value buffers (`rows` rows per sequence)
 * and sees rows max(0, prior + t - window + 1) .. prior + t (window <= 0: all before it); with pos it sees the first
 * min(*pos + 1, rows) rows.  d1, d2 multiples of 8, dv of 16.  q, k1, k2, v in dtype, out in out_dtype. */
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
  int32_t batch, true_width, width, tiles1, tiles2, gated_ld, act, center;
  float eps;
} ajqd_dense_in_args;
/* y1 = norm1(x) w1^T (fp32), gated = act(norm2(x) w_gate^T) * (norm2(x) w_up^T) (bf16).  With x the norms are formed by the
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
int ajqd_latent_decode(const void* q, const void* ring, const int64_t* pos, float* partial, int batch, int heads, int rankp,
                       int rotp, int cap, int chunks, float scale, void* stream);

/* merge of the chunks with the sink (fp32 [heads] or NULL), value expansion uv [heads, vdimp, rankp] bf16, output gate
 * sigmoid(gate[b * gate_ld + h]) (or NULL) -> out bf16 [batch, out_ld], head h at column h * vdimp */
int ajqd_latent_expand(const float* partial, const float* sink, const float* gate, int gate_ld, const void* uv, void* out,
                       int out_ld, int batch, int heads, int chunks, int rankp, int vdimp, void* stream);

#ifdef __cplusplus
}
#endif
#endif /* AJQ_DENSE_H */
