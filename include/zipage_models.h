/* C ABI of the model-side kernels of decoders that need more than the compression library's layer
 * kernels.  Six shared objects, so that a model compiles only what it runs: libzipage_models.so (an
 * fp32 residual stream, attention of prompt runs), libzipage_latent.so (latent attention over pages of
 * latents), libzipage_grouped.so (grouped-query attention, with sinks or of two maps),
 * libzipage_recurrent.so (matrix memory, delta rule), libzipage_linear.so (linear attention with decay) and
 * libzipage_moe.so (mixtures of experts).  Status codes, dtype tags and conventions are those of zipage_hip.h; every entry point here takes ZP_BF16 or ZP_F32 (true 32-bit products), enqueues on
 * `stream`, allocates nothing and may be captured into a HIP graph. */
#ifndef ZIPAGE_MODELS_H
#define ZIPAGE_MODELS_H
#include "zipage_hip.h"

#ifdef __cplusplus
extern "C" {
#endif

/* ------------------------------------------------------------------ libzipage_models.so */

/* x = embed[tokens] * embed_scale (+ pos[positions] when pos is given), fp32, which goes to `result` when given,
 * (+ the row `shift`); with norm_weight also
 * out = x / sqrt(mean(x^2) + eps) * (weight_offset + norm_weight) or, with norm_bias,
 * out = tanh(norm_alpha * x) * (weight_offset + norm_weight) + norm_bias.  Rows are `width` long (multiple
 * of 8, zero padded), the mean runs over norm_width.  embed (vocab, width), pos (max_positions,
 * width) and out are of `dtype`; indices are clamped to the tables. */
int zp_embed_norm(const int64_t* tokens, const int32_t* positions, const void* embed, const void* pos,
                  const float* shift, float* result, float* x, const float* norm_weight,
                  const float* norm_bias, void* out, int32_t n, int32_t width, int32_t norm_width,
                  int64_t vocab, int64_t max_positions, float embed_scale, float eps, float weight_offset,
                  float norm_alpha, int32_t dtype, void* stream);

/* r = x + the branches (x (n, width) fp32; a branch is the sum of `planes` planes (n, width) of dtype, with
 * `weight` RMS-normed times that weight before it is added; up to three branches, two of them normed); written to
 * `result` when given; with a depth average
 * r <- mix[n_hist] * r + sum_{j < n_hist} mix[j] * hist[j] (hist: planes of (n, width) fp32,
 * hist_plane elements apart); plus the row `shift` when given; written to `x_out` when given; with norm_weight also
 * out = rmsnorm(r) * (weight_offset + norm_weight) * out_scale, or with norm_bias
 * out = (tanh(norm_alpha * r) * (weight_offset + norm_weight) + norm_bias) * out_scale.
 * mix NULL: no average. */
typedef struct {
  const void* y;
  const float* weight;
  int32_t planes;
} zp_branch;
int zp_residual_norm(const float* x, const zp_branch* branches, int32_t n_branches, const float* hist,
                     int64_t hist_plane, const float* mix, int32_t n_hist, const float* shift, float* result,
                     float* x_out, const float* norm_weight, const float* norm_bias, void* out, int32_t n,
                     int32_t width, int32_t norm_width, float eps, float weight_offset,
                     float norm_alpha, float out_scale, int32_t dtype, void* stream);

/* Rows z of `in` (in_stride elements apart): a N(z) + b N(z^2) + c N(z^3) + e, powers element by element, N(y) =
 * y / sqrt(mean(y^2) + eps) with the mean over the first norm_width elements; those behind them are zero. */
int zp_normed_powers(const void* in, void* out, int32_t n, int32_t width, int32_t norm_width,
                     int64_t in_stride, int64_t out_stride, float a, float b, float c, float e, float eps,
                     int32_t dtype, void* stream);

/* z > 0: alpha_p z^2 + z / 2;  z <= 0: alpha_n (exp(z) - 1 - z) + z / 2.  count % 8 == 0. */
int zp_xielu(const void* in, void* out, int64_t count, float alpha_p, float alpha_n, int32_t dtype,
             void* stream);

/* max(z, 0)^2.  count % 8 == 0. */
int zp_relu_square(const void* in, void* out, int64_t count, int32_t dtype, void* stream);

/* out (fp32) = cap * tanh(in / cap). */
int zp_softcap(const void* in, float* out, int64_t count, float cap, int32_t dtype, void* stream);

/* out[i] = src[rows[i]], rows of row_bytes (multiple of 16). */
int zp_gather_rows(const void* src, const int32_t* rows, void* out, int32_t n, int32_t row_bytes,
                   int64_t num_rows, void* stream);

/* What an attention does beyond the softmax of scaled products; NULL stands for {0, 1}.
 * softcap > 0: scores s (after the scale) enter the softmax as softcap * tanh(s / softcap).
 * maps 2 (differential attention): a query head holds two queries of D and a key head two keys of D, back to
 * back; both softmaxes weight the same values, and with their results o1, o2 the output is
 *   rms(o1 - balance * o2) * out_scale * sigmoid(gate),  rms over the first `vdim` values with eps,
 * gate (rows gate_stride elements apart, heads of V back to back, of the call's dtype) or NULL: no gate.
 * Sinks are for one map only.
 * turns: (rows of q, V / 2) pairs cos, sin of one map whose values turned by angles of their positions; elements 2 i
 * and 2 i + 1 of every head's output turn back by the query's.  16-byte aligned; NULL: nothing turns. */
typedef struct {
  float softcap;
  int32_t maps;
  float balance, eps;
  int32_t vdim;
  const void* gate;
  int64_t gate_stride;
  const float* turns;
} zp_attention_form;

/* Attention of runs of tokens, bfloat16.  tiles (T, 4) int32, one entry per up to 128 queries of one
 * sequence: first query row, number of queries, row of the run's first key, position of the first
 * query counted from that key (key rows of a run are consecutive positions).  Query head h reads key
 * head h / (H / HK).  A query sees its own position and those before it in the run that lie within
 * `window` (0: no limit) or, with `chunk`, in its own block of `chunk` positions (the run's first key
 * starts a block); at most one of the two is set.  sinks (H,) or NULL: a logit per head that joins the
 * denominator only.  q rows q_stride, k and v rows kv_stride, out rows out_stride elements apart, heads
 * back to back; out is multiplied by out_scale.  With k_shared (rows shared_stride apart) a query head is
 * D + P long and its last P elements meet the row of k_shared, whatever the head. */
int zp_run_attention(const void* q, const void* k, const void* v, const void* k_shared, void* out,
                     const int32_t* tiles, const float* sinks, const zp_attention_form* form, int32_t T,
                     int32_t H, int32_t HK, int32_t D, int32_t P, int32_t V, int32_t window,
                     int32_t chunk, int64_t q_rows, int64_t k_rows, int64_t q_stride, int64_t kv_stride,
                     int64_t shared_stride, int64_t out_stride, float scale, float out_scale,
                     int32_t dtype, void* stream);

/* ------------------------------------------------------------------ libzipage_latent.so */

/* in (n, q_width + c_width + p_width): the first part RMS-normed times q_weight goes to q_out; the second
 * times c_weight, and behind it the third, of which the first `rot` elements turn by positions[i] * freqs[.]
 * (j with j + rot / 2), go to slot slots[i] of the cache (-1 skips) and to c_out when given.  The means run
 * over q_norm and c_norm elements; widths are multiples of 8, zero padded.  c_width and p_width 0: the
 * first part alone. */
int zp_latent_norm_store(const void* in, const float* q_weight, const float* c_weight, void* q_out,
                         void* c_out, void* cache, const int32_t* slots, const int32_t* positions,
                         const float* freqs, int32_t n, int32_t q_width, int32_t c_width,
                         int32_t p_width, int32_t q_norm, int32_t c_norm, int32_t rot,
                         int64_t num_slots, float eps, int32_t dtype, void* stream);

/* x[i, h * head + at ...]: `rot` elements turn in place by positions[i] * freqs[.], j with j + rot / 2. */
int zp_rotate_heads(void* x, const int32_t* positions, const float* freqs, int32_t n, int32_t H,
                    int32_t head, int32_t at, int32_t rot, int64_t x_stride, int32_t dtype,
                    void* stream);

/* out[n, h, :M] = w[h] (M, K) in[n, h, :K]; heads of K + tail and M + tail elements.  The tail passes, its
 * first `rot` elements turned as in zp_rotate_heads.  K a multiple of 32, M of 16, tail of 8. */
int zp_headwise_linear(const void* in, const void* w, void* out, const int32_t* positions,
                       const float* freqs, int32_t n, int32_t H, int32_t K, int32_t M, int32_t tail,
                       int32_t rot, int32_t dtype, void* stream);

/* Attention of single tokens over paged latents.  q (n, H, R + P); cache (num_pages, BS, R + P); token i
 * sees the tokens [max(0, c - window), c) of its sequence, c = context_lens[i] (window 0: all;
 * c = 0: inert, zeros), through row table_rows[i] (NULL: i) of table (B, NB).
 * out[n, h] (R) = sum_j softmax_j(scale * q[n, h] . row_j) row_j[:R].  R a multiple of 32, P of 8.
 * `workspace`: zp_latent_rows_workspace() bytes, 16-byte aligned. */
int64_t zp_latent_rows_workspace(int32_t n, int32_t H, int32_t R, int32_t window, int32_t NB,
                                 int32_t BS, int32_t dtype);
int zp_latent_rows_attention(const void* q, const void* cache, const int32_t* table,
                             const int32_t* context_lens, const int32_t* table_rows, void* out,
                             int32_t n, int32_t H, int32_t R, int32_t P, int32_t BS, int32_t B,
                             int32_t NB, int32_t num_pages, int32_t window, float scale, int32_t dtype,
                             void* workspace, int64_t workspace_bytes, void* stream);

/* ------------------------------------------------------------------ libzipage_grouped.so */

/* What else a store of queries, keys and values does; NULL stands for nothing.
 * norm (H * D + HK * D): weights of RMS norms over the whole of q and the whole of k (means over q_norm and k_norm
 * elements), before they turn.
 * tied: the values are the keys as they are in `in`, which has no value columns; VT = HK * D.
 * value_freqs (V / 2): the values' heads of V turn too, elements 2 i and 2 i + 1 by positions[.] * value_freqs[i];
 * turns (n, V / 2) receives cos and sin of these angles. */
typedef struct {
  const float* norm;
  int32_t q_norm, k_norm;
  float eps;
  int32_t tied;
  int32_t V;
  const float* value_freqs;
  float* turns;
} zp_store_form;

/* Rows `in` (in_stride elements apart) hold q (H heads of D), k (HK of D) and VT value columns; with `bias`
 * (a row of them) it is added first.  The first `rot` dimensions of q's and k's heads turn by positions[i] *
 * freqs[.], dimension j with j + rot / 2.  q goes to q_out, [k | v] to slot slots[i] of the cache (-1
 * skips) and to kv_out when given. */
int zp_rotary_store(const void* in, const float* bias, const int32_t* positions, const float* freqs,
                    const zp_store_form* form, void* q_out, void* kv_out, void* cache, const int32_t* slots,
                    int32_t n, int32_t H, int32_t HK, int32_t D, int32_t VT, int32_t rot,
                    int64_t in_stride, int64_t num_slots, int32_t dtype, void* stream);

/* Attention of single tokens over paged rows [k (HK heads of maps * D) | v (HK of V)].  q (n, H, maps * D);
 * token i is the last of the context_lens[i] tokens of its sequence (0: inert, zeros) in row table_rows[i]
 * (NULL: i) of table (B, NB); window, chunk, sinks, form, out_stride and out_scale as in zp_run_attention,
 * with blocks counted from position 0.  `workspace`: zp_grouped_rows_workspace() bytes. */
int64_t zp_grouped_rows_workspace(int32_t n, int32_t H, int32_t HK, int32_t D, int32_t V, int32_t maps,
                                  int32_t window, int32_t chunk, int32_t NB, int32_t BS,
                                  int32_t dtype);
int zp_grouped_rows_attention(const void* q, const void* cache, const int32_t* table,
                              const int32_t* context_lens, const int32_t* table_rows,
                              const float* sinks, const zp_attention_form* form, void* out, int32_t n,
                              int32_t H, int32_t HK, int32_t D, int32_t V, int32_t BS, int32_t B,
                              int32_t NB, int32_t num_pages, int32_t window, int32_t chunk,
                              int64_t out_stride, float scale, float out_scale, int32_t dtype,
                              void* workspace, int64_t workspace_bytes, void* stream);

/* ------------------------------------------------------------------ libzipage_recurrent.so */

/* The runs of tokens a step holds, one per sequence: token rows row .. row + count - 1, the state slot,
 * the position of the first token (0: the state starts at zero).  rows NULL: row i; max_count > 0 caps
 * the counts; count 0 is inert. */
typedef struct {
  const int32_t *rows, *counts, *slots, *starts;
  int32_t n, max_count, num_slots, num_rows;
} zp_segments;

/* Matrix memory with exponential gates, and the normed, gated read-out.  Rows `in` hold q, k (heads of
 * dk), v, g (heads of dv) from columns q_at, k_at, v_at, g_at; gates (fp32) hold the input gates'
 * and then the forget gates' pre-activations.  dk 32, 64, 128 or 256, dv a multiple of 32 up to 256, zero
 * padded; the norm's mean runs over vdim.  state: (num_slots, heads, dk * dv + dk + 4) fp32. */
typedef struct {
  zp_segments seg;
  const void* in;
  const float *gates, *i_bias, *f_bias, *norm;
  float* state;
  void* out;
  int64_t in_stride, gate_stride, out_stride;
  int32_t heads, dk, dv, vdim, q_at, k_at, v_at, g_at;
  float cap, q_scale, eps, out_scale;
} zp_mlstm;
int zp_mlstm_scan(const zp_mlstm* args, int32_t dtype, void* stream);
/* The same for long runs, 16 tokens at a time on the matrix cores (fp32): bfloat16, dk 32, 64 or 128, dv up
 * to 128, rows given in rising order from first_row on, none longer than `longest`.  `workspace`:
 * zp_mlstm_runs_workspace() bytes for the rows from first_row to the end. */
int64_t zp_mlstm_runs_workspace(int32_t rows, int32_t segments, int32_t heads);
int zp_mlstm_runs(const zp_mlstm* args, int32_t first_row, int32_t longest, void* workspace,
                  int64_t workspace_bytes, int32_t dtype, void* stream);

/* Gated delta rule with a decay per key channel, its short convolutions and gates, and the normed, gated
 * read-out.  Rows `in` hold the projections q, k (kv_heads of dk), v (heads of dv) and from column b_at
 * the step sizes' pre-activations; rows `low` hold the decays' (heads of dk) and from column g_at the
 * output gates' (heads of dv).  filters (taps, 2 * kv_heads * dk + heads * dv), the last tap is the
 * current token's.  state: (num_slots, heads, dk, dv) fp32; conv_state: (num_slots, heads, taps - 1, 2
 * dk + dv) of `dtype`. */
typedef struct {
  zp_segments seg;
  const void *in, *low;
  const float *filters, *a_log, *dt_bias, *norm;
  float* state;
  void *conv_state, *out;
  int64_t in_stride, low_stride, out_stride;
  int32_t heads, kv_heads, dk, dv, vdim, taps, b_at, g_at;
  float q_scale, eps, out_scale;
} zp_delta;
int zp_delta_scan(const zp_delta* args, int32_t dtype, void* stream);
/* The same for long runs (of taps - 1 tokens at least), 16 tokens at a time on the matrix cores (fp32):
 * bfloat16, dk 32, 64 or 128, dv up to 128, rows given in rising order from first_row on, none longer than
 * `longest`.  `workspace`: zp_delta_runs_workspace() bytes for the rows from first_row to the end. */
int64_t zp_delta_runs_workspace(int32_t rows, int32_t segments, int32_t heads, int32_t dk, int32_t dv);
int zp_delta_runs(const zp_delta* args, int32_t first_row, int32_t longest, void* workspace,
                  int64_t workspace_bytes, int32_t dtype, void* stream);

/* ------------------------------------------------------------------ libzipage_linear.so */

/* Linear attention with decay, S <- g S (rows) + k v^T, o = S^T q, and the normed, silu-gated read-out.  Rows `in`
 * hold q, k (heads of dk), v, g (heads of dv) from columns q_at, k_at, v_at, g_at.  The first `rot` dimensions of q's
 * and k's heads turn by position * freqs[.], dimension j with j + rot / 2; q is scaled by q_scale, k by k_scale.
 * Decays: with `low` (rows of heads of dk), sigmoid(low + decay)^inv_tau with `decay` (heads * dk); without it decay
 * (heads) itself.  dk 32, 64, 128 or 256, dv a multiple of 32 up to 256, zero padded; the norm's mean runs over vdim,
 * its weights are (heads * dv).  state: (num_slots, heads, dk, dv) fp32. */
typedef struct {
  zp_segments seg;
  const void *in, *low;
  const float *decay, *freqs, *norm;
  float* state;
  void* out;
  int64_t in_stride, low_stride, out_stride;
  int32_t heads, dk, dv, vdim, rot, q_at, k_at, v_at, g_at;
  float q_scale, k_scale, inv_tau, eps;
} zp_linear;
int zp_linear_scan(const zp_linear* args, int32_t dtype, void* stream);
/* The same for long runs, 16 tokens at a time on the matrix cores (fp32): bfloat16, dk 32, 64 or 128, dv up
 * to 128, rows given in rising order from first_row on, none longer than `longest`.  `workspace`:
 * zp_linear_runs_workspace() bytes for the rows from first_row to the end. */
int64_t zp_linear_runs_workspace(int32_t rows, int32_t segments, int32_t heads, int32_t dk);
int zp_linear_runs(const zp_linear* args, int32_t first_row, int32_t longest, void* workspace,
                   int64_t workspace_bytes, int32_t dtype, void* stream);

/* ------------------------------------------------------------------ libzipage_moe.so */

/* out (n, M) fp32 = x (n, K) w (M, K)^T.  K a multiple of 32, M of 4. */
int zp_small_linear(const void* x, const void* w, float* out, int32_t n, int32_t K, int32_t M,
                    int64_t x_stride, int32_t dtype, void* stream);

/* Per token: scores of the E logits (softmax over them, or each one's sigmoid), the `keep` of `groups` groups
 * with the largest single score, and the `top` best experts of those: ids and scores (n, top).  counts (E +
 * 1) is cleared for the plan. */
enum { ZP_SCORE_SOFTMAX = 0, ZP_SCORE_SIGMOID = 1 };
int zp_moe_select(const float* logits, int32_t* ids, float* weights, int32_t* counts, int32_t n,
                  int32_t E, int32_t top, int32_t groups, int32_t keep, int32_t score,
                  int32_t logits_stride, void* stream);

/* Assignments (token n, slot j), numbered n * (top + shared) + j, in the order of their experts, and the
 * row tiles of the expert products: tiles (max_tiles, 4) of expert, first position in `sorted`, rows.
 * Expert E is the shared one (slot `top` of every token).  zp_moe_tile_rows: rows per tile to plan
 * for; zp_moe_max_tiles: the length of `tiles`. */
int64_t zp_moe_tile_rows(int32_t n, int32_t E, int32_t top, int32_t dtype);
int64_t zp_moe_max_tiles(int32_t n, int32_t E, int32_t top, int32_t shared, int32_t rows);
int64_t zp_moe_plan_workspace(int32_t n, int32_t E, int32_t top);
int zp_moe_plan(const int32_t* ids, int32_t* counts, int32_t* sorted, int32_t* tiles, int32_t* ntiles,
                int32_t n, int32_t E, int32_t top, int32_t shared, int32_t rows, int32_t max_tiles,
                void* workspace, int64_t workspace_bytes, void* stream);

/* Expert products over a plan.  Weights in tile order: [out / 16][in / step][64 lanes][16 bytes], lane (g,
 * r) = 16 g + r holding row r and the g-th 16 bytes of a step of 64 bytes; gate_up interleaves 16
 * rows of the gate with the 16 of `up`.  out of gate_up, by position in `sorted`, with the assignment's
 * weight w (1 for the shared expert):
 *   ZP_GATE_CLAMPED  w g sigmoid(1.702 g) (u + 1), g = min(gate, limit), u = clamp(up, -limit, limit)
 *   ZP_GATE_SILU     g sigmoid(g) u, g = w gate, u = w up: the weight on the expert's input
 * out of down: planes (slots, n, out_stride), an assignment's row in the plane of its slot.  K a multiple
 * of 32, M of 16 (of 32 where it is a later K). */
enum { ZP_GATE_CLAMPED = 0, ZP_GATE_SILU = 1 };
int zp_moe_gate_up(const void* x, const void* w, const void* w_shared, void* out, const int32_t* sorted,
                   const int32_t* tiles, const int32_t* ntiles, const float* weights, int32_t n,
                   int32_t E, int32_t top, int32_t shared, int32_t rows, int32_t max_tiles, int32_t K,
                   int32_t M, int32_t M_shared, int64_t x_stride, int64_t out_stride, int32_t act,
                   float limit, float limit_shared, int32_t dtype, void* stream);
int zp_moe_down(const void* x, const void* w, const void* w_shared, void* out, const int32_t* sorted,
                const int32_t* tiles, const int32_t* ntiles, int32_t n, int32_t E, int32_t top,
                int32_t shared, int32_t rows, int32_t max_tiles, int32_t K, int32_t K_shared,
                int32_t M, int64_t x_stride, int64_t out_stride, int32_t dtype, void* stream);

#ifdef __cplusplus
}
#endif
#endif /* ZIPAGE_MODELS_H */
