/* C ABI of libzipage_models.so: the model-side kernels of decoders that need more than the
 * compression library's layer kernels -- an fp32 residual stream, a depth average, latent
 * attention over pages of latents.  Status codes, dtype tags and conventions are those of
 * zipage_hip.h; every entry point here takes ZP_BF16 or ZP_F32 (true 32-bit products), enqueues on
 * `stream`, allocates nothing and may be captured into a HIP graph. */
#ifndef ZIPAGE_MODELS_H
#define ZIPAGE_MODELS_H
#include "zipage_hip.h"

#ifdef __cplusplus
extern "C" {
#endif

/* x = embed[tokens] (+ pos[positions] when pos is given), fp32; with norm_weight also
 * out = x / sqrt(mean(x^2) + eps) * (weight_offset + norm_weight).  Rows are `width` long (multiple
 * of 8, zero padded), the mean runs over norm_width.  embed (vocab, width), pos (max_positions,
 * width) and out are of `dtype`; indices are clamped to the tables. */
int zp_embed_norm(const int64_t* tokens, const int32_t* positions, const void* embed, const void* pos,
                  float* x, const float* norm_weight, void* out, int32_t n, int32_t width,
                  int32_t norm_width, int64_t vocab, int64_t max_positions, float eps,
                  float weight_offset, int32_t dtype, void* stream);

/* r = x + the sum of y's n_y planes (x (n, width) fp32; y (n_y, n, width) of dtype), written to `result` when given; with a depth average
 * r <- mix[n_hist] * r + sum_{j < n_hist} mix[j] * hist[j] (hist: planes of (n, width) fp32,
 * hist_plane elements apart); written to `x_out` when given; with norm_weight also
 * out = rmsnorm(r) * (weight_offset + norm_weight) * out_scale.  mix NULL: no average. */
int zp_residual_norm(const float* x, const void* y, int32_t n_y, const float* hist,
                     int64_t hist_plane, const float* mix, int32_t n_hist, float* result, float* x_out,
                     const float* norm_weight, void* out, int32_t n, int32_t width,
                     int32_t norm_width, float eps, float weight_offset, float out_scale,
                     int32_t dtype, void* stream);

/* z > 0: alpha_p z^2 + z / 2;  z <= 0: alpha_n (exp(z) - 1 - z) + z / 2.  count % 8 == 0. */
int zp_xielu(const void* in, void* out, int64_t count, float alpha_p, float alpha_n, int32_t dtype,
             void* stream);

/* in (n, q_width + c_width): the first part RMS-normed times q_weight goes to q_out, the second
 * times c_weight to slot slots[i] of the cache (-1 skips) and to c_out when given.  The means run
 * over q_norm and c_norm elements; widths are multiples of 8, zero padded. */
int zp_latent_norm_store(const void* in, const float* q_weight, const float* c_weight, void* q_out,
                         void* c_out, void* cache, const int32_t* slots, int32_t n, int32_t q_width,
                         int32_t c_width, int32_t q_norm, int32_t c_norm, int64_t num_slots, float eps,
                         int32_t dtype, void* stream);

/* out[i] = src[rows[i]], rows of row_bytes (multiple of 16). */
int zp_gather_rows(const void* src, const int32_t* rows, void* out, int32_t n, int32_t row_bytes,
                   int64_t num_rows, void* stream);

/* out[n, h, :] = w[h] (M, K) in[n, h, :]; K a multiple of 32, M of 16. */
int zp_headwise_linear(const void* in, const void* w, void* out, int32_t n, int32_t H, int32_t K,
                       int32_t M, int32_t dtype, void* stream);

/* Attention of single tokens over paged latents.  q (n, H, R); cache (num_pages, BS, R); token i
 * sees the tokens [max(0, c - window), c) of its sequence, c = context_lens[i] (window 0: all;
 * c = 0: inert, zeros), through row table_rows[i] (NULL: i) of table (B, NB).
 * out[n, h] = sum_j softmax_j(scale * q[n, h] . c_j) c_j.  R a multiple of 32.  `workspace`:
 * zp_latent_rows_workspace() bytes, 16-byte aligned. */
int64_t zp_latent_rows_workspace(int32_t n, int32_t H, int32_t R, int32_t window, int32_t NB,
                                 int32_t BS, int32_t dtype);
int zp_latent_rows_attention(const void* q, const void* cache, const int32_t* table,
                             const int32_t* context_lens, const int32_t* table_rows, void* out,
                             int32_t n, int32_t H, int32_t R, int32_t BS, int32_t B, int32_t NB,
                             int32_t num_pages, int32_t window, float scale, int32_t dtype,
                             void* workspace, int64_t workspace_bytes, void* stream);

/* Attention of runs of tokens over expanded keys and values, bfloat16.  tiles (T, 4) int32, one
 * entry per up to 128 queries of one sequence: first query row, number of queries, row of the
 * run's first key, position of the first query counted from that key (key rows of a run are
 * consecutive positions).  A query sees its own position and the window - 1 before it (window 0:
 * all before it in the run).  q rows q_stride, k and v rows kv_stride elements apart; out (rows,
 * H, V). */
int zp_latent_tiles_attention(const void* q, const void* k, const void* v, void* out,
                              const int32_t* tiles, int32_t T, int32_t H, int32_t D, int32_t V,
                              int32_t window, int64_t q_rows, int64_t k_rows, int64_t q_stride,
                              int64_t kv_stride, float scale, int32_t dtype, void* stream);

#ifdef __cplusplus
}
#endif
#endif /* ZIPAGE_MODELS_H */
