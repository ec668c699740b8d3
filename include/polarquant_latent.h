/* polarquant_latent.h — C ABI of libpolarquant_latent.so (gfx950): latent attention and the
 * layer steps around it (no reference counterpart; the Dekipel decoder of
 * polarquant_amd/modeling_dekipel.py).  Conventions and status codes are polarquant.h's.
 *
 * dtype: PQ_F16, PQ_BF16 or PQ_F32 for weights and activations; the residual stream, the convolution's
 * state, scores, softmax and every sum are float32 whatever it is.
 * B sequences of L new tokens each; `pos` is the position of the first of them
 * (tokens the cache holds already), taken from *pos_dev instead when that is not
 * null, so that a step can be replayed from a graph; start[b] (or null: 0) is the
 * position of sequence b's first token, smaller positions being left padding.
 *
 * pq_norm_conv: one launch between two sublayers.
 *     x' = x_in + gnorm(y) * w_post     (y null: x' = x_in, x_out not written)
 *     n  = gnorm(x') * w_pre            gnorm: each of `groups` equal consecutive
 *                                       parts over its own root mean square
 *     h  = n + conv(n)                  conv_w [width, taps], the last tap meets the
 *                                       current token; conv_w null: h = n
 *   state_in / state_out [B, taps - 1, width]: n of the tokens before / up to the
 *   end of this call, oldest first (zeros at a sequence's start).  In place
 *   (x_out == x_in, state_out == state_in) for L <= 32 only.
 *
 * pq_latent_norm: p rows hold q_rank, then (w_kv not null) kv_rank columns;
 *   q_out = rmsnorm(first part) * w_q, cache[b, pos + t] = rmsnorm(second) * w_kv,
 *   cache [B, capacity, kv_rank].
 *
 * pq_relu_sq: y = max(x, 0)^2, n elements, y may be x.
 *
 * pq_head_linear: y[m, h, :] = epilogue(x[m, h, :] w[h]^T) with w [heads, N, K];
 *   PQ_EPI_SIGMOID_GATE multiplies by sigmoid(gate[m, h * N + n]), PQ_EPI_F32 stores
 *   float32.  M <= 16, N % 16 == 0, K % 32 == 0 in a 16-bit dtype stream the weights
 *   through the matrix-core kernels; other sizes and float32 run a plain kernel.
 *
 * pq_latent_decode: q [B, L, H, R] already in the latent space, c [B, capacity, R]
 *   shared by all heads, out [B, L, H, R] = softmax over the keys start[b] <= j <=
 *   pos + t of scale * q . c_j (denominator + exp(sink[h])), applied to c.
 *   16-bit dtypes with R % 8 == 0, R <= 512 cut the context into n_splits slices
 *   (pq_latent_decode_plan) through `workspace`; others run a plain kernel.
 *
 * pq_latent_prefill: q [B, L, H, D], k [B, Lk, H, D] (Lk = pos + L), vt
 *   [B, H * Dv, vt_row_stride] the values with one row per channel (row stride a
 *   multiple of 64, columns past Lk finite), out [B, L, H * Dv], gate as above or
 *   null.  D % 8 == 0, D <= 256, Dv <= 256, 16-bit dtypes (pq_latent_prefill_takes).
 */
#ifndef POLARQUANT_LATENT_H
#define POLARQUANT_LATENT_H

#include "polarquant.h"

#ifdef __cplusplus
extern "C" {
#endif

#define PQ_F32 2             /* beside pq_dtype's two: this library's entry points only */

#define PQ_EPI_PLAIN 0
#define PQ_EPI_RELU_SQ 1
#define PQ_EPI_SIGMOID_GATE 2
#define PQ_EPI_F32 3

int pq_norm_conv(const float *x_in, const void *y, const void *w_post, float *x_out, const void *w_pre, const void *conv_w,
                 const float *state_in, float *state_out, void *h_out, const int32_t *start, const int32_t *pos_dev, int pos,
                 int B, int L, int width, int groups, int taps, float eps, int dtype, void *stream);
int pq_validate_norm_conv(const float *x_in, const void *y, const void *w_post, const float *x_out, const void *w_pre,
                          const void *conv_w, const float *state_in, const float *state_out, const void *h_out,
                          const int32_t *start, const int32_t *pos_dev, int pos, int B, int L, int width, int groups,
                          int taps, int dtype);

int pq_latent_norm(const void *p, int64_t row_stride, const void *w_q, const void *w_kv, void *q_out, void *cache,
                   int64_t capacity, const int32_t *pos_dev, int pos, int B, int L, int q_rank, int kv_rank, float eps,
                   int dtype, void *stream);
int pq_validate_latent_norm(const void *p, int64_t row_stride, const void *w_q, const void *w_kv, const void *q_out,
                            const void *cache, int64_t capacity, const int32_t *pos_dev, int pos, int B, int L, int q_rank,
                            int kv_rank, int dtype);

int pq_relu_sq(const void *x, void *y, size_t n, int dtype, void *stream);

int pq_head_linear(const void *x, int64_t x_row_stride, int64_t x_head_stride, const void *w, const void *gate,
                   int64_t gate_row_stride, void *y, int64_t y_row_stride, int64_t y_head_stride, int M, int heads, int N,
                   int K, int epilogue, int dtype, void *stream);
int pq_validate_head_linear(const void *x, int64_t x_row_stride, int64_t x_head_stride, const void *w, const void *gate,
                            int64_t gate_row_stride, const void *y, int64_t y_row_stride, int64_t y_head_stride, int M,
                            int heads, int N, int K, int epilogue, int dtype);

int pq_latent_decode_plan(int B, int L, int H, int64_t max_keys, int n_cus);
size_t pq_latent_decode_workspace_bytes(int B, int L, int H, int R, int n_splits);
int pq_latent_decode(const void *q, const void *c, int64_t capacity, const float *sink, const int32_t *start,
                     const int32_t *pos_dev, int pos, void *out, int B, int L, int H, int R, float scale, int n_splits,
                     void *workspace, size_t workspace_bytes, int dtype, void *stream);
int pq_validate_latent_decode(const void *q, const void *c, int64_t capacity, const float *sink, const int32_t *start,
                              const int32_t *pos_dev, int pos, const void *out, int B, int L, int H, int R, int n_splits,
                              const void *workspace, size_t workspace_bytes, int dtype);

int pq_latent_prefill_takes(int D, int Dv, int dtype);
int pq_latent_prefill(const void *q, const void *k, const void *vt, int64_t vt_row_stride, const float *sink, const void *gate,
                      int64_t gate_row_stride, const int32_t *start, void *out, int B, int L, int Lk, int H, int D, int Dv,
                      float scale, int dtype, void *stream);
int pq_validate_latent_prefill(const void *q, const void *k, const void *vt, int64_t vt_row_stride, const float *sink,
                               const void *gate, int64_t gate_row_stride, const int32_t *start, const void *out, int B, int L,
                               int Lk, int H, int D, int Dv, int dtype);

#ifdef __cplusplus
}
#endif
#endif /* POLARQUANT_LATENT_H */
