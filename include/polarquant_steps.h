/* polarquant_steps.h — C ABI of libpolarquant_steps.so (gfx950): the steps between a
 * layer's mixers and matrix products, whatever the mixers are (no reference
 * counterpart).  Conventions and status codes are polarquant.h's.
 *
 * dtype: PQ_F16, PQ_BF16 or PQ_F32 for weights and activations; the residual stream, a convolution's
 * state and every sum are float32 whatever it is.
 * B sequences of L new tokens each; `pos` is the position of the first of them, taken
 * from *pos_dev instead when that is not null, so that a step can be replayed from a
 * graph; start[b] (or null: 0) is the position of sequence b's first token, smaller
 * positions being left padding.
 *
 * pq_norm_conv: one launch between two sublayers.
 *     x' = x_in + gnorm(y) * w_post     (y null: x' = x_in, x_out not written)
 *                                       (w_post null: x' = x_in + y)
 *     n  = gnorm(x') * w_pre            gnorm: each of `groups` equal consecutive
 *                                       parts over its own root mean square
 *     h  = n + conv(n)                  conv_w [width, taps], the last tap meets the
 *                                       current token; conv_w null: h = n
 *   state_in / state_out [B, taps - 1, width]: n of the tokens before / up to the
 *   end of this call, oldest first (zeros at a sequence's start).  In place
 *   (x_out == x_in, state_out == state_in) for L <= 32 only.
 *
 * pq_relu_sq: y = max(x, 0)^2, n elements, y may be x.
 *
 * pq_gelu_mul: y = gelu(gate) * up, the tanh form; [rows, cols] with row strides.
 *
 * pq_stream_add: x_out = x + y + e + v; y in the dtype, e float32, v [width] in the
 *   dtype, each or null; x_out may be x.  pq_embed_rows: out[r] = table[ids[r]] * scale.
 * pq_softcap: x <- cap * tanh(x * scale / cap) in place (cap <= 0: x * scale).
 *
 * pq_head_linear: y[m, h, :] = epilogue(x[m, h, :] w[h]^T) with w [heads, N, K];
 *   PQ_EPI_SIGMOID_GATE multiplies by sigmoid(gate[m, h * N + n]), PQ_EPI_F32 stores
 *   float32.  M <= 16, N % 16 == 0, K % 32 == 0 in a 16-bit dtype stream the weights
 *   through the matrix-core kernels; other sizes and float32 run a plain kernel.
 */
#ifndef POLARQUANT_STEPS_H
#define POLARQUANT_STEPS_H

#include "polarquant.h"

#ifdef __cplusplus
extern "C" {
#endif

#define PQ_F32 2             /* beside pq_dtype's two: the entry points of this library and of those built on it */

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

int pq_relu_sq(const void *x, void *y, size_t n, int dtype, void *stream);

int pq_gelu_mul(const void *gate, const void *up, int64_t in_stride, void *y, int64_t out_stride, int64_t rows, int cols,
                int dtype, void *stream);
int pq_stream_add(const float *x, const void *y, const float *e, const void *v, float *x_out, int64_t rows, int width,
                  int dtype, void *stream);
int pq_embed_rows(const void *table, const int64_t *ids, float scale, float *out, int64_t rows, int width, int64_t vocab,
                  int dtype, void *stream);
int pq_softcap(float *x, size_t n, float scale, float cap, void *stream);

int pq_head_linear(const void *x, int64_t x_row_stride, int64_t x_head_stride, const void *w, const void *gate,
                   int64_t gate_row_stride, void *y, int64_t y_row_stride, int64_t y_head_stride, int M, int heads, int N,
                   int K, int epilogue, int dtype, void *stream);
int pq_validate_head_linear(const void *x, int64_t x_row_stride, int64_t x_head_stride, const void *w, const void *gate,
                            int64_t gate_row_stride, const void *y, int64_t y_row_stride, int64_t y_head_stride, int M,
                            int heads, int N, int K, int epilogue, int dtype);

#ifdef __cplusplus
}
#endif
#endif /* POLARQUANT_STEPS_H */
