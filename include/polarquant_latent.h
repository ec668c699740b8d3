/* polarquant_latent.h — C ABI of libpolarquant_latent.so (gfx950): latent attention (no reference counterpart; the Dekipel decoder of
 * polarquant_amd/modeling_dekipel.py).  Conventions and status codes are polarquant.h's.
 *
 * dtype: PQ_F16, PQ_BF16 or PQ_F32 for weights and activations; the residual stream, the convolution's
 * state, scores, softmax and every sum are float32 whatever it is.
 * B sequences of L new tokens each; `pos` is the position of the first of them
 * (tokens the cache holds already), taken from *pos_dev instead when that is not
 * null, so that a step can be replayed from a graph; start[b] (or null: 0) is the
 * position of sequence b's first token, smaller positions being left padding.
 *
 * pq_latent_norm: p rows hold q_rank, then (w_kv not null) kv_rank columns;
 *   q_out = rmsnorm(first part) * w_q, cache[b, pos + t] = rmsnorm(second) * w_kv,
 *   cache [B, capacity, kv_rank].
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

#include "polarquant_steps.h"

#ifdef __cplusplus
extern "C" {
#endif

int pq_latent_norm(const void *p, int64_t row_stride, const void *w_q, const void *w_kv, void *q_out, void *cache,
                   int64_t capacity, const int32_t *pos_dev, int pos, int B, int L, int q_rank, int kv_rank, float eps,
                   int dtype, void *stream);
int pq_validate_latent_norm(const void *p, int64_t row_stride, const void *w_q, const void *w_kv, const void *q_out,
                            const void *cache, int64_t capacity, const int32_t *pos_dev, int pos, int B, int L, int q_rank,
                            int kv_rank, int dtype);

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
