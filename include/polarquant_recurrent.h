/* polarquant_recurrent.h — C ABI of libpolarquant_recurrent.so (gfx950): attention over a
 * sliding window with a distance bias, the gated delta rule, and matrix memories (no
 * reference counterpart; the Kapudra decoder of polarquant_amd/modeling_kapudra.py).
 * Conventions, dtypes and the meaning of pos, pos_dev and start are polarquant_steps.h's.
 *
 * Windowed attention: H query heads read G key heads of size D, values of size Dv; the
 *   ring of a sequence, [G, cap, D] and [G, cap, Dv], holds the key of position j in row
 *   j % cap, cap a multiple of 64 and at least window + PQ_WINDOW_SMALL - 1.
 * pq_qk_norm: q and k, each over all its H * D (G * D) columns, x / rms * w; the keys to
 *   k_out, or (k_out null; L <= PQ_WINDOW_SMALL) keys and values to their ring rows.
 * pq_ring_append: the last min(L, cap) keys and values of a call to the ring.
 * pq_window_attn: out[t, h] = out_scale * softmax over the keys start <= j, 0 <= i - j <
 *   window of (scale * q . k_j - slopes[h] (i - j)), i = pos + t, applied to v.  Keys of
 *   this call come from k_new, v_new (their own row strides) or, with those null, from
 *   the ring like all others.  16-bit dtypes with D, Dv multiples of 8 up to 256 run
 *   matrix-core kernels; calls without k_new cut the window into n_splits slices
 *   (pq_window_plan) through `workspace`.
 *
 * pq_delta_prep: q, k (G heads of dim) and v (H heads of vdim) through a causal
 *   convolution of `taps` per channel (state [B, taps - 1, 2 G dim + H vdim] as in
 *   pq_norm_conv) and silu; 1 / length of each head's q and k (the former also times
 *   dim^-1/2); log_g = -exp(A_log[h]) softplus(a + dt_bias); beta = sigmoid(b).
 * pq_delta_scan: per head, with state rows scaled by g = exp(log_g):
 *     S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q.
 *   state [B, H, vdim, dim] float32, read and written back.
 * pq_memory_gates: log_i = cap tanh((i + b_i) / cap), log_f = log sigmoid(cap tanh((f + b_f) / cap)).
 * pq_memory_scan: m' = max(log_f + m, log_i); S <- exp(log_f + m - m') S + exp(log_i - m') k v^T,
 *   n alike with k alone; o = S^T q q_scale, den = max(|n . q| q_scale, exp(-m')) + 1e-6.
 *   state [B, H, vdim + 1, dim] (the last row is n), m [B, H, (vdim + 16) / 16]
 *   (equal copies, one for every 16 state rows).
 *   Without a workspace both scans go token by token; with one, of pq_scan_workspace_bytes for
 *   any number of tokens, 32 tokens at a time on the matrix cores, as many tokens ahead as it
 *   holds (16-bit dtypes, no pos_dev).
 * pq_head_norm_gate: out = out_scale * rmsnorm(o / den, per head) * w * sigmoid(gate);
 *   w [vdim] for all heads (w_head_stride 0) or [H * vdim] (w_head_stride vdim).
 */
#ifndef POLARQUANT_RECURRENT_H
#define POLARQUANT_RECURRENT_H

#include "polarquant_steps.h"

#ifdef __cplusplus
extern "C" {
#endif

#define PQ_WINDOW_SMALL 16

int pq_qk_norm(const void *q, const void *k, const void *v, int64_t row_stride, const void *w_q, const void *w_k, void *q_out,
               void *k_out, void *k_ring, void *v_ring, const int32_t *pos_dev, int pos, int B, int L, int H, int G, int D,
               int Dv, int cap, float eps, int dtype, void *stream);
int pq_ring_append(const void *k, int64_t k_row_stride, const void *v, int64_t v_row_stride, void *k_ring, void *v_ring,
                   int pos, int B, int L, int G, int D, int Dv, int cap, int dtype, void *stream);
int pq_window_plan(int B, int L, int H, int G, int window, int n_cus);
size_t pq_window_workspace_bytes(int B, int L, int H, int Dv, int n_splits);
int pq_validate_window_attn(const void *q, const void *k_ring, const void *v_ring, const void *k_new, int64_t k_row_stride,
                            const void *v_new, int64_t v_row_stride, const float *slopes, const int32_t *start,
                            const int32_t *pos_dev, int pos, const void *out, int64_t out_row_stride, int B, int L, int H, int G,
                            int D, int Dv, int cap, int window, int n_splits, const void *workspace, size_t workspace_bytes,
                            int dtype);
int pq_window_attn(const void *q, const void *k_ring, const void *v_ring, const void *k_new, int64_t k_row_stride,
                   const void *v_new, int64_t v_row_stride, const float *slopes, const int32_t *start, const int32_t *pos_dev,
                   int pos, void *out, int64_t out_row_stride, int B, int L, int H, int G, int D, int Dv, int cap, int window,
                   float scale, float out_scale, int n_splits, void *workspace, size_t workspace_bytes, int dtype, void *stream);

int pq_validate_delta_prep(int B, int L, int G, int H, int dim, int vdim, int taps, const float *state_in,
                           const float *state_out, int64_t row_stride, int64_t a_row_stride, int dtype);
int pq_delta_prep(const void *q, const void *k, const void *v, const void *b, int64_t row_stride, const void *a,
                  int64_t a_row_stride, const void *w_q, const void *w_k, const void *w_v, const void *A_log,
                  const void *dt_bias, const float *state_in, float *state_out, void *q_out, void *k_out, void *v_out,
                  float *q_inv, float *k_inv, float *log_g, float *beta, const int32_t *start, const int32_t *pos_dev, int pos,
                  int B, int L, int G, int H, int dim, int vdim, int taps, int dtype, void *stream);
size_t pq_scan_workspace_bytes(int delta, int B, int H, int dim, int tokens, int dtype);
int pq_delta_scan(const void *q, const void *k, const void *v, const float *q_inv, const float *k_inv, const float *log_g,
                  const float *beta, float *state, float *o, const int32_t *start, const int32_t *pos_dev, int pos, int B, int L,
                  int G, int H, int dim, int vdim, void *workspace, size_t workspace_bytes, int dtype, void *stream);
int pq_memory_gates(const void *i, const void *f, int64_t row_stride, const void *b_i, const void *b_f, float *log_i,
                    float *log_f, int64_t rows, int H, float cap, int dtype, void *stream);
int pq_memory_scan(const void *q, const void *k, const void *v, int64_t row_stride, const float *log_i, const float *log_f,
                   float *state, float *m, float *o, float *den, float q_scale, const int32_t *start, const int32_t *pos_dev,
                   int pos, int B, int L, int H, int dim, int vdim, void *workspace, size_t workspace_bytes, int dtype,
                   void *stream);
int pq_head_norm_gate(const float *o, const float *den, const void *w, int w_head_stride, const void *gate,
                      int64_t gate_row_stride, void *out, int64_t out_row_stride, int64_t rows, int H, int vdim, float eps,
                      float out_scale, int dtype, void *stream);

#ifdef __cplusplus
}
#endif
#endif /* POLARQUANT_RECURRENT_H */
