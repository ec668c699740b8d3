// C ABI of the latent-attention decoder's kernels: host-side argument checks, then the launchers.
#include "../../include/polarquant_latent.h"
#include "pq_latent_internal.h"

namespace {

inline bool aligned(const void* p, size_t a) { return (reinterpret_cast<uintptr_t>(p) & (a - 1)) == 0; }
inline bool any_dtype(int d) { return d == PQ_F16 || d == PQ_BF16 || d == PQ_F32; }
inline int status(int err) { return err == 0 ? PQ_OK : PQ_ERR_LAUNCH; }
constexpr int64_t kMaxTokens = int64_t{1} << 30;

int check_tokens(int B, int L) {
    if (B < 1 || B > 65535 || L < 1 || static_cast<int64_t>(B) * L > kMaxTokens) return PQ_ERR_BAD_SHAPE;
    return PQ_OK;
}

}  // namespace

extern "C" {

int pq_validate_norm_conv(const float* x_in, const void* y, const void* w_post, const float* x_out, const void* w_pre,
                          const void* conv_w, const float* state_in, const float* state_out, const void* h_out,
                          const int32_t* start, const int32_t* pos_dev, int pos, int B, int L, int width, int groups,
                          int taps, int dtype) {
    if (!x_in || !w_pre || !h_out || (y && (!w_post || !x_out))) return PQ_ERR_NULL_POINTER;
    if (!any_dtype(dtype)) return PQ_ERR_BAD_DTYPE;
    if (int rc = check_tokens(B, L)) return rc;
    if (width < 1 || groups < 1 || width % groups || pos < 0) return PQ_ERR_BAD_SHAPE;
    const int v = (width / groups) % 4 == 0 ? 4 : 1;
    if (width > 4096 * v || groups > 8192) return PQ_ERR_BAD_SHAPE;
    if (conv_w) {
        if (taps < 1 || taps > pq::kConvMaxTaps) return PQ_ERR_BAD_SHAPE;
        if (taps > 1 && (!state_in || !state_out)) return PQ_ERR_NULL_POINTER;
        if (L > pq::kConvInPlaceTokens && taps > 1 && state_in == state_out) return PQ_ERR_BAD_STRIDE;
        if (state_in && (!aligned(state_in, 16) || !aligned(state_out, 16))) return PQ_ERR_MISALIGNED;
        if (L > pq::kConvInPlaceTokens && y && x_out == x_in) return PQ_ERR_BAD_STRIDE;
    }
    if (!aligned(x_in, 16) || (x_out && !aligned(x_out, 16)) || (y && (!aligned(y, 16) || !aligned(w_post, 16))) ||
        !aligned(w_pre, 16) || !aligned(h_out, 16) || (start && !aligned(start, 4)) || (pos_dev && !aligned(pos_dev, 4)))
        return PQ_ERR_MISALIGNED;
    return PQ_OK;
}

int pq_norm_conv(const float* x_in, const void* y, const void* w_post, float* x_out, const void* w_pre, const void* conv_w,
                 const float* state_in, float* state_out, void* h_out, const int32_t* start, const int32_t* pos_dev, int pos,
                 int B, int L, int width, int groups, int taps, float eps, int dtype, void* stream) {
    if (int rc = pq_validate_norm_conv(x_in, y, w_post, x_out, w_pre, conv_w, state_in, state_out, h_out, start, pos_dev, pos, B, L,
                                       width, groups, taps, dtype))
        return rc;
    pq::NormConvArgs a{x_in, y, w_post, x_out, w_pre, conv_w, state_in, state_out, h_out, start, pos_dev,
                       pos, B, L, width, groups, taps, 0, eps};
    return status(pq::launch_norm_conv(a, dtype, static_cast<hipStream_t>(stream)));
}

int pq_validate_latent_norm(const void* p, int64_t row_stride, const void* w_q, const void* w_kv, const void* q_out,
                            const void* cache, int64_t capacity, const int32_t* pos_dev, int pos, int B, int L, int q_rank,
                            int kv_rank, int dtype) {
    if (!p || !w_q || !q_out || (w_kv && !cache)) return PQ_ERR_NULL_POINTER;
    if (!any_dtype(dtype)) return PQ_ERR_BAD_DTYPE;
    if (int rc = check_tokens(B, L)) return rc;
    if (q_rank < 1 || kv_rank < 1 || pos < 0) return PQ_ERR_BAD_SHAPE;
    if (row_stride < static_cast<int64_t>(q_rank) + (w_kv ? kv_rank : 0)) return PQ_ERR_BAD_STRIDE;
    if (w_kv && (capacity < 1 || static_cast<int64_t>(pos) + L > capacity)) return PQ_ERR_BAD_STRIDE;
    if (!aligned(p, 16) || !aligned(w_q, 16) || !aligned(q_out, 16) || (w_kv && (!aligned(w_kv, 16) || !aligned(cache, 16))) ||
        (pos_dev && !aligned(pos_dev, 4)))
        return PQ_ERR_MISALIGNED;
    return PQ_OK;
}

int pq_latent_norm(const void* p, int64_t row_stride, const void* w_q, const void* w_kv, void* q_out, void* cache,
                   int64_t capacity, const int32_t* pos_dev, int pos, int B, int L, int q_rank, int kv_rank, float eps,
                   int dtype, void* stream) {
    if (int rc = pq_validate_latent_norm(p, row_stride, w_q, w_kv, q_out, cache, capacity, pos_dev, pos, B, L, q_rank, kv_rank, dtype))
        return rc;
    pq::LatentNormArgs a{p, row_stride, w_q, w_kv, q_out, cache, capacity, pos_dev, pos, B, L, q_rank, kv_rank, eps};
    return status(pq::launch_latent_norm(a, dtype, static_cast<hipStream_t>(stream)));
}

int pq_relu_sq(const void* x, void* y, size_t n, int dtype, void* stream) {
    if (!x || !y) return PQ_ERR_NULL_POINTER;
    if (!any_dtype(dtype)) return PQ_ERR_BAD_DTYPE;
    if (n < 1 || n > (size_t{1} << 41)) return PQ_ERR_BAD_SHAPE;
    if (!aligned(x, 16) || !aligned(y, 16)) return PQ_ERR_MISALIGNED;
    return status(pq::launch_relu_sq(x, y, n, dtype, static_cast<hipStream_t>(stream)));
}

int pq_validate_head_linear(const void* x, int64_t x_row_stride, int64_t x_head_stride, const void* w, const void* gate,
                            int64_t gate_row_stride, const void* y, int64_t y_row_stride, int64_t y_head_stride, int M,
                            int heads, int N, int K, int epilogue, int dtype) {
    if (!x || !w || !y || (epilogue == PQ_EPI_SIGMOID_GATE && !gate)) return PQ_ERR_NULL_POINTER;
    if (!any_dtype(dtype)) return PQ_ERR_BAD_DTYPE;
    if (M < 1 || M > 65535 || heads < 1 || heads > 65535 || N < 1 || K < 1 || epilogue < 0 || epilogue > PQ_EPI_F32) return PQ_ERR_BAD_SHAPE;
    if (x_row_stride < K || y_row_stride < N || x_head_stride < 0 || y_head_stride < 0 || (heads > 1 && y_head_stride < N)) return PQ_ERR_BAD_STRIDE;
    if (epilogue == PQ_EPI_SIGMOID_GATE && gate_row_stride < static_cast<int64_t>(heads) * N) return PQ_ERR_BAD_STRIDE;
    const size_t e = dtype == PQ_F32 ? 4 : 2;
    if (!aligned(x, e) || !aligned(w, e) || !aligned(y, epilogue == PQ_EPI_F32 ? 4 : e) || (gate && !aligned(gate, e))) return PQ_ERR_MISALIGNED;
    return PQ_OK;
}

// the matrix-core kernels take what their 16-byte loads and 16-column tiles can hold; anything else the plain kernel
static bool head_linear_fits_mfma(const pq::HeadLinearArgs& a, int dtype) {
    return dtype != PQ_F32 && a.M <= 16 && a.N % 16 == 0 && a.K % 32 == 0 && a.x_row % 8 == 0 && a.x_head % 8 == 0 &&
           a.y_row % 4 == 0 && a.y_head % 4 == 0 && aligned(a.x, 16) && aligned(a.w, 16) && aligned(a.y, a.epilogue == PQ_EPI_F32 ? 16 : 8);
}

int pq_head_linear(const void* x, int64_t x_row_stride, int64_t x_head_stride, const void* w, const void* gate,
                   int64_t gate_row_stride, void* y, int64_t y_row_stride, int64_t y_head_stride, int M, int heads, int N,
                   int K, int epilogue, int dtype, void* stream) {
    if (int rc = pq_validate_head_linear(x, x_row_stride, x_head_stride, w, gate, gate_row_stride, y, y_row_stride, y_head_stride, M,
                                         heads, N, K, epilogue, dtype))
        return rc;
    pq::HeadLinearArgs a{x, x_row_stride, x_head_stride, w, gate, gate_row_stride, y, y_row_stride, y_head_stride, M, heads, N, K, epilogue};
    const hipStream_t st = static_cast<hipStream_t>(stream);
    return status(head_linear_fits_mfma(a, dtype) ? pq::launch_head_linear_mfma(a, dtype, st) : pq::launch_head_linear_any(a, dtype, st));
}

int pq_latent_decode_plan(int B, int L, int H, int64_t max_keys, int n_cus) {
    if (B < 1 || L < 1 || H < 1 || max_keys < 1) return 1;
    if (n_cus <= 0) n_cus = 256;
    const int64_t rows = static_cast<int64_t>(L) * H, per = rows <= 16 ? 16 : rows <= 32 ? 32 : 64;
    const int64_t groups = static_cast<int64_t>(B) * ((rows + per - 1) / per);
    // what the compute units hold at once (two workgroups of up to 32 rows, one of 64); every slice costs a partial of R
    // floats per row, so a slice keeps at least 128 keys
    int64_t n = (n_cus * (per <= 32 ? 2 : 1) + groups - 1) / groups, most = (max_keys + 127) / 128;
    n = n < most ? n : most;
    return static_cast<int>(n < 1 ? 1 : n > 512 ? 512 : n);
}

size_t pq_latent_decode_workspace_bytes(int B, int L, int H, int R, int n_splits) {
    if (B < 1 || L < 1 || H < 1 || R < 1 || n_splits < 1) return 0;
    const size_t rows = static_cast<size_t>(B) * n_splits * L * H;
    return (((2 * rows + 3) & ~size_t{3}) + rows * R) * sizeof(float);      // pairs, then accumulators from a 16-byte boundary on
}

int pq_validate_latent_decode(const void* q, const void* c, int64_t capacity, const float* sink, const int32_t* start,
                              const int32_t* pos_dev, int pos, const void* out, int B, int L, int H, int R, int n_splits,
                              const void* workspace, size_t workspace_bytes, int dtype) {
    if (!q || !c || !sink || !out) return PQ_ERR_NULL_POINTER;
    if (!any_dtype(dtype)) return PQ_ERR_BAD_DTYPE;
    if (int rc = check_tokens(B, L)) return rc;
    if (H < 1 || H > 65535 || R < 1 || R > 7168 || static_cast<int64_t>(L) * H > (1 << 24) || pos < 0) return PQ_ERR_BAD_SHAPE;
    if (capacity < 1 || capacity > kMaxTokens || static_cast<int64_t>(pos) + L > capacity) return PQ_ERR_BAD_STRIDE;
    if (!aligned(q, 16) || !aligned(c, 16) || !aligned(out, 16) || !aligned(sink, 4) || (start && !aligned(start, 4)) ||
        (pos_dev && !aligned(pos_dev, 4)))
        return PQ_ERR_MISALIGNED;
    if (pq::latent_decode_mfma(R, dtype)) {
        if (!workspace) return PQ_ERR_NULL_POINTER;
        if (n_splits < 1 || n_splits > 512 || workspace_bytes < pq_latent_decode_workspace_bytes(B, L, H, R, n_splits)) return PQ_ERR_WORKSPACE;
        if (!aligned(workspace, 16)) return PQ_ERR_MISALIGNED;
    }
    return PQ_OK;
}

int pq_latent_decode(const void* q, const void* c, int64_t capacity, const float* sink, const int32_t* start,
                     const int32_t* pos_dev, int pos, void* out, int B, int L, int H, int R, float scale, int n_splits,
                     void* workspace, size_t workspace_bytes, int dtype, void* stream) {
    if (int rc = pq_validate_latent_decode(q, c, capacity, sink, start, pos_dev, pos, out, B, L, H, R, n_splits, workspace, workspace_bytes, dtype))
        return rc;
    pq::LatentDecodeArgs a{q, c, capacity, sink, start, pos_dev, out, static_cast<float*>(workspace), pos, B, L, H, R, n_splits, scale};
    const hipStream_t st = static_cast<hipStream_t>(stream);
    return status(pq::latent_decode_mfma(R, dtype) ? pq::launch_latent_decode(a, dtype, st) : pq::launch_latent_decode_any(a, dtype, st));
}

int pq_latent_prefill_takes(int D, int Dv, int dtype) { return D >= 1 && Dv >= 1 && pq::latent_prefill_mfma(D, Dv, dtype) ? 1 : 0; }

int pq_validate_latent_prefill(const void* q, const void* k, const void* vt, int64_t vt_row_stride, const float* sink,
                               const void* gate, int64_t gate_row_stride, const int32_t* start, const void* out, int B, int L,
                               int Lk, int H, int D, int Dv, int dtype) {
    if (!q || !k || !vt || !sink || !out) return PQ_ERR_NULL_POINTER;
    if (dtype != PQ_F16 && dtype != PQ_BF16) return PQ_ERR_BAD_DTYPE;
    if (int rc = check_tokens(B, L)) return rc;
    if (H < 1 || H > 65535 || !pq_latent_prefill_takes(D, Dv, dtype) || Lk < L || Lk > kMaxTokens || (L + 127) / 128 > 65535) return PQ_ERR_BAD_SHAPE;
    if (vt_row_stride % 64 || vt_row_stride < Lk || (gate && gate_row_stride < static_cast<int64_t>(H) * Dv)) return PQ_ERR_BAD_STRIDE;
    if (!aligned(q, 16) || !aligned(k, 16) || !aligned(vt, 16) || !aligned(out, 8) || (gate && !aligned(gate, 8)) || !aligned(sink, 4) ||
        (start && !aligned(start, 4)))
        return PQ_ERR_MISALIGNED;
    return PQ_OK;
}

int pq_latent_prefill(const void* q, const void* k, const void* vt, int64_t vt_row_stride, const float* sink, const void* gate,
                      int64_t gate_row_stride, const int32_t* start, void* out, int B, int L, int Lk, int H, int D, int Dv,
                      float scale, int dtype, void* stream) {
    if (int rc = pq_validate_latent_prefill(q, k, vt, vt_row_stride, sink, gate, gate_row_stride, start, out, B, L, Lk, H, D, Dv, dtype))
        return rc;
    pq::LatentPrefillArgs a{q, k, vt, sink, gate, gate_row_stride, start, out, vt_row_stride, B, L, Lk, H, D, Dv, scale};
    return status(pq::launch_latent_prefill(a, dtype, static_cast<hipStream_t>(stream)));
}

}  // extern "C"
