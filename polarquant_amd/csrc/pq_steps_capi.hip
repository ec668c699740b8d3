// C ABI of the layer steps: host-side argument checks, then the launchers.
#include "../../include/polarquant_steps.h"
#include "pq_steps_internal.h"
#include "pq_capi_checks.h"

using namespace pq::capi;

extern "C" {

int pq_validate_norm_conv(const float* x_in, const void* y, const void* w_post, const float* x_out, const void* w_pre,
                          const void* conv_w, const float* state_in, const float* state_out, const void* h_out,
                          const int32_t* start, const int32_t* pos_dev, int pos, int B, int L, int width, int groups,
                          int taps, int dtype) {
    if (!x_in || !w_pre || !h_out || (y && !x_out)) return PQ_ERR_NULL_POINTER;
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
    if (!aligned(x_in, 16) || (x_out && !aligned(x_out, 16)) || (y && !aligned(y, 16)) || (w_post && !aligned(w_post, 16)) ||
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

int pq_relu_sq(const void* x, void* y, size_t n, int dtype, void* stream) {
    if (!x || !y) return PQ_ERR_NULL_POINTER;
    if (!any_dtype(dtype)) return PQ_ERR_BAD_DTYPE;
    if (n < 1 || n > (size_t{1} << 41)) return PQ_ERR_BAD_SHAPE;
    if (!aligned(x, 16) || !aligned(y, 16)) return PQ_ERR_MISALIGNED;
    return status(pq::launch_relu_sq(x, y, n, dtype, static_cast<hipStream_t>(stream)));
}

int pq_gelu_mul(const void* gate, const void* up, int64_t in_stride, void* y, int64_t out_stride, int64_t rows, int cols, int dtype, void* stream) {
    if (!gate || !up || !y) return PQ_ERR_NULL_POINTER;
    if (!any_dtype(dtype)) return PQ_ERR_BAD_DTYPE;
    if (rows < 1 || rows > kMaxTokens || cols < 1) return PQ_ERR_BAD_SHAPE;
    if (in_stride < cols || out_stride < cols) return PQ_ERR_BAD_STRIDE;
    pq::GeluMulArgs a{gate, up, y, rows, in_stride, out_stride, cols};
    return status(pq::launch_gelu_mul(a, dtype, static_cast<hipStream_t>(stream)));
}

int pq_stream_add(const float* x, const void* y, const float* e, const void* v, float* x_out, int64_t rows, int width, int dtype, void* stream) {
    if (!x || !x_out) return PQ_ERR_NULL_POINTER;
    if (!any_dtype(dtype)) return PQ_ERR_BAD_DTYPE;
    if (rows < 1 || rows > kMaxTokens || width < 1) return PQ_ERR_BAD_SHAPE;
    pq::StreamAddArgs a{x, y, e, v, x_out, rows, width};
    return status(pq::launch_stream_add(a, dtype, static_cast<hipStream_t>(stream)));
}

int pq_embed_rows(const void* table, const int64_t* ids, float scale, float* out, int64_t rows, int width, int64_t vocab, int dtype, void* stream) {
    if (!table || !ids || !out) return PQ_ERR_NULL_POINTER;
    if (!any_dtype(dtype)) return PQ_ERR_BAD_DTYPE;
    if (rows < 1 || rows > kMaxTokens || width < 1 || vocab < 1) return PQ_ERR_BAD_SHAPE;
    return status(pq::launch_embed_rows(table, ids, scale, out, rows, width, vocab, dtype, static_cast<hipStream_t>(stream)));
}

int pq_softcap(float* x, size_t n, float scale, float cap, void* stream) {
    if (!x) return PQ_ERR_NULL_POINTER;
    if (n < 1 || n > (size_t{1} << 39)) return PQ_ERR_BAD_SHAPE;
    return status(pq::launch_softcap(x, n, scale, cap, static_cast<hipStream_t>(stream)));
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

}  // extern "C"
