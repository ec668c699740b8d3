// C ABI of windowed attention and of the recurrent mixers: host-side argument checks, then the launchers.
#include "../../include/polarquant_recurrent.h"
#include "pq_recurrent_internal.h"
#include "pq_capi_checks.h"

using namespace pq::capi;

namespace {

constexpr int kMaxTaps = 16;
inline hipStream_t S(void* s) { return static_cast<hipStream_t>(s); }
inline size_t elem(int dtype) { return dtype == PQ_F32 ? 4 : 2; }

int check_heads(int H, int G, int D, int Dv) {
    if (H < 1 || H > 65535 || G < 1 || H % G || D < 1 || Dv < 1 || D > 8192 || Dv > 8192) return PQ_ERR_BAD_SHAPE;
    if (static_cast<int64_t>(H) * (D > Dv ? D : Dv) > (1 << 24)) return PQ_ERR_BAD_SHAPE;
    return PQ_OK;
}
int check_scan(int B, int L, int G, int H, int dim, int vdim, int dtype) {
    if (!any_dtype(dtype)) return PQ_ERR_BAD_DTYPE;
    if (int rc = check_tokens(B, L)) return rc;
    if (int rc = check_heads(H, G, dim, vdim)) return rc;
    return dim > pq::kScanMaxDim ? PQ_ERR_BAD_SHAPE : PQ_OK;
}

}  // namespace

extern "C" {

int pq_qk_norm(const void* q, const void* k, const void* v, int64_t row_stride, const void* w_q, const void* w_k, void* q_out,
               void* k_out, void* k_ring, void* v_ring, const int32_t* pos_dev, int pos, int B, int L, int H, int G, int D, int Dv,
               int cap, float eps, int dtype, void* stream) {
    if (!q || !k || !v || !w_q || !w_k || !q_out || !k_ring || !v_ring) return PQ_ERR_NULL_POINTER;
    if (!any_dtype(dtype)) return PQ_ERR_BAD_DTYPE;
    if (int rc = check_tokens(B, L)) return rc;
    if (int rc = check_heads(H, G, D, Dv)) return rc;
    if (pos < 0 || cap < 64 || cap % 64 || (!k_out && L > PQ_WINDOW_SMALL)) return PQ_ERR_BAD_SHAPE;
    if (row_stride < static_cast<int64_t>(H) * D || row_stride < static_cast<int64_t>(G) * Dv) return PQ_ERR_BAD_STRIDE;
    pq::QkNormArgs a{q, k, v, row_stride, w_q, w_k, q_out, k_out, k_ring, v_ring, pos_dev, pos, B, L, H, G, D, Dv, cap, eps};
    return status(pq::launch_qk_norm(a, dtype, S(stream)));
}

int pq_ring_append(const void* k, int64_t k_row_stride, const void* v, int64_t v_row_stride, void* k_ring, void* v_ring, int pos,
                   int B, int L, int G, int D, int Dv, int cap, int dtype, void* stream) {
    if (!k || !v || !k_ring || !v_ring) return PQ_ERR_NULL_POINTER;
    if (!any_dtype(dtype)) return PQ_ERR_BAD_DTYPE;
    if (int rc = check_tokens(B, L)) return rc;
    if (int rc = check_heads(G, G, D, Dv)) return rc;
    if (pos < 0 || cap < 64 || cap % 64) return PQ_ERR_BAD_SHAPE;
    if (k_row_stride < static_cast<int64_t>(G) * D || v_row_stride < static_cast<int64_t>(G) * Dv) return PQ_ERR_BAD_STRIDE;
    pq::RingAppendArgs a{k, v, k_row_stride, v_row_stride, k_ring, v_ring, pos, B, L, G, D, Dv, cap};
    return status(pq::launch_ring_append(a, dtype, S(stream)));
}

int pq_window_plan(int B, int L, int H, int G, int window, int n_cus) {
    if (B < 1 || L < 1 || G < 1 || H < G || window < 1) return 1;
    if (n_cus <= 0) n_cus = 256;
    const int64_t groups = static_cast<int64_t>(B) * G * ((static_cast<int64_t>(L) * (H / G) + 15) / 16);
    // a workgroup per compute unit, each wavefront with a tile of 32 keys or more
    const int64_t tiles = (static_cast<int64_t>(window) + L + 30) / 32 + 1, most = (tiles + 7) / 8;
    int64_t n = n_cus / groups;
    n = n < most ? n : most;
    return static_cast<int>(n < 1 ? 1 : n > 64 ? 64 : n);
}

size_t pq_window_workspace_bytes(int B, int L, int H, int Dv, int n_splits) {
    if (B < 1 || L < 1 || H < 1 || Dv < 1 || n_splits < 2) return 0;
    const size_t rows = static_cast<size_t>(B) * L * H * n_splits;
    return (((2 * rows + 3) & ~size_t{3}) + rows * Dv) * sizeof(float);
}

// what the matrix-core kernels' 16-byte loads and 8-byte stores need; anything else runs the plain kernel
static bool window_fits_mfma(const pq::WindowAttnArgs& a, int dtype) {
    return pq::window_mfma(a.D, a.Dv, dtype) && aligned(a.q, 16) && aligned(a.k_ring, 16) && aligned(a.v_ring, 16) && aligned(a.out, 8) &&
           a.out_row % 4 == 0 && (!a.k_new || (aligned(a.k_new, 16) && aligned(a.v_new, 16) && a.k_row % 8 == 0 && a.v_row % 8 == 0));
}

int pq_validate_window_attn(const void* q, const void* k_ring, const void* v_ring, const void* k_new, int64_t k_row_stride,
                            const void* v_new, int64_t v_row_stride, const float* slopes, const int32_t* start,
                            const int32_t* pos_dev, int pos, const void* out, int64_t out_row_stride, int B, int L, int H, int G, int D,
                            int Dv, int cap, int window, int n_splits, const void* workspace, size_t workspace_bytes, int dtype) {
    if (!q || !k_ring || !v_ring || !out || (!k_new != !v_new)) return PQ_ERR_NULL_POINTER;
    if (!any_dtype(dtype)) return PQ_ERR_BAD_DTYPE;
    if (int rc = check_tokens(B, L)) return rc;
    if (int rc = check_heads(H, G, D, Dv)) return rc;
    if (window < 1 || pos < 0 || static_cast<int64_t>(pos) + L > kMaxTokens || cap < 64 || cap % 64 || static_cast<int64_t>(L) * H > (1 << 30)) return PQ_ERR_BAD_SHAPE;
    if (static_cast<int64_t>(cap) < static_cast<int64_t>(window) + PQ_WINDOW_SMALL - 1) return PQ_ERR_BAD_SHAPE;
    if ((!k_new && L > PQ_WINDOW_SMALL) || (k_new && pos_dev)) return PQ_ERR_BAD_SHAPE;
    if (out_row_stride < static_cast<int64_t>(H) * Dv) return PQ_ERR_BAD_STRIDE;
    if (k_new && (k_row_stride < static_cast<int64_t>(G) * D || v_row_stride < static_cast<int64_t>(G) * Dv)) return PQ_ERR_BAD_STRIDE;
    if (!aligned(q, elem(dtype)) || !aligned(out, elem(dtype)) || (slopes && !aligned(slopes, 4)) || (start && !aligned(start, 4)) || (pos_dev && !aligned(pos_dev, 4)))
        return PQ_ERR_MISALIGNED;
    if (n_splits < 1 || n_splits > 64) return PQ_ERR_WORKSPACE;
    if (!k_new && n_splits > 1 && (!workspace || !aligned(workspace, 16) || workspace_bytes < pq_window_workspace_bytes(B, L, H, Dv, n_splits))) return PQ_ERR_WORKSPACE;
    return PQ_OK;
}

int pq_window_attn(const void* q, const void* k_ring, const void* v_ring, const void* k_new, int64_t k_row_stride, const void* v_new,
                   int64_t v_row_stride, const float* slopes, const int32_t* start, const int32_t* pos_dev, int pos, void* out,
                   int64_t out_row_stride, int B, int L, int H, int G, int D, int Dv, int cap, int window, float scale, float out_scale,
                   int n_splits, void* workspace, size_t workspace_bytes, int dtype, void* stream) {
    if (int rc = pq_validate_window_attn(q, k_ring, v_ring, k_new, k_row_stride, v_new, v_row_stride, slopes, start, pos_dev, pos, out,
                                         out_row_stride, B, L, H, G, D, Dv, cap, window, n_splits, workspace, workspace_bytes, dtype))
        return rc;
    pq::WindowAttnArgs a{q, k_ring, v_ring, k_new, v_new, k_row_stride, v_row_stride, slopes, start, pos_dev, out, out_row_stride,
                         static_cast<float*>(workspace), pos, B, L, H, G, D, Dv, cap, window, n_splits, scale, out_scale};
    if (!window_fits_mfma(a, dtype)) return status(pq::launch_window_plain(a, dtype, S(stream)));
    return status(k_new ? pq::launch_window_prefill(a, dtype, S(stream)) : pq::launch_window_decode(a, dtype, S(stream)));
}

int pq_validate_delta_prep(int B, int L, int G, int H, int dim, int vdim, int taps, const float* state_in, const float* state_out,
                           int64_t row_stride, int64_t a_row_stride, int dtype) {
    if (int rc = check_scan(B, L, G, H, dim, vdim, dtype)) return rc;
    if (taps < 1 || taps > kMaxTaps || vdim > pq::kScanMaxDim) return PQ_ERR_BAD_SHAPE;
    if (taps > 1 && (!state_in || !state_out)) return PQ_ERR_NULL_POINTER;
    if (taps > 1 && L > 32 && state_in == state_out) return PQ_ERR_BAD_STRIDE;      // several workgroups: not in place
    if (row_stride < static_cast<int64_t>(H) * vdim || row_stride < static_cast<int64_t>(G) * dim || a_row_stride < static_cast<int64_t>(H) * dim) return PQ_ERR_BAD_STRIDE;
    return PQ_OK;
}

int pq_delta_prep(const void* q, const void* k, const void* v, const void* b, int64_t row_stride, const void* a, int64_t a_row_stride,
                  const void* w_q, const void* w_k, const void* w_v, const void* A_log, const void* dt_bias, const float* state_in,
                  float* state_out, void* q_out, void* k_out, void* v_out, float* q_inv, float* k_inv, float* log_g, float* beta,
                  const int32_t* start, const int32_t* pos_dev, int pos, int B, int L, int G, int H, int dim, int vdim, int taps, int dtype,
                  void* stream) {
    if (!q || !k || !v || !b || !a || !w_q || !w_k || !w_v || !A_log || !dt_bias || !q_out || !k_out || !v_out || !q_inv || !k_inv || !log_g || !beta)
        return PQ_ERR_NULL_POINTER;
    if (int rc = pq_validate_delta_prep(B, L, G, H, dim, vdim, taps, state_in, state_out, row_stride, a_row_stride, dtype)) return rc;
    pq::DeltaPrepArgs d{q, k, v, b, row_stride, a, a_row_stride, w_q, w_k, w_v, A_log, dt_bias, state_in, state_out, q_out, k_out, v_out,
                        q_inv, k_inv, log_g, beta, start, pos_dev, pos, B, L, G, H, dim, vdim, taps, 0};
    return status(pq::launch_delta_prep(d, dtype, S(stream)));
}

size_t pq_scan_workspace_bytes(int delta, int B, int H, int dim, int tokens, int dtype) {
    if (B < 1 || H < 1 || dim < 1 || dim > pq::kScanMaxDim || tokens < 1 || (dtype != PQ_F16 && dtype != PQ_BF16)) return 0;
    const size_t chunks = (static_cast<size_t>(tokens) + pq::kRecurrentChunk - 1) / pq::kRecurrentChunk;
    return chunks * B * H * pq::chunk_block_bytes(delta != 0, dim, dtype);
}

// a workspace asks for the chunked kernels
static int check_chunks(bool delta, int B, int H, int dim, const void* workspace, size_t bytes, const int32_t* pos_dev, int dtype) {
    if (pos_dev) return PQ_ERR_BAD_SHAPE;
    if (dtype == PQ_F32) return PQ_ERR_BAD_DTYPE;
    if (!aligned(workspace, 16)) return PQ_ERR_MISALIGNED;
    return bytes < pq_scan_workspace_bytes(delta, B, H, dim, 1, dtype) ? PQ_ERR_WORKSPACE : PQ_OK;
}

int pq_delta_scan(const void* q, const void* k, const void* v, const float* q_inv, const float* k_inv, const float* log_g,
                  const float* beta, float* state, float* o, const int32_t* start, const int32_t* pos_dev, int pos, int B, int L, int G,
                  int H, int dim, int vdim, void* workspace, size_t workspace_bytes, int dtype, void* stream) {
    if (!q || !k || !v || !q_inv || !k_inv || !log_g || !beta || !state || !o) return PQ_ERR_NULL_POINTER;
    if (int rc = check_scan(B, L, G, H, dim, vdim, dtype)) return rc;
    if (workspace)
        if (int rc = check_chunks(true, B, H, dim, workspace, workspace_bytes, pos_dev, dtype)) return rc;
    pq::ChunkArgs a{};
    a.workspace = static_cast<char*>(workspace);
    a.q = q; a.k = k; a.v = v;
    a.q_row = a.k_row = static_cast<int64_t>(G) * dim; a.v_row = static_cast<int64_t>(H) * vdim;
    a.q_inv = q_inv; a.k_inv = k_inv; a.log_g = log_g; a.beta = beta; a.state = state; a.o = o; a.start = start; a.pos_dev = pos_dev;
    a.pos = pos; a.B = B; a.L = L; a.G = G; a.H = H; a.dim = dim; a.vdim = vdim;
    return status(workspace ? pq::launch_delta_chunks(a, workspace_bytes, dtype, S(stream)) : pq::launch_delta_scan(a, dtype, S(stream)));
}

int pq_memory_gates(const void* i, const void* f, int64_t row_stride, const void* b_i, const void* b_f, float* log_i, float* log_f,
                    int64_t rows, int H, float cap, int dtype, void* stream) {
    if (!i || !f || !b_i || !b_f || !log_i || !log_f) return PQ_ERR_NULL_POINTER;
    if (!any_dtype(dtype)) return PQ_ERR_BAD_DTYPE;
    if (rows < 1 || rows > kMaxTokens || H < 1 || H > 65535 || !(cap > 0.0f)) return PQ_ERR_BAD_SHAPE;
    if (row_stride < H) return PQ_ERR_BAD_STRIDE;
    pq::MemoryGateArgs a{i, f, row_stride, b_i, b_f, log_i, log_f, rows, H, cap};
    return status(pq::launch_memory_gates(a, dtype, S(stream)));
}

int pq_memory_scan(const void* q, const void* k, const void* v, int64_t row_stride, const float* log_i, const float* log_f, float* state,
                   float* m, float* o, float* den, float q_scale, const int32_t* start, const int32_t* pos_dev, int pos, int B, int L, int H,
                   int dim, int vdim, void* workspace, size_t workspace_bytes, int dtype, void* stream) {
    if (!q || !k || !v || !log_i || !log_f || !state || !m || !o || !den) return PQ_ERR_NULL_POINTER;
    if (int rc = check_scan(B, L, H, H, dim, vdim, dtype)) return rc;
    if (row_stride < static_cast<int64_t>(H) * (dim > vdim ? dim : vdim)) return PQ_ERR_BAD_STRIDE;
    if (workspace && row_stride > (1 << 26)) return PQ_ERR_BAD_STRIDE;      // (a chunk's rows are addressed with 32 bits)
    if (workspace)
        if (int rc = check_chunks(false, B, H, dim, workspace, workspace_bytes, pos_dev, dtype)) return rc;
    pq::ChunkArgs a{};
    a.workspace = static_cast<char*>(workspace);
    a.q = q; a.k = k; a.v = v;
    a.q_row = a.k_row = a.v_row = row_stride;
    a.log_i = log_i; a.log_f = log_f; a.state = state; a.m = m; a.o = o; a.den = den; a.start = start; a.pos_dev = pos_dev;
    a.pos = pos; a.B = B; a.L = L; a.G = H; a.H = H; a.dim = dim; a.vdim = vdim; a.q_scale = q_scale;
    return status(workspace ? pq::launch_memory_chunks(a, workspace_bytes, dtype, S(stream)) : pq::launch_memory_scan(a, dtype, S(stream)));
}

int pq_head_norm_gate(const float* o, const float* den, const void* w, int w_head_stride, const void* gate, int64_t gate_row_stride,
                      void* out, int64_t out_row_stride, int64_t rows, int H, int vdim, float eps, float out_scale, int dtype, void* stream) {
    if (!o || !w || !gate || !out) return PQ_ERR_NULL_POINTER;
    if (!any_dtype(dtype)) return PQ_ERR_BAD_DTYPE;
    if (rows < 1 || rows > kMaxTokens || H < 1 || vdim < 1 || (w_head_stride != 0 && w_head_stride != vdim)) return PQ_ERR_BAD_SHAPE;
    const int64_t cols = static_cast<int64_t>(H) * vdim;
    if (gate_row_stride < cols || out_row_stride < cols) return PQ_ERR_BAD_STRIDE;
    pq::HeadNormGateArgs a{o, den, w, w_head_stride, gate, gate_row_stride, out, out_row_stride, rows, H, vdim, eps, out_scale};
    return status(pq::launch_head_norm_gate(a, dtype, S(stream)));
}

}  // extern "C"
