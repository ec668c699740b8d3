// C ABI of the latent-attention kernels: host-side argument checks, then the launchers.
#include "../../include/polarquant_latent.h"
#include "pq_latent_internal.h"
#include "pq_capi_checks.h"

using namespace pq::capi;

extern "C" {

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
