// Argument blocks and launcher prototypes of the latent-attention kernels (pq_latent_norm.hip, pq_latent_attn.hip),
// shared with their C-ABI translation unit.  Each launcher returns a
// hipError_t cast to int (0 = ok).  dtype: 0 float16, 1 bfloat16, 2 float32.
#pragma once
#include <hip/hip_runtime.h>
#include <stddef.h>
#include <stdint.h>

namespace pq {

struct LatentNormArgs {
    const void* p;           // [B * L, row_stride]: q_rank query-latent columns, then kv_rank latent columns
    int64_t row_stride;
    const void *w_q, *w_kv;  // norm weights; w_kv null: the layer has no latent of its own
    void* q_out;             // [B * L, q_rank]
    void* cache;             // [B, capacity, kv_rank]: rows pos .. pos + L - 1 are written
    int64_t capacity;
    const int32_t* pos_dev;
    int pos, B, L, q_rank, kv_rank;
    float eps;
};
int launch_latent_norm(const LatentNormArgs& a, int dtype, hipStream_t st);

struct LatentDecodeArgs {
    const void* q;           // [B, L, H, R] queries in the latent space
    const void* c;           // [B, capacity, R]
    int64_t capacity;
    const float* sink;       // [H]
    const int32_t* start;
    const int32_t* pos_dev;
    void* out;               // [B, L, H, R]
    float* workspace;
    int pos, B, L, H, R, n_splits;
    float scale;
};
constexpr int kLatentMaxRank = 512;      // of the MFMA kernels; larger ranks run the plain kernel
inline bool latent_decode_mfma(int R, int dtype) { return dtype != 2 && R % 8 == 0 && R >= 8 && R <= kLatentMaxRank; }
int launch_latent_decode(const LatentDecodeArgs& a, int dtype, hipStream_t st);      // partials, then merge
int launch_latent_decode_any(const LatentDecodeArgs& a, int dtype, hipStream_t st);  // any rank, any dtype, no workspace

struct LatentPrefillArgs {
    const void* q;           // [B, L, H, D]
    const void* k;           // [B, Lk, H, D]
    const void* vt;          // [B, H * Dv, ldv]: values, one row per channel
    const float* sink;
    const void* gate;        // [B * L, H * Dv] rows gate_row apart, or null
    int64_t gate_row;
    const int32_t* start;
    void* out;               // [B, L, H * Dv]
    int64_t ldv;
    int B, L, Lk, H, D, Dv;
    float scale;
};
inline bool latent_prefill_mfma(int D, int Dv, int dtype) { return dtype != 2 && D % 8 == 0 && D <= 256 && Dv <= 256; }
int launch_latent_prefill(const LatentPrefillArgs& a, int dtype, hipStream_t st);

}  // namespace pq
