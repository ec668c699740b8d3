// Argument blocks and launcher prototypes of the latent-attention decoder's kernels (pq_latent.hip: the steps around
// the attention; pq_latent_attn.hip: attention), shared with their C-ABI translation unit.  Each launcher returns a
// hipError_t cast to int (0 = ok).  dtype: 0 float16, 1 bfloat16, 2 float32.
#pragma once
#include <hip/hip_runtime.h>
#include <stddef.h>
#include <stdint.h>

namespace pq {

struct NormConvArgs {
    const float* x_in;       // [B, L, W] residual stream
    const void* y;           // [B, L, W] output of the previous sublayer, or null
    const void* w_post;      // [W] weight of the norm applied to y
    float* x_out;            // [B, L, W] x_in + norm(y)
    const void* w_pre;       // [W] weight of the norm applied to the sum
    const void* conv_w;      // [W, taps], or null: no convolution
    const float* state_in;   // [B, taps - 1, W] the last norms of the tokens before this call, oldest first
    float* state_out;
    void* h_out;             // [B, L, W]
    const int32_t* start;    // [B] position of each sequence's first token, or null
    const int32_t* pos_dev;  // position of this call's first token on the device, or null (then `pos`)
    int pos, B, L, W, groups, taps, strip;
    float eps;
};
// A call of at most this many tokens per sequence is worked through by one workgroup per sequence, so that x_out may be
// x_in and state_out may be state_in; longer calls are cut into strips, whose first workgroup reads what the last writes.
constexpr int kConvInPlaceTokens = 32;
constexpr int kConvMaxTaps = 16;
int launch_norm_conv(const NormConvArgs& a, int dtype, hipStream_t st);

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

int launch_relu_sq(const void* x, void* y, size_t n, int dtype, hipStream_t st);

// y[m, h, n] = epilogue(sum_k x[m, h, k] w[h, n, k])
enum { kEpiPlain = 0, kEpiReluSq = 1, kEpiSigmoidGate = 2, kEpiF32 = 3 };
struct HeadLinearArgs {
    const void* x;
    int64_t x_row, x_head;
    const void* w;           // [heads, N, K]
    const void* gate;        // [M, heads * N] rows gate_row apart (kEpiSigmoidGate)
    int64_t gate_row;
    void* y;                 // in the dtype; float32 with kEpiF32
    int64_t y_row, y_head;
    int M, heads, N, K, epilogue;
};
int launch_head_linear_any(const HeadLinearArgs& a, int dtype, hipStream_t st);      // pq_latent.hip: any size, any dtype
int launch_head_linear_mfma(const HeadLinearArgs& a, int dtype, hipStream_t st);     // pq_linear.hip: M <= 16, N % 16 == 0, K % 32 == 0

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
