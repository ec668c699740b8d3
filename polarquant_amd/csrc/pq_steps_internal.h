// Argument blocks and launcher prototypes of the steps between mixers and matrix products (pq_steps.hip,
// pq_head_linear.hip), shared with their C-ABI translation unit.  Each launcher returns a hipError_t cast to int (0 = ok).
// dtype: 0 float16, 1 bfloat16, 2 float32.
#pragma once
#include <hip/hip_runtime.h>
#include <stddef.h>
#include <stdint.h>

namespace pq {

struct NormConvArgs {
    const float* x_in;       // [B, L, W] residual stream
    const void* y;           // [B, L, W] output of the previous sublayer, or null
    const void* w_post;      // [W] weight of the norm applied to y; null: y is added as it is
    float* x_out;            // [B, L, W] x_in + norm(y), or x_in + y
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

int launch_relu_sq(const void* x, void* y, size_t n, int dtype, hipStream_t st);

struct GeluMulArgs {
    const void *gate, *up;   // [rows, cols] rows in_stride apart
    void* y;
    int64_t rows, in_stride, out_stride;
    int cols;
};
int launch_gelu_mul(const GeluMulArgs& a, int dtype, hipStream_t st);

struct StreamAddArgs {
    const float* x;          // [rows, width]
    const void* y;           // sublayer output in the dtype, or null
    const float* e;          // another stream, or null
    const void* v;           // [width], or null
    float* x_out;            // may be x
    int64_t rows;
    int width;
};
int launch_stream_add(const StreamAddArgs& a, int dtype, hipStream_t st);
int launch_embed_rows(const void* table, const int64_t* ids, float scale, float* out, int64_t rows, int width, int64_t vocab, int dtype, hipStream_t st);
int launch_softcap(float* x, size_t n, float scale, float cap, hipStream_t st);

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
int launch_head_linear_any(const HeadLinearArgs& a, int dtype, hipStream_t st);      // pq_steps.hip: any size, any dtype
int launch_head_linear_mfma(const HeadLinearArgs& a, int dtype, hipStream_t st);     // pq_head_linear.hip: M <= 16, N % 16 == 0, K % 32 == 0

}  // namespace pq
