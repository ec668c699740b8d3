// Argument blocks and launcher prototypes of windowed attention (pq_window_attn.hip) and of the recurrent mixers
// (pq_recurrent.hip), shared with their C-ABI translation unit.  Each launcher returns a hipError_t cast to int (0 = ok).
// dtype: 0 float16, 1 bfloat16, 2 float32.
#pragma once
#include <hip/hip_runtime.h>
#include <stddef.h>
#include <stdint.h>

namespace pq {

// ---- windowed attention ----------------------------------------------------------------------------------------------
// The ring of a sequence holds the key of position j in row j % cap; cap is a multiple of 64, so that a tile of 64 keys
// that begins at a multiple of 64 is contiguous.
struct QkNormArgs {
    const void *q, *k, *v;   // columns of the projection output, rows p_row apart: [B * L, H * D], [.., G * D], [.., G * Dv]
    int64_t p_row;
    const void *w_q, *w_k;   // norm weights over all rows of q and of k
    void* q_out;             // [B * L, H * D]
    void* k_out;             // [B * L, G * D], or null: keys and values go to the ring
    void *k_ring, *v_ring;   // [B, G, cap, D], [B, G, cap, Dv]
    const int32_t* pos_dev;
    int pos, B, L, H, G, D, Dv, cap;
    float eps;
};
int launch_qk_norm(const QkNormArgs& a, int dtype, hipStream_t st);

struct RingAppendArgs {
    const void *k, *v;       // [B * L, G * D] rows k_row apart, [B * L, G * Dv] rows v_row apart
    int64_t k_row, v_row;
    void *k_ring, *v_ring;
    int pos, B, L, G, D, Dv, cap;
};
int launch_ring_append(const RingAppendArgs& a, int dtype, hipStream_t st);

struct WindowAttnArgs {
    const void* q;           // [B, L, H, D]
    const void *k_ring, *v_ring;
    const void *k_new, *v_new;   // the call's own keys and values, rows k_row / v_row apart; null: in the ring already
    int64_t k_row, v_row;
    const float* slopes;     // [H] taken off a score per position of distance, or null
    const int32_t* start;    // [B] position of each sequence's first token, or null
    const int32_t* pos_dev;
    void* out;               // [B * L, H * Dv] rows out_row apart
    int64_t out_row;
    float* workspace;
    int pos, B, L, H, G, D, Dv, cap, window, n_splits;
    float scale, out_scale;
};
constexpr int kWindowSmallTokens = 16;       // up to this many new tokens the keys go to the ring first
inline bool window_mfma(int D, int Dv, int dtype) { return dtype != 2 && D % 8 == 0 && Dv % 8 == 0 && D <= 256 && Dv <= 256; }
int launch_window_decode(const WindowAttnArgs& a, int dtype, hipStream_t st);
int launch_window_prefill(const WindowAttnArgs& a, int dtype, hipStream_t st);
int launch_window_plain(const WindowAttnArgs& a, int dtype, hipStream_t st);

// ---- recurrent mixers ------------------------------------------------------------------------------------------------
struct DeltaPrepArgs {
    const void *q, *k, *v, *b;   // columns of the projection output, rows p_row apart: G * dim, G * dim, H * vdim, H
    int64_t p_row;
    const void* a;               // [B * L, H * dim] rows a_row apart: decay input before its bias
    int64_t a_row;
    const void *w_q, *w_k, *w_v; // [channels, taps]
    const void *A_log, *dt_bias; // [H], [H * dim]
    const float* state_in;       // [B, taps - 1, 2 G dim + H vdim], oldest first
    float* state_out;
    void *q_out, *k_out, *v_out; // [B * L, channels] after convolution and silu
    float *q_inv, *k_inv;        // [B * L, G] 1 / length of each head's vector (the query's also times dim^-1/2)
    float* log_g;                // [B * L, H * dim]
    float* beta;                 // [B * L, H]
    const int32_t* start;
    const int32_t* pos_dev;
    int pos, B, L, G, H, dim, vdim, taps, strip;
};
int launch_delta_prep(const DeltaPrepArgs& a, int dtype, hipStream_t st);

struct MemoryGateArgs {
    const void *i, *f;           // [B * L, H] rows p_row apart
    int64_t p_row;
    const void *b_i, *b_f;       // [H]
    float *log_i, *log_f;        // [B * L, H]
    int64_t rows;
    int H;
    float cap;
};
int launch_memory_gates(const MemoryGateArgs& a, int dtype, hipStream_t st);

// State of a head: [columns, dim] float32, one row per value channel (and one for the normalizer n of a matrix memory).
struct ScanArgs {
    const void *q, *k, *v;       // rows q_row, k_row, v_row apart; head h reads q / k head h / (H / G)
    int64_t q_row, k_row, v_row;
    const float *q_inv, *k_inv;  // delta rule: [B * L, G]
    const float* log_g;          // delta rule: [B * L, H * dim]
    const float* beta;           // delta rule: [B * L, H]
    const float *log_i, *log_f;  // matrix memory: [B * L, H]
    float* state;                // [B, H, columns, dim]
    float* m;                    // matrix memory: [B, H, column blocks of 16] running maximum, one copy for each workgroup
    float* o;                    // [B * L, H, vdim]
    float* den;                  // matrix memory: [B * L, H]
    const int32_t* start;
    const int32_t* pos_dev;
    int pos, B, L, G, H, dim, vdim;
    float q_scale;               // matrix memory
};
constexpr int kScanMaxDim = 256;
int launch_delta_scan(const ScanArgs& a, int dtype, hipStream_t st);
int launch_memory_scan(const ScanArgs& a, int dtype, hipStream_t st);

// Both over many tokens, in chunks (pq_recurrent_chunk.hip): 16-bit dtypes, dim <= kScanMaxDim.
constexpr int kRecurrentChunk = 32;
struct ChunkArgs : ScanArgs {
    char* workspace;             // [B, H, chunks] blocks of chunk_block_bytes
    int t0, chunks;              // the segment: its first token in the call, how many chunks
    int prefetch;                // chunks ahead of the walk whose lines are fetched into L2 (set by the launcher)
};
size_t chunk_block_bytes(bool delta, int dim, int dtype);
int launch_delta_chunks(const ChunkArgs& a, size_t workspace_bytes, int dtype, hipStream_t st);
int launch_memory_chunks(const ChunkArgs& a, size_t workspace_bytes, int dtype, hipStream_t st);

struct HeadNormGateArgs {
    const float* o;              // [rows, H, vdim]
    const float* den;            // [rows, H] divisors, or null
    const void* w;               // [vdim] or [H * vdim] (w_head = 0 or vdim)
    int w_head;
    const void* gate;            // [rows, H * vdim] rows gate_row apart
    int64_t gate_row;
    void* out;                   // [rows, H * vdim] rows out_row apart
    int64_t out_row, rows;
    int H, vdim;
    float eps, out_scale;
};
int launch_head_norm_gate(const HeadNormGateArgs& a, int dtype, hipStream_t st);

}  // namespace pq
