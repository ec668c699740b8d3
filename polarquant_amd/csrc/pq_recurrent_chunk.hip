// The recurrences of pq_recurrent.hip over many tokens, 32 at a time on the matrix cores (16-bit models; heads up to 256 wide).
//
// Delta rule.  Within a chunk let L_t be the cumulative log decay of a key channel, S the state before it, and
//     K'_t = e^{L_t} k_t,   Q'_t = e^{L_t} q_t,   K^_s = e^{L_end - L_s} k_s,
//     A_ts = beta_t sum_c k_t k_s e^{L_t - L_s}  (s < t),   P_ts = sum_c q_t k_s e^{L_t - L_s}  (s <= t),
//     T = (1 + A)^{-1} diag(beta).
// Then U = T (V - K' S), O = Q' S + P U, S <- e^{L_end} S + K^^T U: everything but U, O, S is the same for all columns of S and
// needs no earlier chunk.
//
// Matrix memory.  With F_t the cumulative log forget gate, M_t = max_{s <= t} (F_t - F_s + i_s), w_s = e^{F_end - F_s + i_s - M_end}
// and P_ts = q_t.k_s e^{F_t - F_s + i_s - M_t}: m_t = max(F_t + m, M_t), O_t = e^{F_t + m - m_t} q_t S + e^{M_t - m_t} (P V)_t,
// S <- e^{F_end + m - m_end} S + e^{M_end - m_end} sum_s k_s (w_s v_s)^T.
//
//   delta_chunk_kernel, memory_chunk_kernel   what does not depend on the state, a workgroup per chunk and head, written
//                                             in the order in which the matrix cores take their left operands
//   delta_walk_kernel, memory_walk_kernel     the chunks in turn, four wavefronts per head and 16 columns of the state,
//                                             which stays in registers
//
// The products stand for float32 ones: each factor that is not a 16-bit number already is split into two bfloat16 numbers,
// x = hi + lo, and hi hi + hi lo + lo hi is added up in float32 (what is left out is 2^-16 of a term).  State, decays,
// exponentials and sums are float32.
//
// Operand layouts.  The state's accumulators hold channel 16 j + 4 g + i of tile j (g = lane / 16) in register i.  The order of a
// summed index is free as long as both operands agree, so the right operand "32 channels of S" is tiles 2 i and 2 i + 1 as
// they stand, eight values per lane, and left operands list their channels likewise: 32 i + 4 g + 0..3, then 16 more.  The
// same holds for the 32 tokens of R = V - K' S and of U.
#include "pq_mfma.h"
#include "pq_recurrent_internal.h"

namespace pq {

constexpr int kChunk = kRecurrentChunk;
static_assert(kChunk == 32, "two tiles of 16 tokens");
typedef float floatx2_a __attribute__((ext_vector_type(2)));
typedef __bf16 bf16x2_a __attribute__((ext_vector_type(2)));

__device__ __forceinline__ uint32_t pack_bf16(float a, float b) {
    return __builtin_bit_cast(uint32_t, __builtin_convertvector(floatx2_a{a, b}, bf16x2_a));
}
__device__ __forceinline__ void split2(float a, float b, uint32_t& hi, uint32_t& lo) {
    hi = pack_bf16(a, b);
    lo = pack_bf16(a - __uint_as_float(hi << 16), b - __uint_as_float(hi & 0xffff0000u));
}
// two tiles' registers as the right operand of 32 summed indices
__device__ __forceinline__ void split_tiles(const floatx4_a& x, const floatx4_a& y, u32x4_a& hi, u32x4_a& lo) {
    uint32_t h[4], l[4];
    split2(x[0], x[1], h[0], l[0]);
    split2(x[2], x[3], h[1], l[1]);
    split2(y[0], y[1], h[2], l[2]);
    split2(y[2], y[3], h[3], l[3]);
    hi = u32x4_a{h[0], h[1], h[2], h[3]};
    lo = u32x4_a{l[0], l[1], l[2], l[3]};
}
__device__ __forceinline__ floatx4_a mm(u32x4_a a, u32x4_a b, floatx4_a c) { return mma16<BF16>(a, b, c); }
__device__ __forceinline__ void lds_done() { asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory"); }       // this wavefront's own LDS writes

// ---- layout of a chunk's block in the workspace (bytes) -----------------------------------------------------------------------
template <int DP> struct DeltaBlock {
    static constexpr int kMat = kChunk * DP * 2, kSq = kChunk * kChunk * 2;
    static constexpr int k_in = 0, q_in = 2 * kMat, k_out = 4 * kMat, t = 6 * kMat, p = t + 2 * kSq, decay = p + 2 * kSq, size = decay + DP * 4;
};
template <int DP, bool SPLIT> struct MemoryBlock {
    static constexpr int kMat = kChunk * DP * 2, kSq = kChunk * kChunk * 2, parts = SPLIT ? 2 : 1;
    static constexpr int q_in = 0, k_out = parts * kMat, p = 2 * parts * kMat, f = p + 2 * kSq, m = f + kChunk * 4, w = m + kChunk * 4, size = w + kChunk * 4;
};

// a 32 x 32 matrix in LDS (rows of 36 floats, zero above the diagonal) as a left operand: two row tiles, high then low parts
constexpr int kSqRow = 36;
__device__ __forceinline__ void store_square(const float* mat, const float* scale, char* dst, int lane) {
    const int r16 = lane & 15, g = lane >> 4;
#pragma unroll
    for (int rt = 0; rt < 2; rt++) {
        const int t = rt * 16 + r16;
        float x[8];
#pragma unroll
        for (int e = 0; e < 8; e++) {
            const int s = 4 * g + (e & 3) + 16 * (e >> 2);
            x[e] = s <= t ? mat[t * kSqRow + s] * (scale ? scale[s] : 1.0f) : 0.0f;
        }
        u32x4_a hi, lo;
        split_tiles(floatx4_a{x[0], x[1], x[2], x[3]}, floatx4_a{x[4], x[5], x[6], x[7]}, hi, lo);
        *reinterpret_cast<u32x4_a*>(dst + (rt * 64 + lane) * 16) = hi;
        *reinterpret_cast<u32x4_a*>(dst + kChunk * kChunk * 2 + (rt * 64 + lane) * 16) = lo;
    }
}

// ---- delta rule, per chunk -------------------------------------------------------------------------------------------------------
// grid (chunks of the segment, heads, sequences), 2 * DP threads: a thread holds one channel's 16 tokens of one half.
template <typename T, int DP>
__global__ __launch_bounds__(2 * DP) void delta_chunk_kernel(ChunkArgs a) {
    using Blk = DeltaBlock<DP>;
    constexpr int ROW = DP + 8, NW = 2 * DP / kWave, KS = DP / 32;
    extern __shared__ __attribute__((aligned(16))) char sm[];
    uint16_t* arr = reinterpret_cast<uint16_t*>(sm);                 // six [32][ROW]; or three [32][DP] of floats
    constexpr int kArr = kChunk * ROW;
    float* sq = reinterpret_cast<float*>(sm + 6 * kArr * 2);
    float *Am = sq, *Pm = sq + kChunk * kSqRow, *Tm = Pm + kChunk * kSqRow, *tot = Tm + kChunk * kSqRow, *beta = tot + 2 * DP;
    const int tid = threadIdx.x, lane = tid & 63, wv = tid / kWave, c = tid % DP, half = tid / DP;
    const int chunk = blockIdx.x, h = blockIdx.y, b = blockIdx.z, H = a.H, hk = h / (H / a.G), dim = a.dim;
    const int first = a.start ? a.start[b] - a.pos : 0, t0 = a.t0 + chunk * kChunk;
    const size_t row0 = static_cast<size_t>(b) * a.L;
    char* out = a.workspace + (static_cast<size_t>(b * H + h) * gridDim.x + chunk) * Blk::size;
    auto real = [&](int t) { return t >= first && t < a.L; };

    float k[16], q[16], lam[16], cum = 0.0f;
    const bool has = c < dim;
    const int cc = has ? c : 0;
#pragma unroll
    for (int i = 0; i < 16; i++) {
        const int t = t0 + half * 16 + i;
        const size_t row = row0 + (t < a.L ? t : a.L - 1);
        const bool in = has && real(t);
        const float kv = ld1<T>(static_cast<const elem_t<T>*>(a.k) + row * a.k_row + static_cast<size_t>(hk) * dim + cc) * a.k_inv[row * a.G + hk];
        const float qv = ld1<T>(static_cast<const elem_t<T>*>(a.q) + row * a.q_row + static_cast<size_t>(hk) * dim + cc) * a.q_inv[row * a.G + hk];
        const float lg = a.log_g[(row * H + h) * dim + cc] * kLog2e;
        k[i] = in ? kv : 0.0f;
        q[i] = in ? qv : 0.0f;
        cum += in ? lg : 0.0f;
        lam[i] = cum;
    }
    tot[half * DP + c] = cum;
    if (tid < kChunk) beta[tid] = real(t0 + tid) ? a.beta[(row0 + t0 + tid) * H + h] : 0.0f;
    // A and P factor through the middle of the chunk, e^{L_t - r} times e^{r - L_s}, while neither factor leaves the range of a float
    const float far = half ? -lam[15] : lam[0] - cum;
    const bool extreme = __syncthreads_or(!(fabsf(far) <= 100.0f)) != 0;
    const float tot0 = tot[c], tot1 = tot[DP + c];
    if (!extreme) {
#pragma unroll
        for (int i = 0; i < 16; i++) {
            const float rel = half ? lam[i] : lam[i] - cum, e = exp2_hw(rel), ei = exp2_hw(-rel);
            const float x[3] = {k[i] * e, q[i] * e, k[i] * ei};
#pragma unroll
            for (int j = 0; j < 3; j++) {
                const uint16_t hi = f2lo<BF16>(x[j]);
                arr[(2 * j) * kArr + (half * 16 + i) * ROW + c] = hi;
                arr[(2 * j + 1) * kArr + (half * 16 + i) * ROW + c] = f2lo<BF16>(x[j] - lo2f<BF16>(hi));
            }
        }
        __syncthreads();
        const int r16 = lane & 15, g = lane >> 4;
        for (int task = wv; task < 8; task += NW) {                  // matrix, row tile, column tile
            const int mat = task >> 2, rt = (task >> 1) & 1, ct = task & 1;
            float* dst = (mat ? Pm : Am) + (rt * 16 + 4 * g) * kSqRow + ct * 16 + r16;
            if (rt < ct) continue;                                   // (above the diagonal: not read)
            const uint16_t* left = arr + 2 * mat * kArr + (rt * 16 + r16) * ROW + 8 * g;
            const uint16_t* right = arr + 4 * kArr + (ct * 16 + r16) * ROW + 8 * g;
            floatx4_a s0 = {0, 0, 0, 0}, s1 = {0, 0, 0, 0};
            static_for<KS>([&](auto I) {
                constexpr int i = decltype(I)::value;
                const u32x4_a lh = *reinterpret_cast<const u32x4_a*>(left + i * 32), ll = *reinterpret_cast<const u32x4_a*>(left + kArr + i * 32);
                const u32x4_a rh = *reinterpret_cast<const u32x4_a*>(right + i * 32), rl = *reinterpret_cast<const u32x4_a*>(right + kArr + i * 32);
                s0 = mm(lh, rh, s0);
                s1 = mm(lh, rl, s1);
                s1 = mm(ll, rh, s1);
            });
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const int t = rt * 16 + 4 * g + i, s = ct * 16 + r16;
                const float v = s0[i] + s1[i];
                dst[i * kSqRow] = mat ? (s <= t ? v : 0.0f) : (s < t ? v * beta[t] : 0.0f);
            }
        }
    } else {
        float* fl = reinterpret_cast<float*>(sm);
#pragma unroll
        for (int i = 0; i < 16; i++) {
            const int t = half * 16 + i;
            fl[t * DP + c] = k[i];
            fl[(kChunk + t) * DP + c] = q[i];
            fl[(2 * kChunk + t) * DP + c] = lam[i] + (half ? tot0 : 0.0f);
        }
        __syncthreads();
        for (int e = tid; e < kChunk * kChunk; e += 2 * DP) {
            const int t = e / kChunk, s = e % kChunk;
            float ak = 0.0f, pq = 0.0f;
            if (s <= t) {
                for (int ch = 0; ch < dim; ch++) {
                    const float w = fl[s * DP + ch] * exp2_hw(fl[(2 * kChunk + t) * DP + ch] - fl[(2 * kChunk + s) * DP + ch]);
                    ak = __builtin_fmaf(fl[t * DP + ch], w, ak);
                    pq = __builtin_fmaf(fl[(kChunk + t) * DP + ch], w, pq);
                }
            }
            Am[t * kSqRow + s] = s < t ? ak * beta[t] : 0.0f;
            Pm[t * kSqRow + s] = pq;
        }
    }
    __syncthreads();
    // what the walk multiplies by: -K', Q' through LDS, K^ straight from the registers
#pragma unroll
    for (int i = 0; i < 16; i++) {
        const float e = exp2_hw(lam[i] + (half ? tot0 : 0.0f)), x[2] = {-k[i] * e, q[i] * e};
#pragma unroll
        for (int j = 0; j < 2; j++) {
            const uint16_t hi = f2lo<BF16>(x[j]);
            arr[(2 * j) * kArr + (half * 16 + i) * ROW + c] = hi;
            arr[(2 * j + 1) * kArr + (half * 16 + i) * ROW + c] = f2lo<BF16>(x[j] - lo2f<BF16>(hi));
        }
        k[i] *= exp2_hw(cum - lam[i] + (half ? 0.0f : tot1));
    }
#pragma unroll
    for (int g = 0; g < 4; g++) {
        uint32_t hi[2], lo[2];
        split2(k[4 * g], k[4 * g + 1], hi[0], lo[0]);
        split2(k[4 * g + 2], k[4 * g + 3], hi[1], lo[1]);
        char* d = out + Blk::k_out + (((c >> 4) * 64 + g * 16 + (c & 15)) * 8 + half * 4) * 2;
        *reinterpret_cast<u32x2_a*>(d) = u32x2_a{hi[0], hi[1]};
        *reinterpret_cast<u32x2_a*>(d + Blk::kMat) = u32x2_a{lo[0], lo[1]};
    }
    if (half == 0) reinterpret_cast<float*>(out + Blk::decay)[c] = exp2_hw(tot0 + tot1);
    __syncthreads();
    if (wv == 0) {
        // (1 + A)^{-1}: both diagonal blocks by substitution, a lane per column, then the block below them
        const int blk = (lane >> 4) & 1, col = lane & 15, o16 = blk * 16;
        float x[16];
#pragma unroll
        for (int t = 0; t < 16; t++) {
            float s = t == col ? 1.0f : 0.0f;
#pragma unroll
            for (int u = 0; u < t; u++) s = __builtin_fmaf(-Am[(o16 + t) * kSqRow + o16 + u], x[u], s);
            x[t] = s;
        }
        if (lane < 32)
#pragma unroll
            for (int t = 0; t < 16; t++) Tm[(o16 + t) * kSqRow + o16 + col] = x[t];
        lds_done();
        const int i = lane & 15, j4 = (lane >> 4) * 4;
        float4 m4 = make_float4(0, 0, 0, 0);
#pragma unroll
        for (int s = 0; s < 16; s++) {
            const float av = Am[(16 + i) * kSqRow + s];
            const float4 tv = *reinterpret_cast<const float4*>(Tm + s * kSqRow + j4);
            m4.x = __builtin_fmaf(av, tv.x, m4.x); m4.y = __builtin_fmaf(av, tv.y, m4.y);
            m4.z = __builtin_fmaf(av, tv.z, m4.z); m4.w = __builtin_fmaf(av, tv.w, m4.w);
        }
        *reinterpret_cast<float4*>(Tm + i * kSqRow + 16 + j4) = m4;         // (scratch: the block above the diagonal is not read)
        lds_done();
        float4 n4 = make_float4(0, 0, 0, 0);
#pragma unroll
        for (int s = 0; s < 16; s++) {
            const float tv = -Tm[(16 + i) * kSqRow + 16 + s];
            const float4 mv = *reinterpret_cast<const float4*>(Tm + s * kSqRow + 16 + j4);
            n4.x = __builtin_fmaf(tv, mv.x, n4.x); n4.y = __builtin_fmaf(tv, mv.y, n4.y);
            n4.z = __builtin_fmaf(tv, mv.z, n4.z); n4.w = __builtin_fmaf(tv, mv.w, n4.w);
        }
        *reinterpret_cast<float4*>(Tm + (16 + i) * kSqRow + j4) = n4;
        lds_done();
        store_square(Tm, beta, out + Blk::t, lane);
        store_square(Pm, nullptr, out + Blk::p, lane);
    } else {
        for (int u = tid - kWave; u < 4 * 2 * KS * 64; u += 2 * DP - kWave) {
            const int m = u / (2 * KS * 64), rest = u % (2 * KS * 64), rt = rest / (KS * 64), i = rest / 64 % KS, l = rest & 63;
            const uint16_t* s = arr + m * kArr + (rt * 16 + (l & 15)) * ROW + i * 32 + 4 * (l >> 4);
            const u32x2_a w0 = *reinterpret_cast<const u32x2_a*>(s), w1 = *reinterpret_cast<const u32x2_a*>(s + 16);
            *reinterpret_cast<u32x4_a*>(out + m * Blk::kMat + rest * 16) = u32x4_a{w0.x, w0.y, w1.x, w1.y};
        }
    }
}

// ---- delta rule, the chunks in turn --------------------------------------------------------------------------------------------
template <int NT> __device__ __forceinline__ void load_state(const float* sp, int dim, int g, floatx4_a (&S)[NT]) {
    static_for<NT>([&](auto J) {
        constexpr int j = decltype(J)::value;
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int c = 16 * j + 4 * g + i;
            S[j][i] = c < dim ? sp[c] : 0.0f;
        }
    });
}
template <int NT> __device__ __forceinline__ void store_state(float* sp, int dim, int g, const floatx4_a (&S)[NT]) {
    static_for<NT>([&](auto J) {
        constexpr int j = decltype(J)::value;
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int c = 16 * j + 4 * g + i;
            if (c < dim) sp[c] = S[j][i];
        }
    });
}

// A lane's four tokens of a row tile of a chunk, 16 rt + 4 g + i: their values as they are stored (converted when they are used,
// so that nothing waits for them before).  Past the call's last token the last one is read.
template <typename T> struct Rows {
    const uint16_t* v;           // row 0 of the sequence's values, column 0 of the head
    uint32_t stride, col;
    int L, row;                  // row: the first of the four in the chunk
    uint32_t off[4], raw[4];
    __device__ __forceinline__ void offsets(int last) {
#pragma unroll
        for (int i = 0; i < 4; i++) off[i] = static_cast<uint32_t>(row + i < last ? row + i : last) * stride + col;
    }
    __device__ __forceinline__ void load(int t) {
        const uint16_t* base = v + static_cast<size_t>(t) * stride;
        if (L - 1 - t < kChunk - 1) offsets(L - 1 - t);              // uniform: the sequence's last chunk
#pragma unroll
        for (int i = 0; i < 4; i++) raw[i] = base[off[i]];
    }
    __device__ __forceinline__ floatx4_a get() const {
        return floatx4_a{lo2f<T>(static_cast<uint16_t>(raw[0])), lo2f<T>(static_cast<uint16_t>(raw[1])),
                         lo2f<T>(static_cast<uint16_t>(raw[2])), lo2f<T>(static_cast<uint16_t>(raw[3]))};
    }
};
template <typename T> __device__ __forceinline__ Rows<T> rows_of(const ChunkArgs& a, size_t row0, int h, int col, int row) {
    Rows<T> r{static_cast<const uint16_t*>(a.v) + row0 * a.v_row + static_cast<size_t>(h) * a.vdim, static_cast<uint32_t>(a.v_row),
              static_cast<uint32_t>(col), a.L, row, {}, {}};
    r.offsets(kChunk);
    return r;
}
// out: the chunk's first row; left: rows from there to the call's end
__device__ __forceinline__ void store_rows(float* out, uint32_t stride, uint32_t col, int row, int left, const floatx4_a& x) {
    const uint32_t off = row * stride + col;
    if (left >= kChunk) {                                            // uniform
#pragma unroll
        for (int i = 0; i < 4; i++) (out + i * static_cast<size_t>(stride))[off] = x[i];
    } else {
#pragma unroll
        for (int i = 0; i < 4; i++)
            if (row + i < left) (out + i * static_cast<size_t>(stride))[off] = x[i];
    }
}

// Four wavefronts share a walk, one on each SIMD.  The first two carry the state along, half of the channels each, and leave in
// LDS what the other two multiply by Q' and P for the results, a row tile each.  Loads stay in flight across the barriers.
__device__ __forceinline__ void walk_barrier() {
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
}
// chunks whose operands are in flight ahead of the one worked on, each in registers of its own
constexpr int kWalkAhead = 1;
template <int AHEAD, typename F> __device__ __forceinline__ void walk_chunks(int chunks, F&& step) {
    for (int n = 0; n < chunks; n += AHEAD)
        static_for<AHEAD>([&](auto P) {
            if (n + P < chunks) step(P, n + P);
        });
}

// The workgroups of a head fetch the lines of a chunk still further ahead into their L2 in turn, one load each: the operands
// come from the last-level cache or memory.  The value is dropped, a chunk's time or more after the load.
struct LineFetch {
    const char* base;
    int block_bytes, ahead, chunks;
    uint32_t off, got;
    __device__ __forceinline__ void go(int n) {
        const int m = n + ahead < chunks ? n + ahead : chunks - 1;
        got = *reinterpret_cast<const uint32_t*>(base + static_cast<size_t>(m) * block_bytes + off);
    }
    __device__ __forceinline__ void drop() const { asm volatile("" ::"v"(got)); }
};
__device__ __forceinline__ LineFetch line_fetch(const char* base, int block_bytes, const ChunkArgs& a, int lane) {
    const uint32_t off = static_cast<uint32_t>(lane * static_cast<int>(gridDim.y) + static_cast<int>(blockIdx.y)) * 128u, last = block_bytes - 4;
    return LineFetch{base, block_bytes, a.prefetch, a.chunks, off < last ? off : last, 0u};
}

// grid (heads, column blocks of 16, sequences): with a multiple of 8 heads all columns of a head run on one XCD and read its
// operands from one L2.  Every operand is loaded again right after its use (the scheduling barriers keep the compiler from
// moving those loads to where their results are needed).  Two barriers per chunk: the halves of K' S are added up between
// them, while the read-out multiplies the state; U follows the second.
template <typename T, int DP>
__global__ __launch_bounds__(4 * kWave, 1) void delta_walk_kernel(ChunkArgs a) {
    using Blk = DeltaBlock<DP>;
    constexpr int KS = DP / 32, KH = KS / 2, NH = DP / 32, AHEAD = kWalkAhead;
    __shared__ u32x4_a sh_s[2][KS][kWave], sh_u[2][kWave];           // high and low parts
    __shared__ floatx4_a sh_r[2][2][kWave];                          // [half][row tile]
    const int lane = threadIdx.x & 63, wv = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), r16 = lane & 15, g = lane >> 4;
    const int h = blockIdx.x, b = blockIdx.z, H = a.H, col = blockIdx.y * 16 + r16, cc = col < a.vdim ? col : a.vdim - 1;
    const size_t row0 = static_cast<size_t>(b) * a.L;
    const char* base = a.workspace + static_cast<size_t>(b * H + h) * a.chunks * Blk::size;
    const uint32_t lane16 = lane * 16, g16 = g * 16;
    auto at = [&](const char* blk, int off) { return *reinterpret_cast<const u32x4_a*>(blk + off + lane16); };
    if (wv < 2) {
        __builtin_amdgcn_s_setprio(3);                               // (ahead of another segment's chunks on the same compute unit)
        const int c0 = wv * (DP / 2);                                // this wavefront's first channel
        float* sp = a.state + ((static_cast<size_t>(b) * H + h) * a.vdim + cc) * a.dim + c0;
        floatx4_a S[NH], dec[AHEAD][NH];
        load_state<NH>(sp, a.dim - c0, g, S);
        u32x4_a ki[AHEAD][2][2][KH], ko[AHEAD][2][NH], tm[AHEAD][2][2];      // [chunk][part][row tile]..
        Rows<T> v[AHEAD];                                            // of row tile wv
        auto load_ki = [&](auto P, const char* blk) {
            constexpr int p = decltype(P)::value;
            static_for<2 * KH>([&](auto I) {
                constexpr int i = decltype(I)::value, rt = i / KH, k = i % KH;
                const char* src = blk + Blk::k_in + wv * KH * 1024;
                ki[p][0][rt][k] = at(src, (rt * KS + k) * 1024);
                ki[p][1][rt][k] = at(src, Blk::kMat + (rt * KS + k) * 1024);
            });
        };
        auto load_ko = [&](auto P, const char* blk) {
            constexpr int p = decltype(P)::value;
            static_for<NH>([&](auto J) {
                constexpr int j = decltype(J)::value;
                const char* src = blk + Blk::k_out + wv * NH * 1024;
                ko[p][0][j] = at(src, j * 1024);
                ko[p][1][j] = at(src, Blk::kMat + j * 1024);
            });
        };
        auto load_t = [&](auto P, const char* blk) {
            constexpr int p = decltype(P)::value;
            static_for<2>([&](auto I) {
                constexpr int i = decltype(I)::value;
                tm[p][0][i] = at(blk, Blk::t + i * 1024);
                tm[p][1][i] = at(blk, Blk::t + Blk::kSq + i * 1024);
            });
        };
        auto load_dec = [&](auto P, const char* blk) {
            constexpr int p = decltype(P)::value;
            static_for<NH>([&](auto J) {
                constexpr int j = decltype(J)::value;
                dec[p][j] = *reinterpret_cast<const floatx4_a*>(blk + Blk::decay + wv * NH * 64 + j * 64 + g16);
            });
        };
        static_for<AHEAD>([&](auto P) {
            constexpr int p = decltype(P)::value;
            const int n = p < a.chunks ? p : a.chunks - 1;
            const char* blk = base + static_cast<size_t>(n) * Blk::size;
            v[p] = rows_of<T>(a, row0, h, cc, wv * 16 + 4 * g);
            v[p].load(a.t0 + n * kChunk);
            load_ki(P, blk);
            load_dec(P, blk);
            load_t(P, blk);
            load_ko(P, blk);
        });
        auto step = [&](auto P, int n) {
            constexpr int p = decltype(P)::value;
            const int next = n + AHEAD < a.chunks ? n + AHEAD : a.chunks - 1;
            const char* blk = base + static_cast<size_t>(next) * Blk::size;
            const floatx4_a zero = {0, 0, 0, 0}, V = v[p].get();
            floatx4_a R[2] = {wv == 0 ? V : zero, wv == 0 ? zero : V}, R1[2] = {zero, zero};
            __builtin_amdgcn_sched_barrier(0);
            v[p].load(a.t0 + next * kChunk);
            __builtin_amdgcn_sched_barrier(0);
            static_for<KH>([&](auto I) {
                constexpr int i = decltype(I)::value;
                u32x4_a hi, lo;
                split_tiles(S[2 * i], S[2 * i + 1], hi, lo);
                sh_s[0][wv * KH + i][lane] = hi;
                sh_s[1][wv * KH + i][lane] = lo;
#pragma unroll
                for (int rt = 0; rt < 2; rt++) {
                    R[rt] = mm(ki[p][0][rt][i], hi, R[rt]);
                    R1[rt] = mm(ki[p][0][rt][i], lo, R1[rt]);
                    R1[rt] = mm(ki[p][1][rt][i], hi, R1[rt]);
                }
                S[2 * i] *= dec[p][2 * i];
                S[2 * i + 1] *= dec[p][2 * i + 1];
            });
#pragma unroll
            for (int rt = 0; rt < 2; rt++) {
                R[rt] += R1[rt];
                sh_r[wv][rt][lane] = R[rt];
            }
            __builtin_amdgcn_sched_barrier(0);
            load_ki(P, blk);
            load_dec(P, blk);
            __builtin_amdgcn_sched_barrier(0);
            walk_barrier();
            u32x4_a xh, xl;
            split_tiles(R[0] + sh_r[1 - wv][0][lane], R[1] + sh_r[1 - wv][1][lane], xh, xl);
            floatx4_a U[2], U1[2];
#pragma unroll
            for (int rt = 0; rt < 2; rt++) {
                U[rt] = mm(tm[p][0][rt], xh, zero);
                U1[rt] = mm(tm[p][0][rt], xl, zero);
                U1[rt] = mm(tm[p][1][rt], xh, U1[rt]);
            }
            __builtin_amdgcn_sched_barrier(0);
            load_t(P, blk);
            __builtin_amdgcn_sched_barrier(0);
            split_tiles(U[0] + U1[0], U[1] + U1[1], xh, xl);
            if (wv == 0) {
                sh_u[0][lane] = xh;
                sh_u[1][lane] = xl;
            }
            static_for<NH>([&](auto J) { constexpr int j = decltype(J)::value; S[j] = mm(ko[p][0][j], xh, S[j]); });
            static_for<NH>([&](auto J) { constexpr int j = decltype(J)::value; S[j] = mm(ko[p][0][j], xl, S[j]); });
            static_for<NH>([&](auto J) { constexpr int j = decltype(J)::value; S[j] = mm(ko[p][1][j], xh, S[j]); });
            __builtin_amdgcn_sched_barrier(0);
            load_ko(P, blk);
            __builtin_amdgcn_sched_barrier(0);
            walk_barrier();
        };
        walk_chunks<AHEAD>(a.chunks, step);
        if (col < a.vdim) store_state<NH>(sp, a.dim - c0, g, S);
    } else {
        const int rt = wv - 2, row = rt * 16 + 4 * g;
        float* op = a.o + (row0 * H + h) * a.vdim;
        const uint32_t o_stride = static_cast<uint32_t>(H) * a.vdim;
        u32x4_a qi[AHEAD][2][KS], pm[AHEAD][2];
        auto load_q = [&](auto P, const char* blk) {
            constexpr int p = decltype(P)::value;
            static_for<KS>([&](auto I) {
                constexpr int i = decltype(I)::value;
                const char* src = blk + Blk::q_in + rt * KS * 1024;
                qi[p][0][i] = at(src, i * 1024);
                qi[p][1][i] = at(src, Blk::kMat + i * 1024);
            });
        };
        auto load_p = [&](auto P, const char* blk) {
            constexpr int p = decltype(P)::value;
            pm[p][0] = at(blk + rt * 1024, Blk::p);
            pm[p][1] = at(blk + rt * 1024, Blk::p + Blk::kSq);
        };
        static_for<AHEAD>([&](auto P) {
            const char* blk = base + static_cast<size_t>(P < a.chunks ? static_cast<int>(P) : a.chunks - 1) * Blk::size;
            load_q(P, blk);
            load_p(P, blk);
        });
        LineFetch lines = line_fetch(base, Blk::size, a, lane);
        lines.go(0);
        auto step = [&](auto P, int n) {
            constexpr int p = decltype(P)::value;
            const int t = a.t0 + n * kChunk, next = n + AHEAD < a.chunks ? n + AHEAD : a.chunks - 1;
            const char* blk = base + static_cast<size_t>(next) * Blk::size;
            floatx4_a O = {0, 0, 0, 0}, O1 = {0, 0, 0, 0};
            walk_barrier();
            static_for<KS>([&](auto I) {
                constexpr int i = decltype(I)::value;
                const u32x4_a hi = sh_s[0][i][lane], lo = sh_s[1][i][lane];
                O = mm(qi[p][0][i], hi, O);
                O1 = mm(qi[p][0][i], lo, O1);
                O1 = mm(qi[p][1][i], hi, O1);
            });
            __builtin_amdgcn_sched_barrier(0);
            load_q(P, blk);
            __builtin_amdgcn_sched_barrier(0);
            walk_barrier();
            const u32x4_a xh = sh_u[0][lane], xl = sh_u[1][lane];
            O = mm(pm[p][0], xh, O);
            O1 = mm(pm[p][0], xl, O1);
            O1 = mm(pm[p][1], xh, O1);
            __builtin_amdgcn_sched_barrier(0);
            load_p(P, blk);
            if (rt == 0) {
                lines.drop();
                lines.go(n + 1);
            }
            __builtin_amdgcn_sched_barrier(0);                       // (the stores stay behind the loads)
            if (col < a.vdim) store_rows(op + static_cast<size_t>(t) * o_stride, o_stride, col, row, a.L - t, O + O1);
        };
        walk_chunks<AHEAD>(a.chunks, step);
    }
}

// ---- matrix memory, per chunk ------------------------------------------------------------------------------------------------------
// grid (chunks of the segment, heads, sequences), 256 threads
template <typename T, int DP>
__global__ __launch_bounds__(256) void memory_chunk_kernel(ChunkArgs a) {
    constexpr bool SPLIT = __is_same(T, F16);                        // (a bfloat16 number is its own high part)
    using Blk = MemoryBlock<DP, SPLIT>;
    constexpr int ROW = DP + 8, KS = DP / 32, NT = DP / 16, kArr = kChunk * ROW;
    extern __shared__ __attribute__((aligned(16))) char sm[];
    uint16_t* arr = reinterpret_cast<uint16_t*>(sm);                 // [32][ROW]: q, k, and with SPLIT their low parts
    float* Pm = reinterpret_cast<float*>(sm + (SPLIT ? 4 : 2) * kArr * 2);
    float *F = Pm + kChunk * kSqRow, *M = F + kChunk, *I = M + kChunk;
    const int tid = threadIdx.x, lane = tid & 63, wv = tid / kWave, chunk = blockIdx.x, h = blockIdx.y, b = blockIdx.z, H = a.H, dim = a.dim;
    const int first = a.start ? a.start[b] - a.pos : 0, t0 = a.t0 + chunk * kChunk;
    const size_t row0 = static_cast<size_t>(b) * a.L;
    char* out = a.workspace + (static_cast<size_t>(b * H + h) * gridDim.x + chunk) * Blk::size;
    for (int u = tid; u < kChunk * DP; u += 256) {
        const int t = u / DP, c = u % DP;
        const bool in = c < dim && t0 + t >= first && t0 + t < a.L;
        const size_t row = row0 + (t0 + t < a.L ? t0 + t : a.L - 1), cc = static_cast<size_t>(h) * dim + (c < dim ? c : 0);
        const float x[2] = {ld1<T>(static_cast<const elem_t<T>*>(a.q) + row * a.q_row + cc), ld1<T>(static_cast<const elem_t<T>*>(a.k) + row * a.k_row + cc)};
#pragma unroll
        for (int j = 0; j < 2; j++) {
            const uint16_t hi = f2lo<BF16>(in ? x[j] : 0.0f);
            arr[j * kArr + t * ROW + c] = hi;
            if (SPLIT) arr[(2 + j) * kArr + t * ROW + c] = f2lo<BF16>(in ? x[j] - lo2f<BF16>(hi) : 0.0f);
        }
    }
    if (wv == 0) {
        const int t = lane & 31;
        const bool in = t0 + t >= first && t0 + t < a.L;
        const size_t row = row0 + (t0 + t < a.L ? t0 + t : a.L - 1);
        float f = in ? a.log_f[row * H + h] * kLog2e : 0.0f;
        const float li = in ? a.log_i[row * H + h] * kLog2e : -1.0e30f;       // (a token that is not there: no weight, and its k is zero)
#pragma unroll
        for (int d = 1; d < 32; d <<= 1) {
            const float o = __shfl_up(f, d, 32);
            f += t >= d ? o : 0.0f;
        }
        float m = li - f;
#pragma unroll
        for (int d = 1; d < 32; d <<= 1) {
            const float o = __shfl_up(m, d, 32);
            m = t >= d ? fmaxf(m, o) : m;
        }
        m += f;
        const float f_end = __shfl(f, 31, 32), m_end = __shfl(m, 31, 32);
        if (lane < 32) {
            F[t] = f;
            M[t] = m;
            I[t] = li;
            reinterpret_cast<float*>(out + Blk::f)[t] = f;
            reinterpret_cast<float*>(out + Blk::m)[t] = m;
            reinterpret_cast<float*>(out + Blk::w)[t] = in ? exp2_hw(f_end - f + li - m_end) : 0.0f;
        }
    }
    __syncthreads();
    const int r16 = lane & 15, g = lane >> 4;
    if (wv != 1) {                                                   // three lower tiles of q k^T
        const int rt = wv == 0 ? 0 : 1, ct = wv == 3 ? 1 : 0;
        const uint16_t *left = arr + (rt * 16 + r16) * ROW + 8 * g, *right = arr + kArr + (ct * 16 + r16) * ROW + 8 * g;
        floatx4_a s = {0, 0, 0, 0};
        static_for<KS>([&](auto J) {
            constexpr int i = decltype(J)::value;
            const u32x4_a lh = *reinterpret_cast<const u32x4_a*>(left + i * 32), rh = *reinterpret_cast<const u32x4_a*>(right + i * 32);
            s = mm(lh, rh, s);
            if constexpr (SPLIT) {
                s = mm(lh, *reinterpret_cast<const u32x4_a*>(right + 2 * kArr + i * 32), s);
                s = mm(*reinterpret_cast<const u32x4_a*>(left + 2 * kArr + i * 32), rh, s);
            }
        });
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int t = rt * 16 + 4 * g + i, u = ct * 16 + r16;
            Pm[t * kSqRow + u] = u <= t ? s[i] * exp2_hw(F[t] - F[u] + I[u] - M[t]) : 0.0f;
        }
    }
    for (int u = tid; u < Blk::parts * 2 * KS * 64; u += 256) {      // q
        const int part = u / (2 * KS * 64), rest = u % (2 * KS * 64), rt = rest / (KS * 64), i = rest / 64 % KS, l = rest & 63;
        const uint16_t* s = arr + part * 2 * kArr + (rt * 16 + (l & 15)) * ROW + i * 32 + 4 * (l >> 4);
        const u32x2_a w0 = *reinterpret_cast<const u32x2_a*>(s), w1 = *reinterpret_cast<const u32x2_a*>(s + 16);
        *reinterpret_cast<u32x4_a*>(out + Blk::q_in + part * Blk::kMat + rest * 16) = u32x4_a{w0.x, w0.y, w1.x, w1.y};
    }
    for (int u = tid; u < Blk::parts * NT * 64; u += 256) {          // k, a row per channel
        const int part = u / (NT * 64), rest = u % (NT * 64), l = rest & 63, c = (rest >> 6) * 16 + (l & 15), gg = l >> 4;
        const uint16_t* s = arr + (1 + part * 2) * kArr + c;
        uint32_t w[4];
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int t = 4 * gg + 2 * (e & 1) + 16 * (e >> 1);
            w[e] = static_cast<uint32_t>(s[t * ROW]) | (static_cast<uint32_t>(s[(t + 1) * ROW]) << 16);
        }
        *reinterpret_cast<u32x4_a*>(out + Blk::k_out + part * Blk::kMat + rest * 16) = u32x4_a{w[0], w[1], w[2], w[3]};
    }
    __syncthreads();
    if (wv == 0) store_square(Pm, nullptr, out + Blk::p, lane);
}

// grid (heads, column blocks of 16 with the normalizer's column, sequences), four wavefronts as above, the read-out a chunk behind
// (one barrier per chunk, two buffers).  Logarithms to base 2 throughout.
template <typename T, int DP>
__global__ __launch_bounds__(4 * kWave, 1) void memory_walk_kernel(ChunkArgs a) {
    constexpr bool SPLIT = __is_same(T, F16);
    using Blk = MemoryBlock<DP, SPLIT>;
    constexpr int KS = DP / 32, KH = KS / 2, NH = DP / 32, PT = Blk::parts, AHEAD = kWalkAhead;
    __shared__ u32x4_a sh_s[2][2][KS][kWave], sh_v[2][PT][kWave];    // [buffer][part]
    __shared__ float sh_m[2];
    const int lane = threadIdx.x & 63, wv = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), r16 = lane & 15, g = lane >> 4;
    const int h = blockIdx.x, b = blockIdx.z, H = a.H, columns = a.vdim + 1, col = blockIdx.y * 16 + r16;
    const bool value = col < a.vdim, norm = col == a.vdim;
    const size_t row0 = static_cast<size_t>(b) * a.L, head = static_cast<size_t>(b) * H + h;
    const char* base = a.workspace + head * a.chunks * Blk::size;
    const uint32_t lane16 = lane * 16, g16 = g * 16;
    auto at = [&](const char* blk, int off) { return *reinterpret_cast<const u32x4_a*>(blk + off + lane16); };
    auto scalars = [&](const char* blk, int off) { return *reinterpret_cast<const floatx4_a*>(blk + off + g16); };
    if (wv < 2) {
        __builtin_amdgcn_s_setprio(3);
        const int c0 = wv * (DP / 2);
        float* sp = a.state + (head * columns + (col < columns ? col : 0)) * a.dim + c0;
        float* mp = a.m + head * gridDim.y + blockIdx.y;
        floatx4_a S[NH], W[AHEAD][2];
        load_state<NH>(sp, a.dim - c0, g, S);
        float m = *mp * kLog2e, f_end[AHEAD], m_loc[AHEAD];
        u32x4_a ko[AHEAD][PT][NH];
        Rows<T> v[AHEAD][2];
        auto load_ko = [&](auto P, const char* blk) {
            constexpr int p = decltype(P)::value;
            static_for<PT * NH>([&](auto J) {
                constexpr int j = decltype(J)::value, part = j / NH, i = j % NH;
                ko[p][part][i] = at(blk + wv * NH * 1024, Blk::k_out + part * Blk::kMat + i * 1024);
            });
        };
        auto load_rest = [&](auto P, const char* blk, int t) {
            constexpr int p = decltype(P)::value;
            v[p][0].load(t);
            v[p][1].load(t);
            W[p][0] = scalars(blk, Blk::w);
            W[p][1] = scalars(blk, Blk::w + 64);
            f_end[p] = *reinterpret_cast<const float*>(blk + Blk::f + 31 * 4);
            m_loc[p] = *reinterpret_cast<const float*>(blk + Blk::m + 31 * 4);
        };
        static_for<AHEAD>([&](auto P) {
            constexpr int p = decltype(P)::value;
            const int n = p < a.chunks ? p : a.chunks - 1;
            const char* blk = base + static_cast<size_t>(n) * Blk::size;
            v[p][0] = rows_of<T>(a, row0, h, value ? col : 0, 4 * g);
            v[p][1] = rows_of<T>(a, row0, h, value ? col : 0, 16 + 4 * g);
            load_rest(P, blk, a.t0 + n * kChunk);
            load_ko(P, blk);
        });
        auto step = [&](auto P, int n) {
            constexpr int p = decltype(P)::value;
            const int buf = n & 1, next = n + AHEAD < a.chunks ? n + AHEAD : a.chunks - 1;
            const char* blk = base + static_cast<size_t>(next) * Blk::size;
            floatx4_a V[2] = {v[p][0].get(), v[p][1].get()};
            if (!value) V[0] = V[1] = floatx4_a{1, 1, 1, 1};
            const float m_end = fmaxf(f_end[p] + m, m_loc[p]), keep = exp2_hw(f_end[p] + m - m_end), take = exp2_hw(m_loc[p] - m_end);
            u32x4_a xh, xl;
            if (wv == 0) {
                if constexpr (SPLIT) {
                    split_tiles(V[0], V[1], xh, xl);
                    sh_v[buf][0][lane] = xh;
                    sh_v[buf][PT - 1][lane] = xl;
                } else {
                    sh_v[buf][0][lane] = u32x4_a{pack_bf16(V[0][0], V[0][1]), pack_bf16(V[0][2], V[0][3]), pack_bf16(V[1][0], V[1][1]), pack_bf16(V[1][2], V[1][3])};
                }
                if (lane == 0) sh_m[buf] = m;
            }
            split_tiles(V[0] * W[p][0] * take, V[1] * W[p][1] * take, xh, xl);
            __builtin_amdgcn_sched_barrier(0);
            load_rest(P, blk, a.t0 + next * kChunk);
            __builtin_amdgcn_sched_barrier(0);
            static_for<KH>([&](auto I) {
                constexpr int i = decltype(I)::value;
                u32x4_a hi, lo;
                split_tiles(S[2 * i], S[2 * i + 1], hi, lo);
                sh_s[buf][0][wv * KH + i][lane] = hi;
                sh_s[buf][1][wv * KH + i][lane] = lo;
                S[2 * i] *= keep;
                S[2 * i + 1] *= keep;
            });
            static_for<NH>([&](auto J) { constexpr int j = decltype(J)::value; S[j] = mm(ko[p][0][j], xh, S[j]); });
            static_for<NH>([&](auto J) { constexpr int j = decltype(J)::value; S[j] = mm(ko[p][0][j], xl, S[j]); });
            if constexpr (SPLIT) static_for<NH>([&](auto J) { constexpr int j = decltype(J)::value; S[j] = mm(ko[p][PT - 1][j], xh, S[j]); });
            __builtin_amdgcn_sched_barrier(0);
            load_ko(P, blk);
            __builtin_amdgcn_sched_barrier(0);
            m = m_end;
            walk_barrier();
        };
        walk_chunks<AHEAD>(a.chunks, step);
        if (col < columns) store_state<NH>(sp, a.dim - c0, g, S);
        __syncthreads();                                             // (both halves have read the maximum long since)
        if (threadIdx.x == 0) *mp = m / kLog2e;
    } else {
        const int rt = wv - 2, row = rt * 16 + 4 * g;
        float* op = a.o + (row0 * H + h) * a.vdim;
        float* np = a.den + row0 * H + h;
        const uint32_t o_stride = static_cast<uint32_t>(H) * a.vdim;
        u32x4_a qi[AHEAD][PT][KS], pm[AHEAD][2];
        floatx4_a F[AHEAD], M[AHEAD];
        auto load = [&](auto P, const char* blk) {
            constexpr int p = decltype(P)::value;
            static_for<PT * KS>([&](auto I) {
                constexpr int i = decltype(I)::value, part = i / KS, k = i % KS;
                qi[p][part][k] = at(blk + rt * KS * 1024, Blk::q_in + part * Blk::kMat + k * 1024);
            });
            pm[p][0] = at(blk + rt * 1024, Blk::p);
            pm[p][1] = at(blk + rt * 1024, Blk::p + Blk::kSq);
            F[p] = scalars(blk + rt * 64, Blk::f);
            M[p] = scalars(blk + rt * 64, Blk::m);
        };
        static_for<AHEAD>([&](auto P) { load(P, base + static_cast<size_t>(P < a.chunks ? static_cast<int>(P) : a.chunks - 1) * Blk::size); });
        LineFetch lines = line_fetch(base, Blk::size, a, lane);
        lines.go(0);
        auto step = [&](auto P, int n) {
            constexpr int p = decltype(P)::value;
            const int buf = n & 1, t = a.t0 + n * kChunk, next = n + AHEAD < a.chunks ? n + AHEAD : a.chunks - 1;
            walk_barrier();
            const float m = sh_m[buf];
            const u32x4_a vh = sh_v[buf][0][lane];
            floatx4_a O = {0, 0, 0, 0}, O1 = {0, 0, 0, 0}, Pv = {0, 0, 0, 0};
            static_for<KS>([&](auto I) {
                constexpr int i = decltype(I)::value;
                const u32x4_a hi = sh_s[buf][0][i][lane], lo = sh_s[buf][1][i][lane];
                O = mm(qi[p][0][i], hi, O);
                O1 = mm(qi[p][0][i], lo, O1);
                if constexpr (SPLIT) O1 = mm(qi[p][PT - 1][i], hi, O1);
            });
            Pv = mm(pm[p][0], vh, Pv);
            Pv = mm(pm[p][1], vh, Pv);
            if constexpr (SPLIT) Pv = mm(pm[p][0], sh_v[buf][PT - 1][lane], Pv);
            // m_t is the larger of F_t + m and M_t: one of the two weights is 1
            floatx4_a x, mt;
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const float old = F[p][i] + m, d = old - M[p][i], e = exp2_hw(-fabsf(d));
                x[i] = ((d >= 0.0f ? 1.0f : e) * (O[i] + O1[i]) + (d >= 0.0f ? e : 1.0f) * Pv[i]) * a.q_scale;
                mt[i] = fmaxf(old, M[p][i]);
            }
            __builtin_amdgcn_sched_barrier(0);
            load(P, base + static_cast<size_t>(next) * Blk::size);
            if (rt == 0) {
                lines.drop();
                lines.go(n + 1);
            }
            __builtin_amdgcn_sched_barrier(0);                       // (the stores stay behind the loads)
            if (value) store_rows(op + static_cast<size_t>(t) * o_stride, o_stride, col, row, a.L - t, x);
            if (norm) {
#pragma unroll
                for (int i = 0; i < 4; i++) x[i] = fmaxf(fabsf(x[i]), exp2_hw(-mt[i])) + 1e-6f;
                store_rows(np + static_cast<size_t>(t) * H, H, 0, row, a.L - t, x);
            }
        };
        walk_chunks<AHEAD>(a.chunks, step);
        __syncthreads();
    }
}

// ---- launchers -----------------------------------------------------------------------------------------------------------------------
constexpr int kOverlapChunks = 64;        // chunks of a segment from which on a second stream is worth its events
static int padded_dim(int dim) { return dim <= 64 ? 64 : dim <= 128 ? 128 : 256; }

size_t chunk_block_bytes(bool delta, int dim, int dtype) {
    const int dp = padded_dim(dim);
    const size_t mat = static_cast<size_t>(kChunk) * dp * 2, sq = kChunk * kChunk * 2;
    if (delta) return 6 * mat + 4 * sq + dp * 4;
    return (dtype == 0 ? 4 : 2) * mat + 2 * sq + 3 * kChunk * 4;
}

template <typename K>
static int with_lds(K kernel, size_t bytes) {
    if (bytes <= 64 * 1024) return 0;
    return static_cast<int>(hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(bytes)));
}

// one segment: its chunks' operands, or the walk over them
template <typename T, int DP>
static int delta_launch(const ChunkArgs& a, bool walk, hipStream_t st) {
    static_assert(DeltaBlock<DP>::size % 16 == 0, "16-byte operands");
    constexpr size_t lds = 6 * static_cast<size_t>(kChunk) * (DP + 8) * 2 + (3 * kChunk * kSqRow + 2 * DP + kChunk) * sizeof(float);
    static_assert(lds <= 160 * 1024 && 6 * (DP + 8) * 2 >= 3 * DP * 4, "LDS");
    if (walk) {
        hipLaunchKernelGGL((delta_walk_kernel<T, DP>), dim3(a.H, (a.vdim + 15) / 16, a.B), dim3(4 * kWave), 0, st, a);
    } else {
        if (int e = with_lds(&delta_chunk_kernel<T, DP>, lds)) return e;
        hipLaunchKernelGGL((delta_chunk_kernel<T, DP>), dim3(a.chunks, a.H, a.B), dim3(2 * DP), lds, st, a);
    }
    return static_cast<int>(hipGetLastError());
}

template <typename T, int DP>
static int memory_launch(const ChunkArgs& a, bool walk, hipStream_t st) {
    constexpr bool SPLIT = __is_same(T, F16);
    static_assert(MemoryBlock<DP, SPLIT>::size % 16 == 0, "16-byte operands");
    constexpr size_t lds = (SPLIT ? 4 : 2) * static_cast<size_t>(kChunk) * (DP + 8) * 2 + (kChunk * kSqRow + 3 * kChunk) * sizeof(float);
    if (walk) {
        hipLaunchKernelGGL((memory_walk_kernel<T, DP>), dim3(a.H, a.vdim / 16 + 1, a.B), dim3(4 * kWave), 0, st, a);
    } else {
        if (int e = with_lds(&memory_chunk_kernel<T, DP>, lds)) return e;
        hipLaunchKernelGGL((memory_chunk_kernel<T, DP>), dim3(a.chunks, a.H, a.B), dim3(256), lds, st, a);
    }
    return static_cast<int>(hipGetLastError());
}

template <bool DELTA>
static int launch_part(const ChunkArgs& a, bool walk, int dtype, hipStream_t st) {
#define PQ_SEG(T, DP) (DELTA ? delta_launch<T, DP>(a, walk, st) : memory_launch<T, DP>(a, walk, st))
#define PQ_SEG_D(T) (padded_dim(a.dim) == 64 ? PQ_SEG(T, 64) : padded_dim(a.dim) == 128 ? PQ_SEG(T, 128) : PQ_SEG(T, 256))
    return dtype == 0 ? PQ_SEG_D(F16) : PQ_SEG_D(BF16);
#undef PQ_SEG_D
#undef PQ_SEG
}

// A stream beside the caller's, and events to order the two, for each host thread and device (default priority; kept for the
// process).
struct Side {
    hipStream_t stream = nullptr;
    hipEvent_t begin = nullptr, made[2] = {}, used[2] = {};
    int ready = -1;              // -1: not tried, 0: there, otherwise the error
};
static Side& side_of_device() {
    constexpr int kDevices = 16;
    thread_local Side sides[kDevices];
    int dev = 0;
    if (hipGetDevice(&dev) != hipSuccess || dev < 0 || dev >= kDevices) dev = 0;
    Side& s = sides[dev];
    if (s.ready == -1) {
        hipError_t e = hipStreamCreateWithFlags(&s.stream, hipStreamNonBlocking);
        hipEvent_t* events[5] = {&s.begin, &s.made[0], &s.made[1], &s.used[0], &s.used[1]};
        for (hipEvent_t* ev : events)
            if (e == hipSuccess) e = hipEventCreateWithFlags(ev, hipEventDisableTiming);
        s.ready = static_cast<int>(e);
    }
    return s;
}

// The call's chunks in segments that half the workspace holds; the next segment's operands are made, on a stream of their own,
// while a segment is walked (a walk has few wavefronts).  One segment when the whole workspace holds the call.
template <bool DELTA>
static int launch_chunks(const ChunkArgs& args, size_t workspace_bytes, int dtype, hipStream_t st) {
    ChunkArgs a = args;
    const int total = (a.L + kChunk - 1) / kChunk;
    const size_t per = chunk_block_bytes(DELTA, a.dim, dtype) * a.B * a.H;
    const size_t fit = workspace_bytes / per;
    if (fit < 1) return static_cast<int>(hipErrorInvalidValue);
    // lines of up to eight chunks ahead, while those of an XCD's heads take half its 4 MB of L2; with more heads than that there
    // are wavefronts enough to wait in turn
    const size_t live = per * ((a.B * a.H + 7) / 8) / (static_cast<size_t>(a.B) * a.H);
    const size_t ahead = (size_t{2} << 20) / live;
    a.prefetch = ahead < 3 ? 0 : ahead > 8 ? 8 : static_cast<int>(ahead);
    auto segment = [&](int n, int count) {
        a.t0 = n * kChunk;
        a.chunks = n + count < total ? count : total - n;
    };
    // few chunks, or no room for two segments: one after the other
    const bool whole = fit >= static_cast<size_t>(total);
    if ((whole && total < 2 * kOverlapChunks) || fit < 2) {
        const int step = whole ? total : static_cast<int>(fit);
        for (int n = 0; n < total; n += step) {
            segment(n, step);
            if (int e = launch_part<DELTA>(a, false, dtype, st)) return e;
            if (int e = launch_part<DELTA>(a, true, dtype, st)) return e;
        }
        return 0;
    }
    Side& side = side_of_device();
    if (side.ready != 0) return side.ready;
    // segments of a quarter of a call that fits, or of half the workspace
    const int step = whole ? (total + 3) / 4 : static_cast<int>(fit / 2);
    char* const half[2] = {a.workspace, a.workspace + step * per};
#define PQ_TRY(call) do { const int e_ = static_cast<int>(call); if (e_) return e_; } while (0)
    PQ_TRY(hipEventRecord(side.begin, st));
    PQ_TRY(hipStreamWaitEvent(side.stream, side.begin, 0));
    segment(0, step);
    PQ_TRY(launch_part<DELTA>(a, false, dtype, st));
    for (int n = 0, i = 0; n < total; n += step, i++) {
        const int b = i & 1;
        if (n + step < total) {
            if (i > 0) PQ_TRY(hipStreamWaitEvent(side.stream, side.used[1 - b], 0));
            segment(n + step, step);
            a.workspace = half[1 - b];
            PQ_TRY(launch_part<DELTA>(a, false, dtype, side.stream));
            PQ_TRY(hipEventRecord(side.made[1 - b], side.stream));
        }
        if (i > 0) PQ_TRY(hipStreamWaitEvent(st, side.made[b], 0));
        segment(n, step);
        a.workspace = half[b];
        PQ_TRY(launch_part<DELTA>(a, true, dtype, st));
        PQ_TRY(hipEventRecord(side.used[b], st));
    }
#undef PQ_TRY
    return 0;
}
int launch_delta_chunks(const ChunkArgs& a, size_t workspace_bytes, int dtype, hipStream_t st) { return launch_chunks<true>(a, workspace_bytes, dtype, st); }
int launch_memory_chunks(const ChunkArgs& a, size_t workspace_bytes, int dtype, hipStream_t st) { return launch_chunks<false>(a, workspace_bytes, dtype, st); }

}  // namespace pq
