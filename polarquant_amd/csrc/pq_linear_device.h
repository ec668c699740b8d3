// Linear layers of the decode step: y[M, N] = x[M, K] . W[N, K]^T (+ bias) with M <= 16 rows
// (one new token per sequence), the q/k/v, o and MLP projections around the attention call
// (models/modeling_llama_polar.py:47-52, :131 and the decoder layer's MLP, :456-486).
//
// At M <= 16 the product is a stream of the weight matrix through HBM, 2*M flops per weight
// byte: the kernels are laid out for the stream, not for the matrix cores.  Two of them:
// small_m_linear_kernel (any M <= 16, described here) and small_m8_linear_kernel (M <= 8, further
// down: whole-line loads, half the x operand traffic).  A workgroup owns
// 16 output columns (16 rows of W) and splits K over its KSPLIT wavefronts; each wavefront
// keeps two stages of kStage 16-byte loads per lane in flight (ping-pong) and feeds them to
// v_mfma_f32_16x16x32 with the W rows as the A operand and x (rows >= M unused) as the B operand:
// lane l holds W[n0 + l % 16][k + 8 * (l / 16) .. + 8) and x[l % 16][same k], so a 16-byte
// load per lane is one MFMA operand and a wavefront load covers 16 rows x 64 contiguous
// bytes.  The KSPLIT partial 16x16 tiles are added in a fixed order through LDS, so results
// do not depend on scheduling.  x (at most 16 x K) is re-read by every workgroup from L2.
//
// GATED: two weight matrices share the x operand and the epilogue applies
// silu(gate) * up with the eager modules' roundings (gate, up and silu(gate) each rounded
// to the activation dtype), which saves the [M, 2 * N] round trip and one launch.
//
// EPI 0 is the kernel as described (bias, or the gated form); EPI 1 + e is the same stream for one of `heads` independent
// products per launch (blockIdx.y == head, operands `x_head` / N * K / `y_head` elements apart) with epilogue e of
// pq_steps_internal.h: plain, square of relu, times sigmoid(gate), or unrounded float32 output.
#pragma once
#include "pq_device.h"
#include "pq_steps_internal.h"

namespace pq {

typedef float floatx4_l __attribute__((ext_vector_type(4)));
typedef uint32_t u32x4_l __attribute__((ext_vector_type(4)));
typedef _Float16 half8_l __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x8_l __attribute__((ext_vector_type(8)));

template <typename T> __device__ __forceinline__ floatx4_l mfma32(u32x4_l a, u32x4_l b, floatx4_l c);
template <> __device__ __forceinline__ floatx4_l mfma32<F16>(u32x4_l a, u32x4_l b, floatx4_l c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_f16(__builtin_bit_cast(half8_l, a), __builtin_bit_cast(half8_l, b), c, 0, 0, 0);
}
template <> __device__ __forceinline__ floatx4_l mfma32<BF16>(u32x4_l a, u32x4_l b, floatx4_l c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_l, a), __builtin_bit_cast(bf16x8_l, b), c, 0, 0, 0);
}

template <typename T>
__device__ __forceinline__ float rnd_l(float f) { return lo2f<T>(f2lo<T>(f)); }

struct HeadEpi {
    int64_t x_head, w_head, y_head;
    const uint16_t* gate;
    int64_t gate_row;
};

// stores outputs y[r][n .. n + 3] (n: column inside the head) through epilogue EPI - 1
template <typename T, int EPI>
__device__ __forceinline__ void store_head(const float (&s)[4], uint16_t* y, int64_t y_stride, int r, int n, int N, const HeadEpi& he) {
    const size_t o = static_cast<size_t>(r) * y_stride + blockIdx.y * he.y_head + n;
    if constexpr (EPI == 1 + kEpiF32) {
        *reinterpret_cast<float4*>(reinterpret_cast<float*>(y) + o) = make_float4(s[0], s[1], s[2], s[3]);
    } else {
        uint16_t out[4];
#pragma unroll
        for (int i = 0; i < 4; i++) {
            float v = s[i];
            if constexpr (EPI == 1 + kEpiReluSq) {
                v = fmaxf(v, 0.0f);
                v = v * v;
            }
            if constexpr (EPI == 1 + kEpiSigmoidGate)
                v = v / (1.0f + __expf(-lo2f<T>(he.gate[static_cast<size_t>(r) * he.gate_row + static_cast<size_t>(blockIdx.y) * N + n + i])));
            out[i] = f2lo<T>(v);
        }
        *reinterpret_cast<uint2*>(y + o) = make_uint2(static_cast<uint32_t>(out[0]) | (static_cast<uint32_t>(out[1]) << 16),
                                                      static_cast<uint32_t>(out[2]) | (static_cast<uint32_t>(out[3]) << 16));
    }
}

template <bool GATED, int kStage>
struct StageT {
    u32x4_l w[kStage], x[kStage], u[GATED ? kStage : 1];
};

template <typename T, int KSPLIT, bool GATED, int kStage, int EPI = 0>
__global__ __launch_bounds__(kWave * KSPLIT) void small_m_linear_kernel(
    const uint16_t* __restrict__ x, int64_t x_stride, const uint16_t* __restrict__ w, const uint16_t* __restrict__ w_up,
    const uint16_t* __restrict__ bias, uint16_t* __restrict__ y, int64_t y_stride, int M, int K, HeadEpi he) {
    if constexpr (EPI != 0) {
        x += blockIdx.y * he.x_head;
        w += blockIdx.y * he.w_head;
    }
    __shared__ float part[KSPLIT][GATED ? 2 : 1][4][kWave];
    const int lane = threadIdx.x & (kWave - 1), wv = threadIdx.x / kWave;
    const int r = lane & 15, g = lane >> 4;
    const int n0 = blockIdx.x * 16;
    const int klen = K / KSPLIT, steps = klen / 32;
    const int m = r < M ? r : 0;                           // tile columns >= M repeat row 0 and are never stored
    const size_t koff = static_cast<size_t>(wv) * klen + 8 * g;
    const uint16_t* wp = w + static_cast<size_t>(n0 + r) * K + koff;
    const uint16_t* up = GATED ? w_up + static_cast<size_t>(n0 + r) * K + koff : nullptr;
    const uint16_t* xp = x + static_cast<size_t>(m) * x_stride + koff;

    floatx4_l acc[2] = {{0, 0, 0, 0}, {0, 0, 0, 0}}, acu[2] = {{0, 0, 0, 0}, {0, 0, 0, 0}};
    // No branch may sit between a stage's loads and the MFMAs of the other stage: at a join the
    // compiler has to wait for every outstanding load, which would serialize the two stages.  So
    // whole stages run in a branch-free ping-pong loop, and only the tail is predicated.
    auto load = [&](StageT<GATED, kStage>& st, int s0) {
        static_for<kStage>([&](auto U) {
            constexpr int u = decltype(U)::value;
            st.w[u] = *reinterpret_cast<const u32x4_l*>(wp + (s0 + u) * 32);
            if constexpr (GATED) st.u[u] = *reinterpret_cast<const u32x4_l*>(up + (s0 + u) * 32);
            st.x[u] = *reinterpret_cast<const u32x4_l*>(xp + (s0 + u) * 32);
        });
    };
    auto compute = [&](const StageT<GATED, kStage>& st) {
        static_for<kStage>([&](auto U) {
            constexpr int u = decltype(U)::value;
            acc[u & 1] = mfma32<T>(st.w[u], st.x[u], acc[u & 1]);
            if constexpr (GATED) acu[u & 1] = mfma32<T>(st.u[u], st.x[u], acu[u & 1]);
        });
    };
    const int full = steps / kStage;          // whole stages
    if (full > 0) {
        StageT<GATED, kStage> sa, sb;
        load(sa, 0);
        int st = 0;
        while (st + 2 < full) {
            load(sb, (st + 1) * kStage);
            compute(sa);
            load(sa, (st + 2) * kStage);
            compute(sb);
            st += 2;
        }
        if (full - st == 2) {
            load(sb, (st + 1) * kStage);
            compute(sa);
            compute(sb);
        } else {
            compute(sa);
        }
    }
    for (int s1 = full * kStage; s1 < steps; s1++) {      // fewer than kStage steps left
        const u32x4_l wv1 = *reinterpret_cast<const u32x4_l*>(wp + s1 * 32);
        const u32x4_l xv1 = *reinterpret_cast<const u32x4_l*>(xp + s1 * 32);
        acc[0] = mfma32<T>(wv1, xv1, acc[0]);
        if constexpr (GATED) acu[0] = mfma32<T>(*reinterpret_cast<const u32x4_l*>(up + s1 * 32), xv1, acu[0]);
    }
#pragma unroll
    for (int i = 0; i < 4; i++) {
        part[wv][0][i][lane] = acc[0][i] + acc[1][i];
        if constexpr (GATED) part[wv][1][i][lane] = acu[0][i] + acu[1][i];
    }
    __syncthreads();
    if (wv != 0 || r >= M) return;
    // the MFMA result layout: lane (r, g) holds tile rows 4g + i (i < 4) of tile column r = outputs y[r][n0 + 4g + i]
    if constexpr (EPI != 0) {
        float s4[4];
#pragma unroll
        for (int i = 0; i < 4; i++) {
            s4[i] = part[0][0][i][lane];
#pragma unroll
            for (int k = 1; k < KSPLIT; k++) s4[i] += part[k][0][i][lane];
        }
        store_head<T, EPI>(s4, y, y_stride, r, n0 + 4 * g, static_cast<int>(gridDim.x) * 16, he);
        return;
    }
    uint16_t out[4];
#pragma unroll
    for (int i = 0; i < 4; i++) {
        float s = part[0][0][i][lane];
#pragma unroll
        for (int k = 1; k < KSPLIT; k++) s += part[k][0][i][lane];
        if constexpr (GATED) {
            float t = part[0][1][i][lane];
#pragma unroll
            for (int k = 1; k < KSPLIT; k++) t += part[k][1][i][lane];
            const float gv = rnd_l<T>(s), uv = rnd_l<T>(t);
            const float a = rnd_l<T>(gv / (1.0f + __expf(-gv)));
            out[i] = f2lo<T>(a * uv);
        } else {
            if (bias) s += lo2f<T>(bias[n0 + 4 * g + i]);
            out[i] = f2lo<T>(s);
        }
    }
    *reinterpret_cast<uint2*>(y + static_cast<size_t>(r) * y_stride + n0 + 4 * g) =
        make_uint2(static_cast<uint32_t>(out[0]) | (static_cast<uint32_t>(out[1]) << 16),
                   static_cast<uint32_t>(out[2]) | (static_cast<uint32_t>(out[3]) << 16));
}

// M <= 8: each 16 x 16 MFMA tile is used as two 8 x 8 tiles on its diagonal.  Tile rows 0-7 are 8 rows
// of W over the first 32 of a 64-wide k-step, tile rows 8-15 the SAME 8 rows over the second 32; tile
// columns 0-7 are the rows of x over the first 32, columns 8-15 over the second 32.  Then
// y[m][n] = C[n][m] + C[n + 8][m + 8] and the off-diagonal quarters are ignored.  No lane loads a
// duplicate row of x, a wavefront load of W covers 8 rows x 128 contiguous bytes (whole cache lines,
// which is what lets the weight stream carry the non-temporal hint: with half lines the hint drops a
// line before its second half is asked for), and the workgroup's 16 rows of W are two such tiles that
// share one x operand: per 64-wide step two W loads and one x load instead of four and four.
template <bool GATED, int kStage>
struct Stage8T {
    u32x4_l w[2][kStage], x[kStage], u[GATED ? 2 : 1][GATED ? kStage : 1];
};

template <typename T, int KSPLIT, bool GATED, int kStage, int EPI = 0>
__global__ __launch_bounds__(kWave * KSPLIT) void small_m8_linear_kernel(
    const uint16_t* __restrict__ x, int64_t x_stride, const uint16_t* __restrict__ w, const uint16_t* __restrict__ w_up,
    const uint16_t* __restrict__ bias, uint16_t* __restrict__ y, int64_t y_stride, int M, int K, HeadEpi he) {
    if constexpr (EPI != 0) {
        x += blockIdx.y * he.x_head;
        w += blockIdx.y * he.w_head;
    }
    __shared__ float part[KSPLIT][GATED ? 4 : 2][4][kWave];
    const int lane = threadIdx.x & (kWave - 1), wv = threadIdx.x / kWave;
    const int r = lane & 15, g = lane >> 4;
    const int row = r & 7, chunk = (r >> 3) * 4 + g;       // W row inside an 8-row tile == x row; 16-byte piece of the step
    const int n0 = blockIdx.x * 16;
    const int klen = K / KSPLIT, steps = klen / 64;
    const int m = row < M ? row : 0;                       // tile columns >= M repeat row 0 and are never stored
    const size_t koff = static_cast<size_t>(wv) * klen + 8 * chunk;
    const uint16_t* wp = w + static_cast<size_t>(n0 + row) * K + koff;
    const uint16_t* up = GATED ? w_up + static_cast<size_t>(n0 + row) * K + koff : nullptr;
    const uint16_t* xp = x + static_cast<size_t>(m) * x_stride + koff;
    const size_t half_tile = static_cast<size_t>(8) * K;   // rows n0 + 8 .. n0 + 15

    floatx4_l acc[2] = {{0, 0, 0, 0}, {0, 0, 0, 0}}, acu[2] = {{0, 0, 0, 0}, {0, 0, 0, 0}};
    auto ldw = [](const uint16_t* p) { return __builtin_nontemporal_load(reinterpret_cast<const u32x4_l*>(p)); };
    auto load = [&](Stage8T<GATED, kStage>& st, int s0) {          // branch-free, see small_m_linear_kernel
        static_for<kStage>([&](auto U) {
            constexpr int u = decltype(U)::value;
            st.w[0][u] = ldw(wp + (s0 + u) * 64);
            st.w[1][u] = ldw(wp + half_tile + (s0 + u) * 64);
            if constexpr (GATED) {
                st.u[0][u] = ldw(up + (s0 + u) * 64);
                st.u[1][u] = ldw(up + half_tile + (s0 + u) * 64);
            }
            st.x[u] = *reinterpret_cast<const u32x4_l*>(xp + (s0 + u) * 64);
        });
    };
    auto compute = [&](const Stage8T<GATED, kStage>& st) {
        static_for<kStage>([&](auto U) {
            constexpr int u = decltype(U)::value;
            acc[0] = mfma32<T>(st.w[0][u], st.x[u], acc[0]);
            acc[1] = mfma32<T>(st.w[1][u], st.x[u], acc[1]);
            if constexpr (GATED) {
                acu[0] = mfma32<T>(st.u[0][u], st.x[u], acu[0]);
                acu[1] = mfma32<T>(st.u[1][u], st.x[u], acu[1]);
            }
        });
    };
    const int full = steps / kStage;
    if (full > 0) {
        Stage8T<GATED, kStage> sa, sb;
        load(sa, 0);
        int st = 0;
        while (st + 2 < full) {
            load(sb, (st + 1) * kStage);
            compute(sa);
            load(sa, (st + 2) * kStage);
            compute(sb);
            st += 2;
        }
        if (full - st == 2) {
            load(sb, (st + 1) * kStage);
            compute(sa);
            compute(sb);
        } else {
            compute(sa);
        }
    }
    for (int s1 = full * kStage; s1 < steps; s1++) {
        const u32x4_l xv1 = *reinterpret_cast<const u32x4_l*>(xp + s1 * 64);
        acc[0] = mfma32<T>(ldw(wp + s1 * 64), xv1, acc[0]);
        acc[1] = mfma32<T>(ldw(wp + half_tile + s1 * 64), xv1, acc[1]);
        if constexpr (GATED) {
            acu[0] = mfma32<T>(ldw(up + s1 * 64), xv1, acu[0]);
            acu[1] = mfma32<T>(ldw(up + half_tile + s1 * 64), xv1, acu[1]);
        }
    }
#pragma unroll
    for (int i = 0; i < 4; i++) {
        part[wv][0][i][lane] = acc[0][i];
        part[wv][1][i][lane] = acc[1][i];
        if constexpr (GATED) { part[wv][2][i][lane] = acu[0][i]; part[wv][3][i][lane] = acu[1][i]; }
    }
    __syncthreads();
    // lane (r < 8, g < 2) owns outputs y[r][n0 + 8h + 4g + i] (h: which 8-row tile), each the sum of the tile's
    // entry (row 4g + i, column r) and its diagonal partner (row + 8, column + 8), which lane + 40 holds
    if (wv != 0 || r >= 8 || r >= M || g >= 2) return;
#pragma unroll
    for (int h = 0; h < 2; h++) {
        if constexpr (EPI != 0) {
            float s4[4];
#pragma unroll
            for (int i = 0; i < 4; i++) {
                s4[i] = 0.0f;
#pragma unroll
                for (int k = 0; k < KSPLIT; k++) s4[i] += part[k][h][i][lane] + part[k][h][i][lane + 40];
            }
            store_head<T, EPI>(s4, y, y_stride, r, n0 + 8 * h + 4 * g, static_cast<int>(gridDim.x) * 16, he);
            continue;
        }
        uint16_t out[4];
#pragma unroll
        for (int i = 0; i < 4; i++) {
            float s = 0.0f, t = 0.0f;
#pragma unroll
            for (int k = 0; k < KSPLIT; k++) {
                s += part[k][h][i][lane] + part[k][h][i][lane + 40];
                if constexpr (GATED) t += part[k][2 + h][i][lane] + part[k][2 + h][i][lane + 40];
            }
            if constexpr (GATED) {
                const float gv = rnd_l<T>(s), uv = rnd_l<T>(t);
                const float a = rnd_l<T>(gv / (1.0f + __expf(-gv)));
                out[i] = f2lo<T>(a * uv);
            } else {
                if (bias) s += lo2f<T>(bias[n0 + 8 * h + 4 * g + i]);
                out[i] = f2lo<T>(s);
            }
        }
        *reinterpret_cast<uint2*>(y + static_cast<size_t>(r) * y_stride + n0 + 8 * h + 4 * g) =
            make_uint2(static_cast<uint32_t>(out[0]) | (static_cast<uint32_t>(out[1]) << 16),
                       static_cast<uint32_t>(out[2]) | (static_cast<uint32_t>(out[3]) << 16));
    }
}

}  // namespace pq
