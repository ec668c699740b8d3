// Attention over a latent key/value state, with a per-head sink in the softmax's denominator and no positions.
//
//   latent_decode_kernel   few query tokens: queries are already in the latent space, all heads share the cached latents
//                          (read once per row tile), the context is cut into slices; latent_merge_kernel joins them
//   latent_prefill_kernel  many query tokens: keys and values expanded per head beforehand, flash attention, the output
//                          gate in the epilogue
//   latent_plain_kernel    any rank, any dtype (float32 runs here), one wavefront per query row
//
// Both matrix-core kernels compute the TRANSPOSED score tile, S^T = K Q^T, so that a query row is a tile column, i.e. a
// lane: its softmax state is one register, and the weights P^T leave the first product in the layout the second one,
// O^T = V^T P^T, takes its right operand in, once the tokens are numbered accordingly (the order of the summed index is
// free as long as both operands agree).  Scores, their softmax and all sums are float32; latents, queries and weights
// enter the products in the model's 16-bit dtype.
#include "pq_device.h"
#include "pq_latent_internal.h"

namespace pq {

struct F32 {};
typedef float floatx4_a __attribute__((ext_vector_type(4)));
typedef float floatx16_a __attribute__((ext_vector_type(16)));
typedef uint32_t u32x4_a __attribute__((ext_vector_type(4)));
typedef uint32_t u32x2_a __attribute__((ext_vector_type(2)));
typedef _Float16 half8_a __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x8_a __attribute__((ext_vector_type(8)));
typedef short short4_a __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) short4_a lds_short4;
typedef __attribute__((address_space(3))) u32x4_a lds_u32x4;

template <typename T> __device__ __forceinline__ floatx4_a mma16(u32x4_a a, u32x4_a b, floatx4_a c);
template <> __device__ __forceinline__ floatx4_a mma16<F16>(u32x4_a a, u32x4_a b, floatx4_a c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_f16(__builtin_bit_cast(half8_a, a), __builtin_bit_cast(half8_a, b), c, 0, 0, 0);
}
template <> __device__ __forceinline__ floatx4_a mma16<BF16>(u32x4_a a, u32x4_a b, floatx4_a c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_a, a), __builtin_bit_cast(bf16x8_a, b), c, 0, 0, 0);
}
template <typename T> __device__ __forceinline__ floatx16_a mma32(u32x4_a a, u32x4_a b, floatx16_a c);
template <> __device__ __forceinline__ floatx16_a mma32<F16>(u32x4_a a, u32x4_a b, floatx16_a c) {
    return __builtin_amdgcn_mfma_f32_32x32x16_f16(__builtin_bit_cast(half8_a, a), __builtin_bit_cast(half8_a, b), c, 0, 0, 0);
}
template <> __device__ __forceinline__ floatx16_a mma32<BF16>(u32x4_a a, u32x4_a b, floatx16_a c) {
    return __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_a, a), __builtin_bit_cast(bf16x8_a, b), c, 0, 0, 0);
}

constexpr float kLog2e = 1.4426950408889634f;
constexpr float kNone = -1.0e30f;         // running maximum before any key
__device__ __forceinline__ float exp2_hw(float x) { return __builtin_amdgcn_exp2f(x); }

template <typename T> __device__ __forceinline__ uint32_t pack2(float a, float b) {
    return static_cast<uint32_t>(f2lo<T>(a)) | (static_cast<uint32_t>(f2lo<T>(b)) << 16);
}

// ---- decode --------------------------------------------------------------------------------------------------------
// grid (slices, row tiles, sequences); a row is (query token, head), a wavefront owns 16 of them, RW wavefronts share the
// latents of a 32-token tile in LDS (double-buffered, next tile's loads in flight over the current tile's products).
// The same tile serves both products: rows of it (16 bytes per lane) as K, columns of it, transposed on the way out of
// LDS, as V.  16-byte pieces of a row are XOR-swizzled by the token so that neither access meets in few banks.
// Workspace: [B, slices, L * H] pairs (maximum in log2 units, sum), then as many rows of R floats.
constexpr int kDecodeTile = 32;
__device__ __forceinline__ size_t pairs_floats(const LatentDecodeArgs& a) {     // up to the accumulators' 16-byte boundary
    return (2 * static_cast<size_t>(a.B) * a.n_splits * a.L * a.H + 3) & ~static_cast<size_t>(3);
}

template <typename T, int RP, int RW>
__global__ __launch_bounds__(kWave * RW) void latent_decode_kernel(LatentDecodeArgs a) {
    constexpr int CH = RP / 8, NT = kWave * RW, LPT = kDecodeTile * CH / NT, KS = RP / 32, CT = RP / 16;
    static_assert(LPT >= 1 && LPT * NT == kDecodeTile * CH, "whole loads");
    __shared__ __attribute__((aligned(16))) uint16_t tile[2][kDecodeTile * RP];
    const int tid = threadIdx.x, lane = tid & 63, wv = tid / kWave, r16 = lane & 15, g = lane >> 4;
    const int b = blockIdx.z, split = blockIdx.x, R = a.R, rows = a.L * a.H;
    const int n = blockIdx.y * 16 * RW + wv * 16 + r16;
    const bool valid = n < rows;
    const int nc = valid ? n : rows - 1;
    const int pos = a.pos_dev ? *a.pos_dev : a.pos;
    int64_t total = static_cast<int64_t>(pos) + a.L;
    if (total > a.capacity) total = a.capacity;
    const int lo = a.start ? a.start[b] : 0;
    const int len = static_cast<int>(total) - lo;
    const int per = ((len + a.n_splits - 1) / a.n_splits + kDecodeTile - 1) / kDecodeTile * kDecodeTile;
    const int64_t s0 = lo + static_cast<int64_t>(split) * per;
    const int64_t s1 = s0 + per < total ? s0 + per : total;
    const size_t part = (static_cast<size_t>(b) * a.n_splits + split) * rows;
    float* ml = a.workspace + 2 * part;
    float* acc = a.workspace + pairs_floats(a) + part * R;
    if (s0 >= s1) {                                  // uniform over the workgroup
        if (valid && g == 0) { ml[2 * n] = kNone; ml[2 * n + 1] = 0.0f; }
        return;
    }
    auto swz = [](int tok) { return RP >= 128 ? (tok & 15) : ((tok >> 1) & 7); };

    u32x4_a q[KS];
    {
        const uint16_t* qp = static_cast<const uint16_t*>(a.q) + (static_cast<size_t>(b) * rows + nc) * R + 8 * g;
        static_for<KS>([&](auto I) {
            constexpr int i = decltype(I)::value;
            q[i] = u32x4_a{0, 0, 0, 0};
            if (i * 32 + 8 * g < R) q[i] = *reinterpret_cast<const u32x4_a*>(qp + i * 32);
        });
    }
    const int limit = pos + nc / a.H + 1;            // keys this row may see: positions below it
    const float scale2 = a.scale * kLog2e;
    const uint16_t* cb = static_cast<const uint16_t*>(a.c) + static_cast<size_t>(b) * a.capacity * R;

    u32x4_a stage[LPT];
    auto fetch = [&](int64_t key0) {
        static_for<LPT>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const int u = i * NT + tid, tok = u / CH, ch = u % CH;
            const int64_t key = key0 + tok < s1 ? key0 + tok : s1 - 1;       // rows past the slice: a copy, weight zero
            stage[i] = u32x4_a{0, 0, 0, 0};
            if (ch * 8 < R) stage[i] = *reinterpret_cast<const u32x4_a*>(cb + key * R + ch * 8);
        });
    };
    auto put = [&](int buf) {
        static_for<LPT>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const int u = i * NT + tid, tok = u / CH, ch = u % CH;
            *reinterpret_cast<u32x4_a*>(&tile[buf][tok * RP + ((ch ^ swz(tok)) * 8)]) = stage[i];
        });
    };
    floatx4_a o[CT];
    static_for<CT>([&](auto I) { o[decltype(I)::value] = floatx4_a{0, 0, 0, 0}; });
    float m = kNone, l = 0.0f;
    // element offsets inside a tile; pieces 16 apart (8 for the 64-wide rows) differ by a constant
    constexpr int KLOW = KS < 4 ? KS : 4, VLOW = CT < 8 ? CT : 8;
    int koff[KLOW], voff[VLOW];
    static_for<KLOW>([&](auto I) { constexpr int i = decltype(I)::value; koff[i] = r16 * RP + (((i * 4 + g) ^ swz(r16)) * 8); });
    {
        const int row = 4 * g + (r16 >> 2);
        static_for<VLOW>([&](auto I) {
            constexpr int i = decltype(I)::value;
            voff[i] = row * RP + (((i * 2 + ((r16 & 3) >> 1)) ^ swz(row)) * 8) + (r16 & 1) * 4;
        });
    }

    const int ntiles = static_cast<int>((s1 - s0 + kDecodeTile - 1) / kDecodeTile);
    fetch(s0);
    put(0);
    __syncthreads();
    for (int it = 0; it < ntiles; it++) {
        const int buf = it & 1;
        if (it + 1 < ntiles) fetch(s0 + static_cast<int64_t>(it + 1) * kDecodeTile);
        __builtin_amdgcn_sched_barrier(0);
        const uint16_t* base = tile[buf];
        floatx4_a s[2] = {{0, 0, 0, 0}, {0, 0, 0, 0}};
        static_for<KS>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const uint16_t* p = base + koff[i % KLOW] + (i / KLOW) * 128;
            s[0] = mma16<T>(*reinterpret_cast<const u32x4_a*>(p), q[i], s[0]);
            s[1] = mma16<T>(*reinterpret_cast<const u32x4_a*>(p + 16 * RP), q[i], s[1]);
        });
        // this lane: row n, tokens 4g + j and 16 + 4g + j of the tile
        const int64_t key0 = s0 + static_cast<int64_t>(it) * kDecodeTile + 4 * g;
        float p[8], mx = kNone;
#pragma unroll
        for (int u = 0; u < 2; u++)
#pragma unroll
            for (int j = 0; j < 4; j++) {
                const int64_t key = key0 + 16 * u + j;
                const float v = (key < limit && key < s1) ? s[u][j] * scale2 : -INFINITY;
                p[4 * u + j] = v;
                mx = fmaxf(mx, v);
            }
        mx = fmaxf(mx, __shfl_xor(mx, 16));
        mx = fmaxf(mx, __shfl_xor(mx, 32));
        if (__any(mx > m)) {
            const float mn = fmaxf(m, mx), al = exp2_hw(m - mn);
            l *= al;
            static_for<CT>([&](auto I) {
                constexpr int i = decltype(I)::value;
#pragma unroll
                for (int j = 0; j < 4; j++) o[i][j] *= al;
            });
            m = mn;
        }
#pragma unroll
        for (int j = 0; j < 8; j++) { p[j] = exp2_hw(p[j] - m); l += p[j]; }
        const u32x4_a pt = {pack2<T>(p[0], p[1]), pack2<T>(p[2], p[3]), pack2<T>(p[4], p[5]), pack2<T>(p[6], p[7])};
        static_for<CT>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const uint16_t* vp = base + voff[i % VLOW] + (i / VLOW) * 128;
            const short4_a v0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_short4*)(vp));
            const short4_a v1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_short4*)(vp + 16 * RP));
            const u32x2_a w0 = __builtin_bit_cast(u32x2_a, v0), w1 = __builtin_bit_cast(u32x2_a, v1);
            o[i] = mma16<T>(u32x4_a{w0.x, w0.y, w1.x, w1.y}, pt, o[i]);
        });
        if (it + 1 < ntiles) put(buf ^ 1);           // its last readers passed the barrier of the previous iteration
        __syncthreads();
    }
    l += __shfl_xor(l, 16);
    l += __shfl_xor(l, 32);
    if (!valid) return;
    if (g == 0) { ml[2 * n] = m; ml[2 * n + 1] = l; }
    static_for<CT>([&](auto I) {
        constexpr int i = decltype(I)::value;
        const int ch = i * 16 + 4 * g;
        if (ch < R) *reinterpret_cast<float4*>(acc + static_cast<size_t>(n) * R + ch) = make_float4(o[i][0], o[i][1], o[i][2], o[i][3]);
    });
}

// grid (L * H, B), 128 threads: joins the slices of a row; the sink joins the denominator here, once.
constexpr int kMaxSlices = 512;
template <typename T>
__global__ __launch_bounds__(128) void latent_merge_kernel(LatentDecodeArgs a) {
    __shared__ float wgt[kMaxSlices], red[4];
    const int n = blockIdx.x, b = blockIdx.y, rows = a.L * a.H, S = a.n_splits, R = a.R, tid = threadIdx.x;
    const size_t first = static_cast<size_t>(b) * S * rows + n;
    const float sink2 = a.sink[n % a.H] * kLog2e;
    float mx = sink2;
    for (int s = tid; s < S; s += 128) mx = fmaxf(mx, a.workspace[2 * (first + static_cast<size_t>(s) * rows)]);
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o));
    if ((tid & 63) == 0) red[tid >> 6] = mx;
    __syncthreads();
    mx = fmaxf(red[0], red[1]);
    float den = 0.0f;
    for (int s = tid; s < S; s += 128) {
        const float* p = a.workspace + 2 * (first + static_cast<size_t>(s) * rows);
        const float w = p[0] > kNone ? exp2_hw(p[0] - mx) : 0.0f;
        wgt[s] = w;
        den += w * p[1];
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) den += __shfl_xor(den, o);
    if ((tid & 63) == 0) red[2 + (tid >> 6)] = den;
    __syncthreads();
    const float inv = 1.0f / (red[2] + red[3] + exp2_hw(sink2 - mx));
    const float* acc = a.workspace + pairs_floats(a) + first * R;
    for (int ch = tid * 4; ch < R; ch += 512) {
        float4 sum = make_float4(0, 0, 0, 0);
        for (int s = 0; s < S; s++) {
            const float w = wgt[s];
            if (w == 0.0f) continue;                 // (an empty slice's accumulators were never written)
            const float4 v = *reinterpret_cast<const float4*>(acc + static_cast<size_t>(s) * rows * R + ch);
            sum.x = __builtin_fmaf(w, v.x, sum.x); sum.y = __builtin_fmaf(w, v.y, sum.y);
            sum.z = __builtin_fmaf(w, v.z, sum.z); sum.w = __builtin_fmaf(w, v.w, sum.w);
        }
        *reinterpret_cast<uint2*>(static_cast<uint16_t*>(a.out) + (static_cast<size_t>(b) * rows + n) * R + ch) =
            make_uint2(pack2<T>(sum.x * inv, sum.y * inv), pack2<T>(sum.z * inv, sum.w * inv));
    }
}

int launch_latent_decode(const LatentDecodeArgs& a, int dtype, hipStream_t st) {
    const int rows = a.L * a.H;
    // (a single wavefront's share of a 512-wide tile in flight does not fit its registers beside the accumulators)
    const int rw = rows <= 16 && a.R <= 256 ? 1 : rows <= 32 ? 2 : 4;
    dim3 grid(a.n_splits, (rows + 16 * rw - 1) / (16 * rw), a.B), block(kWave * rw);
#define PQ_LD(T, RP)                                                                                                 \
    do {                                                                                                             \
        if (rw == 1 && RP <= 256) hipLaunchKernelGGL((latent_decode_kernel<T, (RP <= 256 ? RP : 256), 1>), grid, block, 0, st, a);                    \
        else if (rw == 2) hipLaunchKernelGGL((latent_decode_kernel<T, RP, 2>), grid, block, 0, st, a);               \
        else hipLaunchKernelGGL((latent_decode_kernel<T, RP, 4>), grid, block, 0, st, a);                            \
    } while (0)
#define PQ_LDT(T)                                                                                                    \
    do {                                                                                                             \
        if (a.R <= 64) PQ_LD(T, 64); else if (a.R <= 128) PQ_LD(T, 128);                                             \
        else if (a.R <= 256) PQ_LD(T, 256); else PQ_LD(T, 512);                                                      \
    } while (0)
    if (dtype == 0) PQ_LDT(F16); else PQ_LDT(BF16);
#undef PQ_LDT
#undef PQ_LD
    int err = static_cast<int>(hipGetLastError());
    if (err) return err;
    dim3 mgrid(rows, a.B), mblock(128);
    if (dtype == 0) hipLaunchKernelGGL(latent_merge_kernel<F16>, mgrid, mblock, 0, st, a);
    else hipLaunchKernelGGL(latent_merge_kernel<BF16>, mgrid, mblock, 0, st, a);
    return static_cast<int>(hipGetLastError());
}

// ---- any rank, any dtype ---------------------------------------------------------------------------------------------
// grid (L * H, B), one wavefront: lane == key for the scores of 64 keys, then lane == channel for the weighted sum.
template <typename T> struct PlainElem { using type = uint16_t; static __device__ float get(uint16_t v) { return lo2f<T>(v); } static __device__ uint16_t put(float f) { return f2lo<T>(f); } };
template <> struct PlainElem<F32> { using type = float; static __device__ float get(float v) { return v; } static __device__ float put(float f) { return f; } };

template <typename T>
__global__ __launch_bounds__(kWave) void latent_plain_kernel(LatentDecodeArgs a) {
    using E = PlainElem<T>;
    using e_t = typename E::type;
    extern __shared__ float sh[];
    float *q = sh, *acc = sh + a.R, *p = sh + 2 * a.R;
    const int n = blockIdx.x, b = blockIdx.y, rows = a.L * a.H, R = a.R, lane = threadIdx.x;
    const int pos = a.pos_dev ? *a.pos_dev : a.pos, lo = a.start ? a.start[b] : 0;
    int64_t limit = static_cast<int64_t>(pos) + n / a.H + 1;
    if (limit > a.capacity) limit = a.capacity;
    const e_t* qp = static_cast<const e_t*>(a.q) + (static_cast<size_t>(b) * rows + n) * R;
    const e_t* cb = static_cast<const e_t*>(a.c) + static_cast<size_t>(b) * a.capacity * R;
    for (int i = lane; i < R; i += kWave) { q[i] = E::get(qp[i]); acc[i] = 0.0f; }
    __syncthreads();
    const float scale2 = a.scale * kLog2e, sink2 = a.sink[n % a.H] * kLog2e;
    float m = sink2, l = 1.0f;                       // the sink: weight 1 at its own maximum, no value
    for (int64_t k0 = lo; k0 < limit; k0 += kWave) {
        const int64_t key = k0 + lane;
        float s = -INFINITY;
        if (key < limit) {
            const e_t* c = cb + key * R;
            float d = 0.0f;
            for (int i = 0; i < R; i++) d = __builtin_fmaf(q[i], E::get(c[i]), d);
            s = d * scale2;
        }
        float mx = s;
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o));
        const float mn = fmaxf(m, mx), al = exp2_hw(m - mn), w = exp2_hw(s - mn);
        m = mn;
        float sum = w;
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) sum += __shfl_xor(sum, o);
        l = l * al + sum;
        p[lane] = w;
        __syncthreads();
        const int cnt = static_cast<int>(limit - k0 < kWave ? limit - k0 : kWave);
        for (int i = lane; i < R; i += kWave) {
            float v = acc[i] * al;
            for (int j = 0; j < cnt; j++) v = __builtin_fmaf(p[j], E::get(cb[(k0 + j) * R + i]), v);
            acc[i] = v;
        }
        __syncthreads();
    }
    e_t* out = static_cast<e_t*>(a.out) + (static_cast<size_t>(b) * rows + n) * R;
    for (int i = lane; i < R; i += kWave) out[i] = E::put(acc[i] / l);
}

int launch_latent_decode_any(const LatentDecodeArgs& a, int dtype, hipStream_t st) {
    dim3 grid(a.L * a.H, a.B), block(kWave);
    const size_t shared = (2 * static_cast<size_t>(a.R) + kWave) * sizeof(float);
    if (dtype == 0) hipLaunchKernelGGL(latent_plain_kernel<F16>, grid, block, shared, st, a);
    else if (dtype == 1) hipLaunchKernelGGL(latent_plain_kernel<BF16>, grid, block, shared, st, a);
    else hipLaunchKernelGGL(latent_plain_kernel<F32>, grid, block, shared, st, a);
    return static_cast<int>(hipGetLastError());
}

// ---- prompt --------------------------------------------------------------------------------------------------------
// grid (heads, query tiles, sequences): consecutive workgroups are different heads of one query tile, so that with a
// multiple of 8 heads the query tiles of a head meet in one XCD's L2.  Four wavefronts with 32 query rows each over
// 64-key tiles, double-buffered in LDS; longest query tiles first.
// K tile: rows of DKP + 8 elements.  V tile: one row per channel, 64 tokens + 8; inside each 16 tokens the order is
// 0-3, 8-11, 4-7, 12-15, so that the 8 tokens a lane half needs for one product are one 16-byte read.
constexpr int kPrefillRows = 128, kPrefillKeys = 64;

template <typename T, int DKP, int DVP>
__global__ __launch_bounds__(256, DKP <= 128 ? 2 : 1) void latent_prefill_kernel(LatentPrefillArgs a) {
    constexpr int KS = DKP / 16, VT = DVP / 32, KROW = DKP + 8, VROW = kPrefillKeys + 8;
    constexpr int KLOADS = kPrefillKeys * (DKP / 8) / 256, VLOADS = DVP * (kPrefillKeys / 8) / 256;
    static_assert(KLOADS * 256 == kPrefillKeys * (DKP / 8) && VLOADS * 256 == DVP * (kPrefillKeys / 8), "whole loads");
    extern __shared__ __attribute__((aligned(16))) uint16_t sm[];
    constexpr int kTileK = kPrefillKeys * KROW, kTileV = DVP * VROW;      // two K tiles, then two V tiles
    auto kt = [&](int buf) { return sm + buf * kTileK; };
    auto vt = [&](int buf) { return sm + 2 * kTileK + buf * kTileV; };
    const int tid = threadIdx.x, lane = tid & 63, wv = tid / kWave, col = lane & 31, hi = lane >> 5;
    const int h = blockIdx.x, b = blockIdx.z, D = a.D, Dv = a.Dv, H = a.H;
    const int tile = static_cast<int>(gridDim.y) - 1 - static_cast<int>(blockIdx.y);
    const int past = a.Lk - a.L;
    const int qw = tile * kPrefillRows + wv * 32;                  // the wavefront's first query token
    const int qi = qw + col;
    const bool valid = qi < a.L;
    const int qc = valid ? qi : a.L - 1;
    const int limit = past + qc;                                   // last key this row sees
    const int lo = a.start ? a.start[b] : 0;
    const int q_last = tile * kPrefillRows + kPrefillRows - 1 < a.L - 1 ? tile * kPrefillRows + kPrefillRows - 1 : a.L - 1;
    const int wave_last = past + (qw + 31 < a.L - 1 ? qw + 31 : a.L - 1);
    const int it0 = lo / kPrefillKeys, it1 = (past + q_last) / kPrefillKeys + 1;

    u32x4_a q[KS];
    {
        const uint16_t* qp = static_cast<const uint16_t*>(a.q) + ((static_cast<size_t>(b) * a.L + qc) * H + h) * D + 8 * hi;
        static_for<KS>([&](auto I) {
            constexpr int i = decltype(I)::value;
            q[i] = u32x4_a{0, 0, 0, 0};
            if (i * 16 + 8 * hi < D) q[i] = *reinterpret_cast<const u32x4_a*>(qp + i * 16);
        });
    }
    const uint16_t* kb = static_cast<const uint16_t*>(a.k) + (static_cast<size_t>(b) * a.Lk * H + h) * D;
    const uint16_t* vb = static_cast<const uint16_t*>(a.vt) + (static_cast<size_t>(b) * H + h) * Dv * a.ldv;
    u32x4_a ks[KLOADS], vs[VLOADS];
    auto fetch = [&](int it) {
        static_for<KLOADS>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const int u = i * 256 + tid, tok = u / (DKP / 8), ch = u % (DKP / 8);
            int key = it * kPrefillKeys + tok;
            key = key < a.Lk ? key : a.Lk - 1;                      // keys past the end: a copy, weight zero
            ks[i] = u32x4_a{0, 0, 0, 0};
            if (ch * 8 < D) ks[i] = *reinterpret_cast<const u32x4_a*>(kb + static_cast<size_t>(key) * H * D + ch * 8);
        });
        static_for<VLOADS>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const int u = i * 256 + tid, ch = u / 8, piece = u % 8;
            vs[i] = u32x4_a{0, 0, 0, 0};
            if (ch < Dv) vs[i] = *reinterpret_cast<const u32x4_a*>(vb + static_cast<size_t>(ch) * a.ldv + it * kPrefillKeys + piece * 8);
        });
    };
    auto put = [&](int buf) {
        static_for<KLOADS>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const int u = i * 256 + tid, tok = u / (DKP / 8), ch = u % (DKP / 8);
            *reinterpret_cast<u32x4_a*>(kt(buf) + tok * KROW + ch * 8) = ks[i];
        });
        static_for<VLOADS>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const int u = i * 256 + tid, ch = u / 8, piece = u % 8;
            uint16_t* d = vt(buf) + ch * VROW + (piece >> 1) * 16 + (piece & 1) * 4;
            *reinterpret_cast<u32x2_a*>(d) = u32x2_a{vs[i].x, vs[i].y};
            *reinterpret_cast<u32x2_a*>(d + 8) = u32x2_a{vs[i].z, vs[i].w};
        });
    };
    floatx16_a o[VT];
    static_for<VT>([&](auto I) {
        constexpr int i = decltype(I)::value;
#pragma unroll
        for (int j = 0; j < 16; j++) o[i][j] = 0.0f;
    });
    float m = kNone, l = 0.0f;
    const float scale2 = a.scale * kLog2e;

    if (it0 < it1) {
        fetch(it0);
        put(it0 & 1);
    }
    __syncthreads();
    for (int it = it0; it < it1; it++) {
        const int buf = it & 1;
        if (it + 1 < it1) fetch(it + 1);
        __builtin_amdgcn_sched_barrier(0);
        const int key0 = it * kPrefillKeys;
        if (key0 <= wave_last) {                                   // uniform over the wavefront
            floatx16_a s[2];
#pragma unroll
            for (int u = 0; u < 2; u++)
#pragma unroll
                for (int j = 0; j < 16; j++) s[u][j] = 0.0f;
            const uint16_t* kp = kt(buf) + col * KROW + 8 * hi;
            static_for<KS>([&](auto I) {
                constexpr int i = decltype(I)::value;
                s[0] = mma32<T>(*reinterpret_cast<const u32x4_a*>(kp + i * 16), q[i], s[0]);
                s[1] = mma32<T>(*reinterpret_cast<const u32x4_a*>(kp + 32 * KROW + i * 16), q[i], s[1]);
            });
            // this lane: query qi, keys key0 + 32 u + 8 (j / 4) + 4 hi + j % 4
            float mx = kNone;
            if (key0 + kPrefillKeys - 1 > past + qw || key0 < lo) {
#pragma unroll
                for (int u = 0; u < 2; u++)
#pragma unroll
                    for (int j = 0; j < 16; j++) {
                        const int key = key0 + 32 * u + 8 * (j >> 2) + 4 * hi + (j & 3);
                        s[u][j] = (key <= limit && key >= lo) ? s[u][j] * scale2 : -INFINITY;
                        mx = fmaxf(mx, s[u][j]);
                    }
            } else {
#pragma unroll
                for (int u = 0; u < 2; u++)
#pragma unroll
                    for (int j = 0; j < 16; j++) {
                        s[u][j] *= scale2;
                        mx = fmaxf(mx, s[u][j]);
                    }
            }
            mx = fmaxf(mx, __shfl_xor(mx, 32));
            if (__any(mx > m)) {
                const float mn = fmaxf(m, mx), al = exp2_hw(m - mn);
                l *= al;
                static_for<VT>([&](auto I) {
                    constexpr int i = decltype(I)::value;
#pragma unroll
                    for (int j = 0; j < 16; j++) o[i][j] *= al;
                });
                m = mn;
            }
            u32x4_a p[4];                                           // right operands of the four 16-token steps
#pragma unroll
            for (int u = 0; u < 2; u++)
#pragma unroll
                for (int j = 0; j < 16; j += 2) {
                    const float e0 = exp2_hw(s[u][j] - m), e1 = exp2_hw(s[u][j + 1] - m);
                    l += e0 + e1;
                    p[2 * u + (j >> 3)][(j & 7) >> 1] = pack2<T>(e0, e1);
                }
            const uint16_t* vp = vt(buf) + col * VROW + 8 * hi;
            static_for<VT>([&](auto I) {
                constexpr int i = decltype(I)::value;
                static_for<4>([&](auto J) {
                    constexpr int j = decltype(J)::value;
                    o[i] = mma32<T>(*reinterpret_cast<const u32x4_a*>(vp + i * 32 * VROW + j * 16), p[j], o[i]);
                });
            });
        }
        if (it + 1 < it1) put(buf ^ 1);
        __syncthreads();
    }
    l += __shfl_xor(l, 32);
    if (!valid) return;
    const float sink2 = a.sink[h] * kLog2e, mf = fmaxf(m, sink2);
    const float al = exp2_hw(m - mf), inv = al / (l * al + exp2_hw(sink2 - mf));
    const size_t row = static_cast<size_t>(b) * a.L + qi;
    uint16_t* out = static_cast<uint16_t*>(a.out) + row * H * Dv + static_cast<size_t>(h) * Dv;
    const uint16_t* gate = a.gate ? static_cast<const uint16_t*>(a.gate) + row * a.gate_row + static_cast<size_t>(h) * Dv : nullptr;
    const bool quads = Dv % 4 == 0 && (!gate || a.gate_row % 4 == 0);
    static_for<VT>([&](auto I) {
        constexpr int i = decltype(I)::value;
#pragma unroll
        for (int j4 = 0; j4 < 4; j4++) {
            const int ch = i * 32 + 8 * j4 + 4 * hi;
            float v[4];
#pragma unroll
            for (int j = 0; j < 4; j++) v[j] = o[i][4 * j4 + j] * inv;
            if (quads && ch + 4 <= Dv) {
                if (gate) {
                    const uint2 gv = *reinterpret_cast<const uint2*>(gate + ch);
                    const uint32_t gw[2] = {gv.x, gv.y};
#pragma unroll
                    for (int j = 0; j < 4; j++) v[j] = v[j] / (1.0f + __expf(-lo2f<T>(static_cast<uint16_t>(gw[j >> 1] >> (16 * (j & 1))))));
                }
                *reinterpret_cast<uint2*>(out + ch) = make_uint2(pack2<T>(v[0], v[1]), pack2<T>(v[2], v[3]));
            } else {
#pragma unroll
                for (int j = 0; j < 4; j++)
                    if (ch + j < Dv) out[ch + j] = f2lo<T>(gate ? v[j] / (1.0f + __expf(-lo2f<T>(gate[ch + j]))) : v[j]);
            }
        }
    });
}

template <typename T, int DKP, int DVP>
static int prefill_one(const LatentPrefillArgs& a, hipStream_t st) {
    constexpr size_t bytes = 2 * 2 * (static_cast<size_t>(kPrefillKeys) * (DKP + 8) + static_cast<size_t>(DVP) * (kPrefillKeys + 8));
    static_assert(bytes <= 160 * 1024, "LDS");
    if (bytes > 64 * 1024) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&latent_prefill_kernel<T, DKP, DVP>),
                                                 hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(bytes));
        if (e != hipSuccess) return static_cast<int>(e);
    }
    dim3 grid(a.H, (a.L + kPrefillRows - 1) / kPrefillRows, a.B), block(256);
    hipLaunchKernelGGL((latent_prefill_kernel<T, DKP, DVP>), grid, block, bytes, st, a);
    return static_cast<int>(hipGetLastError());
}

template <typename T>
static int prefill_dims(const LatentPrefillArgs& a, hipStream_t st) {
    if (a.D <= 64 && a.Dv <= 64) return prefill_one<T, 64, 64>(a, st);
    if (a.D <= 128 && a.Dv <= 128) return prefill_one<T, 128, 128>(a, st);
    if (a.D <= 192 && a.Dv <= 128) return prefill_one<T, 192, 128>(a, st);
    return prefill_one<T, 256, 256>(a, st);
}

int launch_latent_prefill(const LatentPrefillArgs& a, int dtype, hipStream_t st) {
    return dtype == 0 ? prefill_dims<F16>(a, st) : prefill_dims<BF16>(a, st);
}

}  // namespace pq
