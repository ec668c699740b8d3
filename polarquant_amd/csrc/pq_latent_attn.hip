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
#include "pq_mfma.h"
#include "pq_latent_internal.h"

namespace pq {

// ---- decode --------------------------------------------------------------------------------------------------------
// grid (slices, row tiles, sequences); a row is (query token, head), a workgroup owns 16 * RT of them and walks its slice
// 32 keys at a time.  The latent's channels are divided among its wavefronts: each holds its channels of the queries and of
// the output, loads its channels of the keys (the next tile's while it works on the current one) and keeps them in LDS of
// its own.  Per tile, each wavefront multiplies its channels of K and Q^T, the partial scores are added up through LDS (the
// only barrier), every wavefront runs the softmax of all rows, and multiplies its channels of V^T, the same LDS tile
// transposed on the way out, with P^T.  So each key is read from HBM once, and from LDS once per product, for all rows.
// 16-byte pieces of a key's row are XOR-swizzled by the key so that neither access meets in few banks.
// Workspace: [B, slices, L * H] pairs (maximum in log2 units, sum), then as many rows of R floats.
constexpr int kDecodeTile = 32;
__device__ __forceinline__ size_t pairs_floats(const LatentDecodeArgs& a) {     // up to the accumulators' 16-byte boundary
    return (2 * static_cast<size_t>(a.B) * a.n_splits * a.L * a.H + 3) & ~static_cast<size_t>(3);
}
template <int RP> struct DecodeShape {
    static constexpr int CW = RP / 4 < 32 ? 32 : RP / 4;       // channels per wavefront
    static constexpr int NW = RP / CW;                         // wavefronts
};

template <typename T, int RP, int RT>
__global__ __launch_bounds__(kWave * DecodeShape<RP>::NW, RT <= 2 ? 2 : 1) void latent_decode_kernel(LatentDecodeArgs a) {
    constexpr int CW = DecodeShape<RP>::CW, NW = DecodeShape<RP>::NW, CH = CW / 8, KS = CW / 32, CT = CW / 16;
    constexpr int LPT = kDecodeTile * CH / kWave, RPW = 16 / CH;           // loads per lane; rows per 256 bytes of LDS
    __shared__ __attribute__((aligned(16))) uint16_t tiles[NW][kDecodeTile * CW];
    __shared__ floatx4_a exch[2][NW][2 * RT][kWave];
    const int tid = threadIdx.x, lane = tid & 63, wv = tid / kWave, r16 = lane & 15, g = lane >> 4;
    const int b = blockIdx.z, split = blockIdx.x, R = a.R, rows = a.L * a.H, n0 = blockIdx.y * 16 * RT;
    const int pos = a.pos_dev ? *a.pos_dev : a.pos;
    const int total = static_cast<int>(static_cast<int64_t>(pos) + a.L < a.capacity ? pos + a.L : a.capacity);   // (below 2^30)
    const int lo = a.start ? a.start[b] : 0;
    const int per = ((total - lo + a.n_splits - 1) / a.n_splits + kDecodeTile - 1) / kDecodeTile * kDecodeTile;
    const int64_t begin = lo + static_cast<int64_t>(split) * per;
    const int s0 = static_cast<int>(begin < total ? begin : total), s1 = begin + per < total ? s0 + per : total;
    const size_t part = (static_cast<size_t>(b) * a.n_splits + split) * rows;
    float* ml = a.workspace + 2 * part;
    float* acc = a.workspace + pairs_floats(a) + part * R;
    if (s0 >= s1) {                                  // uniform over the workgroup
        if (tid < 16 * RT && n0 + tid < rows) { ml[2 * (n0 + tid)] = kNone; ml[2 * (n0 + tid) + 1] = 0.0f; }
        return;
    }
    auto swz = [](int tok) { return (tok / RPW) % CH; };
    const int c0 = wv * CW;                          // this wavefront's first channel

    const uint16_t* cb = static_cast<const uint16_t*>(a.c) + static_cast<size_t>(b) * a.capacity * R;
    uint16_t* tile = tiles[wv];

    u32x4_a stage[LPT];
    uint32_t off[LPT], col[LPT];                     // elements from the tile's first key
    static_for<LPT>([&](auto I) {
        constexpr int i = decltype(I)::value;
        const int u = i * kWave + lane, c = c0 + (u % CH) * 8;
        col[i] = c < R ? c : 0;
        off[i] = static_cast<uint32_t>(u / CH) * R + col[i];
    });
    auto fetch = [&](int key0) {
        const uint16_t* base = cb + static_cast<int64_t>(key0) * R;
        const int last = s1 - 1 - key0;              // uniform
        static_for<LPT>([&](auto I) {
            constexpr int i = decltype(I)::value;
            // no branch around a load (it would be waited for at the join): rows past the slice are a copy with weight
            // zero, columns past R a copy that meets zeros of q and whose output columns are never stored
            const int tok = (i * kWave + lane) / CH;
            stage[i] = *reinterpret_cast<const u32x4_a*>(base + (tok <= last ? off[i] : static_cast<uint32_t>(last) * R + col[i]));
        });
    };
    fetch(s0);
    __builtin_amdgcn_sched_barrier(0);
    u32x4_a q[RT][KS];
    int limit[RT];                                   // keys a row may see: positions below it
    static_for<RT>([&](auto J) {
        constexpr int j = decltype(J)::value;
        const int n = n0 + j * 16 + r16 < rows ? n0 + j * 16 + r16 : rows - 1;
        limit[j] = pos + n / a.H + 1;
        const uint16_t* qp = static_cast<const uint16_t*>(a.q) + (static_cast<size_t>(b) * rows + n) * R;
        static_for<KS>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const int c = c0 + i * 32 + 8 * g;
            const u32x4_a t = *reinterpret_cast<const u32x4_a*>(qp + (c < R ? c : 0));
            q[j][i] = c < R ? t : u32x4_a{0, 0, 0, 0};
        });
    });
    const int first_limit = pos + n0 / a.H + 1;      // the smallest of them: tiles below it need no mask
    const float scale2 = a.scale * kLog2e;
    auto put = [&]() {
        static_for<LPT>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const int u = i * kWave + lane, tok = u / CH, ch = u % CH;
            *reinterpret_cast<u32x4_a*>(tile + tok * CW + ((ch ^ swz(tok)) * 8)) = stage[i];
        });
    };
    floatx4_a o[RT][CT];
    static_for<RT>([&](auto J) { static_for<CT>([&](auto I) { o[decltype(J)::value][decltype(I)::value] = floatx4_a{0, 0, 0, 0}; }); });
    float m[RT], l[RT];
    static_for<RT>([&](auto J) { m[decltype(J)::value] = kNone; l[decltype(J)::value] = 0.0f; });
    int koff[KS], voff[CT];                          // elements inside the tile
    static_for<KS>([&](auto I) { constexpr int i = decltype(I)::value; koff[i] = r16 * CW + (((i * 4 + g) ^ swz(r16)) * 8); });
    {
        const int row = 4 * g + (r16 >> 2);
        static_for<CT>([&](auto I) {
            constexpr int i = decltype(I)::value;
            voff[i] = row * CW + (((i * 2 + ((r16 & 3) >> 1)) ^ swz(row)) * 8) + (r16 & 1) * 4;
        });
    }
    static_assert((16 / RPW) % CH == 0, "rows 16 apart are swizzled alike");

    const int ntiles = (s1 - s0 + kDecodeTile - 1) / kDecodeTile;
    put();
    for (int it = 0; it < ntiles; it++) {
        if (it + 1 < ntiles) fetch(s0 + (it + 1) * kDecodeTile);
        __builtin_amdgcn_sched_barrier(0);
        u32x4_a k[2][KS];
        static_for<KS>([&](auto I) {
            constexpr int i = decltype(I)::value;
            k[0][i] = *reinterpret_cast<const u32x4_a*>(tile + koff[i]);
            k[1][i] = *reinterpret_cast<const u32x4_a*>(tile + koff[i] + 16 * CW);
        });
        floatx4_a s[RT][2];
        static_for<RT>([&](auto J) { constexpr int j = decltype(J)::value; s[j][0] = s[j][1] = floatx4_a{0, 0, 0, 0}; });
        static_for<KS>([&](auto I) {
            constexpr int i = decltype(I)::value;
            static_for<RT>([&](auto J) {
                constexpr int j = decltype(J)::value;
                s[j][0] = mma16<T>(k[0][i], q[j][i], s[j][0]);
                s[j][1] = mma16<T>(k[1][i], q[j][i], s[j][1]);
            });
        });
        // the second product's operands, ahead of the exchange
        u32x4_a v[CT];
        static_for<CT>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const u32x2_a w0 = __builtin_bit_cast(u32x2_a, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_short4*)(tile + voff[i])));
            const u32x2_a w1 = __builtin_bit_cast(u32x2_a, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_short4*)(tile + voff[i] + 16 * CW)));
            v[i] = u32x4_a{w0.x, w0.y, w1.x, w1.y};
        });
        floatx4_a(*ex)[2 * RT][kWave] = exch[it & 1];
        static_for<RT>([&](auto J) {
            constexpr int j = decltype(J)::value;
            ex[wv][2 * j][lane] = s[j][0];
            ex[wv][2 * j + 1][lane] = s[j][1];
        });
        __syncthreads();     // (the other buffer's readers are done before they arrive here)
        const int tile0 = s0 + it * kDecodeTile, key0 = tile0 + 4 * g;
        const bool whole = tile0 + kDecodeTile <= first_limit && tile0 + kDecodeTile <= s1;
        static_for<RT>([&](auto J) {
            constexpr int j = decltype(J)::value;
            // this lane: row r16 of row tile j, keys key0 + jj and key0 + 16 + jj
            float p[8], mx = kNone;
#pragma unroll
            for (int u = 0; u < 2; u++) {
                floatx4_a t = ex[0][2 * j + u][lane];
#pragma unroll
                for (int w = 1; w < NW; w++) t += ex[w][2 * j + u][lane];
#pragma unroll
                for (int jj = 0; jj < 4; jj++) p[4 * u + jj] = t[jj] * scale2;
            }
            if (!whole) {
#pragma unroll
                for (int e = 0; e < 8; e++) {
                    const int key = key0 + 16 * (e >> 2) + (e & 3);
                    if (key >= limit[j] || key >= s1) p[e] = -INFINITY;
                }
            }
#pragma unroll
            for (int e = 0; e < 8; e++) mx = fmaxf(mx, p[e]);
            mx = fmaxf(mx, __shfl_xor(mx, 16));
            mx = fmaxf(mx, __shfl_xor(mx, 32));
            if (__any(mx > m[j])) {
                const float mn = fmaxf(m[j], mx), al = exp2_hw(m[j] - mn);
                l[j] *= al;
                static_for<CT>([&](auto I) {
                    constexpr int i = decltype(I)::value;
                    o[j][i] *= al;
                });
                m[j] = mn;
            }
#pragma unroll
            for (int e = 0; e < 8; e++) { p[e] = exp2_hw(p[e] - m[j]); l[j] += p[e]; }
            const u32x4_a pt = {pack2<T>(p[0], p[1]), pack2<T>(p[2], p[3]), pack2<T>(p[4], p[5]), pack2<T>(p[6], p[7])};
            static_for<CT>([&](auto I) {
                constexpr int i = decltype(I)::value;
                o[j][i] = mma16<T>(v[i], pt, o[j][i]);
            });
        });
        if (it + 1 < ntiles) put();
    }
    static_for<RT>([&](auto J) {
        constexpr int j = decltype(J)::value;
        const int n = n0 + j * 16 + r16;
        float ls = l[j] + __shfl_xor(l[j], 16);
        ls += __shfl_xor(ls, 32);
        if (n < rows) {
            if (g == 0 && wv == 0) { ml[2 * n] = m[j]; ml[2 * n + 1] = ls; }
            static_for<CT>([&](auto I) {
                constexpr int i = decltype(I)::value;
                const int c = c0 + i * 16 + 4 * g;
                if (c < R) *reinterpret_cast<float4*>(acc + static_cast<size_t>(n) * R + c) = make_float4(o[j][i][0], o[j][i][1], o[j][i][2], o[j][i][3]);
            });
        }
    });
}

// grid (L * H, channel blocks of 64, B), 256 threads: joins the slices of a row; the sink joins the denominator here, once.
// 16 lanes hold a block's channels, the 16 groups of them take the slices in turn.
constexpr int kMaxSlices = 512;
template <typename T>
__global__ __launch_bounds__(256) void latent_merge_kernel(LatentDecodeArgs a) {
    __shared__ float wgt[kMaxSlices], red[8];
    __shared__ float4 sums[16][16];
    const int n = blockIdx.x, b = blockIdx.z, rows = a.L * a.H, S = a.n_splits, R = a.R, tid = threadIdx.x;
    const int ch = blockIdx.y * 64 + (tid & 15) * 4, grp = tid >> 4;
    const int cc = ch < R ? ch : 0;
    const size_t first = static_cast<size_t>(b) * S * rows + n;
    const float sink2 = a.sink[n % a.H] * kLog2e;
    float mx = sink2, den = 0.0f;
    for (int s = tid; s < S; s += 256) mx = fmaxf(mx, a.workspace[2 * (first + static_cast<size_t>(s) * rows)]);
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o));
    if ((tid & 63) == 0) red[tid >> 6] = mx;
    __syncthreads();
    mx = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
    for (int s = tid; s < S; s += 256) {
        const float* p = a.workspace + 2 * (first + static_cast<size_t>(s) * rows);
        const float w = p[0] > kNone ? exp2_hw(p[0] - mx) : 0.0f;
        wgt[s] = w;
        den += w * p[1];
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) den += __shfl_xor(den, o);
    if ((tid & 63) == 0) red[4 + (tid >> 6)] = den;
    __syncthreads();
    const float* acc = a.workspace + pairs_floats(a) + first * R + cc;
    float4 sum = make_float4(0, 0, 0, 0);
#pragma unroll 4
    for (int s = grp; s < S; s += 16) {
        const float w = wgt[s];
        const float4 v = *reinterpret_cast<const float4*>(acc + static_cast<size_t>(s) * rows * R);
        const bool live = w != 0.0f;                 // (an empty slice's accumulators were never written)
        sum.x = __builtin_fmaf(w, live ? v.x : 0.0f, sum.x); sum.y = __builtin_fmaf(w, live ? v.y : 0.0f, sum.y);
        sum.z = __builtin_fmaf(w, live ? v.z : 0.0f, sum.z); sum.w = __builtin_fmaf(w, live ? v.w : 0.0f, sum.w);
    }
    sums[grp][tid & 15] = sum;
    __syncthreads();
    if (grp != 0 || ch >= R) return;
    for (int j = 1; j < 16; j++) {
        const float4 v = sums[j][tid];
        sum.x += v.x; sum.y += v.y; sum.z += v.z; sum.w += v.w;
    }
    const float inv = 1.0f / (red[4] + red[5] + red[6] + red[7] + exp2_hw(sink2 - mx));
    *reinterpret_cast<uint2*>(static_cast<uint16_t*>(a.out) + (static_cast<size_t>(b) * rows + n) * R + ch) =
        make_uint2(pack2<T>(sum.x * inv, sum.y * inv), pack2<T>(sum.z * inv, sum.w * inv));
}

int launch_latent_decode(const LatentDecodeArgs& a, int dtype, hipStream_t st) {
    const int rows = a.L * a.H;
    const int rt = rows <= 16 ? 1 : rows <= 32 ? 2 : 4;
    dim3 grid(a.n_splits, (rows + 16 * rt - 1) / (16 * rt), a.B);
#define PQ_LD1(T, RP, RT) hipLaunchKernelGGL((latent_decode_kernel<T, RP, RT>), grid, dim3(kWave * DecodeShape<RP>::NW), 0, st, a)
#define PQ_LD(T, RP) do { if (rt == 1) PQ_LD1(T, RP, 1); else if (rt == 2) PQ_LD1(T, RP, 2); else PQ_LD1(T, RP, 4); } while (0)
#define PQ_LDT(T)                                                                                                    \
    do {                                                                                                             \
        if (a.R <= 64) PQ_LD(T, 64); else if (a.R <= 128) PQ_LD(T, 128);                                             \
        else if (a.R <= 256) PQ_LD(T, 256); else PQ_LD(T, 512);                                                      \
    } while (0)
    if (dtype == 0) PQ_LDT(F16); else PQ_LDT(BF16);
#undef PQ_LDT
#undef PQ_LD
#undef PQ_LD1
    int err = static_cast<int>(hipGetLastError());
    if (err) return err;
    dim3 mgrid(rows, (a.R + 63) / 64, a.B), mblock(256);
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
        const uint16_t* qp = static_cast<const uint16_t*>(a.q) + ((static_cast<size_t>(b) * a.L + qc) * H + h) * D;
        static_for<KS>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const int c = i * 16 + 8 * hi;
            const u32x4_a t = *reinterpret_cast<const u32x4_a*>(qp + (c < D ? c : 0));
            q[i] = c < D ? t : u32x4_a{0, 0, 0, 0};
        });
    }
    const uint16_t* kb = static_cast<const uint16_t*>(a.k) + (static_cast<size_t>(b) * a.Lk * H + h) * D;
    const uint16_t* vb = static_cast<const uint16_t*>(a.vt) + (static_cast<size_t>(b) * H + h) * Dv * a.ldv;
    u32x4_a ks[KLOADS], vs[VLOADS];
    const uint32_t k_row = static_cast<uint32_t>(H) * D;
    auto fetch = [&](int it) {
        const uint16_t* kbase = kb + static_cast<size_t>(it) * kPrefillKeys * k_row;
        const int last = a.Lk - 1 - it * kPrefillKeys;             // uniform
        static_for<KLOADS>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const int u = i * 256 + tid, tok = u / (DKP / 8), ch = u % (DKP / 8);
            // no branch around a load (it would be waited for at the join): keys past the end are a copy with weight zero,
            // columns past D a copy that meets zeros of q
            ks[i] = *reinterpret_cast<const u32x4_a*>(kbase + (static_cast<uint32_t>(tok <= last ? tok : last) * k_row + (ch * 8 < D ? ch * 8 : 0)));
        });
        static_for<VLOADS>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const int u = i * 256 + tid, piece = u % 8, ch = u / 8 < Dv ? u / 8 : Dv - 1;      // (rows past Dv are never stored)
            vs[i] = *reinterpret_cast<const u32x4_a*>(vb + static_cast<size_t>(ch) * a.ldv + it * kPrefillKeys + piece * 8);
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
