// Attention over a sliding window of grouped keys, with a bias per position of distance and norms of q and k over the whole
// projection.
//
//   qk_norm_kernel         norms of q and of k, the latter and v written to the ring (short calls) or k to a buffer
//   ring_append_kernel     the last keys and values of a long call, into the ring
//   window_decode_kernel   few query tokens, from the ring: the window cut into slices; window_merge_kernel joins them
//   window_prefill_kernel  many query tokens: flash attention over ring and new keys
//   window_plain_kernel    any size, any dtype (float32 runs here), one wavefront per query row
//
// The matrix-core kernels compute S^T = K Q^T, so that a query row is a lane: its softmax state is one register, and the weights
// P^T leave the first product in the layout in which the second one, O^T = V^T P^T, takes its right operand.  Scores,
// bias, softmax and all sums are float32; q, k, v and the weights enter the products in the model's 16-bit dtype.
#include "pq_mfma.h"
#include "pq_recurrent_internal.h"

namespace pq {

// ---- norms and append -------------------------------------------------------------------------------------------------
// A workgroup per token.
template <typename T, int V>
__global__ __launch_bounds__(256) void qk_norm_kernel(QkNormArgs a) {
    __shared__ float part[2][4];
    const int tid = threadIdx.x, wv = tid >> 6, tok = blockIdx.x, b = tok / a.L, t = tok - b * a.L;
    const int nq = a.H * a.D, nk = a.G * a.D, nv = a.G * a.Dv;
    const elem_t<T>* q = static_cast<const elem_t<T>*>(a.q) + static_cast<size_t>(tok) * a.p_row;
    const elem_t<T>* k = static_cast<const elem_t<T>*>(a.k) + static_cast<size_t>(tok) * a.p_row;
    const elem_t<T>* v = static_cast<const elem_t<T>*>(a.v) + static_cast<size_t>(tok) * a.p_row;
    float sq = 0.0f, sk = 0.0f, x[V], w[V];
    for (int i = tid * V; i < nq; i += 256 * V) {
        ldv<T, V>(q, i, x);
#pragma unroll
        for (int j = 0; j < V; j++) sq = __builtin_fmaf(x[j], x[j], sq);
    }
    for (int i = tid * V; i < nk; i += 256 * V) {
        ldv<T, V>(k, i, x);
#pragma unroll
        for (int j = 0; j < V; j++) sk = __builtin_fmaf(x[j], x[j], sk);
    }
    sq = wave_sum(sq);
    sk = wave_sum(sk);
    if ((tid & 63) == 0) { part[0][wv] = sq; part[1][wv] = sk; }
    __syncthreads();
    sq = part[0][0] + part[0][1] + part[0][2] + part[0][3];
    sk = part[1][0] + part[1][1] + part[1][2] + part[1][3];
    const float rq = 1.0f / sqrtf(sq / static_cast<float>(nq) + a.eps), rk = 1.0f / sqrtf(sk / static_cast<float>(nk) + a.eps);
    for (int i = tid * V; i < nq; i += 256 * V) {
        ldv<T, V>(q, i, x);
        ldv<T, V>(a.w_q, i, w);
#pragma unroll
        for (int j = 0; j < V; j++) x[j] = x[j] * rq * w[j];
        stv<T, V>(static_cast<elem_t<T>*>(a.q_out) + static_cast<size_t>(tok) * nq, i, x);
    }
    const int pos = (a.pos_dev ? *a.pos_dev : a.pos) + t;
    const int slot = (pos < 0 ? 0 : pos) % a.cap;
    auto ring = [&](void* base, int i, int width) {
        const int g = i / width;
        return static_cast<elem_t<T>*>(base) + ((static_cast<size_t>(b) * a.G + g) * a.cap + slot) * width + (i - g * width);
    };
    for (int i = tid * V; i < nk; i += 256 * V) {
        ldv<T, V>(k, i, x);
        ldv<T, V>(a.w_k, i, w);
#pragma unroll
        for (int j = 0; j < V; j++) x[j] = x[j] * rk * w[j];
        if (a.k_out) stv<T, V>(static_cast<elem_t<T>*>(a.k_out) + static_cast<size_t>(tok) * nk, i, x);
        else stv<T, V>(ring(a.k_ring, i, a.D), 0, x);
    }
    if (a.k_out) return;
    for (int i = tid * V; i < nv; i += 256 * V) {
        ldv<T, V>(v, i, x);
        stv<T, V>(ring(a.v_ring, i, a.Dv), 0, x);
    }
}

int launch_qk_norm(const QkNormArgs& a, int dtype, hipStream_t st) {
    const size_t align = dtype == 2 ? 16 : 8;
    auto ok = [&](const void* p) { return reinterpret_cast<uintptr_t>(p) % align == 0; };
    const bool v4 = a.D % 4 == 0 && a.Dv % 4 == 0 && a.p_row % 4 == 0 && ok(a.q) && ok(a.k) && ok(a.v) && ok(a.w_q) && ok(a.w_k) &&
                    ok(a.q_out) && ok(a.k_out) && ok(a.k_ring) && ok(a.v_ring);
    dim3 grid(static_cast<unsigned>(a.B * a.L)), block(256);
#define PQ_QN(T) do { if (v4) hipLaunchKernelGGL((qk_norm_kernel<T, 4>), grid, block, 0, st, a); \
                      else hipLaunchKernelGGL((qk_norm_kernel<T, 1>), grid, block, 0, st, a); } while (0)
    if (dtype == 0) PQ_QN(F16); else if (dtype == 1) PQ_QN(BF16); else PQ_QN(F32);
#undef PQ_QN
    return static_cast<int>(hipGetLastError());
}

// grid (rows kept, sequences)
template <typename E>
__global__ __launch_bounds__(256) void ring_append_kernel(RingAppendArgs a) {
    const int b = blockIdx.y, t = a.L - static_cast<int>(gridDim.x) + static_cast<int>(blockIdx.x), slot = (a.pos + t) % a.cap;
    const size_t row = static_cast<size_t>(b) * a.L + t;
    const E *k = static_cast<const E*>(a.k) + row * a.k_row, *v = static_cast<const E*>(a.v) + row * a.v_row;
    E *kr = static_cast<E*>(a.k_ring), *vr = static_cast<E*>(a.v_ring);
    for (int i = threadIdx.x; i < a.G * a.D; i += 256) {
        const int g = i / a.D;
        kr[((static_cast<size_t>(b) * a.G + g) * a.cap + slot) * a.D + (i - g * a.D)] = k[i];
    }
    for (int i = threadIdx.x; i < a.G * a.Dv; i += 256) {
        const int g = i / a.Dv;
        vr[((static_cast<size_t>(b) * a.G + g) * a.cap + slot) * a.Dv + (i - g * a.Dv)] = v[i];
    }
}

int launch_ring_append(const RingAppendArgs& a, int dtype, hipStream_t st) {
    dim3 grid(static_cast<unsigned>(a.L < a.cap ? a.L : a.cap), static_cast<unsigned>(a.B)), block(256);
    if (dtype == 2) hipLaunchKernelGGL(ring_append_kernel<float>, grid, block, 0, st, a);
    else hipLaunchKernelGGL(ring_append_kernel<uint16_t>, grid, block, 0, st, a);
    return static_cast<int>(hipGetLastError());
}

// ---- decode --------------------------------------------------------------------------------------------------------------
// grid (slices, key heads x row tiles, sequences); a row is (query token, query head of the group), a workgroup owns 16 of them.
// Its wavefronts take the window's 32-key tiles in turn, each with a softmax of its own: keys go from the ring straight into
// operand registers, values through an LDS tile of the wavefront's own and out of it transposed, the next tile's loads in
// flight.  At the end the wavefronts are joined through LDS; with one slice that is the result, otherwise a partial:
// workspace [B, G, L * H / G, slices] pairs (maximum in log2 units, sum), then as many rows of Dv floats.
constexpr int kTile = 32, kVPad = 16;
constexpr int decode_waves(int width) { return width <= 128 ? 8 : 4; }       // (wider heads: more registers each)
__device__ __forceinline__ size_t window_pairs(const WindowAttnArgs& a) {      // floats, up to a 16-byte boundary
    return (2 * static_cast<size_t>(a.B) * a.L * a.H * a.n_splits + 3) & ~static_cast<size_t>(3);
}

template <typename T, int DKP, int DVP>
__global__ __launch_bounds__(kWave * decode_waves(DVP), 1) void window_decode_kernel(WindowAttnArgs a) {
    constexpr int kDecodeWaves = decode_waves(DVP), KS = DKP / 32, CT = DVP / 16, CH = DVP / 8, LPT = kTile * CH / kWave, VROW = DVP + kVPad;
    extern __shared__ __attribute__((aligned(16))) uint16_t sm[];
    __shared__ float wm[kDecodeWaves][16], wl[kDecodeWaves][16];
    const int tid = threadIdx.x, lane = tid & 63, wv = tid / kWave, r16 = lane & 15, g4 = lane >> 4;
    const int rep = a.H / a.G, rows = a.L * rep, row_tiles = (rows + 15) / 16;
    const int g = blockIdx.y / row_tiles, n0 = (blockIdx.y - g * row_tiles) * 16, b = blockIdx.z, split = blockIdx.x;
    const int pos = a.pos_dev ? *a.pos_dev : a.pos, lo = a.start ? a.start[b] : 0, D = a.D, Dv = a.Dv;
    const int n = n0 + r16 < rows ? n0 + r16 : rows - 1, i_row = pos + n / rep, h = g * rep + n % rep;
    int key_lo = pos + n0 / rep - a.window + 1;                      // of the tile's first token
    key_lo = key_lo > lo ? key_lo : lo;
    key_lo = key_lo > 0 ? key_lo : 0;
    const int last_row = n0 + 15 < rows ? n0 + 15 : rows - 1, key_hi = pos + last_row / rep;
    const int tile0 = key_lo / kTile, tiles = key_hi >= key_lo ? key_hi / kTile - tile0 + 1 : 0;
    const int step = a.n_splits * kDecodeWaves;
    const size_t head = static_cast<size_t>(b) * a.G + g;
    const uint16_t* kr = static_cast<const uint16_t*>(a.k_ring) + head * a.cap * D;
    const uint16_t* vr = static_cast<const uint16_t*>(a.v_ring) + head * a.cap * Dv;
    uint16_t* vt = sm + wv * kTile * VROW;

    u32x4_a q[KS], k[2][KS], stage[LPT];
    const uint16_t* qp = static_cast<const uint16_t*>(a.q) + ((static_cast<size_t>(b) * a.L + n / rep) * a.H + h) * D;
    static_for<KS>([&](auto I) {
        constexpr int i = decltype(I)::value;
        const int c = i * 32 + 8 * g4;
        const u32x4_a t = *reinterpret_cast<const u32x4_a*>(qp + (c < D ? c : 0));
        q[i] = c < D ? t : u32x4_a{0, 0, 0, 0};
    });
    // whole tiles are inside the ring; columns past D are a copy that meets zeros of q, columns past Dv are never stored
    auto fetch = [&](int tile) {
        const int slot = (tile0 + tile) * kTile % a.cap;
        const uint16_t* kp = kr + static_cast<size_t>(slot + r16) * D;
        static_for<KS>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const int c = i * 32 + 8 * g4 < D ? i * 32 + 8 * g4 : 0;
            k[0][i] = *reinterpret_cast<const u32x4_a*>(kp + c);
            k[1][i] = *reinterpret_cast<const u32x4_a*>(kp + 16 * static_cast<size_t>(D) + c);
        });
        const uint16_t* vp = vr + static_cast<size_t>(slot) * Dv;
        static_for<LPT>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const int u = i * kWave + lane, tok = u / CH, c = (u % CH) * 8;
            stage[i] = *reinterpret_cast<const u32x4_a*>(vp + static_cast<size_t>(tok) * Dv + (c < Dv ? c : 0));
        });
    };
    floatx4_a o[CT];
    static_for<CT>([&](auto I) { o[decltype(I)::value] = floatx4_a{0, 0, 0, 0}; });
    float m = kNone, l = 0.0f;
    const float scale2 = a.scale * kLog2e, slope2 = a.slopes ? a.slopes[h] * kLog2e : 0.0f;
    int tile = split * kDecodeWaves + wv;
    if (tile < tiles) fetch(tile);
    for (; tile < tiles; tile += step) {
        floatx4_a s[2] = {floatx4_a{0, 0, 0, 0}, floatx4_a{0, 0, 0, 0}};
        static_for<KS>([&](auto I) {
            constexpr int i = decltype(I)::value;
            s[0] = mma16<T>(k[0][i], q[i], s[0]);
            s[1] = mma16<T>(k[1][i], q[i], s[1]);
        });
        static_for<LPT>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const int u = i * kWave + lane;
            *reinterpret_cast<u32x4_a*>(vt + (u / CH) * VROW + (u % CH) * 8) = stage[i];
        });
        if (tile + step < tiles) fetch(tile + step);
        __builtin_amdgcn_wave_barrier();
        // this lane: row r16, keys key0 + jj and key0 + 16 + jj
        const int key0 = (tile0 + tile) * kTile + 4 * g4;
        float p[8], mx = kNone;
#pragma unroll
        for (int e = 0; e < 8; e++) {
            const int key = key0 + 16 * (e >> 2) + (e & 3), back = i_row - key;
            const bool seen = back >= 0 && back < a.window && key >= lo;
            p[e] = seen ? __builtin_fmaf(-slope2, static_cast<float>(back), s[e >> 2][e & 3] * scale2) : -INFINITY;
            mx = fmaxf(mx, p[e]);
        }
        mx = fmaxf(mx, __shfl_xor(mx, 16));
        mx = fmaxf(mx, __shfl_xor(mx, 32));
        const float mn = fmaxf(m, mx), al = exp2_hw(m - mn);
        m = mn;
        l *= al;
#pragma unroll
        for (int e = 0; e < 8; e++) { p[e] = exp2_hw(p[e] - m); l += p[e]; }
        const u32x4_a pt = {pack2<T>(p[0], p[1]), pack2<T>(p[2], p[3]), pack2<T>(p[4], p[5]), pack2<T>(p[6], p[7])};
        static_for<CT>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const uint16_t* vp = vt + (4 * g4 + (r16 >> 2)) * VROW + i * 16 + (r16 & 3) * 4;
            const u32x2_a w0 = __builtin_bit_cast(u32x2_a, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_short4*)vp));
            const u32x2_a w1 = __builtin_bit_cast(u32x2_a, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_short4*)(vp + 16 * VROW)));
            o[i] *= al;
            o[i] = mma16<T>(u32x4_a{w0.x, w0.y, w1.x, w1.y}, pt, o[i]);
        });
        __builtin_amdgcn_wave_barrier();
    }
    l += __shfl_xor(l, 16);
    l += __shfl_xor(l, 32);
    __syncthreads();                                                 // the tiles' memory takes the wavefronts' results
    float* acc = reinterpret_cast<float*>(sm);                       // [wavefront][row][DVP]
    if (g4 == 0) { wm[wv][r16] = m; wl[wv][r16] = l; }
    static_for<CT>([&](auto I) {
        constexpr int i = decltype(I)::value;
        *reinterpret_cast<float4*>(acc + (wv * 16 + r16) * DVP + i * 16 + 4 * g4) = make_float4(o[i][0], o[i][1], o[i][2], o[i][3]);
    });
    __syncthreads();
    for (int e = tid; e < 16 * DVP / 4; e += kWave * kDecodeWaves) {
        const int r = e / (DVP / 4), c = (e - r * (DVP / 4)) * 4, nr = n0 + r;
        if (nr >= rows || c >= Dv) continue;
        float mx = wm[0][r];
#pragma unroll
        for (int w = 1; w < kDecodeWaves; w++) mx = fmaxf(mx, wm[w][r]);
        float4 sum = make_float4(0, 0, 0, 0);
        float den = 0.0f;
#pragma unroll
        for (int w = 0; w < kDecodeWaves; w++) {
            const float f = exp2_hw(wm[w][r] - mx);
            const float4 x = *reinterpret_cast<const float4*>(acc + (w * 16 + r) * DVP + c);
            den = __builtin_fmaf(f, wl[w][r], den);
            sum.x = __builtin_fmaf(f, x.x, sum.x); sum.y = __builtin_fmaf(f, x.y, sum.y);
            sum.z = __builtin_fmaf(f, x.z, sum.z); sum.w = __builtin_fmaf(f, x.w, sum.w);
        }
        if (a.n_splits == 1) {
            const float inv = den > 0.0f ? a.out_scale / den : 0.0f;
            uint16_t* out = static_cast<uint16_t*>(a.out) + (static_cast<size_t>(b) * a.L + nr / rep) * a.out_row + (g * rep + nr % rep) * static_cast<size_t>(Dv) + c;
            *reinterpret_cast<uint2*>(out) = make_uint2(pack2<T>(sum.x * inv, sum.y * inv), pack2<T>(sum.z * inv, sum.w * inv));
        } else {
            const size_t idx = (head * rows + nr) * a.n_splits + split;
            if (c == 0) { a.workspace[2 * idx] = mx; a.workspace[2 * idx + 1] = den; }
            *reinterpret_cast<float4*>(a.workspace + window_pairs(a) + idx * Dv + c) = sum;
        }
    }
}

// grid (L * H, sequences), a thread per channel and turn
template <typename T>
__global__ __launch_bounds__(128) void window_merge_kernel(WindowAttnArgs a) {
    const int rep = a.H / a.G, rows = a.L * rep, S = a.n_splits, b = blockIdx.y, t = blockIdx.x / a.H, h = blockIdx.x - t * a.H;
    const size_t idx = ((static_cast<size_t>(b) * a.G + h / rep) * rows + t * rep + h % rep) * S;
    const float *ml = a.workspace + 2 * idx, *acc = a.workspace + window_pairs(a) + idx * a.Dv;
    float mx = kNone, den = 0.0f;
    for (int s = 0; s < S; s++) mx = fmaxf(mx, ml[2 * s]);
    for (int s = 0; s < S; s++) den = __builtin_fmaf(exp2_hw(ml[2 * s] - mx), ml[2 * s + 1], den);
    const float inv = den > 0.0f ? a.out_scale / den : 0.0f;
    uint16_t* out = static_cast<uint16_t*>(a.out) + (static_cast<size_t>(b) * a.L + t) * a.out_row + static_cast<size_t>(h) * a.Dv;
    for (int c = threadIdx.x; c < a.Dv; c += 128) {
        float sum = 0.0f;
        for (int s = 0; s < S; s++) sum = __builtin_fmaf(exp2_hw(ml[2 * s] - mx), acc[static_cast<size_t>(s) * a.Dv + c], sum);
        out[c] = f2lo<T>(sum * inv);
    }
}

template <typename T, int P>
static int window_decode_one(const WindowAttnArgs& a, hipStream_t st) {
    constexpr int kDecodeWaves = decode_waves(P);
    constexpr size_t bytes = 2 * static_cast<size_t>(kDecodeWaves) * kTile * (P + kVPad);
    static_assert(bytes >= sizeof(float) * kDecodeWaves * 16 * P && bytes + 2048 <= 160 * 1024, "LDS");
    if (bytes > 64 * 1024 - 2048) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&window_decode_kernel<T, P, P>),
                                                 hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(bytes));
        if (e != hipSuccess) return static_cast<int>(e);
    }
    const int row_tiles = (a.L * (a.H / a.G) + 15) / 16;
    dim3 grid(a.n_splits, a.G * row_tiles, a.B);
    hipLaunchKernelGGL((window_decode_kernel<T, P, P>), grid, dim3(kWave * kDecodeWaves), bytes, st, a);
    int err = static_cast<int>(hipGetLastError());
    if (err || a.n_splits == 1) return err;
    hipLaunchKernelGGL(window_merge_kernel<T>, dim3(a.L * a.H, a.B), dim3(128), 0, st, a);
    return static_cast<int>(hipGetLastError());
}

template <typename T>
static int window_decode_dims(const WindowAttnArgs& a, hipStream_t st) {
    const int widest = a.D > a.Dv ? a.D : a.Dv;
    return widest <= 64 ? window_decode_one<T, 64>(a, st) : widest <= 128 ? window_decode_one<T, 128>(a, st) : window_decode_one<T, 256>(a, st);
}
int launch_window_decode(const WindowAttnArgs& a, int dtype, hipStream_t st) {
    return dtype == 0 ? window_decode_dims<F16>(a, st) : window_decode_dims<BF16>(a, st);
}

// ---- any size, any dtype ---------------------------------------------------------------------------------------------------
// grid (L * H, B), one wavefront: lane == key for the scores of 64 keys, then lane == channel for the weighted sum.
template <typename T>
__global__ __launch_bounds__(kWave) void window_plain_kernel(WindowAttnArgs a) {
    extern __shared__ float sh[];
    const int D = a.D, Dv = a.Dv, lane = threadIdx.x, b = blockIdx.y, t = blockIdx.x / a.H, h = blockIdx.x - t * a.H, g = h / (a.H / a.G);
    float *q = sh, *acc = sh + D, *p = acc + Dv;
    const int pos = a.pos_dev ? *a.pos_dev : a.pos, i_row = pos + t;
    const size_t row = static_cast<size_t>(b) * a.L + t, head = static_cast<size_t>(b) * a.G + g;
    const elem_t<T>* qp = static_cast<const elem_t<T>*>(a.q) + (row * a.H + h) * D;
    for (int i = lane; i < D; i += kWave) q[i] = ld1<T>(qp + i);
    for (int i = lane; i < Dv; i += kWave) acc[i] = 0.0f;
    __syncthreads();
    auto at = [&](const void* ring, const void* fresh, int64_t fresh_row, int width, int key) {
        return fresh && key >= pos ? static_cast<const elem_t<T>*>(fresh) + (static_cast<size_t>(b) * a.L + key - pos) * fresh_row + static_cast<size_t>(g) * width
                                   : static_cast<const elem_t<T>*>(ring) + (head * a.cap + key % a.cap) * width;
    };
    const float slope2 = a.slopes ? a.slopes[h] * kLog2e : 0.0f, scale2 = a.scale * kLog2e;
    int lo = a.start ? a.start[b] : 0;
    lo = lo > i_row - a.window + 1 ? lo : i_row - a.window + 1;
    lo = lo > 0 ? lo : 0;
    float m = kNone, l = 0.0f;
    for (int k0 = lo; k0 <= i_row; k0 += kWave) {
        const int key = k0 + lane;
        float s = -INFINITY;
        if (key <= i_row) {
            const elem_t<T>* kp = at(a.k_ring, a.k_new, a.k_row, D, key);
            float d = 0.0f;
            for (int i = 0; i < D; i++) d = __builtin_fmaf(q[i], ld1<T>(kp + i), d);
            s = __builtin_fmaf(-slope2, static_cast<float>(i_row - key), d * scale2);
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
        const int cnt = i_row + 1 - k0 < kWave ? i_row + 1 - k0 : kWave;
        for (int i = lane; i < Dv; i += kWave) {
            float v = acc[i] * al;
            for (int j = 0; j < cnt; j++) v = __builtin_fmaf(p[j], ld1<T>(at(a.v_ring, a.v_new, a.v_row, Dv, k0 + j) + i), v);
            acc[i] = v;
        }
        __syncthreads();
    }
    const float inv = l > 0.0f ? a.out_scale / l : 0.0f;
    elem_t<T>* out = static_cast<elem_t<T>*>(a.out) + row * a.out_row + static_cast<size_t>(h) * Dv;
    for (int i = lane; i < Dv; i += kWave) out[i] = cv1<T>(acc[i] * inv);
}

int launch_window_plain(const WindowAttnArgs& a, int dtype, hipStream_t st) {
    dim3 grid(a.L * a.H, a.B), block(kWave);
    const size_t shared = (static_cast<size_t>(a.D) + a.Dv + kWave) * sizeof(float);
    if (dtype == 0) hipLaunchKernelGGL(window_plain_kernel<F16>, grid, block, shared, st, a);
    else if (dtype == 1) hipLaunchKernelGGL(window_plain_kernel<BF16>, grid, block, shared, st, a);
    else hipLaunchKernelGGL(window_plain_kernel<F32>, grid, block, shared, st, a);
    return static_cast<int>(hipGetLastError());
}

// ---- prompt --------------------------------------------------------------------------------------------------------------
// grid (heads, query tiles, sequences).  Four wavefronts with 32 query rows each over 64-key tiles, double-buffered in LDS; a
// wavefront passes over tiles that its rows' windows do not touch.  A key of an earlier call comes from the ring, one of this
// call from its own buffer.
constexpr int kPromptRows = 128, kPromptKeys = 64;

template <typename T, int DKP, int DVP>
__global__ __launch_bounds__(256, DKP <= 128 ? 2 : 1) void window_prefill_kernel(WindowAttnArgs a) {
    constexpr int KS = DKP / 16, VT = DVP / 32, KROW = DKP + 8, VROW = DVP + 16, KCH = DKP / 8, VCH = DVP / 8;
    constexpr int KLOADS = kPromptKeys * KCH / 256, VLOADS = kPromptKeys * VCH / 256;
    static_assert(KLOADS * 256 == kPromptKeys * KCH && VLOADS * 256 == kPromptKeys * VCH, "whole loads");
    extern __shared__ __attribute__((aligned(16))) uint16_t sm[];
    auto kt = [&](int buf) { return sm + buf * (kPromptKeys * KROW); };
    auto vt = [&](int buf) { return sm + 2 * (kPromptKeys * KROW) + buf * (kPromptKeys * VROW); };
    const int tid = threadIdx.x, lane = tid & 63, wv = tid / kWave, col = lane & 31, hi = lane >> 5;
    const int h = blockIdx.x, b = blockIdx.z, D = a.D, Dv = a.Dv, H = a.H, g = h / (H / a.G), window = a.window, past = a.pos;
    const int q_tile = blockIdx.y * kPromptRows, qw = q_tile + wv * 32;                 // first query tokens of workgroup and wavefront
    const int qi = qw + col;
    const bool valid = qi < a.L;
    const int qc = valid ? qi : a.L - 1, limit = past + qc;                             // this row's position
    const int lo = a.start ? a.start[b] : 0;
    const int q_last = q_tile + kPromptRows - 1 < a.L - 1 ? q_tile + kPromptRows - 1 : a.L - 1;
    const int wave_last = past + (qw + 31 < a.L - 1 ? qw + 31 : a.L - 1), wave_first = past + (qw < a.L - 1 ? qw : a.L - 1);
    int key_lo = past + q_tile - window + 1;
    key_lo = key_lo > lo ? key_lo : lo;
    key_lo = key_lo > 0 ? key_lo : 0;
    const int it0 = key_lo / kPromptKeys, it1 = (past + q_last) / kPromptKeys + 1, key_end = past + a.L - 1;

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
    const size_t head = static_cast<size_t>(b) * a.G + g;
    const uint16_t* kr = static_cast<const uint16_t*>(a.k_ring) + head * a.cap * D;
    const uint16_t* vr = static_cast<const uint16_t*>(a.v_ring) + head * a.cap * Dv;
    const uint16_t* kn = static_cast<const uint16_t*>(a.k_new) + static_cast<size_t>(b) * a.L * a.k_row + static_cast<size_t>(g) * D;
    const uint16_t* vn = static_cast<const uint16_t*>(a.v_new) + static_cast<size_t>(b) * a.L * a.v_row + static_cast<size_t>(g) * Dv;
    u32x4_a ks[KLOADS], vs[VLOADS];
    auto fetch = [&](int it) {
        const int key0 = it * kPromptKeys, slot0 = key0 % a.cap;
        // no branch around a load (it would be waited for at the join): keys past the end are a copy with weight zero, columns
        // past D a copy that meets zeros of q, columns past Dv a copy that is never stored
        auto row = [&](int tok, const uint16_t* ring, int width, const uint16_t* fresh, int64_t fresh_row) {
            const int key = key0 + tok < key_end ? key0 + tok : key_end;
            return key < past ? ring + static_cast<size_t>(slot0 + tok) * width : fresh + static_cast<size_t>(key - past) * fresh_row;
        };
        static_for<KLOADS>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const int u = i * 256 + tid, tok = u / KCH, c = (u % KCH) * 8;
            ks[i] = *reinterpret_cast<const u32x4_a*>(row(tok, kr, D, kn, a.k_row) + (c < D ? c : 0));
        });
        static_for<VLOADS>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const int u = i * 256 + tid, tok = u / VCH, c = (u % VCH) * 8;
            vs[i] = *reinterpret_cast<const u32x4_a*>(row(tok, vr, Dv, vn, a.v_row) + (c < Dv ? c : 0));
        });
    };
    auto put = [&](int buf) {
        static_for<KLOADS>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const int u = i * 256 + tid;
            *reinterpret_cast<u32x4_a*>(kt(buf) + (u / KCH) * KROW + (u % KCH) * 8) = ks[i];
        });
        static_for<VLOADS>([&](auto I) {
            constexpr int i = decltype(I)::value;
            const int u = i * 256 + tid;
            *reinterpret_cast<u32x4_a*>(vt(buf) + (u / VCH) * VROW + (u % VCH) * 8) = vs[i];
        });
    };
    floatx16_a o[VT];
    static_for<VT>([&](auto I) {
        constexpr int i = decltype(I)::value;
#pragma unroll
        for (int j = 0; j < 16; j++) o[i][j] = 0.0f;
    });
    float m = kNone, l = 0.0f;
    const float scale2 = a.scale * kLog2e, slope2 = a.slopes ? a.slopes[h] * kLog2e : 0.0f;

    if (it0 < it1) {
        fetch(it0);
        put(it0 & 1);
    }
    __syncthreads();
    for (int it = it0; it < it1; it++) {
        const int buf = it & 1;
        if (it + 1 < it1) fetch(it + 1);
        __builtin_amdgcn_sched_barrier(0);
        const int key0 = it * kPromptKeys;
        if (key0 <= wave_last && key0 + kPromptKeys - 1 > wave_first - window) {        // uniform over the wavefront
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
            const float base = -slope2 * static_cast<float>(limit - key0 - 4 * hi);
            const bool whole = key0 + kPromptKeys - 1 <= wave_first && key0 > wave_last - window && key0 >= lo;
#pragma unroll
            for (int u = 0; u < 2; u++)
#pragma unroll
                for (int j = 0; j < 16; j++) {
                    const int e = 32 * u + 8 * (j >> 2) + (j & 3);
                    s[u][j] = __builtin_fmaf(s[u][j], scale2, __builtin_fmaf(slope2, static_cast<float>(e), base));
                }
            if (!whole) {
#pragma unroll
                for (int u = 0; u < 2; u++)
#pragma unroll
                    for (int j = 0; j < 16; j++) {
                        const int key = key0 + 32 * u + 8 * (j >> 2) + 4 * hi + (j & 3);
                        if (key > limit || limit - key >= window || key < lo) s[u][j] = -INFINITY;
                    }
            }
#pragma unroll
            for (int u = 0; u < 2; u++)
#pragma unroll
                for (int j = 0; j < 16; j++) mx = fmaxf(mx, s[u][j]);
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
            // 16 lanes read 4 tokens x 16 channels and get them transposed: a lane ends up with its channel's tokens 4 hi .. and
            // 8 + 4 hi .. of a 16-token step, the order in which p holds them
            const int r16 = lane & 15;
            const uint16_t* vp = vt(buf) + (4 * hi + (r16 >> 2)) * VROW + ((lane >> 4) & 1) * 16 + (r16 & 3) * 4;
            static_for<VT>([&](auto I) {
                constexpr int i = decltype(I)::value;
                static_for<4>([&](auto J) {
                    constexpr int j = decltype(J)::value;
                    const u32x2_a w0 = __builtin_bit_cast(u32x2_a, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_short4*)(vp + i * 32 + j * 16 * VROW)));
                    const u32x2_a w1 = __builtin_bit_cast(u32x2_a, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_short4*)(vp + i * 32 + (j * 16 + 8) * VROW)));
                    o[i] = mma32<T>(u32x4_a{w0.x, w0.y, w1.x, w1.y}, p[j], o[i]);
                });
            });
        }
        if (it + 1 < it1) put(buf ^ 1);
        __syncthreads();
    }
    l += __shfl_xor(l, 32);
    if (!valid) return;
    const float inv = l > 0.0f ? a.out_scale / l : 0.0f;
    uint16_t* out = static_cast<uint16_t*>(a.out) + (static_cast<size_t>(b) * a.L + qi) * a.out_row + static_cast<size_t>(h) * Dv;
    static_for<VT>([&](auto I) {
        constexpr int i = decltype(I)::value;
#pragma unroll
        for (int j4 = 0; j4 < 4; j4++) {
            const int ch = i * 32 + 8 * j4 + 4 * hi;
            if (ch < Dv)
                *reinterpret_cast<uint2*>(out + ch) = make_uint2(pack2<T>(o[i][4 * j4] * inv, o[i][4 * j4 + 1] * inv),
                                                                 pack2<T>(o[i][4 * j4 + 2] * inv, o[i][4 * j4 + 3] * inv));
        }
    });
}

template <typename T, int P>
static int window_prefill_one(const WindowAttnArgs& a, hipStream_t st) {
    constexpr size_t bytes = 2 * 2 * static_cast<size_t>(kPromptKeys) * ((P + 8) + (P + 16));
    static_assert(bytes <= 160 * 1024, "LDS");
    if (bytes > 64 * 1024) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&window_prefill_kernel<T, P, P>),
                                                 hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(bytes));
        if (e != hipSuccess) return static_cast<int>(e);
    }
    dim3 grid(a.H, (a.L + kPromptRows - 1) / kPromptRows, a.B), block(256);
    hipLaunchKernelGGL((window_prefill_kernel<T, P, P>), grid, block, bytes, st, a);
    return static_cast<int>(hipGetLastError());
}

template <typename T>
static int window_prefill_dims(const WindowAttnArgs& a, hipStream_t st) {
    const int widest = a.D > a.Dv ? a.D : a.Dv;
    return widest <= 64 ? window_prefill_one<T, 64>(a, st) : widest <= 128 ? window_prefill_one<T, 128>(a, st) : window_prefill_one<T, 256>(a, st);
}
int launch_window_prefill(const WindowAttnArgs& a, int dtype, hipStream_t st) {
    return dtype == 0 ? window_prefill_dims<F16>(a, st) : window_prefill_dims<BF16>(a, st);
}

}  // namespace pq
