// Mixers with a matrix-valued state per head: the gated delta rule and the matrix memory.
//
//   delta_prep_kernel      short convolutions + silu of q, k, v, lengths of the heads' vectors, log decays, step sizes
//   memory_gates_kernel    capped input and forget gates of a matrix memory, as logarithms
//   scan_kernel            either recurrence, token by token, any size and dtype
//   head_norm_gate_kernel  RMS norm per head of what was read out, its weight, the output gate
//
// State and everything that enters a recurrence are float32; q, k, v come in the model's dtype.
#include "pq_elem.h"
#include "pq_recurrent_internal.h"

namespace pq {

// (one instruction each, exact to about a unit in the last place)
__device__ __forceinline__ float exp_fast(float x) { return __builtin_amdgcn_exp2f(x * 1.4426950408889634f); }
__device__ __forceinline__ float sigmoid(float z) { return __builtin_amdgcn_rcpf(1.0f + exp_fast(-z)); }
// max(z, 0) + log(1 + e), e = e^-|z|: for small e by its series, 1 + e would lose it
__device__ __forceinline__ float softplus(float z) {
    const float e = exp_fast(-fabsf(z));
    const float series = e * __builtin_fmaf(e, __builtin_fmaf(e, __builtin_fmaf(e, -0.25f, 0.33333334f), -0.5f), 1.0f);
    return fmaxf(z, 0.0f) + (e < 0.01f ? series : __builtin_amdgcn_logf(1.0f + e) * 0.6931471805599453f);
}

// V (1 or 2) consecutive elements at p
template <typename T, int V> __device__ __forceinline__ void ldvec(const elem_t<T>* p, float (&o)[V]) {
    if constexpr (V == 1) {
        o[0] = ld1<T>(p);
    } else if constexpr (__is_same(T, F32)) {
        const float2 v = *reinterpret_cast<const float2*>(p);
        o[0] = v.x; o[1] = v.y;
    } else {
        const uint32_t v = *reinterpret_cast<const uint32_t*>(p);
        o[0] = lo2f<T>(static_cast<uint16_t>(v & 0xffffu)); o[1] = lo2f<T>(static_cast<uint16_t>(v >> 16));
    }
}
template <typename T, int V> __device__ __forceinline__ void stvec(elem_t<T>* p, const float (&o)[V]) {
    if constexpr (V == 1) *p = cv1<T>(o[0]);
    else if constexpr (__is_same(T, F32)) *reinterpret_cast<float2*>(p) = make_float2(o[0], o[1]);
    else *reinterpret_cast<uint32_t*>(p) = static_cast<uint32_t>(f2lo<T>(o[0])) | (static_cast<uint32_t>(f2lo<T>(o[1])) << 16);
}

// ---- what enters the delta rule ------------------------------------------------------------------------------------------
// A wavefront per (sequence, strip of tokens, head's vector): first the G query heads, the G key heads, the H value heads,
// then the H heads' decays and step sizes.  It walks its strip with the last taps - 1 inputs of its channels in registers and
// the next four tokens' in flight; a strip that does not begin the call reads those before it from the projection, the first
// takes them from the state.  A lane's i-th piece is V channels from (lane + 64 i) V on.
constexpr int kPrepGroup = 4;

template <typename T, int TAPS, int NC, int V>
__global__ __launch_bounds__(256) void delta_prep_kernel(DeltaPrepArgs a) {
    const int lane = threadIdx.x & 63, unit = blockIdx.y * 4 + (threadIdx.x >> 6), b = blockIdx.z, G = a.G, H = a.H, L = a.L;
    if (unit >= 2 * G + 2 * H) return;
    const int t0 = blockIdx.x * a.strip, t1 = t0 + a.strip < L ? t0 + a.strip : L;
    const int first_tok = a.start ? a.start[b] - (a.pos_dev ? *a.pos_dev : a.pos) : 0;      // tokens before it are padding
    const size_t row0 = static_cast<size_t>(b) * L;
    const bool is_q = unit < G, is_k = !is_q && unit < 2 * G, is_g = unit >= 2 * G + H;
    const int head = is_q ? unit : is_k ? unit - G : is_g ? unit - 2 * G - H : unit - 2 * G, width = is_q || is_k || is_g ? a.dim : a.vdim;
    bool own[NC];
    int ch[NC];
#pragma unroll
    for (int i = 0; i < NC; i++) {
        own[i] = (lane + 64 * i) * V < width;
        ch[i] = own[i] ? (lane + 64 * i) * V : 0;
    }
    const int64_t src_row = is_g ? a.a_row : a.p_row;
    const elem_t<T>* src = static_cast<const elem_t<T>*>(is_q ? a.q : is_k ? a.k : is_g ? a.a : a.v) + row0 * src_row + static_cast<size_t>(head) * width;
    float x[kPrepGroup][NC][V];
    auto fetch = [&](int t) {
#pragma unroll
        for (int d = 0; d < kPrepGroup; d++) {
            const elem_t<T>* r = src + static_cast<size_t>(t + d < t1 ? t + d : t1 - 1) * src_row;
#pragma unroll
            for (int i = 0; i < NC; i++) ldvec<T, V>(r + ch[i], x[d][i]);
        }
    };
    fetch(t0);
    if (is_g) {
        const float rate = -expf(ld1<T>(static_cast<const elem_t<T>*>(a.A_log) + head));
        float bias[NC][V], now[kPrepGroup][NC][V];
#pragma unroll
        for (int i = 0; i < NC; i++) ldvec<T, V>(static_cast<const elem_t<T>*>(a.dt_bias) + static_cast<size_t>(head) * width + ch[i], bias[i]);
        for (int t = t0 + lane; t < t1; t += 64)
            a.beta[(row0 + t) * H + head] = sigmoid(ld1<T>(static_cast<const elem_t<T>*>(a.b) + (row0 + t) * a.p_row + head));
        for (int t = t0; t < t1; t += kPrepGroup) {
#pragma unroll
            for (int d = 0; d < kPrepGroup; d++)
#pragma unroll
                for (int i = 0; i < NC; i++)
#pragma unroll
                    for (int j = 0; j < V; j++) now[d][i][j] = x[d][i][j];
            fetch(t + kPrepGroup < t1 ? t + kPrepGroup : t);
#pragma unroll
            for (int d = 0; d < kPrepGroup; d++) {
                if (t + d >= t1) break;
                float* lr = a.log_g + ((row0 + t + d) * H + head) * width;
#pragma unroll
                for (int i = 0; i < NC; i++) {
                    float y[V];
#pragma unroll
                    for (int j = 0; j < V; j++) y[j] = rate * softplus(now[d][i][j] + bias[i][j]);
                    if (own[i]) stvec<F32, V>(lr + ch[i], y);
                }
            }
        }
        return;
    }
    const int channels = (is_q || is_k ? G : H) * width, all = 2 * G * a.dim + H * a.vdim;
    const int state_c = (is_q ? 0 : is_k ? G * a.dim : 2 * G * a.dim) + head * width;
    const elem_t<T>* w = static_cast<const elem_t<T>*>(is_q ? a.w_q : is_k ? a.w_k : a.w_v) + static_cast<size_t>(head) * width * a.taps;
    elem_t<T>* dst = static_cast<elem_t<T>*>(is_q ? a.q_out : is_k ? a.k_out : a.v_out) + row0 * channels + static_cast<size_t>(head) * width;
    float* inv = is_q ? a.q_inv : a.k_inv;
    const float unit_scale = is_q ? 1.0f / sqrtf(static_cast<float>(a.dim)) : 1.0f;
    const int taps = a.taps, shift = TAPS - taps;            // a shorter filter: zero taps in front
    float cw[TAPS][NC][V], hist[TAPS][NC][V];                // hist[TAPS - 1] is the current token
#pragma unroll
    for (int j = 0; j < TAPS; j++) {
        const int tap = j - shift, t = t0 + j - TAPS;        // hist[j] before the first shift: input of token t0 + j - TAPS
#pragma unroll
        for (int i = 0; i < NC; i++) {
#pragma unroll
            for (int k = 0; k < V; k++) {
                cw[j][i][k] = tap >= 0 ? ld1<T>(w + (ch[i] + k) * taps + tap) : 0.0f;
                float y = 0.0f;
                if (j > 0 && tap > 0) {                      // (hist[0] is shifted out at once)
                    if (t0 > 0) y = t >= first_tok && t >= 0 ? ld1<T>(src + t * src_row + ch[i] + k) : 0.0f;
                    else y = a.state_in[(static_cast<size_t>(b) * (taps - 1) + tap - 1) * all + state_c + ch[i] + k];
                }
                hist[j][i][k] = y;
            }
        }
    }
    for (int t = t0; t < t1; t += kPrepGroup) {
        float now[kPrepGroup][NC][V];
#pragma unroll
        for (int d = 0; d < kPrepGroup; d++)
#pragma unroll
            for (int i = 0; i < NC; i++)
#pragma unroll
                for (int k = 0; k < V; k++) now[d][i][k] = x[d][i][k];
        fetch(t + kPrepGroup < t1 ? t + kPrepGroup : t);
#pragma unroll
        for (int d = 0; d < kPrepGroup; d++) {
            if (t + d >= t1) break;                          // uniform
            const bool real = t + d >= first_tok;
            float ss = 0.0f;
#pragma unroll
            for (int i = 0; i < NC; i++) {
                float y[V];
#pragma unroll
                for (int k = 0; k < V; k++) {
#pragma unroll
                    for (int j = 0; j + 1 < TAPS; j++) hist[j][i][k] = hist[j + 1][i][k];
                    hist[TAPS - 1][i][k] = real ? now[d][i][k] : 0.0f;
                    float s = 0.0f;
#pragma unroll
                    for (int j = 0; j < TAPS; j++) s = __builtin_fmaf(cw[j][i][k], hist[j][i][k], s);
                    const elem_t<T> r = cv1<T>(s * sigmoid(s));      // (lengths are those of what is stored)
                    y[k] = ld1<T>(&r);
                    ss = own[i] ? __builtin_fmaf(y[k], y[k], ss) : ss;
                }
                if (own[i]) stvec<T, V>(dst + static_cast<size_t>(t + d) * channels + ch[i], y);
            }
            if (is_q || is_k) {
                ss = wave_sum(ss);
                if (lane == 0) inv[(row0 + t + d) * G + head] = unit_scale / sqrtf(ss + 1e-6f);
            }
        }
    }
    if (t1 == L) {
#pragma unroll
        for (int j = 1; j < TAPS; j++) {
            const int row = j - shift - 1;
            if (row < 0) continue;
#pragma unroll
            for (int i = 0; i < NC; i++)
                if (own[i]) stvec<F32, V>(a.state_out + (static_cast<size_t>(b) * (taps - 1) + row) * all + state_c + ch[i], hist[j][i]);
        }
    }
}

int launch_delta_prep(const DeltaPrepArgs& args, int dtype, hipStream_t st) {
    DeltaPrepArgs a = args;
    a.strip = 32;
    const int widest = a.dim > a.vdim ? a.dim : a.vdim, least = a.dim < a.vdim ? a.dim : a.vdim;
    // two channels at a time where heads are wide and all rows begin at even channels
    const size_t align = dtype == 2 ? 8 : 4;
    auto ok = [&](const void* p) { return reinterpret_cast<uintptr_t>(p) % align == 0; };
    auto ok8 = [&](const void* p) { return reinterpret_cast<uintptr_t>(p) % 8 == 0; };
    const bool v2 = least >= 96 && a.dim % 2 == 0 && a.vdim % 2 == 0 && a.p_row % 2 == 0 && a.a_row % 2 == 0 && ok(a.q) && ok(a.k) && ok(a.v) && ok(a.a) &&
                    ok(a.dt_bias) && ok(a.q_out) && ok(a.k_out) && ok(a.v_out) && ok8(a.log_g) && ok8(a.state_out);
    const int per = (widest + 64 * (v2 ? 2 : 1) - 1) / (64 * (v2 ? 2 : 1));
    dim3 grid(static_cast<unsigned>((a.L + a.strip - 1) / a.strip), static_cast<unsigned>((2 * a.G + 2 * a.H + 3) / 4), static_cast<unsigned>(a.B)), block(256);
#define PQ_DP(T, TP, N, VV) hipLaunchKernelGGL((delta_prep_kernel<T, TP, N, VV>), grid, block, 0, st, a)
#define PQ_DP_N(T, TP)                                                                                               \
    do {                                                                                                             \
        if (v2) { if (per <= 1) PQ_DP(T, TP, 1, 2); else PQ_DP(T, TP, 2, 2); }                                       \
        else if (per <= 1) PQ_DP(T, TP, 1, 1); else if (per <= 2) PQ_DP(T, TP, 2, 1); else PQ_DP(T, TP, 4, 1);       \
    } while (0)
#define PQ_DP_T(T) do { if (a.taps <= 4) PQ_DP_N(T, 4); else PQ_DP_N(T, 16); } while (0)
    if (dtype == 0) PQ_DP_T(F16); else if (dtype == 1) PQ_DP_T(BF16); else PQ_DP_T(F32);
#undef PQ_DP_T
#undef PQ_DP_N
#undef PQ_DP
    return static_cast<int>(hipGetLastError());
}

// ---- gates of a matrix memory ------------------------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void memory_gates_kernel(MemoryGateArgs a) {
    const int64_t n = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
    if (n >= a.rows * a.H) return;
    const int64_t row = n / a.H;
    const int h = static_cast<int>(n - row * a.H);
    const float i = ld1<T>(static_cast<const elem_t<T>*>(a.i) + row * a.p_row + h) + ld1<T>(static_cast<const elem_t<T>*>(a.b_i) + h);
    const float f = ld1<T>(static_cast<const elem_t<T>*>(a.f) + row * a.p_row + h) + ld1<T>(static_cast<const elem_t<T>*>(a.b_f) + h);
    a.log_i[n] = a.cap * tanhf(i / a.cap);
    a.log_f[n] = -softplus(-(a.cap * tanhf(f / a.cap)));
}

int launch_memory_gates(const MemoryGateArgs& a, int dtype, hipStream_t st) {
    dim3 grid(static_cast<unsigned>((a.rows * a.H + 255) / 256)), block(256);
    if (dtype == 0) hipLaunchKernelGGL(memory_gates_kernel<F16>, grid, block, 0, st, a);
    else if (dtype == 1) hipLaunchKernelGGL(memory_gates_kernel<BF16>, grid, block, 0, st, a);
    else hipLaunchKernelGGL(memory_gates_kernel<F32>, grid, block, 0, st, a);
    return static_cast<int>(hipGetLastError());
}

// ---- token by token ------------------------------------------------------------------------------------------------------
// grid (column blocks of 16, heads, sequences).  16 lanes hold a column of the state, RPL rows each; a wavefront four columns.
// Columns are independent.  Delta rule: S' = g S, d = S'^T k, e = S'^T q, u = beta (v - d), S = S' + k u, o = e + (q.k) u, so
// that one reduction over the 16 lanes gives d, e and q.k.  Matrix memory: S = a S + b k v, o = S^T q, the normalizer being one
// more column whose v is 1.
__device__ __forceinline__ float row16_sum(float v) {
    v += __uint_as_float(row_rotate<8>(__float_as_uint(v)));
    v += __uint_as_float(row_rotate<4>(__float_as_uint(v)));
    v += __uint_as_float(row_rotate<2>(__float_as_uint(v)));
    v += __uint_as_float(row_rotate<1>(__float_as_uint(v)));
    return v;
}

template <typename T, bool DELTA, int RPL>
__global__ __launch_bounds__(256) void scan_kernel(ScanArgs a) {
    const int lane = threadIdx.x & 63, part = lane & 15, h = blockIdx.y, b = blockIdx.z, H = a.H, L = a.L, dim = a.dim;
    const int columns = a.vdim + (DELTA ? 0 : 1), col = blockIdx.x * 16 + (threadIdx.x >> 4), r0 = part * RPL;
    const bool live = col < columns, value = col < a.vdim;
    const int hk = h / (H / a.G);
    int first = a.start ? a.start[b] - (a.pos_dev ? *a.pos_dev : a.pos) : 0;
    first = first < 0 ? 0 : first > L ? L : first;
    float S[RPL];
    float* sp = a.state + ((static_cast<size_t>(b) * H + h) * columns + (live ? col : 0)) * dim;
#pragma unroll
    for (int i = 0; i < RPL; i++) S[i] = r0 + i < dim ? sp[r0 + i] : 0.0f;
    float* mp = DELTA ? nullptr : a.m + (static_cast<size_t>(b) * H + h) * gridDim.x + blockIdx.x;
    float m = DELTA ? 0.0f : *mp;
    if (!DELTA) __syncthreads();                     // (read by all before one writes it)
    const size_t row0 = static_cast<size_t>(b) * L;
    for (int t = 0; t < first; t++) {
        if (part == 0 && value) a.o[((row0 + t) * H + h) * a.vdim + col] = 0.0f;
        if (part == 0 && !DELTA && col == a.vdim) a.den[(row0 + t) * H + h] = 1.0f;
    }
    struct Tok { float q[RPL], k[RPL], g[RPL], v, x, y, z; };
    auto load = [&](int t, Tok& d) {
        const size_t row = row0 + (t < L ? t : L - 1);
        const elem_t<T>* qp = static_cast<const elem_t<T>*>(a.q) + row * a.q_row + static_cast<size_t>(hk) * dim;
        const elem_t<T>* kp = static_cast<const elem_t<T>*>(a.k) + row * a.k_row + static_cast<size_t>(hk) * dim;
        const float* gp = DELTA ? a.log_g + (row * H + h) * dim : nullptr;
#pragma unroll
        for (int i = 0; i < RPL; i++) {
            const int r = r0 + i < dim ? r0 + i : 0;
            d.q[i] = ld1<T>(qp + r);
            d.k[i] = ld1<T>(kp + r);
            if (DELTA) d.g[i] = gp[r];
        }
        d.v = ld1<T>(static_cast<const elem_t<T>*>(a.v) + row * a.v_row + static_cast<size_t>(h) * a.vdim + (value ? col : 0));
        if (DELTA) {
            d.x = a.q_inv[row * a.G + hk];
            d.y = a.k_inv[row * a.G + hk];
            d.z = a.beta[row * H + h];
        } else {
            d.x = a.log_i[row * H + h];
            d.y = a.log_f[row * H + h];
        }
    };
    auto step = [&](int t, Tok& d) {
        const size_t row = row0 + t;
        if constexpr (DELTA) {
            float e0 = 0.0f, e1 = 0.0f, e2 = 0.0f;
#pragma unroll
            for (int i = 0; i < RPL; i++) {
                const bool in = r0 + i < dim;
                const float k = in ? d.k[i] * d.y : 0.0f, q = in ? d.q[i] * d.x : 0.0f;
                S[i] *= exp_fast(d.g[i]);
                e0 = __builtin_fmaf(S[i], k, e0);
                e1 = __builtin_fmaf(S[i], q, e1);
                e2 = __builtin_fmaf(k, q, e2);
                d.k[i] = k;
            }
            e0 = row16_sum(e0);
            e1 = row16_sum(e1);
            e2 = row16_sum(e2);
            const float u = d.z * (d.v - e0);
#pragma unroll
            for (int i = 0; i < RPL; i++) S[i] = __builtin_fmaf(d.k[i], u, S[i]);
            if (part == 0 && live) a.o[(row * H + h) * a.vdim + col] = __builtin_fmaf(e2, u, e1);
        } else {
            const float mn = fmaxf(d.y + m, d.x), fa = exp_fast(d.y + m - mn), ib = exp_fast(d.x - mn) * (value ? d.v : 1.0f);
            m = mn;
            float e = 0.0f;
#pragma unroll
            for (int i = 0; i < RPL; i++) {
                const bool in = r0 + i < dim;
                S[i] = __builtin_fmaf(in ? d.k[i] : 0.0f, ib, fa * S[i]);
                e = __builtin_fmaf(S[i], in ? d.q[i] : 0.0f, e);
            }
            e = row16_sum(e) * a.q_scale;
            if (part == 0 && value) a.o[(row * H + h) * a.vdim + col] = e;
            if (part == 0 && col == a.vdim) a.den[row * H + h] = fmaxf(fabsf(e), exp_fast(-m)) + 1e-6f;
        }
    };
    // the next token's operands are in flight while one is worked on
    Tok t0, t1;
    if (first < L) load(first, t0);
    int t = first;
    for (; t + 1 < L; t += 2) {
        load(t + 1, t1);
        step(t, t0);
        load(t + 2, t0);
        step(t + 1, t1);
    }
    if (t < L) step(t, t0);
    if (live) {
#pragma unroll
        for (int i = 0; i < RPL; i++)
            if (r0 + i < dim) sp[r0 + i] = S[i];
    }
    if (!DELTA && threadIdx.x == 0) *mp = m;
}

template <bool DELTA>
static int launch_scan(const ScanArgs& a, int dtype, hipStream_t st) {
    const int columns = a.vdim + (DELTA ? 0 : 1);
    dim3 grid(static_cast<unsigned>((columns + 15) / 16), static_cast<unsigned>(a.H), static_cast<unsigned>(a.B)), block(256);
#define PQ_S(T)                                                                                                      \
    do {                                                                                                             \
        if (a.dim <= 64) hipLaunchKernelGGL((scan_kernel<T, DELTA, 4>), grid, block, 0, st, a);                      \
        else if (a.dim <= 128) hipLaunchKernelGGL((scan_kernel<T, DELTA, 8>), grid, block, 0, st, a);                \
        else hipLaunchKernelGGL((scan_kernel<T, DELTA, 16>), grid, block, 0, st, a);                                 \
    } while (0)
    if (dtype == 0) PQ_S(F16); else if (dtype == 1) PQ_S(BF16); else PQ_S(F32);
#undef PQ_S
    return static_cast<int>(hipGetLastError());
}
int launch_delta_scan(const ScanArgs& a, int dtype, hipStream_t st) { return launch_scan<true>(a, dtype, st); }
int launch_memory_scan(const ScanArgs& a, int dtype, hipStream_t st) { return launch_scan<false>(a, dtype, st); }

// ---- read-out --------------------------------------------------------------------------------------------------------------
// LPH lanes per (token, head), V channels per lane and turn.
template <typename T, int V, int LPH>
__global__ __launch_bounds__(256) void head_norm_gate_kernel(HeadNormGateArgs a) {
    const int64_t n = static_cast<int64_t>(blockIdx.x) * (256 / LPH) + threadIdx.x / LPH;
    if (n >= a.rows * a.H) return;
    const int lane = threadIdx.x % LPH, h = static_cast<int>(n % a.H);
    const int64_t row = n / a.H;
    const float* o = a.o + n * a.vdim;
    const float div = a.den ? 1.0f / a.den[n] : 1.0f;
    const elem_t<T>* gate = static_cast<const elem_t<T>*>(a.gate) + row * a.gate_row + static_cast<size_t>(h) * a.vdim;
    const elem_t<T>* w = static_cast<const elem_t<T>*>(a.w) + static_cast<size_t>(h) * a.w_head;
    elem_t<T>* out = static_cast<elem_t<T>*>(a.out) + row * a.out_row + static_cast<size_t>(h) * a.vdim;
    const bool once = a.vdim <= LPH * V;                     // every lane has one piece, which stays in its registers
    const int c0 = lane * V;
    float x0[V], g0[V], w0[V];
#pragma unroll
    for (int j = 0; j < V; j++) x0[j] = g0[j] = w0[j] = 0.0f;
    if (c0 < a.vdim) {
        ldv<F32, V>(o, c0, x0);
        ldv<T, V>(gate, c0, g0);
        ldv<T, V>(w, c0, w0);
    }
    float ss = 0.0f;
#pragma unroll
    for (int j = 0; j < V; j++) {
        const float x = x0[j] * div;
        ss = __builtin_fmaf(x, x, ss);
    }
    if (!once) {
        for (int c = c0 + LPH * V; c < a.vdim; c += LPH * V) {
            float x[V];
            ldv<F32, V>(o, c, x);
#pragma unroll
            for (int j = 0; j < V; j++) {
                x[j] *= div;
                ss = __builtin_fmaf(x[j], x[j], ss);
            }
        }
    }
    ss = row16_sum(ss);
    if (LPH >= 32) ss += __shfl_xor(ss, 16);
    if (LPH >= 64) ss += __shfl_xor(ss, 32);
    const float r = div * a.out_scale / sqrtf(ss / static_cast<float>(a.vdim) + a.eps);
    if (c0 < a.vdim) {
#pragma unroll
        for (int j = 0; j < V; j++) x0[j] = x0[j] * r * w0[j] * sigmoid(g0[j]);
        stv<T, V>(out, c0, x0);
    }
    if (!once) {
        for (int c = c0 + LPH * V; c < a.vdim; c += LPH * V) {
            float x[V], g[V], wv[V];
            ldv<F32, V>(o, c, x);
            ldv<T, V>(gate, c, g);
            ldv<T, V>(w, c, wv);
#pragma unroll
            for (int j = 0; j < V; j++) x[j] = x[j] * r * wv[j] * sigmoid(g[j]);
            stv<T, V>(out, c, x);
        }
    }
}

int launch_head_norm_gate(const HeadNormGateArgs& a, int dtype, hipStream_t st) {
    const size_t align = dtype == 2 ? 16 : 8;
    auto ok = [&](const void* p, size_t n) { return reinterpret_cast<uintptr_t>(p) % n == 0; };
    const bool v4 = a.vdim % 4 == 0 && a.gate_row % 4 == 0 && a.out_row % 4 == 0 && ok(a.gate, align) && ok(a.out, align) && ok(a.w, align) && ok(a.o, 16);
    const int pieces = v4 ? a.vdim / 4 : a.vdim, lph = pieces <= 16 ? 16 : pieces <= 32 ? 32 : 64;
    dim3 grid(static_cast<unsigned>((a.rows * a.H + 256 / lph - 1) / (256 / lph))), block(256);
#define PQ_HN(T, V)                                                                                                  \
    do {                                                                                                             \
        if (lph == 16) hipLaunchKernelGGL((head_norm_gate_kernel<T, V, 16>), grid, block, 0, st, a);                 \
        else if (lph == 32) hipLaunchKernelGGL((head_norm_gate_kernel<T, V, 32>), grid, block, 0, st, a);            \
        else hipLaunchKernelGGL((head_norm_gate_kernel<T, V, 64>), grid, block, 0, st, a);                           \
    } while (0)
#define PQ_HN_T(T) do { if (v4) PQ_HN(T, 4); else PQ_HN(T, 1); } while (0)
    if (dtype == 0) PQ_HN_T(F16); else if (dtype == 1) PQ_HN_T(BF16); else PQ_HN_T(F32);
#undef PQ_HN_T
#undef PQ_HN
    return static_cast<int>(hipGetLastError());
}

}  // namespace pq
