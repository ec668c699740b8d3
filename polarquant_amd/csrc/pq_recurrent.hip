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

__device__ __forceinline__ float softplus(float z) { return fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }

// ---- what enters the delta rule ------------------------------------------------------------------------------------------
// A wavefront per (sequence, strip of tokens, head's vector): first the G query heads, the G key heads, the H value heads,
// then the H heads' decays and step sizes.  It walks its strip with the last taps - 1 inputs of its channels in registers;
// a strip that does not begin the call reads them from the projection, the first takes them from the state.  Channel
// lane + 64 i is a lane's i-th.
template <typename T, int TAPS, int NC>
__global__ __launch_bounds__(256) void delta_prep_kernel(DeltaPrepArgs a) {
    const int lane = threadIdx.x & 63, unit = blockIdx.y * 4 + (threadIdx.x >> 6), b = blockIdx.z, G = a.G, H = a.H, L = a.L;
    if (unit >= 2 * G + 2 * H) return;
    const int t0 = blockIdx.x * a.strip, t1 = t0 + a.strip < L ? t0 + a.strip : L;
    const int first_tok = a.start ? a.start[b] - (a.pos_dev ? *a.pos_dev : a.pos) : 0;      // tokens before it are padding
    const size_t row0 = static_cast<size_t>(b) * L;
    if (unit >= 2 * G + H) {
        const int h = unit - 2 * G - H;
        const float rate = -expf(ld1<T>(static_cast<const elem_t<T>*>(a.A_log) + h));
        float bias[NC];
#pragma unroll
        for (int i = 0; i < NC; i++) {
            const int c = lane + 64 * i;
            bias[i] = ld1<T>(static_cast<const elem_t<T>*>(a.dt_bias) + static_cast<size_t>(h) * a.dim + (c < a.dim ? c : 0));
        }
        for (int t = t0; t < t1; t++) {
            const elem_t<T>* ar = static_cast<const elem_t<T>*>(a.a) + (row0 + t) * a.a_row + static_cast<size_t>(h) * a.dim;
            float* lr = a.log_g + ((row0 + t) * H + h) * a.dim;
#pragma unroll
            for (int i = 0; i < NC; i++) {
                const int c = lane + 64 * i;
                if (c < a.dim) lr[c] = rate * softplus(ld1<T>(ar + c) + bias[i]);
            }
            if (lane == 0) a.beta[(row0 + t) * H + h] = sigmoid(ld1<T>(static_cast<const elem_t<T>*>(a.b) + (row0 + t) * a.p_row + h));
        }
        return;
    }
    const bool is_q = unit < G, is_k = !is_q && unit < 2 * G;
    const int head = is_q ? unit : is_k ? unit - G : unit - 2 * G, width = is_q || is_k ? a.dim : a.vdim;
    const int channels = (is_q || is_k ? G : H) * width, all = 2 * G * a.dim + H * a.vdim;
    const int state_c = (is_q ? 0 : is_k ? G * a.dim : 2 * G * a.dim) + head * width;
    const elem_t<T>* src = static_cast<const elem_t<T>*>(is_q ? a.q : is_k ? a.k : a.v) + row0 * a.p_row + static_cast<size_t>(head) * width;
    const elem_t<T>* w = static_cast<const elem_t<T>*>(is_q ? a.w_q : is_k ? a.w_k : a.w_v) + static_cast<size_t>(head) * width * a.taps;
    elem_t<T>* dst = static_cast<elem_t<T>*>(is_q ? a.q_out : is_k ? a.k_out : a.v_out) + row0 * channels + static_cast<size_t>(head) * width;
    float* inv = is_q ? a.q_inv : a.k_inv;
    const float unit_scale = is_q ? 1.0f / sqrtf(static_cast<float>(a.dim)) : 1.0f;
    const int taps = a.taps, shift = TAPS - taps;            // a shorter filter: zero taps in front
    float cw[TAPS][NC], hist[TAPS][NC];                      // hist[TAPS - 1] is the current token
    int ch[NC];
#pragma unroll
    for (int i = 0; i < NC; i++) ch[i] = lane + 64 * i < width ? lane + 64 * i : 0;
#pragma unroll
    for (int j = 0; j < TAPS; j++) {
        const int tap = j - shift, t = t0 + j - TAPS;        // hist[j] before the first shift: input of token t0 + j - TAPS
#pragma unroll
        for (int i = 0; i < NC; i++) {
            cw[j][i] = tap >= 0 ? ld1<T>(w + ch[i] * taps + tap) : 0.0f;
            float x = 0.0f;
            if (j > 0 && tap > 0) {                          // (hist[0] is shifted out at once)
                if (t0 > 0) x = t >= first_tok && t >= 0 ? ld1<T>(src + t * a.p_row + ch[i]) : 0.0f;
                else x = a.state_in[(static_cast<size_t>(b) * (taps - 1) + tap - 1) * all + state_c + ch[i]];
            }
            hist[j][i] = x;
        }
    }
    for (int t = t0; t < t1; t++) {
        const bool real = t >= first_tok;
        float ss = 0.0f, y[NC];
#pragma unroll
        for (int i = 0; i < NC; i++) {
#pragma unroll
            for (int j = 0; j + 1 < TAPS; j++) hist[j][i] = hist[j + 1][i];
            hist[TAPS - 1][i] = real ? ld1<T>(src + t * a.p_row + ch[i]) : 0.0f;
            float s = 0.0f;
#pragma unroll
            for (int j = 0; j < TAPS; j++) s = __builtin_fmaf(cw[j][i], hist[j][i], s);
            const elem_t<T> r = cv1<T>(s / (1.0f + expf(-s)));
            y[i] = ld1<T>(&r);
            if (lane + 64 * i < width) {
                dst[static_cast<size_t>(t) * channels + ch[i]] = r;
                ss = __builtin_fmaf(y[i], y[i], ss);
            }
        }
        if (is_q || is_k) {
            ss = wave_sum(ss);
            if (lane == 0) inv[(row0 + t) * G + head] = unit_scale / sqrtf(ss + 1e-6f);
        }
    }
    if (t1 == L) {
#pragma unroll
        for (int j = 1; j < TAPS; j++) {
            const int row = j - shift - 1;
            if (row < 0) continue;
#pragma unroll
            for (int i = 0; i < NC; i++)
                if (lane + 64 * i < width) a.state_out[(static_cast<size_t>(b) * (taps - 1) + row) * all + state_c + ch[i]] = hist[j][i];
        }
    }
}

int launch_delta_prep(const DeltaPrepArgs& args, int dtype, hipStream_t st) {
    DeltaPrepArgs a = args;
    a.strip = 32;
    const int widest = a.dim > a.vdim ? a.dim : a.vdim;
    dim3 grid(static_cast<unsigned>((a.L + a.strip - 1) / a.strip), static_cast<unsigned>((2 * a.G + 2 * a.H + 3) / 4), static_cast<unsigned>(a.B)), block(256);
#define PQ_DP(T, TP, N) hipLaunchKernelGGL((delta_prep_kernel<T, TP, N>), grid, block, 0, st, a)
#define PQ_DP_N(T, TP) do { if (widest <= 64) PQ_DP(T, TP, 1); else if (widest <= 128) PQ_DP(T, TP, 2); else PQ_DP(T, TP, 4); } while (0)
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
                S[i] *= expf(d.g[i]);
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
            const float mn = fmaxf(d.y + m, d.x), fa = expf(d.y + m - mn), ib = expf(d.x - mn) * (value ? d.v : 1.0f);
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
            if (part == 0 && col == a.vdim) a.den[row * H + h] = fmaxf(fabsf(e), expf(-m)) + 1e-6f;
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
// A wavefront per (token, head), 4 channels per lane and turn.
template <typename T, int V>
__global__ __launch_bounds__(256) void head_norm_gate_kernel(HeadNormGateArgs a) {
    const int64_t n = static_cast<int64_t>(blockIdx.x) * 4 + (threadIdx.x >> 6);
    if (n >= a.rows * a.H) return;
    const int lane = threadIdx.x & 63, h = static_cast<int>(n % a.H);
    const int64_t row = n / a.H;
    const float* o = a.o + n * a.vdim;
    const float div = a.den ? 1.0f / a.den[n] : 1.0f;
    float ss = 0.0f, x[V];
    for (int c = lane * V; c < a.vdim; c += 64 * V) {
        ldv<F32, V>(o, c, x);
#pragma unroll
        for (int j = 0; j < V; j++) {
            x[j] *= div;
            ss = __builtin_fmaf(x[j], x[j], ss);
        }
    }
    ss = wave_sum(ss);
    const float r = div * a.out_scale / sqrtf(ss / static_cast<float>(a.vdim) + a.eps);
    const elem_t<T>* gate = static_cast<const elem_t<T>*>(a.gate) + row * a.gate_row + static_cast<size_t>(h) * a.vdim;
    const elem_t<T>* w = static_cast<const elem_t<T>*>(a.w) + static_cast<size_t>(h) * a.w_head;
    elem_t<T>* out = static_cast<elem_t<T>*>(a.out) + row * a.out_row + static_cast<size_t>(h) * a.vdim;
    for (int c = lane * V; c < a.vdim; c += 64 * V) {
        float g[V], wv[V];
        ldv<F32, V>(o, c, x);
        ldv<T, V>(gate, c, g);
        ldv<T, V>(w, c, wv);
#pragma unroll
        for (int j = 0; j < V; j++) x[j] = x[j] * r * wv[j] * sigmoid(g[j]);
        stv<T, V>(out, c, x);
    }
}

int launch_head_norm_gate(const HeadNormGateArgs& a, int dtype, hipStream_t st) {
    dim3 grid(static_cast<unsigned>((a.rows * a.H + 3) / 4)), block(256);
    const size_t align = dtype == 2 ? 16 : 8;
    auto ok = [&](const void* p, size_t n) { return reinterpret_cast<uintptr_t>(p) % n == 0; };
    const bool v4 = a.vdim % 4 == 0 && a.gate_row % 4 == 0 && a.out_row % 4 == 0 && ok(a.gate, align) && ok(a.out, align) && ok(a.w, align) && ok(a.o, 16);
#define PQ_HN(T) do { if (v4) hipLaunchKernelGGL((head_norm_gate_kernel<T, 4>), grid, block, 0, st, a); \
                      else hipLaunchKernelGGL((head_norm_gate_kernel<T, 1>), grid, block, 0, st, a); } while (0)
    if (dtype == 0) PQ_HN(F16); else if (dtype == 1) PQ_HN(BF16); else PQ_HN(F32);
#undef PQ_HN
    return static_cast<int>(hipGetLastError());
}

}  // namespace pq
