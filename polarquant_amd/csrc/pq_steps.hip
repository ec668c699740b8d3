// The steps between a layer's mixers and matrix products, whatever the mixers are.
//
//   norm_conv_kernel    residual add of a normed sublayer output, grouped RMS norm of the sum, causal convolution over
//                       time with its per-sequence state: everything between two sublayers in one launch
//   stream_add_kernel   residual stream + sublayer output + another stream + one vector
//   embed_rows_kernel   scaled embedding rows as the float32 stream
//   relu_sq_kernel      square of relu
//   gelu_mul_kernel     gelu (tanh form) of one product times another
//   softcap_kernel      scale and soft cap of logits
//   head_linear_kernel  per-head (or plain) matrix product for sizes and dtypes the matrix-core kernels do not take
//
// All of this is fp32 arithmetic on whatever the operands' dtype is; results are rounded to it once.
#include "pq_elem.h"
#include "pq_steps_internal.h"

namespace pq {

// ---- residual add + grouped norms + causal convolution ----------------------------------------------------------------
// A workgroup walks a strip of consecutive tokens of one sequence; a thread owns the same NC pieces of V channels for all
// of them, so that the last taps - 1 norms (the convolution's inputs) stay in its registers.  A strip that does not begin
// the call recomputes the norms of the taps - 1 tokens before it (from x_in and y, which nobody overwrites in a call of
// several strips); the first strip takes them from the state.  TAPS is the register depth: shorter filters are padded
// with zero taps in front.
//
// Sums over a group: where every wavefront's piece lies in one group (`wave_groups`), wavefront sums go through LDS once;
// otherwise every piece's sum does, and wavefronts add them up group by group.
template <typename T, int TAPS, int V, int NC>
__global__ __launch_bounds__(512) void norm_conv_kernel(NormConvArgs a) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int tid = threadIdx.x, nthr = blockDim.x, nw = nthr / kWave, wv = tid / kWave, lane = tid & (kWave - 1);
    const int b = blockIdx.y, W = a.W, L = a.L, taps = a.taps;
    const int t0 = blockIdx.x * a.strip, t1 = t0 + a.strip < L ? t0 + a.strip : L;
    const int gs = W / a.groups, pieces = W / V, ppg = gs / V;       // pieces, pieces per group
    const bool one_group = a.groups == 1, wave_groups = one_group || (ppg % kWave) == 0;
    const int spg = one_group ? nw : ppg / kWave;                    // wavefront sums per group
    const float inv_gs = 1.0f / static_cast<float>(gs);
    const int begin = (TAPS > 0 && t0 > 0) ? t0 - (taps - 1) : t0;   // strips are longer than the filter
    int phase = 0;

    bool own[NC];
    uint32_t ch[NC];
#pragma unroll
    for (int k = 0; k < NC; k++) {
        const int q = k * nthr + tid;
        own[k] = q < pieces;
        ch[k] = (own[k] ? q : 0) * V;
    }
    // rows of this sequence; without y something that exists is loaded in its place and not used
    const float* xr = a.x_in + static_cast<size_t>(b) * L * W;
    const elem_t<T>* yr = a.y ? static_cast<const elem_t<T>*>(a.y) + static_cast<size_t>(b) * L * W : static_cast<const elem_t<T>*>(a.w_pre);
    const size_t y_stride = a.y ? W : 0;
    // tokens in flight ahead of the one being worked on: what a compute unit holds of them is what keeps HBM busy
    constexpr int AHEAD = NC == 1 ? 3 : 1;
    float xc[NC][V], yc[NC][V], xn[AHEAD][NC][V], yn[AHEAD][NC][V];
    auto fetch = [&](int t, float (&x)[NC][V], float (&y)[NC][V]) {
        const float* xp = xr + static_cast<size_t>(t) * W;
        const elem_t<T>* yp = yr + t * y_stride;
#pragma unroll
        for (int k = 0; k < NC; k++) {
            ldv<F32, V>(xp, ch[k], x[k]);
            ldv<T, V>(yp, ch[k], y[k]);
        }
    };
    fetch(begin, xc, yc);
#pragma unroll
    for (int d = 0; d < AHEAD; d++) fetch(begin + d + 1 < t1 ? begin + d + 1 : begin, xn[d], yn[d]);

    // 1 / sqrt(mean square of the group + eps) for each of this thread's pieces
    auto group_scale = [&](const float (&v)[NC][V], float (&r)[NC]) {
        float s[NC];
#pragma unroll
        for (int k = 0; k < NC; k++) {
            s[k] = 0.0f;
#pragma unroll
            for (int i = 0; i < V; i++) s[k] = __builtin_fmaf(v[k][i], v[k][i], s[k]);
            if (!own[k]) s[k] = 0.0f;
        }
        if (wave_groups) {
            float* buf = lds + (phase & 1) * (NC * 8);
            phase++;
            if (one_group) {
#pragma unroll
                for (int k = 1; k < NC; k++) s[0] += s[k];
                s[0] = wave_sum(s[0]);
                if (lane == 0) buf[wv] = s[0];
            } else {
#pragma unroll
                for (int k = 0; k < NC; k++) {
                    const float ws = wave_sum(s[k]);
                    if (lane == 0) buf[k * nw + wv] = ws;
                }
            }
            __syncthreads();
#pragma unroll
            for (int k = 0; k < NC; k++) {
                if (k > 0 && one_group) { r[k] = r[0]; continue; }
                const int slot = k * nw + wv, slots = one_group ? nw : NC * nw, group = one_group ? 0 : slot / spg;
                float sum = 0.0f;
                if ((spg & 3) == 0 && (group + 1) * spg <= slots) {
                    for (int j = 0; j < spg; j += 4) {
                        const float4 p = *reinterpret_cast<const float4*>(buf + group * spg + j);
                        sum += (p.x + p.y) + (p.z + p.w);
                    }
                } else {
                    for (int j = 0; j < spg; j++) sum += buf[group * spg + j < slots ? group * spg + j : 0];
                }
                r[k] = rsqrtf(sum * inv_gs + a.eps);
            }
        } else {
            float* buf = lds;
            float* rs = lds + NC * nthr;
#pragma unroll
            for (int k = 0; k < NC; k++) buf[k * nthr + tid] = s[k];
            __syncthreads();
            for (int g = wv; g < a.groups; g += nw) {
                float sum = 0.0f;
                for (int j = lane; j < ppg; j += kWave) sum += buf[g * ppg + j];
                sum = wave_sum(sum);
                if (lane == 0) rs[g] = rsqrtf(sum * inv_gs + a.eps);
            }
            __syncthreads();
#pragma unroll
            for (int k = 0; k < NC; k++) r[k] = rs[ch[k] / gs];
        }
    };

    float wpre[NC][V], wpost[NC][V];
    constexpr int RING = TAPS > 1 ? TAPS - 1 : 1;
    float ring[RING][NC][V], cw[TAPS > 0 ? TAPS : 1][NC][V];
#pragma unroll
    for (int k = 0; k < NC; k++) {
        ldv<T, V>(a.w_pre, ch[k], wpre[k]);
        ldv<T, V>(a.w_post ? a.w_post : a.w_pre, ch[k], wpost[k]);
    }
    // (loads of what a shorter filter or a later strip does not have go to an address that exists and are dropped: with a
    // branch around each, every one would be waited for before the next)
    if constexpr (TAPS > 0) {
        const elem_t<T>* w = static_cast<const elem_t<T>*>(a.conv_w);
        if (taps == TAPS && V == 4 && TAPS % 4 == 0) {
#pragma unroll
            for (int k = 0; k < NC; k++)
#pragma unroll
                for (int i = 0; i < V; i++)
#pragma unroll
                    for (int j = 0; j + 4 <= TAPS; j += 4) {
                        float c4[4];
                        ldv<T, 4>(w, (ch[k] + i) * static_cast<size_t>(TAPS) + j, c4);
#pragma unroll
                        for (int jj = 0; jj < 4; jj++) cw[j + jj][k][i] = c4[jj];
                    }
        } else {
#pragma unroll
            for (int j = 0; j < TAPS; j++) {
                const int tap = j - (TAPS - taps);           // of the real filter; negative: padding
#pragma unroll
                for (int k = 0; k < NC; k++)
#pragma unroll
                    for (int i = 0; i < V; i++) {
                        const float c1 = ld1<T>(w + (ch[k] + i) * static_cast<size_t>(taps) + (tap >= 0 ? tap : 0));
                        cw[j][k][i] = tap >= 0 ? c1 : 0.0f;
                    }
            }
        }
        const float* state = taps > 1 ? a.state_in : a.x_in;
#pragma unroll
        for (int j = 0; j < TAPS - 1; j++) {
            const int row = j - (TAPS - taps);
#pragma unroll
            for (int k = 0; k < NC; k++) {
                ldv<F32, V>(state, (static_cast<size_t>(b) * (taps - 1) + (row >= 0 ? row : 0)) * W + ch[k], ring[j][k]);
                const bool has = t0 == 0 && row >= 0;
#pragma unroll
                for (int i = 0; i < V; i++) ring[j][k][i] = has ? ring[j][k][i] : 0.0f;
            }
        }
    }
    const int first_tok = a.start ? a.start[b] - (a.pos_dev ? *a.pos_dev : a.pos) : 0;      // tokens before it are padding

    for (int t = begin; t < t1; t++) {
        const size_t row = (static_cast<size_t>(b) * L + t) * W;
        if (a.y) {
            if (a.w_post) {
                float r[NC];
                group_scale(yc, r);
#pragma unroll
                for (int k = 0; k < NC; k++)
#pragma unroll
                    for (int i = 0; i < V; i++) xc[k][i] = __builtin_fmaf(wpost[k][i], yc[k][i] * r[k], xc[k][i]);
            } else {
#pragma unroll
                for (int k = 0; k < NC; k++)
#pragma unroll
                    for (int i = 0; i < V; i++) xc[k][i] += yc[k][i];
            }
            if (t >= t0)
#pragma unroll
                for (int k = 0; k < NC; k++)
                    if (own[k]) stv<F32, V>(a.x_out + row, ch[k], xc[k]);
        }
        float r[NC];
        group_scale(xc, r);
        const bool real = t >= first_tok;
#pragma unroll
        for (int k = 0; k < NC; k++) {
            float h[V], o[V];
#pragma unroll
            for (int i = 0; i < V; i++) {
                h[i] = real ? wpre[k][i] * (xc[k][i] * r[k]) : 0.0f;
                o[i] = h[i];
            }
            if constexpr (TAPS > 0) {
#pragma unroll
                for (int i = 0; i < V; i++) {
                    float c = cw[TAPS - 1][k][i] * h[i];
#pragma unroll
                    for (int j = 0; j < TAPS - 1; j++) c = __builtin_fmaf(cw[j][k][i], ring[j][k][i], c);
                    o[i] += real ? c : 0.0f;
#pragma unroll
                    for (int j = 0; j + 1 < TAPS - 1; j++) ring[j][k][i] = ring[j + 1][k][i];
                    if constexpr (TAPS > 1) ring[TAPS > 1 ? TAPS - 2 : 0][k][i] = h[i];
                }
            }
            if (t >= t0 && own[k]) stv<T, V>(static_cast<elem_t<T>*>(a.h_out) + row, ch[k], o);
        }
#pragma unroll
        for (int k = 0; k < NC; k++)
#pragma unroll
            for (int i = 0; i < V; i++) {
                xc[k][i] = xn[0][k][i];
                yc[k][i] = yn[0][k][i];
#pragma unroll
                for (int d = 0; d + 1 < AHEAD; d++) { xn[d][k][i] = xn[d + 1][k][i]; yn[d][k][i] = yn[d + 1][k][i]; }
            }
        fetch(t + AHEAD + 1 < t1 ? t + AHEAD + 1 : t, xn[AHEAD - 1], yn[AHEAD - 1]);
    }
    if constexpr (TAPS > 1) {
        if (t1 == L) {
#pragma unroll
            for (int j = 0; j < TAPS - 1; j++) {
                const int row = j - (TAPS - taps);
                if (row < 0) continue;
#pragma unroll
                for (int k = 0; k < NC; k++)
                    if (own[k]) stv<F32, V>(a.state_out + (static_cast<size_t>(b) * (taps - 1) + row) * W, ch[k], ring[j][k]);
            }
        }
    }
}

int launch_norm_conv(const NormConvArgs& args, int dtype, hipStream_t st) {
    NormConvArgs a = args;
    const int taps = a.conv_w ? a.taps : 0;
    if (!a.conv_w) a.taps = 1;
    const int V = ((a.W / a.groups) % 4 == 0) ? 4 : 1;
    const int pieces = a.W / V;
    const int nthr = pieces <= 256 ? 256 : 512;
    const int per = (pieces + nthr - 1) / nthr;
    const int NC = per <= 1 ? 1 : per <= 2 ? 2 : per <= 4 ? 4 : 8;
    if (per > 8) return static_cast<int>(hipErrorInvalidValue);
    a.strip = a.L <= kConvInPlaceTokens ? a.L : 32;
    const size_t shared = (static_cast<size_t>(NC) * nthr + a.groups) * sizeof(float);
    if (shared > 64 * 1024) return static_cast<int>(hipErrorInvalidValue);
    dim3 grid(static_cast<unsigned>((a.L + a.strip - 1) / a.strip), static_cast<unsigned>(a.B)), block(nthr);
#define PQ_NC(T, TP, VV, N) hipLaunchKernelGGL((norm_conv_kernel<T, TP, VV, N>), grid, block, shared, st, a)
#define PQ_NC_N(T, TP, VV)                                                                                           \
    do {                                                                                                             \
        if (NC == 1) PQ_NC(T, TP, VV, 1); else if (NC == 2) PQ_NC(T, TP, VV, 2);                                     \
        else if (NC == 4) PQ_NC(T, TP, VV, 4); else PQ_NC(T, TP, VV, 8);                                             \
    } while (0)
#define PQ_NC_V(T, TP) do { if (V == 4) PQ_NC_N(T, TP, 4); else PQ_NC_N(T, TP, 1); } while (0)
#define PQ_NC_T(T)                                                                                                   \
    do {                                                                                                             \
        if (taps == 0) PQ_NC_V(T, 0);                                                                                \
        else if (taps <= 4) PQ_NC_V(T, 4);                                                                           \
        else if (taps <= 8) PQ_NC_V(T, 8);                                                                           \
        else PQ_NC_V(T, 16);                                                                                         \
    } while (0)
    if (dtype == 0) PQ_NC_T(F16); else if (dtype == 1) PQ_NC_T(BF16); else PQ_NC_T(F32);
#undef PQ_NC_T
#undef PQ_NC_V
#undef PQ_NC_N
#undef PQ_NC
    return static_cast<int>(hipGetLastError());
}

// ---- square of relu ----------------------------------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void relu_sq_kernel(const void* __restrict__ x, void* __restrict__ y, size_t n) {
    const size_t i = (static_cast<size_t>(blockIdx.x) * 256 + threadIdx.x) * 8;
    if (i + 8 <= n) {
        float v[2][4];
        ldv<T, 4>(x, i, v[0]);
        ldv<T, 4>(x, i + 4, v[1]);
#pragma unroll
        for (int k = 0; k < 2; k++)
#pragma unroll
            for (int j = 0; j < 4; j++) { const float r = fmaxf(v[k][j], 0.0f); v[k][j] = r * r; }
        stv<T, 4>(y, i, v[0]);
        stv<T, 4>(y, i + 4, v[1]);
    } else {
        for (size_t j = i; j < n; j++) {
            const float r = fmaxf(ld1<T>(static_cast<const elem_t<T>*>(x) + j), 0.0f);
            static_cast<elem_t<T>*>(y)[j] = cv1<T>(r * r);
        }
    }
}

int launch_relu_sq(const void* x, void* y, size_t n, int dtype, hipStream_t st) {
    dim3 grid(static_cast<unsigned>((n + 2047) / 2048)), block(256);
    if (dtype == 0) hipLaunchKernelGGL(relu_sq_kernel<F16>, grid, block, 0, st, x, y, n);
    else if (dtype == 1) hipLaunchKernelGGL(relu_sq_kernel<BF16>, grid, block, 0, st, x, y, n);
    else hipLaunchKernelGGL(relu_sq_kernel<F32>, grid, block, 0, st, x, y, n);
    return static_cast<int>(hipGetLastError());
}

// ---- gelu (tanh form) times --------------------------------------------------------------------------------------------
// 0.5 z (1 + tanh u) = z / (1 + exp(-2 u)), u = sqrt(2 / pi) (z + 0.044715 z^3)
__device__ __forceinline__ float gelu_tanh(float z) {
    const float u2 = 1.5957691216057308f * __builtin_fmaf(0.044715f * z * z, z, z);
    return z * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(u2 * -1.4426950408889634f));
}

// grid (column pieces, rows)
template <typename T, int V>
__global__ __launch_bounds__(256) void gelu_mul_kernel(GeluMulArgs a) {
    const int c = (blockIdx.x * 256 + threadIdx.x) * V;
    if (c >= a.cols) return;
    for (int64_t row = blockIdx.y; row < a.rows; row += gridDim.y) {
        float g[V], u[V];
        ldv<T, V>(a.gate, row * a.in_stride + c, g);
        ldv<T, V>(a.up, row * a.in_stride + c, u);
#pragma unroll
        for (int j = 0; j < V; j++) u[j] *= gelu_tanh(g[j]);
        stv<T, V>(a.y, row * a.out_stride + c, u);
    }
}

int launch_gelu_mul(const GeluMulArgs& a, int dtype, hipStream_t st) {
    const size_t align = dtype == 2 ? 16 : 8;
    auto ok = [&](const void* p) { return reinterpret_cast<uintptr_t>(p) % align == 0; };
    const bool v4 = a.cols % 4 == 0 && a.in_stride % 4 == 0 && a.out_stride % 4 == 0 && ok(a.gate) && ok(a.up) && ok(a.y);
    const int per = v4 ? 1024 : 256;
    dim3 grid(static_cast<unsigned>((a.cols + per - 1) / per), static_cast<unsigned>(a.rows < 32768 ? a.rows : 32768)), block(256);
#define PQ_GM(T) do { if (v4) hipLaunchKernelGGL((gelu_mul_kernel<T, 4>), grid, block, 0, st, a); \
                      else hipLaunchKernelGGL((gelu_mul_kernel<T, 1>), grid, block, 0, st, a); } while (0)
    if (dtype == 0) PQ_GM(F16); else if (dtype == 1) PQ_GM(BF16); else PQ_GM(F32);
#undef PQ_GM
    return static_cast<int>(hipGetLastError());
}

// ---- streams --------------------------------------------------------------------------------------------------------------
// x_out = x (+ y) (+ e) (+ v), v one vector for every row.  grid (column pieces, rows)
template <typename T>
__global__ __launch_bounds__(256) void stream_add_kernel(StreamAddArgs a) {
    const int c = blockIdx.x * 256 + threadIdx.x;
    if (c >= a.width) return;
    const float v = a.v ? ld1<T>(static_cast<const elem_t<T>*>(a.v) + c) : 0.0f;
    for (int64_t row = blockIdx.y; row < a.rows; row += gridDim.y) {
        const size_t i = static_cast<size_t>(row) * a.width + c;
        float x = a.x[i];
        if (a.y) x += ld1<T>(static_cast<const elem_t<T>*>(a.y) + i);
        if (a.e) x += a.e[i];
        a.x_out[i] = x + v;
    }
}

int launch_stream_add(const StreamAddArgs& a, int dtype, hipStream_t st) {
    dim3 grid(static_cast<unsigned>((a.width + 255) / 256), static_cast<unsigned>(a.rows < 32768 ? a.rows : 32768)), block(256);
    if (dtype == 0) hipLaunchKernelGGL(stream_add_kernel<F16>, grid, block, 0, st, a);
    else if (dtype == 1) hipLaunchKernelGGL(stream_add_kernel<BF16>, grid, block, 0, st, a);
    else hipLaunchKernelGGL(stream_add_kernel<F32>, grid, block, 0, st, a);
    return static_cast<int>(hipGetLastError());
}

template <typename T>
__global__ __launch_bounds__(256) void embed_rows_kernel(const void* table, const int64_t* ids, float scale, float* out, int64_t rows, int width, int64_t vocab) {
    const int c = blockIdx.x * 256 + threadIdx.x;
    if (c >= width) return;
    for (int64_t row = blockIdx.y; row < rows; row += gridDim.y) {
        int64_t id = ids[row];
        id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);          // (never past the table)
        out[static_cast<size_t>(row) * width + c] = ld1<T>(static_cast<const elem_t<T>*>(table) + static_cast<size_t>(id) * width + c) * scale;
    }
}

int launch_embed_rows(const void* table, const int64_t* ids, float scale, float* out, int64_t rows, int width, int64_t vocab, int dtype, hipStream_t st) {
    dim3 grid(static_cast<unsigned>((width + 255) / 256), static_cast<unsigned>(rows < 32768 ? rows : 32768)), block(256);
    if (dtype == 0) hipLaunchKernelGGL(embed_rows_kernel<F16>, grid, block, 0, st, table, ids, scale, out, rows, width, vocab);
    else if (dtype == 1) hipLaunchKernelGGL(embed_rows_kernel<BF16>, grid, block, 0, st, table, ids, scale, out, rows, width, vocab);
    else hipLaunchKernelGGL(embed_rows_kernel<F32>, grid, block, 0, st, table, ids, scale, out, rows, width, vocab);
    return static_cast<int>(hipGetLastError());
}

// ---- logits ---------------------------------------------------------------------------------------------------------------
__global__ __launch_bounds__(256) void softcap_kernel(float* x, size_t n, float scale, float cap) {
    const size_t i = static_cast<size_t>(blockIdx.x) * 256 + threadIdx.x;
    if (i >= n) return;
    const float z = x[i] * scale;
    x[i] = cap > 0.0f ? cap * tanhf(z / cap) : z;
}

int launch_softcap(float* x, size_t n, float scale, float cap, hipStream_t st) {
    hipLaunchKernelGGL(softcap_kernel, dim3(static_cast<unsigned>((n + 255) / 256)), dim3(256), 0, st, x, n, scale, cap);
    return static_cast<int>(hipGetLastError());
}

// ---- per-head product, any size ------------------------------------------------------------------------------------------
// A wavefront per output: lanes stride over k, then a butterfly sum.  grid (N / 4 rounded up, heads, M).
template <typename T>
__global__ __launch_bounds__(256) void head_linear_kernel(HeadLinearArgs a) {
    const int lane = threadIdx.x & 63, n = blockIdx.x * 4 + (threadIdx.x >> 6), h = blockIdx.y, m = blockIdx.z;
    if (n >= a.N) return;
    const elem_t<T>* x = static_cast<const elem_t<T>*>(a.x) + m * a.x_row + h * a.x_head;
    const elem_t<T>* w = static_cast<const elem_t<T>*>(a.w) + (static_cast<size_t>(h) * a.N + n) * a.K;
    float s = 0.0f;
    for (int k = lane; k < a.K; k += 64) s = __builtin_fmaf(ld1<T>(x + k), ld1<T>(w + k), s);
    s = wave_sum(s);
    if (lane != 0) return;
    if (a.epilogue == kEpiReluSq) {
        s = fmaxf(s, 0.0f);
        s = s * s;
    } else if (a.epilogue == kEpiSigmoidGate) {
        const float g = ld1<T>(static_cast<const elem_t<T>*>(a.gate) + m * a.gate_row + static_cast<size_t>(h) * a.N + n);
        s = s / (1.0f + __expf(-g));
    }
    const size_t o = m * a.y_row + h * a.y_head + n;
    if (a.epilogue == kEpiF32) static_cast<float*>(a.y)[o] = s;
    else static_cast<elem_t<T>*>(a.y)[o] = cv1<T>(s);
}

int launch_head_linear_any(const HeadLinearArgs& a, int dtype, hipStream_t st) {
    dim3 grid(static_cast<unsigned>((a.N + 3) / 4), static_cast<unsigned>(a.heads), static_cast<unsigned>(a.M)), block(256);
    if (dtype == 0) hipLaunchKernelGGL(head_linear_kernel<F16>, grid, block, 0, st, a);
    else if (dtype == 1) hipLaunchKernelGGL(head_linear_kernel<BF16>, grid, block, 0, st, a);
    else hipLaunchKernelGGL(head_linear_kernel<F32>, grid, block, 0, st, a);
    return static_cast<int>(hipGetLastError());
}

}  // namespace pq
