// RMS norms of the query latent and of the key/value latent, the latter written to its cache row.  fp32 arithmetic on
// whatever the operands' dtype is; results are rounded to it once.
#include "pq_elem.h"
#include "pq_latent_internal.h"

namespace pq {

// ---- norms of the two latents ---------------------------------------------------------------------------------------
// A wavefront per token when there are many (WIDE false), a workgroup per token otherwise.
template <typename T, int V, bool WIDE>
__global__ __launch_bounds__(256) void latent_norm_kernel(LatentNormArgs a) {
    __shared__ float part[2][4];
    const int wv = threadIdx.x >> 6, n_tok = a.B * a.L;
    const int first = (WIDE ? static_cast<int>(threadIdx.x) : static_cast<int>(threadIdx.x & 63)) * V, step = (WIDE ? 256 : 64) * V;
    int tok = WIDE ? static_cast<int>(blockIdx.x) : static_cast<int>(blockIdx.x) * 4 + wv;
    if (!WIDE && tok >= n_tok) return;
    const int b = tok / a.L, t = tok - b * a.L;
    const int Q = a.q_rank, R = a.w_kv ? a.kv_rank : 0;
    const elem_t<T>* p = static_cast<const elem_t<T>*>(a.p) + static_cast<size_t>(tok) * a.row_stride;
    float sq = 0.0f, sc = 0.0f, v[V];
    for (int i = first; i < Q + R; i += step) {
        ldv<T, V>(p, i, v);
        float s = 0.0f;
#pragma unroll
        for (int j = 0; j < V; j++) s = __builtin_fmaf(v[j], v[j], s);
        sq += i < Q ? s : 0.0f;
        sc += i < Q ? 0.0f : s;
    }
    sq = wave_sum(sq);
    sc = wave_sum(sc);
    if (WIDE) {
        if ((threadIdx.x & 63) == 0) { part[0][wv] = sq; part[1][wv] = sc; }
        __syncthreads();
        sq = part[0][0] + part[0][1] + part[0][2] + part[0][3];
        sc = part[1][0] + part[1][1] + part[1][2] + part[1][3];
    }
    const float rq = rsqrtf(sq / static_cast<float>(Q) + a.eps), rc = R ? rsqrtf(sc / static_cast<float>(R) + a.eps) : 0.0f;
    int64_t pos = (a.pos_dev ? *a.pos_dev : a.pos) + t;
    pos = pos < 0 ? 0 : (pos >= a.capacity ? a.capacity - 1 : pos);          // (never past the cache)
    elem_t<T>* qo = static_cast<elem_t<T>*>(a.q_out) + static_cast<size_t>(tok) * Q;
    elem_t<T>* co = static_cast<elem_t<T>*>(a.cache) + (static_cast<size_t>(b) * a.capacity + pos) * R;
    for (int i = first; i < Q + R; i += step) {
        const bool is_q = i < Q;
        float w[V];
        ldv<T, V>(p, i, v);
        ldv<T, V>(is_q ? a.w_q : a.w_kv, is_q ? i : i - Q, w);
        const float r = is_q ? rq : rc;
#pragma unroll
        for (int j = 0; j < V; j++) v[j] = w[j] * (v[j] * r);
        stv<T, V>(is_q ? qo : co, is_q ? i : i - Q, v);
    }
}

int launch_latent_norm(const LatentNormArgs& a, int dtype, hipStream_t st) {
    const bool v4 = a.q_rank % 4 == 0 && (!a.w_kv || a.kv_rank % 4 == 0) && a.row_stride % 4 == 0;
    const int n_tok = a.B * a.L;
    const bool wide = n_tok < 1024;
    dim3 grid(static_cast<unsigned>(wide ? n_tok : (n_tok + 3) / 4)), block(256);
#define PQ_LN1(T, V) do { if (wide) hipLaunchKernelGGL((latent_norm_kernel<T, V, true>), grid, block, 0, st, a); \
                          else hipLaunchKernelGGL((latent_norm_kernel<T, V, false>), grid, block, 0, st, a); } while (0)
#define PQ_LN(T) do { if (v4) PQ_LN1(T, 4); else PQ_LN1(T, 1); } while (0)
    if (dtype == 0) PQ_LN(F16); else if (dtype == 1) PQ_LN(BF16); else PQ_LN(F32);
#undef PQ_LN
#undef PQ_LN1
    return static_cast<int>(hipGetLastError());
}

}  // namespace pq
