// Launcher of the per-head products at <= 16 rows (kernels: pq_linear_device.h).
#include "pq_linear_device.h"

namespace pq {

// The same two kernels for `heads` products per launch; K of a head is short (a head's dimension, a latent's rank), so
// fewer wavefronts split it: each keeps at least two k-steps.
int launch_head_linear_mfma(const HeadLinearArgs& a, int dtype, hipStream_t st) {
    const bool m8 = a.M <= 8 && (a.K % 64) == 0;
    const int kstep = m8 ? 64 : 32;
    int ks = (m8 && a.K >= 8192) ? 8 : 4;
    while (ks > 1 && ((a.K % (kstep * ks)) != 0 || a.K / (kstep * ks) < 2)) ks >>= 1;
    dim3 grid(a.N / 16, a.heads), block(kWave * ks);
    const HeadEpi he{a.x_head, static_cast<int64_t>(a.N) * a.K, a.y_head, static_cast<const uint16_t*>(a.gate), a.gate_row};
#define PQ_H(KERNEL, T, KS, S, E)                                                                                    \
    hipLaunchKernelGGL((KERNEL<T, KS, false, S, 1 + E>), grid, block, 0, st, (const uint16_t*)a.x, a.x_row,          \
                       (const uint16_t*)a.w, nullptr, nullptr, (uint16_t*)a.y, a.y_row, a.M, a.K, he)
#define PQ_H8(T, E)                                                                                                  \
    do {                                                                                                             \
        if (ks == 8) PQ_H(small_m8_linear_kernel, T, 8, 2, E);                                                       \
        else if (ks == 4) PQ_H(small_m8_linear_kernel, T, 4, 1, E);                                                  \
        else if (ks == 2) PQ_H(small_m8_linear_kernel, T, 2, 1, E);                                                  \
        else PQ_H(small_m8_linear_kernel, T, 1, 1, E);                                                               \
    } while (0)
#define PQ_H16(T, E)                                                                                                 \
    do {                                                                                                             \
        if (ks == 4) PQ_H(small_m_linear_kernel, T, 4, 4, E);                                                        \
        else if (ks == 2) PQ_H(small_m_linear_kernel, T, 2, 4, E);                                                   \
        else PQ_H(small_m_linear_kernel, T, 1, 4, E);                                                                \
    } while (0)
#define PQ_HE(T, E) do { if (m8) PQ_H8(T, E); else PQ_H16(T, E); } while (0)
#define PQ_HT(T)                                                                                                     \
    do {                                                                                                             \
        if (a.epilogue == kEpiReluSq) PQ_HE(T, kEpiReluSq);                                                          \
        else if (a.epilogue == kEpiSigmoidGate) PQ_HE(T, kEpiSigmoidGate);                                           \
        else if (a.epilogue == kEpiF32) PQ_HE(T, kEpiF32);                                                           \
        else PQ_HE(T, kEpiPlain);                                                                                    \
    } while (0)
    if (dtype == 0) PQ_HT(F16); else PQ_HT(BF16);
#undef PQ_HT
#undef PQ_HE
#undef PQ_H16
#undef PQ_H8
#undef PQ_H
    return static_cast<int>(hipGetLastError());
}

}  // namespace pq
