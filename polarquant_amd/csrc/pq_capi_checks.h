// Argument checks that the C-ABI translation units share.
#pragma once
#include <stddef.h>
#include <stdint.h>

namespace pq {
namespace capi {

inline bool aligned(const void* p, size_t a) { return (reinterpret_cast<uintptr_t>(p) & (a - 1)) == 0; }
inline bool any_dtype(int d) { return d == PQ_F16 || d == PQ_BF16 || d == PQ_F32; }
inline int status(int err) { return err == 0 ? PQ_OK : PQ_ERR_LAUNCH; }
constexpr int64_t kMaxTokens = int64_t{1} << 30;

inline int check_tokens(int B, int L) {
    if (B < 1 || B > 65535 || L < 1 || static_cast<int64_t>(B) * L > kMaxTokens) return PQ_ERR_BAD_SHAPE;
    return PQ_OK;
}

}  // namespace capi
}  // namespace pq
