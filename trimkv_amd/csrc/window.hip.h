// Sliding-window attention with kept first tokens over a ring of keys and values: what its prompt and decode kernels share.
//
// Position i sees j iff j <= i and (i - j < size or j < keep).  Keys arrive as they are scored (rotated, if at all), so a sequence needs
// exactly keep + size rows however long it is: the first `keep` tokens own their rows, later ones overwrite the row of the
// token that has just left the window.  After a token is stored, the rows in use are its visible set.
//
// Scores, maxima, exponentials and sums are fp32; scores are scaled after the product.  The sigmoid output gate (a number per
// value or one per head) is applied on the way out.  With a sink the denominator has one more term, a score of 0 without a value.
#pragma once

#include "hybrid.hip.h"

namespace trimkv {

constexpr float WA_NEG = -1.0e30f;

struct WindowArgs {
    const void* q; const void* k; const void* v;      // portion, [T][heads][padded dim]
    const void* rk; const void* rv;                   // rings [slot][G][keep + size][padded dim]
    const int32_t* cu; const int32_t* slots; const int32_t* seen;
    const void* gate; int64_t gate_stride; void* out;
    int H, G, D, Dv, Dp, Dvp, keep, size;
    float scale_log2;
    int chunk, splits; float* ws;                     // decode: rows per workgroup; partial results
    int vec;                                          // gate and out may be accessed four elements at a time
    int head_gate;                                    // one gate per head instead of one per value
    int sink;                                         // the softmax denominator starts at exp(0)
};
template <typename T>
__device__ __forceinline__ float window_gate(const WindowArgs& a, int64_t t, int h, int d) {
    return sigmoid_fast(ld((const T*)a.gate + t * a.gate_stride + (a.head_gate ? h : h * a.Dv + d)));
}
// what the sink adds to a sum of weights exp2(score - m)
__device__ __forceinline__ float window_sink(const WindowArgs& a, float m) { return a.sink ? exp2f(-m) : 0.0f; }

inline int window_common(const char* fn, const WindowArgs& a, int batch, int dtype) {
    if (!a.q || !a.rk || !a.rv || !a.slots || !a.seen || !a.gate || !a.out) return fail(TRIMKV_ERR_NULL, "%s: null pointer argument", fn);
    HY_CHECK_DTYPE(fn, dtype);
    if (batch <= 0 || batch > 65535 || a.H <= 0 || a.G <= 0 || a.H % a.G || a.D <= 0 || a.Dv <= 0 || a.Dp < a.D || a.Dvp < a.Dv || a.Dp % 8 || a.Dvp % 8 || a.keep < 0 || a.size <= 0)
        return fail(TRIMKV_ERR_SHAPE, "%s: bad sizes batch=%d heads=%d kv_heads=%d dim=%d/%d vdim=%d/%d keep=%d window=%d", fn, batch, a.H, a.G, a.D, a.Dp, a.Dv, a.Dvp, a.keep, a.size);
    if (a.Dp > 512 || a.Dvp > 512) return fail(TRIMKV_ERR_UNSUPPORTED, "%s: head sizes up to 512 (got %d, %d)", fn, a.D, a.Dv);
    if ((int64_t)batch * a.H > 65535 * 16) return fail(TRIMKV_ERR_SHAPE, "%s: too many (sequence, head) pairs", fn);
    if (((uintptr_t)a.q | (uintptr_t)a.rk | (uintptr_t)a.rv) & 15) return fail(TRIMKV_ERR_SHAPE, "%s: q and the rings must be 16-byte aligned", fn);
    return 0;
}

}  // namespace trimkv
