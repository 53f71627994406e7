// Mixture of experts with squared-ReLU experts -- gfx950.
//
//   trimkv_moe_route   sigmoid scores, choice scores with a correction, groups of neighbouring experts of which the best are
//                      open (a group's score: its two largest choice scores), top-k; weights are the plain scores
//   trimkv_moe_plan    (token, choice) rows ordered by expert, and the list of row tiles of the grouped products
//   trimkv_moe_gemm    one product per expert over its rows: up (rows gathered by token, squared ReLU) or down (rows
//                      scattered back to (token, choice) order)
//
// Expert weights are [E][n padded][k padded] with zeros in the padding (both padded to multiples of 64), activations rows
// of k padded elements, so that no kernel has a tail along k.
#include "hybrid.hip.h"
#include <type_traits>

namespace trimkv {

constexpr int ROUTE_MAX_E = 1024;

__global__ __launch_bounds__(256) void route_kernel(const float* z, const float* correction, int32_t* ids, float* weights, int tokens, int E, int top, int count, int keep) {
    extern __shared__ float rt[];                 // per wavefront: choice [E], group [count]
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
    const int t = blockIdx.x * 4 + w;
    float* choice = rt + w * (E + count);
    float* group = choice + E;
    const bool live = t < tokens;
    const float* zr = z + (int64_t)min(t, tokens - 1) * E;
    for (int e = lane; e < E; e += 64) choice[e] = sigmoid_f(zr[e]) + correction[e];
    __syncthreads();
    const int per = E / count;
    for (int g = lane; g < count; g += 64) {
        float a = -INFINITY, b = -INFINITY;
        for (int e = g * per; e < (g + 1) * per; ++e) {
            const float c = choice[e];
            if (c > a) { b = a; a = c; } else if (c > b) b = c;
        }
        group[g] = per > 1 ? a + b : a;
    }
    __syncthreads();
    float c[ROUTE_MAX_E / 64];
#pragma unroll
    for (int i = 0; i < ROUTE_MAX_E / 64; ++i) {
        const int e = i * 64 + lane;
        c[i] = -INFINITY;
        if (e < E) {
            const int g = e / per;
            int better = 0;
            for (int o = 0; o < count; ++o) better += group[o] > group[g] || (group[o] == group[g] && o < g);
            if (better < keep) c[i] = choice[e];
        }
    }
    for (int j = 0; j < top; ++j) {
        float best = -INFINITY;
        int at = 0x7fffffff;
#pragma unroll
        for (int i = 0; i < ROUTE_MAX_E / 64; ++i)
            if (c[i] > best) { best = c[i]; at = i * 64 + lane; }
#pragma unroll
        for (int d = 32; d > 0; d >>= 1) {
            const float bo = __shfl_xor(best, d, 64);
            const int ao = __shfl_xor(at, d, 64);
            if (bo > best || (bo == best && ao < at)) { best = bo; at = ao; }
        }
        at = min(at, E - 1);                      // non-finite logits: stay in bounds
#pragma unroll
        for (int i = 0; i < ROUTE_MAX_E / 64; ++i)
            if (i * 64 + lane == at) c[i] = -INFINITY;
        if (live && lane == 0) {
            ids[(int64_t)t * top + j] = at;
            weights[(int64_t)t * top + j] = sigmoid_f(zr[at]);
        }
    }
}

// One workgroup orders all rows (a step's few thousand, or a prompt's tens of thousands): counts, offsets and scatter in LDS.
__global__ __launch_bounds__(1024) void plan_kernel(const int32_t* ids, int rows, int E, int tile, int32_t* order, int32_t* offsets, int32_t* tiles) {
    extern __shared__ int32_t pl[];               // cursor [E], tile cursor [E]
    int32_t* cursor = pl; int32_t* tcur = pl + E;
    const int tid = threadIdx.x;
    for (int e = tid; e < E; e += 1024) cursor[e] = 0;
    __syncthreads();
    for (int i = tid; i < rows; i += 1024) atomicAdd(&cursor[ids[i]], 1);
    __syncthreads();
    if (tid < 64) {                               // exclusive sums over experts, 64 at a time
        int base = 0, tbase = 0;
        for (int e0 = 0; e0 < E; e0 += 64) {
            const int e = e0 + tid, c = e < E ? cursor[e] : 0, nt = (c + tile - 1) / tile;
            int s = c, ts = nt;
#pragma unroll
            for (int d = 1; d < 64; d <<= 1) {
                const int o = __shfl_up(s, d, 64), to = __shfl_up(ts, d, 64);
                if (tid >= d) { s += o; ts += to; }
            }
            if (e < E) { offsets[e] = base + s - c; cursor[e] = base + s - c; tcur[e] = tbase + ts - nt; }
            base += __shfl(s, 63, 64);
            tbase += __shfl(ts, 63, 64);
        }
        if (tid == 0) { offsets[E] = base; tiles[0] = tbase; }
    }
    __syncthreads();
    // tiles[1 + 2 i] = expert, tiles[2 + 2 i] = first row of tile i
    for (int e = tid; e < E; e += 1024) {
        const int first = cursor[e], c = (e + 1 < E ? cursor[e + 1] : rows) - first;
        for (int x = 0; x * tile < c; ++x) { tiles[1 + 2 * (tcur[e] + x)] = e; tiles[2 + 2 * (tcur[e] + x)] = first + x * tile; }
    }
    __syncthreads();
    for (int i = tid; i < rows; i += 1024) order[atomicAdd(&cursor[ids[i]], 1)] = i;
}

struct GroupedArgs {
    const void* x; int64_t xs;                    // activations; up: row = order[i] / top, down: row = i
    const void* w;                                // [E][np][kp]
    void* y; int64_t ys;                          // up: row i; down: row order[i]
    const int32_t* order; const int32_t* offsets; const int32_t* tiles;
    int top, n, np, kp;
};
// squared ReLU of the up product; the down product passes
template <bool UP> __device__ __forceinline__ float expert_act(float f) { return UP ? (f > 0.0f ? f * f : 0.0f) : f; }

// General form: 16 rows x 64 outputs per workgroup, fp32 arithmetic.
template <typename T, bool UP>
__global__ __launch_bounds__(256) void grouped_simple_kernel(GroupedArgs a) {
    __shared__ float xs[16][17];
    __shared__ float wsm[64][17];
    if ((int)blockIdx.x >= a.tiles[0]) return;
    const int e = a.tiles[1 + 2 * blockIdx.x], m0 = a.tiles[2 + 2 * blockIdx.x], mend = a.offsets[e + 1];
    const int tid = threadIdx.x, n0 = blockIdx.y * 64;
    const int tn = tid & 63, tm = tid >> 6;
    const T* w = (const T*)a.w + (int64_t)e * a.np * a.kp;
    float acc[4] = {0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < a.kp; k0 += 16) {
        {
            const int r = tid >> 4, c = tid & 15, i = min(m0 + r, mend - 1);
            const int64_t row = UP ? a.order[i] / a.top : i;
            xs[r][c] = ld((const T*)a.x + row * a.xs + k0 + c);
        }
        for (int x = tid; x < 1024; x += 256) wsm[x >> 4][x & 15] = ld(w + (int64_t)(n0 + (x >> 4)) * a.kp + k0 + (x & 15));
        __syncthreads();
#pragma unroll
        for (int c = 0; c < 16; ++c)
#pragma unroll
            for (int y = 0; y < 4; ++y) acc[y] = fmaf(xs[tm * 4 + y][c], wsm[tn][c], acc[y]);
        __syncthreads();
    }
#pragma unroll
    for (int y = 0; y < 4; ++y) {
        const int i = m0 + tm * 4 + y;
        if (i < mend && n0 + tn < a.n) st((T*)a.y + (UP ? (int64_t)i : (int64_t)a.order[i]) * a.ys + n0 + tn, expert_act<UP>(acc[y]));
    }
}

}  // namespace trimkv

using namespace trimkv;

extern "C" int trimkv_moe_route(const float* logits, const float* correction, int32_t* ids, float* weights, int tokens, int experts, int top, int groups,
                                int keep_groups, void* stream) {
    const char* fn = "trimkv_moe_route";
    if (!logits || !correction || !ids || !weights) return fail(TRIMKV_ERR_NULL, "%s: null pointer argument", fn);
    if (tokens <= 0 || experts <= 0 || experts > ROUTE_MAX_E || groups <= 0 || experts % groups || keep_groups < 1 || keep_groups > groups || top < 1 ||
        top > keep_groups * (experts / groups))
        return fail(TRIMKV_ERR_SHAPE, "%s: bad sizes tokens=%d experts=%d top=%d groups=%d keep=%d", fn, tokens, experts, top, groups, keep_groups);
    hipLaunchKernelGGL(route_kernel, dim3((tokens + 3) / 4), dim3(256), 4 * (experts + groups) * sizeof(float), (hipStream_t)stream, logits, correction, ids, weights,
                       tokens, experts, top, groups, keep_groups);
    return launch_status(fn);
}

extern "C" int trimkv_moe_plan(const int32_t* ids, int rows, int experts, int tile, int32_t* order, int32_t* offsets, int32_t* tiles, void* stream) {
    const char* fn = "trimkv_moe_plan";
    if (!ids || !order || !offsets || !tiles) return fail(TRIMKV_ERR_NULL, "%s: null pointer argument", fn);
    if (rows <= 0 || experts <= 0 || experts > ROUTE_MAX_E || tile <= 0) return fail(TRIMKV_ERR_SHAPE, "%s: bad sizes rows=%d experts=%d tile=%d", fn, rows, experts, tile);
    hipLaunchKernelGGL(plan_kernel, dim3(1), dim3(1024), 2 * experts * sizeof(int32_t), (hipStream_t)stream, ids, rows, experts, tile, order, offsets, tiles);
    return launch_status(fn);
}

extern "C" int trimkv_moe_gemm(const void* x, int64_t x_stride, const void* w, void* y, int64_t y_stride, const int32_t* order, const int32_t* offsets,
                               const int32_t* tiles, int rows, int experts, int tile, int top, int n, int n_padded, int k_padded, int up, int dtype, void* stream) {
    const char* fn = "trimkv_moe_gemm";
    if (!x || !w || !y || !order || !offsets || !tiles) return fail(TRIMKV_ERR_NULL, "%s: null pointer argument", fn);
    HY_CHECK_DTYPE(fn, dtype);
    if (rows <= 0 || experts <= 0 || top <= 0 || n <= 0 || n > n_padded || n_padded % 64 || k_padded <= 0 || k_padded % 64 || x_stride < k_padded || y_stride < n)
        return fail(TRIMKV_ERR_SHAPE, "%s: bad sizes rows=%d experts=%d n=%d/%d k=%d", fn, rows, experts, n, n_padded, k_padded);
    if (tile != 16) return fail(TRIMKV_ERR_SHAPE, "%s: row tiles of 16 (got %d)", fn, tile);
    GroupedArgs a{x, x_stride, w, y, y_stride, order, offsets, tiles, top, n, n_padded, k_padded};
    hipStream_t s = (hipStream_t)stream;
    const int most = rows < experts ? rows : (rows - experts) / tile + experts;     // no more row tiles than this
    const dim3 grid(most, n_padded / 64);
    HY_BY_DTYPE(dtype, T,
        if (up) hipLaunchKernelGGL((grouped_simple_kernel<T, true>), grid, dim3(256), 0, s, a);
        else hipLaunchKernelGGL((grouped_simple_kernel<T, false>), grid, dim3(256), 0, s, a));
    return launch_status(fn);
}
