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

// fp32: 16 rows x 64 outputs per workgroup.
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

// bf16, a handful of rows per expert (decode): 16 rows x 64 outputs per workgroup, 16 outputs per wavefront, operands straight
// from memory (lane l: 8 consecutive k of weight row, or token row, l % 16 at k-group l / 16).  The launch is bound by the
// stream of weights; UNROLL loads of them are in flight per lane.
template <bool UP>
__global__ __launch_bounds__(256) void grouped_skinny_kernel(GroupedArgs a) {
    constexpr int UNROLL = 8;
    if ((int)blockIdx.x >= a.tiles[0]) return;
    const int e = a.tiles[1 + 2 * blockIdx.x], m0 = a.tiles[2 + 2 * blockIdx.x], mend = a.offsets[e + 1];
    const int lane = threadIdx.x & 63, r = lane & 15, kg = lane >> 4, n0 = blockIdx.y * 64 + (threadIdx.x >> 6) * 16;
    const int i = min(m0 + r, mend - 1);
    const uint16_t* xr = (const uint16_t*)a.x + (UP ? (int64_t)(a.order[i] / a.top) : (int64_t)i) * a.xs + kg * 8;
    const uint16_t* wr = (const uint16_t*)a.w + ((int64_t)e * a.np + n0 + r) * a.kp + kg * 8;
    hy_f32x4 acc[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
    for (int k = 0; k < a.kp; k += 32 * UNROLL) {
        hy_u32x4 wf[UNROLL], xf[UNROLL];
#pragma unroll
        for (int u = 0; u < UNROLL; ++u) wf[u] = __builtin_nontemporal_load((const hy_u32x4*)(wr + min(k + 32 * u, a.kp - 32)));
#pragma unroll
        for (int u = 0; u < UNROLL; ++u) {
            xf[u] = *(const hy_u32x4*)(xr + min(k + 32 * u, a.kp - 32));
            if (k + 32 * u >= a.kp) xf[u] = hy_u32x4{0u, 0u, 0u, 0u};
        }
#pragma unroll
        for (int u = 0; u < UNROLL; ++u) acc[u & 1] = mfma16(__builtin_bit_cast(hy_bf16x8, wf[u]), __builtin_bit_cast(hy_bf16x8, xf[u]), acc[u & 1]);
    }
    // lane holds outputs n0 + 4 kg .. + 3 of row r
    if (m0 + r >= mend) return;
    uint16_t* y = (uint16_t*)a.y + (UP ? (int64_t)(m0 + r) : (int64_t)a.order[m0 + r]) * a.ys + n0 + 4 * kg;
#pragma unroll
    for (int v = 0; v < 4; ++v)
        if (n0 + 4 * kg + v < a.n) y[v] = f32_to_bf16_bits(expert_act<UP>(acc[0][v] + acc[1][v]));
}

// bf16, many rows per expert (prompts): 128 rows x 128 outputs per workgroup, 64 x 64 per wavefront on 32x32x16 MFMAs, 64 k per
// step through two LDS buffers filled by LDS-direct loads (whose lanes gather token rows as they please).  Row r keeps its
// 16-byte piece c at c ^ ((r / 2) % 8), so that the rows of a fragment read fall on different banks.
template <bool UP>
__global__ __launch_bounds__(256) void grouped_big_kernel(GroupedArgs a, int n_tiles) {
    extern __shared__ __attribute__((aligned(16))) char gb_lds[];
    HY_LDS char* const lds3 = (HY_LDS char*)gb_lds;
    const uint32_t lds0 = (uint32_t)(uintptr_t)lds3;
    // an XCD takes a contiguous share of the row tiles and walks it in blocks of 4 row tiles x all outputs: the rows and the
    // weights that neighbouring workgroups read stay in its L2
    const int total = a.tiles[0], share = (total + 7) / 8, turn = blockIdx.x >> 3;
    const int blk = turn / (4 * n_tiles), in = turn - blk * 4 * n_tiles;
    const int first = blk * 4, rows_here = min(4, share - first);
    if (rows_here <= 0) return;
    const int rt_ = first + in % rows_here, nt = in / rows_here;
    const int rt = (blockIdx.x & 7) * share + rt_;
    if (nt >= n_tiles || rt >= total) return;
    const int e = a.tiles[1 + 2 * rt], m0 = a.tiles[2 + 2 * rt], mend = a.offsets[e + 1], n0 = nt * 128;
    const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6), j = lane & 31, hl = lane >> 5;
    const int wm = w & 1, wn = w >> 1;
    const uint16_t* xp[4]; const uint16_t* wp[4];
#pragma unroll
    for (int x = 0; x < 4; ++x) {
        const int row = x * 32 + (tid >> 3), piece = (tid & 7) ^ ((row >> 1) & 7);
        const int i = min(m0 + row, mend - 1);
        xp[x] = (const uint16_t*)a.x + (UP ? (int64_t)(a.order[i] / a.top) : (int64_t)i) * a.xs + piece * 8;
        wp[x] = (const uint16_t*)a.w + ((int64_t)e * a.np + min(n0 + row, a.np - 1)) * a.kp + piece * 8;
    }
    auto request = [&](int k, int buf) __attribute__((always_inline)) {
        const uint32_t dst = lds0 + buf * 32768 + w * 1024;
#pragma unroll
        for (int x = 0; x < 4; ++x) load_to_lds16(xp[x] + k, dst + x * 4096);
#pragma unroll
        for (int x = 0; x < 4; ++x) load_to_lds16(wp[x] + k, dst + 16384 + x * 4096);
    };
    hy_f32x16 acc[2][2];
#pragma unroll
    for (int x = 0; x < 2; ++x)
#pragma unroll
        for (int y = 0; y < 2; ++y)
#pragma unroll
            for (int v = 0; v < 16; ++v) acc[x][y][v] = 0.0f;
    const int sw = (j >> 1) & 7;
    HY_LDS char* const xr = lds3 + (wm * 64 + j) * 128;
    HY_LDS char* const wr = lds3 + 16384 + (wn * 64 + j) * 128;
    request(0, 0);
    const int steps = a.kp / 64;
    for (int s = 0; s < steps; ++s) {
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();
        if (s + 1 < steps) request((s + 1) * 64, (s + 1) & 1);
        const int off = (s & 1) * 32768;
#pragma unroll
        for (int ks = 0; ks < 4; ++ks) {
            const int po = off + (((2 * ks + hl) ^ sw) << 4);
            hy_bf16x8 xf[2], wf[2];
#pragma unroll
            for (int y = 0; y < 2; ++y) { xf[y] = *(const HY_LDS hy_bf16x8*)(xr + y * 4096 + po); wf[y] = *(const HY_LDS hy_bf16x8*)(wr + y * 4096 + po); }
#pragma unroll
            for (int x = 0; x < 2; ++x)
#pragma unroll
                for (int y = 0; y < 2; ++y) acc[x][y] = mfma32(wf[x], xf[y], acc[x][y]);
        }
    }
    // acc[x][y]: outputs n0 + wn 64 + 32 x + 8 (v / 4) + 4 hl + v % 4 of row m0 + wm 64 + 32 y + j
#pragma unroll
    for (int y = 0; y < 2; ++y) {
        const int i = m0 + wm * 64 + 32 * y + j;
        if (i >= mend) continue;
        uint16_t* yr = (uint16_t*)a.y + (UP ? (int64_t)i : (int64_t)a.order[i]) * a.ys;
#pragma unroll
        for (int x = 0; x < 2; ++x)
#pragma unroll
            for (int c = 0; c < 4; ++c) {
                const int n = n0 + wn * 64 + 32 * x + 8 * c + 4 * hl;
                float f[4];
#pragma unroll
                for (int v = 0; v < 4; ++v) f[v] = expert_act<UP>(acc[x][y][4 * c + v]);
                if (n + 3 < a.n && a.ys % 4 == 0) *(uint2*)(yr + n) = make_uint2(pack2(f[0], f[1]), pack2(f[2], f[3]));
                else
#pragma unroll
                    for (int v = 0; v < 4; ++v)
                        if (n + v < a.n) yr[n + v] = f32_to_bf16_bits(f[v]);
            }
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
    if (tile != 16 && !(tile == 128 && dtype == TRIMKV_BF16)) return fail(TRIMKV_ERR_SHAPE, "%s: row tiles of 16, or of 128 in bf16 (got %d)", fn, tile);
    if (((uintptr_t)x | (uintptr_t)w | (uintptr_t)y) & 15 || x_stride % 8) return fail(TRIMKV_ERR_SHAPE, "%s: x, w and y must be 16-byte aligned", fn);
    GroupedArgs a{x, x_stride, w, y, y_stride, order, offsets, tiles, top, n, n_padded, k_padded};
    hipStream_t s = (hipStream_t)stream;
    const int most = rows < experts ? rows : (rows - experts) / tile + experts;     // no more row tiles than this
    const dim3 grid(most, n_padded / 64);
    if (tile == 128) {
        const int n_tiles = (n_padded + 127) / 128, blocks = 8 * (((most + 7) / 8 + 3) / 4) * 4 * n_tiles;
        if (up) hipLaunchKernelGGL((grouped_big_kernel<true>), dim3(blocks), dim3(256), 65536, s, a, n_tiles);
        else hipLaunchKernelGGL((grouped_big_kernel<false>), dim3(blocks), dim3(256), 65536, s, a, n_tiles);
    } else if (dtype == TRIMKV_BF16) {
        if (up) hipLaunchKernelGGL((grouped_skinny_kernel<true>), grid, dim3(256), 0, s, a);
        else hipLaunchKernelGGL((grouped_skinny_kernel<false>), grid, dim3(256), 0, s, a);
    } else {
        if (up) hipLaunchKernelGGL((grouped_simple_kernel<float, true>), grid, dim3(256), 0, s, a);
        else hipLaunchKernelGGL((grouped_simple_kernel<float, false>), grid, dim3(256), 0, s, a);
    }
    return launch_status(fn);
}
