// Mixture of experts with squared-ReLU experts -- gfx950.
//
//   trimkv_moe_route   sigmoid scores, choice scores with a correction, groups of neighbouring experts of which the best are
//                      open (a group's score: its two largest choice scores), top-k; weights are the plain scores
//   trimkv_moe_plan    (token, choice) rows ordered by expert, and the list of row tiles of the grouped products
//   trimkv_moe_gemm    one product per expert over its rows: up (rows gathered by token, squared ReLU) or down (rows
//                      scattered back to (token, choice) order)
//
// Expert weights are stored in the order in which the matrix cores take them: blocks of 32 outputs x 16 k, in a block first
// k 0..7 of the 32 outputs, then k 8..15 (lane l of a wavefront: output l % 32, k 8 (l / 32) .. + 7), so that a load
// instruction reads 1 KiB in one piece: [E][n padded / 32][k padded / 16][2][32][8].  n and k are padded with zeros to
// multiples of 64, activations are rows of k padded elements: no kernel has a tail along k.
#include "hybrid.hip.h"
#include <type_traits>

namespace trimkv {

constexpr int ROUTE_MAX_E = 1024;

// NE: 64-expert slices, rounded up
template <int NE>
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
    float c[NE];
#pragma unroll
    for (int i = 0; i < NE; ++i) {
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
        for (int i = 0; i < NE; ++i)
            if (c[i] > best) { best = c[i]; at = i * 64 + lane; }
#pragma unroll
        for (int d = 32; d > 0; d >>= 1) {
            const float bo = __shfl_xor(best, d, 64);
            const int ao = __shfl_xor(at, d, 64);
            if (bo > best || (bo == best && ao < at)) { best = bo; at = ao; }
        }
        at = min(at, E - 1);                      // non-finite logits: stay in bounds
#pragma unroll
        for (int i = 0; i < NE; ++i)
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

// element (n, k) of an expert's matrix
__device__ __forceinline__ int64_t packed_at(int n, int k, int kp) { return ((int64_t)(n >> 5) * (kp >> 4) + (k >> 4)) * 512 + ((k >> 3) & 1) * 256 + (n & 31) * 8 + (k & 7); }

// fp32: 16 rows x 64 outputs per workgroup.
template <bool UP>
__global__ __launch_bounds__(256) void grouped_f32_kernel(GroupedArgs a) {
    __shared__ float xs[16][17];
    __shared__ float wsm[64][17];
    if ((int)blockIdx.x >= a.tiles[0]) return;
    const int e = a.tiles[1 + 2 * blockIdx.x], m0 = a.tiles[2 + 2 * blockIdx.x], mend = a.offsets[e + 1];
    const int tid = threadIdx.x, n0 = blockIdx.y * 64;
    const int tn = tid & 63, tm = tid >> 6;
    const float* w = (const float*)a.w + (int64_t)e * a.np * a.kp;
    float acc[4] = {0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < a.kp; k0 += 16) {
        {
            const int r = tid >> 4, c = tid & 15, i = min(m0 + r, mend - 1);
            const int64_t row = UP ? a.order[i] / a.top : i;
            xs[r][c] = ((const float*)a.x)[row * a.xs + k0 + c];
        }
        for (int x = tid; x < 1024; x += 256) wsm[x >> 4][x & 15] = w[packed_at(n0 + (x >> 4), k0 + (x & 15), a.kp)];
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
        if (i < mend && n0 + tn < a.n) ((float*)a.y)[(UP ? (int64_t)i : (int64_t)a.order[i]) * a.ys + n0 + tn] = expert_act<UP>(acc[y]);
    }
}

// four consecutive outputs from n on
template <bool UP>
__device__ __forceinline__ void store_outputs(const GroupedArgs& a, uint16_t* yr, int n, float f0, float f1, float f2, float f3) {
    f0 = expert_act<UP>(f0); f1 = expert_act<UP>(f1); f2 = expert_act<UP>(f2); f3 = expert_act<UP>(f3);
    if (n + 3 < a.n && a.ys % 4 == 0) { *(uint2*)(yr + n) = make_uint2(pack2(f0, f1), pack2(f2, f3)); return; }
    if (n < a.n) yr[n] = f32_to_bf16_bits(f0);
    if (n + 1 < a.n) yr[n + 1] = f32_to_bf16_bits(f1);
    if (n + 2 < a.n) yr[n + 2] = f32_to_bf16_bits(f2);
    if (n + 3 < a.n) yr[n + 3] = f32_to_bf16_bits(f3);
}

// bf16, a handful of rows per expert (decode): 32 rows x 32 outputs per workgroup, whose KS wavefronts share the k of them;
// operands straight from memory.  The launch is bound by the stream of weights; UNROLL loads of them are in flight per lane.
template <bool UP, int KS>
__global__ __launch_bounds__(KS * 64) void grouped_skinny_kernel(GroupedArgs a) {
    constexpr int UNROLL = 8;
    __shared__ hy_f32x4 part[KS - 1][4][64];
    if ((int)blockIdx.x >= a.tiles[0]) return;
    const int e = a.tiles[1 + 2 * blockIdx.x], m0 = a.tiles[2 + 2 * blockIdx.x], mend = a.offsets[e + 1];
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, j = lane & 31, hl = lane >> 5;
    const int nb = blockIdx.y, kb16 = a.kp >> 4, span = (kb16 + KS - 1) / KS, s0 = w * span, s1 = min(kb16, s0 + span);
    const int i = min(m0 + j, mend - 1);
    const uint16_t* xr = (const uint16_t*)a.x + (UP ? (int64_t)(a.order[i] / a.top) : (int64_t)i) * a.xs + hl * 8;
    const uint16_t* wr = (const uint16_t*)a.w + ((int64_t)e * (a.np >> 5) + nb) * kb16 * 512 + lane * 8;
    hy_f32x16 acc;
#pragma unroll
    for (int v = 0; v < 16; ++v) acc[v] = 0.0f;
    for (int s = s0; s < s1; s += UNROLL) {
        hy_u32x4 wf[UNROLL], xf[UNROLL];
#pragma unroll
        for (int u = 0; u < UNROLL; ++u) wf[u] = __builtin_nontemporal_load((const hy_u32x4*)(wr + (int64_t)min(s + u, s1 - 1) * 512));
#pragma unroll
        for (int u = 0; u < UNROLL; ++u) {
            xf[u] = *(const hy_u32x4*)(xr + min(s + u, s1 - 1) * 16);
            if (s + u >= s1) xf[u] = hy_u32x4{0u, 0u, 0u, 0u};
        }
#pragma unroll
        for (int u = 0; u < UNROLL; ++u) acc = mfma32(__builtin_bit_cast(hy_bf16x8, wf[u]), __builtin_bit_cast(hy_bf16x8, xf[u]), acc);
    }
    if (w) {
#pragma unroll
        for (int c = 0; c < 4; ++c) part[w - 1][c][lane] = hy_f32x4{acc[4 * c], acc[4 * c + 1], acc[4 * c + 2], acc[4 * c + 3]};
    }
    __syncthreads();
    if (w || m0 + j >= mend) return;
    // lane holds outputs 32 nb + 8 (v / 4) + 4 hl + v % 4 of row j
    uint16_t* y = (uint16_t*)a.y + (UP ? (int64_t)(m0 + j) : (int64_t)a.order[m0 + j]) * a.ys;
#pragma unroll
    for (int c = 0; c < 4; ++c) {
        hy_f32x4 f = {acc[4 * c], acc[4 * c + 1], acc[4 * c + 2], acc[4 * c + 3]};
#pragma unroll
        for (int x = 0; x < KS - 1; ++x) f += part[x][c][lane];
        store_outputs<UP>(a, y, nb * 32 + 8 * c + 4 * hl, f[0], f[1], f[2], f[3]);
    }
}

// bf16, many rows per expert (prompts): WM YT x 32 rows by WN XT x 32 outputs per workgroup of WM WN wavefronts, each XT x YT
// tiles of 32x32x16 MFMAs.  Steps of 32 k rotate through four LDS buffers filled by LDS-direct loads, three steps ahead: the
// weights lane-linear as they lie in memory, token rows gathered, the 16-byte piece c of row r at c ^ ((r / 4) % 4), so that
// the rows of a fragment read fall on different banks.
template <bool UP, int XT, int YT, int WN, int WM>
__global__ __launch_bounds__(WN * WM * 64) void grouped_big_kernel(GroupedArgs a, int n_tiles) {
    constexpr int THREADS = WN * WM * 64, TM = WM * YT * 32, TN = WN * XT * 32, RL = THREADS / 4, XB = TM * 64, BUF = (TM + TN) * 64;
    constexpr int XL = TM / RL, WL = TN / 16 / (WN * WM);
    static_assert(TM % RL == 0 && TN / 16 % (WN * WM) == 0, "whole loads");
    extern __shared__ __attribute__((aligned(16))) char gb_lds[];
    HY_LDS char* const lds3 = (HY_LDS char*)gb_lds;
    const uint32_t lds0 = (uint32_t)(uintptr_t)lds3;
    // an XCD takes a contiguous share of the row tiles and walks it in blocks of 4 row tiles x all outputs: the rows and the
    // weights that neighbouring workgroups read stay in its L2
    const int total = a.tiles[0], share = (total + 7) / 8, turn = blockIdx.x >> 3;
    const int blk = turn / (4 * n_tiles), in = turn - blk * 4 * n_tiles;
    const int first = blk * 4, rows_here = min(4, share - first);
    if (rows_here <= 0) return;
    const int nt = in / rows_here, rt = (blockIdx.x & 7) * share + first + in % rows_here;
    if (nt >= n_tiles || rt >= total) return;
    const int e = a.tiles[1 + 2 * rt], m0 = a.tiles[2 + 2 * rt], mend = a.offsets[e + 1], n0 = nt * TN;
    const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6), j = lane & 31, hl = lane >> 5;
    const int wm = w % WM, wn = w / WM, kb16 = a.kp >> 4;
    const uint16_t* xp[XL]; const char* wp[WL];
    const int lrow = tid >> 2, piece = ((tid & 3) ^ ((lrow >> 2) & 3)) * 8;       // RL is a multiple of 16: one swizzle for all loads
#pragma unroll
    for (int x = 0; x < XL; ++x) {
        const int i = min(m0 + x * RL + lrow, mend - 1);
        xp[x] = (const uint16_t*)a.x + (UP ? (int64_t)(a.order[i] / a.top) : (int64_t)i) * a.xs + piece;
    }
#pragma unroll
    for (int x = 0; x < WL; ++x) {                                                // block w WL + x of the step: outputs / 2, k half % 2
        const int b = w * WL + x, nb = min((n0 >> 5) + (b >> 1), (a.np >> 5) - 1);
        wp[x] = (const char*)a.w + (((int64_t)e * (a.np >> 5) + nb) * kb16 + (b & 1)) * 1024;
    }
    const uint32_t woff = lane * 16;
    const int steps = a.kp / 32;
    auto request = [&](int s, int buf) __attribute__((always_inline)) {
        const int sc = min(s, steps - 1);                                         // past the end: re-read, never used
        const uint32_t dst = lds0 + buf * BUF;
#pragma unroll
        for (int x = 0; x < XL; ++x) load_to_lds16(xp[x] + sc * 32, dst + x * RL * 64 + w * 1024);
#pragma unroll
        for (int x = 0; x < WL; ++x) load_to_lds16_at(wp[x] + (int64_t)sc * 2048, woff, dst + XB + (w * WL + x) * 1024);
    };
    hy_f32x16 acc[XT][YT];
#pragma unroll
    for (int x = 0; x < XT; ++x)
#pragma unroll
        for (int y = 0; y < YT; ++y)
#pragma unroll
            for (int v = 0; v < 16; ++v) acc[x][y][v] = 0.0f;
    const int sw = (j >> 2) & 3;
    HY_LDS char* const xr = lds3 + (wm * YT * 32 + j) * 64;
    HY_LDS char* const wr = lds3 + XB + wn * XT * 2048 + lane * 16;
    request(0, 0);
    request(1, 1);
    request(2, 2);
    for (int s = 0; s < steps; ++s) {
        asm volatile("s_waitcnt vmcnt(%0)" :: "n"(2 * (XL + WL)) : "memory");     // step s is here; two more are on their way
        __syncthreads();
        request(s + 3, (s + 3) & 3);
        const int off = (s & 3) * BUF;
        hy_bf16x8 xf[2][YT], wf[2][XT];
#pragma unroll
        for (int ks = 0; ks < 2; ++ks) {
            const int po = off + (((2 * ks + hl) ^ sw) << 4);
#pragma unroll
            for (int y = 0; y < YT; ++y) xf[ks][y] = *(const HY_LDS hy_bf16x8*)(xr + y * 2048 + po);
#pragma unroll
            for (int x = 0; x < XT; ++x) wf[ks][x] = *(const HY_LDS hy_bf16x8*)(wr + off + x * 2048 + ks * 1024);
        }
#pragma unroll
        for (int ks = 0; ks < 2; ++ks)
#pragma unroll
            for (int x = 0; x < XT; ++x)
#pragma unroll
                for (int y = 0; y < YT; ++y) acc[x][y] = mfma32(wf[ks][x], xf[ks][y], acc[x][y]);
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");       // nothing may land in LDS after the workgroup has gone
    // acc[x][y]: outputs n0 + (wn XT + x) 32 + 8 (v / 4) + 4 hl + v % 4 of row m0 + (wm YT + y) 32 + j
#pragma unroll
    for (int y = 0; y < YT; ++y) {
        const int i = m0 + (wm * YT + y) * 32 + j;
        if (i >= mend) continue;
        uint16_t* yr = (uint16_t*)a.y + (UP ? (int64_t)i : (int64_t)a.order[i]) * a.ys;
#pragma unroll
        for (int x = 0; x < XT; ++x)
#pragma unroll
            for (int c = 0; c < 4; ++c)
                store_outputs<UP>(a, yr, n0 + (wn * XT + x) * 32 + 8 * c + 4 * hl, acc[x][y][4 * c], acc[x][y][4 * c + 1], acc[x][y][4 * c + 2], acc[x][y][4 * c + 3]);
    }
}

template <bool UP, int XT, int YT, int WN, int WM>
static int launch_big(const GroupedArgs& a, int most, hipStream_t s) {
    constexpr int LDS = 4 * (WM * YT + WN * XT) * 32 * 64;
    static bool opted_in[64] = {};
    int dev = 0;
    if (hipGetDevice(&dev) != hipSuccess || dev < 0 || dev >= 64) dev = -1;
    if (dev < 0 || !opted_in[dev]) {
        hipError_t e = hipFuncSetAttribute((const void*)grouped_big_kernel<UP, XT, YT, WN, WM>, hipFuncAttributeMaxDynamicSharedMemorySize, LDS);
        if (e != hipSuccess) return (int)e;
        if (dev >= 0) opted_in[dev] = true;
    }
    const int n_tiles = (a.np + WN * XT * 32 - 1) / (WN * XT * 32), blocks = 8 * (((most + 7) / 8 + 3) / 4) * 4 * n_tiles;
    hipLaunchKernelGGL((grouped_big_kernel<UP, XT, YT, WN, WM>), dim3(blocks), dim3(WN * WM * 64), LDS, s, a, n_tiles);
    return 0;
}

}  // namespace trimkv

using namespace trimkv;

extern "C" const char* trimkv_moe_last_error(void) { return err_buf(); }

extern "C" int trimkv_moe_route(const float* logits, const float* correction, int32_t* ids, float* weights, int tokens, int experts, int top, int groups,
                                int keep_groups, void* stream) {
    const char* fn = "trimkv_moe_route";
    if (!logits || !correction || !ids || !weights) return fail(TRIMKV_ERR_NULL, "%s: null pointer argument", fn);
    if (tokens <= 0 || experts <= 0 || experts > ROUTE_MAX_E || groups <= 0 || experts % groups || keep_groups < 1 || keep_groups > groups || top < 1 ||
        top > keep_groups * (experts / groups))
        return fail(TRIMKV_ERR_SHAPE, "%s: bad sizes tokens=%d experts=%d top=%d groups=%d keep=%d", fn, tokens, experts, top, groups, keep_groups);
    auto go = [&](auto ne) {
        hipLaunchKernelGGL((route_kernel<decltype(ne)::value>), dim3((tokens + 3) / 4), dim3(256), 4 * (experts + groups) * sizeof(float), (hipStream_t)stream,
                           logits, correction, ids, weights, tokens, experts, top, groups, keep_groups);
    };
    if (experts <= 64) go(std::integral_constant<int, 1>{});
    else if (experts <= 128) go(std::integral_constant<int, 2>{});
    else if (experts <= 256) go(std::integral_constant<int, 4>{});
    else go(std::integral_constant<int, ROUTE_MAX_E / 64>{});
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
    if (dtype == TRIMKV_F32 ? tile != 16 : tile != 32 && tile != 256) return fail(TRIMKV_ERR_SHAPE, "%s: row tiles of 16 in fp32, of 32 or 256 in bf16 (got %d)", fn, tile);
    if (((uintptr_t)x | (uintptr_t)w | (uintptr_t)y) & 15 || x_stride % 8) return fail(TRIMKV_ERR_SHAPE, "%s: x, w and y must be 16-byte aligned", fn);
    GroupedArgs a{x, x_stride, w, y, y_stride, order, offsets, tiles, top, n, n_padded, k_padded};
    hipStream_t s = (hipStream_t)stream;
    const int most = rows < experts ? rows : (rows - experts) / tile + experts;     // no more row tiles than this
    const dim3 grid(most, n_padded / 64);
    if (tile == 256) {
        const int rc = up ? launch_big<true, 2, 4, 4, 2>(a, most, s) : launch_big<false, 2, 4, 4, 2>(a, most, s);
        if (rc) return fail(rc, "%s: hipFuncSetAttribute failed (%d)", fn, rc);
    } else if (dtype == TRIMKV_BF16) {
        const dim3 g(most, n_padded / 32);
        if ((int64_t)most * n_padded / 32 < 2048) {
            if (up) hipLaunchKernelGGL((grouped_skinny_kernel<true, 8>), g, dim3(512), 0, s, a);
            else hipLaunchKernelGGL((grouped_skinny_kernel<false, 8>), g, dim3(512), 0, s, a);
        } else {
            if (up) hipLaunchKernelGGL((grouped_skinny_kernel<true, 4>), g, dim3(256), 0, s, a);
            else hipLaunchKernelGGL((grouped_skinny_kernel<false, 4>), g, dim3(256), 0, s, a);
        }
    } else {
        if (up) hipLaunchKernelGGL((grouped_f32_kernel<true>), grid, dim3(256), 0, s, a);
        else hipLaunchKernelGGL((grouped_f32_kernel<false>), grid, dim3(256), 0, s, a);
    }
    return launch_status(fn);
}
