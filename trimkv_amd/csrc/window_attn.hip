// Sliding-window attention of prompts and their portions -- gfx950 (masks, ring and arithmetic: window.hip.h).
//
//   window_prefill_kernel  on the matrix cores (bf16): keys are the ring (what earlier portions left) and then the portion's own
//                          rows; tiles that no query of the workgroup sees are skipped
//   window_rows_kernel     the same for fp32 and for head sizes beyond the tiles: one wavefront per query
//
// In the prefill kernel the probabilities enter the second product as two bf16 terms each (17 bits).
#include "window.hip.h"

namespace trimkv {

// ---- general form: one wavefront per (token, query head) ---------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void window_rows_kernel(WindowArgs a) {
    const int b = blockIdx.y, lane = threadIdx.x & 63;
    const int t0 = a.cu[b], len = a.cu[b + 1] - t0;
    const int unit = blockIdx.x * 4 + (threadIdx.x >> 6);
    const int t = unit / a.H, h = unit - t * a.H;
    if (t >= len) return;
    const int g = h / (a.H / a.G), slot = a.slots[b], past = a.seen[2 * slot], i = past + t;
    const int cap = a.keep + a.size, nring = min(past, cap), nkeys = nring + t + 1;
    const T* q = (const T*)a.q + ((int64_t)(t0 + t) * a.H + h) * a.Dp;
    const T* rk = (const T*)a.rk + ((int64_t)slot * a.G + g) * cap * a.Dp;
    const T* rv = (const T*)a.rv + ((int64_t)slot * a.G + g) * cap * a.Dvp;
    const T* pk = (const T*)a.k + ((int64_t)t0 * a.G + g) * a.Dp;
    const T* pv = (const T*)a.v + ((int64_t)t0 * a.G + g) * a.Dvp;
    float m = WA_NEG, l = 0.0f, acc[8];
#pragma unroll
    for (int c = 0; c < 8; ++c) acc[c] = 0.0f;
    for (int base = 0; base < nkeys; base += 64) {
        const int x = base + lane;
        const int pos = x < nring ? ring_position(x, past, a.keep, a.size) : past + x - nring;
        const bool see = x < nkeys && (i - pos < a.size || pos < a.keep);
        if (__builtin_amdgcn_ballot_w64(see) == 0) continue;
        float s = WA_NEG;
        if (see) {
            const T* kr = x < nring ? rk + (int64_t)x * a.Dp : pk + (int64_t)(x - nring) * a.G * a.Dp;
            float d = 0.0f;
            for (int e = 0; e < a.D; ++e) d += ld(q + e) * ld(kr + e);
            s = d * a.scale_log2;
        }
        const float mn = fmaxf(m, wave_max_f(s)), alpha = exp2f(m - mn);
        const float p = see ? exp2f(s - mn) : 0.0f;
        m = mn;
        l = l * alpha + wave_sum_f(p);
#pragma unroll
        for (int c = 0; c < 8; ++c) acc[c] *= alpha;
        const int cnt = min(64, nkeys - base);
        for (int y = 0; y < cnt; ++y) {
            const float py = __shfl(p, y, 64);
            if (py == 0.0f) continue;                 // wavefront-uniform
            const int xx = base + y;
            const T* vr = xx < nring ? rv + (int64_t)xx * a.Dvp : pv + (int64_t)(xx - nring) * a.G * a.Dvp;
#pragma unroll
            for (int c = 0; c < 8; ++c)
                if (c * 64 + lane < a.Dv) acc[c] += py * ld(vr + c * 64 + lane);
        }
    }
    const float inv = 1.0f / (l + window_sink(a, m));
    T* o = (T*)a.out + ((int64_t)(t0 + t) * a.H + h) * a.Dv;
#pragma unroll
    for (int c = 0; c < 8; ++c) {
        const int d = c * 64 + lane;
        if (d < a.Dv) st(o + d, acc[c] * inv * window_gate<T>(a, t0 + t, h, d));
    }
}

// ---- prompts on the matrix cores -------------------------------------------------------------------
// A workgroup owns 128 rows = consecutive query times x the query heads of one KV head, 32 rows per wavefront.  Per tile of
// 64 keys a wavefront computes S^T[key][row] = K . Q^T and O^T[d][row] += V^T . P^T on 32x32x16 MFMAs: the row is the MFMA
// column (lane % 32), so maxima and sums live in the lane that needs them and the probabilities a lane holds after the first
// product are its operand of the second.  Layout (half hl = lane / 32): A, B hold k = 8 hl + 0..7 of row / column lane % 32;
// register v of C holds row 8 (v / 4) + 4 hl + v % 4.  Tiles come by LDS-direct loads, two buffers in turn.
//   K: 16-byte piece c of row r sits at c ^ swz(r), so that the rows of a fragment read fall on different banks
//   V: row-major too, read with ds_read_b64_tr_b16 (4 keys of one d per lane); its 32-byte pairs are swizzled by row
template <int D>
struct WindowTile {
    static constexpr int BN = 64, PIECES = D / 8, TILE = BN * D * 2, LOADS = BN * PIECES / 256;
    static __device__ __forceinline__ int kswz(int r) { return D == 64 ? (r >> 1) & 7 : r & 15; }
    static __device__ __forceinline__ int vswz(int r) { return D == 64 ? 4 * ((r >> 1) & 1) : 4 * (r & 3); }   // in 16-byte pieces
};

// Tiles are laid out for D features; products stop at USED of them.
template <int D, int USED>
__global__ __launch_bounds__(256, D <= 128 ? 2 : 1) void window_prefill_kernel(WindowArgs a) {
    using W = WindowTile<D>;
    constexpr int KS = USED / 16, DB = USED / 32;
    extern __shared__ __attribute__((aligned(16))) char wa_lds[];
    HY_LDS char* const lds3 = (HY_LDS char*)wa_lds;
    const uint32_t lds0 = (uint32_t)(uintptr_t)lds3;
    const int tid = threadIdx.x, lane = tid & 63;
    const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int j = lane & 31, hl = lane >> 5;
    // workgroups go to the 8 XCDs in turn; the tiles of one (sequence, KV head) read the same keys, so they share an XCD
    int pair = blockIdx.y, tile = (int)gridDim.x - 1 - (int)blockIdx.x;
    if ((gridDim.y & 7) == 0) {
        const int lin = (int)blockIdx.y * (int)gridDim.x + (int)blockIdx.x, turn = lin >> 3;
        pair = (lin & 7) + 8 * (turn / (int)gridDim.x);
        tile = (int)gridDim.x - 1 - turn % (int)gridDim.x;
    }
    const int b = pair / a.G, g = pair - b * a.G;
    const int tok0 = a.cu[b], len = a.cu[b + 1] - tok0;
    const int per = a.H / a.G, BT = 128 / per, q0 = tile * BT;
    if (q0 >= len) return;                                        // workgroup-uniform, before any barrier
    const int slot = a.slots[b], past = a.seen[2 * slot], cap = a.keep + a.size, nring = min(past, cap);
    const int r = w * 32 + j, t = q0 + r / per, h = g * per + r % per;
    const bool ok = r < BT * per && t < len;
    const int tc = min(t, len - 1), i = past + tc;
    const int q1 = min(len - 1, q0 + BT - 1);                     // the workgroup's last query time
    const int tw0 = min(q0 + (w * 32) / per, len - 1), tw1 = min(q0 + (w * 32 + 31) / per, q1);

    const bf16_t* Q = (const bf16_t*)a.q + ((int64_t)(tok0 + tc) * a.H + h) * a.Dp;
    hy_bf16x8 qf[KS];
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
        const int e0 = ks * 16 + hl * 8;
        const hy_u32x4 raw = *(const hy_u32x4*)(Q + min(e0, a.Dp - 8));
        qf[ks] = __builtin_bit_cast(hy_bf16x8, e0 < a.Dp ? raw : hy_u32x4{0u, 0u, 0u, 0u});
    }
    hy_f32x16 o[DB];
#pragma unroll
    for (int db = 0; db < DB; ++db)
#pragma unroll
        for (int v = 0; v < 16; ++v) o[db][v] = 0.0f;
    float m = WA_NEG, l = 0.0f;

    const char* rk = (const char*)a.rk + ((int64_t)slot * a.G + g) * cap * a.Dp * 2;
    const char* rv = (const char*)a.rv + ((int64_t)slot * a.G + g) * cap * a.Dvp * 2;
    const char* pk = (const char*)a.k + ((int64_t)tok0 * a.G + g) * a.Dp * 2;
    const char* pv = (const char*)a.v + ((int64_t)tok0 * a.G + g) * a.Dvp * 2;

    // tiles: the ring, then the portion's kept rows, then its window
    const int nr = (nring + 63) / 64;
    const int nkept = (max(0, min(a.keep - past, q1 + 1)) + 63) / 64;
    const int wt0 = max(nkept, max(0, q0 - a.size + 1) / 64);
    const int total = nr + nkept + max(0, q1 / 64 + 1 - wt0);
    // a load instruction of the workgroup covers RL rows; what a lane fetches of them does not depend on the tile, so a tile
    // whose rows all exist needs scalar addresses only
    constexpr int RL = 256 / W::PIECES;
    const int lrow = tid / W::PIECES, lpos = tid % W::PIECES;
    int kcol[2], vcol[2];                                  // swizzles repeat after 16 rows
#pragma unroll
    for (int x = 0; x < 2; ++x) {
        kcol[x] = min((lpos ^ W::kswz(lrow + x * RL)) * 16, a.Dp * 2 - 16);
        vcol[x] = min((lpos ^ W::vswz(lrow + x * RL)) * 16, a.Dvp * 2 - 16);
    }
    auto request = [&](int n, int buf) __attribute__((always_inline)) {
        const bool ring = n < nr;
        const int k0 = 64 * (ring ? n : n - nr < nkept ? n - nr : wt0 + n - nr - nkept);
        const int last = ring ? nring - 1 : len - 1;
        const char* kb = ring ? rk : pk;
        const char* vb = ring ? rv : pv;
        const int ks = ring ? a.Dp * 2 : a.G * a.Dp * 2, vs = ring ? a.Dvp * 2 : a.G * a.Dvp * 2;
        const uint32_t dst = lds0 + buf * 2 * W::TILE + w * 1024;
        if (k0 + 63 <= last) {
            const char* kt = kb + (int64_t)k0 * ks;
            const char* vt = vb + (int64_t)k0 * vs;
            const uint32_t ko = lrow * ks, vo = lrow * vs;
#pragma unroll
            for (int x = 0; x < W::LOADS; ++x) {
                load_to_lds16_at(kt + x * RL * ks, ko + kcol[x & 1], dst + x * 4096);
                load_to_lds16_at(vt + x * RL * vs, vo + vcol[x & 1], dst + W::TILE + x * 4096);
            }
        } else {
#pragma unroll
            for (int x = 0; x < W::LOADS; ++x) {
                const int64_t key = min(k0 + x * RL + lrow, last);
                load_to_lds16(kb + key * ks + kcol[x & 1], dst + x * 4096);
                load_to_lds16(vb + key * vs + vcol[x & 1], dst + W::TILE + x * 4096);
            }
        }
    };
    const int kx = 4 * hl + ((lane & 15) >> 2), jh = (lane >> 4) & 1;   // the transposing read: key of this lane, half of the 32 d
    auto k_frag = [&](int off, int blk, int ks) __attribute__((always_inline)) {
        const int row = blk * 32 + j;
        return *(const HY_LDS hy_bf16x8*)(lds3 + off + row * (D * 2) + (((2 * ks + hl) ^ W::kswz(j)) << 4));
    };
    auto v_frag = [&](int off, int st_, int db) __attribute__((always_inline)) {
        HY_LDS char* p = lds3 + off + W::TILE + (st_ * 16 + kx) * (D * 2) + ((((2 * db + jh) * 2) ^ W::vswz(kx)) << 4) + (lane & 3) * 8;
        const hy_s16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((HY_LDS hy_s16x4*)p);
        const hy_s16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((HY_LDS hy_s16x4*)(p + 8 * D * 2));
        return __builtin_bit_cast(hy_bf16x8, __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7));
    };

    request(0, 0);
    for (int n = 0; n < total; ++n) {
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();                                   // tile n is complete, tile n - 1 is no longer read
        if (n + 1 < total) request(n + 1, (n + 1) & 1);
        const bool ring = n < nr;
        const int k0 = 64 * (ring ? n : n - nr < nkept ? n - nr : wt0 + n - nr - nkept);
        if (!ring && k0 > tw1) continue;                   // wavefront-uniform: nothing of the tile is visible yet
        if (!ring && k0 + 63 <= tw0 - a.size && past + k0 >= a.keep) continue;   // ... or any more
        const int off = (n & 1) * 2 * W::TILE;
        // operands are requested AHEAD steps before the MFMA that takes them; the fences keep the compiler from moving them back
        constexpr int AHEAD = 3;
        __builtin_amdgcn_s_setprio(1);                     // the wavefront that can feed the matrix cores goes first
        hy_f32x16 s[2];
#pragma unroll
        for (int v = 0; v < 16; ++v) s[0][v] = s[1][v] = 0.0f;
        {
            hy_bf16x8 kf[2 * KS];
#pragma unroll
            for (int x = 0; x < AHEAD; ++x) kf[x] = k_frag(off, x & 1, x >> 1);
#pragma unroll
            for (int x = 0; x < 2 * KS; ++x) {
                if (x + AHEAD < 2 * KS) kf[x + AHEAD] = k_frag(off, (x + AHEAD) & 1, (x + AHEAD) >> 1);
                s[x & 1] = mfma32(kf[x], qf[x >> 1], s[x & 1]);
                __builtin_amdgcn_sched_barrier(0);
            }
        }
        hy_bf16x8 vf[4 * DB];
#pragma unroll
        for (int x = 0; x < AHEAD; ++x) vf[x] = v_frag(off, x / DB, x % DB);
        __builtin_amdgcn_s_setprio(0);
        const bool whole = !ring && k0 + 63 <= tw0 && (k0 > tw1 - a.size || past + k0 + 63 < a.keep);
        if (!whole) {
            asm volatile("" :::);                          // keeps this a branch
            if (ring) {
#pragma unroll 1
                for (int v = 0; v < 16; ++v) {
                    // (rarely taken: a loop over registers through a compare, not 32 copies of the slot arithmetic)
                    const int x = k0 + 8 * (v >> 2) + 4 * hl + (v & 3);
                    bool see[2];
#pragma unroll
                    for (int blk = 0; blk < 2; ++blk) {
                        const int slot_ = x + 32 * blk, pos = ring_position(slot_, past, a.keep, a.size);
                        see[blk] = slot_ < nring && (i - pos < a.size || pos < a.keep);
                    }
#pragma unroll
                    for (int u = 0; u < 16; ++u) {
                        s[0][u] = u == v && !see[0] ? WA_NEG : s[0][u];
                        s[1][u] = u == v && !see[1] ? WA_NEG : s[1][u];
                    }
                }
            } else {
                const int x1 = i - past, x0 = x1 - a.size, xk = a.keep - past;    // rows up to x1 and beyond x0 or below xk
#pragma unroll
                for (int blk = 0; blk < 2; ++blk)
#pragma unroll
                    for (int v = 0; v < 16; ++v) {
                        const int x = k0 + blk * 32 + 8 * (v >> 2) + 4 * hl + (v & 3);
                        const bool see = (x <= x1) & ((x > x0) | (x < xk));
                        s[blk][v] = see ? s[blk][v] : WA_NEG;
                    }
            }
        }
        float tm = s[0][0];
#pragma unroll
        for (int v = 0; v < 16; ++v) tm = fmaxf(tm, fmaxf(s[0][v], s[1][v]));
        tm = tm > 0.5f * WA_NEG ? tm * a.scale_log2 : WA_NEG;
        // the reference moves only when some row outgrows it by 2^6 (or has none yet)
        if (__builtin_amdgcn_ballot_w64(tm > m + 6.0f) != 0) {
            const float mn = fmaxf(m, fmaxf(tm, __shfl_xor(tm, 32, 64)));
            const float alpha = __builtin_amdgcn_exp2f(m - mn);
            m = mn;
            l *= alpha;
#pragma unroll
            for (int db = 0; db < DB; ++db)
#pragma unroll
                for (int v = 0; v < 16; ++v) o[db][v] *= alpha;
        }
        const float ref = m > 0.5f * WA_NEG ? m : 0.0f;    // a row that has seen nothing: its scores give exp2(-huge) = 0
        const float sc = a.scale_log2;
        // the exponentials of the next 16 keys run between the MFMAs of these
        hy_u32x4 hi[2], lo[2];
        auto weigh = [&](int st_, int x) __attribute__((always_inline)) {
            const int v = (st_ & 1) * 8 + 2 * x;
            const float p0 = __builtin_amdgcn_exp2f(fmaf(s[st_ >> 1][v], sc, -ref)), p1 = __builtin_amdgcn_exp2f(fmaf(s[st_ >> 1][v + 1], sc, -ref));
            l += p0 + p1;
            uint32_t tw[2];
            split2<2>(p0, p1, tw);
            hi[st_ & 1][x] = tw[0]; lo[st_ & 1][x] = tw[1];
        };
#pragma unroll
        for (int x = 0; x < 4; ++x) weigh(0, x);
        __builtin_amdgcn_s_setprio(1);
#pragma unroll
        for (int st_ = 0; st_ < 4; ++st_) {
#pragma unroll
            for (int db = 0; db < DB; ++db) {
                const int x = st_ * DB + db;
                if (x + AHEAD < 4 * DB) vf[x + AHEAD] = v_frag(off, (x + AHEAD) / DB, (x + AHEAD) % DB);
                o[db] = mfma32(vf[x], __builtin_bit_cast(hy_bf16x8, hi[st_ & 1]), o[db]);
                if (st_ < 3 && db < 2) weigh(st_ + 1, db);
                __builtin_amdgcn_sched_barrier(0);
            }
#pragma unroll
            for (int db = 0; db < DB; ++db) {
                o[db] = mfma32(vf[st_ * DB + db], __builtin_bit_cast(hy_bf16x8, lo[st_ & 1]), o[db]);
                if (st_ < 3 && db < 2) weigh(st_ + 1, 2 + db);
                __builtin_amdgcn_sched_barrier(0);
            }
        }
        __builtin_amdgcn_s_setprio(0);
    }
    l += __shfl_xor(l, 32, 64);                            // the halves of a row hold disjoint keys
    if (!ok) return;
    float inv = 1.0f / (l + window_sink(a, m));
    const bf16_t* gr = (const bf16_t*)a.gate + (int64_t)(tok0 + t) * a.gate_stride + h * a.Dv;
    if (a.head_gate) inv *= window_gate<bf16_t>(a, tok0 + t, h, 0);
    bf16_t* orow = (bf16_t*)a.out + ((int64_t)(tok0 + t) * a.H + h) * a.Dv;
#pragma unroll
    for (int db = 0; db < DB; ++db) {
#pragma unroll
        for (int c = 0; c < 4; ++c) {
            const int d = db * 32 + 8 * c + 4 * hl;
            if (a.vec) {
                if (d >= a.Dv) continue;
                if (a.head_gate) st4(orow + d, make_float4(o[db][4 * c] * inv, o[db][4 * c + 1] * inv, o[db][4 * c + 2] * inv, o[db][4 * c + 3] * inv));
                else {
                    const float4 gt = ld4(gr + d);
                    st4(orow + d, make_float4(o[db][4 * c] * inv * sigmoid_fast(gt.x), o[db][4 * c + 1] * inv * sigmoid_fast(gt.y),
                                              o[db][4 * c + 2] * inv * sigmoid_fast(gt.z), o[db][4 * c + 3] * inv * sigmoid_fast(gt.w)));
                }
            } else {
#pragma unroll
                for (int x = 0; x < 4; ++x)
                    if (d + x < a.Dv) st(orow + d + x, o[db][4 * c + x] * inv * (a.head_gate ? 1.0f : sigmoid_fast(ld(gr + d + x))));
            }
        }
    }
}

template <int D, int USED = D>
static int launch_window_prefill(const WindowArgs& a, int batch, int max_len, hipStream_t s) {
    constexpr int LDS = 4 * WindowTile<D>::TILE;
    static bool opted_in[64] = {};
    int dev = 0;
    if (hipGetDevice(&dev) != hipSuccess || dev < 0 || dev >= 64) dev = -1;
    if (dev < 0 || !opted_in[dev]) {
        hipError_t e = hipFuncSetAttribute((const void*)window_prefill_kernel<D, USED>, hipFuncAttributeMaxDynamicSharedMemorySize, LDS);
        if (e != hipSuccess) return (int)e;
        if (dev >= 0) opted_in[dev] = true;
    }
    const int bt = 128 / (a.H / a.G);
    hipLaunchKernelGGL((window_prefill_kernel<D, USED>), dim3((max_len + bt - 1) / bt, batch * a.G), dim3(256), LDS, s, a);
    return 0;
}

}  // namespace trimkv

using namespace trimkv;

extern "C" int trimkv_window_prefill(const void* q, const void* k, const void* v, const void* ring_k, const void* ring_v, const int32_t* cu,
                                     const int32_t* slots, const int32_t* seen, const void* gate, int64_t gate_stride, void* out, int batch, int max_len,
                                     int heads, int kv_heads, int dim, int vdim, int dim_stride, int vdim_stride, int keep_first, int window,
                                     float scale, int head_gate, int sink, int dtype, void* stream) {
    const char* fn = "trimkv_window_prefill";
    WindowArgs a{};
    a.q = q; a.k = k; a.v = v; a.rk = ring_k; a.rv = ring_v; a.cu = cu; a.slots = slots; a.seen = seen; a.gate = gate; a.gate_stride = gate_stride; a.out = out;
    a.H = heads; a.G = kv_heads; a.D = dim; a.Dv = vdim; a.Dp = dim_stride; a.Dvp = vdim_stride; a.keep = keep_first; a.size = window;
    a.scale_log2 = scale * 1.4426950408889634f; a.splits = 1; a.head_gate = head_gate; a.sink = sink;
    if (int rc = window_common(fn, a, batch, dtype)) return rc;
    if (!k || !v || !cu) return fail(TRIMKV_ERR_NULL, "%s: null pointer argument", fn);
    if (max_len <= 0 || (int64_t)batch * kv_heads > 65535) return fail(TRIMKV_ERR_SHAPE, "%s: bad sizes max_len=%d batch*kv_heads=%lld", fn, max_len, (long long)batch * kv_heads);
    hipStream_t s = (hipStream_t)stream;
    const int per = heads / kv_heads, big = dim_stride > vdim_stride ? dim_stride : vdim_stride;
    const bool aligned = !(((uintptr_t)k | (uintptr_t)v) & 15);
    if (dtype == TRIMKV_BF16 && big <= 256 && per <= 128 && aligned && scale > 0.0f) {
        a.vec = vdim % 4 == 0 && !((uintptr_t)out & 7) && (head_gate || (gate_stride % 4 == 0 && !((uintptr_t)gate & 7)));
        const int rc = big <= 64 ? launch_window_prefill<64>(a, batch, max_len, s) : big <= 96 ? launch_window_prefill<128, 96>(a, batch, max_len, s) : big <= 128 ? launch_window_prefill<128>(a, batch, max_len, s)
                                                                                               : launch_window_prefill<256>(a, batch, max_len, s);
        if (rc) return fail(rc, "%s: hipFuncSetAttribute failed (%d)", fn, rc);
        return launch_status(fn);
    }
    const int64_t units = (int64_t)max_len * heads;
    HY_BY_DTYPE(dtype, T, hipLaunchKernelGGL((window_rows_kernel<T>), dim3((unsigned)((units + 3) / 4), batch), dim3(256), 0, s, a));
    return launch_status(fn);
}
