// Sliding-window attention with kept first tokens over a ring of keys and values -- gfx950.
//
// Position i sees j iff j <= i and (i - j < size or j < keep).  Keys arrive as they are scored (rotated, if at all), so a sequence needs
// exactly keep + size rows however long it is: the first `keep` tokens own their rows, later ones overwrite the row of the
// token that has just left the window.  After a token is stored, the rows in use are its visible set, and the decode kernel
// walks them in storage order without any mask.
//
//   window_decode_kernel   one new token per sequence; rows split over workgroups (split-K), all query heads of a KV head
//                          share the rows; 64 / L rows per load instruction, L lanes with 8 features each per row
//   window_prefill_kernel  prompts and their portions on the matrix cores (bf16): keys are the ring (what earlier portions
//                          left) and then the portion's own rows; tiles that no query of the workgroup sees are skipped
//   window_rows_kernel     the same for fp32 and for head sizes beyond the tiles: one wavefront per query
//
// Scores, maxima, exponentials and sums are fp32; scores are scaled after the product.  In the prefill kernel the
// probabilities enter the second product as two bf16 terms each (17 bits).  The sigmoid output gate (a number per value or one
// per head) is applied on the way out.  With a sink the denominator has one more term, a score of 0 without a value.
#include "hybrid.hip.h"
#include <type_traits>

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

// ---- decode --------------------------------------------------------------------------------------
template <int CTRL>
__device__ __forceinline__ float dpp_add(float v) {
    return v + __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xf, 0xf, true));
}
// sum over aligned groups of L lanes, result in every lane
template <int L>
__device__ __forceinline__ float group_sum(float v) {
    v = dpp_add<0xB1>(v);                        // quad_perm 1,0,3,2
    v = dpp_add<0x4E>(v);                        // quad_perm 2,3,0,1
    if constexpr (L >= 8) v = dpp_add<0x141>(v); // row_half_mirror
    if constexpr (L >= 16) v = dpp_add<0x140>(v);// row_mirror
    if constexpr (L >= 32) v += __shfl_xor(v, 16, 64);
    if constexpr (L >= 64) v += __shfl_xor(v, 32, 64);
    return v;
}

struct Row8 { float f[8]; };
__device__ __forceinline__ hy_u32x4 raw8(const bf16_t* p) { return __builtin_nontemporal_load((const hy_u32x4*)p); }
__device__ __forceinline__ void widen(hy_u32x4 r, float (&f)[8]) {
#pragma unroll
    for (int x = 0; x < 4; ++x) { f[2 * x] = __uint_as_float(r[x] << 16); f[2 * x + 1] = __uint_as_float(r[x] & 0xffff0000u); }
}
struct Raw8f { float4 lo, hi; };
__device__ __forceinline__ Raw8f raw8(const float* p) { return {*(const float4*)p, *(const float4*)(p + 4)}; }
__device__ __forceinline__ void widen(Raw8f r, float (&f)[8]) {
    f[0] = r.lo.x; f[1] = r.lo.y; f[2] = r.lo.z; f[3] = r.lo.w; f[4] = r.hi.x; f[5] = r.hi.y; f[6] = r.hi.z; f[7] = r.hi.w;
}

template <typename T, int L, int GQ>
__global__ __launch_bounds__(256) void window_decode_kernel(WindowArgs a) {
    constexpr int R = 64 / L, U = GQ >= 8 ? 2 : 4, WAVES = 4;
    extern __shared__ float lds[];                  // [WAVES][GQ][L * 8 + 2]
    const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
    const int per = a.H / a.G, passes = (per + GQ - 1) / GQ;
    const int split = blockIdx.x, g = blockIdx.y / passes, h0 = (blockIdx.y % passes) * GQ, b = blockIdx.z;
    const int nh = min(GQ, per - h0);
    const int slot = a.slots[b], cap = a.keep + a.size;
    const int n = min(a.seen[2 * slot] + 1, cap);
    const int r0 = split * a.chunk, r1 = min(n, r0 + a.chunk);
    const int e = (lane % L) * 8, sub = lane / L;
    const bool kin = e < a.Dp, vin = e < a.Dvp;     // padded dims are multiples of 8
    const T* rk = (const T*)a.rk + ((int64_t)slot * a.G + g) * cap * a.Dp + (kin ? e : 0);
    const T* rv = (const T*)a.rv + ((int64_t)slot * a.G + g) * cap * a.Dvp + (vin ? e : 0);
    float q[GQ][8];
#pragma unroll
    for (int x = 0; x < GQ; ++x) {
        widen(raw8((const T*)a.q + ((int64_t)b * a.H + g * per + h0 + min(x, nh - 1)) * a.Dp + (kin ? e : 0)), q[x]);
#pragma unroll
        for (int y = 0; y < 8; ++y) q[x][y] = kin ? q[x][y] * a.scale_log2 : 0.0f;
    }
    float m[GQ], l[GQ], acc[GQ][8];
#pragma unroll
    for (int x = 0; x < GQ; ++x) {
        m[x] = WA_NEG; l[x] = 0.0f;
#pragma unroll
        for (int y = 0; y < 8; ++y) acc[x][y] = 0.0f;
    }
    using Raw = decltype(raw8((const T*)nullptr));
    for (int base = r0 + wv * R * U; base < r1; base += WAVES * R * U) {
        Raw kr[U], vr[U];
#pragma unroll
        for (int u = 0; u < U; ++u) kr[u] = raw8(rk + (int64_t)min(base + u * R + sub, r1 - 1) * a.Dp);
#pragma unroll
        for (int u = 0; u < U; ++u) vr[u] = raw8(rv + (int64_t)min(base + u * R + sub, r1 - 1) * a.Dvp);
        float s[U][GQ];
#pragma unroll
        for (int u = 0; u < U; ++u) {
            float kf[8];
            widen(kr[u], kf);
            const bool in = base + u * R + sub < r1;
#pragma unroll
            for (int x = 0; x < GQ; ++x) {
                float d = 0.0f;
#pragma unroll
                for (int y = 0; y < 8; ++y) d = fmaf(q[x][y], kf[y], d);
                d = group_sum<L>(d);
                s[u][x] = in ? d : WA_NEG;
            }
        }
#pragma unroll
        for (int x = 0; x < GQ; ++x) {
            float mn = m[x];
#pragma unroll
            for (int u = 0; u < U; ++u) mn = fmaxf(mn, s[u][x]);
            const float alpha = __builtin_amdgcn_exp2f(m[x] - mn);
            m[x] = mn;
            float ps = 0.0f;
#pragma unroll
            for (int u = 0; u < U; ++u) { s[u][x] = s[u][x] > 0.5f * WA_NEG ? __builtin_amdgcn_exp2f(s[u][x] - mn) : 0.0f; ps += s[u][x]; }
            l[x] = l[x] * alpha + ps;
#pragma unroll
            for (int y = 0; y < 8; ++y) acc[x][y] *= alpha;
        }
#pragma unroll
        for (int u = 0; u < U; ++u) {
            float vf[8];
            widen(vr[u], vf);
#pragma unroll
            for (int x = 0; x < GQ; ++x)
#pragma unroll
                for (int y = 0; y < 8; ++y) acc[x][y] = fmaf(s[u][x], vf[y], acc[x][y]);
        }
    }
    // lanes that hold the same features of different rows meet, then the wavefronts
    constexpr int ROW = L * 8 + 2;
#pragma unroll
    for (int x = 0; x < GQ; ++x) {
#pragma unroll
        for (int d = L; d < 64; d <<= 1) {
            const float mo = __shfl_xor(m[x], d, 64), lo = __shfl_xor(l[x], d, 64), mn = fmaxf(m[x], mo);
            const float f0 = __builtin_amdgcn_exp2f(m[x] - mn), f1 = __builtin_amdgcn_exp2f(mo - mn);
            m[x] = mn;
            l[x] = l[x] * f0 + lo * f1;
#pragma unroll
            for (int y = 0; y < 8; ++y) acc[x][y] = acc[x][y] * f0 + __shfl_xor(acc[x][y], d, 64) * f1;
        }
        float* row = lds + (wv * GQ + x) * ROW;
        if (sub == 0) {
#pragma unroll
            for (int y = 0; y < 8; ++y) row[e + y] = acc[x][y];
            if (lane == 0) { row[L * 8] = m[x]; row[L * 8 + 1] = l[x]; }
        }
    }
    __syncthreads();
    for (int idx = tid; idx < nh * a.Dv; idx += 256) {
        const int x = idx / a.Dv, d = idx - x * a.Dv;
        float mm = WA_NEG;
#pragma unroll
        for (int w = 0; w < WAVES; ++w) mm = fmaxf(mm, lds[(w * GQ + x) * ROW + L * 8]);
        float num = 0.0f, den = 0.0f;
#pragma unroll
        for (int w = 0; w < WAVES; ++w) {
            const float* row = lds + (w * GQ + x) * ROW;
            const float f = __builtin_amdgcn_exp2f(row[L * 8] - mm);
            num += row[d] * f;
            den += row[L * 8 + 1] * f;
        }
        const int h = g * per + h0 + x;
        if (a.splits == 1) {
            st((T*)a.out + ((int64_t)b * a.H + h) * a.Dv + d, num / (den + window_sink(a, mm)) * window_gate<T>(a, b, h, d));
        } else {
            float* w = a.ws + (((int64_t)b * a.H + h) * a.splits + split) * (a.Dv + 2);
            w[d] = num;
            if (d == 0) { w[a.Dv] = mm; w[a.Dv + 1] = den; }
        }
    }
}

template <typename T>
__global__ __launch_bounds__(256) void window_combine_kernel(WindowArgs a) {
    __shared__ float f[256];                        // a split's share of the result
    __shared__ float part[4];
    const int64_t bh = blockIdx.x;
    const int64_t b = bh / a.H;
    const int h = (int)(bh - b * a.H), tid = threadIdx.x, row = a.Dv + 2;
    const float* w = a.ws + bh * a.splits * row;
    const float m = tid < a.splits ? w[tid * row + a.Dv] : WA_NEG, l = tid < a.splits ? w[tid * row + a.Dv + 1] : 0.0f;
    const float wm = wave_max_f(m);
    if ((tid & 63) == 0) part[tid >> 6] = wm;
    __syncthreads();
    const float mm = fmaxf(fmaxf(part[0], part[1]), fmaxf(part[2], part[3]));
    __syncthreads();
    const float e = __builtin_amdgcn_exp2f(m - mm);
    const float inv = 1.0f / (block_sum_f(l * e, part, 4) + window_sink(a, mm));
    f[tid] = e * inv;
    __syncthreads();
    for (int d = tid; d < a.Dv; d += 256) {
        float num = 0.0f;
#pragma unroll 8
        for (int s = 0; s < a.splits; ++s) num += w[s * row + d] * f[s];
        st((T*)a.out + bh * a.Dv + d, num * window_gate<T>(a, b, h, d));
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

template <typename T, int L>
static void launch_window_decode(const WindowArgs& a, int batch, hipStream_t s) {
    const int per = a.H / a.G;
    auto go = [&](auto gq) {
        constexpr int GQ = decltype(gq)::value;
        const int passes = (per + GQ - 1) / GQ;
        hipLaunchKernelGGL((window_decode_kernel<T, L, GQ>), dim3(a.splits, a.G * passes, batch), dim3(256), 4 * GQ * (L * 8 + 2) * sizeof(float), s, a);
    };
    if (per == 1) go(std::integral_constant<int, 1>{});
    else if (per == 2) go(std::integral_constant<int, 2>{});
    else if (per <= 4 || L >= 64) go(std::integral_constant<int, 4>{});
    else go(std::integral_constant<int, 8>{});
}

static int window_common(const char* fn, const WindowArgs& a, int batch, int dtype) {
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

using namespace trimkv;

extern "C" int trimkv_window_decode_splits(int batch, int kv_heads, int capacity) {
    if (batch <= 0 || kv_heads <= 0 || capacity <= 0) return 1;
    // enough workgroups to fill the chip, at least 128 rows for each
    const int64_t pairs = (int64_t)batch * kv_heads;
    int64_t s = (2048 + pairs - 1) / pairs;
    const int most = (capacity + 127) / 128;
    s = s < 1 ? 1 : s > most ? most : s;
    return (int)(s > 256 ? 256 : s);
}

extern "C" int trimkv_window_decode(const void* q, const void* ring_k, const void* ring_v, const int32_t* slots, const int32_t* seen,
                                    const void* gate, int64_t gate_stride, void* out, int batch, int heads, int kv_heads, int dim, int vdim,
                                    int dim_stride, int vdim_stride, int keep_first, int window, float scale, int head_gate, int sink, int splits, float* workspace,
                                    int dtype, void* stream) {
    const char* fn = "trimkv_window_decode";
    WindowArgs a{};
    a.q = q; a.rk = ring_k; a.rv = ring_v; a.slots = slots; a.seen = seen; a.gate = gate; a.gate_stride = gate_stride; a.out = out;
    a.H = heads; a.G = kv_heads; a.D = dim; a.Dv = vdim; a.Dp = dim_stride; a.Dvp = vdim_stride; a.keep = keep_first; a.size = window;
    a.scale_log2 = scale * 1.4426950408889634f; a.splits = splits; a.ws = workspace; a.head_gate = head_gate; a.sink = sink;
    if (int rc = window_common(fn, a, batch, dtype)) return rc;
    if (splits < 1 || splits > 256 || (splits > 1 && !workspace)) return fail(TRIMKV_ERR_WORKSPACE, "%s: splits=%d needs a workspace", fn, splits);
    const int cap = keep_first + window;
    a.chunk = (cap + splits - 1) / splits;
    const int lanes = ((dim_stride > vdim_stride ? dim_stride : vdim_stride) + 7) / 8;
    hipStream_t s = (hipStream_t)stream;
    HY_BY_DTYPE(dtype, T,
        if (lanes <= 4) launch_window_decode<T, 4>(a, batch, s);
        else if (lanes <= 8) launch_window_decode<T, 8>(a, batch, s);
        else if (lanes <= 16) launch_window_decode<T, 16>(a, batch, s);
        else if (lanes <= 32) launch_window_decode<T, 32>(a, batch, s);
        else launch_window_decode<T, 64>(a, batch, s));
    int rc = launch_status(fn);
    if (rc || splits == 1) return rc;
    HY_BY_DTYPE(dtype, T, hipLaunchKernelGGL((window_combine_kernel<T>), dim3(batch * heads), dim3(256), 0, s, a));
    return launch_status(fn);
}

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
