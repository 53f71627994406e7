// Sliding-window attention of one new token per sequence -- gfx950 (masks, ring and arithmetic: window.hip.h).
//
//   window_decode_kernel   walks the rows in use in storage order without any mask; rows split over workgroups (split-K), all
//                          query heads of a KV head share the rows; 64 / L rows per load instruction, L lanes with 8 features
//                          each per row
//   window_combine_kernel  the splits' shares
#include "window.hip.h"
#include <type_traits>

namespace trimkv {

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
