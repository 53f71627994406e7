// The row-wise work of the hybrid decoders, one launch each; the residual stream is fp32.
//
//   trimkv_embed_scaled    x = table[id] * scale, or x += ..., optionally normed for the first sublayer
//   trimkv_linear_f32      fp32 rows times a narrow matrix with fp32 results (routers, gates of a recurrence)
//   trimkv_residual_norm   x += mult * w * rms(y), y one row or a weighted sum of several (the experts of a token); the new x
//                          or its norm for the next sublayer goes along in the matrices' dtype
//   trimkv_rms_rows        w * rms(x) of chosen rows
//   trimkv_qkv_norm        RMS norm over the whole q and the whole k projection; q, k, v into head-major padded rows, or k
//                          and v straight into the window ring (decode)
//   trimkv_rotary_table    cosines and sines of a step's positions, once for all layers that turn alike
//   trimkv_qkv_heads       bias, RMS norm per head and rotary positions; q, k, v go where trimkv_qkv_norm puts them
//   trimkv_silu_gate       silu(gate) * up
//   trimkv_soft_cap        cap * tanh(x / cap) in fp32
//   trimkv_ring_store      the rows of a prompt that outlive it, into the window ring
//   trimkv_head_norm_gate  per-head RMS norm, weight and sigmoid gate behind a recurrence
//   trimkv_advance         tokens and steps seen per sequence slot
#include "hybrid.hip.h"
#include <type_traits>

namespace trimkv {

// ---- embedding -------------------------------------------------------------------------------
struct EmbedArgs {
    const int64_t* ids; const void* table; float scale;
    float* x; void* xh; const float* norm_w; float eps;
    int vocab, width, xs, add;
};
template <typename T>
__global__ __launch_bounds__(256) void embed_kernel(EmbedArgs a) {
    __shared__ float part[4];
    const int64_t t = blockIdx.x;
    const int64_t id = min(max(a.ids[t], (int64_t)0), (int64_t)a.vocab - 1);
    const T* src = (const T*)a.table + id * a.width;
    float* xr = a.x + t * a.xs;
    T* hr = (T*)a.xh + t * a.xs;
    float ss = 0.0f;
    for (int i = threadIdx.x; i < a.xs; i += 256) {
        float f = i < a.width ? ld(src + i) * a.scale : 0.0f;
        if (a.add) f += xr[i];
        xr[i] = f;
        ss += f * f;
        if (a.xh && !a.norm_w) st(hr + i, f);
    }
    if (!a.norm_w) return;
    const float inv = 1.0f / sqrtf(block_sum_f(ss, part, 4) / (float)a.width + a.eps);
    for (int i = threadIdx.x; i < a.xs; i += 256)        // a thread re-reads what it wrote itself
        st(hr + i, i < a.width ? xr[i] * inv * a.norm_w[i] : 0.0f);
}
// width and stride multiples of 4, width up to 1024 NV: a row stays in registers
template <typename T, int NV>
__global__ __launch_bounds__(256) void embed_vec_kernel(EmbedArgs a) {
    __shared__ float part[4];
    const int64_t t = blockIdx.x;
    const int64_t id = min(max(a.ids[t], (int64_t)0), (int64_t)a.vocab - 1);
    const T* src = (const T*)a.table + id * a.width;
    float* xr = a.x + t * a.xs;
    T* hr = (T*)a.xh + t * a.xs;
    const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
    float4 f[NV];
    float ss = 0.0f;
#pragma unroll
    for (int v = 0; v < NV; ++v) {
        const int i = (v * 256 + threadIdx.x) * 4;
        f[v] = zero;
        if (i < a.width) {
            f[v] = ld4(src + i);
            f[v].x *= a.scale; f[v].y *= a.scale; f[v].z *= a.scale; f[v].w *= a.scale;
            if (a.add) {
                const float4 o = *(const float4*)(xr + i);
                f[v].x += o.x; f[v].y += o.y; f[v].z += o.z; f[v].w += o.w;
            }
        }
        if (i < a.xs) {
            *(float4*)(xr + i) = f[v];
            if (a.xh && !a.norm_w) st4(hr + i, f[v]);
        }
        ss += f[v].x * f[v].x + f[v].y * f[v].y + f[v].z * f[v].z + f[v].w * f[v].w;
    }
    if (!a.norm_w) return;
    const float inv = 1.0f / sqrtf(block_sum_f(ss, part, 4) / (float)a.width + a.eps);
#pragma unroll
    for (int v = 0; v < NV; ++v) {
        const int i = (v * 256 + threadIdx.x) * 4;
        if (i >= a.xs) continue;
        const float4 w = i < a.width ? *(const float4*)(a.norm_w + i) : zero;
        st4(hr + i, make_float4(f[v].x * inv * w.x, f[v].y * inv * w.y, f[v].z * inv * w.z, f[v].w * inv * w.w));
    }
}

// ---- fp32 rows times a narrow matrix ---------------------------------------------------------
// General form: one wavefront per (row, output).
template <typename T>
__global__ __launch_bounds__(256) void linear_f32_kernel(const float* x, int64_t xs, const T* w, int64_t ws, float* out, int64_t units, int n, int k) {
    const int64_t unit = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (unit >= units) return;
    const int64_t t = unit / n;
    const int o = (int)(unit - t * n), lane = threadIdx.x & 63;
    const float* xr = x + t * xs;
    const T* wr = w + o * ws;
    float acc = 0.0f;
    for (int i = lane * 4; i < k; i += 256) {
        const float4 a = ld4(xr + i), b = ld4(wr + i);
        acc += a.x * b.x + a.y * b.y + a.z * b.z + a.w * b.w;
    }
    acc = wave_sum_f(acc);
    if (lane == 0) out[unit] = acc;
}

// bf16 weights on the matrix cores: a row's fp32 values are split exactly into three bf16 terms, so every product is an
// fp32 product.  A workgroup owns 16 rows and 16 * NT outputs; its WAVES wavefronts split k and meet in LDS.
// Operands straight from memory: lane l holds 8 consecutive k of row (or output) l % 16 at k-group l / 16.
template <int NT, int WAVES>
__global__ __launch_bounds__(WAVES * 64) void linear_f32_mfma_kernel(const float* x, int64_t xs, const bf16_t* w, int64_t ws, float* out, int rows, int n, int k) {
    __shared__ float part[WAVES][NT][256];
    const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, r = lane & 15, kg = lane >> 4;
    const int row0 = blockIdx.x * 16, n0 = blockIdx.y * 16 * NT;
    const float* xr = x + (int64_t)min(row0 + r, rows - 1) * xs;
    const bf16_t* wr[NT];
#pragma unroll
    for (int j = 0; j < NT; ++j) wr[j] = w + (int64_t)min(n0 + 16 * j + r, n - 1) * ws;
    hy_f32x4 acc[NT];
#pragma unroll
    for (int j = 0; j < NT; ++j) acc[j] = {0.f, 0.f, 0.f, 0.f};
    constexpr int UN = NT == 1 ? 4 : 1;                 // k-steps whose operands are requested together
    for (int i0 = wv * 32; i0 < k; i0 += UN * WAVES * 32) {     // k is a multiple of 32
        float4 a[UN], b[UN];
        hy_u32x4 wf[UN][NT];
#pragma unroll
        for (int u = 0; u < UN; ++u) {
            const int i = min(i0 + u * WAVES * 32, k - 32) + kg * 8;
            a[u] = *(const float4*)(xr + i);
            b[u] = *(const float4*)(xr + i + 4);
#pragma unroll
            for (int j = 0; j < NT; ++j) wf[u][j] = *(const hy_u32x4*)(wr[j] + i);
        }
#pragma unroll
        for (int u = 0; u < UN; ++u) {
            if (i0 + u * WAVES * 32 >= k) break;
            uint32_t s0[3], s1[3], s2[3], s3[3];
            split2<3>(a[u].x, a[u].y, s0); split2<3>(a[u].z, a[u].w, s1); split2<3>(b[u].x, b[u].y, s2); split2<3>(b[u].z, b[u].w, s3);
#pragma unroll
            for (int e = 2; e >= 0; --e) {
                const hy_bf16x8 xf = __builtin_bit_cast(hy_bf16x8, (hy_u32x4){s0[e], s1[e], s2[e], s3[e]});
#pragma unroll
                for (int j = 0; j < NT; ++j) acc[j] = mfma16(xf, __builtin_bit_cast(hy_bf16x8, wf[u][j]), acc[j]);
            }
        }
    }
#pragma unroll
    for (int j = 0; j < NT; ++j) *(hy_f32x4*)&part[wv][j][lane * 4] = acc[j];
    __syncthreads();
    for (int e = tid; e < NT * 256; e += WAVES * 64) {
        const int j = e >> 8, idx = e & 255;
        float s = 0.0f;
#pragma unroll
        for (int v = 0; v < WAVES; ++v) s += part[v][j][idx];
        const int l = idx >> 2, row = row0 + 4 * (l >> 4) + (idx & 3), col = n0 + 16 * j + (l & 15);
        if (row < rows && col < n) out[(int64_t)row * n + col] = s;
    }
}

// ---- residual += mult * w * rms(y) --------------------------------------------------------------------
struct ResidualNormArgs {
    const void* y; int64_t y_stride; const float* y_weight; int top;
    float* x; const float* w; void* xh; int width, xs; float eps;
    float mult; const float* next_w;                  // next_w: xh = next_w * rms(new x) instead of a copy
};
// NV > 0: rows of up to 1024 NV elements, four at a time, held in registers; everything is requested before the reduction.
template <typename T, int NV>
__global__ __launch_bounds__(256) void residual_norm_kernel(ResidualNormArgs a) {
    extern __shared__ float row[];     // NV = 0: width floats, y of this token summed over its experts
    __shared__ float part[4], part2[4];
    const int64_t t = blockIdx.x;
    const int tid = threadIdx.x;
    const T* y = (const T*)a.y + t * a.top * a.y_stride;
    float* xr = a.x + t * a.xs;
    T* hr = (T*)a.xh + t * a.xs;
    float ss = 0.0f;
    if constexpr (NV > 0) {
        float4 s[NV], f[NV], w[NV];
#pragma unroll
        for (int v = 0; v < NV; ++v) {
            const int i = (v * 256 + tid) * 4;
            s[v] = make_float4(0.f, 0.f, 0.f, 0.f);
            if (i < a.width) {
                f[v] = *(const float4*)(xr + i);
                w[v] = *(const float4*)(a.w + i);
                if (!a.y_weight) s[v] = ld4(y + i);
            }
        }
        if (a.y_weight)
            for (int j = 0; j < a.top; ++j) {
                const float wt = a.y_weight[t * a.top + j];
#pragma unroll
                for (int v = 0; v < NV; ++v) {
                    const int i = (v * 256 + tid) * 4;
                    if (i < a.width) {
                        const float4 e = ld4(y + j * a.y_stride + i);
                        s[v].x += wt * e.x; s[v].y += wt * e.y; s[v].z += wt * e.z; s[v].w += wt * e.w;
                    }
                }
            }
#pragma unroll
        for (int v = 0; v < NV; ++v) ss += s[v].x * s[v].x + s[v].y * s[v].y + s[v].z * s[v].z + s[v].w * s[v].w;
        const float inv = a.mult / sqrtf(block_sum_f(ss, part, 4) / (float)a.width + a.eps);
        float s2 = 0.0f;
#pragma unroll
        for (int v = 0; v < NV; ++v) {
            const int i = (v * 256 + tid) * 4;
            if (i < a.width) {
                f[v].x += s[v].x * inv * w[v].x; f[v].y += s[v].y * inv * w[v].y; f[v].z += s[v].z * inv * w[v].z; f[v].w += s[v].w * inv * w[v].w;
                *(float4*)(xr + i) = f[v];
                if (a.next_w) {
                    s2 += f[v].x * f[v].x + f[v].y * f[v].y + f[v].z * f[v].z + f[v].w * f[v].w;
                    w[v] = *(const float4*)(a.next_w + i);
                } else if (a.xh) st4(hr + i, f[v]);
            }
        }
        if (!a.next_w) return;
        const float inv2 = 1.0f / sqrtf(block_sum_f(s2, part2, 4) / (float)a.width + a.eps);
#pragma unroll
        for (int v = 0; v < NV; ++v) {
            const int i = (v * 256 + tid) * 4;
            if (i < a.width) st4(hr + i, make_float4(f[v].x * inv2 * w[v].x, f[v].y * inv2 * w[v].y, f[v].z * inv2 * w[v].z, f[v].w * inv2 * w[v].w));
        }
    } else {
        for (int i = tid; i < a.width; i += 256) {
            float s = 0.0f;
            if (a.y_weight) for (int j = 0; j < a.top; ++j) s += a.y_weight[t * a.top + j] * ld(y + j * a.y_stride + i);
            else s = ld(y + i);
            row[i] = s;
            ss += s * s;
        }
        const float inv = a.mult / sqrtf(block_sum_f(ss, part, 4) / (float)a.width + a.eps);
        float s2 = 0.0f;
        for (int i = tid; i < a.width; i += 256) {      // a thread re-reads what it wrote itself
            const float f = xr[i] + row[i] * inv * a.w[i];
            xr[i] = f;
            row[i] = f;
            s2 += f * f;
            if (a.xh && !a.next_w) st(hr + i, f);
        }
        if (!a.next_w) return;
        const float inv2 = 1.0f / sqrtf(block_sum_f(s2, part2, 4) / (float)a.width + a.eps);
        for (int i = tid; i < a.width; i += 256) st(hr + i, row[i] * inv2 * a.next_w[i]);
    }
}

template <typename T>
__global__ __launch_bounds__(256) void rms_rows_kernel(const float* x, int xs, const int64_t* rows, const float* w, T* out, int width, float eps) {
    __shared__ float part[4];
    const int64_t t = blockIdx.x;
    const float* xr = x + (rows ? rows[t] : t) * xs;
    float ss = 0.0f;
    for (int i = threadIdx.x; i < width; i += 256) ss += xr[i] * xr[i];
    const float inv = 1.0f / sqrtf(block_sum_f(ss, part, 4) / (float)width + eps);
    for (int i = threadIdx.x; i < width; i += 256) st(out + t * width + i, xr[i] * inv * w[i]);
}

// ---- q and k normed over all their heads ---------------------------------------------------------
struct QkvNormArgs {
    const void* p; int64_t p_stride; int q_off, k_off, v_off;
    const float* qw; const float* kw; float eps;
    int H, G, D, Dv, Dp, Dvp;
    void* q; void* k; void* v;                       // [T][heads][padded dim]
    const int32_t* slots; const int32_t* seen;       // both given: k and v rows go into the rings k, v [slot][G][cap][padded dim]
    int keep, size;
};
// rows of heads without padding and multiples of 8 apart: eight elements at a time
struct Eight { float f[8]; };
__device__ __forceinline__ Eight ld8(const bf16_t* p) {
    const hy_u32x4 r = *(const hy_u32x4*)p;
    Eight e;
#pragma unroll
    for (int x = 0; x < 4; ++x) { e.f[2 * x] = __uint_as_float(r[x] << 16); e.f[2 * x + 1] = __uint_as_float(r[x] & 0xffff0000u); }
    return e;
}
__device__ __forceinline__ Eight ld8(const float* p) {
    const float4 a = *(const float4*)p, b = *(const float4*)(p + 4);
    return {{a.x, a.y, a.z, a.w, b.x, b.y, b.z, b.w}};
}
__device__ __forceinline__ void st8(bf16_t* p, Eight e) { *(hy_u32x4*)p = hy_u32x4{pack2(e.f[0], e.f[1]), pack2(e.f[2], e.f[3]), pack2(e.f[4], e.f[5]), pack2(e.f[6], e.f[7])}; }
__device__ __forceinline__ void st8(float* p, Eight e) { *(float4*)p = make_float4(e.f[0], e.f[1], e.f[2], e.f[3]); *(float4*)(p + 4) = make_float4(e.f[4], e.f[5], e.f[6], e.f[7]); }

template <typename T>
__global__ __launch_bounds__(256) void qkv_norm_vec_kernel(QkvNormArgs a) {
    __shared__ float part[4];
    const int64_t t = blockIdx.x;
    const int tid = threadIdx.x, kind = blockIdx.y;
    const T* row = (const T*)a.p + t * a.p_stride;
    const T* src = row + (kind ? a.k_off : a.q_off);
    const float* wt = kind ? a.kw : a.qw;
    const int n = (kind ? a.G : a.H) * a.D;
    constexpr int HOLD = 2;                               // held in registers between the two passes; longer rows are read again
    Eight held[HOLD];
    float ss = 0.0f;
#pragma unroll
    for (int v = 0; v < HOLD; ++v) {
        const int i = (v * 256 + tid) * 8;
        if (i < n) {
            held[v] = ld8(src + i);
#pragma unroll
            for (int x = 0; x < 8; ++x) ss += held[v].f[x] * held[v].f[x];
        }
    }
    for (int i = (HOLD * 256 + tid) * 8; i < n; i += 2048) {
        const Eight e = ld8(src + i);
#pragma unroll
        for (int x = 0; x < 8; ++x) ss += e.f[x] * e.f[x];
    }
    int64_t kstep = a.D, vstep = a.Dv, k0 = t * a.G * a.D, v0 = t * a.G * a.Dv;
    if (kind && a.slots) {
        const int slot = a.slots[t], cap = a.keep + a.size, r = ring_slot(a.seen[2 * slot], a.keep, a.size);
        kstep = (int64_t)cap * a.D; vstep = (int64_t)cap * a.Dv;
        k0 = (int64_t)slot * a.G * kstep + (int64_t)r * a.D; v0 = (int64_t)slot * a.G * vstep + (int64_t)r * a.Dv;
    }
    if (kind)
        for (int i = tid * 8; i < a.G * a.Dv; i += 2048) {
            const int g = i / a.Dv;
            st8((T*)a.v + v0 + g * vstep + (i - g * a.Dv), ld8(row + a.v_off + i));
        }
    const float inv = 1.0f / sqrtf(block_sum_f(ss, part, 4) / (float)n + a.eps);
    auto put = [&](int i, Eight e) __attribute__((always_inline)) {
        const Eight w = ld8(wt + i);
#pragma unroll
        for (int x = 0; x < 8; ++x) e.f[x] *= inv * w.f[x];
        if (!kind) { st8((T*)a.q + t * n + i, e); return; }
        const int g = i / a.D;
        st8((T*)a.k + k0 + g * kstep + (i - g * a.D), e);
    };
#pragma unroll
    for (int v = 0; v < HOLD; ++v)
        if ((v * 256 + tid) * 8 < n) put((v * 256 + tid) * 8, held[v]);
    for (int i = (HOLD * 256 + tid) * 8; i < n; i += 2048) put(i, ld8(src + i));
}

template <typename T>
__global__ __launch_bounds__(256) void qkv_norm_kernel(QkvNormArgs a) {
    __shared__ float part[4];
    const int64_t t = blockIdx.x;
    const int tid = threadIdx.x;
    const T* row = (const T*)a.p + t * a.p_stride;
    const int nq = a.H * a.D, nk = a.G * a.D;
    const int kind = blockIdx.y;                      // 0: q; 1: k and v
    const T* src = row + (kind ? a.k_off : a.q_off);
    const int n = kind ? nk : nq;
    float ss = 0.0f;
    for (int i = tid; i < n; i += 256) { const float f = ld(src + i); ss += f * f; }
    const float inv = 1.0f / sqrtf(block_sum_f(ss, part, 4) / (float)n + a.eps);
    if (kind == 0) {
        T* dst = (T*)a.q + t * a.H * a.Dp;
        for (int i = tid; i < a.H * a.Dp; i += 256) {
            const int h = i / a.Dp, d = i - h * a.Dp, e = h * a.D + d;
            st(dst + i, d < a.D ? ld(src + e) * inv * a.qw[e] : 0.0f);
        }
        return;
    }
    int64_t kstep = a.Dp, vstep = a.Dvp, k0 = t * a.G * a.Dp, v0 = t * a.G * a.Dvp;
    if (a.slots) {
        const int slot = a.slots[t], cap = a.keep + a.size, r = ring_slot(a.seen[2 * slot], a.keep, a.size);
        kstep = (int64_t)cap * a.Dp; vstep = (int64_t)cap * a.Dvp;
        k0 = (int64_t)slot * a.G * kstep + (int64_t)r * a.Dp; v0 = (int64_t)slot * a.G * vstep + (int64_t)r * a.Dvp;
    }
    for (int i = tid; i < a.G * a.Dp; i += 256) {
        const int g = i / a.Dp, d = i - g * a.Dp, e = g * a.D + d;
        st((T*)a.k + k0 + g * kstep + d, d < a.D ? ld(src + e) * inv * a.kw[e] : 0.0f);
    }
    const T* vs = row + a.v_off;
    for (int i = tid; i < a.G * a.Dvp; i += 256) {
        const int g = i / a.Dvp, d = i - g * a.Dvp;
        st((T*)a.v + v0 + g * vstep + d, d < a.Dv ? ld(vs + g * a.Dv + d) : 0.0f);
    }
}

// ---- rotary positions, bias and a norm per head ----------------------------------------------------
// table [tokens][rot]: cosines of the rot / 2 pairs, then their sines.  Angles in fp64: exact positions, and no table of all
// positions to keep.
__global__ __launch_bounds__(64) void rotary_table_kernel(const double* freq, const int32_t* cu, const int32_t* slots, const int32_t* seen, float* table, int half) {
    const int b = blockIdx.y, t0 = cu[b], i = blockIdx.x;
    if (i >= cu[b + 1] - t0) return;
    const double pos = (double)(seen[2 * slots[b]] + i);
    float* row = table + (int64_t)(t0 + i) * 2 * half;
    for (int j = threadIdx.x; j < half; j += 64) {
        double s, c;
        sincos(pos * freq[j], &s, &c);
        row[j] = (float)c;
        row[half + j] = (float)s;
    }
}

struct QkvHeadsArgs {
    const void* p; int64_t p_stride; int q_off, k_off, v_off;
    const float* bias; const float* qw; const float* kw; const float* table;      // each may be absent (the two weights together)
    float eps;
    int H, G, D, Dv, Dp, Dvp, rot;
    void* q; void* k; void* v;
    const int32_t* slots; const int32_t* seen; int keep, size;
};
// where head idx of q (kind 0), k (1) or v (2) of token t goes
template <typename T>
__device__ __forceinline__ T* qkv_heads_row(const QkvHeadsArgs& a, int64_t t, int kind, int idx) {
    if (kind == 0) return (T*)a.q + (t * a.H + idx) * a.Dp;
    T* base = (T*)(kind == 1 ? a.k : a.v);
    const int n = kind == 1 ? a.Dp : a.Dvp;
    if (!a.slots) return base + (t * a.G + idx) * n;
    const int slot = a.slots[t], cap = a.keep + a.size;
    return base + (((int64_t)slot * a.G + idx) * cap + ring_slot(a.seen[2 * slot], a.keep, a.size)) * n;
}

// LH lanes of sixteen values per head: below the rotated size eight values and their eight partners, behind it neighbours.
// A workgroup keeps to one token, so its lanes' cosines and sines stay in registers over its heads.
template <typename T, int LH>
__global__ __launch_bounds__(256) void qkv_heads_vec_kernel(QkvHeadsArgs a) {
    const int64_t t = blockIdx.x;
    const int sub = threadIdx.x / LH, l = threadIdx.x % LH, groups = blockDim.x / LH;
    const int half = a.rot / 2, rl = a.rot / 16, heads = a.H + 2 * a.G;
    const bool turned = l < rl;
    const int e0 = turned ? 8 * l : a.rot + 16 * (l - rl), e1 = turned ? half + 8 * l : e0 + 8;
    const T* row = (const T*)a.p + t * a.p_stride;
    Eight c, s, w0, w1;
#pragma unroll
    for (int x = 0; x < 8; ++x) { c.f[x] = 1.0f; s.f[x] = 0.0f; w0.f[x] = w1.f[x] = 1.0f; }
    if (turned) {
        c = ld8(a.table + t * a.rot + 8 * l);
        s = ld8(a.table + t * a.rot + half + 8 * l);
    }
    int held = -1;                                    // whose norm weights w0, w1 hold
    for (int h = blockIdx.y * groups + sub; h < heads; h += gridDim.y * groups) {
        const int kind = h < a.H ? 0 : h < a.H + a.G ? 1 : 2;
        const int idx = kind == 0 ? h : kind == 1 ? h - a.H : h - a.H - a.G;
        const int n = kind == 2 ? a.Dv : a.D, off = kind == 0 ? a.q_off + idx * a.D : kind == 1 ? a.k_off + idx * a.D : a.v_off + idx * a.Dv;
        const int i0 = kind == 2 ? 16 * l : e0, i1 = kind == 2 ? 16 * l + 8 : e1;
        const bool in0 = i0 < n, in1 = i1 < n;
        Eight x0, x1;
#pragma unroll
        for (int x = 0; x < 8; ++x) x0.f[x] = x1.f[x] = 0.0f;
        if (in0) x0 = ld8(row + off + i0);
        if (in1) x1 = ld8(row + off + i1);
        if (a.bias) {
            if (in0) { const Eight b = ld8(a.bias + off + i0);
#pragma unroll
                for (int x = 0; x < 8; ++x) x0.f[x] += b.f[x]; }
            if (in1) { const Eight b = ld8(a.bias + off + i1);
#pragma unroll
                for (int x = 0; x < 8; ++x) x1.f[x] += b.f[x]; }
        }
        if (kind < 2) {
            float inv = 1.0f;
            if (a.qw) {
                if (held != kind) {
                    const float* w = kind ? a.kw : a.qw;
                    if (in0) w0 = ld8(w + i0);
                    if (in1) w1 = ld8(w + i1);
                    held = kind;
                }
                float ss = 0.0f;
#pragma unroll
                for (int x = 0; x < 8; ++x) ss += x0.f[x] * x0.f[x] + x1.f[x] * x1.f[x];
#pragma unroll
                for (int d = LH / 2; d > 0; d >>= 1) ss += __shfl_xor(ss, d, 64);
                inv = 1.0f / sqrtf(ss / (float)a.D + a.eps);
            }
#pragma unroll
            for (int x = 0; x < 8; ++x) {
                const float u = x0.f[x] * inv * w0.f[x], v = x1.f[x] * inv * w1.f[x];
                x0.f[x] = u * c.f[x] - v * s.f[x];
                x1.f[x] = v * c.f[x] + u * s.f[x];
            }
        }
        T* dst = qkv_heads_row<T>(a, t, kind, idx);
        if (in0) st8(dst + i0, x0);
        if (in1) st8(dst + i1, x1);
    }
}

// General form: one wavefront per (token, head), partners read again.
template <typename T>
__global__ __launch_bounds__(256) void qkv_heads_kernel(QkvHeadsArgs a, int64_t units) {
    const int64_t unit = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (unit >= units) return;
    const int heads = a.H + 2 * a.G, lane = threadIdx.x & 63;
    const int64_t t = unit / heads;
    const int h = (int)(unit - t * heads);
    const int kind = h < a.H ? 0 : h < a.H + a.G ? 1 : 2;
    const int idx = kind == 0 ? h : kind == 1 ? h - a.H : h - a.H - a.G;
    const int n = kind == 2 ? a.Dv : a.D, off = kind == 0 ? a.q_off + idx * a.D : kind == 1 ? a.k_off + idx * a.D : a.v_off + idx * a.Dv;
    const T* src = (const T*)a.p + t * a.p_stride + off;
    const float* w = kind == 0 ? a.qw : kind == 1 ? a.kw : nullptr;
    const int rot = kind == 2 ? 0 : a.rot, half = rot / 2;
    float inv = 1.0f;
    if (w) {
        float ss = 0.0f;
        for (int i = lane; i < n; i += 64) { const float f = ld(src + i) + (a.bias ? a.bias[off + i] : 0.0f); ss += f * f; }
        inv = 1.0f / sqrtf(wave_sum_f(ss) / (float)n + a.eps);
    }
    auto value = [&](int i) { return (ld(src + i) + (a.bias ? a.bias[off + i] : 0.0f)) * inv * (w ? w[i] : 1.0f); };
    T* dst = qkv_heads_row<T>(a, t, kind, idx);
    for (int i = lane; i < (kind == 2 ? a.Dvp : a.Dp); i += 64) {
        float f = i < n ? value(i) : 0.0f;
        if (i < rot) {
            const int j = i < half ? i : i - half;
            const float c = a.table[t * rot + j], s = a.table[t * rot + half + j];
            f = i < half ? f * c - value(i + half) * s : f * c + value(i - half) * s;
        }
        st(dst + i, f);
    }
}

// ---- silu(gate) * up -----------------------------------------------------------------------------
__device__ __forceinline__ float silu_gate(const bf16_t*, float g, float u) { return g * sigmoid_fast(g) * u; }
__device__ __forceinline__ float silu_gate(const float*, float g, float u) { return g * sigmoid_f(g) * u; }

template <typename T, int PER>
__global__ __launch_bounds__(256) void silu_gate_kernel(const T* gate, const T* up, int64_t stride, T* out, int per_row, int64_t n) {
    for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (int64_t)gridDim.x * 256) {
        const int64_t t = i / per_row;
        const int64_t at = t * stride + (i - t * per_row) * PER;
        if constexpr (PER == 8) {
            Eight g = ld8(gate + at);
            const Eight u = ld8(up + at);
#pragma unroll
            for (int x = 0; x < 8; ++x) g.f[x] = silu_gate(out, g.f[x], u.f[x]);
            st8(out + i * 8, g);
        } else st(out + i, silu_gate(out, ld(gate + at), ld(up + at)));
    }
}

template <typename T>
__global__ __launch_bounds__(256) void soft_cap_kernel(const T* x, float* out, int64_t n, float cap) {
    const int64_t i = ((int64_t)blockIdx.x * 256 + threadIdx.x) * 4;
    if (i + 4 <= n) {
        const float4 f = ld4(x + i);
        *(float4*)(out + i) = make_float4(cap * tanhf(f.x / cap), cap * tanhf(f.y / cap), cap * tanhf(f.z / cap), cap * tanhf(f.w / cap));
    } else
        for (int64_t j = i; j < n; ++j) out[j] = cap * tanhf(ld(x + j) / cap);
}

// ---- a prompt's surviving rows into the ring -----------------------------------------------------
// Rows are multiples of 16 bytes: kc pieces of 16 for a token's keys of one head, vc for its values.
__global__ __launch_bounds__(256) void ring_store_kernel(const uint4* k, const uint4* v, const int32_t* cu, const int32_t* slots, const int32_t* seen,
                                                         uint4* rk, uint4* rv, int G, int kc, int vc, int keep, int size) {
    const int b = blockIdx.y, slot = slots[b], t0 = cu[b], len = cu[b + 1] - t0, past = seen[2 * slot];
    const int i = blockIdx.x;                          // token of the portion
    if (i >= len) return;
    const int pos = past + i;
    if (pos >= keep && pos < past + len - size) return;     // a later token takes its slot
    const int cap = keep + size, r = ring_slot(pos, keep, size);
    for (int e = threadIdx.x; e < G * (kc + vc); e += 256) {
        const bool key = e < G * kc;
        const int n = key ? kc : vc, at = key ? e : e - G * kc, g = at / n;
        (key ? rk : rv)[(((int64_t)slot * G + g) * cap + r) * n + (at - g * n)] = (key ? k : v)[(int64_t)(t0 + i) * G * n + at];
    }
}

// ---- behind a recurrence: rms per head, weight, sigmoid gate -------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void head_norm_gate_kernel(const T* o, const T* g, int64_t g_stride, const float* w, T* out, int64_t units, int H, int Dv, float eps) {
    const int64_t unit = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (unit >= units) return;
    const int64_t t = unit / H;
    const int h = (int)(unit - t * H), lane = threadIdx.x & 63;
    const T* src = o + unit * Dv;
    const T* gr = g + t * g_stride + h * Dv;
    float ss = 0.0f;
    for (int i = lane; i < Dv; i += 64) { const float f = ld(src + i); ss += f * f; }
    const float inv = 1.0f / sqrtf(wave_sum_f(ss) / (float)Dv + eps);
    for (int i = lane; i < Dv; i += 64) st(out + unit * Dv + i, ld(src + i) * inv * w[h * Dv + i] * sigmoid_fast(ld(gr + i)));
}

// Dv a multiple of 8: LH lanes with eight values each per head, 64 / LH heads per wavefront and pass, two passes on their way
// together
template <typename T, int LH>
__global__ __launch_bounds__(256) void head_norm_gate_vec_kernel(const T* o, const T* g, int64_t g_stride, const float* w, T* out, int64_t units, int H, int Dv, float eps) {
    constexpr int PER = 4 * 64 / LH, U = 2;
    const int sub = threadIdx.x / LH, i = (threadIdx.x % LH) * 8;
    const bool in = i < Dv;
    Eight s[U], gt[U];
    int64_t unit[U];
    int h[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
        unit[u] = min((int64_t)blockIdx.x * PER * U + u * PER + sub, units - 1);      // past the end: the last one again, same values
        const int64_t t = unit[u] / H;
        h[u] = (int)(unit[u] - t * H);
        s[u] = ld8(o + unit[u] * Dv + (in ? i : 0));
        gt[u] = ld8(g + t * g_stride + h[u] * Dv + (in ? i : 0));
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
        float ss = 0.0f;
#pragma unroll
        for (int x = 0; x < 8; ++x) ss += s[u].f[x] * s[u].f[x];
        if (!in) ss = 0.0f;
#pragma unroll
        for (int d = LH / 2; d > 0; d >>= 1) ss += __shfl_xor(ss, d, 64);
        const float inv = 1.0f / sqrtf(ss / (float)Dv + eps);
        if (in) {
            const Eight wt = ld8(w + h[u] * Dv + i);
#pragma unroll
            for (int x = 0; x < 8; ++x) s[u].f[x] *= inv * wt.f[x] * sigmoid_fast(gt[u].f[x]);
            st8(out + unit[u] * Dv + i, s[u]);
        }
    }
}

__global__ void advance_kernel(int32_t* seen, const int32_t* slots, const int32_t* cu, int batch) {
    const int b = blockIdx.x * 64 + threadIdx.x;
    if (b >= batch) return;
    const int slot = slots[b];
    seen[2 * slot] += cu[b + 1] - cu[b];
    seen[2 * slot + 1] += 1;
}

}  // namespace trimkv

using namespace trimkv;

extern "C" const char* trimkv_hybrid_last_error(void) { return err_buf(); }

extern "C" int trimkv_embed_scaled(const int64_t* ids, const void* table, float scale, float* x, void* xh, const float* norm_weight, float eps, int add,
                                   int tokens, int vocab, int width, int x_stride, int dtype, void* stream) {
    const char* fn = "trimkv_embed_scaled";
    if (!ids || !table || !x || (norm_weight && !xh)) return fail(TRIMKV_ERR_NULL, "%s: null pointer argument", fn);
    HY_CHECK_DTYPE(fn, dtype);
    if (tokens <= 0 || vocab <= 0 || width <= 0 || x_stride < width) return fail(TRIMKV_ERR_SHAPE, "%s: bad sizes tokens=%d vocab=%d width=%d stride=%d", fn, tokens, vocab, width, x_stride);
    EmbedArgs a{ids, table, scale, x, xh, norm_weight, eps, vocab, width, x_stride, add};
    const bool vec = width % 4 == 0 && x_stride % 4 == 0 && !(((uintptr_t)table | (uintptr_t)x | (uintptr_t)xh | (uintptr_t)norm_weight) & 15);
    HY_BY_DTYPE(dtype, T,
        if (vec && x_stride <= 1024) hipLaunchKernelGGL((embed_vec_kernel<T, 1>), dim3(tokens), dim3(256), 0, (hipStream_t)stream, a);
        else if (vec && x_stride <= 4096) hipLaunchKernelGGL((embed_vec_kernel<T, 4>), dim3(tokens), dim3(256), 0, (hipStream_t)stream, a);
        else hipLaunchKernelGGL((embed_kernel<T>), dim3(tokens), dim3(256), 0, (hipStream_t)stream, a));
    return launch_status(fn);
}

extern "C" int trimkv_linear_f32(const float* x, int64_t x_stride, const void* w, int64_t w_stride, float* out, int rows, int n, int k, int dtype, void* stream) {
    const char* fn = "trimkv_linear_f32";
    if (!x || !w || !out) return fail(TRIMKV_ERR_NULL, "%s: null pointer argument", fn);
    HY_CHECK_DTYPE(fn, dtype);
    if (rows <= 0 || n <= 0 || k <= 0 || k % 4 || x_stride < k || w_stride < k || x_stride % 4 || w_stride % 8)
        return fail(TRIMKV_ERR_SHAPE, "%s: bad sizes rows=%d n=%d k=%d strides %lld %lld", fn, rows, n, k, (long long)x_stride, (long long)w_stride);
    if (((uintptr_t)x | (uintptr_t)w) & 15) return fail(TRIMKV_ERR_SHAPE, "%s: x and w must be 16-byte aligned", fn);
    hipStream_t st_ = (hipStream_t)stream;
    if (dtype == TRIMKV_BF16 && k % 32 == 0) {
        const bf16_t* wb = (const bf16_t*)w;
        if (rows >= 2048 && n > 16)
            hipLaunchKernelGGL((linear_f32_mfma_kernel<4, 4>), dim3((rows + 15) / 16, (n + 63) / 64), dim3(256), 0, st_, x, x_stride, wb, w_stride, out, rows, n, k);
        else if (rows >= 2048)
            hipLaunchKernelGGL((linear_f32_mfma_kernel<1, 4>), dim3((rows + 15) / 16, (n + 15) / 16), dim3(256), 0, st_, x, x_stride, wb, w_stride, out, rows, n, k);
        else
            hipLaunchKernelGGL((linear_f32_mfma_kernel<1, 16>), dim3((rows + 15) / 16, (n + 15) / 16), dim3(1024), 0, st_, x, x_stride, wb, w_stride, out, rows, n, k);
        return launch_status(fn);
    }
    const int64_t units = (int64_t)rows * n;
    HY_BY_DTYPE(dtype, T, hipLaunchKernelGGL((linear_f32_kernel<T>), dim3((unsigned)((units + 3) / 4)), dim3(256), 0, st_, x, x_stride, (const T*)w, w_stride, out, units, n, k));
    return launch_status(fn);
}

extern "C" int trimkv_residual_norm(const void* y, int64_t y_stride, const float* y_weight, int top, float* x, const float* w, float mult, void* xh,
                                    const float* next_w, int tokens, int width, int x_stride, float eps, int dtype, void* stream) {
    const char* fn = "trimkv_residual_norm";
    if (!y || !x || !w || (next_w && !xh)) return fail(TRIMKV_ERR_NULL, "%s: null pointer argument", fn);
    HY_CHECK_DTYPE(fn, dtype);
    if (tokens <= 0 || width <= 0 || width > 16384 || top < 1 || x_stride < width || y_stride < width)
        return fail(TRIMKV_ERR_SHAPE, "%s: bad sizes tokens=%d width=%d top=%d", fn, tokens, width, top);
    if (!y_weight && top != 1) return fail(TRIMKV_ERR_SHAPE, "%s: several rows per token need weights", fn);
    ResidualNormArgs a{y, y_stride, y_weight, top, x, w, xh, width, x_stride, eps, mult, next_w};
    const bool vec = width % 4 == 0 && x_stride % 4 == 0 && y_stride % 4 == 0 && !(((uintptr_t)y | (uintptr_t)x | (uintptr_t)w | (uintptr_t)xh | (uintptr_t)next_w) & 15);
    const size_t lds = (size_t)width * 4;
    HY_BY_DTYPE(dtype, T,
        if (vec && width <= 1024) hipLaunchKernelGGL((residual_norm_kernel<T, 1>), dim3(tokens), dim3(256), 0, (hipStream_t)stream, a);
        else if (vec && width <= 2048) hipLaunchKernelGGL((residual_norm_kernel<T, 2>), dim3(tokens), dim3(256), 0, (hipStream_t)stream, a);
        else if (vec && width <= 4096) hipLaunchKernelGGL((residual_norm_kernel<T, 4>), dim3(tokens), dim3(256), 0, (hipStream_t)stream, a);
        else if (vec && width <= 8192) hipLaunchKernelGGL((residual_norm_kernel<T, 8>), dim3(tokens), dim3(256), 0, (hipStream_t)stream, a);
        else hipLaunchKernelGGL((residual_norm_kernel<T, 0>), dim3(tokens), dim3(256), lds, (hipStream_t)stream, a));
    return launch_status(fn);
}

extern "C" int trimkv_rms_rows(const float* x, int x_stride, const int64_t* rows, const float* w, void* out, int count, int width, float eps, int dtype, void* stream) {
    const char* fn = "trimkv_rms_rows";
    if (!x || !w || !out) return fail(TRIMKV_ERR_NULL, "%s: null pointer argument", fn);
    HY_CHECK_DTYPE(fn, dtype);
    if (count <= 0 || width <= 0 || x_stride < width) return fail(TRIMKV_ERR_SHAPE, "%s: bad sizes count=%d width=%d", fn, count, width);
    HY_BY_DTYPE(dtype, T, hipLaunchKernelGGL((rms_rows_kernel<T>), dim3(count), dim3(256), 0, (hipStream_t)stream, x, x_stride, rows, w, (T*)out, width, eps));
    return launch_status(fn);
}

extern "C" int trimkv_qkv_norm(const void* proj, int64_t proj_stride, int q_off, int k_off, int v_off, const float* q_weight, const float* k_weight, float eps,
                               int heads, int kv_heads, int dim, int vdim, int dim_stride, int vdim_stride, void* q, void* k, void* v,
                               const int32_t* slots, const int32_t* seen, int keep_first, int window, int tokens, int dtype, void* stream) {
    const char* fn = "trimkv_qkv_norm";
    if (!proj || !q_weight || !k_weight || !q || !k || !v || (!slots != !seen)) return fail(TRIMKV_ERR_NULL, "%s: null pointer argument", fn);
    HY_CHECK_DTYPE(fn, dtype);
    if (tokens <= 0 || heads <= 0 || kv_heads <= 0 || dim <= 0 || vdim <= 0 || dim_stride < dim || vdim_stride < vdim || (slots && (window <= 0 || keep_first < 0)))
        return fail(TRIMKV_ERR_SHAPE, "%s: bad sizes tokens=%d heads=%d kv_heads=%d dim=%d vdim=%d", fn, tokens, heads, kv_heads, dim, vdim);
    QkvNormArgs a{proj, proj_stride, q_off, k_off, v_off, q_weight, k_weight, eps, heads, kv_heads, dim, vdim, dim_stride, vdim_stride, q, k, v, slots, seen, keep_first, window};
    const bool vec = dim_stride == dim && vdim_stride == vdim && dim % 8 == 0 && vdim % 8 == 0 && proj_stride % 8 == 0 && (q_off | k_off | v_off) % 8 == 0 &&
                     !(((uintptr_t)proj | (uintptr_t)q_weight | (uintptr_t)k_weight | (uintptr_t)q | (uintptr_t)k | (uintptr_t)v) & 15);
    if (vec) {
        HY_BY_DTYPE(dtype, T, hipLaunchKernelGGL((qkv_norm_vec_kernel<T>), dim3(tokens, 2), dim3(256), 0, (hipStream_t)stream, a));
        return launch_status(fn);
    }
    HY_BY_DTYPE(dtype, T, hipLaunchKernelGGL((qkv_norm_kernel<T>), dim3(tokens, 2), dim3(256), 0, (hipStream_t)stream, a));
    return launch_status(fn);
}

extern "C" int trimkv_rotary_table(const double* freq, const int32_t* cu, const int32_t* slots, const int32_t* seen, float* table, int batch, int max_len, int rot_dims, void* stream) {
    const char* fn = "trimkv_rotary_table";
    if (!freq || !cu || !slots || !seen || !table) return fail(TRIMKV_ERR_NULL, "%s: null pointer argument", fn);
    if (batch <= 0 || batch > 65535 || max_len <= 0 || rot_dims <= 0 || rot_dims % 2) return fail(TRIMKV_ERR_SHAPE, "%s: bad sizes batch=%d max_len=%d rot_dims=%d", fn, batch, max_len, rot_dims);
    hipLaunchKernelGGL(rotary_table_kernel, dim3(max_len, batch), dim3(64), 0, (hipStream_t)stream, freq, cu, slots, seen, table, rot_dims / 2);
    return launch_status(fn);
}

extern "C" int trimkv_qkv_heads(const void* proj, int64_t proj_stride, int q_off, int k_off, int v_off, const float* bias, const float* q_weight, const float* k_weight, float eps,
                                const float* table, int rot_dims, int heads, int kv_heads, int dim, int vdim, int dim_stride, int vdim_stride, void* q, void* k, void* v,
                                const int32_t* slots, const int32_t* seen, int keep_first, int window, int tokens, int dtype, void* stream) {
    const char* fn = "trimkv_qkv_heads";
    if (!proj || !q || !k || !v || (!slots != !seen) || (!q_weight != !k_weight) || (!table && rot_dims)) return fail(TRIMKV_ERR_NULL, "%s: null pointer argument", fn);
    HY_CHECK_DTYPE(fn, dtype);
    if (tokens <= 0 || heads <= 0 || kv_heads <= 0 || dim <= 0 || vdim <= 0 || dim_stride < dim || vdim_stride < vdim || rot_dims < 0 || rot_dims > dim || rot_dims % 2 ||
        (slots && (window <= 0 || keep_first < 0)))
        return fail(TRIMKV_ERR_SHAPE, "%s: bad sizes tokens=%d heads=%d kv_heads=%d dim=%d vdim=%d rot_dims=%d", fn, tokens, heads, kv_heads, dim, vdim, rot_dims);
    QkvHeadsArgs a{proj, proj_stride, q_off, k_off, v_off, bias, q_weight, k_weight, table, eps, heads, kv_heads, dim, vdim, dim_stride, vdim_stride, rot_dims, q, k, v, slots, seen, keep_first, window};
    hipStream_t s = (hipStream_t)stream;
    const int units = heads + 2 * kv_heads;
    const int lanes_qk = rot_dims / 16 + (dim - rot_dims + 15) / 16, lanes_v = (vdim + 15) / 16, lanes = lanes_qk > lanes_v ? lanes_qk : lanes_v;
    const bool vec = dim_stride == dim && vdim_stride == vdim && dim % 8 == 0 && vdim % 8 == 0 && rot_dims % 16 == 0 && lanes <= 32 && proj_stride % 8 == 0 &&
                     (q_off | k_off | v_off) % 8 == 0 &&
                     !(((uintptr_t)proj | (uintptr_t)bias | (uintptr_t)q_weight | (uintptr_t)k_weight | (uintptr_t)table | (uintptr_t)q | (uintptr_t)k | (uintptr_t)v) & 15);
    if (vec) {
        auto go = [&](auto lh) {
            constexpr int LH = decltype(lh)::value;
            // few tokens: one head per group of lanes; many: a workgroup walks the heads of its token in equal turns
            int threads = 256, waste = 1 << 30;
            for (int n = 256; n >= 64; n /= 2) {
                const int groups = n / LH, idle = (units + groups - 1) / groups * groups - units;
                if (idle < waste) { waste = idle; threads = n; }
            }
            const int groups = threads / LH, spread = tokens < 1024 ? (units + groups - 1) / groups : 1;
            HY_BY_DTYPE(dtype, T, hipLaunchKernelGGL((qkv_heads_vec_kernel<T, LH>), dim3(tokens, spread), dim3(threads), 0, s, a));
        };
        if (lanes <= 4) go(std::integral_constant<int, 4>{});
        else if (lanes <= 8) go(std::integral_constant<int, 8>{});
        else if (lanes <= 16) go(std::integral_constant<int, 16>{});
        else go(std::integral_constant<int, 32>{});
        return launch_status(fn);
    }
    const int64_t n = (int64_t)tokens * units;
    HY_BY_DTYPE(dtype, T, hipLaunchKernelGGL((qkv_heads_kernel<T>), dim3((unsigned)((n + 3) / 4)), dim3(256), 0, s, a, n));
    return launch_status(fn);
}

extern "C" int trimkv_silu_gate(const void* gate, const void* up, int64_t stride, void* out, int tokens, int inter, int dtype, void* stream) {
    const char* fn = "trimkv_silu_gate";
    if (!gate || !up || !out) return fail(TRIMKV_ERR_NULL, "%s: null pointer argument", fn);
    HY_CHECK_DTYPE(fn, dtype);
    if (tokens <= 0 || inter <= 0 || stride < inter) return fail(TRIMKV_ERR_SHAPE, "%s: bad sizes tokens=%d inter=%d stride=%lld", fn, tokens, inter, (long long)stride);
    const bool vec = inter % 8 == 0 && stride % 8 == 0 && !(((uintptr_t)gate | (uintptr_t)up | (uintptr_t)out) & 15);
    const int per_row = vec ? inter / 8 : inter;
    const int64_t n = (int64_t)tokens * per_row, blocks = (n + 255) / 256;
    const dim3 grid((unsigned)(blocks < 65536 ? blocks : 65536));
    HY_BY_DTYPE(dtype, T,
        if (vec) hipLaunchKernelGGL((silu_gate_kernel<T, 8>), grid, dim3(256), 0, (hipStream_t)stream, (const T*)gate, (const T*)up, stride, (T*)out, per_row, n);
        else hipLaunchKernelGGL((silu_gate_kernel<T, 1>), grid, dim3(256), 0, (hipStream_t)stream, (const T*)gate, (const T*)up, stride, (T*)out, per_row, n));
    return launch_status(fn);
}

extern "C" int trimkv_soft_cap(const void* x, float* out, int64_t count, float cap, int dtype, void* stream) {
    const char* fn = "trimkv_soft_cap";
    if (!x || !out) return fail(TRIMKV_ERR_NULL, "%s: null pointer argument", fn);
    HY_CHECK_DTYPE(fn, dtype);
    const int64_t blocks = (count + 1023) / 1024;
    if (count <= 0 || blocks > 0x7fffffffLL || !(cap > 0.0f)) return fail(TRIMKV_ERR_SHAPE, "%s: bad sizes count=%lld cap=%g", fn, (long long)count, (double)cap);
    if (((uintptr_t)x | (uintptr_t)out) & 15) return fail(TRIMKV_ERR_SHAPE, "%s: x and out must be 16-byte aligned", fn);
    HY_BY_DTYPE(dtype, T, hipLaunchKernelGGL((soft_cap_kernel<T>), dim3((unsigned)blocks), dim3(256), 0, (hipStream_t)stream, (const T*)x, out, count, cap));
    return launch_status(fn);
}

extern "C" int trimkv_ring_store(const void* k, const void* v, const int32_t* cu, const int32_t* slots, const int32_t* seen, void* ring_k, void* ring_v,
                                 int batch, int max_len, int kv_heads, int dim_stride, int vdim_stride, int keep_first, int window, int dtype, void* stream) {
    const char* fn = "trimkv_ring_store";
    if (!k || !v || !cu || !slots || !seen || !ring_k || !ring_v) return fail(TRIMKV_ERR_NULL, "%s: null pointer argument", fn);
    HY_CHECK_DTYPE(fn, dtype);
    if (batch <= 0 || batch > 65535 || max_len <= 0 || kv_heads <= 0 || dim_stride <= 0 || vdim_stride <= 0 || keep_first < 0 || window <= 0)
        return fail(TRIMKV_ERR_SHAPE, "%s: bad sizes batch=%d max_len=%d kv_heads=%d keep=%d window=%d", fn, batch, max_len, kv_heads, keep_first, window);
    const int per = dtype == TRIMKV_BF16 ? 8 : 4;
    if (dim_stride % 8 || vdim_stride % 8 || (((uintptr_t)k | (uintptr_t)v | (uintptr_t)ring_k | (uintptr_t)ring_v) & 15))
        return fail(TRIMKV_ERR_SHAPE, "%s: padded sizes must be multiples of 8 and pointers 16-byte aligned", fn);
    hipLaunchKernelGGL(ring_store_kernel, dim3(max_len, batch), dim3(256), 0, (hipStream_t)stream, (const uint4*)k, (const uint4*)v, cu, slots, seen,
                       (uint4*)ring_k, (uint4*)ring_v, kv_heads, dim_stride / per, vdim_stride / per, keep_first, window);
    return launch_status(fn);
}

extern "C" int trimkv_head_norm_gate(const void* o, const void* gate, int64_t gate_stride, const float* w, void* out, int tokens, int heads, int vdim, float eps, int dtype, void* stream) {
    const char* fn = "trimkv_head_norm_gate";
    if (!o || !gate || !w || !out) return fail(TRIMKV_ERR_NULL, "%s: null pointer argument", fn);
    HY_CHECK_DTYPE(fn, dtype);
    if (tokens <= 0 || heads <= 0 || vdim <= 0) return fail(TRIMKV_ERR_SHAPE, "%s: bad sizes tokens=%d heads=%d vdim=%d", fn, tokens, heads, vdim);
    const int64_t units = (int64_t)tokens * heads;
    if (vdim % 8 == 0 && vdim <= 512 && gate_stride % 8 == 0 && !(((uintptr_t)o | (uintptr_t)gate | (uintptr_t)w | (uintptr_t)out) & 15)) {
        auto go = [&](auto lh) {
            constexpr int LH = decltype(lh)::value, PER = 4 * 64 / LH * 2;
            HY_BY_DTYPE(dtype, T, hipLaunchKernelGGL((head_norm_gate_vec_kernel<T, LH>), dim3((unsigned)((units + PER - 1) / PER)), dim3(256), 0, (hipStream_t)stream,
                                                     (const T*)o, (const T*)gate, gate_stride, w, (T*)out, units, heads, vdim, eps));
        };
        if (vdim <= 64) go(std::integral_constant<int, 8>{});
        else if (vdim <= 128) go(std::integral_constant<int, 16>{});
        else if (vdim <= 256) go(std::integral_constant<int, 32>{});
        else go(std::integral_constant<int, 64>{});
        return launch_status(fn);
    }
    HY_BY_DTYPE(dtype, T, hipLaunchKernelGGL((head_norm_gate_kernel<T>), dim3((unsigned)((units + 3) / 4)), dim3(256), 0, (hipStream_t)stream, (const T*)o, (const T*)gate, gate_stride, w, (T*)out, units, heads, vdim, eps));
    return launch_status(fn);
}

extern "C" int trimkv_advance(int32_t* seen, const int32_t* slots, const int32_t* cu, int batch, void* stream) {
    const char* fn = "trimkv_advance";
    if (!seen || !slots || !cu) return fail(TRIMKV_ERR_NULL, "%s: null pointer argument", fn);
    if (batch <= 0) return fail(TRIMKV_ERR_SHAPE, "%s: bad batch %d", fn, batch);
    hipLaunchKernelGGL(advance_kernel, dim3((batch + 63) / 64), dim3(64), 0, (hipStream_t)stream, seen, slots, cu, batch);
    return launch_status(fn);
}
