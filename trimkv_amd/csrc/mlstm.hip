// mLSTM matrix memory (xLSTM) -- gfx950.  Per head, with log gates i_t, f_t (soft-capped; f through logsigmoid):
//
//   m_t = max(f_t + m_{t-1}, i_t)          a_t = exp(f_t + m_{t-1} - m_t)      c_t = exp(i_t - m_t)
//   S_t = a_t S_{t-1} + c_t k_t v_t^T      n_t = a_t n_{t-1} + c_t k_t
//   o_t = S_t^T q_t / (max(|n_t . q_t|, exp(-m_t)) + 1e-6),   S_0 = 0, n_0 = 0, m_0 = 0
//
// State per sequence slot: S [H][D][Dv] and, twice, (n, m) [H][D + 1], all fp32.  n and m are needed by every workgroup of
// a head while S is split over workgroups by value columns, so a step reads (n, m) from the copy of the parity of the
// slot's step count and writes the other one.  A slot whose token count is 0 starts from the zero state whatever it holds.
//
//   mlstm_recurrent_kernel  token by token; decode, and any portion in fp32
//   mlstm_chunk_kernel      prompts in bf16 on the matrix cores, 64 tokens at a time
#include "hybrid.hip.h"
#include <type_traits>

namespace trimkv {

struct MlstmArgs {
    const void* p; int64_t p_stride; int q_off, k_off, v_off;   // projection rows [T][p_stride]
    const float* gates;                                         // [T][2 H]: W_i h, then W_f h
    const float* ib; const float* fb; float cap;
    float* S; float* nm;                                        // nm: [2][slots][H][D + 1]
    const int32_t* cu; const int32_t* slots; const int32_t* seen;
    void* o;                                                    // [T][H][Dv] in the activations' type
    int H, D, Dv, nslots;
    float qscale;
};

__device__ __forceinline__ float log_input_gate(float z, float cap) { return cap * tanhf(z / cap); }
__device__ __forceinline__ float log_forget_gate(float z, float cap) { return log_sigmoid_exact(cap * tanhf(z / cap)); }

// A workgroup owns 64 value columns of one head: lane = column, wavefront w = rows w KW .. of S.
template <typename T, int KMAX>
__global__ __launch_bounds__(256) void mlstm_recurrent_kernel(MlstmArgs a) {
    extern __shared__ float ms[];                 // n [D], q [D], k [D], red [4][64], part [4]
    float* const n = ms; float* const q = n + a.D; float* const k = q + a.D; float* const red = k + a.D; float* const part = red + 256;
    const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
    const int h = blockIdx.y, b = blockIdx.z, col = blockIdx.x * 64 + lane;
    const bool cin = col < a.Dv;
    const int t0 = a.cu[b], len = a.cu[b + 1] - t0;
    const int slot = a.slots[b];
    const bool fresh = a.seen[2 * slot] == 0;
    const int parity = a.seen[2 * slot + 1] & 1;
    const int KW = (a.D + 3) / 4, d0 = w * KW, nd = max(0, min(KW, a.D - d0));
    const int64_t copy = (int64_t)a.nslots * a.H * (a.D + 1), at = ((int64_t)slot * a.H + h) * (a.D + 1);
    const float* nm_in = a.nm + parity * copy + at;
    float* nm_out = a.nm + (1 - parity) * copy + at;
    float* Sp = a.S + (((int64_t)slot * a.H + h) * a.D + d0) * a.Dv + (cin ? col : 0);
    // a token's operands are requested one token ahead (the first ones before the state)
    float q_next[2], k_next[2], v_next, zi, zf;
    auto fetch = [&](int t) __attribute__((always_inline)) {
        const int64_t tok = t0 + min(t, len - 1);
        const T* row = (const T*)a.p + tok * a.p_stride;
#pragma unroll
        for (int x = 0; x < 2; ++x) {
            const int d = min(tid + 256 * x, a.D - 1);
            q_next[x] = ld(row + a.q_off + h * a.D + d);
            k_next[x] = ld(row + a.k_off + h * a.D + d);
        }
        v_next = ld(row + a.v_off + h * a.Dv + (cin ? col : 0));
        zi = a.gates[tok * 2 * a.H + h];
        zf = a.gates[tok * 2 * a.H + a.H + h];
    };
    fetch(0);
    float s[KMAX];
#pragma unroll
    for (int x = 0; x < KMAX; ++x) s[x] = fresh || x >= nd ? 0.0f : Sp[(int64_t)x * a.Dv];
    for (int d = tid; d < a.D; d += 256) n[d] = fresh ? 0.0f : nm_in[d];
    float m = fresh ? 0.0f : nm_in[a.D];
    const float ib = a.ib[h], fb = a.fb[h];
    for (int t = 0; t < len; ++t) {
        const int64_t tok = t0 + t;
        const float li = log_input_gate(zi + ib, a.cap), lf = log_forget_gate(zf + fb, a.cap), v = v_next;
        const float mn = fmaxf(lf + m, li), keep = expf(lf + m - mn), add = expf(li - mn);
        m = mn;
        float qn = 0.0f;
#pragma unroll
        for (int x = 0; x < 2; ++x) {
            const int d = tid + 256 * x;
            if (d < a.D) {
                const float qq = q_next[x] * a.qscale, kk = k_next[x];
                q[d] = qq; k[d] = kk;
                const float nn = keep * n[d] + add * kk;
                n[d] = nn;
                qn += nn * qq;
            }
        }
        if (t + 1 < len) fetch(t + 1);
        qn = block_sum_f(qn, part, 4);            // its barrier also publishes q and k
        const float av = add * v;
        float num = 0.0f;
#pragma unroll
        for (int x = 0; x < KMAX; ++x)
            if (x < nd) {
                s[x] = keep * s[x] + k[d0 + x] * av;
                num += s[x] * q[d0 + x];
            }
        red[w * 64 + lane] = num;
        __syncthreads();
        if (w == 0 && cin) {
            num = red[lane] + red[64 + lane] + red[128 + lane] + red[192 + lane];
            st((T*)a.o + (tok * a.H + h) * a.Dv + col, num / (fmaxf(fabsf(qn), expf(-m)) + 1e-6f));
        }
        __syncthreads();                          // red, part, q and k are free again
    }
    if (cin) {
#pragma unroll
        for (int x = 0; x < KMAX; ++x)
            if (x < nd) Sp[(int64_t)x * a.Dv] = s[x];
    }
    if (blockIdx.x == 0) {
        for (int d = tid; d < a.D; d += 256) nm_out[d] = n[d];
        if (tid == 0) nm_out[a.D] = m;
    }
}

// ---- prompts: 64 tokens at a time on the matrix cores -----------------------------------------------
// Inside a chunk, with F_t = f_1 + .. + f_t, d_s = i_s - F_s and M_t = max(m_0, max_{s<=t} d_s), the recurrence unrolls to
//
//   m_t = F_t + M_t,   o_t ~ sum_{s<=t} exp(d_s - M_t) (q_t.k_s) v_s + exp(m_0 - M_t) S_0^T q_t,   n.q alike without v,
//   S_C = exp(m_0 - M_C) S_0 + sum_s exp(d_s - M_C) k_s v_s^T.
//
// q, k, v are bf16; everything that multiplies them is fp32 and enters the matrix cores as a sum of bf16 terms: the weighted v
// that goes into the state as three (fp32 products), S and the weighted scores on their way to an output as two (17 bits).
// The state itself stays in fp32 accumulators.  A workgroup owns 128 value columns of one head, a wavefront 32:
// its part of S stays in the accumulators, whose layout (column = lane % 32, rows 8 (v / 4) + 4 half + v % 4) is the operand
// layout of S_0^T q with k taken in the order 4 half + 0..3, 8 + 4 half + 0..3 of every 16.  The same order is used along s
// (V and K are read transposed, ds_read_b64_tr_b16).
//
// Long prompts are cut into segments that run side by side: pass 1 computes every segment's own contribution to the state,
// mlstm_join_kernel chains them into the state each segment starts from, pass 2 computes the outputs.
struct ChunkArgs {
    MlstmArgs a;
    float* seg_S; float* seg_n; float* seg_g; float* seg_m;     // [batch][H][nseg] x (D Dv, D, 2: sum of f and stabiliser, 1)
    int seg_len, nseg;
};
enum { CHUNK_WHOLE = 0, CHUNK_LOCAL = 1, CHUNK_OUTPUT = 2 };

template <int DKT>
struct ChunkCfg {
    static constexpr int DK = 32 * DKT, NBUF = 1;       // two workgroups fit a CU and hide each other's loads
    static constexpr int QB = 64 * DK * 2, VB = 64 * 256, BUF = 2 * QB + VB;
    static constexpr int PROW = 144, PPLANE = 64 * PROW;
    static constexpr int P0 = NBUF * BUF, F0 = P0 + 2 * PPLANE;
    static constexpr int LDS = F0 + (6 * 64 + DK + 64 + 96 + 256) * 4;
    // position of 16-byte piece c of row r: rows that one read instruction touches together fall on different banks
    static __device__ __forceinline__ int swz(int r) {
        return DK == 32 ? (r >> 2) & 3 : DK == 64 ? (((r >> 1) & 1) << 2) | ((r >> 2) & 3) : ((r & 3) << 2) | ((r >> 2) & 3);
    }
    static __device__ __forceinline__ int vswz(int r) { return ((r & 3) << 2) | ((r >> 2) & 3); }
};

__device__ __forceinline__ float wave_scan_add(float v, int lane) {
#pragma unroll
    for (int d = 1; d < 64; d <<= 1) { const float o = __shfl_up(v, d, 64); if (lane >= d) v += o; }
    return v;
}
__device__ __forceinline__ float wave_scan_max(float v, int lane) {
#pragma unroll
    for (int d = 1; d < 64; d <<= 1) { const float o = __shfl_up(v, d, 64); if (lane >= d) v = fmaxf(v, o); }
    return v;
}
// The chunk kernels keep gates and stabilisers in units of log 2, so that an exponential is one instruction; the state's m is
// converted on the way in and out.
constexpr float LOG2E = 1.4426950408889634f, LN2 = 0.6931471805599453f;
__device__ __forceinline__ float exp_fast(float x) { return __builtin_amdgcn_exp2f(x); }

template <int DKT, int MODE, bool FULL>     // FULL: dim is exactly 32 DKT
__global__ __launch_bounds__(256, DKT <= 4 ? 2 : 1) void mlstm_chunk_kernel(ChunkArgs ca) {
    using C = ChunkCfg<DKT>;
    constexpr int DK = C::DK, NB = C::NBUF;
    const MlstmArgs& a = ca.a;
    extern __shared__ __attribute__((aligned(16))) char ck_lds[];
    HY_LDS char* const lds3 = (HY_LDS char*)ck_lds;
    const uint32_t lds0 = (uint32_t)(uintptr_t)lds3;
    float* const gF = (float*)(ck_lds + C::F0);      // [2][64] each
    float* const gD = gF + 128; float* const gM = gD + 128;
    float* const n = gM + 128; float* const qn = n + DK; float* const dsum = qn + 64;
    float* const wgt = dsum + 96;                     // [4][64]: every wavefront's own copy of exp(d_s - M_C)
    const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6), j = lane & 31, hl = lane >> 5;
    const int vt = (a.Dv + 127) / 128, seg = blockIdx.x / vt, dv0 = (blockIdx.x % vt) * 128, h = blockIdx.y, b = blockIdx.z;
    const int t0 = a.cu[b], len_all = a.cu[b + 1] - t0;
    const int first = MODE == CHUNK_WHOLE ? 0 : seg * ca.seg_len;
    const int len = MODE == CHUNK_WHOLE ? len_all : min(len_all - first, ca.seg_len);
    if (len <= 0) return;                             // workgroup-uniform, before any barrier
    const int slot = a.slots[b];
    const bool fresh = a.seen[2 * slot] == 0;
    const int parity = a.seen[2 * slot + 1] & 1;
    const int64_t sat = ((int64_t)b * a.H + h) * ca.nseg + seg;
    const int64_t copy = (int64_t)a.nslots * a.H * (a.D + 1), at = ((int64_t)slot * a.H + h) * (a.D + 1);
    const int col = dv0 + w * 32 + j;
    const bool live = dv0 + w * 32 < a.Dv;            // wavefront-uniform

    hy_f32x16 S[DKT];
    float m0;
    {
        const bool zero = MODE == CHUNK_LOCAL || (MODE == CHUNK_WHOLE && fresh);
        const float* src = MODE == CHUNK_OUTPUT ? ca.seg_S + sat * a.D * a.Dv : a.S + ((int64_t)slot * a.H + h) * a.D * a.Dv;
        const float* nsrc = MODE == CHUNK_OUTPUT ? ca.seg_n + sat * a.D : a.nm + parity * copy + at;
#pragma unroll
        for (int db = 0; db < DKT; ++db)
#pragma unroll
            for (int v = 0; v < 16; ++v) {
                const int d = db * 32 + 8 * (v >> 2) + 4 * hl + (v & 3);
                S[db][v] = zero || (!FULL && d >= a.D) || col >= a.Dv ? 0.0f : src[(int64_t)d * a.Dv + col];
            }
        for (int d = tid; d < DK; d += 256) n[d] = zero || d >= a.D ? 0.0f : nsrc[d];
        m0 = MODE == CHUNK_LOCAL ? -1.0e30f : MODE == CHUNK_OUTPUT ? ca.seg_m[sat] : fresh ? 0.0f : a.nm[parity * copy + at + a.D] * LOG2E;
    }
    const bf16_t* base = (const bf16_t*)a.p + (int64_t)(t0 + first) * a.p_stride;
    auto request = [&](int c, int buf) __attribute__((always_inline)) {
        const uint32_t dst = lds0 + buf * C::BUF + w * 1024;
#pragma unroll
        for (int x = 0; x < 64 * (DK / 8) / 256; ++x) {
            const int p = x * 256 + tid, row = p / (DK / 8), pos = p % (DK / 8);
            const bf16_t* r = base + (int64_t)min(c * 64 + row, len - 1) * a.p_stride + h * a.D + min((pos ^ C::swz(row)) * 8, a.D - 8);
            if (MODE != CHUNK_LOCAL) load_to_lds16(r + a.q_off, dst + x * 4096);
            load_to_lds16(r + a.k_off, dst + C::QB + x * 4096);
        }
#pragma unroll
        for (int x = 0; x < 4; ++x) {
            const int p = x * 256 + tid, row = p >> 4, pos = p & 15;
            load_to_lds16(base + (int64_t)min(c * 64 + row, len - 1) * a.p_stride + a.v_off + h * a.Dv + min(dv0 + (pos ^ C::vswz(row)) * 8, a.Dv - 8),
                          dst + 2 * C::QB + x * 4096);
        }
    };
    const float ib = a.ib[h], fb = a.fb[h];
    float zi = 0.0f, zf = 0.0f;                       // raw gates of the chunk after next, on their way
    auto fetch_gates = [&](int c) __attribute__((always_inline)) {        // one wavefront, lane = token of chunk c
        const float* g = a.gates + (int64_t)(t0 + first + min(c * 64 + lane, len - 1)) * 2 * a.H + h;
        zi = g[0];
        zf = g[a.H];
    };
    auto gates = [&](int c, int buf) __attribute__((always_inline)) {
        const int t = c * 64 + lane;
        const float li = t < len ? log_input_gate(zi + ib, a.cap) * LOG2E : -1.0e30f;
        const float lf = t < len ? log_forget_gate(zf + fb, a.cap) * LOG2E : 0.0f;
        const float F = wave_scan_add(lf, lane), d = li - F;
        gF[buf * 64 + lane] = F;
        gD[buf * 64 + lane] = d;
        gM[buf * 64 + lane] = wave_scan_max(d, lane);
    };
    // transposing read of 8 rows (16 st + 4 hl + 0..3, + 8) at column 32 db + lane % 32
    const int kx = 4 * hl + ((lane & 15) >> 2), pc = 2 * ((lane >> 4) & 1) + ((lane & 3) >> 1), pb = (lane & 1) * 8;
    auto tr_read = [&](int off, int row_bytes, int sw0, int sw1, int st_, int db) __attribute__((always_inline)) {
        HY_LDS char* p = lds3 + off + (st_ * 16 + kx) * row_bytes + pb;
        const hy_s16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((HY_LDS hy_s16x4*)(p + (((4 * db + pc) ^ sw0) << 4)));
        const hy_s16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((HY_LDS hy_s16x4*)(p + 8 * row_bytes + (((4 * db + pc) ^ sw1) << 4)));
        return __builtin_bit_cast(hy_bf16x8, __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7));
    };
    const int ksw0 = C::swz(kx), ksw1 = C::swz(kx + 8), vsw0 = C::vswz(kx), vsw1 = C::vswz(kx + 8);

    const int nchunks = (len + 63) / 64;
    float fsum = 0.0f;
    request(0, 0);
    if (w == 3) { fetch_gates(0); gates(0, 0); fetch_gates(1); }
    for (int c = 0; c < nchunks; ++c) {
        const int buf = NB == 2 ? c & 1 : 0, gb = (c & 1) * 64, off = buf * C::BUF;
        if (c == 0 || NB == 1) asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();                              // chunk c and its gates are there; chunk c - 1 is done with
        if (NB == 2 && c + 1 < nchunks) request(c + 1, buf ^ 1);
        if (w == 3 && c + 1 < nchunks) { gates(c + 1, (c + 1) & 1); fetch_gates(c + 2); }
        const float Mc = fmaxf(m0, gM[gb + 63]);
        float* const ws = wgt + w * 64;
        ws[lane] = exp_fast(gD[gb + lane] - Mc);
        hy_f32x16 o[2];
        if (MODE != CHUNK_LOCAL) {
            if (w < 3) {                              // scores, weighted: blocks (s, t) = (0, 0), (0, 1), (1, 1)
                const int sb = w == 2, tb = w >= 1;
                hy_f32x16 p;
#pragma unroll
                for (int v = 0; v < 16; ++v) p[v] = 0.0f;
#pragma unroll
                for (int ks = 0; ks < DK / 16; ++ks) {
                    const int kr = sb * 32 + j, qr = tb * 32 + j, pcs = 2 * ks + hl;
                    const hy_bf16x8 kf = *(const HY_LDS hy_bf16x8*)(lds3 + off + C::QB + kr * DK * 2 + ((pcs ^ C::swz(kr)) << 4));
                    hy_u32x4 qf = *(const HY_LDS hy_u32x4*)(lds3 + off + qr * DK * 2 + ((pcs ^ C::swz(qr)) << 4));
                    if (!FULL && pcs * 8 >= a.D) qf = hy_u32x4{0u, 0u, 0u, 0u};
                    p = mfma32(kf, __builtin_bit_cast(hy_bf16x8, qf), p);
                }
                const int t = tb * 32 + j;
                const float M = fmaxf(m0, gM[gb + t]);
                float sum = 0.0f;
#pragma unroll
                for (int x = 0; x < 4; ++x) {
                    const float4 d = *(const float4*)(gD + gb + sb * 32 + 8 * x + 4 * hl);
                    const float dd[4] = {d.x, d.y, d.z, d.w};
                    float q[4];
#pragma unroll
                    for (int y = 0; y < 4; ++y) {
                        const int s = sb * 32 + 8 * x + 4 * hl + y;
                        q[y] = s <= t ? p[4 * x + y] * a.qscale * exp_fast(dd[y] - M) : 0.0f;
                        sum += q[y];
                    }
                    uint32_t e0[2], e1[2];
                    split2<2>(q[0], q[1], e0);
                    split2<2>(q[2], q[3], e1);
#pragma unroll
                    for (int e = 0; e < 2; ++e)
                        *(uint2*)(ck_lds + C::P0 + e * C::PPLANE + t * C::PROW + (sb * 32 + 8 * x + 4 * hl) * 2) = make_uint2(e0[e], e1[e]);
                }
                sum += __shfl_xor(sum, 32, 64);
                if (hl == 0) dsum[w * 32 + j] = sum;
            } else {                                  // n_0 . q_t, lane = t
                float acc = 0.0f;
                for (int pcs = 0; pcs * 8 < a.D; ++pcs) {
                    const hy_u32x4 q = *(const HY_LDS hy_u32x4*)(lds3 + off + lane * DK * 2 + ((pcs ^ C::swz(lane)) << 4));
                    const float4 na = *(const float4*)(n + pcs * 8), nb = *(const float4*)(n + pcs * 8 + 4);
                    acc += __uint_as_float(q[0] << 16) * na.x + __uint_as_float(q[0] & 0xffff0000u) * na.y + __uint_as_float(q[1] << 16) * na.z + __uint_as_float(q[1] & 0xffff0000u) * na.w;
                    acc += __uint_as_float(q[2] << 16) * nb.x + __uint_as_float(q[2] & 0xffff0000u) * nb.y + __uint_as_float(q[3] << 16) * nb.z + __uint_as_float(q[3] & 0xffff0000u) * nb.w;
                }
                qn[lane] = acc * a.qscale;
            }
#pragma unroll
            for (int v = 0; v < 16; ++v) o[0][v] = o[1][v] = 0.0f;
            if (live) {                               // S_0^T q
#pragma unroll
                for (int db = 0; db < DKT; ++db)
#pragma unroll
                    for (int st_ = 0; st_ < 2; ++st_) {
                        uint32_t e0[2], e1[2], e2[2], e3[2];
                        split2<2>(S[db][8 * st_], S[db][8 * st_ + 1], e0);
                        split2<2>(S[db][8 * st_ + 2], S[db][8 * st_ + 3], e1);
                        split2<2>(S[db][8 * st_ + 4], S[db][8 * st_ + 5], e2);
                        split2<2>(S[db][8 * st_ + 6], S[db][8 * st_ + 7], e3);
                        const int pcs = db * 4 + st_ * 2;
#pragma unroll
                        for (int tb = 0; tb < 2; ++tb) {
                            const int r = tb * 32 + j;
                            const HY_LDS char* qp = lds3 + off + r * DK * 2 + hl * 8;
                            hy_u32x2 lo = *(const HY_LDS hy_u32x2*)(qp + ((pcs ^ C::swz(r)) << 4)), hi = *(const HY_LDS hy_u32x2*)(qp + (((pcs + 1) ^ C::swz(r)) << 4));
                            if (!FULL && pcs * 8 >= a.D) lo = hy_u32x2{0u, 0u};
                            if (!FULL && pcs * 8 + 8 >= a.D) hi = hy_u32x2{0u, 0u};
                            const hy_bf16x8 qf = __builtin_bit_cast(hy_bf16x8, __builtin_shufflevector(lo, hi, 0, 1, 2, 3));
#pragma unroll
                            for (int e = 1; e >= 0; --e)
                                o[tb] = mfma32(__builtin_bit_cast(hy_bf16x8, (hy_u32x4){e0[e], e1[e], e2[e], e3[e]}), qf, o[tb]);
                        }
                    }
            }
            __syncthreads();                          // weighted scores and sums are there
#pragma unroll
            for (int tb = 0; tb < 2; ++tb) {
                const float f = exp_fast(m0 - fmaxf(m0, gM[gb + tb * 32 + j])) * a.qscale;
#pragma unroll
                for (int v = 0; v < 16; ++v) o[tb][v] *= f;
            }
        }
        if (live) {
            const float keep = exp_fast(m0 - Mc);
#pragma unroll
            for (int db = 0; db < DKT; ++db)
#pragma unroll
                for (int v = 0; v < 16; ++v) S[db][v] *= keep;
#pragma unroll
            for (int st_ = 0; st_ < 4; ++st_) {
                const hy_bf16x8 vf = tr_read(off + 2 * C::QB, 256, vsw0, vsw1, st_, w);
                if (MODE != CHUNK_LOCAL) {
#pragma unroll
                    for (int tb = 0; tb < 2; ++tb) {
                        if (tb == 0 && st_ >= 2) continue;
#pragma unroll
                        for (int e = 1; e >= 0; --e) {
                            const char* pp = ck_lds + C::P0 + e * C::PPLANE + (tb * 32 + j) * C::PROW + (16 * st_ + 4 * hl) * 2;
                            const uint2 lo = *(const uint2*)pp, hi = *(const uint2*)(pp + 16);
                            o[tb] = mfma32(vf, __builtin_bit_cast(hy_bf16x8, (hy_u32x4){lo.x, lo.y, hi.x, hi.y}), o[tb]);
                        }
                    }
                }
                const hy_u32x4 vr = __builtin_bit_cast(hy_u32x4, vf);
                const float4 d0 = *(const float4*)(ws + 16 * st_ + 4 * hl), d1 = *(const float4*)(ws + 16 * st_ + 4 * hl + 8);
                uint32_t e0[3], e1[3], e2[3], e3[3];
                split2<3>(__uint_as_float(vr[0] << 16) * d0.x, __uint_as_float(vr[0] & 0xffff0000u) * d0.y, e0);
                split2<3>(__uint_as_float(vr[1] << 16) * d0.z, __uint_as_float(vr[1] & 0xffff0000u) * d0.w, e1);
                split2<3>(__uint_as_float(vr[2] << 16) * d1.x, __uint_as_float(vr[2] & 0xffff0000u) * d1.y, e2);
                split2<3>(__uint_as_float(vr[3] << 16) * d1.z, __uint_as_float(vr[3] & 0xffff0000u) * d1.w, e3);
#pragma unroll
                for (int db = 0; db < DKT; ++db) {
                    const hy_bf16x8 kf = tr_read(off + C::QB, DK * 2, ksw0, ksw1, st_, db);
#pragma unroll
                    for (int e = 2; e >= 0; --e)
                        S[db] = mfma32(kf, __builtin_bit_cast(hy_bf16x8, (hy_u32x4){e0[e], e1[e], e2[e], e3[e]}), S[db]);
                }
            }
        }
        // n: 16 pairs of features per wavefront and pass, four quarters of the tokens side by side
        {
            const float keep = exp_fast(m0 - Mc);
            const int pr = lane & 15, qt = lane >> 4;
#pragma unroll
            for (int pass = 0; pass < (DK + 127) / 128; ++pass) {
                const int d = pass * 128 + (w * 16 + pr) * 2;
                if (d < DK) {                         // DK = 32, 64: the first wavefronts only
                    float x = 0.0f, y = 0.0f;
#pragma unroll
                    for (int i = 0; i < 16; ++i) {
                        const int s = qt * 16 + i;
                        const uint32_t k2 = *(const HY_LDS uint32_t*)(lds3 + off + C::QB + s * DK * 2 + (((d >> 3) ^ C::swz(s)) << 4) + (d & 7) * 2);
                        const float f = ws[s];
                        x += f * __uint_as_float(k2 << 16);
                        y += f * __uint_as_float(k2 & 0xffff0000u);
                    }
                    x += __shfl_xor(x, 16, 64); y += __shfl_xor(y, 16, 64);
                    x += __shfl_xor(x, 32, 64); y += __shfl_xor(y, 32, 64);
                    if (qt == 0) { n[d] = keep * n[d] + x; n[d + 1] = keep * n[d + 1] + y; }
                }
            }
        }
        if (NB == 2) asm volatile("s_waitcnt vmcnt(0)" ::: "memory");   // the next chunk, requested a chunk ago: not the stores below
        if (live) {
            if (MODE != CHUNK_LOCAL) {
#pragma unroll
                for (int tb = 0; tb < 2; ++tb) {
                    const int t = tb * 32 + j;
                    const float M = fmaxf(m0, gM[gb + t]);
                    const float den = dsum[tb * 32 + j] + (tb ? dsum[64 + j] : 0.0f) + exp_fast(m0 - M) * qn[t];
                    const float inv = 1.0f / (fmaxf(fabsf(den), exp_fast(-(gF[gb + t] + M))) + 1e-6f);
                    bf16_t* orow = (bf16_t*)a.o + ((int64_t)(t0 + first + c * 64 + t) * a.H + h) * a.Dv + dv0 + w * 32;
                    if (c * 64 + t < len) {
#pragma unroll
                        for (int x = 0; x < 4; ++x) {
                            const int d = 8 * x + 4 * hl;           // Dv is a multiple of 8: four columns are in or out together
                            if (dv0 + w * 32 + d < a.Dv)
                                *(uint2*)(orow + d) = make_uint2(pack2(o[tb][4 * x] * inv, o[tb][4 * x + 1] * inv), pack2(o[tb][4 * x + 2] * inv, o[tb][4 * x + 3] * inv));
                        }
                    }
                }
            }
        }
        if (MODE == CHUNK_LOCAL) fsum += gF[gb + 63];
        m0 = gF[gb + 63] + Mc;
        if (NB == 1 && c + 1 < nchunks) {
            __syncthreads();
            request(c + 1, 0);
        }
    }
    if (MODE == CHUNK_OUTPUT) return;
    __syncthreads();                                  // n is complete
    float* dst = MODE == CHUNK_LOCAL ? ca.seg_S + sat * a.D * a.Dv : a.S + ((int64_t)slot * a.H + h) * a.D * a.Dv;
    if (live && col < a.Dv) {
#pragma unroll
        for (int db = 0; db < DKT; ++db)
#pragma unroll
            for (int v = 0; v < 16; ++v) {
                const int d = db * 32 + 8 * (v >> 2) + 4 * hl + (v & 3);
                if (FULL || d < a.D) dst[(int64_t)d * a.Dv + col] = S[db][v];
            }
    }
    if (dv0 == 0) {
        float* nd = MODE == CHUNK_LOCAL ? ca.seg_n + sat * a.D : a.nm + (1 - parity) * copy + at;
        for (int d = tid; d < a.D; d += 256) nd[d] = n[d];
        if (tid == 0) {
            if (MODE == CHUNK_LOCAL) { ca.seg_g[2 * sat] = fsum; ca.seg_g[2 * sat + 1] = m0; }
            else nd[a.D] = m0 * LN2;
        }
    }
}

// Chains the segments' contributions: every segment's own state is replaced by the state it starts from, and the state behind
// the last one becomes the sequence's.  One thread per element of S (then of n); the scalars are recomputed by everyone.
__global__ __launch_bounds__(256) void mlstm_join_kernel(ChunkArgs ca) {
    const MlstmArgs& a = ca.a;
    const int h = blockIdx.y, b = blockIdx.z, len = a.cu[b + 1] - a.cu[b], slot = a.slots[b];
    const int e = blockIdx.x * 256 + threadIdx.x, nS = a.D * a.Dv;
    if (e >= nS + a.D) return;
    const bool fresh = a.seen[2 * slot] == 0;
    const int parity = a.seen[2 * slot + 1] & 1;
    const int64_t copy = (int64_t)a.nslots * a.H * (a.D + 1), at = ((int64_t)slot * a.H + h) * (a.D + 1);
    const float* in = a.nm + parity * copy + at;
    float* S = a.S + ((int64_t)slot * a.H + h) * nS;
    float m = fresh ? 0.0f : in[a.D] * LOG2E, cur = fresh ? 0.0f : e < nS ? S[e] : in[e - nS];
    const int64_t s0 = ((int64_t)b * a.H + h) * ca.nseg;
    for (int s = 0; s < ca.nseg && s * ca.seg_len < len; ++s) {
        float* p = e < nS ? ca.seg_S + (s0 + s) * nS + e : ca.seg_n + (s0 + s) * a.D + (e - nS);
        const float own = *p, f = ca.seg_g[2 * (s0 + s)], ms = ca.seg_g[2 * (s0 + s) + 1];
        *p = cur;
        if (e == 0) ca.seg_m[s0 + s] = m;
        const float mn = fmaxf(f + m, ms);
        cur = exp_fast(f + m - mn) * cur + exp_fast(ms - mn) * own;
        m = mn;
    }
    float* out = a.nm + (1 - parity) * copy + at;
    if (e < nS) S[e] = cur; else out[e - nS] = cur;
    if (e == 0) out[a.D] = m * LN2;
}

template <int DKT, int MODE, bool FULL>
static int launch_chunk(const ChunkArgs& c, dim3 grid, hipStream_t s) {
    static bool opted_in[64] = {};
    int dev = 0;
    if (hipGetDevice(&dev) != hipSuccess || dev < 0 || dev >= 64) dev = -1;
    if (dev < 0 || !opted_in[dev]) {
        hipError_t e = hipFuncSetAttribute((const void*)mlstm_chunk_kernel<DKT, MODE, FULL>, hipFuncAttributeMaxDynamicSharedMemorySize, ChunkCfg<DKT>::LDS);
        if (e != hipSuccess) return (int)e;
        if (dev >= 0) opted_in[dev] = true;
    }
    hipLaunchKernelGGL((mlstm_chunk_kernel<DKT, MODE, FULL>), grid, dim3(256), ChunkCfg<DKT>::LDS, s, c);
    return 0;
}
template <int DKT, bool FULL>
static int launch_chunked(const ChunkArgs& c, int batch, hipStream_t s) {
    const MlstmArgs& a = c.a;
    const int vt = (a.Dv + 127) / 128;
    if (c.nseg == 1) return launch_chunk<DKT, CHUNK_WHOLE, FULL>(c, dim3(vt, a.H, batch), s);
    if (int rc = launch_chunk<DKT, CHUNK_LOCAL, FULL>(c, dim3(vt * c.nseg, a.H, batch), s)) return rc;
    hipLaunchKernelGGL(mlstm_join_kernel, dim3((a.D * a.Dv + a.D + 255) / 256, a.H, batch), dim3(256), 0, s, c);
    return launch_chunk<DKT, CHUNK_OUTPUT, FULL>(c, dim3(vt * c.nseg, a.H, batch), s);
}
// the chunk kernel reads 16-byte pieces of rows and holds one head's query/key features in registers
static bool chunk_fits(int64_t proj_stride, int q_off, int k_off, int v_off, int dim, int vdim, int dtype, int max_len, const void* proj) {
    return dtype == TRIMKV_BF16 && max_len > 1 && dim <= 256 && dim % 8 == 0 && vdim % 8 == 0 && proj_stride % 8 == 0 && (q_off | k_off | v_off) % 8 == 0 && !((uintptr_t)proj & 15);
}
static int chunk_segments(int batch, int max_len, int heads, int vdim) {
    const int64_t wgs = (int64_t)batch * heads * ((vdim + 127) / 128);
    int64_t n = (512 + wgs - 1) / wgs;                // two rounds of the chip
    const int most = max_len / 256;                   // at least four chunks each
    n = n > most ? most : n;
    return n < 1 ? 1 : (int)n;
}

}  // namespace trimkv

using namespace trimkv;

extern "C" const char* trimkv_mlstm_last_error(void) { return err_buf(); }

extern "C" int64_t trimkv_mlstm_workspace(int batch, int max_len, int heads, int dim, int vdim, int dtype) {
    if (batch <= 0 || max_len <= 1 || heads <= 0 || dim <= 0 || vdim <= 0 || dtype != TRIMKV_BF16) return 0;
    const int n = chunk_segments(batch, max_len, heads, vdim);
    return n == 1 ? 0 : (int64_t)batch * heads * n * ((int64_t)dim * vdim + dim + 3);
}

extern "C" int trimkv_mlstm(const void* proj, int64_t proj_stride, int q_off, int k_off, int v_off, const float* gates, const float* i_bias,
                            const float* f_bias, float gate_cap, float* state, float* norm_state, const int32_t* cu, const int32_t* slots, const int32_t* seen,
                            void* out, int batch, int max_len, int heads, int dim, int vdim, int num_slots, float q_scale, float* workspace, int dtype, void* stream) {
    const char* fn = "trimkv_mlstm";
    if (!proj || !gates || !i_bias || !f_bias || !state || !norm_state || !cu || !slots || !seen || !out) return fail(TRIMKV_ERR_NULL, "%s: null pointer argument", fn);
    HY_CHECK_DTYPE(fn, dtype);
    if (batch <= 0 || batch > 65535 || max_len <= 0 || heads <= 0 || heads > 65535 || dim <= 0 || vdim <= 0 || num_slots <= 0 || gate_cap <= 0.0f)
        return fail(TRIMKV_ERR_SHAPE, "%s: bad sizes batch=%d max_len=%d heads=%d dim=%d vdim=%d", fn, batch, max_len, heads, dim, vdim);
    if (max_len > (1 << 24) || (int64_t)heads * batch > (1 << 24)) return fail(TRIMKV_ERR_SHAPE, "%s: too many tokens or heads", fn);
    if (dim > 512) return fail(TRIMKV_ERR_UNSUPPORTED, "%s: query/key sizes up to 512 (got %d)", fn, dim);
    MlstmArgs a{proj, proj_stride, q_off, k_off, v_off, gates, i_bias, f_bias, gate_cap, state, norm_state, cu, slots, seen, out, heads, dim, vdim, num_slots, q_scale};
    hipStream_t s = (hipStream_t)stream;
    if (chunk_fits(proj_stride, q_off, k_off, v_off, dim, vdim, dtype, max_len, proj)) {
        ChunkArgs c{a};
        c.nseg = chunk_segments(batch, max_len, heads, vdim);
        if (c.nseg > 1) {
            if (!workspace) return fail(TRIMKV_ERR_WORKSPACE, "%s: a prompt of %d tokens needs a workspace (trimkv_mlstm_workspace)", fn, max_len);
            c.seg_len = ((max_len + c.nseg - 1) / c.nseg + 63) / 64 * 64;
            const int64_t n = (int64_t)batch * heads * c.nseg;
            c.seg_S = workspace; c.seg_n = c.seg_S + n * dim * vdim; c.seg_g = c.seg_n + n * dim; c.seg_m = c.seg_g + 2 * n;
        }
        int rc;
        if (dim == 256) rc = launch_chunked<8, true>(c, batch, s);
        else if (dim == 128) rc = launch_chunked<4, true>(c, batch, s);
        else if (dim == 64) rc = launch_chunked<2, true>(c, batch, s);
        else rc = dim <= 32 ? launch_chunked<1, false>(c, batch, s) : dim < 64 ? launch_chunked<2, false>(c, batch, s) : dim < 128 ? launch_chunked<4, false>(c, batch, s)
                                                                                                                     : launch_chunked<8, false>(c, batch, s);
        if (rc) return fail(rc, "%s: hipFuncSetAttribute failed (%d)", fn, rc);
        return launch_status(fn);
    }
    const dim3 grid((vdim + 63) / 64, heads, batch);
    const size_t lds = (3 * dim + 256 + 4) * sizeof(float);
    const int kw = (dim + 3) / 4;
    HY_BY_DTYPE(dtype, T,
        if (kw <= 16) hipLaunchKernelGGL((mlstm_recurrent_kernel<T, 16>), grid, dim3(256), lds, s, a);
        else if (kw <= 32) hipLaunchKernelGGL((mlstm_recurrent_kernel<T, 32>), grid, dim3(256), lds, s, a);
        else if (kw <= 64) hipLaunchKernelGGL((mlstm_recurrent_kernel<T, 64>), grid, dim3(256), lds, s, a);
        else hipLaunchKernelGGL((mlstm_recurrent_kernel<T, 128>), grid, dim3(256), lds, s, a));
    return launch_status(fn);
}
