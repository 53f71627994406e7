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
    float* o;                                                   // [T][H][Dv]
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
    float s[KMAX];
#pragma unroll
    for (int x = 0; x < KMAX; ++x) s[x] = fresh || x >= nd ? 0.0f : Sp[(int64_t)x * a.Dv];
    for (int d = tid; d < a.D; d += 256) n[d] = fresh ? 0.0f : nm_in[d];
    float m = fresh ? 0.0f : nm_in[a.D];
    const float ib = a.ib[h], fb = a.fb[h];
    for (int t = 0; t < len; ++t) {
        const int64_t tok = t0 + t;
        const T* row = (const T*)a.p + tok * a.p_stride;
        const float li = log_input_gate(a.gates[tok * 2 * a.H + h] + ib, a.cap);
        const float lf = log_forget_gate(a.gates[tok * 2 * a.H + a.H + h] + fb, a.cap);
        const float v = ld(row + a.v_off + h * a.Dv + (cin ? col : 0));
        const float mn = fmaxf(lf + m, li), keep = expf(lf + m - mn), add = expf(li - mn);
        m = mn;
        float qn = 0.0f;
        for (int d = tid; d < a.D; d += 256) {
            const float qq = ld(row + a.q_off + h * a.D + d) * a.qscale, kk = ld(row + a.k_off + h * a.D + d);
            q[d] = qq; k[d] = kk;
            const float nn = keep * n[d] + add * kk;
            n[d] = nn;
            qn += nn * qq;
        }
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
            a.o[(tok * a.H + h) * a.Dv + col] = num / (fmaxf(fabsf(qn), expf(-m)) + 1e-6f);
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

}  // namespace trimkv

using namespace trimkv;

extern "C" int trimkv_mlstm(const void* proj, int64_t proj_stride, int q_off, int k_off, int v_off, const float* gates, const float* i_bias,
                            const float* f_bias, float gate_cap, float* state, float* norm_state, const int32_t* cu, const int32_t* slots, const int32_t* seen,
                            float* out, int batch, int max_len, int heads, int dim, int vdim, int num_slots, float q_scale, int dtype, void* stream) {
    const char* fn = "trimkv_mlstm";
    if (!proj || !gates || !i_bias || !f_bias || !state || !norm_state || !cu || !slots || !seen || !out) return fail(TRIMKV_ERR_NULL, "%s: null pointer argument", fn);
    HY_CHECK_DTYPE(fn, dtype);
    if (batch <= 0 || batch > 65535 || max_len <= 0 || heads <= 0 || heads > 65535 || dim <= 0 || vdim <= 0 || num_slots <= 0 || gate_cap <= 0.0f)
        return fail(TRIMKV_ERR_SHAPE, "%s: bad sizes batch=%d max_len=%d heads=%d dim=%d vdim=%d", fn, batch, max_len, heads, dim, vdim);
    if (dim > 512) return fail(TRIMKV_ERR_UNSUPPORTED, "%s: query/key sizes up to 512 (got %d)", fn, dim);
    MlstmArgs a{proj, proj_stride, q_off, k_off, v_off, gates, i_bias, f_bias, gate_cap, state, norm_state, cu, slots, seen, out, heads, dim, vdim, num_slots, q_scale};
    hipStream_t s = (hipStream_t)stream;
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
