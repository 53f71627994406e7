/*
 * trimkv_hybrid.h -- C ABI of the kernels of decoders that mix windowed attention with recurrent layers, dense feed-forwards
 * and routed experts, on MI355X (gfx950).  libtrimkv_hybrid.so holds all but trimkv_mlstm* (libtrimkv_mlstm.so) and
 * trimkv_moe_* (libtrimkv_moe.so), so that a decoder needs only what it uses.
 *
 * Conventions as in trimkv_hip.h: device pointers throughout, work enqueued on `stream`, no allocation and no host
 * synchronisation, 0 / negative trimkv_status / positive hipError_t, text of the last error of the calling thread from
 * trimkv_hybrid_last_error() (trimkv_mlstm_last_error(), trimkv_moe_last_error() of the other two).  `dtype` is the type of activations and matrices: TRIMKV_BF16 or TRIMKV_F32 (everything in
 * true fp32).  Norm weights, biases, gates, router logits, recurrent state and the residual stream are fp32 always.
 *
 * Batches are packed: the tokens of all sequences of a step lie one after the other, sequence b owns tokens
 * cu[b] .. cu[b+1]-1 (cu [batch+1] int32).  What a sequence leaves behind lives in a slot, slots[b] (int32); seen [slots][2]
 * int32 holds the tokens and the steps a slot has seen before this step (trimkv_advance moves both on at its end).  Slot
 * contents of a slot with 0 tokens are never read.
 */
#ifndef TRIMKV_HYBRID_H
#define TRIMKV_HYBRID_H

#include "trimkv_hip.h"

#ifdef __cplusplus
extern "C" {
#endif

const char* trimkv_hybrid_last_error(void);
const char* trimkv_mlstm_last_error(void);
const char* trimkv_moe_last_error(void);

/* x[t] = table[ids[t]] * scale as fp32 rows of x_stride elements (zeros behind `width`), or, with `add`, x[t] += that; xh
 * (optional): the same in dtype, or with norm_weight (needs xh) its RMS norm times that weight.  Ids outside [0, vocab) are
 * clamped. */
int trimkv_embed_scaled(const int64_t* ids, const void* table, float scale, float* x, void* xh, const float* norm_weight, float eps, int add,
                        int tokens, int vocab, int width, int x_stride, int dtype, void* stream);

/* out[t][o] = sum_k x[t][k] w[o][k], fp32 x and out, fp32 products and sums (bf16 w on the matrix cores: x split exactly into
 * three bf16 terms).  k and x_stride multiples of 4, w_stride a multiple of 8; 16-byte aligned. */
int trimkv_linear_f32(const float* x, int64_t x_stride, const void* w, int64_t w_stride, float* out, int rows, int n, int k, int dtype, void* stream);

/* x[t] += mult * w * y' / sqrt(mean(y'^2) + eps), y' = y[t] or, with y_weight [tokens][top], sum_j y_weight[t][j] * y[t * top + j].
 * xh (optional): the new x in dtype, same stride, or with next_w (needs xh) its RMS norm times that weight. width <= 16384. */
int trimkv_residual_norm(const void* y, int64_t y_stride, const float* y_weight, int top, float* x, const float* w, float mult, void* xh,
                         const float* next_w, int tokens, int width, int x_stride, float eps, int dtype, void* stream);

/* out[i] = w * x[r] / sqrt(mean(x[r]^2) + eps) with r = rows[i] (NULL: r = i); out [count][width] in dtype. */
int trimkv_rms_rows(const float* x, int x_stride, const int64_t* rows, const float* w, void* out, int count, int width, float eps, int dtype, void* stream);

/* RMS norm of q over all its heads at once, likewise k (weights of those sizes); v is copied.  proj rows hold q, k, v at
 * element offsets q_off, k_off, v_off.  Outputs [tokens][heads][dim_stride] / [tokens][kv_heads][(v)dim_stride], zeros behind
 * dim / vdim.  With slots and seen (one token per sequence): k and v are the window rings and the token goes into its slot. */
int trimkv_qkv_norm(const void* proj, int64_t proj_stride, int q_off, int k_off, int v_off, const float* q_weight, const float* k_weight, float eps,
                    int heads, int kv_heads, int dim, int vdim, int dim_stride, int vdim_stride, void* q, void* k, void* v,
                    const int32_t* slots, const int32_t* seen, int keep_first, int window, int tokens, int dtype, void* stream);

/* Cosines and sines of the positions of a step: table [tokens][rot_dims], the cosines of the rot_dims / 2 pairs, then their
 * sines; token i of sequence b stands at seen + i and pair j turns by that times freq[j] (fp64, radians per position). */
int trimkv_rotary_table(const double* freq, const int32_t* cu, const int32_t* slots, const int32_t* seen, float* table, int batch, int max_len,
                        int rot_dims, void* stream);

/* q, k, v heads of projection rows (layout and destinations as in trimkv_qkv_norm): + bias (optional; fp32, indexed like a row
 * of proj), RMS norm of each q and k head over its dim with one weight [dim] for all heads (optional, both or neither), rotation
 * of the pairs (i, i + rot_dims / 2) of q and k by the token's row of the table (rot_dims 0: none). */
int trimkv_qkv_heads(const void* proj, int64_t proj_stride, int q_off, int k_off, int v_off, const float* bias, const float* q_weight,
                     const float* k_weight, float eps, const float* table, int rot_dims, int heads, int kv_heads, int dim, int vdim,
                     int dim_stride, int vdim_stride, void* q, void* k, void* v, const int32_t* slots, const int32_t* seen, int keep_first,
                     int window, int tokens, int dtype, void* stream);

/* out[t][i] = silu(gate[t][i]) * up[t][i]; gate and up rows `stride` apart, out [tokens][inter]; computed in fp32. */
int trimkv_silu_gate(const void* gate, const void* up, int64_t stride, void* out, int tokens, int inter, int dtype, void* stream);

/* out[i] = cap * tanh(x[i] / cap), fp32 out; 16-byte aligned. */
int trimkv_soft_cap(const void* x, float* out, int64_t count, float cap, int dtype, void* stream);

/* Window rings [slot][kv_heads][keep_first + window][dim_stride]: position p < keep_first owns row p, a later one row
 * keep_first + (p - keep_first) % window.  Stores those tokens of a portion that no later token of it overwrites.
 * Padded sizes are multiples of 8, pointers 16-byte aligned. */
int trimkv_ring_store(const void* k, const void* v, const int32_t* cu, const int32_t* slots, const int32_t* seen, void* ring_k, void* ring_v,
                      int batch, int max_len, int kv_heads, int dim_stride, int vdim_stride, int keep_first, int window, int dtype, void* stream);

/* Attention of portions: position i sees j <= i with i - j < window or j < keep_first; earlier tokens from the rings (which
 * must not hold this portion yet), the portion's own from k and v.  out [tokens][heads * vdim] = attention * sigmoid(gate),
 * gate rows gate_stride apart with a number per output value or, with head_gate, per head.  sink: the softmax denominator has one
 * more term, exp(0). Padded sizes are multiples of 8 up to 512. */
int trimkv_window_prefill(const void* q, const void* k, const void* v, const void* ring_k, const void* ring_v, const int32_t* cu,
                          const int32_t* slots, const int32_t* seen, const void* gate, int64_t gate_stride, void* out, int batch, int max_len,
                          int heads, int kv_heads, int dim, int vdim, int dim_stride, int vdim_stride, int keep_first, int window,
                          float scale, int head_gate, int sink, int dtype, void* stream);

/* Attention of one new token per sequence, already stored in the rings (seen does not count it yet).  splits > 1: rows of a
 * sequence are split over that many workgroups, workspace [batch][heads][splits][vdim + 2] floats. */
int trimkv_window_decode_splits(int batch, int kv_heads, int capacity);
int trimkv_window_decode(const void* q, const void* ring_k, const void* ring_v, const int32_t* slots, const int32_t* seen,
                         const void* gate, int64_t gate_stride, void* out, int batch, int heads, int kv_heads, int dim, int vdim,
                         int dim_stride, int vdim_stride, int keep_first, int window, float scale, int head_gate, int sink, int splits, float* workspace,
                         int dtype, void* stream);

/* mLSTM over portions (equations in csrc/mlstm.hip). gates [tokens][2 heads]: W_i h, W_f h without biases.  state
 * [slot][heads][dim][vdim]; norm_state [2][num_slots][heads][dim + 1] (n and m, by parity of the slot's steps).
 * out [tokens][heads][vdim] in dtype, before the head norm.  dim up to 512.  workspace: trimkv_mlstm_workspace(...) floats (0: NULL will do), for the states
 * between the segments of long bf16 prompts. */
int64_t trimkv_mlstm_workspace(int batch, int max_len, int heads, int dim, int vdim, int dtype);
int trimkv_mlstm(const void* proj, int64_t proj_stride, int q_off, int k_off, int v_off, const float* gates, const float* i_bias,
                 const float* f_bias, float gate_cap, float* state, float* norm_state, const int32_t* cu, const int32_t* slots, const int32_t* seen,
                 void* out, int batch, int max_len, int heads, int dim, int vdim, int num_slots, float q_scale, float* workspace, int dtype, void* stream);

/* out[t][h][:] = w[h] * o / sqrt(mean(o^2) + eps) * sigmoid(gate), o [tokens][heads][vdim] in dtype; norm and gate in fp32. */
int trimkv_head_norm_gate(const void* o, const void* gate, int64_t gate_stride, const float* w, void* out, int tokens, int heads, int vdim, float eps, int dtype, void* stream);

/* seen[slots[b]] += {cu[b+1] - cu[b], 1}. */
int trimkv_advance(int32_t* seen, const int32_t* slots, const int32_t* cu, int batch, void* stream);

/* Sigmoid routing: choice = sigmoid(logits) + correction; `keep_groups` of `groups` equal groups of neighbours with the
 * largest sums of their two largest choices are open; the `top` largest open choices win (lower index first among equals).
 * weights: the plain sigmoids of the chosen. experts <= 1024. */
int trimkv_moe_route(const float* logits, const float* correction, int32_t* ids, float* weights, int tokens, int experts, int top, int groups,
                     int keep_groups, void* stream);

/* Orders rows = tokens * top by expert: order [rows], offsets [experts + 1], tiles [1 + 2 * most]: their number, then
 * (expert, first row) of every run of up to `tile` rows; most = rows < experts ? rows : (rows - experts) / tile + experts. */
int trimkv_moe_plan(const int32_t* ids, int rows, int experts, int tile, int32_t* order, int32_t* offsets, int32_t* tiles, void* stream);

/* One product per expert.  w: n and k padded with zeros to multiples of 64, stored in blocks of 32 outputs x 16 k as the matrix
 * cores take them, [experts][n_padded / 32][k_padded / 16][2][32][8]: first k 0..7 of the block's 32 outputs, then k 8..15.
 * up: y[i] = relu(w x[order[i] / top])^2; else y[order[i]] = w x[i].  x rows hold k_padded elements.  `tile` as in the plan:
 * 16 in fp32, in bf16 32 (a few rows per expert) or 256. */
int trimkv_moe_gemm(const void* x, int64_t x_stride, const void* w, void* y, int64_t y_stride, const int32_t* order, const int32_t* offsets,
                    const int32_t* tiles, int rows, int experts, int tile, int top, int n, int n_padded, int k_padded, int up, int dtype, void* stream);

#ifdef __cplusplus
}
#endif
#endif
