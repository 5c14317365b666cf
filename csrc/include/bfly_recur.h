// Host-side launch API of csrc/kernels/recur.hip, forget.hip and pooled.hip: linear attention with a
// constant decay per head or a forget gate per channel, the selective scan, gated norms over whole rows or
// per head, and the preparation of pooled-block attention (norms over whole projections, paged append, block means). Every launcher is
// stream-ordered, allocation-free and synchronisation-free. `f32`: the activation element type is
// float (else bf16); norms, recurrences and their states are f32 in both.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

namespace bfly {

// Linear attention with a constant decay per head over packed rows: S <- decay[h] S + k v^T, o = S^T q, q, k
// [T, H, D] and v [T, H, Dv] rows of the activation type with row strides, first passed through silu when
// act == 1. dpow [H, n_pow]: dpow[h][i] = decay[h]^i, n_pow >= 65. state f32 [slots, H, D, Dv], o f32
// [T, H, Dv]. one_row: sequence s has the one row s. Sequences without a slot (-1) leave zeros. nrot > 0: the
// first 2 nrot dims of q and k are rotated (after act), dimension i with i + nrot, by cs [T, 2, nrot] (cosines,
// sines); k is multiplied by k_scale.
void launch_decay_scan(const void* q, long q_ld, const void* k, long k_ld, const void* v, long v_ld, const float* dpow,
                       int n_pow, float* state, const int* state_slots, const int* row_cu, int nseq,
                       const int* positions, int act, const float* cs, int nrot, float k_scale, float* o, int T, int H,
                       int D, int Dv, bool one_row, bool f32, hipStream_t s);
// Linear attention with a forget gate per head and channel over packed rows: f = lower + (1 - lower) sigmoid(z +
// f_bias), S <- diag(f) S + (1 - f) v^T, o = S^T act(q). q, z [T, H, D], v [T, H, Dv] rows of the activation type with
// row strides; f_bias, lower f32 [H * D]; state, o, one_row as above.
void launch_forget_scan(const void* q, long q_ld, const void* z, long z_ld, const void* v, long v_ld, const float* f_bias,
                        const float* lower, float* state, const int* state_slots, const int* row_cu, int nseq,
                        const int* positions, int act, float* o, int T, int H, int D, int Dv, bool one_row, bool f32,
                        hipStream_t s);
// out[t, h] = o[t, h] / sqrt(mean(o[t, h]^2) + eps) * w * act(gate[t, h]) * mul per head of Dv values; o f32 [T, H, Dv]
// contiguous, w f32 [Dv] (nullable), gate (nullable; act 0 sigmoid, 1 silu) and out rows of the activation type
void launch_head_norm_gate(const float* o, const float* w, float eps, const void* gate, long g_ld, int act, float mul,
                           void* out, long out_ld, int T, int H, int Dv, bool f32, hipStream_t s);
// out[t] = o[t] / sqrt(mean(o[t]^2) + eps) * w * sigmoid(gate[t]) * mul over whole rows of N values; o f32
// contiguous, gate (nullable) and out of the activation type with row strides
void launch_row_norm_gate(const float* o, const float* w, float eps, const void* gate, long g_ld, float mul, void* out,
                          long out_ld, int T, int N, bool f32, hipStream_t s);
// Selective scan over packed rows, per channel c and state n: dt = softplus(dtr + dt_bias), S <- exp(-exp(a_log)
// dt) S + dt x B, y = S . C + d x, out = y * silu(z). x, z, B, C rows of the activation type with row strides, dtr
// f32 [T, C] rows; a_log f32 [C, N], state f32 [slots, C, N], out [T, C] contiguous. N <= 256 (returns < 0 else).
int launch_selective_scan(const void* x, long x_ld, const float* dtr, long dt_ld, const void* b, long b_ld, const void* c,
                          long c_ld, const void* z, long z_ld, const float* a_log, const float* dt_bias, const float* d,
                          float* state, const int* state_slots, const int* row_cu, int nseq, const int* positions,
                          void* out, int T, int C, int N, bool f32, hipStream_t s);

// launch_selective_scan for a step whose sequence s has the one row s, with dtr = wdt low: low [T, R] rows, wdt [C, R]
int launch_selective_step(const void* x, long x_ld, const void* low, long l_ld, const void* wdt, int R, const void* b,
                          long b_ld, const void* c, long c_ld, const void* z, long z_ld, const float* a_log,
                          const float* dt_bias, const float* d, float* state, const int* state_slots, const int* positions,
                          void* out, int T, int C, int N, bool f32, hipStream_t s);

// RMS norm of a token's whole query row [H * D] and key row [G * D] (weights qw, kw of those sizes; nullptr: no
// norm), the queries copied to q_out [T, H, Dp] (zero padded), keys and values appended to K [blocks, G, BS, Dp],
// V [blocks, G, Dvp, BS] at slots[t] >= 0. pool > 0 (only for steps in which every row is a sequence of its
// own): a row that completes a block of `pool` positions also writes the block's mean key and value.
void launch_qk_norm_rows_kv(const void* q, long q_ld, const void* k, long k_ld, const void* v, long v_ld, const float* qw,
                            const float* kw, float eps, const int* slots, void* k_cache, void* v_cache, void* q_out, int T,
                            int H, int G, int D, int Dv, int Dp, int Dvp, int bs, int pool, int pool_rows, void* k_pool,
                            void* v_pool, const int* positions, const int* row_seq, const int* tables, int max_blocks,
                            bool f32, hipStream_t s);
// Block means: every row whose position completes a block of `pool` positions averages the block's cached keys
// and values into k_pool [blocks, G, pool_rows, Dp], v_pool [.., Dvp] (block b: the page n of its last
// position, index b - floor(n BS / pool)).
void launch_pool_blocks(const void* k_cache, const void* v_cache, const int* tables, int max_blocks, const int* row_seq,
                        const int* positions, const int* slots, int pool, int pool_rows, void* k_pool, void* v_pool,
                        int T, int G, int Dp, int Dvp, int bs, bool f32, hipStream_t s);

}  // namespace bfly
