// Sequence mixers for heterogeneous layer stacks, generic in head count, head sizes and element
// type (bf16 or f32 activations / caches; scores, softmax, angles, decays and state are f32):
//   rope_partial_kv_kernel    interleaved-pair rotary on the first 2 * nrot dims of q / k heads,
//                             fused with the paged append of k and v
//                             (K [blocks, G, BS, D] rows, V [blocks, G, Dv, BS] transposed: a
//                             page's keys are contiguous for the P V operand)
//   attn_window_paged_kernel  attention of packed rows over the paged cache: causal sliding
//                             window plus the always-visible first `keep_first` positions, and a
//                             per-head sink logit that only enters the softmax denominator
//   gla_scan_kernel           gated linear attention S <- diag(a) S + k v^T, o = S^T q with the
//                             state pooled in per-sequence slots
//   gla_out_kernel            per-head RMS norm of o, times silu(gate)
// Rows of a step are packed: sequence s owns rows row_cu[s] .. row_cu[s+1] (one row for a
// decoded token, several for a prompt chunk), positions[] gives each row's position.
#include <algorithm>

#include "bfly_common.h"
#include "bfly_mixers.h"

namespace bfly {

#include "attn_window.inc"

namespace {

template <typename T>
__global__ __launch_bounds__(256) void rope_partial_kv_kernel(T* __restrict__ q, long q_ld, T* __restrict__ k, long k_ld,
                                                              const T* __restrict__ v, long v_ld,
                                                              const int* __restrict__ positions,
                                                              const float* __restrict__ inv_freq, int nrot,
                                                              const int* __restrict__ slots, T* __restrict__ k_cache,
                                                              T* __restrict__ v_cache, int H, int G, int D, int Dv,
                                                              int bs) {
  const long t = blockIdx.x;
  const float p = (float)positions[t];
  const int slot = (slots && k) ? slots[t] : -1;
  // rotated pairs of the q heads, then of the k heads
  const int nq = H * nrot, nk = k ? G * nrot : 0;
  for (int i = threadIdx.x; i < nq + nk; i += blockDim.x) {
    const bool isq = i < nq;
    const int j = isq ? i : i - nq;
    const int h = j / nrot, r = j % nrot;
    T* ptr = (isq ? q + t * q_ld : k + t * k_ld) + (long)h * D + 2 * r;
    const float a = p * inv_freq[r];
    double sd, cd;
    sincos((double)a, &sd, &cd);
    const float c = (float)cd, s = (float)sd;
    const float u = (float)ptr[0], w = (float)ptr[1];
    ptr[0] = (T)(u * c - w * s);
    ptr[1] = (T)(w * c + u * s);
  }
  if (slot < 0) return;
  __syncthreads();      // the rotated k is read back below
  const long blk = slot / bs, off = slot % bs;
  for (int i = threadIdx.x; i < G * D; i += blockDim.x) {
    const int g = i / D, d = i % D;
    k_cache[((blk * G + g) * bs + off) * D + d] = k[t * k_ld + i];
  }
  for (int i = threadIdx.x; i < G * Dv; i += blockDim.x) {
    const int g = i / Dv, d = i % Dv;
    v_cache[((blk * G + g) * Dv + d) * bs + off] = v[t * v_ld + i];
  }
}

// row -> sequence map of a packed step (rows outside every sequence: -1)
__global__ void row_seq_kernel(const int* __restrict__ row_cu, int nseq, int* __restrict__ row_seq, int T) {
  const int t = blockIdx.x * blockDim.x + threadIdx.x;
  if (t >= T) return;
  int s = -1;
  for (int i = 0; i < nseq; ++i)
    if (t >= row_cu[i] && t < row_cu[i + 1]) { s = i; break; }
  row_seq[t] = s;
}

// Workgroup = (sequence, head, 64-column slice of Dv), 8 waves; wave w owns 8 columns. A lane is
// (column c = lane & 7, row group gg = lane >> 3) and keeps the NR rows d = gg * NR .. + NR - 1 of
// its column's state in registers, so a token costs NR fused updates per lane and three shuffles to
// sum the eight row groups: no barrier inside the token loop. Tokens are staged 16 at a time:
// their decays (a = exp(log sigmoid(z) / tau), f32), keys, scaled queries and values go to LDS in
// one pass (rows past D are zero, so the row loop needs no bound), the outputs of the 16 tokens
// leave through LDS in another.
template <typename T, int NR>
__global__ __launch_bounds__(512) void gla_scan_kernel(const T* __restrict__ q, long q_ld, const T* __restrict__ k,
                                                       long k_ld, const T* __restrict__ v, long v_ld,
                                                       const T* __restrict__ z, long z_ld, float* __restrict__ state,
                                                       const int* __restrict__ state_slots,
                                                       const int* __restrict__ row_cu,
                                                       const int* __restrict__ positions, float inv_tau,
                                                       float q_scale, float* __restrict__ o, int H, int D, int Dv) {
  constexpr int TB = 16, DP = 8 * NR, NT = 512;
  __shared__ __attribute__((aligned(16))) float sa[TB * DP], sk[TB * DP], sq[TB * DP];
  __shared__ float sv[TB][64], so[TB][64];
  const int s = blockIdx.x, h = blockIdx.y, c0 = blockIdx.z * 64;
  const int w = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int cl = 8 * w + (lane & 7), gg = lane >> 3;
  const int col = c0 + cl;
  const bool live = col < Dv;
  const int r0 = row_cu[s], r1 = row_cu[s + 1];
  const int slot = state_slots[s];
  if (r1 <= r0) return;
  if (slot < 0) {      // padding sequence of a fixed-shape step: defined output, no state
    for (int i = threadIdx.x; i < (r1 - r0) * 64; i += NT)
      if (c0 + (i & 63) < Dv) o[((long)(r0 + (i >> 6)) * H + h) * Dv + c0 + (i & 63)] = 0.f;
    return;
  }
  float* S = state + ((long)slot * H + h) * D * Dv;
  float st[NR];
  const bool fresh = positions[r0] == 0;
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int d = gg * NR + i;
    st[i] = (!fresh && live && d < D) ? S[(long)d * Dv + col] : 0.f;
  }
  for (int t0 = r0; t0 < r1; t0 += TB) {
    const int nb = min(TB, r1 - t0);
    for (int i = threadIdx.x; i < nb * DP; i += NT) {
      const int tt = i / DP, d = i - tt * DP;
      float a = 0.f, kk = 0.f, qq = 0.f;
      if (d < D) {
        const long t = t0 + tt;
        const float zz = (float)z[t * z_ld + (long)h * D + d];
        // log sigmoid(z) = -softplus(-z), stable on both sides
        float ls;
        if constexpr (sizeof(T) == 2) {   // bf16 inputs: hardware exp / log (f32, ~1 ulp)
          ls = zz < 0.f ? zz - __logf(1.f + __expf(zz)) : -__logf(1.f + __expf(-zz));
          a = __expf(ls * inv_tau);
        } else {
          ls = zz < 0.f ? zz - log1pf(expf(zz)) : -log1pf(expf(-zz));
          a = expf(ls * inv_tau);
        }
        kk = (float)k[t * k_ld + (long)h * D + d];
        qq = (float)q[t * q_ld + (long)h * D + d] * q_scale;
      }
      sa[i] = a;
      sk[i] = kk;
      sq[i] = qq;
    }
    for (int i = threadIdx.x; i < nb * 64; i += NT) {
      const int tt = i >> 6, c = i & 63;
      sv[tt][c] = (c0 + c < Dv) ? (float)v[(long)(t0 + tt) * v_ld + (long)h * Dv + c0 + c] : 0.f;
    }
    __syncthreads();
    for (int tt = 0; tt < nb; ++tt) {
      const float vv = sv[tt][cl];
      const f32x4* pa = reinterpret_cast<const f32x4*>(sa + tt * DP + gg * NR);
      const f32x4* pk = reinterpret_cast<const f32x4*>(sk + tt * DP + gg * NR);
      const f32x4* pq = reinterpret_cast<const f32x4*>(sq + tt * DP + gg * NR);
      float po = 0.f;
#pragma unroll
      for (int i4 = 0; i4 < NR / 4; ++i4) {
        const f32x4 a4 = pa[i4], k4 = pk[i4], q4 = pq[i4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          st[4 * i4 + j] = fmaf(a4[j], st[4 * i4 + j], k4[j] * vv);
          po = fmaf(q4[j], st[4 * i4 + j], po);
        }
      }
      po += __shfl_xor(po, 8, 64);
      po += __shfl_xor(po, 16, 64);
      po += __shfl_xor(po, 32, 64);
      if (gg == 0) so[tt][cl] = po;
    }
    __syncthreads();
    for (int i = threadIdx.x; i < nb * 64; i += NT) {
      const int tt = i >> 6, c = i & 63;
      if (c0 + c < Dv) o[((long)(t0 + tt) * H + h) * Dv + c0 + c] = so[tt][c];
    }
    // (the next block's staging overwrites sa / sk / sq / sv, which every wave finished reading
    // at the barrier above; so is rewritten only after the next block's first barrier)
  }
  if (live) {
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int d = gg * NR + i;
      if (d < D) S[(long)d * Dv + col] = st[i];
    }
  }
}

template <typename T>
__global__ __launch_bounds__(64) void gla_out_kernel(const float* __restrict__ o, const T* __restrict__ g, long g_ld,
                                                     const float* __restrict__ norm_w, float eps, T* __restrict__ out,
                                                     int H, int Dv) {
  const long t = blockIdx.x;
  const int h = blockIdx.y, lane = threadIdx.x;
  const float* row = o + (t * H + h) * Dv;
  float ss = 0.f;
  for (int d = lane; d < Dv; d += 64) ss = fmaf(row[d], row[d], ss);
  ss = wave_sum(ss);
  const float r = 1.f / sqrtf(ss / (float)Dv + eps);
  for (int d = lane; d < Dv; d += 64) {
    const float gg = (float)g[t * g_ld + (long)h * Dv + d];
    const float y = row[d] * r * norm_w[d];
    out[(t * H + h) * Dv + d] = (T)(y * (gg / (1.f + expf(-gg))));
  }
}

}  // namespace

void launch_rope_partial_kv(void* q, long q_ld, void* k, long k_ld, const void* v, long v_ld, const int* positions,
                            const float* inv_freq, int nrot, const int* slots, void* k_cache, void* v_cache,
                            int T, int H, int G, int D, int Dv, int block_size, bool f32, hipStream_t s) {
  if (T <= 0) return;
  if (f32)
    rope_partial_kv_kernel<float><<<T, 256, 0, s>>>((float*)q, q_ld, (float*)k, k_ld, (const float*)v, v_ld, positions,
                                                    inv_freq, nrot, slots, (float*)k_cache, (float*)v_cache, H, G, D,
                                                    Dv, block_size);
  else
    rope_partial_kv_kernel<bf16><<<T, 256, 0, s>>>((bf16*)q, q_ld, (bf16*)k, k_ld, (const bf16*)v, v_ld, positions,
                                                   inv_freq, nrot, slots, (bf16*)k_cache, (bf16*)v_cache, H, G, D, Dv,
                                                   block_size);
}

void launch_row_seq(const int* row_cu, int nseq, int* row_seq, int T, hipStream_t s) {
  if (T <= 0) return;
  row_seq_kernel<<<(T + 255) / 256, 256, 0, s>>>(row_cu, nseq, row_seq, T);
}

// launch_attn_window_mfma with AttnMod's extensions (attn_ext.hip)
bool launch_attn_window_mfma_ext(const void* q, long q_ld, const void* k_cache, const void* v_cache, const int* tables,
                                 int max_blocks, const int* row_cu, int nseq, const int* positions, float scale,
                                 int window, int keep_first, const float* sink, const float* out_scale, void* out, int T,
                                 int H, int G, int D, int Dv, int block_size, float* part, long part_floats,
                                 hipStream_t s, const AttnMod& md);

bool launch_attn_window_mfma(const void* q, long q_ld, const void* k_cache, const void* v_cache, const int* tables,
                             int max_blocks, const int* row_cu, int nseq, const int* positions, float scale, int window,
                             int keep_first, const float* sink, const float* out_scale, void* out, int T, int H, int G,
                             int D, int Dv, int block_size, bool fold, float* part, long part_floats, hipStream_t s,
                             const AttnMod& md) {
  if (md.ext())
    return launch_attn_window_mfma_ext(q, q_ld, k_cache, v_cache, tables, max_blocks, row_cu, nseq, positions, scale, window,
                                       keep_first, sink, out_scale, out, T, H, G, D, Dv, block_size, part, part_floats, s,
                                       md);
  return attn_mfma_launch<0>(q, q_ld, k_cache, v_cache, tables, max_blocks, row_cu, nseq, positions, scale, window,
                             keep_first, sink, out_scale, out, T, H, G, D, Dv, block_size, fold, part, part_floats, s, md);
}

void launch_attn_window_paged(const void* q, long q_ld, const void* k_cache, const void* v_cache, const int* tables,
                              int max_blocks, const int* row_seq, int nseq, const int* positions, float scale,
                              int window, int keep_first, const float* sink, const float* out_scale, void* out, int T,
                              int H, int G, int D, int Dv, int block_size, bool f32, hipStream_t s, const AttnMod& md) {
  if (T <= 0) return;
  (void)nseq;
  dim3 grid(T, H);
  const size_t sm = (size_t)(D + 64 + 2) * sizeof(float) + 64 * sizeof(long);
  if (f32)
    attn_window_paged_kernel<float><<<grid, 64, sm, s>>>((const float*)q, q_ld, (const float*)k_cache,
                                                         (const float*)v_cache, tables, max_blocks, row_seq, positions,
                                                         scale, window, keep_first, sink, out_scale, out, H, G,
                                                         D, Dv, block_size, md);
  else
    attn_window_paged_kernel<bf16><<<grid, 64, sm, s>>>((const bf16*)q, q_ld, (const bf16*)k_cache,
                                                        (const bf16*)v_cache, tables, max_blocks, row_seq, positions,
                                                        scale, window, keep_first, sink, out_scale, out, H, G, D,
                                                        Dv, block_size, md);
}

template <typename T>
static int gla_scan_t(const T* q, long q_ld, const T* k, long k_ld, const T* v, long v_ld, const T* z, long z_ld,
                      float* state, const int* state_slots, const int* row_cu, int nseq, const int* positions,
                      float tau, float q_scale, float* o, int H, int D, int Dv, hipStream_t s) {
  dim3 grid(nseq, H, (Dv + 63) / 64);
  const float it = 1.f / tau;
#define BFLY_GLA(NR)                                                                                              \
  gla_scan_kernel<T, NR><<<grid, 512, 0, s>>>(q, q_ld, k, k_ld, v, v_ld, z, z_ld, state, state_slots, row_cu, positions, \
                                              it, q_scale, o, H, D, Dv)
  if (D <= 32) BFLY_GLA(4);
  else if (D <= 64) BFLY_GLA(8);
  else if (D <= 128) BFLY_GLA(16);
  else if (D <= 256) BFLY_GLA(32);
  else return -1;
#undef BFLY_GLA
  return 0;
}

int launch_gla_scan(const void* q, long q_ld, const void* k, long k_ld, const void* v, long v_ld, const void* z,
                    long z_ld, float* state, const int* state_slots, const int* row_cu, int nseq,
                    const int* positions, float tau, float q_scale, float* o, int T, int H, int D, int Dv, bool f32,
                    hipStream_t s) {
  if (T <= 0 || nseq <= 0) return 0;
  if (f32)
    return gla_scan_t<float>((const float*)q, q_ld, (const float*)k, k_ld, (const float*)v, v_ld, (const float*)z, z_ld,
                             state, state_slots, row_cu, nseq, positions, tau, q_scale, o, H, D, Dv, s);
  return gla_scan_t<bf16>((const bf16*)q, q_ld, (const bf16*)k, k_ld, (const bf16*)v, v_ld, (const bf16*)z, z_ld, state,
                          state_slots, row_cu, nseq, positions, tau, q_scale, o, H, D, Dv, s);
}

void launch_gla_out(const float* o, const void* g, long g_ld, const float* norm_w, float eps, void* out, int T, int H,
                    int Dv, bool f32, hipStream_t s) {
  if (T <= 0) return;
  dim3 grid(T, H);
  if (f32) gla_out_kernel<float><<<grid, 64, 0, s>>>(o, (const float*)g, g_ld, norm_w, eps, (float*)out, H, Dv);
  else gla_out_kernel<bf16><<<grid, 64, 0, s>>>(o, (const bf16*)g, g_ld, norm_w, eps, (bf16*)out, H, Dv);
}

}  // namespace bfly
