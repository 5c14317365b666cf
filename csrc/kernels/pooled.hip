// Preparation of pooled-block attention, generic in every size and in the element type (bf16 or f32):
//   qk_norm_rows_kv_kernel   RMS norms over a token's whole query and key projections, a padded query copy,
//                            the paged append, and in steps of one row per sequence the block means
//   pool_blocks_kernel       mean key and value of every block that a row of the step completes
// Block b of P positions lives in the page n of its last position, at index b - floor(n BS / P) of that page's
// ceil(BS / P) pooled rows: pooled rows are handed out, reused and freed with the pages themselves.
#include <algorithm>

#include "bfly_common.h"
#include "bfly_recur.h"

namespace bfly {

namespace {

template <typename T>
struct PoolArgs {
  int pool, pool_rows, max_blocks;
  T* k_pool;
  T* v_pool;
  const int* positions;
  const int* row_seq;
  const int* tables;
};

// The mean of block b = (p + 1) / P - 1, whose last position p is in the cache, for key / value head g. Entries
// [0, Dp) are the key's, [Dp, Dp + Dvp) the value's; the sum runs over ascending positions.
template <typename T>
__device__ __forceinline__ void pool_block(const T* k_cache, const T* v_cache, int p, const int* tab, int g, int G, int Dp, int Dvp, int bs,
                                           const PoolArgs<T>& pa, int i) {
  const int P = pa.pool, b = (p + 1) / P - 1, first = b * P;
  float a = 0.f;
  int page = first / bs, off = first - page * bs;
  for (int j = 0; j < P;) {
    const long blk = tab[page];
    const int run = min(P - j, bs - off);
    // (eight loads in flight; the sum stays in ascending order)
    const bool key = i < Dp;
    const T* src = key ? k_cache + ((blk * G + g) * bs + off) * Dp + i : v_cache + ((blk * G + g) * Dvp + (i - Dp)) * bs + off;
    const long step = key ? Dp : 1;
    int u = 0;
    for (; u + 8 <= run; u += 8) {
      float x[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) x[e] = (float)src[(u + e) * step];
#pragma unroll
      for (int e = 0; e < 8; ++e) a += x[e];
    }
    for (; u < run; ++u) a += (float)src[u * step];
    j += run;
    ++page;
    off = 0;
  }
  a /= (float)P;
  const int n = p / bs;
  const long row = ((long)tab[n] * G + g) * pa.pool_rows + (b - (n * bs) / P);
  if (i < Dp) pa.k_pool[row * Dp + i] = (T)a;
  else pa.v_pool[row * Dvp + (i - Dp)] = (T)a;
}

// One workgroup per row. The sums of squares of the query and the key row are taken together.
template <typename T, int V>
__global__ __launch_bounds__(256) void qk_norm_rows_kv_kernel(const T* __restrict__ q, long q_ld,
                                                              const T* __restrict__ k, long k_ld,
                                                              const T* __restrict__ v, long v_ld,
                                                              const float* __restrict__ qw,
                                                              const float* __restrict__ kw, float eps,
                                                              const int* __restrict__ slots, T* __restrict__ k_cache,
                                                              T* __restrict__ v_cache, T* __restrict__ q_out, int H,
                                                              int G, int D, int Dv, int Dp, int Dvp, int bs,
                                                              PoolArgs<T> pa) {
  typedef T tv __attribute__((ext_vector_type(V)));
  typedef float fv __attribute__((ext_vector_type(V)));
  __shared__ float red[16];
  const long t = blockIdx.x;
  const int nq = H * D, nk = G * D, tid = threadIdx.x;
  const T *qr = q + t * q_ld, *kr = k + t * k_ld, *vr = v + t * v_ld;
  float rq = 1.f, rk = 1.f;
  if (qw) {
    float ss = 0.f;
    for (int c = V * tid; c < nq; c += V * 256) {
      const tv x = *reinterpret_cast<const tv*>(qr + c);
#pragma unroll
      for (int e = 0; e < V; ++e) ss = fmaf((float)x[e], (float)x[e], ss);
    }
    rq = 1.f / sqrtf(block_sum(ss, red) / (float)nq + eps);
  }
  if (kw) {
    float ss = 0.f;
    for (int c = V * tid; c < nk; c += V * 256) {
      const tv x = *reinterpret_cast<const tv*>(kr + c);
#pragma unroll
      for (int e = 0; e < V; ++e) ss = fmaf((float)x[e], (float)x[e], ss);
    }
    rk = 1.f / sqrtf(block_sum(ss, red) / (float)nk + eps);
  }
  for (int c = V * tid; c < nq; c += V * 256) {
    const tv x = *reinterpret_cast<const tv*>(qr + c);
    const fv w = qw ? *reinterpret_cast<const fv*>(qw + c) : fv(1.f);
    tv y;
#pragma unroll
    for (int e = 0; e < V; ++e) y[e] = (T)((float)x[e] * rq * w[e]);
    const int h = c / D;
    *reinterpret_cast<tv*>(q_out + (t * H + h) * Dp + (c - h * D)) = y;
  }
  if (Dp > D)
    for (int i = tid; i < H * (Dp - D); i += 256) q_out[(t * H + i / (Dp - D)) * Dp + D + i % (Dp - D)] = (T)0.f;
  const int slot = slots[t];
  if (slot < 0) return;
  const long blk = slot / bs, off = slot % bs;
  for (int c = V * tid; c < nk; c += V * 256) {
    const tv x = *reinterpret_cast<const tv*>(kr + c);
    const fv w = kw ? *reinterpret_cast<const fv*>(kw + c) : fv(1.f);
    tv y;
#pragma unroll
    for (int e = 0; e < V; ++e) y[e] = (T)((float)x[e] * rk * w[e]);
    const int g = c / D;
    *reinterpret_cast<tv*>(k_cache + ((blk * G + g) * bs + off) * Dp + (c - g * D)) = y;
  }
  for (int c = tid; c < G * Dv; c += 256) {
    const int g = c / Dv;
    v_cache[((blk * G + g) * Dvp + (c - g * Dv)) * bs + off] = vr[c];
  }
  // one row per sequence: the block's other positions are in the cache since earlier steps, this
  // one's since the writes above
  if (pa.pool > 0) {
    const int p = pa.positions[t], s = pa.row_seq[t];
    if (s >= 0 && (p + 1) % pa.pool == 0) {      // (the whole workgroup)
      __threadfence_block();
      __syncthreads();
      const int* tab = pa.tables + (long)s * pa.max_blocks;
      for (int i = tid; i < G * (Dp + Dvp); i += 256)
        pool_block(k_cache, v_cache, p, tab, i / (Dp + Dvp), G, Dp, Dvp, bs, pa, i % (Dp + Dvp));
    }
  }
}

// Workgroup = (32 rows of the step, key / value head): every wave finds the rows that complete a block and
// all threads average those blocks one after the other.
template <typename T>
__global__ __launch_bounds__(256) void pool_blocks_kernel(const T* __restrict__ k_cache, const T* __restrict__ v_cache,
                                                          const int* __restrict__ slots, int T_, int G, int Dp, int Dvp,
                                                          int bs, PoolArgs<T> pa) {
  const int lane = threadIdx.x & 63, t = blockIdx.x * 32 + lane;
  int s = -1, p = 0;
  if (lane < 32 && t < T_) {
    p = pa.positions[t];
    s = slots[t] >= 0 && (p + 1) % pa.pool == 0 ? pa.row_seq[t] : -1;
  }
  unsigned long long todo = __ballot(s >= 0);
  while (todo) {
    const int l = __ffsll(todo) - 1;
    todo &= todo - 1;
    const int* tab = pa.tables + (long)__shfl(s, l) * pa.max_blocks;
    const int pl = __shfl(p, l);
    for (int i = threadIdx.x; i < Dp + Dvp; i += 256)
      pool_block(k_cache, v_cache, pl, tab, (int)blockIdx.y, G, Dp, Dvp, bs, pa, i);
  }
}

template <typename T>
void qk_norm_rows_t(const T* q, long q_ld, const T* k, long k_ld, const T* v, long v_ld, const float* qw, const float* kw,
                    float eps, const int* slots, T* k_cache, T* v_cache, T* q_out, int T_, int H, int G, int D, int Dv,
                    int Dp, int Dvp, int bs, const PoolArgs<T>& pa, hipStream_t s) {
  const bool vec = D % 4 == 0 && Dp % 4 == 0 && q_ld % 4 == 0 && k_ld % 4 == 0 &&
                   reinterpret_cast<uintptr_t>(q) % (4 * sizeof(T)) == 0 &&
                   reinterpret_cast<uintptr_t>(k) % (4 * sizeof(T)) == 0;
  if (vec)
    qk_norm_rows_kv_kernel<T, 4><<<T_, 256, 0, s>>>(q, q_ld, k, k_ld, v, v_ld, qw, kw, eps, slots, k_cache, v_cache, q_out, H,
                                                    G, D, Dv, Dp, Dvp, bs, pa);
  else
    qk_norm_rows_kv_kernel<T, 1><<<T_, 256, 0, s>>>(q, q_ld, k, k_ld, v, v_ld, qw, kw, eps, slots, k_cache, v_cache, q_out, H,
                                                    G, D, Dv, Dp, Dvp, bs, pa);
}

}  // namespace

void launch_qk_norm_rows_kv(const void* q, long q_ld, const void* k, long k_ld, const void* v, long v_ld, const float* qw,
                            const float* kw, float eps, const int* slots, void* k_cache, void* v_cache, void* q_out, int T,
                            int H, int G, int D, int Dv, int Dp, int Dvp, int bs, int pool, int pool_rows, void* k_pool,
                            void* v_pool, const int* positions, const int* row_seq, const int* tables, int max_blocks,
                            bool f32, hipStream_t s) {
  if (T <= 0) return;
  if (f32)
    qk_norm_rows_t<float>((const float*)q, q_ld, (const float*)k, k_ld, (const float*)v, v_ld, qw, kw, eps, slots,
                          (float*)k_cache, (float*)v_cache, (float*)q_out, T, H, G, D, Dv, Dp, Dvp, bs,
                          {pool, pool_rows, max_blocks, (float*)k_pool, (float*)v_pool, positions, row_seq, tables}, s);
  else
    qk_norm_rows_t<bf16>((const bf16*)q, q_ld, (const bf16*)k, k_ld, (const bf16*)v, v_ld, qw, kw, eps, slots,
                         (bf16*)k_cache, (bf16*)v_cache, (bf16*)q_out, T, H, G, D, Dv, Dp, Dvp, bs,
                         {pool, pool_rows, max_blocks, (bf16*)k_pool, (bf16*)v_pool, positions, row_seq, tables}, s);
}

void launch_pool_blocks(const void* k_cache, const void* v_cache, const int* tables, int max_blocks, const int* row_seq,
                        const int* positions, const int* slots, int pool, int pool_rows, void* k_pool, void* v_pool,
                        int T, int G, int Dp, int Dvp, int bs, bool f32, hipStream_t s) {
  if (T <= 0 || pool <= 0) return;
  if (f32)
    pool_blocks_kernel<float><<<dim3((T + 31) / 32, G), 256, 0, s>>>(
        (const float*)k_cache, (const float*)v_cache, slots, T, G, Dp, Dvp, bs,
        {pool, pool_rows, max_blocks, (float*)k_pool, (float*)v_pool, positions, row_seq, tables});
  else
    pool_blocks_kernel<bf16><<<dim3((T + 31) / 32, G), 256, 0, s>>>(
        (const bf16*)k_cache, (const bf16*)v_cache, slots, T, G, Dp, Dvp, bs,
        {pool, pool_rows, max_blocks, (bf16*)k_pool, (bf16*)v_pool, positions, row_seq, tables});
}

}  // namespace bfly
