// Linear attention with a gate per head and channel as decay and its complement as key, and the norm per head that
// follows a linear attention; generic in every size and in the activation type (bf16 or f32; gates, decays, states
// and the recurrence are f32 in both):
//   forget_chunk_kernel, forget_step_kernel   f = l + (1 - l) sigmoid(z + b), S <- diag(f) S + (1 - f) v^T, o = S^T q,
//                                             in chunks on the f32 matrix cores or row by row
//   head_norm_gate_kernel                     RMS norm per head, times an optional weight, a gate and a factor
// Rows of a step are packed: sequence s owns rows row_cu[s] .. row_cu[s+1]; a sequence whose first row is at
// position 0 starts from a zero state whatever its slot holds.
#include <algorithm>
#include <type_traits>

#include "bfly_recur.h"
#include "bfly_recur_dev.h"

namespace bfly {

namespace {

// sigmoid(x) and its complement, each with its own relative accuracy
template <bool FAST>
__device__ __forceinline__ void sigmoid2(float x, float& s, float& c) {
  const float e = FAST ? __expf(-fabsf(x)) : expf(-fabsf(x));
  const float r = FAST ? __builtin_amdgcn_rcpf(1.f + e) : 1.f / (1.f + e);
  s = x < 0.f ? e * r : r;
  c = x < 0.f ? r : e * r;
}

// One element at a byte offset below 2^31 from a uniform base. (Rows of one chunk; callers clamp row and channel to the
// tensor.)
__device__ __forceinline__ __amdgpu_buffer_rsrc_t rows_rsrc(const void* base) {
  return __builtin_amdgcn_make_buffer_rsrc(const_cast<void*>(base), (short)0, 0x7fffffff, 0x00027000);
}
template <typename T>
__device__ __forceinline__ T row_load(__amdgpu_buffer_rsrc_t r, int off) {
  if constexpr (sizeof(T) == 2) return __builtin_bit_cast(T, __builtin_amdgcn_raw_buffer_load_b16(r, off, 0, 0));
  else return __builtin_bit_cast(T, __builtin_amdgcn_raw_buffer_load_b32(r, off, 0, 0));
}

// sum over the 32 lanes of a half wave, in its upper sixteen lanes
__device__ __forceinline__ float half_sum(float v) {
  v = row16_sum(v);
  return v + __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x142, 0xA, 0xF, false));
}

// Chunks of 16 rows. Workgroup = (sequence, head, 64 value columns), eight waves: wave & 3 names 16 columns, wave >> 2 a half
// of the state's rows. With F_t = f_0 .. f_t and B_j = f_(j+1) .. f_(n-1) (products per channel over the chunk's rows)
// and S the state before it,
//   o_t = (q_t F_t) S + sum_(j <= t) (sum_d q_td k_jd f_(j+1)d .. f_td) v_j,      S <- diag(F_(n-1)) S + sum_j (k_j B_j) v_j^T
// with k = 1 - f. Only products of decays occur, never quotients, so gates of any size are safe. The inputs of one
// channel are held by two lanes of a wave, eight rows each, which form the running products on the way into LDS: the
// first DP of 2 DP roles stage q, f and q F, the others k and k B. The products with the state and with v run on the f32
// matrix cores (16x16x4 tiles); a wave keeps its part of the state in the accumulator layout (tile i, element e: row d =
// 16 i + 4 gg + e of lane group gg), which is also the B operand of (q F) S. Of the 16 x 16 weights of the second sum the
// block t >= 8 > j is such a product too, with the decays split at row 8 (both factors are the lanes' own running
// products); the two 8 x 8 blocks on the diagonal are formed on the vector units while the matrix cores are busy: 32
// lanes per row t share its channels, and q_t times the decays so far is carried down j. Rows past the sequence have f = 1,
// k = q = 0. D <= 16 NT, NT even.
template <typename T, int NT>
__global__ __launch_bounds__(512, NT <= 8 ? 4 : 2) void forget_chunk_kernel(const T* __restrict__ q, long q_ld, const T* __restrict__ z,
                                                           long z_ld, const T* __restrict__ v, long v_ld,
                                                           const float* __restrict__ f_bias,
                                                           const float* __restrict__ lower, float* __restrict__ state,
                                                           const int* __restrict__ state_slots,
                                                           const int* __restrict__ row_cu,
                                                           const int* __restrict__ positions, int act, int vec,
                                                           float* __restrict__ o, int H, int D, int Dv) {
  constexpr int C = 16, DP = 16 * NT, NH = NT / 2, NU = (DP + 127) / 128, KP = 128 * NU + 4, VP = 68, PP = C + 4;
  constexpr int NI = (2 * DP + 255) / 256, HC = C / 2, NP = NT < 8 ? NT : 8;
  constexpr bool FAST = sizeof(T) == 2, WHOLE = NI * 256 == 2 * DP;
  extern __shared__ __attribute__((aligned(16))) float smem[];
  float* sq = smem;                     // [C][KP] q
  float* sk = sq + C * KP;              // [C][KP] k
  float* sf = sk + C * KP;              // [C + 1][KP] f; row C holds ones
  float* sqf = sf + (C + 1) * KP;       // [C][KP] q F
  float* skb = sqf + C * KP;            // [C][KP] k B
  float* sqh = skb + C * KP;            // [HC][KP] q times the decays from row 8 on, of rows 8 .. 15
  float* skh = sqh + HC * KP;           // [HC][KP] k times the decays up to row 7, of rows 0 .. 7
  float* sv = skh + HC * KP;            // [C][VP]
  float* so = sv + C * VP;              // [C][VP] (q F) S over the second half of the state's rows
  float* sp = so + C * VP;              // [C][PP] weights; those of rows 8 .. 15 on columns 0 .. 7 come as the sum of
  float* sph = sp + C * PP;             // [NP][HC][HC] the waves' parts
  float* sl = sph + NP * HC * HC;       // [DP] F of the last row
  const int s = blockIdx.x, h = blockIdx.y, c0 = blockIdx.z * 64;
  const int r0 = __builtin_amdgcn_readfirstlane(row_cu[s]), r1 = __builtin_amdgcn_readfirstlane(row_cu[s + 1]);
  if (r1 <= r0) return;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, m = lane & 15, gg = lane >> 4;
  const int slot = state_slots[s];
  if (slot < 0) {      // padding sequence of a fixed-shape step: defined output, no state
    for (int i = tid; i < (r1 - r0) * 64; i += 512)
      if (c0 + (i & 63) < Dv) o[((long)(r0 + (i >> 6)) * H + h) * Dv + c0 + (i & 63)] = 0.f;
    return;
  }
  const int cl = 16 * (wave & 3) + m, col = c0 + cl, d0 = (wave >> 2) * 16 * NH;
  const bool live = col < Dv;
  float* S = state + ((long)slot * H + h) * D * Dv + col;
  const bool fresh = positions[r0] == 0;
  f32x4 st[NH];
#pragma unroll
  for (int i = 0; i < NH; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int d = d0 + 16 * i + 4 * gg + e;
      st[i][e] = (!fresh && live && d < D) ? S[(long)d * Dv] : 0.f;
    }
  for (int i = tid; i < KP; i += 512) sf[C * KP + i] = 1.f;
  if (tid < HC * HC) sp[(tid / HC) * PP + HC + tid % HC] = 0.f;      // (above the diagonal blocks, never written again)
  if (DP < 128 * NU) {      // columns that no role stages
    constexpr int R = 128 * NU - DP > 0 ? 128 * NU - DP : 1;
    for (int i = tid; i < C * R; i += 512) {
      const int at = (i / R) * KP + DP + i % R;
      sq[at] = sk[at] = 0.f;
      sf[at] = 1.f;
    }
  }
  // this thread's roles: channel, rows ra .. ra + 7, bias and lower bound
  const int role = 32 * wave + (lane & 31), hf = lane >> 5, ra = HC * hf;
  float rb[NI], rl[NI];
#pragma unroll
  for (int u = 0; u < NI; ++u) {
    const int idx = role + 256 * u, d = min(idx < DP ? idx : idx - DP, D - 1);
    rb[u] = f_bias[(long)h * D + d];
    rl[u] = lower[(long)h * D + d];
  }
  // the next chunk's inputs as they are stored (rows past the sequence: its last row again)
  typedef T t4 __attribute__((ext_vector_type(4)));
  T rq[NI][HC], rz[NI][HC];
  t4 rv;
  auto fetch = [&](int t0) {
    const __amdgpu_buffer_rsrc_t qb = rows_rsrc(q + (long)t0 * q_ld + (long)h * D);
    const __amdgpu_buffer_rsrc_t zb = rows_rsrc(z + (long)t0 * z_ld + (long)h * D);
    const int qs = (int)q_ld * (int)sizeof(T), zs = (int)z_ld * (int)sizeof(T), last = r1 - 1 - t0;
#pragma unroll
    for (int u = 0; u < NI; ++u) {
      const int idx = role + 256 * u;
      const int d = min(idx < DP ? idx : idx - DP, D - 1) * (int)sizeof(T);
      if (idx < DP) {
#pragma unroll
        for (int i = 0; i < HC; ++i) rq[u][i] = row_load<T>(qb, __umul24(min(ra + i, last), qs) + d);
      }
      if (WHOLE || idx < 2 * DP) {
#pragma unroll
        for (int i = 0; i < HC; ++i) rz[u][i] = row_load<T>(zb, __umul24(min(ra + i, last), zs) + d);
      }
    }
    if (tid >= 256) return;
    const T* vr = v + (long)min(t0 + (tid >> 4), r1 - 1) * v_ld + (long)h * Dv;
    const int c = c0 + 4 * (tid & 15);
    if (vec & 2) {
      rv = *reinterpret_cast<const t4*>(vr + min(c, Dv - 4));
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) rv[e] = vr[min(c + e, Dv - 1)];
    }
  };
  // Gates of this thread's channels into LDS. No branch on rows or channels: a row past the sequence is set to f = 1, k =
  // q = 0 by factors (`tail`: the last chunk has such rows), a channel past D has q = 0 (its state row is never read or
  // stored). The running products cross from one half of the rows to the other between lanes l and l + 32.
  auto stage = [&](int n, auto tail) {
#pragma unroll
    for (int u = 0; u < NI; ++u) {
      const int idx = role + 256 * u;
      const float one = 1.f - rl[u];
      if (idx < DP) {
        const float qm = idx < D ? 1.f : 0.f;
        float F = 1.f, w[HC];
#pragma unroll
        for (int i = 0; i < HC; ++i) {
          float sg, cg;
          sigmoid2<FAST>((float)rz[u][i] + rb[u], sg, cg);
          float f = fmaf(one, sg, rl[u]), qv = act_in<FAST>((float)rq[u][i], act) * qm;
          if (decltype(tail)::value) {
            const float in = ra + i < n ? 1.f : 0.f;
            f = fmaf(in, f, 1.f - in);
            qv *= in;
          }
          F *= f;
          sq[(ra + i) * KP + idx] = qv;
          sf[(ra + i) * KP + idx] = f;
          w[i] = qv * F;
        }
        const float Fo = __shfl_xor(F, 32, 64), by = hf ? Fo : 1.f;
#pragma unroll
        for (int i = 0; i < HC; ++i) {
          sqf[(ra + i) * KP + idx] = w[i] * by;
          if (hf) sqh[i * KP + idx] = w[i];
        }
        if (hf == 0) sl[idx] = F * Fo;
      } else if (WHOLE || idx < 2 * DP) {
        const int d = idx - DP;
        float B = 1.f, w[HC];
#pragma unroll
        for (int i = HC - 1; i >= 0; --i) {
          float sg, cg;
          sigmoid2<FAST>((float)rz[u][i] + rb[u], sg, cg);
          float f = fmaf(one, sg, rl[u]), k = one * cg;
          if (decltype(tail)::value) {
            const float in = ra + i < n ? 1.f : 0.f;
            f = fmaf(in, f, 1.f - in);
            k *= in;
          }
          sk[(ra + i) * KP + d] = k;
          w[i] = k * B;
          B *= f;
        }
        const float Bo = __shfl_xor(B, 32, 64), by = hf ? 1.f : Bo;
#pragma unroll
        for (int i = 0; i < HC; ++i) {
          skb[(ra + i) * KP + d] = w[i] * by;
          if (!hf) skh[i * KP + d] = w[i];
        }
      }
    }
    if (tid < 256) {
      const int t = tid >> 4, c = 4 * (tid & 15);
      f32x4 a;
#pragma unroll
      for (int e = 0; e < 4; ++e) a[e] = (t < n && c0 + c + e < Dv) ? (float)rv[e] : 0.f;
      *reinterpret_cast<f32x4*>(sv + t * VP + c) = a;
    }
  };
  fetch(r0);
  for (int t0 = r0; t0 < r1; t0 += C) {
    const int n = min(C, r1 - t0);
    if (n == C) stage(n, std::false_type{});
    else stage(n, std::true_type{});
    if (t0 + C < r1) fetch(t0 + C);      // in flight during the products below
    __syncthreads();
    // (q F) S, then the new state
    f32x4 oc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < NH; ++i) {
      const f32x4 a = *reinterpret_cast<const f32x4*>(sqf + m * KP + d0 + 16 * i + 4 * gg);
#pragma unroll
      for (int e = 0; e < 4; ++e) oc = mfma_f32(a[e], st[i][e], oc);
    }
    float bv[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) bv[e] = sv[(4 * gg + e) * VP + cl];
#pragma unroll
    for (int i = 0; i < NH; ++i) {
      st[i] *= *reinterpret_cast<const f32x4*>(sl + d0 + 16 * i + 4 * gg);
#pragma unroll
      for (int e = 0; e < 4; ++e) st[i] = mfma_f32(skb[(4 * gg + e) * KP + d0 + 16 * i + m], bv[e], st[i]);
    }
    // weights of rows 8 .. 15 on columns 0 .. 7: this wave's channels
    if (wave < NP) {
      f32x4 w = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < (NT + 7) / 8; ++i) {
        const int at = (m & 7) * KP + 16 * (wave + 8 * i) + 4 * gg;
        if (NT % 8 && wave + 8 * i >= NT) break;
        const f32x4 a = *reinterpret_cast<const f32x4*>(sqh + at), b = *reinterpret_cast<const f32x4*>(skh + at);
#pragma unroll
        for (int e = 0; e < 4; ++e) w = mfma_f32(a[e], b[e], w);
      }
      if (m < HC && gg < 2) {
#pragma unroll
        for (int e = 0; e < 4; ++e) sph[(wave * HC + 4 * gg + e) * HC + m] = w[e];
      }
    }
    // the diagonal blocks: rows tb and 8 + tb, 32 lanes each share the row's channels, lane 16 + j keeps column j
    {
      const int tb = wave < 4 ? wave : 11 - wave, l4 = 4 * (lane & 31);      // (SIMDs get rows of equal work)
      f32x4 qd[NU];
#pragma unroll
      for (int u = 0; u < NU; ++u) qd[u] = *reinterpret_cast<const f32x4*>(sq + (ra + tb) * KP + 128 * u + l4);
      float keep = 0.f;
#pragma unroll
      for (int j = HC - 1; j >= 0; --j) {
        if (j > tb) continue;
        const float* fr = sf + (j < tb ? ra + j + 1 : C) * KP + l4;      // (its own column: not decayed yet)
        const float* kr = sk + (ra + j) * KP + l4;
        float w = 0.f;
#pragma unroll
        for (int u = 0; u < NU; ++u) {
          qd[u] *= *reinterpret_cast<const f32x4*>(fr + 128 * u);
          const f32x4 kk = *reinterpret_cast<const f32x4*>(kr + 128 * u);
#pragma unroll
          for (int e = 0; e < 4; ++e) w = fmaf(qd[u][e], kk[e], w);
        }
        w = half_sum(w);
        keep = m == j ? w : keep;
      }
      if ((lane & 16) && m < HC) sp[(ra + tb) * PP + ra + m] = keep;
    }
    if (wave >= 4) {
#pragma unroll
      for (int e = 0; e < 4; ++e) so[(4 * gg + e) * VP + cl] = oc[e];
    }
    __syncthreads();
    if (wave < 4) {
      f32x4 a = *reinterpret_cast<const f32x4*>(sp + m * PP + 4 * gg);
      if (m >= HC && gg < 2) {
        a = *reinterpret_cast<const f32x4*>(sph + (m - HC) * HC + 4 * gg);
#pragma unroll
        for (int i = 1; i < NP; ++i) a += *reinterpret_cast<const f32x4*>(sph + (i * HC + m - HC) * HC + 4 * gg);
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) oc[e] += so[(4 * gg + e) * VP + cl];
#pragma unroll
      for (int e = 0; e < 4; ++e) oc = mfma_f32(a[e], bv[e], oc);
      if (live) {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int t = 4 * gg + e;
          if (t < n) o[((long)(t0 + t) * H + h) * Dv + col] = oc[e];
        }
      }
    }
    // (the next chunk's staging writes nothing that is read after the barrier above; sp, sph and so are rewritten only
    // after its own first barrier)
  }
  int De = D;
  asm volatile("" : "+s"(De));      // (the bounds are compared anew: kept masks would fill the scalar registers)
  if (live) {
#pragma unroll
    for (int i = 0; i < NH; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int d = d0 + 16 * i + 4 * gg + e;
        if (d < De) S[(long)d * Dv] = st[i][e];
      }
  }
}

// The same recurrence row by row, for steps of one row per sequence (decoding) and for any D. Workgroup =
// (sequence, head, 64 value columns): 16 lanes of four columns by 16 groups of state rows; the state is read and
// written in place, the row groups' partial read-outs are summed in LDS.
template <typename T>
__global__ __launch_bounds__(256) void forget_step_kernel(const T* __restrict__ q, long q_ld, const T* __restrict__ z,
                                                          long z_ld, const T* __restrict__ v, long v_ld,
                                                          const float* __restrict__ f_bias,
                                                          const float* __restrict__ lower, float* __restrict__ state,
                                                          const int* __restrict__ state_slots,
                                                          const int* __restrict__ row_cu,
                                                          const int* __restrict__ positions, int act, int vec,
                                                          float* __restrict__ o, int H, int D, int Dv) {
  constexpr bool FAST = sizeof(T) == 2;
  extern __shared__ __attribute__((aligned(16))) float smem[];
  float* sq = smem;            // [D]
  float* sk = smem + D;        // [D]
  float* sf = smem + 2 * D;    // [D]
  __shared__ f32x4 red[16][16];
  const int s = blockIdx.x, h = blockIdx.y, c0 = blockIdx.z * 64;
  const int r0 = row_cu ? row_cu[s] : s, r1 = row_cu ? row_cu[s + 1] : s + 1;
  const int tid = threadIdx.x, cg = tid & 15, dg = tid >> 4;
  const int slot = state_slots[s], c = c0 + 4 * cg;
  if (slot < 0) {
    for (int i = tid; i < (r1 - r0) * 64; i += 256)
      if (c0 + (i & 63) < Dv) o[((long)(r0 + (i >> 6)) * H + h) * Dv + c0 + (i & 63)] = 0.f;
    return;
  }
  float* S = state + ((long)slot * H + h) * D * Dv;
  const bool sv4 = (vec & 4) && c + 3 < Dv;      // 16-byte state rows
  for (int t = r0; t < r1; ++t) {
    for (int d = tid; d < D; d += 256) {
      const float lo = lower[(long)h * D + d];
      float sg, cg2;
      sigmoid2<FAST>((float)z[(long)t * z_ld + (long)h * D + d] + f_bias[(long)h * D + d], sg, cg2);
      sq[d] = act_in<FAST>((float)q[(long)t * q_ld + (long)h * D + d], act);
      sk[d] = (1.f - lo) * cg2;
      sf[d] = lo + (1.f - lo) * sg;
    }
    const f32x4 vv = load4(v + (long)t * v_ld + (long)h * Dv, c, Dv, vec & 2);
    __syncthreads();
    const bool fresh = positions[t] == 0;
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    if (c < Dv)
#pragma unroll 8
      for (int d = dg; d < D; d += 16) {
        float* Sr = S + (long)d * Dv + c;
        f32x4 x = {0.f, 0.f, 0.f, 0.f};
        if (!fresh) {
          if (sv4) x = *reinterpret_cast<const f32x4*>(Sr);
          else
#pragma unroll
            for (int e = 0; e < 4; ++e) x[e] = c + e < Dv ? Sr[e] : 0.f;
        }
        const float kd = sk[d], qd = sq[d], fd = sf[d];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          x[e] = fmaf(fd, x[e], kd * vv[e]);
          acc[e] = fmaf(qd, x[e], acc[e]);
        }
        if (sv4) *reinterpret_cast<f32x4*>(Sr) = x;
        else
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if (c + e < Dv) Sr[e] = x[e];
      }
    red[dg][cg] = acc;
    __syncthreads();
    if (tid < 64 && c0 + tid < Dv) {
      float a = 0.f;
#pragma unroll
      for (int g = 0; g < 16; ++g) a += red[g][tid >> 2][tid & 3];
      o[((long)t * H + h) * Dv + c0 + tid] = a;
    }
    __syncthreads();
  }
}

// L lanes per (row, head), V values per access
template <typename T, int V, int L>
__global__ __launch_bounds__(256) void head_norm_gate_kernel(const float* __restrict__ o, const float* __restrict__ w,
                                                             float eps, const T* __restrict__ gate, long g_ld, int act,
                                                             float mul, T* __restrict__ out, long out_ld, long n, int H,
                                                             int Dv) {
  typedef float fv __attribute__((ext_vector_type(V)));
  typedef T tv __attribute__((ext_vector_type(V)));
  const long item = blockIdx.x * (long)(256 / L) + threadIdx.x / L;      // t * H + h
  const int l = threadIdx.x % L;
  if (item >= n) return;      // (whole groups of L lanes leave; a group never spans waves)
  const long t = item / H;
  const int h = (int)(item - t * H);
  const float* row = o + item * Dv;
  fv x0 = fv(0.f);
  float ss = 0.f;
  for (int c = V * l; c < Dv; c += V * L) {
    const fv x = *reinterpret_cast<const fv*>(row + c);
    if (c < V * L) x0 = x;
#pragma unroll
    for (int e = 0; e < V; ++e) ss = fmaf(x[e], x[e], ss);
  }
#pragma unroll
  for (int d = L / 2; d > 0; d >>= 1) ss += __shfl_xor(ss, d, 64);
  const float r = mul / sqrtf(ss / (float)Dv + eps);
  for (int c = V * l; c < Dv; c += V * L) {
    const fv x = c < V * L ? x0 : *reinterpret_cast<const fv*>(row + c);
    fv f;
#pragma unroll
    for (int e = 0; e < V; ++e) f[e] = x[e] * r;
    if (w) f *= *reinterpret_cast<const fv*>(w + c);
    if (gate) {
      const tv gv = *reinterpret_cast<const tv*>(gate + t * g_ld + (long)h * Dv + c);
#pragma unroll
      for (int e = 0; e < V; ++e) {
        const float g = (float)gv[e], sg = 1.f / (1.f + expf(-g));
        f[e] *= act == 1 ? g * sg : sg;
      }
    }
    tv y;
#pragma unroll
    for (int e = 0; e < V; ++e) y[e] = (T)f[e];
    *reinterpret_cast<tv*>(out + t * out_ld + (long)h * Dv + c) = y;
  }
}

template <typename T, int NT>
void forget_chunk_launch(const T* q, long q_ld, const T* z, long z_ld, const T* v, long v_ld, const float* f_bias,
                         const float* lower, float* state, const int* state_slots, const int* row_cu, int nseq,
                         const int* positions, int act, int vec, float* o, int H, int D, int Dv, hipStream_t s) {
  constexpr int DP = 16 * NT, KP = (DP + 127) / 128 * 128 + 4;
  constexpr size_t lds = (size_t)(97 * KP + 2 * 16 * 68 + 16 * 20 + 64 * (NT < 8 ? NT : 8) + DP) * sizeof(float);
  static bool once = false;
  if (!once) {
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&forget_chunk_kernel<T, NT>),
                              hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    once = true;
  }
  dim3 grid(nseq, H, (Dv + 63) / 64);
  forget_chunk_kernel<T, NT><<<grid, 512, lds, s>>>(q, q_ld, z, z_ld, v, v_ld, f_bias, lower, state, state_slots, row_cu,
                                                    positions, act, vec, o, H, D, Dv);
}

template <typename T>
void forget_scan_t(const T* q, long q_ld, const T* z, long z_ld, const T* v, long v_ld, const float* f_bias,
                   const float* lower, float* state, const int* state_slots, const int* row_cu, int nseq,
                   const int* positions, int act, float* o, int H, int D, int Dv, bool one_row, hipStream_t s) {
  int vec = 0;      // 2: v rows, 4: state rows in four-element accesses
  if (Dv % 4 == 0 && rows_aligned(v, v_ld, sizeof(T))) vec |= 2;
  if (Dv % 4 == 0) vec |= 4;
  if (one_row || D > 256) {
    dim3 grid(nseq, H, (Dv + 63) / 64);
    forget_step_kernel<T><<<grid, 256, 3 * (size_t)D * sizeof(float), s>>>(
        q, q_ld, z, z_ld, v, v_ld, f_bias, lower, state, state_slots, one_row ? nullptr : row_cu, positions, act, vec, o, H, D,
        Dv);
    return;
  }
#define BFLY_FCH(NT)                                                                                                  \
  forget_chunk_launch<T, NT>(q, q_ld, z, z_ld, v, v_ld, f_bias, lower, state, state_slots, row_cu, nseq, positions, act, \
                             vec, o, H, D, Dv, s)
  if (D <= 32) BFLY_FCH(2);
  else if (D <= 64) BFLY_FCH(4);
  else if (D <= 96) BFLY_FCH(6);
  else if (D <= 128) BFLY_FCH(8);
  else if (D <= 192) BFLY_FCH(12);
  else BFLY_FCH(16);
#undef BFLY_FCH
}

template <typename T, int V>
void head_norm_gate_t(const float* o, const float* w, float eps, const T* gate, long g_ld, int act, float mul, T* out,
                      long out_ld, int T_, int H, int Dv, hipStream_t s) {
  const long n = (long)T_ * H;
#define BFLY_HNG(L)                                                                                                  \
  head_norm_gate_kernel<T, V, L><<<(int)((n + 256 / L - 1) / (256 / L)), 256, 0, s>>>(o, w, eps, gate, g_ld, act, mul, out, \
                                                                                      out_ld, n, H, Dv)
  if (Dv <= 8 * V) BFLY_HNG(8);
  else if (Dv <= 16 * V) BFLY_HNG(16);
  else if (Dv <= 32 * V) BFLY_HNG(32);
  else BFLY_HNG(64);
#undef BFLY_HNG
}

}  // namespace

void launch_forget_scan(const void* q, long q_ld, const void* z, long z_ld, const void* v, long v_ld, const float* f_bias,
                        const float* lower, float* state, const int* state_slots, const int* row_cu, int nseq,
                        const int* positions, int act, float* o, int T, int H, int D, int Dv, bool one_row, bool f32,
                        hipStream_t s) {
  if (T <= 0 || nseq <= 0) return;
  if (f32)
    forget_scan_t<float>((const float*)q, q_ld, (const float*)z, z_ld, (const float*)v, v_ld, f_bias, lower, state,
                         state_slots, row_cu, nseq, positions, act, o, H, D, Dv, one_row, s);
  else
    forget_scan_t<bf16>((const bf16*)q, q_ld, (const bf16*)z, z_ld, (const bf16*)v, v_ld, f_bias, lower, state, state_slots,
                        row_cu, nseq, positions, act, o, H, D, Dv, one_row, s);
}

void launch_head_norm_gate(const float* o, const float* w, float eps, const void* gate, long g_ld, int act, float mul,
                           void* out, long out_ld, int T, int H, int Dv, bool f32, hipStream_t s) {
  if (T <= 0 || H <= 0) return;
  const size_t esz = f32 ? 4 : 2;
  const bool vec = Dv % 4 == 0 && rows_aligned(out, out_ld, esz) && (!gate || rows_aligned(gate, g_ld, esz)) &&
                   (!w || rows_aligned(w, 0, 4));
#define BFLY_HN(TT, V) head_norm_gate_t<TT, V>(o, w, eps, (const TT*)gate, g_ld, act, mul, (TT*)out, out_ld, T, H, Dv, s)
  if (f32) { if (vec) BFLY_HN(float, 4); else BFLY_HN(float, 1); }
  else { if (vec) BFLY_HN(bf16, 4); else BFLY_HN(bf16, 1); }
#undef BFLY_HN
}

}  // namespace bfly
