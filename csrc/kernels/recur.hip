// Recurrent mixers with pooled per-sequence state, generic in every size and in the activation type (bf16
// or f32; decays, step sizes, states and all recurrences are f32 in both):
//   decay_chunk_kernel, decay_step_kernel   linear attention with a constant decay per head, S <- decay S +
//                                           k v^T, o = S^T q, in chunks on the f32 matrix cores or row by row; queries
//                                           and keys optionally rotated by position as they are loaded
//   selective_scan_kernel, selective_step_kernel
//                                           S <- exp(dt A) S + dt x B, y = S C + d x, out = y silu(z), over many
//                                           rows per sequence or one row each (with dt's projection)
//   row_norm_gate_kernel                    RMS norm of whole rows, times a sigmoid gate and a factor
// Rows of a step are packed: sequence s owns rows row_cu[s] .. row_cu[s+1]; a sequence whose first row is at
// position 0 starts from a zero state whatever its slot holds.
#include <algorithm>

#include "bfly_recur.h"
#include "bfly_recur_dev.h"

namespace bfly {

namespace {

// Linear attention with decay in chunks of C rows. Workgroup = (sequence, head, 64 value columns), four
// waves of 16 columns each. With local row indices 0 .. n - 1 of a chunk and S the state before it,
//   o_t = decay^(t + 1) q_t S + sum_(j <= t) decay^(t - j) (q_t . k_j) v_j,
//   S  <- decay^n S + sum_j decay^(n - 1 - j) k_j v_j^T,
// all four products on the f32 matrix cores (16x16x4 tiles, f32 operands and accumulators): nothing is
// rounded below f32. A wave keeps its columns' state in the accumulator layout (tile i, element e: row
// d = 16 i + 4 gg + e of lane group gg), which is also the B operand of the q S product when step e of
// tile i takes d = 16 i + 4 gg + e from group gg; q, k and the weights then come from LDS as 16-byte
// reads. The chunk's (q . k) decay tiles at or below the diagonal are dealt to the waves and shared
// through LDS. Rows past the sequence and dimensions past D are staged as zeros. D <= 16 NT.
// ROT: the first 2 nrot dimensions of q and k are rotated in LDS (dimension i with i + nrot) by the row's
// cosines and sines cs[t][2][nrot]; k is multiplied by k_scale either way.
template <typename T, int NT, int C, bool ROT>
__global__ __launch_bounds__(256) void decay_chunk_kernel(const T* __restrict__ q, long q_ld, const T* __restrict__ k,
                                                          long k_ld, const T* __restrict__ v, long v_ld,
                                                          const float* __restrict__ dpow, int n_pow,
                                                          float* __restrict__ state,
                                                          const int* __restrict__ state_slots,
                                                          const int* __restrict__ row_cu,
                                                          const int* __restrict__ positions, int act, int vec,
                                                          const float* __restrict__ cs, int nrot, float k_scale,
                                                          float* __restrict__ o, int H, int D, int Dv) {
  constexpr int DP = 16 * NT, KP = DP + 4, VP = 68, PP = C + 4, TT = C / 16;
  extern __shared__ __attribute__((aligned(16))) float smem[];
  float* sq = smem;                  // [C][KP]
  float* sk = sq + C * KP;           // [C][KP]
  float* sv = sk + C * KP;           // [C][VP]
  float* sp = sv + C * VP;           // [C][PP]
  float* sd = sp + C * PP;           // [C + 1] powers of the decay
  const int s = blockIdx.x, h = blockIdx.y, c0 = blockIdx.z * 64;
  const int r0 = row_cu[s], r1 = row_cu[s + 1];
  if (r1 <= r0) return;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, m = lane & 15, gg = lane >> 4;
  const int slot = state_slots[s];
  if (slot < 0) {      // padding sequence of a fixed-shape step: defined output, no state
    for (int i = tid; i < (r1 - r0) * 64; i += 256)
      if (c0 + (i & 63) < Dv) o[((long)(r0 + (i >> 6)) * H + h) * Dv + c0 + (i & 63)] = 0.f;
    return;
  }
  const int cl = 16 * wave + m, col = c0 + cl;
  const bool live = col < Dv;
  float* S = state + ((long)slot * H + h) * D * Dv + col;
  const bool fresh = positions[r0] == 0;
  f32x4 st[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int d = 16 * i + 4 * gg + e;
      st[i][e] = (!fresh && live && d < D) ? S[(long)d * Dv] : 0.f;
    }
  for (int i = tid; i <= C; i += 256) sd[i] = dpow[(long)h * n_pow + i];
  // A chunk's inputs travel to registers as they are stored while the chunk before is computed (rows past the
  // sequence: its last row again, so no load hangs on a branch; staged as zeros).
  typedef T t4 __attribute__((ext_vector_type(4)));
  constexpr int NQ = (C * (DP / 4) + 255) / 256, NV = C * 16 / 256;
  t4 rq[NQ], rk[NQ], rv[NV];
  // rotation: four pairs of a row per thread, DP / 8 threads per row; their cosines and sines travel along
  constexpr int NR = ROT ? (C * (DP / 8) + 255) / 256 : 1;
  f32x4 rc[NR], rs[NR];
  auto fetch4 = [&](const T* row, int c, int size, bool v4) {
    if (v4) return *reinterpret_cast<const t4*>(row + min(c, size - 4));
    t4 r;
#pragma unroll
    for (int e = 0; e < 4; ++e) r[e] = row[min(c + e, size - 1)];
    return r;
  };
  auto fetch = [&](int t0) {
#pragma unroll
    for (int j = 0; j < NQ; ++j) {
      const int i = tid + 256 * j, d = 4 * (i % (DP / 4));
      const long t = min(t0 + i / (DP / 4), r1 - 1);
      rq[j] = fetch4(q + t * q_ld + (long)h * D, d, D, vec & 1);
      rk[j] = fetch4(k + t * k_ld + (long)h * D, d, D, vec & 1);
    }
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int i = tid + 256 * j;
      const long t = min(t0 + (i >> 4), r1 - 1);
      rv[j] = fetch4(v + t * v_ld + (long)h * Dv, c0 + 4 * (i & 15), Dv, vec & 2);
    }
    if constexpr (ROT) {
      if (vec & 8) {
#pragma unroll
        for (int j = 0; j < NR; ++j) {
          const int i = tid + 256 * j;
          const float* row = cs + (long)min(t0 + i / (DP / 8), r1 - 1) * 2 * nrot + min(4 * (i % (DP / 8)), nrot - 4);
          rc[j] = *reinterpret_cast<const f32x4*>(row);
          rs[j] = *reinterpret_cast<const f32x4*>(row + nrot);
        }
      }
    }
  };
  auto stage4 = [&](const t4& r, bool row, int c, int size) {
    f32x4 a;
#pragma unroll
    for (int e = 0; e < 4; ++e) a[e] = (row && c + e < size) ? act_in<sizeof(T) == 2>((float)r[e], act) : 0.f;
    return a;
  };
  auto rotate4 = [&](float* row, int i, const f32x4& c, const f32x4& sn) {      // pairs i .. i + 3
    const f32x4 u = *reinterpret_cast<const f32x4*>(row + i), w = *reinterpret_cast<const f32x4*>(row + nrot + i);
    *reinterpret_cast<f32x4*>(row + i) = u * c - w * sn;
    *reinterpret_cast<f32x4*>(row + nrot + i) = w * c + u * sn;
  };
  fetch(r0);
  for (int t0 = r0; t0 < r1; t0 += C) {
    const int n = min(C, r1 - t0);
#pragma unroll
    for (int j = 0; j < NQ; ++j) {
      const int i = tid + 256 * j, t = i / (DP / 4), d = 4 * (i % (DP / 4));
      if (NQ * 256 != C * (DP / 4) && t >= C) break;
      *reinterpret_cast<f32x4*>(sq + t * KP + d) = stage4(rq[j], t < n, d, D);
      *reinterpret_cast<f32x4*>(sk + t * KP + d) = stage4(rk[j], t < n, d, D) * k_scale;
    }
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int i = tid + 256 * j, t = i >> 4, c = 4 * (i & 15);
      *reinterpret_cast<f32x4*>(sv + t * VP + c) = stage4(rv[j], t < n, c0 + c, Dv);
    }
    if constexpr (ROT) {
      __syncthreads();
      if (vec & 8) {      // nrot % 4 == 0
#pragma unroll
        for (int j = 0; j < NR; ++j) {
          const int i = tid + 256 * j, t = i / (DP / 8), d = 4 * (i % (DP / 8));
          if (t < C && d < nrot) {
            rotate4(sq + t * KP, d, rc[j], rs[j]);
            rotate4(sk + t * KP, d, rc[j], rs[j]);
          }
        }
      } else {
        for (int i = tid; i < n * nrot; i += 256) {
          const int t = i / nrot, d = i - t * nrot;
          const float c = cs[(long)(t0 + t) * 2 * nrot + d], sn = cs[(long)(t0 + t) * 2 * nrot + nrot + d];
          float* qr = sq + t * KP + d;
          float* kr = sk + t * KP + d;
          const float qu = qr[0], qw = qr[nrot], ku = kr[0], kw = kr[nrot];
          qr[0] = qu * c - qw * sn;
          qr[nrot] = qw * c + qu * sn;
          kr[0] = ku * c - kw * sn;
          kr[nrot] = kw * c + ku * sn;
        }
      }
    }
    if (t0 + C < r1) fetch(t0 + C);      // in flight during the products below
    __syncthreads();
    // (q . k) decay^(t - j): the tiles at or below the diagonal, dealt to the waves
    for (int tile = wave; tile < TT * (TT + 1) / 2; tile += 4) {
      int tt = 0, jt = tile;
      while (jt > tt) { ++tt; jt -= tt; }
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < NT; ++i) {
        const f32x4 a = *reinterpret_cast<const f32x4*>(sq + (16 * tt + m) * KP + 16 * i + 4 * gg);
        const f32x4 b = *reinterpret_cast<const f32x4*>(sk + (16 * jt + m) * KP + 16 * i + 4 * gg);
#pragma unroll
        for (int e = 0; e < 4; ++e) acc = mfma_f32(a[e], b[e], acc);
      }
      const int j = 16 * jt + m;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int t = 16 * tt + 4 * gg + e;
        sp[t * PP + j] = j <= t ? acc[e] * sd[t - j] : 0.f;
      }
    }
    __syncthreads();
    f32x4 oc[TT];
#pragma unroll
    for (int tt = 0; tt < TT; ++tt) oc[tt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < NT; ++i)
#pragma unroll
      for (int tt = 0; tt < TT; ++tt) {
        const f32x4 a = *reinterpret_cast<const f32x4*>(sq + (16 * tt + m) * KP + 16 * i + 4 * gg);
#pragma unroll
        for (int e = 0; e < 4; ++e) oc[tt] = mfma_f32(a[e], st[i][e], oc[tt]);
      }
#pragma unroll
    for (int tt = 0; tt < TT; ++tt)
#pragma unroll
      for (int e = 0; e < 4; ++e) oc[tt][e] *= sd[16 * tt + 4 * gg + e + 1];
    const float dn = sd[n];
#pragma unroll
    for (int i = 0; i < NT; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) st[i][e] *= dn;
#pragma unroll
    for (int jt = 0; jt < TT; ++jt) {
      float bv[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) bv[e] = sv[(16 * jt + 4 * gg + e) * VP + cl];
#pragma unroll
      for (int tt = jt; tt < TT; ++tt) {
        const f32x4 a = *reinterpret_cast<const f32x4*>(sp + (16 * tt + m) * PP + 16 * jt + 4 * gg);
#pragma unroll
        for (int e = 0; e < 4; ++e) oc[tt] = mfma_f32(a[e], bv[e], oc[tt]);
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int j = 16 * jt + 4 * gg + e;
        bv[e] = j < n ? bv[e] * sd[n - 1 - j] : 0.f;
      }
#pragma unroll
      for (int e = 0; e < 4; ++e)
#pragma unroll
        for (int i = 0; i < NT; ++i) st[i] = mfma_f32(sk[(16 * jt + 4 * gg + e) * KP + 16 * i + m], bv[e], st[i]);
    }
    if (live) {
#pragma unroll
      for (int tt = 0; tt < TT; ++tt)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int t = 16 * tt + 4 * gg + e;
          if (t < n) o[((long)(t0 + t) * H + h) * Dv + col] = oc[tt][e];
        }
    }
    __syncthreads();      // every wave has left sq / sk / sv / sp before the next chunk is staged
  }
  if (live) {
#pragma unroll
    for (int i = 0; i < NT; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int d = 16 * i + 4 * gg + e;
        if (d < D) S[(long)d * Dv] = st[i][e];
      }
  }
}

// The same recurrence row by row, for steps of one row per sequence (decoding) and for any D. Workgroup =
// (sequence, head, 64 value columns): 16 lanes of four columns by 16 groups of state rows; the state
// is read and written in place, the row groups' partial read-outs are summed in LDS.
template <typename T>
__global__ __launch_bounds__(256) void decay_step_kernel(const T* __restrict__ q, long q_ld, const T* __restrict__ k,
                                                         long k_ld, const T* __restrict__ v, long v_ld,
                                                         const float* __restrict__ dpow, int n_pow,
                                                         float* __restrict__ state, const int* __restrict__ state_slots,
                                                         const int* __restrict__ row_cu,
                                                         const int* __restrict__ positions, int act, int vec,
                                                         const float* __restrict__ cs, int nrot, float k_scale,
                                                         float* __restrict__ o, int H, int D, int Dv) {
  extern __shared__ __attribute__((aligned(16))) float smem[];
  float* sq = smem;            // [D]
  float* sk = smem + D;        // [D]
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
  const float lam = dpow[(long)h * n_pow + 1];
  float* S = state + ((long)slot * H + h) * D * Dv;
  const bool sv4 = (vec & 4) && c + 3 < Dv;      // 16-byte state rows
  for (int t = r0; t < r1; ++t) {
    const T* qr = q + (long)t * q_ld + (long)h * D;
    const T* kr = k + (long)t * k_ld + (long)h * D;
    for (int d = tid; d < D; d += 256) {
      float qv = act_in<sizeof(T) == 2>((float)qr[d], act), kv = act_in<sizeof(T) == 2>((float)kr[d], act);
      if (d < 2 * nrot) {      // rotated with its partner: (u c - w s, w c + u s)
        const bool hi = d >= nrot;
        const int i = hi ? d - nrot : d, m = hi ? i : d + nrot;
        const float c = cs[(long)t * 2 * nrot + i], sn = cs[(long)t * 2 * nrot + nrot + i];
        const float qm = act_in<sizeof(T) == 2>((float)qr[m], act), km = act_in<sizeof(T) == 2>((float)kr[m], act);
        qv = hi ? qv * c + qm * sn : qv * c - qm * sn;
        kv = hi ? kv * c + km * sn : kv * c - km * sn;
      }
      sq[d] = qv;
      sk[d] = kv * k_scale;
    }
    f32x4 vv = load4(v + (long)t * v_ld + (long)h * Dv, c, Dv, vec & 2);
#pragma unroll
    for (int e = 0; e < 4; ++e) vv[e] = act_in<sizeof(T) == 2>(vv[e], act);
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
        const float kd = sk[d], qd = sq[d];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          x[e] = fmaf(lam, x[e], kd * vv[e]);
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

// softplus, silu and exp(dt A) of the selective scan. FAST (bf16 activations): the hardware exp / log /
// reciprocal, and for small e = exp(v) the series of log(1 + e), which keeps its relative accuracy there; a
// true-f32 run uses the precise functions.
template <bool FAST>
__device__ __forceinline__ float softplus(float v) {
  if (!FAST) return v > 20.f ? v : log1pf(expf(v));
  const float e = __expf(v);
  const float small = e * (1.f - e * (0.5f - e * (1.f / 3.f - e * 0.25f)));
  return v > 20.f ? v : e < 0.03125f ? small : __logf(1.f + e);
}
template <bool FAST>
__device__ __forceinline__ float silu_f(float v) {
  if (FAST) return v * __builtin_amdgcn_rcpf(1.f + __expf(-v));
  return v / (1.f + expf(-v));
}
constexpr float kLog2e = 1.4426950408889634f;

// Selective scan. Workgroup = (sequence, 64 channels); the four lanes of a quad share a channel and keep NS
// of its N states each in registers (N <= 4 NS; states past N have B = C = 0). Tokens are staged 16 at a
// time: step sizes dt = softplus(dtr + bias), dt x, and the B and C rows go to LDS, the next block's inputs
// travel to registers meanwhile; a token then costs NS exponentials and fused updates per lane and two
// cross-lane moves, with no barrier inside the token loop. Rows past the sequence are staged with dt = 0
// and x = 0 (they leave the state as it is), so the loop has a fixed length and its LDS reads are
// scheduled ahead. The outputs leave through LDS, where the skip d x and the gate silu(z) are applied by
// the threads that hold x and z.
template <typename T, int NS>
__global__ __launch_bounds__(256) void selective_scan_kernel(const T* __restrict__ x, long x_ld,
                                                             const float* __restrict__ dtr, long dt_ld,
                                                             const T* __restrict__ b, long b_ld,
                                                             const T* __restrict__ cc, long c_ld,
                                                             const T* __restrict__ z, long z_ld,
                                                             const float* __restrict__ a_log,
                                                             const float* __restrict__ dt_bias,
                                                             const float* __restrict__ dskip,
                                                             float* __restrict__ state,
                                                             const int* __restrict__ state_slots,
                                                             const int* __restrict__ row_cu,
                                                             const int* __restrict__ positions, T* __restrict__ out,
                                                             int C, int N) {
  constexpr int TB = 16, NP = 4 * NS, PT = TB * 64 / 256, PB = (TB * NP + 255) / 256;
  __shared__ __attribute__((aligned(16))) float sB[TB * NP], sC[TB * NP];
  __shared__ float sdt[TB][64], sdx[TB][64], sy[TB][64];
  const int s = blockIdx.x, c0 = blockIdx.y * 64;
  const int r0 = row_cu[s], r1 = row_cu[s + 1];
  if (r1 <= r0) return;
  const int tid = threadIdx.x, cl = tid >> 2, qd = tid & 3, ch = c0 + cl;
  const int slot = state_slots[s];
  const int cs = c0 + (tid & 63), tr = tid >> 6;      // this thread's channel and first row when staging
  if (slot < 0) {      // padding sequence of a fixed-shape step: defined output, no state
    for (int t = r0 + tr; t < r1; t += 4)
      if (cs < C) out[(long)t * C + cs] = (T)0.f;
    return;
  }
  float* S = state + ((long)slot * C + ch) * N + qd * NS;
  const bool fresh = positions[r0] == 0;
  constexpr bool FAST = sizeof(T) == 2;
  float st[NS], A[NS];
#pragma unroll
  for (int i = 0; i < NS; ++i) {
    const bool ok = ch < C && qd * NS + i < N;
    st[i] = (ok && !fresh) ? S[i] : 0.f;
    A[i] = ok ? -expf(a_log[(long)ch * N + qd * NS + i]) : 0.f;
    if (FAST) A[i] *= kLog2e;      // exp2 of (dt A log2 e)
  }
  const float bias = cs < C ? dt_bias[cs] : 0.f, ds = cs < C ? dskip[cs] : 0.f;
  // the next block's inputs as they are stored (rows and columns past the end: the last one again, so no
  // load hangs on a branch; such values meet dt = 0 or B = C = 0)
  T rx[PT], rz[PT], rb[PB], rc[PB];
  float rd[PT];
  const int csc = min(cs, C - 1);
  auto fetch = [&](int t0) {
#pragma unroll
    for (int j = 0; j < PT; ++j) {
      const long t = min(t0 + tr + 4 * j, r1 - 1);
      rx[j] = x[t * x_ld + csc];
      rz[j] = z[t * z_ld + csc];
      rd[j] = dtr[t * dt_ld + csc];
    }
#pragma unroll
    for (int j = 0; j < PB; ++j) {
      const int i = tid + 256 * j, tt = i / NP, n = min(i - tt * NP, N - 1);
      const long t = min(t0 + tt, r1 - 1);
      rb[j] = b[t * b_ld + n];
      rc[j] = cc[t * c_ld + n];
    }
  };
  fetch(r0);
  for (int t0 = r0; t0 < r1; t0 += TB) {
    const int nb = min(TB, r1 - t0);
    float cx[PT], cz[PT];
#pragma unroll
    for (int j = 0; j < PT; ++j) {
      const float dt = tr + 4 * j < nb ? softplus<FAST>(rd[j] + bias) : 0.f;
      cx[j] = (float)rx[j];
      cz[j] = (float)rz[j];
      sdt[tr + 4 * j][tid & 63] = dt;
      sdx[tr + 4 * j][tid & 63] = dt * cx[j];
    }
#pragma unroll
    for (int j = 0; j < PB; ++j) {
      const int i = tid + 256 * j;
      if (i < TB * NP) {
        const bool in = i % NP < N;
        sB[i] = in ? (float)rb[j] : 0.f;
        sC[i] = in ? (float)rc[j] : 0.f;
      }
    }
    __syncthreads();
    if (t0 + TB < r1) fetch(t0 + TB);        // in flight during the token loop
    float ys[TB / 4];      // lane qd of a quad keeps the outputs of tokens qd, qd + 4, ... (no store in the loop)
#pragma unroll
    for (int tt = 0; tt < TB; ++tt) {
      const float dt = sdt[tt][cl], dx = sdx[tt][cl];
      const float* pb = sB + tt * NP + qd * NS;
      const float* pc = sC + tt * NP + qd * NS;
      float y0 = 0.f, y1 = 0.f;
#pragma unroll
      for (int i = 0; i < NS; ++i) {
        const float a = FAST ? __builtin_amdgcn_exp2f(dt * A[i]) : expf(dt * A[i]);
        st[i] = fmaf(a, st[i], dx * pb[i]);
        if (i & 1) y1 = fmaf(st[i], pc[i], y1);
        else y0 = fmaf(st[i], pc[i], y0);
      }
      const float y = quad_sum(y0 + y1);
      if ((tt & 3) == 0) ys[tt >> 2] = y;
      else ys[tt >> 2] = qd == (tt & 3) ? y : ys[tt >> 2];
    }
#pragma unroll
    for (int j = 0; j < TB / 4; ++j) sy[4 * j + qd][cl] = ys[j];
    __syncthreads();
#pragma unroll
    for (int j = 0; j < PT; ++j) {
      const int tt = tr + 4 * j;
      if (tt < nb && cs < C) {
        const float y = fmaf(ds, cx[j], sy[tt][tid & 63]);
        out[(long)(t0 + tt) * C + cs] = (T)(y * silu_f<FAST>(cz[j]));
      }
    }
    // (the next block's staging overwrites sdt / sdx / sB / sC, which every wave finished reading at the
    // barrier above; sy is rewritten only after the next block's first barrier)
  }
  if (ch < C) {
#pragma unroll
    for (int i = 0; i < NS; ++i)
      if (qd * NS + i < N) S[i] = st[i];
  }
}

// Decoding: row s is sequence s's one row. Same workgroup shape and lanes as above; the step sizes' low-rank
// projection dtr = W low (W [C, R], low [R] per row) happens here too, a quad sharing the dot product
// of its channel.
template <typename T, int NS>
__global__ __launch_bounds__(256) void selective_step_kernel(const T* __restrict__ x, long x_ld,
                                                             const T* __restrict__ low, long l_ld,
                                                             const T* __restrict__ wdt, int R, int vec,
                                                             const T* __restrict__ b, long b_ld,
                                                             const T* __restrict__ cc, long c_ld,
                                                             const T* __restrict__ z, long z_ld,
                                                             const float* __restrict__ a_log,
                                                             const float* __restrict__ dt_bias,
                                                             const float* __restrict__ dskip,
                                                             float* __restrict__ state,
                                                             const int* __restrict__ state_slots,
                                                             const int* __restrict__ positions, T* __restrict__ out,
                                                             int C, int N) {
  extern __shared__ __attribute__((aligned(16))) float slow[];      // [R]
  constexpr bool FAST = sizeof(T) == 2;
  const long t = blockIdx.x;
  const int tid = threadIdx.x, cl = tid >> 2, qd = tid & 3, ch = blockIdx.y * 64 + cl;
  const int slot = state_slots[t];
  if (slot < 0) {      // padding row
    if (ch < C && qd == 0) out[t * C + ch] = (T)0.f;
    return;
  }
  const bool ok = ch < C, fresh = positions[t] == 0;
  float* S = state + ((long)slot * C + ch) * N + qd * NS;
  float st[NS], A[NS], bv[NS], cv[NS];
#pragma unroll
  for (int i = 0; i < NS; ++i) {
    const bool in = ok && qd * NS + i < N;
    st[i] = (in && !fresh) ? S[i] : 0.f;
    A[i] = in ? a_log[(long)ch * N + qd * NS + i] : 0.f;
    bv[i] = in ? (float)b[t * b_ld + qd * NS + i] : 0.f;
    cv[i] = in ? (float)cc[t * c_ld + qd * NS + i] : 0.f;
  }
  const float xv = ok ? (float)x[t * x_ld + ch] : 0.f, zv = ok ? (float)z[t * z_ld + ch] : 0.f;
  // (the first 128 columns of the projection's row travel to registers before the barrier)
  typedef T t8 __attribute__((ext_vector_type(8)));
  t8 w0[4];
  const T* wr = wdt + (long)ch * R;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int r = 8 * qd + 32 * j;
    if (ok && vec && r < R) w0[j] = *reinterpret_cast<const t8*>(wr + r);
    else w0[j] = t8((T)0.f);
  }
  for (int r = tid; r < R; r += 256) slow[r] = (float)low[t * l_ld + r];
  __syncthreads();
  float acc = 0.f;
  if (ok) {
    if (vec) {      // R % 8 == 0
      float a1 = 0.f;
      auto dot8 = [&](const t8& wv, int r) {
        const f32x4 l0 = *reinterpret_cast<const f32x4*>(slow + r), l1 = *reinterpret_cast<const f32x4*>(slow + r + 4);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          acc = fmaf((float)wv[e], l0[e], acc);
          a1 = fmaf((float)wv[4 + e], l1[e], a1);
        }
      };
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (8 * qd + 32 * j < R) dot8(w0[j], 8 * qd + 32 * j);
      for (int r = 8 * qd + 128; r < R; r += 32) dot8(*reinterpret_cast<const t8*>(wr + r), r);
      acc += a1;
    } else {
      for (int r = qd; r < R; r += 4) acc = fmaf((float)wr[r], slow[r], acc);
    }
  }
  const float dt = ok ? softplus<FAST>(quad_sum(acc) + dt_bias[ch]) : 0.f, dx = dt * xv;
  float y = 0.f;
#pragma unroll
  for (int i = 0; i < NS; ++i) {
    const float a = FAST ? __builtin_amdgcn_exp2f(-dt * kLog2e * __expf(A[i])) : expf(-dt * expf(A[i]));
    st[i] = fmaf(a, st[i], dx * bv[i]);
    y = fmaf(st[i], cv[i], y);
    if (ok && qd * NS + i < N) S[i] = st[i];
  }
  y = quad_sum(y);
  if (ok && qd == 0) {
    y = fmaf(dskip[ch], xv, y);
    out[t * C + ch] = (T)(y * silu_f<FAST>(zv));
  }
}

template <typename T, int V>
__global__ __launch_bounds__(256) void row_norm_gate_kernel(const float* __restrict__ o, const float* __restrict__ w,
                                                            float eps, const T* __restrict__ gate, long g_ld, float mul,
                                                            T* __restrict__ out, long out_ld, int N) {
  typedef float fv __attribute__((ext_vector_type(V)));
  typedef T tv __attribute__((ext_vector_type(V)));
  __shared__ float red[16];
  const long t = blockIdx.x;
  const float* row = o + t * N;
  float ss = 0.f;
  for (int c = V * threadIdx.x; c < N; c += V * 256) {
    const fv x = *reinterpret_cast<const fv*>(row + c);
#pragma unroll
    for (int e = 0; e < V; ++e) ss = fmaf(x[e], x[e], ss);
  }
  const float r = mul / sqrtf(block_sum(ss, red) / (float)N + eps);
  for (int c = V * threadIdx.x; c < N; c += V * 256) {
    const fv x = *reinterpret_cast<const fv*>(row + c), wv = *reinterpret_cast<const fv*>(w + c);
    tv y;
    if (gate) {
      const tv gv = *reinterpret_cast<const tv*>(gate + t * g_ld + c);
#pragma unroll
      for (int e = 0; e < V; ++e) y[e] = (T)(x[e] * r * wv[e] / (1.f + expf(-(float)gv[e])));
    } else {
#pragma unroll
      for (int e = 0; e < V; ++e) y[e] = (T)(x[e] * r * wv[e]);
    }
    *reinterpret_cast<tv*>(out + t * out_ld + c) = y;
  }
}

template <typename T, int NT, int C, bool ROT>
void decay_chunk_launch(const T* q, long q_ld, const T* k, long k_ld, const T* v, long v_ld, const float* dpow, int n_pow,
                        float* state, const int* state_slots, const int* row_cu, int nseq, const int* positions, int act,
                        int vec, const float* cs, int nrot, float k_scale, float* o, int H, int D, int Dv, hipStream_t s) {
  constexpr size_t lds = (size_t)(2 * C * (16 * NT + 4) + C * 68 + C * (C + 4) + C + 1) * sizeof(float);
  static bool once = false;
  if (!once) {
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&decay_chunk_kernel<T, NT, C, ROT>),
                              hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    once = true;
  }
  dim3 grid(nseq, H, (Dv + 63) / 64);
  decay_chunk_kernel<T, NT, C, ROT><<<grid, 256, lds, s>>>(q, q_ld, k, k_ld, v, v_ld, dpow, n_pow, state, state_slots,
                                                           row_cu, positions, act, vec, cs, nrot, k_scale, o, H, D, Dv);
}

template <typename T>
void decay_scan_t(const T* q, long q_ld, const T* k, long k_ld, const T* v, long v_ld, const float* dpow, int n_pow,
                  float* state, const int* state_slots, const int* row_cu, int nseq, const int* positions, int act,
                  const float* cs, int nrot, float k_scale, float* o, int H, int D, int Dv, bool one_row, hipStream_t s) {
  int vec = 0;      // 1: q and k rows, 2: v rows, 4: state rows, 8: rotated pairs in four-element accesses
  if (D % 4 == 0 && rows_aligned(q, q_ld, sizeof(T)) && rows_aligned(k, k_ld, sizeof(T))) vec |= 1;
  if (Dv % 4 == 0 && rows_aligned(v, v_ld, sizeof(T))) vec |= 2;
  if (Dv % 4 == 0) vec |= 4;
  if (nrot > 0 && nrot % 4 == 0 && rows_aligned(cs, 2 * nrot, sizeof(float))) vec |= 8;
  if (one_row || D > 256) {
    dim3 grid(nseq, H, (Dv + 63) / 64);
    decay_step_kernel<T><<<grid, 256, 2 * (size_t)D * sizeof(float), s>>>(
        q, q_ld, k, k_ld, v, v_ld, dpow, n_pow, state, state_slots, one_row ? nullptr : row_cu, positions, act, vec, cs, nrot,
        k_scale, o, H, D, Dv);
    return;
  }
#define BFLY_DCH2(NT, C, ROT)                                                                                          \
  decay_chunk_launch<T, NT, C, ROT>(q, q_ld, k, k_ld, v, v_ld, dpow, n_pow, state, state_slots, row_cu, nseq, positions, \
                                    act, vec, cs, nrot, k_scale, o, H, D, Dv, s)
#define BFLY_DCH(NT, C)                                                 \
  {                                                                     \
    if (nrot > 0) BFLY_DCH2(NT, C, true); else BFLY_DCH2(NT, C, false); \
  }
  if (D <= 32) BFLY_DCH(2, 64)
  else if (D <= 64) BFLY_DCH(4, 64)
  else if (D <= 96) BFLY_DCH(6, 64)
  else if (D <= 128) BFLY_DCH(8, 64)
  else if (D <= 192) BFLY_DCH(12, 32)
  else BFLY_DCH(16, 32)
#undef BFLY_DCH
#undef BFLY_DCH2
}

template <typename T>
int selective_step_t(const T* x, long x_ld, const T* low, long l_ld, const T* wdt, int R, const T* b, long b_ld, const T* c,
                     long c_ld, const T* z, long z_ld, const float* a_log, const float* dt_bias, const float* d, float* state,
                     const int* state_slots, const int* positions, T* out, int T_, int C, int N, hipStream_t s) {
  dim3 grid(T_, (C + 63) / 64);
  const int vec = R % 8 == 0 && reinterpret_cast<uintptr_t>(wdt) % (8 * sizeof(T)) == 0;
#define BFLY_SST(NS)                                                                                                  \
  selective_step_kernel<T, NS><<<grid, 256, R * sizeof(float), s>>>(x, x_ld, low, l_ld, wdt, R, vec, b, b_ld, c, c_ld, z, \
                                                                    z_ld, a_log, dt_bias, d, state, state_slots, positions, \
                                                                    out, C, N)
  if (N <= 4) BFLY_SST(1);
  else if (N <= 8) BFLY_SST(2);
  else if (N <= 16) BFLY_SST(4);
  else if (N <= 32) BFLY_SST(8);
  else if (N <= 64) BFLY_SST(16);
  else if (N <= 128) BFLY_SST(32);
  else if (N <= 256) BFLY_SST(64);
  else return -1;
#undef BFLY_SST
  return 0;
}

template <typename T>
int selective_scan_t(const T* x, long x_ld, const float* dtr, long dt_ld, const T* b, long b_ld, const T* c, long c_ld,
                     const T* z, long z_ld, const float* a_log, const float* dt_bias, const float* d, float* state,
                     const int* state_slots, const int* row_cu, int nseq, const int* positions, T* out, int C, int N,
                     hipStream_t s) {
  dim3 grid(nseq, (C + 63) / 64);
#define BFLY_SSC(NS)                                                                                               \
  selective_scan_kernel<T, NS><<<grid, 256, 0, s>>>(x, x_ld, dtr, dt_ld, b, b_ld, c, c_ld, z, z_ld, a_log, dt_bias, d, \
                                                    state, state_slots, row_cu, positions, out, C, N)
  if (N <= 4) BFLY_SSC(1);
  else if (N <= 8) BFLY_SSC(2);
  else if (N <= 16) BFLY_SSC(4);
  else if (N <= 32) BFLY_SSC(8);
  else if (N <= 64) BFLY_SSC(16);
  else if (N <= 128) BFLY_SSC(32);
  else if (N <= 256) BFLY_SSC(64);
  else return -1;
#undef BFLY_SSC
  return 0;
}

}  // namespace

void launch_decay_scan(const void* q, long q_ld, const void* k, long k_ld, const void* v, long v_ld, const float* dpow,
                       int n_pow, float* state, const int* state_slots, const int* row_cu, int nseq,
                       const int* positions, int act, const float* cs, int nrot, float k_scale, float* o, int T, int H,
                       int D, int Dv, bool one_row, bool f32, hipStream_t s) {
  if (T <= 0 || nseq <= 0) return;
  if (f32)
    decay_scan_t<float>((const float*)q, q_ld, (const float*)k, k_ld, (const float*)v, v_ld, dpow, n_pow, state,
                        state_slots, row_cu, nseq, positions, act, cs, nrot, k_scale, o, H, D, Dv, one_row, s);
  else
    decay_scan_t<bf16>((const bf16*)q, q_ld, (const bf16*)k, k_ld, (const bf16*)v, v_ld, dpow, n_pow, state, state_slots,
                       row_cu, nseq, positions, act, cs, nrot, k_scale, o, H, D, Dv, one_row, s);
}

void launch_row_norm_gate(const float* o, const float* w, float eps, const void* gate, long g_ld, float mul, void* out,
                          long out_ld, int T, int N, bool f32, hipStream_t s) {
  if (T <= 0) return;
  const size_t esz = f32 ? 4 : 2;
  const bool vec = N % 4 == 0 && rows_aligned(out, out_ld, esz) && (!gate || rows_aligned(gate, g_ld, esz));
#define BFLY_RNG(TT, V) \
  row_norm_gate_kernel<TT, V><<<T, 256, 0, s>>>(o, w, eps, (const TT*)gate, g_ld, mul, (TT*)out, out_ld, N)
  if (f32) { if (vec) BFLY_RNG(float, 4); else BFLY_RNG(float, 1); }
  else { if (vec) BFLY_RNG(bf16, 4); else BFLY_RNG(bf16, 1); }
#undef BFLY_RNG
}

int launch_selective_scan(const void* x, long x_ld, const float* dtr, long dt_ld, const void* b, long b_ld, const void* c,
                          long c_ld, const void* z, long z_ld, const float* a_log, const float* dt_bias, const float* d,
                          float* state, const int* state_slots, const int* row_cu, int nseq, const int* positions,
                          void* out, int T, int C, int N, bool f32, hipStream_t s) {
  if (T <= 0 || nseq <= 0) return 0;
  if (f32)
    return selective_scan_t<float>((const float*)x, x_ld, dtr, dt_ld, (const float*)b, b_ld, (const float*)c, c_ld,
                                   (const float*)z, z_ld, a_log, dt_bias, d, state, state_slots, row_cu, nseq, positions,
                                   (float*)out, C, N, s);
  return selective_scan_t<bf16>((const bf16*)x, x_ld, dtr, dt_ld, (const bf16*)b, b_ld, (const bf16*)c, c_ld, (const bf16*)z,
                                z_ld, a_log, dt_bias, d, state, state_slots, row_cu, nseq, positions, (bf16*)out, C, N, s);
}

int launch_selective_step(const void* x, long x_ld, const void* low, long l_ld, const void* wdt, int R, const void* b,
                          long b_ld, const void* c, long c_ld, const void* z, long z_ld, const float* a_log,
                          const float* dt_bias, const float* d, float* state, const int* state_slots, const int* positions,
                          void* out, int T, int C, int N, bool f32, hipStream_t s) {
  if (T <= 0) return 0;
  if (f32)
    return selective_step_t<float>((const float*)x, x_ld, (const float*)low, l_ld, (const float*)wdt, R, (const float*)b, b_ld,
                                   (const float*)c, c_ld, (const float*)z, z_ld, a_log, dt_bias, d, state, state_slots,
                                   positions, (float*)out, T, C, N, s);
  return selective_step_t<bf16>((const bf16*)x, x_ld, (const bf16*)low, l_ld, (const bf16*)wdt, R, (const bf16*)b, b_ld,
                                (const bf16*)c, c_ld, (const bf16*)z, z_ld, a_log, dt_bias, d, state, state_slots, positions,
                                (bf16*)out, T, C, N, s);
}

}  // namespace bfly
