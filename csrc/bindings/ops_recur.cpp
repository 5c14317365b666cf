// torch.ops.bfly.* registrations of csrc/kernels/recur.hip, forget.hip and pooled.hip
// (csrc/include/bfly_recur.h). Shapes, strides and index tensors are validated on the host before any launch.
#include <ATen/ATen.h>
#include <ATen/hip/impl/HIPStreamMasqueradingAsCUDA.h>
#include <torch/library.h>

#include "bfly_recur.h"

namespace {

using at::Tensor;
using c10::optional;

inline hipStream_t cur_stream() { return at::hip::getCurrentHIPStreamMasqueradingAsCUDA().stream(); }

inline bool is_f32(const Tensor& t) {
  TORCH_CHECK(t.scalar_type() == at::kFloat || t.scalar_type() == at::kBFloat16, "expected a bf16 or f32 tensor");
  return t.scalar_type() == at::kFloat;
}
#define CHK_SAME(a, b) TORCH_CHECK((a).scalar_type() == (b).scalar_type(), #a " and " #b " must have one element type")
#define CHK_F32(t) \
  TORCH_CHECK((t).is_cuda() && (t).scalar_type() == at::kFloat && (t).is_contiguous(), #t " must be contiguous f32 on the GPU")
#define CHK_I32(t) \
  TORCH_CHECK((t).is_cuda() && (t).scalar_type() == at::kInt && (t).is_contiguous(), #t " must be contiguous int32 on the GPU")
// [T, heads, size] view of a (possibly wider) row: heads packed, rows strided
#define CHK_HEADS(t)                                                                                            \
  TORCH_CHECK((t).is_cuda() && (t).dim() == 3 && (t).stride(2) == 1 && (t).stride(1) == (t).size(2),            \
              #t " must be [T, heads, size] rows on the GPU")
#define CHK_ROWS(t) TORCH_CHECK((t).is_cuda() && (t).dim() == 2 && (t).stride(1) == 1, #t " must be rows on the GPU")

const float* opt_f32(const optional<Tensor>& t, int64_t n, const char* what) {
  if (!t.has_value()) return nullptr;
  TORCH_CHECK(t->is_cuda() && t->scalar_type() == at::kFloat && t->is_contiguous() && t->numel() == n, what);
  return t->data_ptr<float>();
}

// a packed step's description (slot numbers come from the block manager that sized the pool)
void check_step(const Tensor& state_slots, const Tensor& row_cu, const Tensor& positions, int64_t T, const char* what) {
  CHK_I32(state_slots); CHK_I32(row_cu); CHK_I32(positions);
  TORCH_CHECK(row_cu.numel() == state_slots.numel() + 1 && positions.numel() == T, what, ": row_cu / positions");
}

void decay_scan(const Tensor& q, const Tensor& k, const Tensor& v, const Tensor& dpow, Tensor& state,
                const Tensor& state_slots, const Tensor& row_cu, const Tensor& positions, int64_t act, bool one_row,
                Tensor& o, const optional<Tensor>& cs, double k_scale) {
  CHK_HEADS(q); CHK_HEADS(k); CHK_HEADS(v); CHK_SAME(k, q); CHK_SAME(v, q);
  CHK_F32(dpow); CHK_F32(state); CHK_F32(o);
  const int64_t T = q.size(0), H = q.size(1), D = q.size(2), Dv = v.size(2);
  TORCH_CHECK(k.sizes() == q.sizes() && v.size(0) == T && v.size(1) == H, "decay_scan: q, k [T, H, D], v [T, H, Dv]");
  TORCH_CHECK(dpow.dim() == 2 && dpow.size(0) == H && dpow.size(1) >= 65, "decay_scan: dpow [H, >= 65]");
  TORCH_CHECK(state.dim() == 4 && state.size(1) == H && state.size(2) == D && state.size(3) == Dv,
              "decay_scan: state [slots, H, D, Dv]");
  check_step(state_slots, row_cu, positions, T, "decay_scan");
  TORCH_CHECK(!one_row || state_slots.numel() == T, "decay_scan: one_row needs one row per sequence");
  TORCH_CHECK(act == 0 || act == 1, "decay_scan: act");
  TORCH_CHECK(D <= 8192, "decay_scan: key size");
  const float* csp = nullptr;
  int64_t nrot = 0;
  if (cs.has_value()) {
    CHK_F32(*cs);
    TORCH_CHECK(cs->dim() == 3 && cs->size(0) == T && cs->size(1) == 2 && 2 * cs->size(2) <= D,
                "decay_scan: cs [T, 2, n], 2 n <= D");
    csp = cs->data_ptr<float>();
    nrot = cs->size(2);
  }
  TORCH_CHECK(o.dim() == 3 && o.size(0) == T && o.size(1) == H && o.size(2) == Dv, "decay_scan: o [T, H, Dv]");
  bfly::launch_decay_scan(q.data_ptr(), q.stride(0), k.data_ptr(), k.stride(0), v.data_ptr(), v.stride(0),
                          dpow.data_ptr<float>(), (int)dpow.size(1), state.data_ptr<float>(), state_slots.data_ptr<int>(),
                          row_cu.data_ptr<int>(), (int)state_slots.numel(), positions.data_ptr<int>(), (int)act,
                          csp, (int)nrot, (float)k_scale, o.data_ptr<float>(), (int)T, (int)H, (int)D, (int)Dv, one_row,
                          is_f32(q), cur_stream());
}

void forget_scan(const Tensor& q, const Tensor& z, const Tensor& v, const Tensor& f_bias, const Tensor& lower, Tensor& state,
                 const Tensor& state_slots, const Tensor& row_cu, const Tensor& positions, int64_t act, bool one_row,
                 Tensor& o) {
  CHK_HEADS(q); CHK_HEADS(z); CHK_HEADS(v); CHK_SAME(z, q); CHK_SAME(v, q);
  CHK_F32(f_bias); CHK_F32(lower); CHK_F32(state); CHK_F32(o);
  const int64_t T = q.size(0), H = q.size(1), D = q.size(2), Dv = v.size(2);
  TORCH_CHECK(z.sizes() == q.sizes() && v.size(0) == T && v.size(1) == H, "forget_scan: q, z [T, H, D], v [T, H, Dv]");
  TORCH_CHECK(f_bias.numel() == H * D && lower.numel() == H * D, "forget_scan: f_bias, lower [H * D]");
  TORCH_CHECK(state.dim() == 4 && state.size(1) == H && state.size(2) == D && state.size(3) == Dv,
              "forget_scan: state [slots, H, D, Dv]");
  check_step(state_slots, row_cu, positions, T, "forget_scan");
  TORCH_CHECK(!one_row || state_slots.numel() == T, "forget_scan: one_row needs one row per sequence");
  TORCH_CHECK((act == 0 || act == 1) && D <= 4096, "forget_scan: act / key size");
  TORCH_CHECK(q.stride(0) < (1 << 21) && z.stride(0) < (1 << 21), "forget_scan: row strides");      // (24-bit byte offsets)
  TORCH_CHECK(o.dim() == 3 && o.size(0) == T && o.size(1) == H && o.size(2) == Dv, "forget_scan: o [T, H, Dv]");
  bfly::launch_forget_scan(q.data_ptr(), q.stride(0), z.data_ptr(), z.stride(0), v.data_ptr(), v.stride(0),
                           f_bias.data_ptr<float>(), lower.data_ptr<float>(), state.data_ptr<float>(),
                           state_slots.data_ptr<int>(), row_cu.data_ptr<int>(), (int)state_slots.numel(),
                           positions.data_ptr<int>(), (int)act, o.data_ptr<float>(), (int)T, (int)H, (int)D, (int)Dv, one_row,
                           is_f32(q), cur_stream());
}

void head_norm_gate(const Tensor& o, const optional<Tensor>& w, double eps, const optional<Tensor>& gate, int64_t act,
                    double mul, Tensor& out) {
  CHK_F32(o); CHK_ROWS(out);
  TORCH_CHECK(o.dim() == 3, "head_norm_gate: o [T, H, Dv]");
  const int64_t T = o.size(0), H = o.size(1), Dv = o.size(2);
  TORCH_CHECK(out.size(0) == T && out.size(1) == H * Dv && (act == 0 || act == 1), "head_norm_gate: out [T, H * Dv] / act");
  const float* wp = opt_f32(w, Dv, "head_norm_gate: w f32 [Dv]");
  const void* gp = nullptr;
  int64_t gld = 0;
  if (gate.has_value()) {
    CHK_ROWS(*gate); CHK_SAME(*gate, out);
    TORCH_CHECK(gate->sizes() == out.sizes(), "head_norm_gate: gate [T, H * Dv]");
    gp = gate->data_ptr();
    gld = gate->stride(0);
  }
  bfly::launch_head_norm_gate(o.data_ptr<float>(), wp, (float)eps, gp, gld, (int)act, (float)mul, out.data_ptr(), out.stride(0),
                              (int)T, (int)H, (int)Dv, is_f32(out), cur_stream());
}

void row_norm_gate(const Tensor& o, const Tensor& w, double eps, const optional<Tensor>& gate, double mul, Tensor& out) {
  CHK_F32(o); CHK_F32(w); CHK_ROWS(out);
  TORCH_CHECK(o.dim() == 2 && out.sizes() == o.sizes() && w.numel() == o.size(1), "row_norm_gate: o, out [T, N], w [N]");
  const void* gp = nullptr;
  int64_t gld = 0;
  if (gate.has_value()) {
    CHK_ROWS(*gate); CHK_SAME(*gate, out);
    TORCH_CHECK(gate->sizes() == o.sizes(), "row_norm_gate: gate [T, N]");
    gp = gate->data_ptr();
    gld = gate->stride(0);
  }
  bfly::launch_row_norm_gate(o.data_ptr<float>(), w.data_ptr<float>(), (float)eps, gp, gld, (float)mul, out.data_ptr(),
                             out.stride(0), (int)o.size(0), (int)o.size(1), is_f32(out), cur_stream());
}

// checks shared by the scan and the step: x, z [T, C], B, C [T, N] rows, a_log [C, N], state [slots, C, N]
void check_selective(const Tensor& x, const Tensor& b, const Tensor& c, const Tensor& z, const Tensor& a_log,
                     const Tensor& dt_bias, const Tensor& d, const Tensor& state, const Tensor& out) {
  CHK_ROWS(x); CHK_ROWS(b); CHK_ROWS(c); CHK_ROWS(z); CHK_ROWS(out);
  CHK_SAME(b, x); CHK_SAME(c, x); CHK_SAME(z, x); CHK_SAME(out, x);
  CHK_F32(a_log); CHK_F32(dt_bias); CHK_F32(d); CHK_F32(state);
  const int64_t T = x.size(0), C = x.size(1), N = a_log.size(1);
  TORCH_CHECK(a_log.dim() == 2 && a_log.size(0) == C && dt_bias.numel() == C && d.numel() == C && z.sizes() == x.sizes(),
              "selective scan: x, z [T, C], a_log [C, N], dt_bias, d [C]");
  TORCH_CHECK(b.size(0) == T && b.size(1) == N && c.sizes() == b.sizes(), "selective scan: B, C [T, N]");
  TORCH_CHECK(state.dim() == 3 && state.size(1) == C && state.size(2) == N, "selective scan: state [slots, C, N]");
  TORCH_CHECK(out.is_contiguous() && out.sizes() == x.sizes(), "selective scan: out [T, C]");
}

void selective_step(const Tensor& x, const Tensor& low, const Tensor& wdt, const Tensor& b, const Tensor& c, const Tensor& z,
                    const Tensor& a_log, const Tensor& dt_bias, const Tensor& d, Tensor& state, const Tensor& state_slots,
                    const Tensor& positions, Tensor& out) {
  check_selective(x, b, c, z, a_log, dt_bias, d, state, out);
  CHK_ROWS(low); CHK_SAME(low, x); CHK_SAME(wdt, x); CHK_I32(state_slots); CHK_I32(positions);
  const int64_t T = x.size(0), C = x.size(1), N = a_log.size(1), R = low.size(1);
  TORCH_CHECK(low.size(0) == T && wdt.is_cuda() && wdt.is_contiguous() && wdt.dim() == 2 && wdt.size(0) == C &&
                  wdt.size(1) == R && R <= 8192, "selective_step: low [T, R], wdt [C, R]");
  TORCH_CHECK(state_slots.numel() == T && positions.numel() == T, "selective_step: one row per sequence");
  const int rc = bfly::launch_selective_step(
      x.data_ptr(), x.stride(0), low.data_ptr(), low.stride(0), wdt.data_ptr(), (int)R, b.data_ptr(), b.stride(0),
      c.data_ptr(), c.stride(0), z.data_ptr(), z.stride(0), a_log.data_ptr<float>(), dt_bias.data_ptr<float>(),
      d.data_ptr<float>(), state.data_ptr<float>(), state_slots.data_ptr<int>(), positions.data_ptr<int>(), out.data_ptr(),
      (int)T, (int)C, (int)N, is_f32(x), cur_stream());
  TORCH_CHECK(rc == 0, "selective_step: ", N, " states per channel are not supported (<= 256)");
}

void selective_scan(const Tensor& x, const Tensor& dtr, const Tensor& b, const Tensor& c, const Tensor& z,
                    const Tensor& a_log, const Tensor& dt_bias, const Tensor& d, Tensor& state, const Tensor& state_slots,
                    const Tensor& row_cu, const Tensor& positions, Tensor& out) {
  check_selective(x, b, c, z, a_log, dt_bias, d, state, out);
  CHK_ROWS(dtr);
  const int64_t T = x.size(0), C = x.size(1), N = a_log.size(1);
  TORCH_CHECK(dtr.scalar_type() == at::kFloat && dtr.size(0) == T && dtr.size(1) == C, "selective_scan: dtr f32 [T, C]");
  check_step(state_slots, row_cu, positions, T, "selective_scan");
  const int rc = bfly::launch_selective_scan(
      x.data_ptr(), x.stride(0), dtr.data_ptr<float>(), dtr.stride(0), b.data_ptr(), b.stride(0), c.data_ptr(), c.stride(0),
      z.data_ptr(), z.stride(0), a_log.data_ptr<float>(), dt_bias.data_ptr<float>(), d.data_ptr<float>(),
      state.data_ptr<float>(), state_slots.data_ptr<int>(), row_cu.data_ptr<int>(), (int)state_slots.numel(),
      positions.data_ptr<int>(), out.data_ptr(), (int)T, (int)C, (int)N, is_f32(x), cur_stream());
  TORCH_CHECK(rc == 0, "selective_scan: ", N, " states per channel are not supported (<= 256)");
}

// caches K [blocks, G, BS, Dp], V [blocks, G, Dvp, BS] and pooled rows [blocks, G, ceil(BS / pool), Dp or Dvp]
void check_pool(const Tensor& kc, const Tensor& vc, int64_t pool, const Tensor& kp, const Tensor& vp, const char* what) {
  const int64_t bs = kc.size(2), pr = (bs + pool - 1) / pool;
  CHK_SAME(kp, kc); CHK_SAME(vp, kc);
  TORCH_CHECK(kp.is_cuda() && vp.is_cuda() && kp.is_contiguous() && vp.is_contiguous() && kp.dim() == 4 && vp.dim() == 4 &&
                  kp.size(0) == kc.size(0) && kp.size(1) == kc.size(1) && kp.size(2) == pr && kp.size(3) == kc.size(3) &&
                  vp.size(0) == kc.size(0) && vp.size(1) == kc.size(1) && vp.size(2) == pr && vp.size(3) == vc.size(2),
              what, ": pooled caches [blocks, G, ceil(BS / pool), size]");
}

void check_caches(const Tensor& kc, const Tensor& vc, const char* what) {
  TORCH_CHECK(kc.is_cuda() && vc.is_cuda() && kc.dim() == 4 && vc.dim() == 4 && kc.is_contiguous() && vc.is_contiguous() &&
                  vc.size(0) == kc.size(0) && vc.size(1) == kc.size(1) && vc.size(3) == kc.size(2),
              what, ": caches K [blocks, G, BS, Dp], V [blocks, G, Dvp, BS]");
}

void qk_norm_rows_kv(const Tensor& q, const Tensor& k, const Tensor& v, const optional<Tensor>& qw,
                     const optional<Tensor>& kw, double eps, const Tensor& slots, Tensor& k_cache, Tensor& v_cache,
                     Tensor& q_out, int64_t pool, const optional<Tensor>& k_pool, const optional<Tensor>& v_pool,
                     const optional<Tensor>& positions, const optional<Tensor>& row_seq, const optional<Tensor>& tables) {
  CHK_HEADS(q); CHK_HEADS(k); CHK_HEADS(v); CHK_SAME(k, q); CHK_SAME(v, q); CHK_SAME(k_cache, q); CHK_SAME(v_cache, q);
  CHK_SAME(q_out, q); CHK_I32(slots);
  check_caches(k_cache, v_cache, "qk_norm_rows_kv");
  const int64_t T = q.size(0), H = q.size(1), D = q.size(2), G = k.size(1), Dv = v.size(2);
  const int64_t Dp = k_cache.size(3), Dvp = v_cache.size(2), bs = k_cache.size(2);
  TORCH_CHECK(k.size(0) == T && k.size(2) == D && v.size(0) == T && v.size(1) == G && k_cache.size(1) == G && Dp >= D &&
                  Dvp >= Dv && slots.numel() == T, "qk_norm_rows_kv: shapes");
  TORCH_CHECK(q_out.is_cuda() && q_out.is_contiguous() && q_out.dim() == 3 && q_out.size(0) == T && q_out.size(1) == H &&
                  q_out.size(2) == Dp, "qk_norm_rows_kv: q_out [T, H, Dp]");
  const float* qwp = opt_f32(qw, H * D, "qk_norm_rows_kv: query weight f32 [H * D]");
  const float* kwp = opt_f32(kw, G * D, "qk_norm_rows_kv: key weight f32 [G * D]");
  TORCH_CHECK(pool >= 0, "qk_norm_rows_kv: pool");
  void *kp = nullptr, *vp = nullptr;
  const int *pos = nullptr, *rs = nullptr, *tab = nullptr;
  int64_t pr = 0, mb = 0;
  if (pool > 0) {
    TORCH_CHECK(k_pool.has_value() && v_pool.has_value() && positions.has_value() && row_seq.has_value() &&
                    tables.has_value(), "qk_norm_rows_kv: pooling needs the pooled caches and the step's description");
    check_pool(k_cache, v_cache, pool, *k_pool, *v_pool, "qk_norm_rows_kv");
    CHK_I32(*positions); CHK_I32(*row_seq); CHK_I32(*tables);
    TORCH_CHECK(positions->numel() == T && row_seq->numel() == T && tables->dim() == 2 && tables->size(0) == T,
                "qk_norm_rows_kv: pooling in the same launch takes steps of one row per sequence");
    kp = k_pool->data_ptr(); vp = v_pool->data_ptr();
    pos = positions->data_ptr<int>(); rs = row_seq->data_ptr<int>(); tab = tables->data_ptr<int>();
    pr = k_pool->size(2); mb = tables->size(1);
  }
  bfly::launch_qk_norm_rows_kv(q.data_ptr(), q.stride(0), k.data_ptr(), k.stride(0), v.data_ptr(), v.stride(0), qwp, kwp,
                               (float)eps, slots.data_ptr<int>(), k_cache.data_ptr(), v_cache.data_ptr(), q_out.data_ptr(),
                               (int)T, (int)H, (int)G, (int)D, (int)Dv, (int)Dp, (int)Dvp, (int)bs, (int)pool, (int)pr, kp,
                               vp, pos, rs, tab, (int)mb, is_f32(q), cur_stream());
}

void pool_blocks(const Tensor& k_cache, const Tensor& v_cache, const Tensor& tables, const Tensor& row_seq,
                 const Tensor& positions, const Tensor& slots, int64_t pool, Tensor& k_pool, Tensor& v_pool) {
  CHK_SAME(v_cache, k_cache);
  CHK_I32(tables); CHK_I32(row_seq); CHK_I32(positions); CHK_I32(slots);
  check_caches(k_cache, v_cache, "pool_blocks");
  TORCH_CHECK(pool >= 1, "pool_blocks: pool >= 1");
  check_pool(k_cache, v_cache, pool, k_pool, v_pool, "pool_blocks");
  const int64_t T = positions.numel();
  TORCH_CHECK(tables.dim() == 2 && row_seq.numel() == T && slots.numel() == T, "pool_blocks: index shapes");
  bfly::launch_pool_blocks(k_cache.data_ptr(), v_cache.data_ptr(), tables.data_ptr<int>(), (int)tables.size(1),
                           row_seq.data_ptr<int>(), positions.data_ptr<int>(), slots.data_ptr<int>(), (int)pool,
                           (int)k_pool.size(2), k_pool.data_ptr(), v_pool.data_ptr(), (int)T, (int)k_cache.size(1),
                           (int)k_cache.size(3), (int)v_cache.size(2), (int)k_cache.size(2), is_f32(k_cache), cur_stream());
}

}  // namespace

TORCH_LIBRARY_FRAGMENT(bfly, m) {
  m.def("decay_scan(Tensor q, Tensor k, Tensor v, Tensor dpow, Tensor(a!) state, Tensor state_slots, Tensor row_cu, "
        "Tensor positions, int act, bool one_row, Tensor(b!) o, Tensor? cs=None, float k_scale=1.0) -> ()");
  m.def("forget_scan(Tensor q, Tensor z, Tensor v, Tensor f_bias, Tensor lower, Tensor(a!) state, Tensor state_slots, "
        "Tensor row_cu, Tensor positions, int act, bool one_row, Tensor(b!) o) -> ()");
  m.def("head_norm_gate(Tensor o, Tensor? w, float eps, Tensor? gate, int act, float mul, Tensor(a!) out) -> ()");
  m.def("row_norm_gate(Tensor o, Tensor w, float eps, Tensor? gate, float mul, Tensor(a!) out) -> ()");
  m.def("selective_scan(Tensor x, Tensor dtr, Tensor b, Tensor c, Tensor z, Tensor a_log, Tensor dt_bias, Tensor d, "
        "Tensor(a!) state, Tensor state_slots, Tensor row_cu, Tensor positions, Tensor(b!) out) -> ()");
  m.def("selective_step(Tensor x, Tensor low, Tensor wdt, Tensor b, Tensor c, Tensor z, Tensor a_log, Tensor dt_bias, "
        "Tensor d, Tensor(a!) state, Tensor state_slots, Tensor positions, Tensor(b!) out) -> ()");
  m.def("qk_norm_rows_kv(Tensor q, Tensor k, Tensor v, Tensor? qw, Tensor? kw, float eps, Tensor slots, "
        "Tensor(a!) k_cache, Tensor(b!) v_cache, Tensor(c!) q_out, int pool, Tensor(d!)? k_pool, Tensor(e!)? v_pool, "
        "Tensor? positions, Tensor? row_seq, Tensor? tables) -> ()");
  m.def("pool_blocks(Tensor k_cache, Tensor v_cache, Tensor tables, Tensor row_seq, Tensor positions, Tensor slots, "
        "int pool, Tensor(a!) k_pool, Tensor(b!) v_pool) -> ()");
}

TORCH_LIBRARY_IMPL(bfly, CUDA, m) {
  m.impl("decay_scan", &decay_scan);
  m.impl("forget_scan", &forget_scan);
  m.impl("head_norm_gate", &head_norm_gate);
  m.impl("row_norm_gate", &row_norm_gate);
  m.impl("selective_scan", &selective_scan);
  m.impl("selective_step", &selective_step);
  m.impl("qk_norm_rows_kv", &qk_norm_rows_kv);
  m.impl("pool_blocks", &pool_blocks);
}
