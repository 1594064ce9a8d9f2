// Gated linear attention: per head a state S [D, V] from zero whose rows decay by a gate per key channel,
//
//   f = sigmoid(z + b)^(1 / tau),  z = W_2 (W_1 h)  (a low-rank pair),   S = diag(f) S + k v',   y = S' q     (q times a constant)
//   out = y / sqrt(mean(y^2) + eps) * gain * silu(g)
//
// The kernels are gated_rule.h's: a walk over a request's rows (a decoded token is one of one row; W_2 is applied inside it), and the
// rule in chunks for long portions, which reads z as a float32 product.
#include "gated_rule.h"

namespace {
RuleArgs linear_rule(const void* raw, long ld, int off_q, int off_k, int off_v, int off_g, const float* bias, float inv_tau, float q_scale,
                     const float* gain, float eps, float* state, long slot_stride, const int* cu, const int* slot, void* out, int H, int D, int V) {
  RuleArgs a{};
  a.raw = raw; a.ld = ld; a.off_q = off_q; a.off_k = off_k; a.off_v = off_v; a.off_g = off_g;
  a.bias = bias; a.inv_tau = inv_tau; a.q_scale = q_scale; a.gain = gain; a.eps = eps;
  a.state = state; a.slot_stride = slot_stride; a.cu = cu; a.slot = slot; a.out = out; a.H = H; a.D = D; a.V = V;
  return a;
}
int check(const char* what, const RuleArgs& a, int dtype) {
  GIBBS_REQUIRE(a.raw && a.bias && a.gain && a.state && a.slot && a.out, "%s: null operand", what);
  GIBBS_REQUIRE(a.H > 0 && a.H <= 65535 && a.D > 0 && a.V > 0 && a.off_q >= 0 && a.off_k >= 0 && a.off_v >= 0 && a.off_g >= 0 && a.inv_tau > 0.f,
                "%s: heads=%d D=%d V=%d", what, a.H, a.D, a.V);
  GIBBS_REQUIRE(a.ld >= std::max(std::max(a.off_q, a.off_k) + (long)a.H * a.D, std::max(a.off_v, a.off_g) + (long)a.H * a.V), "%s: rows of %ld values are too short", what, a.ld);
  GIBBS_REQUIRE(a.slot_stride >= (long)a.H * a.D * a.V, "%s: a slot of %ld floats is too small", what, a.slot_stride);
  GIBBS_REQUIRE(dtype == GIBBS_F32 || dtype == GIBBS_BF16, "%s: unknown dtype %d", what, dtype);
  return 0;
}
}  // namespace

// Whether the row kernel and the rule in chunks take a head's sizes, and the floats of workspace that the latter needs.
GIBBS_EXPORT int gibbs_gated_linear_rows_take(int D, int V) { return rule_rows_take(D, V); }
GIBBS_EXPORT int gibbs_gated_linear_chunks_take(int D, int V) { return rule_chunks_take(D, V); }
GIBBS_EXPORT long gibbs_gated_linear_chunks_workspace(int rows, int n_req, int H, int D, int V) { return rule_chunks_workspace(rows, n_req, H, D, V); }

// raw: projected rows (row stride ld) with q and k (heads * dim), v and g (heads * vdim) and the low-rank columns of the gate (`rank` of
// them) at their offsets; w_z [heads * dim, rank] in the rows' type; bias [heads * dim]; gain [vdim].  state [slots][heads][dim]
// [vdim].  cu null: row n is request n's; else the rows cu[r] .. cu[r + 1].  out [.., heads * vdim] in the rows' type.
GIBBS_EXPORT int gibbs_gated_linear_rows(const void* raw, long ld, int off_q, int off_k, int off_v, int off_g, int off_z, const void* w_z, int rank,
                                         const float* bias, float inv_tau, float q_scale, const float* gain, float eps, float* state,
                                         long slot_stride, const int* cu, const int* slot, void* out, int dtype, int n_req, int H, int D, int V,
                                         hipStream_t stream) {
  RuleArgs a = linear_rule(raw, ld, off_q, off_k, off_v, off_g, bias, inv_tau, q_scale, gain, eps, state, slot_stride, cu, slot, out, H, D, V);
  if (check("gated_linear_rows", a, dtype)) return 1;
  GIBBS_REQUIRE(w_z && rank > 0 && off_z >= 0 && ld >= (long)off_z + rank && n_req > 0 && rule_rows_take(D, V), "gated_linear_rows: requests=%d rank=%d, states of %d x %d", n_req, rank, D, V);
  a.w_z = w_z; a.off_z = off_z; a.rank = rank;
  a.vec_z = rank % 8 == 0 && off_z % 8 == 0 && ld % 8 == 0 && ((uintptr_t)raw % 16) == 0 && ((uintptr_t)w_z % 16) == 0;
  if (dtype == GIBBS_F32 ? launch_rule_rows<float, RULE_LINEAR>(a, n_req, stream) : launch_rule_rows<bf16, RULE_LINEAR>(a, n_req, stream)) return 1;
  GIBBS_LAUNCH_STATUS("gated_linear_rows");
}

// The rows cu[0] .. of n_req requests (raw and out are addressed by the step's rows, cu may start above 0), n_rows in all; z [n_rows,
// heads * dim] float32: the gate's projection of those rows, without the bias.
GIBBS_EXPORT int gibbs_gated_linear_chunks(const void* raw, long ld, int off_q, int off_k, int off_v, int off_g, const float* z, const float* bias,
                                           float inv_tau, float q_scale, const float* gain, float eps, float* state, long slot_stride,
                                           const int* cu, const int* slot, void* out, float* workspace, int dtype, int n_rows, int n_req, int H,
                                           int D, int V, hipStream_t stream) {
  RuleArgs a = linear_rule(raw, ld, off_q, off_k, off_v, off_g, bias, inv_tau, q_scale, gain, eps, state, slot_stride, cu, slot, out, H, D, V);
  if (check("gated_linear_chunks", a, dtype)) return 1;
  GIBBS_REQUIRE(z && cu && workspace && n_rows > 0 && n_req > 0 && n_req <= 65535 && rule_chunks_take(D, V), "gated_linear_chunks: rows=%d requests=%d, states of %d x %d", n_rows, n_req, D, V);
  a.z = z;
  const int places = ceil_div(n_rows, CHUNK) + n_req;      // (more than the requests' chunks can be)
  if (dtype == GIBBS_F32 ? launch_chunks<float, RULE_LINEAR>(a, workspace, places, n_req, stream) : launch_chunks<bf16, RULE_LINEAR>(a, workspace, places, n_req, stream)) return 1;
  GIBBS_LAUNCH_STATUS("gated_linear_chunks");
}
