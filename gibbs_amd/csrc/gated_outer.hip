// The gated outer-product recurrence around its walk (recurrent.hip): per head, with a gate f per channel,
//
//   q = silu(a),  f = l + (1 - l) sigmoid(z + b),  k = 1 - f = (1 - l) sigmoid(-(z + b))        (a, z, v: projected rows)
//   S = diag(f) S + k v',   y = S' q                                                          (S [D, V] from zero)
//   out = y / sqrt(mean(y^2) + eps) * gain
//
//   prep   q, f, k, v of a step's rows as float32, for the walk over ragged portions
//   step   everything above in one kernel for a step of one token per request (gated_rule.h)
//   chunks the rule for long portions, regrouped into products on the matrix cores (gated_rule.h)
//
// Everything behind the projections is float32, and so is the state.
#include "gated_rule.h"

namespace {
// raw [N, ld]: rows [a: H D | z: H D | v: H V]
template <typename T>
__global__ __launch_bounds__(256) void gated_outer_prep_kernel(const T* __restrict__ raw, long ld, const float* __restrict__ bias,
                                                               const float* __restrict__ lower, float* __restrict__ q, float* __restrict__ f,
                                                               float* __restrict__ k, float* __restrict__ v, int n_rows, int C, int HV) {
  const long item = (long)blockIdx.x * blockDim.x + threadIdx.x;
  const int per = C + HV;
  if (item >= (long)n_rows * per) return;
  const int n = (int)(item / per), c = (int)(item % per);
  const T* row = raw + (size_t)n * ld;
  if (c >= C) {
    v[(size_t)n * HV + c - C] = to_float(row[C + c]);
    return;
  }
  const float a = to_float(row[c]);
  const Gate g = gate_of(to_float(row[C + c]) + bias[c], lower[c]);
  q[(size_t)n * C + c] = a * sigm(a);
  f[(size_t)n * C + c] = g.f;
  k[(size_t)n * C + c] = g.k;
}

RuleArgs complement_rule(const void* raw, long ld, const float* bias, const float* lower, const float* gain, float eps, float* state, long slot_stride,
                         const int* cu, const int* slot, void* out, int H, int D, int V) {
  RuleArgs a{};
  a.raw = raw; a.ld = ld; a.off_q = 0; a.off_k = H * D; a.off_v = 2 * H * D;
  a.bias = bias; a.lower = lower; a.gain = gain; a.eps = eps;
  a.state = state; a.slot_stride = slot_stride; a.cu = cu; a.slot = slot; a.out = out; a.H = H; a.D = D; a.V = V;
  return a;
}
}  // namespace

// Whether the rule in chunks takes a head's sizes, and the floats of workspace that `rows` rows of `n_req` requests need.
GIBBS_EXPORT int gibbs_gated_outer_chunks_take(int D, int V) {
  return rule_chunks_take(D, V);
}
GIBBS_EXPORT long gibbs_gated_outer_chunks_workspace(int rows, int n_req, int H, int D, int V) {
  return rule_chunks_workspace(rows, n_req, H, D, V);
}
// The rows cu[0] .. of n_req requests (cu may start above 0): raw and out are addressed by the step's rows.  n_rows: the rows in
// all.  out: [.., H * V] in the activation type, normed per head; the requests' states are read and left as the rule leaves them.
GIBBS_EXPORT int gibbs_gated_outer_chunks(const void* raw, long ld, int dtype, const float* bias, const float* lower, const float* gain, float eps,
                                          float* state, long slot_stride, const int* cu, const int* slot, void* out, float* workspace,
                                          int n_rows, int n_req, int H, int D, int V, hipStream_t stream) {
  GIBBS_REQUIRE(raw && bias && lower && gain && state && cu && slot && out && workspace && n_rows > 0 && n_req > 0 && n_req <= 65535,
                "gated_outer_chunks: null operand or no rows");
  GIBBS_REQUIRE(H > 0 && H <= 65535 && gibbs_gated_outer_chunks_take(D, V) && ld >= (long)H * (2 * D + V) && slot_stride >= (long)H * D * V,
                "gated_outer_chunks: heads=%d D=%d V=%d", H, D, V);
  const int places = ceil_div(n_rows, CHUNK) + n_req;      // (more than the requests' chunks can be)
  const RuleArgs a = complement_rule(raw, ld, bias, lower, gain, eps, state, slot_stride, cu, slot, out, H, D, V);
  if (dtype == GIBBS_F32) { if (launch_chunks<float, RULE_COMPLEMENT>(a, workspace, places, n_req, stream)) return 1; }
  else if (dtype == GIBBS_BF16) { if (launch_chunks<bf16, RULE_COMPLEMENT>(a, workspace, places, n_req, stream)) return 1; }
  else return gibbs_fail("gated_outer_chunks: unknown dtype %d", dtype);
  GIBBS_LAUNCH_STATUS("gated_outer_chunks");
}

GIBBS_EXPORT int gibbs_gated_outer_prep(const void* raw, long ld, int dtype, const float* bias, const float* lower, float* q, float* f, float* k,
                                        float* v, int n_rows, int H, int D, int V, hipStream_t stream) {
  GIBBS_REQUIRE(raw && bias && lower && q && f && k && v && n_rows > 0 && H > 0 && D > 0 && V > 0 && ld >= (long)H * (2 * D + V),
                "gated_outer_prep: bad operands rows=%d heads=%d D=%d V=%d", n_rows, H, D, V);
  const int grid = ceil_div((long)n_rows * H * (D + V), 256);
  if (dtype == GIBBS_F32)
    gated_outer_prep_kernel<float><<<grid, 256, 0, stream>>>((const float*)raw, ld, bias, lower, q, f, k, v, n_rows, H * D, H * V);
  else if (dtype == GIBBS_BF16)
    gated_outer_prep_kernel<bf16><<<grid, 256, 0, stream>>>((const bf16*)raw, ld, bias, lower, q, f, k, v, n_rows, H * D, H * V);
  else
    return gibbs_fail("gated_outer_prep: unknown dtype %d", dtype);
  GIBBS_LAUNCH_STATUS("gated_outer_prep");
}

// Whether the step kernel takes a head's sizes.
GIBBS_EXPORT int gibbs_gated_outer_step_takes(int D, int V) { return rule_rows_take(D, V) && D <= 256 && V <= STEP_THREADS; }

// Row n is request n.  out: [n_req, H * V] in the activation type.
GIBBS_EXPORT int gibbs_gated_outer_step(const void* raw, long ld, int dtype, const float* bias, const float* lower, const float* gain, float eps,
                                        float* state, long slot_stride, const int* slot, void* out, int n_req, int H, int D, int V,
                                        hipStream_t stream) {
  GIBBS_REQUIRE(raw && bias && lower && gain && state && slot && out && n_req > 0 && H > 0 && H <= 65535 && ld >= (long)H * (2 * D + V),
                "gated_outer_step: bad operands rows=%d heads=%d", n_req, H);
  GIBBS_REQUIRE(gibbs_gated_outer_step_takes(D, V) && slot_stride >= (long)H * D * V, "gated_outer_step: states of %d x %d", D, V);
  const RuleArgs a = complement_rule(raw, ld, bias, lower, gain, eps, state, slot_stride, nullptr, slot, out, H, D, V);
  if (dtype == GIBBS_F32) { if (launch_rule_rows<float, RULE_COMPLEMENT>(a, n_req, stream)) return 1; }
  else if (dtype == GIBBS_BF16) { if (launch_rule_rows<bf16, RULE_COMPLEMENT>(a, n_req, stream)) return 1; }
  else return gibbs_fail("gated_outer_step: unknown dtype %d", dtype);
  GIBBS_LAUNCH_STATUS("gated_outer_step");
}
