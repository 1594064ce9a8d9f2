// What a differential attention does around the scores (the attention itself is the framework's: a map is a query head whose
// query is zero where the other map's key lies).
//
//   prepare  projected rows [q: H x 2 maps x dim | k: G x 2 maps x dim | v: G x vdim | ..] become
//              queries  q_out[n][2 h + c] (size ks): zeros, but for entries c dim .. c dim + dim - 1 = turn(norm(q_(h,c)))
//              keys     page row of kv head g (size ks): [turn(norm(k_(g,1))) | turn(norm(k_(g,2))) | zeros]
//              values   page row of kv head g (size vs): [v_g | zeros]
//            norm: x / sqrt(mean(x^2) + eps) * gain over dim; turn: the first `rot` entries by the row's position (pairs half-split
//            or interleaved), the rest pass
//   finish   o[n][h] = (a_1 - lambda a_2) / sqrt(mean(.^2) + eps) * out_scale * sigmoid(gate[n][h]), a_c = att[n][2 h + c][:vdim]
//
// Norms, angles and the combination are float32; lambda is one number on the device.
#include "common.h"
#include "lane8.h"

namespace {
struct DiffPrepareArgs {
  const float* q_gain;      // [dim]
  const float* k_gain;      // [dim]
  const float* inv_freq;    // [rot / 2] or null: no rotation
  const float2* cs_table;   // [table_len, rot / 2] of (cos, sin), or null
  int rot, variant, table_len;
  float eps;
  const int* pos;
  const int* row_req;
  const int* table;
  int max_pages, page_size, num_pages;
  int H, G, dim, vdim, ks, vs;
  long ld;
};

// LPH lanes share one map of a head of q or k, or one head of v.
template <typename T, int LPH>
__global__ __launch_bounds__(256) void diff_prepare_kernel(const T* __restrict__ rows, T* __restrict__ q_out, T* __restrict__ kpages,
                                                           T* __restrict__ vpages, DiffPrepareArgs a) {
  const int n = blockIdx.x;
  const int it = blockIdx.y * (blockDim.x / LPH) + threadIdx.x / LPH, lane = threadIdx.x % LPH;
  const int q_items = 2 * a.H, k_items = 2 * a.G;
  if (it >= q_items + k_items + a.G) return;
  const T* row = rows + (size_t)n * a.ld;
  const int p = a.pos[n];
  const bool is_q = it < q_items, is_v = it >= q_items + k_items;
  const int g = is_q ? 0 : (is_v ? it - q_items - k_items : (it - q_items) / 2);
  size_t at = 0;      // where the position's row of kv head g lies, in rows
  if (!is_q) {
    const int page = a.table[(size_t)a.row_req[n] * a.max_pages + p / a.page_size];
    if (page < 0 || page >= a.num_pages) return;      // (the host never asks for another; never write outside the pool)
    at = ((size_t)page * a.G + g) * a.page_size + p % a.page_size;
  }
  if (is_v) {
    const T* src = row + (size_t)(q_items + k_items) * a.dim + (size_t)g * a.vdim;
    T* dst = vpages + at * a.vs;
    for (int e = lane; e < a.vs; e += LPH) dst[e] = e < a.vdim ? src[e] : from_float<T>(0.f);
    return;
  }
  const T* src = row + (size_t)it * a.dim;
  const int c = it % 2;                               // the map
  T* head = is_q ? q_out + ((size_t)n * q_items + it) * a.ks : kpages + at * a.ks;
  T* dst = head + (size_t)c * a.dim;
  const float* gain = is_q ? a.q_gain : a.k_gain;
  float ss = 0.f;
  for (int e = lane; e < a.dim; e += LPH) { const float x = to_float(src[e]); ss = fmaf(x, x, ss); }
  const float inv = 1.0f / sqrtf((LPH == WAVE ? wave_sum(ss) : group_sum<LPH>(ss)) / (float)a.dim + a.eps);
  const int half = a.inv_freq ? a.rot / 2 : 0;
  for (int j = lane; j < half; j += LPH) {
    const int i0 = a.variant == 0 ? j : 2 * j, i1 = a.variant == 0 ? j + half : 2 * j + 1;
    const float x0 = to_float(src[i0]) * inv * gain[i0], x1 = to_float(src[i1]) * inv * gain[i1];
    float co, si;
    if (a.cs_table && p < a.table_len) {
      const float2 cs = a.cs_table[(size_t)p * half + j];
      co = cs.x;
      si = cs.y;
    } else {
      rope_cos_sin((float)p * a.inv_freq[j], &co, &si);
    }
    dst[i0] = from_float<T>(x0 * co - x1 * si);
    dst[i1] = from_float<T>(x1 * co + x0 * si);
  }
  for (int e = 2 * half + lane; e < a.dim; e += LPH) dst[e] = from_float<T>(to_float(src[e]) * inv * gain[e]);
  // zeros: a query's other map and what lies behind both; behind both of a key's (its second map's lanes write them)
  if (is_q) {
    for (int e = lane; e < a.ks - a.dim; e += LPH) {
      head[(c == 1 && e < a.dim) ? e : e + a.dim] = from_float<T>(0.f);
    }
  } else if (c == 1) {
    for (int e = 2 * a.dim + lane; e < a.ks; e += LPH) head[e] = from_float<T>(0.f);
  }
}

// LPH lanes share a head; TA: the type of the attention's outputs.
template <typename T, typename TA, int LPH>
__global__ __launch_bounds__(256) void diff_finish_kernel(const TA* __restrict__ att, int vs, const T* __restrict__ gate, long ld_gate,
                                                          const float* __restrict__ lambda, float eps, float out_scale, T* __restrict__ o,
                                                          int n_rows, int H, int V) {
  const long item = (long)blockIdx.x * (blockDim.x / LPH) + threadIdx.x / LPH;
  const int lane = threadIdx.x % LPH;
  if (item >= (long)n_rows * H) return;
  const int n = (int)(item / H), h = (int)(item % H);
  const float lam = *lambda;
  const TA* a1 = att + (size_t)item * 2 * vs;
  const TA* a2 = a1 + vs;
  float ss = 0.f;
  for (int e = lane; e < V; e += LPH) {
    const float d = to_float(a1[e]) - lam * to_float(a2[e]);
    ss = fmaf(d, d, ss);
  }
  float f = out_scale / sqrtf((LPH == WAVE ? wave_sum(ss) : group_sum<LPH>(ss)) / (float)V + eps);
  if (gate) f /= 1.0f + expf(-to_float(gate[(size_t)n * ld_gate + h]));
  for (int e = lane; e < V; e += LPH) o[(size_t)item * V + e] = from_float<T>((to_float(a1[e]) - lam * to_float(a2[e])) * f);
}
}  // namespace

GIBBS_EXPORT int gibbs_diff_prepare(const void* rows, long ld, void* q_out, void* kpages, void* vpages, int dtype, const float* q_gain,
                                    const float* k_gain, float eps, const float* inv_freq, int rot, int variant, const float* cs_table,
                                    int table_len, const int* pos, const int* row_req, const int* table, int max_pages, int page_size,
                                    int num_pages, int n_rows, int H, int G, int dim, int vdim, int ks, int vs, hipStream_t stream) {
  GIBBS_REQUIRE(rows && q_out && kpages && vpages && q_gain && k_gain && pos && row_req && table && n_rows > 0, "diff_prepare: null operand or no rows");
  GIBBS_REQUIRE(H > 0 && G > 0 && dim > 0 && vdim > 0 && ks >= 2 * dim && vs >= vdim && ld >= (long)2 * (H + G) * dim + (long)G * vdim,
                "diff_prepare: bad sizes heads=%d kv=%d dim=%d vdim=%d stored %d, %d", H, G, dim, vdim, ks, vs);
  GIBBS_REQUIRE(max_pages > 0 && page_size > 0 && num_pages > 0, "diff_prepare: bad cache geometry");
  GIBBS_REQUIRE(!inv_freq || (rot > 0 && rot % 2 == 0 && rot <= dim && (variant == 0 || variant == 1)), "diff_prepare: %d turned entries of a map of %d", rot, dim);
  DiffPrepareArgs a{q_gain, k_gain, inv_freq, (const float2*)cs_table, inv_freq ? rot : 0, variant, cs_table && inv_freq ? table_len : 0, eps, pos, row_req,
                    table, max_pages, page_size, num_pages, H, G, dim, vdim, ks, vs, ld};
  const bool narrow = dim <= 128 && vdim <= 256;
  const dim3 grid(n_rows, ceil_div(2 * H + 3 * G, narrow ? 16 : 4));
  GIBBS_REQUIRE(grid.y <= 65535, "diff_prepare: too many heads (%d)", H);
  if (dtype == GIBBS_F32) {
    if (narrow) diff_prepare_kernel<float, 16><<<grid, 256, 0, stream>>>((const float*)rows, (float*)q_out, (float*)kpages, (float*)vpages, a);
    else diff_prepare_kernel<float, 64><<<grid, 256, 0, stream>>>((const float*)rows, (float*)q_out, (float*)kpages, (float*)vpages, a);
  } else if (dtype == GIBBS_BF16) {
    if (narrow) diff_prepare_kernel<bf16, 16><<<grid, 256, 0, stream>>>((const bf16*)rows, (bf16*)q_out, (bf16*)kpages, (bf16*)vpages, a);
    else diff_prepare_kernel<bf16, 64><<<grid, 256, 0, stream>>>((const bf16*)rows, (bf16*)q_out, (bf16*)kpages, (bf16*)vpages, a);
  } else {
    return gibbs_fail("diff_prepare: unknown dtype %d", dtype);
  }
  GIBBS_LAUNCH_STATUS("diff_prepare");
}

// att: [n_rows, 2 H, vs] in the activation type; gate: rows of H values (stride ld_gate) or null; o: [n_rows, H * V].
GIBBS_EXPORT int gibbs_diff_finish(const void* att, int vs, const void* gate, long ld_gate, const float* lambda, float eps, float out_scale,
                                   void* o, int dtype, int n_rows, int H, int V, hipStream_t stream) {
  GIBBS_REQUIRE(att && lambda && o && n_rows > 0 && H > 0 && V > 0 && vs >= V && (!gate || ld_gate >= H), "diff_finish: bad operands rows=%d heads=%d V=%d", n_rows, H, V);
  const int lph = V <= 128 ? 16 : 64;
  const int grid = ceil_div((long)n_rows * H, 256 / lph);
#define DIFF_FINISH(T) \
  do { \
    if (lph == 16) diff_finish_kernel<T, T, 16><<<grid, 256, 0, stream>>>((const T*)att, vs, (const T*)gate, ld_gate, lambda, eps, out_scale, (T*)o, n_rows, H, V); \
    else diff_finish_kernel<T, T, 64><<<grid, 256, 0, stream>>>((const T*)att, vs, (const T*)gate, ld_gate, lambda, eps, out_scale, (T*)o, n_rows, H, V); \
  } while (0)
  if (dtype == GIBBS_F32) DIFF_FINISH(float);
  else if (dtype == GIBBS_BF16) DIFF_FINISH(bf16);
  else return gibbs_fail("diff_finish: unknown dtype %d", dtype);
#undef DIFF_FINISH
  GIBBS_LAUNCH_STATUS("diff_finish");
}
