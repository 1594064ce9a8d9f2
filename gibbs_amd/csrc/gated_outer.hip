// The gated outer-product recurrence around its walk (recurrent.hip): per head, with a gate f per channel,
//
//   q = silu(a),  f = l + (1 - l) sigmoid(z + b),  k = 1 - f = (1 - l) sigmoid(-(z + b))        (a, z, v: projected rows)
//   S = diag(f) S + k v',   y = S' q                                                          (S [D, V] from zero)
//   out = y / sqrt(mean(y^2) + eps) * gain
//
//   prep   q, f, k, v of a step's rows as float32, for the walk over ragged portions
//   step   everything above in one kernel for a step of one token per request: a workgroup owns one head of one request and
//          streams its state once, in whole rows
//
// Everything behind the projections is float32, and so is the state.
#include "common.h"

namespace {
__device__ __forceinline__ float sigm(float z) { return 1.0f / (1.0f + expf(-z)); }
struct Gate { float f, k; };
__device__ __forceinline__ Gate gate_of(float z, float l) {
  // (both exponentials taken with a negative argument: no overflow, and 1 - f without cancellation)
  const float e = expf(-fabsf(z)), inv = 1.0f / (1.0f + e);
  const float s = z >= 0.f ? inv : e * inv, t = z >= 0.f ? e * inv : inv;
  return Gate{fmaf(1.0f - l, s, l), (1.0f - l) * t};
}

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

// Thread (tx, group): columns tx VEC .. and rows group, group + groups, ...; y by groups, added in group order.
constexpr int STEP_THREADS = 512, STEP_ROWS = 8;
template <typename T, int VEC>
__global__ __launch_bounds__(STEP_THREADS) void gated_outer_step_kernel(const T* __restrict__ raw, long ld, const float* __restrict__ bias,
                                                                        const float* __restrict__ lower, const float* __restrict__ gain, float eps,
                                                                        float* __restrict__ state, long slot_stride, const int* __restrict__ slot,
                                                                        T* __restrict__ out, int H, int D, int V, int lanes) {
  extern __shared__ float part[];      // [groups][V]
  __shared__ float sq[256], sf[256], sk[256], scratch[16];
  const int n = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int tx = tid % lanes, group = tid / lanes, groups = STEP_THREADS / lanes;
  const int j0 = tx * VEC;
  const bool live = j0 < V;
  const T* row = raw + (size_t)n * ld;
  float* st = state + (size_t)slot[n] * slot_stride + (size_t)h * D * V + j0;
  // the first rows of the state are asked for before anything else
  float s[STEP_ROWS][VEC];
  auto ask = [&](int i0) {
#pragma unroll
    for (int u = 0; u < STEP_ROWS; ++u) {
      const int i = i0 + u * groups;
      if (live && i < D) {
        if constexpr (VEC == 4) { const float4 t = *(const float4*)(st + (size_t)i * V); s[u][0] = t.x; s[u][1] = t.y; s[u][2] = t.z; s[u][3] = t.w; }
        else s[u][0] = st[(size_t)i * V];
      }
    }
  };
  ask(group);
  const int C = H * D;
  for (int i = tid; i < D; i += STEP_THREADS) {
    const int c = h * D + i;
    const float a = to_float(row[c]);
    const Gate g = gate_of(to_float(row[C + c]) + bias[c], lower[c]);
    sq[i] = a * sigm(a);
    sf[i] = g.f;
    sk[i] = g.k;
  }
  float v[VEC], y[VEC];
#pragma unroll
  for (int e = 0; e < VEC; ++e) {
    v[e] = live ? to_float(row[2 * C + h * V + j0 + e]) : 0.f;
    y[e] = 0.f;
  }
  __syncthreads();
  for (int i0 = group; i0 < D; i0 += STEP_ROWS * groups) {
    if (i0 != group) ask(i0);
#pragma unroll
    for (int u = 0; u < STEP_ROWS; ++u) {
      const int i = i0 + u * groups;
      if (live && i < D) {
        const float f = sf[i], k = sk[i], q = sq[i];
#pragma unroll
        for (int e = 0; e < VEC; ++e) {
          s[u][e] = fmaf(f, s[u][e], k * v[e]);
          y[e] = fmaf(s[u][e], q, y[e]);
        }
        if constexpr (VEC == 4) *(float4*)(st + (size_t)i * V) = make_float4(s[u][0], s[u][1], s[u][2], s[u][3]);
        else st[(size_t)i * V] = s[u][0];
      }
    }
  }
  if (live) {
#pragma unroll
    for (int e = 0; e < VEC; ++e) part[group * V + j0 + e] = y[e];
  }
  __syncthreads();
  float ss = 0.f;
  for (int j = tid; j < V; j += STEP_THREADS) {
    float t = part[j];
    for (int g = 1; g < groups; ++g) t += part[g * V + j];
    part[j] = t;
    ss = fmaf(t, t, ss);
  }
  const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / (float)V + eps);
  for (int j = tid; j < V; j += STEP_THREADS) out[((size_t)n * H + h) * V + j] = from_float<T>(part[j] * inv * gain[j]);
}
}  // namespace

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
GIBBS_EXPORT int gibbs_gated_outer_step_takes(int D, int V) { return D > 0 && D <= 256 && V > 0 && V <= STEP_THREADS; }

// Row n is request n.  out: [n_req, H * V] in the activation type.
GIBBS_EXPORT int gibbs_gated_outer_step(const void* raw, long ld, int dtype, const float* bias, const float* lower, const float* gain, float eps,
                                        float* state, long slot_stride, const int* slot, void* out, int n_req, int H, int D, int V,
                                        hipStream_t stream) {
  GIBBS_REQUIRE(raw && bias && lower && gain && state && slot && out && n_req > 0 && H > 0 && H <= 65535 && ld >= (long)H * (2 * D + V),
                "gated_outer_step: bad operands rows=%d heads=%d", n_req, H);
  GIBBS_REQUIRE(gibbs_gated_outer_step_takes(D, V) && slot_stride >= (long)H * D * V, "gated_outer_step: states of %d x %d", D, V);
  const bool vec = V % 4 == 0 && slot_stride % 4 == 0 && ((uintptr_t)state % 16) == 0;

  int lanes = 1;
  while (lanes < (vec ? V / 4 : V)) lanes *= 2;
  const size_t lds = (size_t)(STEP_THREADS / lanes) * V * sizeof(float);
  const dim3 grid(n_req, H);
#define GATED_STEP(T, VEC) \
  gated_outer_step_kernel<T, VEC><<<grid, STEP_THREADS, lds, stream>>>((const T*)raw, ld, bias, lower, gain, eps, state, slot_stride, slot, (T*)out, H, D, V, lanes)
  if (dtype == GIBBS_F32) { if (vec) GATED_STEP(float, 4); else GATED_STEP(float, 1); }
  else if (dtype == GIBBS_BF16) { if (vec) GATED_STEP(bf16, 4); else GATED_STEP(bf16, 1); }
  else return gibbs_fail("gated_outer_step: unknown dtype %d", dtype);
#undef GATED_STEP
  GIBBS_LAUNCH_STATUS("gated_outer_step");
}
