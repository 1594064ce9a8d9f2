// Gated activation of a feed-forward:  out[n, f] = act(gu[n, f]) * gu[n, F + f], where the
// gate and up projections were computed as one product against [W_gate; W_up].
// The activation (activation.h: silu, two gelus, relu) is computed in float32.
#include "activation.h"
#include "lane8.h"

template <typename T>
__global__ void glu_kernel(const T* __restrict__ gu, T* __restrict__ out, int F, int act) {
  const int n = blockIdx.x;
  const int f = blockIdx.y * blockDim.x + threadIdx.x;
  if (f >= F) return;
  const float g = to_float(gu[(size_t)n * 2 * F + f]);
  const float u = to_float(gu[(size_t)n * 2 * F + F + f]);
  out[(size_t)n * F + f] = from_float<T>(activate(g, act) * u);
}

// 8 elements (16 bytes of bfloat16) per thread: the pass is bound by memory traffic.
__global__ void glu_bf16x8_kernel(const bf16* __restrict__ gu, bf16* __restrict__ out, int F, int act) {
  const int n = blockIdx.x;
  const int f = (blockIdx.y * blockDim.x + threadIdx.x) * 8;
  if (f >= F) return;
  const uint4 gr = *(const uint4*)(gu + (size_t)n * 2 * F + f);
  const uint4 ur = *(const uint4*)(gu + (size_t)n * 2 * F + F + f);
  const uint32_t gw[4] = {gr.x, gr.y, gr.z, gr.w}, uw[4] = {ur.x, ur.y, ur.z, ur.w};
  uint32_t ow[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const float g0 = __uint_as_float(gw[i] << 16), g1 = __uint_as_float(gw[i] & 0xffff0000u);
    const float u0 = __uint_as_float(uw[i] << 16), u1 = __uint_as_float(uw[i] & 0xffff0000u);
    const bf16 a0 = (bf16)(activate(g0, act) * u0);
    const bf16 a1 = (bf16)(activate(g1, act) * u1);
    ow[i] = (uint32_t)__builtin_bit_cast(unsigned short, a0) | ((uint32_t)__builtin_bit_cast(unsigned short, a1) << 16);
  }
  *(uint4*)(out + (size_t)n * F + f) = make_uint4(ow[0], ow[1], ow[2], ow[3]);
}

// The clamped variant (activation.h: the gate capped from above, the up value clipped, gate * sigmoid(alpha * gate) * (1 + up)).
template <typename T>
__global__ void glu_clamped_kernel(const T* __restrict__ gu, T* __restrict__ out, int F, float alpha, float limit) {
  const int n = blockIdx.x;
  const int f = blockIdx.y * blockDim.x + threadIdx.x;
  if (f >= F) return;
  out[(size_t)n * F + f] = from_float<T>(clamped_swish_product(to_float(gu[(size_t)n * 2 * F + f]), to_float(gu[(size_t)n * 2 * F + F + f]), alpha, limit));
}

// 8 elements per thread, as glu_bf16x8_kernel.
__global__ void glu_clamped_bf16x8_kernel(const bf16* __restrict__ gu, bf16* __restrict__ out, int F, float alpha, float limit) {
  const int n = blockIdx.x;
  const int f = (blockIdx.y * blockDim.x + threadIdx.x) * 8;
  if (f >= F) return;
  const uint4 gr = *(const uint4*)(gu + (size_t)n * 2 * F + f);
  const uint4 ur = *(const uint4*)(gu + (size_t)n * 2 * F + F + f);
  const uint32_t gw[4] = {gr.x, gr.y, gr.z, gr.w}, uw[4] = {ur.x, ur.y, ur.z, ur.w};
  uint32_t ow[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const float g0 = __uint_as_float(gw[i] << 16), g1 = __uint_as_float(gw[i] & 0xffff0000u);
    const float u0 = __uint_as_float(uw[i] << 16), u1 = __uint_as_float(uw[i] & 0xffff0000u);
    const bf16 a0 = (bf16)clamped_swish_product(g0, u0, alpha, limit);
    const bf16 a1 = (bf16)clamped_swish_product(g1, u1, alpha, limit);
    ow[i] = (uint32_t)__builtin_bit_cast(unsigned short, a0) | ((uint32_t)__builtin_bit_cast(unsigned short, a1) << 16);
  }
  *(uint4*)(out + (size_t)n * F + f) = make_uint4(ow[0], ow[1], ow[2], ow[3]);
}

GIBBS_EXPORT int gibbs_glu_clamped(const void* gu, void* out, int dtype, int n, int F, float alpha, float limit, hipStream_t stream) {
  GIBBS_REQUIRE(n >= 0 && F > 0 && F <= 65535 * 256, "glu: bad sizes n=%d F=%d", n, F);
  if (n == 0) return 0;
  dim3 grid(n, ceil_div(F, 256));
  if (dtype == GIBBS_F32)
    glu_clamped_kernel<float><<<grid, 256, 0, stream>>>((const float*)gu, (float*)out, F, alpha, limit);
  else if (dtype == GIBBS_BF16 && F % 8 == 0 && ((uintptr_t)gu % 16) == 0 && ((uintptr_t)out % 16) == 0)
    glu_clamped_bf16x8_kernel<<<dim3(n, ceil_div(F, 8 * 256)), 256, 0, stream>>>((const bf16*)gu, (bf16*)out, F, alpha, limit);
  else if (dtype == GIBBS_BF16)
    glu_clamped_kernel<bf16><<<grid, 256, 0, stream>>>((const bf16*)gu, (bf16*)out, F, alpha, limit);
  else
    return gibbs_fail("glu: unknown dtype %d", dtype);
  GIBBS_LAUNCH_STATUS("glu");
}

GIBBS_EXPORT int gibbs_glu(const void* gu, void* out, int dtype, int n, int F, int act, hipStream_t stream) {
  GIBBS_REQUIRE(n >= 0 && F > 0, "glu: bad sizes n=%d F=%d", n, F);
  GIBBS_REQUIRE(act >= 0 && act < ACT_COUNT, "glu: unknown activation %d", act);
  GIBBS_REQUIRE(F <= 65535 * 256, "glu: width %d too large", F);
  if (n == 0) return 0;
  dim3 grid(n, ceil_div(F, 256));
  if (dtype == GIBBS_F32)
    glu_kernel<float><<<grid, 256, 0, stream>>>((const float*)gu, (float*)out, F, act);
  else if (dtype == GIBBS_BF16 && F % 8 == 0 && ((uintptr_t)gu % 16) == 0 && ((uintptr_t)out % 16) == 0)
    glu_bf16x8_kernel<<<dim3(n, ceil_div(F, 8 * 256)), 256, 0, stream>>>((const bf16*)gu, (bf16*)out, F, act);
  else if (dtype == GIBBS_BF16)
    glu_kernel<bf16><<<grid, 256, 0, stream>>>((const bf16*)gu, (bf16*)out, F, act);
  else
    return gibbs_fail("glu: unknown dtype %d", dtype);
  GIBBS_LAUNCH_STATUS("glu");
}

// out[n, c] = act(z[n, c]) (* table[ids[n]][c]), c < F; columns from F to ld_out are zeros.  float32 arithmetic.
namespace {
__device__ __forceinline__ void act_load8(const bf16* p, float* f) { unpack8(*(const uint4*)p, f); }
__device__ __forceinline__ void act_load8(const float* p, float* f) {
  const float4 a = *(const float4*)p, b = *(const float4*)(p + 4);
  f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w; f[4] = b.x; f[5] = b.y; f[6] = b.z; f[7] = b.w;
}
__device__ __forceinline__ void act_store8(bf16* p, const float* f) { *(uint4*)p = pack8(f); }
__device__ __forceinline__ void act_store8(float* p, const float* f) {
  *(float4*)p = make_float4(f[0], f[1], f[2], f[3]);
  *(float4*)(p + 4) = make_float4(f[4], f[5], f[6], f[7]);
}
template <typename T, int V>
__global__ void act_rows_kernel(const T* __restrict__ z, T* __restrict__ out, long ld_out, int act, const T* __restrict__ mult, long mult_ld,
                                const int* __restrict__ ids, int vocab, int n_rows, int F) {
  const int per = (int)(ld_out / V);
  const long item = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (item >= (long)n_rows * per) return;
  const int n = (int)(item / per), c = (int)(item % per) * V;
  const T* m = mult ? mult + (size_t)min(max(ids[n], 0), vocab - 1) * mult_ld + c : nullptr;      // (never read outside the table)
  float f[V];
  if constexpr (V == 8) {
    float x[8], y[8];
    act_load8(z + (size_t)n * F + c, x);
    if (m) act_load8(m, y);
#pragma unroll
    for (int i = 0; i < 8; ++i) f[i] = activate(x[i], act) * (m ? y[i] : 1.0f);
    act_store8(out + (size_t)n * ld_out + c, f);
  } else {
    f[0] = c < F ? activate(to_float(z[(size_t)n * F + c]), act) * (m ? to_float(m[0]) : 1.0f) : 0.f;
    out[(size_t)n * ld_out + c] = from_float<T>(f[0]);
  }
}
}  // namespace
GIBBS_EXPORT int gibbs_act_rows(const void* z, void* out, long ld_out, int dtype, int act, const void* mult, long mult_ld, const int* ids, int vocab,
                                int n_rows, int F, hipStream_t stream) {
  GIBBS_REQUIRE(z && out && n_rows > 0 && F > 0 && ld_out >= F, "act_rows: bad operands rows=%d width=%d", n_rows, F);
  GIBBS_REQUIRE((act >= 0 && act < ACT_COUNT) || act == ACT_RELU_SQUARED, "act_rows: unknown activation %d", act);
  GIBBS_REQUIRE(!mult || (ids && vocab > 0 && mult_ld >= F), "act_rows: a table without the rows' tokens, or rows of %ld entries", mult_ld);
  const bool x8 = F % 8 == 0 && ld_out == F && ((uintptr_t)z % 16) == 0 && ((uintptr_t)out % 16) == 0 && (!mult || (mult_ld % 8 == 0 && ((uintptr_t)mult % 16) == 0));
  const int grid = ceil_div((long)n_rows * (ld_out / (x8 ? 8 : 1)), 256);
#define ACT_ROWS(T, V) act_rows_kernel<T, V><<<grid, 256, 0, stream>>>((const T*)z, (T*)out, ld_out, act, (const T*)mult, mult_ld, ids, vocab, n_rows, F)
  if (dtype == GIBBS_F32) { if (x8) ACT_ROWS(float, 8); else ACT_ROWS(float, 1); }
  else if (dtype == GIBBS_BF16) { if (x8) ACT_ROWS(bf16, 8); else ACT_ROWS(bf16, 1); }
  else return gibbs_fail("act_rows: unknown dtype %d", dtype);
#undef ACT_ROWS
  GIBBS_LAUNCH_STATUS("act_rows");
}
