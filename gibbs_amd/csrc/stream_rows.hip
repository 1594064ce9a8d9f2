// Readers of the residual stream for sublayers that are not normed on their way in, and the normed embedding.
//
//   embed_norm    x[n] = table[id] / sqrt(mean(table[id]^2) + eps) * gain
//   stream_rows   out[n] = x[n] in the activation type
//   stream_shift  out[n] = x[n] + (before(n) - x[n]) * mu, before(n) the request's previous row: the row above, or for the
//                 first row that a request brings its state (zeros at a sequence's start); the request's last row
//                 becomes its state
//
// The stream, the mixing and the state are float32.  Four values a thread where rows allow it (16-byte accesses).
#include "common.h"

namespace {
template <int V> struct Vals { float v[V]; };
template <int V> __device__ __forceinline__ Vals<V> load_vals(const float* p) {
  Vals<V> r;
  if constexpr (V == 4) { const float4 t = *(const float4*)p; r.v[0] = t.x; r.v[1] = t.y; r.v[2] = t.z; r.v[3] = t.w; }
  else r.v[0] = *p;
  return r;
}
template <int V> __device__ __forceinline__ Vals<V> load_vals(const bf16* p) {
  Vals<V> r;
  if constexpr (V == 4) {
    const uint2 t = *(const uint2*)p;
    r.v[0] = __uint_as_float(t.x << 16); r.v[1] = __uint_as_float(t.x & 0xffff0000u);
    r.v[2] = __uint_as_float(t.y << 16); r.v[3] = __uint_as_float(t.y & 0xffff0000u);
  } else {
    r.v[0] = (float)*p;
  }
  return r;
}
template <int V> __device__ __forceinline__ void store_vals(float* p, const Vals<V>& r) {
  if constexpr (V == 4) *(float4*)p = make_float4(r.v[0], r.v[1], r.v[2], r.v[3]);
  else *p = r.v[0];
}
template <int V> __device__ __forceinline__ void store_vals(bf16* p, const Vals<V>& r) {
  if constexpr (V == 4) {
    union { bf16 h[4]; uint2 u; } o;
#pragma unroll
    for (int i = 0; i < 4; ++i) o.h[i] = (bf16)r.v[i];
    *(uint2*)p = o.u;
  } else {
    *p = (bf16)r.v[0];
  }
}

template <typename T, int V>
__global__ void embed_norm_kernel(const T* __restrict__ table, const int* __restrict__ ids, float* __restrict__ x, const float* __restrict__ gain,
                                  float eps, int W, int vocab) {
  __shared__ float scratch[16];
  const int n = blockIdx.x;
  int id = ids[n];
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);      // (never read outside the table)
  const T* row = table + (size_t)id * W;
  float ss = 0.f;
  for (int i = threadIdx.x * V; i < W; i += blockDim.x * V) {
    const Vals<V> r = load_vals<V>(row + i);
#pragma unroll
    for (int e = 0; e < V; ++e) ss = fmaf(r.v[e], r.v[e], ss);
  }
  const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / (float)W + eps);
  for (int i = threadIdx.x * V; i < W; i += blockDim.x * V) {
    Vals<V> r = load_vals<V>(row + i);
#pragma unroll
    for (int e = 0; e < V; ++e) r.v[e] = r.v[e] * inv * (gain ? gain[i + e] : 1.f);
    store_vals<V>(x + (size_t)n * W + i, r);
  }
}

template <typename T, int V>
__global__ void stream_rows_kernel(const float* __restrict__ x, T* __restrict__ out, long count) {
  const long i = ((long)blockIdx.x * blockDim.x + threadIdx.x) * V;
  if (i < count) store_vals<V>(out + i, load_vals<V>(x + i));
}

// A thread owns V channels of one row.  The first row's thread is the only one that touches the request's state in its
// channels: it reads the old row and then leaves the request's last row there (the stream itself is not written here).
template <typename T, int V>
__global__ __launch_bounds__(256) void stream_shift_kernel(const float* __restrict__ x, const float* __restrict__ mu, float* __restrict__ state,
                                                           long slot_stride, const int* __restrict__ row_req, const int* __restrict__ cu,
                                                           const int* __restrict__ slot, T* __restrict__ out, int n_rows, int W) {
  const int per_row = W / V;
  const long item = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (item >= (long)n_rows * per_row) return;
  const int n = (int)(item / per_row), c = (int)(item % per_row) * V;
  const int r = row_req[n], first = cu[r];
  const Vals<V> cur = load_vals<V>(x + (size_t)n * W + c), m = load_vals<V>(mu + c);
  Vals<V> before;
  if (n > first) {
    before = load_vals<V>(x + (size_t)(n - 1) * W + c);
  } else {
    float* st = state + (size_t)slot[r] * slot_stride + c;
    before = load_vals<V>(st);
    store_vals<V>(st, load_vals<V>(x + (size_t)(cu[r + 1] - 1) * W + c));
  }
  Vals<V> o;
#pragma unroll
  for (int e = 0; e < V; ++e) o.v[e] = fmaf(before.v[e] - cur.v[e], m.v[e], cur.v[e]);
  store_vals<V>(out + (size_t)n * W + c, o);
}
}  // namespace

#define STREAM_BY_DTYPE(dtype, what, call_f32, call_bf16)  \
  do {                                                     \
    if ((dtype) == GIBBS_F32) { call_f32; }                \
    else if ((dtype) == GIBBS_BF16) { call_bf16; }         \
    else return gibbs_fail(what ": unknown dtype %d", (dtype)); \
  } while (0)

GIBBS_EXPORT int gibbs_embed_norm(const void* table, int dtype, const int* ids, float* x, const float* gain, float eps, int n, int hidden,
                                  int vocab, hipStream_t stream) {
  GIBBS_REQUIRE(table && ids && x && n >= 0 && hidden > 0 && vocab > 0, "embed_norm: bad sizes n=%d hidden=%d", n, hidden);
  if (n == 0) return 0;
  const bool vec = hidden % 4 == 0 && ((uintptr_t)table % 16) == 0 && ((uintptr_t)x % 16) == 0;
  const int threads = hidden >= 2048 ? 512 : (hidden >= 512 ? 256 : 64);
#define EMBED_NORM(T, V) embed_norm_kernel<T, V><<<n, threads, 0, stream>>>((const T*)table, ids, x, gain, eps, hidden, vocab)
  if (vec) STREAM_BY_DTYPE(dtype, "embed_norm", EMBED_NORM(float, 4), EMBED_NORM(bf16, 4));
  else STREAM_BY_DTYPE(dtype, "embed_norm", EMBED_NORM(float, 1), EMBED_NORM(bf16, 1));
#undef EMBED_NORM
  GIBBS_LAUNCH_STATUS("embed_norm");
}

GIBBS_EXPORT int gibbs_stream_rows(const float* x, void* out, int dtype, long count, hipStream_t stream) {
  GIBBS_REQUIRE(x && out && count > 0, "stream_rows: bad operands");
  const bool vec = count % 4 == 0 && ((uintptr_t)x % 16) == 0 && ((uintptr_t)out % 16) == 0;
#define STREAM_ROWS(T, V) stream_rows_kernel<T, V><<<ceil_div(count / V, 256), 256, 0, stream>>>(x, (T*)out, count)
  if (vec) STREAM_BY_DTYPE(dtype, "stream_rows", STREAM_ROWS(float, 4), STREAM_ROWS(bf16, 4));
  else STREAM_BY_DTYPE(dtype, "stream_rows", STREAM_ROWS(float, 1), STREAM_ROWS(bf16, 1));
#undef STREAM_ROWS
  GIBBS_LAUNCH_STATUS("stream_rows");
}

GIBBS_EXPORT int gibbs_stream_shift(const float* x, const float* mu, float* state, long slot_stride, const int* row_req, const int* cu,
                                    const int* slot, void* out, int dtype, int n_rows, int hidden, hipStream_t stream) {
  GIBBS_REQUIRE(x && mu && state && row_req && cu && slot && out && n_rows > 0 && hidden > 0 && slot_stride >= hidden,
                "stream_shift: bad operands rows=%d hidden=%d", n_rows, hidden);
  const bool vec = hidden % 4 == 0 && slot_stride % 4 == 0 && ((uintptr_t)x % 16) == 0 && ((uintptr_t)mu % 16) == 0 && ((uintptr_t)state % 16) == 0 &&
                   ((uintptr_t)out % 16) == 0;
#define STREAM_SHIFT(T, V) \
  stream_shift_kernel<T, V><<<ceil_div((long)n_rows * (hidden / V), 256), 256, 0, stream>>>(x, mu, state, slot_stride, row_req, cu, slot, (T*)out, n_rows, hidden)
  if (vec) STREAM_BY_DTYPE(dtype, "stream_shift", STREAM_SHIFT(float, 4), STREAM_SHIFT(bf16, 4));
  else STREAM_BY_DTYPE(dtype, "stream_shift", STREAM_SHIFT(float, 1), STREAM_SHIFT(bf16, 1));
#undef STREAM_SHIFT
  GIBBS_LAUNCH_STATUS("stream_shift");
}
