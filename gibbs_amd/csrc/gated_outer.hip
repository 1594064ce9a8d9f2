// The gated outer-product recurrence around its walk (recurrent.hip): per head, with a gate f per channel,
//
//   q = silu(a),  f = l + (1 - l) sigmoid(z + b),  k = 1 - f = (1 - l) sigmoid(-(z + b))        (a, z, v: projected rows)
//   S = diag(f) S + k v',   y = S' q                                                          (S [D, V] from zero)
//   out = y / sqrt(mean(y^2) + eps) * gain
//
//   prep   q, f, k, v of a step's rows as float32, for the walk over ragged portions
//   step   everything above in one kernel for a step of one token per request: a workgroup owns one head of one request and
//          streams its state once, in whole rows
//   chunks the rule for long portions, regrouped into products on the matrix cores (float32 operands): see below
//
// Everything behind the projections is float32, and so is the state.
#include "common.h"
#include "lane8.h"
#include <algorithm>

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

// ------------------------------------------------------------------------------------------------ the rule in chunks
// A request's rows in chunks of 64 tokens, a chunk in segments of 16.  With b_t the sum of log f (per channel) over the tokens
// of t's segment up to t, B_J a segment's whole sum, and S_0 the state in front of the chunk:
//   y_t = sum_(s <= t) A_ts v_s + (q_t e^(sum up to t))' S_0      A_ts = sum_i q_ti k_si e^(sum of log f_i over s < . <= t)
//   S_64 = diag(e^(all)) S_0 + U,   U = sum_s (k_s e^(sum behind s)) v_s'
// Three kernels: U and the chunk's decay per (chunk, head); the states in front of the chunks, per element in order; and per
// (chunk, head) the scores A, both terms of y, and the head's norm.  The products run on the matrix cores with float32
// operands.  Every exponent is a sum over few segments, and the two factors that a score's decay is split into never grow:
//   s in an earlier segment than t   e^(b_t) and e^(B_J - b_s + segments between)
//   s in the first half of t's segment, t in the second   both about the border between the halves
//   both in the same half (8 tokens)   about the half's middle: a factor may grow over at most four tokens, and log2 f is kept
//   above -28 here (f at least 3.7e-9: what is left of the state then is below the rounding of what is added), 2^112
// so nothing overflows that is used.  Logarithms are to base 2: the vector unit's own exponential, logarithm and reciprocal
// (one unit in the last place) are what the many factors cost.  The order of additions differs from the walk's: results
// agree to rounding.
constexpr int CHUNK = 64, SEG = 16, CT = 512, CWAVES = CT / WAVE, MAX_VT = 2;
constexpr float LOG2E = 1.44269504088896340736f;
__device__ __forceinline__ float exp2_of(float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ float rcp_of(float x) { return __builtin_amdgcn_rcpf(x); }
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float floatx4;
struct ChunkedArgs {
  const void* raw;            // [rows, ld]: [a | z | v]
  long ld;
  const float* bias; const float* lower; const float* gain;
  float eps;
  float* u;                   // [places, H, D, V]: U, then the state in front of each chunk
  float* decay;               // [places, H, D]
  float* state; long slot_stride;
  const int* cu; const int* slot;
  void* out;                  // [rows, H * V]
  int n_req, H, D, V;
  int d_shift, v_shift;       // log2 of the next powers of two of D's multiple of 16 and of V / 8
  int v8;                     // values are loaded 8 at a time
};
// the request and the chunk of it that place `p` stands for (false: none)
__device__ __forceinline__ bool chunk_of(const ChunkedArgs& a, int p, int* t0, int* rows) {
  for (int r = 0; r < a.n_req; ++r) {
    const int first = a.cu[r], len = a.cu[r + 1] - first, n = (len + CHUNK - 1) / CHUNK;
    if (p < n) {
      *t0 = first + p * CHUNK;
      *rows = min(CHUNK, len - p * CHUNK);
      return true;
    }
    p -= n;
  }
  return false;
}
// q (optional), k and b of the chunk's tokens into LDS rows of `lq` floats (channels from D to Dp and tokens beyond the end:
// q = k = 0, no decay), and the segments' sums tot [4][lq].
template <typename T, bool Q>
__device__ __forceinline__ void chunk_gates(const ChunkedArgs& a, int h, int t0, int rows, int Dp, int lq, float* sq, float* sk, float* sb, float* tot) {
  const int C = a.H * a.D, span = 1 << a.d_shift;
  for (int idx = threadIdx.x; idx < (CHUNK / SEG) * span; idx += CT) {
    const int seg = idx >> a.d_shift, i = idx & (span - 1);
    if (i >= Dp) continue;
    const bool live = i < a.D;
    const int c = h * a.D + (live ? i : 0);
    const T* at = (const T*)a.raw + (size_t)t0 * a.ld + c;
    T z[SEG], q[SEG];
#pragma unroll
    for (int t = 0; t < SEG; ++t) {      // (rows beyond the end: the last one again, masked below)
      const T* row = at + (size_t)min(seg * SEG + t, rows - 1) * a.ld;
      z[t] = row[C];
      if constexpr (Q) q[t] = row[0];
    }
    const float bias = a.bias[c], l = a.lower[c];
    float run = 0.f;
#pragma unroll
    for (int t = 0; t < SEG; ++t) {
      const int row = seg * SEG + t;
      const bool in = live && row < rows;
      const float x = to_float(z[t]) + bias;
      const float e = exp2_of(-fabsf(x) * LOG2E), inv = rcp_of(1.0f + e), ei = e * inv;
      const float f = fmaf(1.0f - l, x >= 0.f ? inv : ei, l), k = (1.0f - l) * (x >= 0.f ? ei : inv);
      run += in ? __builtin_amdgcn_logf(fmaxf(f, 3.7252903e-9f)) : 0.f;
      sk[row * lq + i] = in ? k : 0.f;
      sb[row * lq + i] = run;
      if constexpr (Q) {
        const float y = to_float(q[t]);
        sq[row * lq + i] = in ? y * rcp_of(1.0f + exp2_of(-y * LOG2E)) : 0.f;
      }
    }
    tot[seg * lq + i] = run;
  }
}
__device__ __forceinline__ void load_eight(const bf16* p, float* f) { unpack8(*(const uint4*)p, f); }
__device__ __forceinline__ void load_eight(const float* p, float* f) {
  const float4 a = *(const float4*)p, b = *(const float4*)(p + 4);
  f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w; f[4] = b.x; f[5] = b.y; f[6] = b.z; f[7] = b.w;
}
template <typename T>
__device__ __forceinline__ void chunk_values(const ChunkedArgs& a, int h, int t0, int rows, int Vp, int lv, float* sv) {
  const T* at = (const T*)a.raw + (size_t)t0 * a.ld + 2 * a.H * a.D + h * a.V;
  if (a.v8) {
    const int span = 1 << a.v_shift;
#pragma unroll 2
    for (int idx = threadIdx.x; idx < CHUNK * span; idx += CT) {
      const int t = idx >> a.v_shift, j = (idx & (span - 1)) * 8;
      if (j >= Vp) continue;
      float f[8] = {};
      if (t < rows && j < a.V) load_eight(at + (size_t)t * a.ld + j, f);
      *(float4*)(sv + t * lv + j) = make_float4(f[0], f[1], f[2], f[3]);
      *(float4*)(sv + t * lv + j + 4) = make_float4(f[4], f[5], f[6], f[7]);
    }
    return;
  }
  for (int idx = threadIdx.x; idx < CHUNK * Vp; idx += CT) {
    const int t = idx / Vp, j = idx % Vp;
    sv[t * lv + j] = (t < rows && j < a.V) ? to_float(at[(size_t)t * a.ld + j]) : 0.f;
  }
}

template <typename T>
__global__ __launch_bounds__(CT) void gated_outer_chunk_state_kernel(ChunkedArgs a) {
  extern __shared__ float lds[];
  const int Dp = (a.D + 15) / 16 * 16, Vp = (a.V + 15) / 16 * 16, lq = Dp + 4, lv = Vp + 4;
  float* sk = lds;                        // [CHUNK][lq]
  float* sb = sk + CHUNK * lq;            // [CHUNK][lq]
  float* sv = sb + CHUNK * lq;            // [CHUNK][lv]
  float* tot = sv + CHUNK * lv;           // [4][lq]
  int t0, rows;
  if (!chunk_of(a, blockIdx.x, &t0, &rows)) return;
  const int h = blockIdx.y;
  chunk_gates<T, false>(a, h, t0, rows, Dp, lq, nullptr, sk, sb, tot);
  chunk_values<T>(a, h, t0, rows, Vp, lv, sv);
  __syncthreads();
  // k_s times the decay from behind s to the chunk's end
  for (int idx = threadIdx.x; idx < (CHUNK / SEG) << a.d_shift; idx += CT) {
    const int seg = idx >> a.d_shift, i = idx & ((1 << a.d_shift) - 1);
    if (i >= Dp) continue;
    float rest = tot[seg * lq + i];
    for (int m = seg + 1; m < CHUNK / SEG; ++m) rest += tot[m * lq + i];
#pragma unroll
    for (int t = seg * SEG; t < seg * SEG + SEG; ++t) sk[t * lq + i] *= exp2_of(rest - sb[t * lq + i]);
  }
  if (threadIdx.x < a.D) {
    const int i = threadIdx.x;
    a.decay[((size_t)blockIdx.x * a.H + h) * a.D + i] = exp2_of(tot[i] + tot[lq + i] + tot[2 * lq + i] + tot[3 * lq + i]);
  }
  __syncthreads();
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE, lr = lane % 16, g = lane / 16;
  float* u = a.u + ((size_t)blockIdx.x * a.H + h) * a.D * a.V;
  for (int n0 = wave * 16; n0 < Vp; n0 += CWAVES * 16) {
    for (int m0 = 0; m0 < Dp; m0 += 64) {           // four channel tiles at a time
      floatx4 acc[4] = {};
      for (int s0 = 0; s0 < CHUNK; s0 += 16) {
        float vb[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) vb[j] = sv[(s0 + g * 4 + j) * lv + n0 + lr];
#pragma unroll
        for (int m = 0; m < 4; ++m) {
          if (m0 + m * 16 >= Dp) break;
#pragma unroll
          for (int j = 0; j < 4; ++j)
            acc[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(sk[(s0 + g * 4 + j) * lq + m0 + m * 16 + lr], vb[j], acc[m], 0, 0, 0);
        }
      }
      const int col = n0 + lr;
#pragma unroll
      for (int m = 0; m < 4; ++m)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int row = m0 + m * 16 + g * 4 + i;
          if (row < a.D && col < a.V) u[(size_t)row * a.V + col] = acc[m][i];
        }
    }
  }
}

// Per element of a request's state, over its chunks in order: u becomes the state in front of each chunk, the slot's state the
// one behind the last.  Four chunks' values are asked for at a time.
__global__ __launch_bounds__(256) void gated_outer_chunk_scan_kernel(ChunkedArgs a) {
  const int r = blockIdx.y;
  const size_t per = (size_t)a.H * a.D * a.V, e = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (e >= per) return;
  int place = 0;
  for (int q = 0; q < r; ++q) place += (a.cu[q + 1] - a.cu[q] + CHUNK - 1) / CHUNK;
  const int n = (a.cu[r + 1] - a.cu[r] + CHUNK - 1) / CHUNK;
  const size_t channel = e / a.V;      // h D + i
  float* state = a.state + (size_t)a.slot[r] * a.slot_stride + e;
  float* u = a.u + (size_t)place * per + e;
  const float* dec = a.decay + (size_t)place * a.H * a.D + channel;
  float S = *state;
  constexpr int AHEAD = 8;
  for (int c0 = 0; c0 < n; c0 += AHEAD) {
    float own[AHEAD], d[AHEAD];
#pragma unroll
    for (int k = 0; k < AHEAD; ++k) {
      const int c = min(c0 + k, n - 1);
      own[k] = u[(size_t)c * per];
      d[k] = dec[(size_t)c * a.H * a.D];
    }
#pragma unroll
    for (int k = 0; k < AHEAD; ++k)
      if (c0 + k < n) {
        u[(size_t)(c0 + k) * per] = S;
        S = fmaf(d[k], S, own[k]);
      }
  }
  *state = S;
}

enum { PASS_EARLIER = 0, PASS_HALF = 1, PASS_BORDER = 2 };
template <typename T>
__global__ __launch_bounds__(CT) void gated_outer_chunk_out_kernel(ChunkedArgs a) {
  extern __shared__ float lds[];
  const int Dp = (a.D + 15) / 16 * 16, Vp = (a.V + 15) / 16 * 16, lq = Dp + 4, lv = Vp + 4;
  constexpr int la = CHUNK + 4;
  float* sq = lds;                        // [CHUNK][lq]
  float* sk = sq + CHUNK * lq;            // [CHUNK][lq]
  float* sb = sk + CHUNK * lq;            // [CHUNK][lq]
  float* sv = sb + CHUNK * lq;            // [CHUNK][lv]
  float* sA = sv + CHUNK * lv;            // [CHUNK][la]
  float* tot = sA + CHUNK * la;           // [4][lq]
  float* red = tot + 4 * lq;              // [CWAVES][CHUNK]
  int t0, rows;
  if (!chunk_of(a, blockIdx.x, &t0, &rows)) return;
  const int h = blockIdx.y;
  chunk_gates<T, true>(a, h, t0, rows, Dp, lq, sq, sk, sb, tot);
  chunk_values<T>(a, h, t0, rows, Vp, lv, sv);
  __syncthreads();
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE, lr = lane % 16, g = lane / 16;
  const int segs = (rows + SEG - 1) / SEG;
  // the scores' tiles: six of pairs of segments, and two passes for each segment with itself
  for (int p = wave; p < 14; p += CWAVES) {
    const int kind = p < 6 ? PASS_EARLIER : (p < 10 ? PASS_HALF : PASS_BORDER);
    const int I = kind == PASS_EARLIER ? (p < 1 ? 1 : (p < 3 ? 2 : 3)) : (p - 6) % 4;
    const int J = kind == PASS_EARLIER ? (p < 1 ? 0 : (p < 3 ? p - 1 : p - 3)) : I;
    if (I >= segs) continue;
    const float* qr = sq + (I * SEG + lr) * lq;
    const float* bq = sb + (I * SEG + lr) * lq;
    const float* kr = sk + (J * SEG + lr) * lq;
    const float* bk = sb + (J * SEG + lr) * lq;
    const float* ref = kind == PASS_EARLIER ? tot + J * lq : sb + (I * SEG + (kind == PASS_BORDER ? 7 : (lr < 8 ? 3 : 11))) * lq;
    floatx4 acc = {};
    for (int c0 = 0; c0 < Dp; c0 += 16) {
      const int ch = c0 + g * 4;
      const float4 q4 = *(const float4*)(qr + ch), x4 = *(const float4*)(bq + ch), k4 = *(const float4*)(kr + ch), y4 = *(const float4*)(bk + ch);
      float4 r4 = *(const float4*)(ref + ch);
      float eq[4] = {x4.x, x4.y, x4.z, x4.w};
      if (kind == PASS_EARLIER) {
        for (int m = J + 1; m < I; ++m) {
          const float4 t4 = *(const float4*)(tot + m * lq + ch);
          r4.x += t4.x; r4.y += t4.y; r4.z += t4.z; r4.w += t4.w;
        }
      } else {
        eq[0] -= r4.x; eq[1] -= r4.y; eq[2] -= r4.z; eq[3] -= r4.w;
      }
      const float qv[4] = {q4.x, q4.y, q4.z, q4.w}, kv[4] = {k4.x, k4.y, k4.z, k4.w};
      const float ek[4] = {r4.x - y4.x, r4.y - y4.y, r4.z - y4.z, r4.w - y4.w};
#pragma unroll
      for (int j = 0; j < 4; ++j) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(qv[j] * exp2_of(eq[j]), kv[j] * exp2_of(ek[j]), acc, 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = g * 4 + i;             // in its segment
      float* dst = sA + (I * SEG + t) * la + J * SEG + lr;
      if (kind == PASS_EARLIER) *dst = acc[i];
      else if (kind == PASS_BORDER) { if (t >= 8 && lr < 8) *dst = acc[i]; }
      else if (!(t >= 8 && lr < 8)) *dst = (t / 8 == lr / 8 && lr <= t) ? acc[i] : 0.f;
    }
  }
  __syncthreads();
  // q_t times the decay from the chunk's start to t
  for (int idx = threadIdx.x; idx < (CHUNK / SEG) << a.d_shift; idx += CT) {
    const int seg = idx >> a.d_shift, i = idx & ((1 << a.d_shift) - 1);
    if (i >= Dp) continue;
    float before = 0.f;
    for (int m = 0; m < seg; ++m) before += tot[m * lq + i];
#pragma unroll
    for (int t = seg * SEG; t < seg * SEG + SEG; ++t) sq[t * lq + i] *= exp2_of(before + sb[t * lq + i]);
  }
  __syncthreads();
  const float* s0 = a.u + ((size_t)blockIdx.x * a.H + h) * a.D * a.V;
  floatx4 acc[MAX_VT][CHUNK / SEG] = {};
#pragma unroll
  for (int v = 0; v < MAX_VT; ++v) {
    const int n0 = (wave + v * CWAVES) * 16, col = n0 + lr;
    if (n0 >= Vp) break;
    for (int c = 0; c < segs * SEG; c += 16) {
      float vb[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) vb[j] = sv[(c + g * 4 + j) * lv + col];
#pragma unroll
      for (int I = 0; I < CHUNK / SEG; ++I) {
        if (I < c / SEG || I >= segs) continue;
        const float4 a4 = *(const float4*)(sA + (I * SEG + lr) * la + c + g * 4);
        const float av[4] = {a4.x, a4.y, a4.z, a4.w};
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[v][I] = __builtin_amdgcn_mfma_f32_16x16x4f32(av[j], vb[j], acc[v][I], 0, 0, 0);
      }
    }
#pragma unroll 2
    for (int c = 0; c < Dp; c += 16) {
      float sb4[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int i = c + g * 4 + j;
        sb4[j] = (i < a.D && col < a.V) ? s0[(size_t)i * a.V + col] : 0.f;
      }
#pragma unroll
      for (int I = 0; I < CHUNK / SEG; ++I) {
        const float4 q4 = *(const float4*)(sq + (I * SEG + lr) * lq + c + g * 4);
        const float qv[4] = {q4.x, q4.y, q4.z, q4.w};
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[v][I] = __builtin_amdgcn_mfma_f32_16x16x4f32(qv[j], sb4[j], acc[v][I], 0, 0, 0);
      }
    }
  }
  // the heads' norm over V: a row's squares over the 16 columns of a tile, then over the waves (in order)
#pragma unroll
  for (int I = 0; I < CHUNK / SEG; ++I)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      float ss = 0.f;
#pragma unroll
      for (int v = 0; v < MAX_VT; ++v) ss = fmaf(acc[v][I][i], acc[v][I][i], ss);
      ss = group_sum<16>(ss);
      if (lr == 0) red[wave * CHUNK + I * SEG + g * 4 + i] = ss;
    }
  __syncthreads();
  if (threadIdx.x < CHUNK) {
    float total = 0.f;
#pragma unroll
    for (int w = 0; w < CWAVES; ++w) total += red[w * CHUNK + threadIdx.x];
    red[threadIdx.x] = 1.0f / sqrtf(total / (float)a.V + a.eps);
  }
  __syncthreads();
#pragma unroll
  for (int v = 0; v < MAX_VT; ++v) {
    const int col = (wave + v * CWAVES) * 16 + lr;
    if (col >= a.V) break;
    const float gain = a.gain[col];
    T* out = (T*)a.out + ((size_t)t0 * a.H + h) * a.V + col;
#pragma unroll
    for (int I = 0; I < CHUNK / SEG; ++I)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = I * SEG + g * 4 + i;
        if (t < rows) out[(size_t)t * a.H * a.V] = from_float<T>(acc[v][I][i] * red[t] * gain);
      }
  }
}
size_t chunk_state_lds(int D, int V) {
  const int lq = (D + 15) / 16 * 16 + 4, lv = (V + 15) / 16 * 16 + 4;
  return (size_t)(2 * CHUNK * lq + CHUNK * lv + 4 * lq) * sizeof(float);
}
size_t chunk_out_lds(int D, int V) {
  const int lq = (D + 15) / 16 * 16 + 4, lv = (V + 15) / 16 * 16 + 4;
  return (size_t)(3 * CHUNK * lq + CHUNK * lv + CHUNK * (CHUNK + 4) + 4 * lq + CWAVES * CHUNK) * sizeof(float);
}
constexpr size_t LDS_BYTES = 160 * 1024;
template <typename T>
int launch_chunks(const ChunkedArgs& a, int places, hipStream_t stream) {
  const size_t lds1 = chunk_state_lds(a.D, a.V), lds2 = chunk_out_lds(a.D, a.V);
  static bool raised = false;      // (one flag per instantiation)
  if (!raised) {
    if (hipFuncSetAttribute((const void*)gated_outer_chunk_state_kernel<T>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)LDS_BYTES) != hipSuccess ||
        hipFuncSetAttribute((const void*)gated_outer_chunk_out_kernel<T>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)LDS_BYTES) != hipSuccess)
      return gibbs_fail("gated_outer_chunks: the kernels' LDS could not be reserved");
    raised = true;
  }
  const dim3 grid(places, a.H);
  gated_outer_chunk_state_kernel<T><<<grid, CT, lds1, stream>>>(a);
  gated_outer_chunk_scan_kernel<<<dim3(ceil_div((long)a.H * a.D * a.V, 256), a.n_req), 256, 0, stream>>>(a);
  gated_outer_chunk_out_kernel<T><<<grid, CT, lds2, stream>>>(a);
  return 0;
}
}  // namespace

// Whether the rule in chunks takes a head's sizes, and the floats of workspace that `rows` rows of `n_req` requests need.
GIBBS_EXPORT int gibbs_gated_outer_chunks_take(int D, int V) {
  return D > 0 && V > 0 && V <= MAX_VT * CWAVES * 16 && D <= CT && chunk_out_lds(D, V) <= LDS_BYTES;
}
GIBBS_EXPORT long gibbs_gated_outer_chunks_workspace(int rows, int n_req, int H, int D, int V) {
  return ((long)ceil_div(rows, CHUNK) + n_req) * H * D * ((long)V + 1);
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
  ChunkedArgs a{raw, ld, bias, lower, gain, eps, workspace, workspace + (size_t)places * H * D * V, state, slot_stride, cu, slot, out, n_req, H, D, V, 4, 0, 0};
  while ((1 << a.d_shift) < D) ++a.d_shift;
  while ((1 << a.v_shift) * 8 < V) ++a.v_shift;
  if (V % 16) a.v_shift = std::max(a.v_shift, 1);      // (the zeros up to the next multiple of 16 are written as well)
  a.v8 = V % 8 == 0 && ld % 8 == 0 && (2L * H * D) % 8 == 0 && ((uintptr_t)raw % 16) == 0;
  if (dtype == GIBBS_F32) { if (launch_chunks<float>(a, places, stream)) return 1; }
  else if (dtype == GIBBS_BF16) { if (launch_chunks<bf16>(a, places, stream)) return 1; }
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
