// Kernels of an outer-product state that decays channel by channel, S = diag(f) S + k v', read-out S' q normed per head, times a gain
// [vdim]: token by token (`gated_rule_rows_kernel`: gates, state, read-out and norm in one kernel) and in chunks on the matrix cores
// (float32 operands).  Two rules share them; they differ in where q, k and f come from and in what follows the norm:
//
//   RULE_COMPLEMENT  (gated_outer.hip)   rows [a | z | v]: q = silu(a), f = l + (1 - l) sigmoid(z + b), k = 1 - f
//   RULE_LINEAR      (gated_linear.hip)  rows with q, k, v, g and a low-rank z at their offsets: q and k as projected (q times a
//                                        constant), f = sigmoid(z + b)^(1 / tau); the normed read-out times silu(g)
//
// Everything behind the projections is float32, and so is the state.
#pragma once
#include "common.h"
#include "lane8.h"
#include <algorithm>

namespace {
enum { RULE_COMPLEMENT = 0, RULE_LINEAR = 1 };
__device__ __forceinline__ float sigm(float z) { return 1.0f / (1.0f + expf(-z)); }
struct Gate { float f, k; };
__device__ __forceinline__ Gate gate_of(float z, float l) {
  // (both exponentials taken with a negative argument: no overflow, and 1 - f without cancellation)
  const float e = expf(-fabsf(z)), inv = 1.0f / (1.0f + e);
  const float s = z >= 0.f ? inv : e * inv, t = z >= 0.f ? e * inv : inv;
  return Gate{fmaf(1.0f - l, s, l), (1.0f - l) * t};
}
__device__ __forceinline__ void load_eight(const bf16* p, float* f) { unpack8(*(const uint4*)p, f); }
__device__ __forceinline__ void load_eight(const float* p, float* f) {
  const float4 a = *(const float4*)p, b = *(const float4*)(p + 4);
  f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w; f[4] = b.x; f[5] = b.y; f[6] = b.z; f[7] = b.w;
}
struct RuleArgs {
  const void* raw; long ld;     // projected rows: q at off_q, k at off_k (RULE_COMPLEMENT: a and z), v at off_v, g at off_g
  int off_q, off_k, off_v, off_g;
  const float* bias;            // [H D]: added to z
  const float* lower;           // [H D]: RULE_COMPLEMENT
  const float* gain; float eps;
  float q_scale, inv_tau;       // RULE_LINEAR
  // RULE_LINEAR: z of a row.  Rows kernel: from the low-rank columns at off_z (`rank` of them) and w_z [H D, rank] in the rows' type;
  // chunks: z [rows, H D] float32, counted from the first request's first row
  const void* w_z; int off_z, rank, vec_z;
  const float* z;
  float* state; long slot_stride;
  const int* cu; const int* slot;
  void* out;                    // [rows, H V]
  int H, D, V;
};

// A workgroup owns one head of one request and walks the request's rows in order (cu null: one row, row n is request n's); the state is
// streamed in whole rows, and stays in registers over a walk of several rows where it fits.
// Thread (tx, group): columns tx VEC .. and rows group, group + groups, ...; y by groups, added in group order.
constexpr int STEP_THREADS = 512, STEP_ROWS = 8;
template <typename T, int VEC, int RULE>
__global__ __launch_bounds__(STEP_THREADS) void gated_rule_rows_kernel(RuleArgs a, int lanes) {
  extern __shared__ float lds[];
  __shared__ float scratch[16];
  const int r = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, H = a.H, D = a.D, V = a.V;
  float* sq = lds;                     // [D]
  float* sf = sq + D;                  // [D]
  float* sk = sf + D;                  // [D]
  float* part = sk + D;                // [groups][V]
  const int tx = tid % lanes, group = tid / lanes, groups = STEP_THREADS / lanes;
  const int j0 = tx * VEC;
  const bool live = j0 < V;
  float* st = a.state + (size_t)a.slot[r] * a.slot_stride + (size_t)h * D * V + j0;
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
  auto put = [&](int i0) {
#pragma unroll
    for (int u = 0; u < STEP_ROWS; ++u) {
      const int i = i0 + u * groups;
      if (live && i < D) {
        if constexpr (VEC == 4) *(float4*)(st + (size_t)i * V) = make_float4(s[u][0], s[u][1], s[u][2], s[u][3]);
        else st[(size_t)i * V] = s[u][0];
      }
    }
  };
  const bool resident = D <= STEP_ROWS * groups;      // the whole state in registers over the walk
  ask(group);
  const int first = a.cu ? a.cu[r] : r, last = a.cu ? a.cu[r + 1] : r + 1, C = H * D;
  for (int n = first; n < last; ++n) {
    const T* row = (const T*)a.raw + (size_t)n * a.ld;
    for (int i = tid; i < D; i += STEP_THREADS) {
      const int c = h * D + i;
      if constexpr (RULE == RULE_COMPLEMENT) {
        const float x = to_float(row[a.off_q + c]);
        const Gate g = gate_of(to_float(row[a.off_k + c]) + a.bias[c], a.lower[c]);
        sq[i] = x * sigm(x);
        sf[i] = g.f;
        sk[i] = g.k;
      } else {
        float z = 0.f;
        const T* w = (const T*)a.w_z + (size_t)c * a.rank;
        if (a.vec_z) {
          for (int e0 = 0; e0 < a.rank; e0 += 8) {
            float x[8], y[8];
            load_eight(row + a.off_z + e0, x);
            load_eight(w + e0, y);
#pragma unroll
            for (int e = 0; e < 8; ++e) z = fmaf(x[e], y[e], z);
          }
        } else {
          for (int e = 0; e < a.rank; ++e) z = fmaf(to_float(row[a.off_z + e]), to_float(w[e]), z);
        }
        z += a.bias[c];
        sq[i] = to_float(row[a.off_q + c]) * a.q_scale;
        sk[i] = to_float(row[a.off_k + c]);
        sf[i] = expf((fminf(z, 0.f) - log1pf(expf(-fabsf(z)))) * a.inv_tau);
      }
    }
    float v[VEC], y[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      v[e] = live ? to_float(row[a.off_v + h * V + j0 + e]) : 0.f;
      y[e] = 0.f;
    }
    __syncthreads();
    for (int i0 = group; i0 < D; i0 += STEP_ROWS * groups) {
      if (!resident && (i0 != group || n != first)) ask(i0);
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
        }
      }
      if (!resident || n + 1 == last) put(i0);
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
    const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / (float)V + a.eps);
    T* out = (T*)a.out + ((size_t)n * H + h) * V;
    for (int j = tid; j < V; j += STEP_THREADS) {
      float o = part[j] * inv * a.gain[j];
      if constexpr (RULE == RULE_LINEAR) {
        const float g = to_float(row[a.off_g + h * V + j]);
        o *= g * sigm(g);
      }
      out[j] = from_float<T>(o);
    }
    __syncthreads();                   // (the next row writes part and the channels again)
  }
}
inline int rule_lanes(int V, bool vec) {
  int lanes = 1;
  while (lanes < (vec ? V / 4 : V)) lanes *= 2;
  return lanes;
}
inline int rule_rows_take(int D, int V) { return D > 0 && D <= 3072 && V > 0 && (V <= STEP_THREADS || (V % 4 == 0 && V <= 4 * STEP_THREADS)); }
template <typename T, int RULE>
int launch_rule_rows(const RuleArgs& a, int n_req, hipStream_t stream) {
  const bool vec = a.V % 4 == 0 && a.slot_stride % 4 == 0 && ((uintptr_t)a.state % 16) == 0;
  GIBBS_REQUIRE(vec || a.V <= STEP_THREADS, "gated rule: values of %d that are not aligned to 16 bytes", a.V);
  const int lanes = rule_lanes(a.V, vec);
  const size_t lds = ((size_t)3 * a.D + (size_t)(STEP_THREADS / lanes) * a.V) * sizeof(float);
  const dim3 grid(n_req, a.H);
  if (vec) gated_rule_rows_kernel<T, 4, RULE><<<grid, STEP_THREADS, lds, stream>>>(a, lanes);
  else gated_rule_rows_kernel<T, 1, RULE><<<grid, STEP_THREADS, lds, stream>>>(a, lanes);
  return 0;
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
  RuleArgs r;
  float* u;                   // [places, H, D, V]: U, then the state in front of each chunk
  float* decay;               // [places, H, D]
  int n_req;
  int d_shift, v_shift;       // log2 of the next powers of two of D's multiple of 16 and of V / 8
  int v8;                     // values are loaded 8 at a time
};
// the request and the chunk of it that place `p` stands for (false: none)
__device__ __forceinline__ bool chunk_of(const ChunkedArgs& a, int p, int* t0, int* rows) {
  for (int r = 0; r < a.n_req; ++r) {
    const int first = a.r.cu[r], len = a.r.cu[r + 1] - first, n = (len + CHUNK - 1) / CHUNK;
    if (p < n) {
      *t0 = first + p * CHUNK;
      *rows = min(CHUNK, len - p * CHUNK);
      return true;
    }
    p -= n;
  }
  return false;
}
// log2(sigmoid(x)): behind 1 + e the logarithm of a small e is taken by its series (1 + e would have rounded it away)
__device__ __forceinline__ float log2_sigmoid(float x) {
  const float e = exp2_of(-fabsf(x) * LOG2E);
  const float tail = e < 0.03125f ? e * LOG2E * fmaf(e, fmaf(e, fmaf(e, -0.25f, 0.33333333f), -0.5f), 1.0f) : __builtin_amdgcn_logf(1.0f + e);
  return fmaf(fminf(x, 0.f), LOG2E, -tail);
}
// q (optional), k and b of the chunk's tokens into LDS rows of `lq` floats (channels from D to Dp and tokens beyond the end:
// q = k = 0, no decay), and the segments' sums tot [4][lq].
template <typename T, bool Q, int RULE>
__device__ __forceinline__ void chunk_gates(const ChunkedArgs& ca, int h, int t0, int rows, int Dp, int lq, float* sq, float* sk, float* sb, float* tot) {
  const RuleArgs& a = ca.r;
  const int C = a.H * a.D, span = 1 << ca.d_shift;
  for (int idx = threadIdx.x; idx < (CHUNK / SEG) * span; idx += CT) {
    const int seg = idx >> ca.d_shift, i = idx & (span - 1);
    if (i >= Dp) continue;
    const bool live = i < a.D;
    const int c = h * a.D + (live ? i : 0);
    const T* at = (const T*)a.raw + (size_t)t0 * a.ld + c;
    T z[SEG], q[SEG];
    float zf[RULE == RULE_LINEAR ? SEG : 1];
#pragma unroll
    for (int t = 0; t < SEG; ++t) {      // (rows beyond the end: the last one again, masked below)
      const int tt = min(seg * SEG + t, rows - 1);
      const T* row = at + (size_t)tt * a.ld;
      z[t] = row[a.off_k];
      if constexpr (RULE == RULE_LINEAR) zf[t] = a.z[(size_t)(t0 - a.cu[0] + tt) * C + c];
      if constexpr (Q) q[t] = row[a.off_q];
    }
    const float bias = a.bias[c], l = RULE == RULE_COMPLEMENT ? a.lower[c] : 0.f;
    float run = 0.f;
#pragma unroll
    for (int t = 0; t < SEG; ++t) {
      const int row = seg * SEG + t;
      const bool in = live && row < rows;
      float k, lf;
      if constexpr (RULE == RULE_COMPLEMENT) {
        const float x = to_float(z[t]) + bias;
        const float e = exp2_of(-fabsf(x) * LOG2E), inv = rcp_of(1.0f + e), ei = e * inv;
        const float f = fmaf(1.0f - l, x >= 0.f ? inv : ei, l);
        k = (1.0f - l) * (x >= 0.f ? ei : inv);
        lf = __builtin_amdgcn_logf(fmaxf(f, 3.7252903e-9f));
      } else {
        k = to_float(z[t]);
        lf = fmaxf(log2_sigmoid(zf[t] + bias) * a.inv_tau, -28.0f);
      }
      run += in ? lf : 0.f;
      sk[row * lq + i] = in ? k : 0.f;
      sb[row * lq + i] = run;
      if constexpr (Q) {
        const float y = to_float(q[t]);
        sq[row * lq + i] = !in ? 0.f : (RULE == RULE_COMPLEMENT ? y * rcp_of(1.0f + exp2_of(-y * LOG2E)) : y * a.q_scale);
      }
    }
    tot[seg * lq + i] = run;
  }
}
template <typename T>
__device__ __forceinline__ void chunk_values(const ChunkedArgs& ca, int h, int t0, int rows, int Vp, int lv, float* sv) {
  const RuleArgs& a = ca.r;
  const T* at = (const T*)a.raw + (size_t)t0 * a.ld + a.off_v + h * a.V;
  if (ca.v8) {
    const int span = 1 << ca.v_shift;
#pragma unroll 2
    for (int idx = threadIdx.x; idx < CHUNK * span; idx += CT) {
      const int t = idx >> ca.v_shift, j = (idx & (span - 1)) * 8;
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

template <typename T, int RULE>
__global__ __launch_bounds__(CT) void gated_rule_chunk_state_kernel(ChunkedArgs ca) {
  extern __shared__ float lds[];
  const RuleArgs& a = ca.r;
  const int Dp = (a.D + 15) / 16 * 16, Vp = (a.V + 15) / 16 * 16, lq = Dp + 4, lv = Vp + 4;
  float* sk = lds;                        // [CHUNK][lq]
  float* sb = sk + CHUNK * lq;            // [CHUNK][lq]
  float* sv = sb + CHUNK * lq;            // [CHUNK][lv]
  float* tot = sv + CHUNK * lv;           // [4][lq]
  int t0, rows;
  if (!chunk_of(ca, blockIdx.x, &t0, &rows)) return;
  const int h = blockIdx.y;
  chunk_gates<T, false, RULE>(ca, h, t0, rows, Dp, lq, nullptr, sk, sb, tot);
  chunk_values<T>(ca, h, t0, rows, Vp, lv, sv);
  __syncthreads();
  // k_s times the decay from behind s to the chunk's end
  for (int idx = threadIdx.x; idx < (CHUNK / SEG) << ca.d_shift; idx += CT) {
    const int seg = idx >> ca.d_shift, i = idx & ((1 << ca.d_shift) - 1);
    if (i >= Dp) continue;
    float rest = tot[seg * lq + i];
    for (int m = seg + 1; m < CHUNK / SEG; ++m) rest += tot[m * lq + i];
#pragma unroll
    for (int t = seg * SEG; t < seg * SEG + SEG; ++t) sk[t * lq + i] *= exp2_of(rest - sb[t * lq + i]);
  }
  if (threadIdx.x < a.D) {
    const int i = threadIdx.x;
    ca.decay[((size_t)blockIdx.x * a.H + h) * a.D + i] = exp2_of(tot[i] + tot[lq + i] + tot[2 * lq + i] + tot[3 * lq + i]);
  }
  __syncthreads();
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE, lr = lane % 16, g = lane / 16;
  float* u = ca.u + ((size_t)blockIdx.x * a.H + h) * a.D * a.V;
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
__global__ __launch_bounds__(256) void gated_rule_chunk_scan_kernel(ChunkedArgs ca) {
  const RuleArgs& a = ca.r;
  const int r = blockIdx.y;
  const size_t per = (size_t)a.H * a.D * a.V, e = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (e >= per) return;
  int place = 0;
  for (int q = 0; q < r; ++q) place += (a.cu[q + 1] - a.cu[q] + CHUNK - 1) / CHUNK;
  const int n = (a.cu[r + 1] - a.cu[r] + CHUNK - 1) / CHUNK;
  const size_t channel = e / a.V;      // h D + i
  float* state = a.state + (size_t)a.slot[r] * a.slot_stride + e;
  float* u = ca.u + (size_t)place * per + e;
  const float* dec = ca.decay + (size_t)place * a.H * a.D + channel;
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
template <typename T, int RULE>
__global__ __launch_bounds__(CT) void gated_rule_chunk_out_kernel(ChunkedArgs ca) {
  extern __shared__ float lds[];
  const RuleArgs& a = ca.r;
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
  if (!chunk_of(ca, blockIdx.x, &t0, &rows)) return;
  const int h = blockIdx.y;
  chunk_gates<T, true, RULE>(ca, h, t0, rows, Dp, lq, sq, sk, sb, tot);
  chunk_values<T>(ca, h, t0, rows, Vp, lv, sv);
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
  for (int idx = threadIdx.x; idx < (CHUNK / SEG) << ca.d_shift; idx += CT) {
    const int seg = idx >> ca.d_shift, i = idx & ((1 << ca.d_shift) - 1);
    if (i >= Dp) continue;
    float before = 0.f;
    for (int m = 0; m < seg; ++m) before += tot[m * lq + i];
#pragma unroll
    for (int t = seg * SEG; t < seg * SEG + SEG; ++t) sq[t * lq + i] *= exp2_of(before + sb[t * lq + i]);
  }
  __syncthreads();
  const float* s0 = ca.u + ((size_t)blockIdx.x * a.H + h) * a.D * a.V;
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
    const T* gate = (const T*)a.raw + (size_t)t0 * a.ld + a.off_g + h * a.V + col;
#pragma unroll
    for (int I = 0; I < CHUNK / SEG; ++I)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = I * SEG + g * 4 + i;
        if (t >= rows) continue;
        float o = acc[v][I][i] * red[t] * gain;
        if constexpr (RULE == RULE_LINEAR) {
          const float g = to_float(gate[(size_t)t * a.ld]);
          o *= g * sigm(g);
        }
        out[(size_t)t * a.H * a.V] = from_float<T>(o);
      }
  }
}
inline size_t chunk_state_lds(int D, int V) {
  const int lq = (D + 15) / 16 * 16 + 4, lv = (V + 15) / 16 * 16 + 4;
  return (size_t)(2 * CHUNK * lq + CHUNK * lv + 4 * lq) * sizeof(float);
}
inline size_t chunk_out_lds(int D, int V) {
  const int lq = (D + 15) / 16 * 16 + 4, lv = (V + 15) / 16 * 16 + 4;
  return (size_t)(3 * CHUNK * lq + CHUNK * lv + CHUNK * (CHUNK + 4) + 4 * lq + CWAVES * CHUNK) * sizeof(float);
}
constexpr size_t LDS_BYTES = 160 * 1024;
template <typename T, int RULE>
int launch_chunks(const RuleArgs& r, float* workspace, int places, int n_req, hipStream_t stream) {
  ChunkedArgs a{r, workspace, workspace + (size_t)places * r.H * r.D * r.V, n_req, 4, 0, 0};
  while ((1 << a.d_shift) < r.D) ++a.d_shift;
  while ((1 << a.v_shift) * 8 < r.V) ++a.v_shift;
  if (r.V % 16) a.v_shift = std::max(a.v_shift, 1);      // (the zeros up to the next multiple of 16 are written as well)
  a.v8 = r.V % 8 == 0 && r.ld % 8 == 0 && r.off_v % 8 == 0 && ((uintptr_t)r.raw % 16) == 0;
  const size_t lds1 = chunk_state_lds(r.D, r.V), lds2 = chunk_out_lds(r.D, r.V);
  static bool raised = false;      // (one flag per instantiation)
  if (!raised) {
    if (hipFuncSetAttribute((const void*)gated_rule_chunk_state_kernel<T, RULE>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)LDS_BYTES) != hipSuccess ||
        hipFuncSetAttribute((const void*)gated_rule_chunk_out_kernel<T, RULE>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)LDS_BYTES) != hipSuccess)
      return gibbs_fail("gated rule in chunks: the kernels' LDS could not be reserved");
    raised = true;
  }
  const dim3 grid(places, r.H);
  gated_rule_chunk_state_kernel<T, RULE><<<grid, CT, lds1, stream>>>(a);
  gated_rule_chunk_scan_kernel<<<dim3(ceil_div((long)r.H * r.D * r.V, 256), n_req), 256, 0, stream>>>(a);
  gated_rule_chunk_out_kernel<T, RULE><<<grid, CT, lds2, stream>>>(a);
  return 0;
}
inline int rule_chunks_take(int D, int V) { return D > 0 && V > 0 && V <= MAX_VT * CWAVES * 16 && D <= CT && chunk_out_lds(D, V) <= LDS_BYTES; }
inline long rule_chunks_workspace(int rows, int n_req, int H, int D, int V) { return ((long)ceil_div(rows, CHUNK) + n_req) * H * D * ((long)V + 1); }
}  // namespace
