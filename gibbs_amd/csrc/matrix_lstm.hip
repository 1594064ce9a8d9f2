// A matrix memory with exponential gates and a normaliser (mLSTM).  Per head, with q, k [D], v [V] of a row, both gates one number
// per head, a = cap tanh((w_i . h + b_i) / cap) and log f = log sigmoid(cap tanh((w_f . h + b_f) / cap)), S [D, V], n [D] and m from 0:
//
//   m' = max(log f + m, a),  keep = exp(log f + m - m'),  take = exp(a - m')
//   S = keep S + take k v',  n = keep n + take k,  m = m'
//   o = S' q / (max(|n . q|, exp(-m)) + 1e-6)
//   out = o / sqrt(mean(o^2) + eps) * gain * sigmoid(g)
//
//   rows    a workgroup per (request, head) walks the request's rows in order: gates, state, read-out, norm and output gate in one
//           kernel.  A decoded token is a walk of one row; the state is streamed once in whole rows, and stays in registers
//           over a walk of several rows where it fits
//   chunks  long portions: a scan for the gates (m is a maximum of sums: an associative scan of pairs), then the rule over chunks of
//           64 tokens as products on the matrix cores with float32 operands
//
// Everything behind the projections is float32, and so is the state; the gates' own projections are float32 sums that are not
// rounded in between.  A slot holds S [H][D][V], and n [H][D] with m [H] behind it.
#include "common.h"
#include "lane8.h"
#include <algorithm>

namespace {
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float floatx4;
constexpr float LOG2E = 1.44269504088896340736f;
constexpr float TINY = 1e-6f;
__device__ __forceinline__ float exp2_of(float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ float sigm(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float log_sigm(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ void load_eight(const bf16* p, float* f) { unpack8(*(const uint4*)p, f); }
__device__ __forceinline__ void load_eight(const float* p, float* f) {
  const float4 a = *(const float4*)p, b = *(const float4*)(p + 4);
  f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w; f[4] = b.x; f[5] = b.y; f[6] = b.z; f[7] = b.w;
}

struct LstmArgs {
  const void* raw; long ld;             // projected rows: q at off_q, k at off_k (H D each), v at off_v, g at off_g (H V each)
  int off_q, off_k, off_v, off_g;
  const void* h; int W;                 // the rows that the gates' projections read [rows, W]
  const void* w_gates;                  // [2 H, W]: w_i of every head, then w_f
  const float* b_gates;                 // [2 H]
  const float* gain;                    // [H V]
  float cap, eps, q_scale;
  float* state; float* norm_state; long slot_stride;
  const int* cu;                        // null: row n is request n's
  const int* slot;
  void* out;                            // [rows, H V]
  int H, D, V;
  int vec;                              // rows of h and w_gates take 8 values at a time
};

// Thread (tx, group): columns tx VEC .. and rows group, group + groups, ...; y by groups, added in group order.
constexpr int STEP_THREADS = 512, STEP_ROWS = 8;
template <typename T, int VEC>
__global__ __launch_bounds__(STEP_THREADS) void matrix_lstm_rows_kernel(LstmArgs a, int lanes) {
  extern __shared__ float lds[];
  __shared__ float scratch[16], scratch2[16];
  const int r = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, D = a.D, V = a.V, H = a.H;
  const int tx = tid % lanes, group = tid / lanes, groups = STEP_THREADS / lanes;
  float* sq = lds;                // [D]
  float* sk = sq + D;             // [D]
  float* sn = sk + D;             // [D]
  float* part = sn + D;           // [groups][V]
  const int j0 = tx * VEC;
  const bool live = j0 < V;
  float* st = a.state + (size_t)a.slot[r] * a.slot_stride + (size_t)h * D * V + j0;
  float* ns = a.norm_state + (size_t)a.slot[r] * a.slot_stride;
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
  const int first = a.cu ? a.cu[r] : r, last = a.cu ? a.cu[r + 1] : r + 1;
  float m = ns[(size_t)H * D + h];
  for (int i = tid; i < D; i += STEP_THREADS) sn[i] = ns[(size_t)h * D + i];
  const T* wi = (const T*)a.w_gates + (size_t)h * a.W;
  const T* wf = (const T*)a.w_gates + (size_t)(H + h) * a.W;
  for (int n = first; n < last; ++n) {
    const T* row = (const T*)a.raw + (size_t)n * a.ld;
    const T* hr = (const T*)a.h + (size_t)n * a.W;
    float di = 0.f, df = 0.f;
    if (a.vec) {
      for (int c = tid * 8; c < a.W; c += STEP_THREADS * 8) {
        float x[8], p[8], q[8];
        load_eight(hr + c, x);
        load_eight(wi + c, p);
        load_eight(wf + c, q);
#pragma unroll
        for (int e = 0; e < 8; ++e) { di = fmaf(x[e], p[e], di); df = fmaf(x[e], q[e], df); }
      }
    } else {
      for (int c = tid; c < a.W; c += STEP_THREADS) {
        const float x = to_float(hr[c]);
        di = fmaf(x, to_float(wi[c]), di);
        df = fmaf(x, to_float(wf[c]), df);
      }
    }
    float v[VEC], y[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      v[e] = live ? to_float(row[a.off_v + h * V + j0 + e]) : 0.f;
      y[e] = 0.f;
    }
    di = block_sum(di, scratch);
    df = block_sum(df, scratch2);
    const float gate_in = a.cap * tanhf((di + a.b_gates[h]) / a.cap), gate_keep = log_sigm(a.cap * tanhf((df + a.b_gates[H + h]) / a.cap));
    const float above = fmaxf(gate_keep + m, gate_in);
    const float keep = expf(gate_keep + m - above), take = expf(gate_in - above);
    m = above;
    float nq = 0.f;
    for (int i = tid; i < D; i += STEP_THREADS) {      // (a thread's own entries of n: no one else touches them)
      const float q = to_float(row[a.off_q + h * D + i]) * a.q_scale, k = to_float(row[a.off_k + h * D + i]) * take;
      const float x = fmaf(keep, sn[i], k);
      sq[i] = q;
      sk[i] = k;
      sn[i] = x;
      nq = fmaf(x, q, nq);
    }
    nq = block_sum(nq, scratch);                       // (its barriers also publish sq and sk)
    for (int i0 = group; i0 < D; i0 += STEP_ROWS * groups) {
      if (!resident && (i0 != group || n != first)) ask(i0);
#pragma unroll
      for (int u = 0; u < STEP_ROWS; ++u) {
        const int i = i0 + u * groups;
        if (live && i < D) {
          const float k = sk[i], q = sq[i];
#pragma unroll
          for (int e = 0; e < VEC; ++e) {
            s[u][e] = fmaf(keep, s[u][e], k * v[e]);
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
    const float inv_den = 1.0f / (fmaxf(fabsf(nq), expf(-m)) + TINY);
    float ss = 0.f;
    for (int j = tid; j < V; j += STEP_THREADS) {
      float t = part[j];
      for (int g = 1; g < groups; ++g) t += part[g * V + j];
      t *= inv_den;
      part[j] = t;
      ss = fmaf(t, t, ss);
    }
    const float inv = 1.0f / sqrtf(block_sum(ss, scratch2) / (float)V + a.eps);
    T* out = (T*)a.out + ((size_t)n * H + h) * V;
    for (int j = tid; j < V; j += STEP_THREADS)
      out[j] = from_float<T>(part[j] * inv * a.gain[h * V + j] * sigm(to_float(row[a.off_g + h * V + j])));
    __syncthreads();                                   // (the next row writes part, sq and sk again)
  }
  for (int i = tid; i < D; i += STEP_THREADS) ns[(size_t)h * D + i] = sn[i];
  if (tid == 0) ns[(size_t)H * D + h] = m;
}

// ------------------------------------------------------------------------------------------------ the rule in chunks
// With c_t the sum of log2(keep) over the chunk's tokens up to t, and S_0, n_0 in front of the chunk:
//   S_t = 2^(c_t) S_0 + sum_(s <= t) 2^(c_t - c_s) take_s k_s v_s'      (n likewise, with 1 for v)
// so  S_t' q_t = 2^(c_t) S_0' q_t + sum_s A_ts v_s,  n_t . q_t = 2^(c_t) n_0 . q_t + sum_s A_ts,  A_ts = (q_t . k_s) take_s 2^(c_t - c_s),
// and the chunk's own part of S and n is sum_s 2^(c_64 - c_s) take_s k_s (v_s' or 1).  The exponents are never positive.
constexpr int CHUNK = 64, CT = 512, CWAVES = CT / WAVE, DB = 64, VB = 128;
constexpr int LDB = DB + 4;
struct LstmChunkArgs {
  LstmArgs a;
  int n_req, rows;                      // rows in all; arrays over rows count from the first request's first row
  const float* gates;                   // [2 H, rows]: the gates' projections
  float* keep;                          // [H, rows]: log2(keep)
  float* take;                          // [H, rows]
  float* level;                         // [H, rows]: m behind the row
  float* u;                             // [places, H, D, V]: a chunk's own part, then S in front of it
  float* un;                            // [places, H, D]: the same of n
  float* decay;                         // [places, H]: 2^(c_64)
};
// the request and the chunk of it that place `p` stands for (false: none); t0: the chunk's first row, counted from cu[0]
__device__ __forceinline__ bool chunk_of(const LstmChunkArgs& c, int p, int* t0, int* rows) {
  const int base = c.a.cu[0];
  for (int r = 0; r < c.n_req; ++r) {
    const int first = c.a.cu[r], len = c.a.cu[r + 1] - first, n = (len + CHUNK - 1) / CHUNK;
    if (p < n) {
      *t0 = first - base + p * CHUNK;
      *rows = min(CHUNK, len - p * CHUNK);
      return true;
    }
    p -= n;
  }
  return false;
}

// The gates of a request's rows for one head.  m_t = max(log f_t + m_(t-1), a_t): the map m -> max(x + m, y) of a row follows
// another as (x1 + x2, max(x2 + y1, y2)), so m is a scan of pairs over the rows, GT at a time.  (Sums of log f that matter are no longer
// than the gates' cap allows: whatever lies farther below is under the maximum.)
constexpr int GT = 512;
__global__ __launch_bounds__(GT) void matrix_lstm_gates_kernel(LstmChunkArgs c) {
  __shared__ float wx[GT / WAVE], wy[GT / WAVE], sm[GT];
  const int r = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid % WAVE, wave = tid / WAVE;
  const LstmArgs& a = c.a;
  const int first = a.cu[r] - a.cu[0], len = a.cu[r + 1] - a.cu[r];
  float* ms = a.norm_state + (size_t)a.slot[r] * a.slot_stride + (size_t)a.H * a.D + h;
  float m0 = *ms;
  const float* gi = c.gates + (size_t)h * c.rows + first;
  const float* gf = c.gates + (size_t)(a.H + h) * c.rows + first;
  for (int t0 = 0; t0 < len; t0 += GT) {
    const int t = t0 + tid;
    const bool in = t < len;
    float lf = 0.f, li = -INFINITY;      // (rows beyond the end change nothing)
    if (in) {
      lf = log_sigm(a.cap * tanhf((gf[t] + a.b_gates[a.H + h]) / a.cap));
      li = a.cap * tanhf((gi[t] + a.b_gates[h]) / a.cap);
    }
    float x = lf, y = li;
#pragma unroll
    for (int o = 1; o < WAVE; o <<= 1) {
      const float px = __shfl_up(x, o, WAVE), py = __shfl_up(y, o, WAVE);
      if (lane >= o) {
        y = fmaxf(x + py, y);
        x += px;
      }
    }
    if (lane == WAVE - 1) { wx[wave] = x; wy[wave] = y; }
    __syncthreads();
    float before = m0;                   // m in front of this wave's rows
    for (int w = 0; w < wave; ++w) before = fmaxf(wx[w] + before, wy[w]);
    const float m = fmaxf(x + before, y);
    sm[tid] = m;
    __syncthreads();
    const float prev = tid > 0 ? sm[tid - 1] : m0;
    if (in) {
      const size_t at = (size_t)h * c.rows + first + t;
      c.keep[at] = (lf + prev - m) * LOG2E;
      c.take[at] = expf(li - m);
      c.level[at] = m;
    }
    m0 = sm[GT - 1];
    __syncthreads();
  }
  if (tid == 0) *ms = m0;
}

// c_t of the chunk's tokens (the first wave; tokens beyond the end: as the last real one)
__device__ __forceinline__ float wave_cumulative(float x, int lane) {
#pragma unroll
  for (int o = 1; o < WAVE; o <<= 1) {
    const float y = __shfl_up(x, o, WAVE);
    if (lane >= o) x += y;
  }
  return x;
}
// `width` channels from column `col` of the chunk's projected rows into LDS rows of `ldl` floats, times a factor (scale[t] if given);
// channels from `have` to `width` and rows beyond the end are zeros.
template <typename T>
__device__ __forceinline__ void chunk_columns(const LstmArgs& a, int t0, int rows, long col, int have, int width, const float* scale, float factor,
                                              float* dst, int ldl) {
  const T* at = (const T*)a.raw + (size_t)(a.cu[0] + t0) * a.ld + col;
  if (a.vec && have % 8 == 0 && (((uintptr_t)at) % 16) == 0) {
    const int per = width / 8;
    for (int idx = threadIdx.x; idx < CHUNK * per; idx += CT) {
      const int t = idx / per, j = (idx % per) * 8;
      float f[8] = {};
      if (t < rows && j < have) load_eight(at + (size_t)t * a.ld + j, f);
      const float w = scale ? factor * scale[t] : factor;
#pragma unroll
      for (int e = 0; e < 8; ++e) f[e] *= w;
      *(float4*)(dst + t * ldl + j) = make_float4(f[0], f[1], f[2], f[3]);
      *(float4*)(dst + t * ldl + j + 4) = make_float4(f[4], f[5], f[6], f[7]);
    }
    return;
  }
  for (int idx = threadIdx.x; idx < CHUNK * width; idx += CT) {
    const int t = idx / width, j = idx % width;
    const float w = scale ? factor * scale[t] : factor;
    dst[t * ldl + j] = (t < rows && j < have) ? to_float(at[(size_t)t * a.ld + j]) * w : 0.f;
  }
}

// A chunk's own part of S (128 x 128 of it a workgroup) and of n.
template <typename T>
__global__ __launch_bounds__(CT) void matrix_lstm_chunk_state_kernel(LstmChunkArgs c, int v_blocks) {
  constexpr int DS = 128, LK = DS + 4, LV = VB + 4;
  extern __shared__ float lds[];
  float* sk = lds;                 // [CHUNK][LK]
  float* sv = sk + CHUNK * LK;     // [CHUNK][LV]
  __shared__ float weight[CHUNK];
  int t0, rows;
  if (!chunk_of(c, blockIdx.x, &t0, &rows)) return;
  const LstmArgs& a = c.a;
  const int h = blockIdx.y, d0 = (blockIdx.z / v_blocks) * DS, v0 = (blockIdx.z % v_blocks) * VB;
  const int dw = min(DS, a.D - d0), vw = min(VB, a.V - v0), dp = (dw + 15) / 16 * 16, vp = (vw + 15) / 16 * 16;
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE, lr = lane % 16, g = lane / 16;
  chunk_columns<T>(a, t0, rows, a.off_v + (long)h * a.V + v0, vw, vp, nullptr, 1.f, sv, LV);
  if (wave == 0) {
    const size_t at = (size_t)h * c.rows + t0 + lane;
    const float cum = wave_cumulative(lane < rows ? c.keep[at] : 0.f, lane);
    const float all = __shfl(cum, WAVE - 1, WAVE);
    weight[lane] = lane < rows ? c.take[at] * exp2_of(all - cum) : 0.f;
    if (lane == 0 && blockIdx.z == 0) c.decay[(size_t)blockIdx.x * a.H + h] = exp2_of(all);
  }
  __syncthreads();
  chunk_columns<T>(a, t0, rows, a.off_k + (long)h * a.D + d0, dw, dp, weight, 1.f, sk, LK);
  __syncthreads();
  if (v0 == 0 && threadIdx.x < dw) {
    float sum = 0.f;
    for (int t = 0; t < CHUNK; ++t) sum += sk[t * LK + threadIdx.x];
    c.un[((size_t)blockIdx.x * a.H + h) * a.D + d0 + threadIdx.x] = sum;
  }
  float* u = c.u + (((size_t)blockIdx.x * a.H + h) * a.D + d0) * a.V + v0;
  const int n0 = wave * 16;
  if (n0 >= vp) return;
  for (int m0 = 0; m0 < dp; m0 += 64) {           // four channel tiles at a time
    floatx4 acc[4] = {};
    for (int s0 = 0; s0 < CHUNK; s0 += 16) {
      float vb[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) vb[j] = sv[(s0 + g * 4 + j) * LV + n0 + lr];
#pragma unroll
      for (int m = 0; m < 4; ++m) {
        if (m0 + m * 16 >= dp) break;
#pragma unroll
        for (int j = 0; j < 4; ++j)
          acc[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(sk[(s0 + g * 4 + j) * LK + m0 + m * 16 + lr], vb[j], acc[m], 0, 0, 0);
      }
    }
#pragma unroll
    for (int m = 0; m < 4; ++m)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int row = m0 + m * 16 + g * 4 + i;
        if (row < dw && n0 + lr < vw) u[(size_t)row * a.V + n0 + lr] = acc[m][i];
      }
  }
}

// Per element of a request's S and n, over its chunks in order: u becomes what stands in front of each chunk, the slot's state what
// stands behind the last.
__global__ __launch_bounds__(256) void matrix_lstm_chunk_scan_kernel(LstmChunkArgs c) {
  const LstmArgs& a = c.a;
  const int r = blockIdx.y;
  const size_t per_s = (size_t)a.H * a.D * a.V, per_n = (size_t)a.H * a.D;
  size_t e = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (e >= per_s + per_n) return;
  const bool of_n = e >= per_s;
  if (of_n) e -= per_s;
  int place = 0;
  for (int q = 0; q < r; ++q) place += (a.cu[q + 1] - a.cu[q] + CHUNK - 1) / CHUNK;
  const int n = (a.cu[r + 1] - a.cu[r] + CHUNK - 1) / CHUNK;
  const int h = (int)(e / (of_n ? (size_t)a.D : (size_t)a.D * a.V));
  const size_t per = of_n ? per_n : per_s;
  float* state = (of_n ? a.norm_state : a.state) + (size_t)a.slot[r] * a.slot_stride + e;
  float* u = (of_n ? c.un : c.u) + (size_t)place * per + e;
  const float* dec = c.decay + (size_t)place * a.H + h;
  float S = *state;
  constexpr int AHEAD = 8;
  for (int c0 = 0; c0 < n; c0 += AHEAD) {
    float own[AHEAD], d[AHEAD];
#pragma unroll
    for (int k = 0; k < AHEAD; ++k) {
      const int at = min(c0 + k, n - 1);
      own[k] = u[(size_t)at * per];
      d[k] = dec[(size_t)at * a.H];
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

// The chunk's outputs: q and k come through LDS 64 channels at a time; the scores' tiles (ten of 16 x 16 on and below the diagonal) and
// S_0' q_t stay in registers across them.  VT: tiles of 16 values a wave.
template <typename T, int VT>
__global__ __launch_bounds__(CT) void matrix_lstm_chunk_out_kernel(LstmChunkArgs c) {
  __shared__ __attribute__((aligned(16))) float sq[CHUNK * LDB], sk[CHUNK * LDB], sA[CHUNK * LDB];
  __shared__ float cum[CHUNK], take[CHUNK], den[CHUNK], red[CWAVES][CHUNK];
  int t0, rows;
  if (!chunk_of(c, blockIdx.x, &t0, &rows)) return;
  const LstmArgs& a = c.a;
  const int h = blockIdx.y, D = a.D, V = a.V;
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE, lr = lane % 16, g = lane / 16;
  if (wave == 0) {
    const size_t at = (size_t)h * c.rows + t0 + lane;
    cum[lane] = wave_cumulative(lane < rows ? c.keep[at] : 0.f, lane);
    take[lane] = lane < rows ? c.take[at] : 0.f;
    den[lane] = lane < rows ? expf(-c.level[at]) : 1.f;
  }
  const int segs = (rows + 15) / 16;
  const float* s0 = c.u + ((size_t)blockIdx.x * a.H + h) * D * V;
  const float* n0 = c.un + ((size_t)blockIdx.x * a.H + h) * D;
  // tiles (I, J) of the scores: number p of the lower triangle, row by row; a wave has p = wave and p = wave + 8
  int tI[2], tJ[2];
#pragma unroll
  for (int x = 0; x < 2; ++x) {
    const int p = wave + x * CWAVES;
    tI[x] = p < 1 ? 0 : (p < 3 ? 1 : (p < 6 ? 2 : (p < 10 ? 3 : 4)));
    tJ[x] = p - tI[x] * (tI[x] + 1) / 2;
  }
  floatx4 score[2] = {}, acc[VT][4] = {};
  const int t_nq = threadIdx.x / 8, part = threadIdx.x % 8;      // (n . q: eight threads a token)
  float nq = 0.f;
  for (int d0 = 0; d0 < D; d0 += DB) {
    const int dw = min(DB, D - d0), dp = (dw + 15) / 16 * 16;
    __syncthreads();
    chunk_columns<T>(a, t0, rows, a.off_q + (long)h * D + d0, dw, dp, nullptr, a.q_scale, sq, LDB);
    chunk_columns<T>(a, t0, rows, a.off_k + (long)h * D + d0, dw, dp, nullptr, 1.f, sk, LDB);
    __syncthreads();
#pragma unroll
    for (int x = 0; x < 2; ++x) {
      if (tI[x] >= segs) continue;
      const float* qr = sq + (tI[x] * 16 + lr) * LDB + g * 4;
      const float* kr = sk + (tJ[x] * 16 + lr) * LDB + g * 4;
      for (int ch = 0; ch < dp; ch += 16) {
        const float4 q4 = *(const float4*)(qr + ch), k4 = *(const float4*)(kr + ch);
        score[x] = __builtin_amdgcn_mfma_f32_16x16x4f32(q4.x, k4.x, score[x], 0, 0, 0);
        score[x] = __builtin_amdgcn_mfma_f32_16x16x4f32(q4.y, k4.y, score[x], 0, 0, 0);
        score[x] = __builtin_amdgcn_mfma_f32_16x16x4f32(q4.z, k4.z, score[x], 0, 0, 0);
        score[x] = __builtin_amdgcn_mfma_f32_16x16x4f32(q4.w, k4.w, score[x], 0, 0, 0);
      }
    }
    for (int i = part; i < dw; i += 8) nq = fmaf(sq[t_nq * LDB + i], n0[d0 + i], nq);
#pragma unroll
    for (int v = 0; v < VT; ++v) {
      const int col = (wave + v * CWAVES) * 16 + lr;
      if ((wave + v * CWAVES) * 16 >= V) break;
#pragma unroll 2
      for (int ch = 0; ch < dp; ch += 16) {
        float sb[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int i = d0 + ch + g * 4 + j;
          sb[j] = (i < D && col < V) ? s0[(size_t)i * V + col] : 0.f;
        }
#pragma unroll
        for (int I = 0; I < 4; ++I) {
          const float4 q4 = *(const float4*)(sq + (I * 16 + lr) * LDB + ch + g * 4);
          const float qv[4] = {q4.x, q4.y, q4.z, q4.w};
#pragma unroll
          for (int j = 0; j < 4; ++j) acc[v][I] = __builtin_amdgcn_mfma_f32_16x16x4f32(qv[j], sb[j], acc[v][I], 0, 0, 0);
        }
      }
    }
  }
  // A_ts = (q_t . k_s) take_s 2^(c_t - c_s) for s <= t, else 0
#pragma unroll
  for (int x = 0; x < 2; ++x) {
    if (tI[x] >= segs) continue;
    const int s = tJ[x] * 16 + lr;
    const float ts = take[s], cs = cum[s];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = tI[x] * 16 + g * 4 + i;
      sA[t * LDB + s] = s <= t ? score[x][i] * ts * exp2_of(cum[t] - cs) : 0.f;
    }
  }
  __syncthreads();
  {
    nq *= exp2_of(cum[t_nq]);
    if (t_nq < segs * 16)
      for (int s = part; s <= t_nq; s += 8) nq += sA[t_nq * LDB + s];
    nq = group_sum<8>(nq);
    if (part == 0) den[t_nq] = 1.0f / (fmaxf(fabsf(nq), den[t_nq]) + TINY);
  }
#pragma unroll
  for (int I = 0; I < 4; ++I)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float e = exp2_of(cum[I * 16 + g * 4 + i]);
#pragma unroll
      for (int v = 0; v < VT; ++v) acc[v][I][i] *= e;
    }
  const T* values = (const T*)a.raw + (size_t)(a.cu[0] + t0) * a.ld + a.off_v + (long)h * V;
#pragma unroll
  for (int v = 0; v < VT; ++v) {
    const int col = (wave + v * CWAVES) * 16 + lr;
    if ((wave + v * CWAVES) * 16 >= V) break;
    for (int s = 0; s < segs * 16; s += 16) {
      float vb[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int t = s + g * 4 + j;
        vb[j] = (t < rows && col < V) ? to_float(values[(size_t)t * a.ld + col]) : 0.f;
      }
#pragma unroll
      for (int I = 0; I < 4; ++I) {
        if (I < s / 16 || I >= segs) continue;
        const float4 a4 = *(const float4*)(sA + (I * 16 + lr) * LDB + s + g * 4);
        const float av[4] = {a4.x, a4.y, a4.z, a4.w};
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[v][I] = __builtin_amdgcn_mfma_f32_16x16x4f32(av[j], vb[j], acc[v][I], 0, 0, 0);
      }
    }
  }
  __syncthreads();                        // (den is ready)
  // o, and the heads' norm over V: a row's squares over the 16 columns of a tile, then over the waves (in order)
#pragma unroll
  for (int I = 0; I < 4; ++I)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = I * 16 + g * 4 + i;
      const float d = den[t];
      float ss = 0.f;
#pragma unroll
      for (int v = 0; v < VT; ++v) {
        acc[v][I][i] *= d;
        ss = fmaf(acc[v][I][i], acc[v][I][i], ss);
      }
      ss = group_sum<16>(ss);
      if (lr == 0) red[wave][t] = ss;
    }
  __syncthreads();
  if (threadIdx.x < CHUNK) {
    float total = 0.f;
#pragma unroll
    for (int w = 0; w < CWAVES; ++w) total += red[w][threadIdx.x];
    den[threadIdx.x] = 1.0f / sqrtf(total / (float)V + a.eps);
  }
  __syncthreads();
#pragma unroll
  for (int v = 0; v < VT; ++v) {
    const int col = (wave + v * CWAVES) * 16 + lr;
    if (col >= V) break;
    const float gain = a.gain[h * V + col];
    const size_t row0 = (size_t)(a.cu[0] + t0);
    const T* gate = (const T*)a.raw + row0 * a.ld + a.off_g + (long)h * V + col;
    T* out = (T*)a.out + (row0 * a.H + h) * V + col;
#pragma unroll
    for (int I = 0; I < 4; ++I)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = I * 16 + g * 4 + i;
        if (t < rows) out[(size_t)t * a.H * V] = from_float<T>(acc[v][I][i] * den[t] * gain * sigm(to_float(gate[(size_t)t * a.ld])));
      }
  }
}

template <typename T>
int launch_chunks(const LstmChunkArgs& c, int places, hipStream_t stream) {
  const LstmArgs& a = c.a;
  constexpr size_t LDS_STATE = (size_t)CHUNK * (128 + 4 + VB + 4) * sizeof(float);
  static bool raised = false;      // (one flag per instantiation)
  if (!raised) {
    if (hipFuncSetAttribute((const void*)matrix_lstm_chunk_state_kernel<T>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)LDS_STATE) != hipSuccess)
      return gibbs_fail("matrix_lstm_chunks: the kernel's LDS could not be reserved");
    raised = true;
  }
  matrix_lstm_gates_kernel<<<dim3(c.n_req, a.H), GT, 0, stream>>>(c);
  const int v_blocks = ceil_div(a.V, VB), d_blocks = ceil_div(a.D, 128);
  matrix_lstm_chunk_state_kernel<T><<<dim3(places, a.H, v_blocks * d_blocks), CT, LDS_STATE, stream>>>(c, v_blocks);
  matrix_lstm_chunk_scan_kernel<<<dim3(ceil_div((long)a.H * a.D * (a.V + 1L), 256), c.n_req), 256, 0, stream>>>(c);
  const dim3 grid(places, a.H);
  if (a.V <= 128) matrix_lstm_chunk_out_kernel<T, 1><<<grid, CT, 0, stream>>>(c);
  else if (a.V <= 256) matrix_lstm_chunk_out_kernel<T, 2><<<grid, CT, 0, stream>>>(c);
  else matrix_lstm_chunk_out_kernel<T, 4><<<grid, CT, 0, stream>>>(c);
  return 0;
}
int step_lanes(int V, bool vec) {
  int lanes = 1;
  while (lanes < (vec ? V / 4 : V)) lanes *= 2;
  return lanes;
}
size_t rows_lds(int D, int V, int lanes) { return ((size_t)3 * D + (size_t)(STEP_THREADS / lanes) * V) * sizeof(float); }
}  // namespace

// Whether the row kernel takes a head's sizes, whether the rule in chunks does, and the floats of workspace that `rows` rows of
// `n_req` requests need in chunks.
GIBBS_EXPORT int gibbs_matrix_lstm_rows_take(int D, int V) {
  return D > 0 && D <= 3072 && V > 0 && (V <= STEP_THREADS || (V % 4 == 0 && V <= 4 * STEP_THREADS));
}
GIBBS_EXPORT int gibbs_matrix_lstm_chunks_take(int D, int V) { return D > 0 && V > 0 && V <= 4 * CWAVES * 16; }
GIBBS_EXPORT long gibbs_matrix_lstm_chunks_workspace(int rows, int n_req, int H, int D, int V) {
  const long places = (long)ceil_div(rows, CHUNK) + n_req;
  return 3L * H * rows + places * H * ((long)D * V + D + 1);
}

// raw: projected rows (row stride ld) with q, k, v and the output gate's columns at their offsets; h [.., W]: the rows that the gates'
// projections w_gates [2 heads, W] (w_i of every head, then w_f; the rows' type) read; b_gates [2 heads]; gain [heads * vdim].
// state [slots][heads][dim][vdim] and norm_state [slots]([heads][dim], then [heads]), slot_stride apart.  cu null: row n is
// request n's; else the rows cu[r] .. cu[r + 1].  out [.., heads * vdim] in the rows' type.
#define GIBBS_LSTM_OPERANDS                                                                                                              \
  const void *raw, long ld, int off_q, int off_k, int off_v, int off_g, const void *h, int W, const void *w_gates, const float *b_gates, \
      const float *gain, float cap, float eps, float q_scale, float *state, float *norm_state, long slot_stride, const int *cu, const int *slot, void *out
namespace {
int fill(LstmArgs* a, const char* what, int dtype, int H, int D, int V, GIBBS_LSTM_OPERANDS) {
  GIBBS_REQUIRE(raw && h && w_gates && b_gates && gain && state && norm_state && slot && out && W > 0, "%s: null operand", what);
  GIBBS_REQUIRE(H > 0 && H <= 65535 && D > 0 && V > 0 && cap > 0.f && off_q >= 0 && off_k >= 0 && off_v >= 0 && off_g >= 0, "%s: heads=%d D=%d V=%d cap=%g", what, H, D, V, cap);
  GIBBS_REQUIRE(ld >= std::max(std::max(off_q, off_k) + (long)H * D, std::max(off_v, off_g) + (long)H * V), "%s: rows of %ld values are too short", what, ld);
  GIBBS_REQUIRE(slot_stride >= (long)H * D * V && slot_stride >= (long)H * (D + 1), "%s: a slot of %ld floats is too small", what, slot_stride);
  GIBBS_REQUIRE(dtype == GIBBS_F32 || dtype == GIBBS_BF16, "%s: unknown dtype %d", what, dtype);
  *a = LstmArgs{raw, ld, off_q, off_k, off_v, off_g, h, W, w_gates, b_gates, gain, cap, eps, q_scale, state, norm_state, slot_stride, cu, slot, out, H, D, V, 0};
  a->vec = W % 8 == 0 && ld % 8 == 0 && ((uintptr_t)h % 16) == 0 && ((uintptr_t)w_gates % 16) == 0 && ((uintptr_t)raw % 16) == 0;
  return 0;
}
}  // namespace

GIBBS_EXPORT int gibbs_matrix_lstm_rows(GIBBS_LSTM_OPERANDS, int dtype, int n_req, int H, int D, int V, hipStream_t stream) {
  LstmArgs a;
  if (fill(&a, "matrix_lstm_rows", dtype, H, D, V, raw, ld, off_q, off_k, off_v, off_g, h, W, w_gates, b_gates, gain, cap, eps, q_scale, state, norm_state,
           slot_stride, cu, slot, out))
    return 1;
  GIBBS_REQUIRE(n_req > 0 && gibbs_matrix_lstm_rows_take(D, V), "matrix_lstm_rows: requests=%d, states of %d x %d", n_req, D, V);
  const bool vec = V % 4 == 0 && slot_stride % 4 == 0 && ((uintptr_t)state % 16) == 0;
  GIBBS_REQUIRE(vec || V <= STEP_THREADS, "matrix_lstm_rows: values of %d that are not aligned to 16 bytes", V);
  const int lanes = step_lanes(V, vec);
  const size_t lds = rows_lds(D, V, lanes);
  const dim3 grid(n_req, H);
  if (dtype == GIBBS_F32) {
    if (vec) matrix_lstm_rows_kernel<float, 4><<<grid, STEP_THREADS, lds, stream>>>(a, lanes);
    else matrix_lstm_rows_kernel<float, 1><<<grid, STEP_THREADS, lds, stream>>>(a, lanes);
  } else {
    if (vec) matrix_lstm_rows_kernel<bf16, 4><<<grid, STEP_THREADS, lds, stream>>>(a, lanes);
    else matrix_lstm_rows_kernel<bf16, 1><<<grid, STEP_THREADS, lds, stream>>>(a, lanes);
  }
  GIBBS_LAUNCH_STATUS("matrix_lstm_rows");
}

// The rows cu[0] .. of n_req requests (raw, h and out are addressed by the step's rows, cu may start above 0), n_rows in all; gates
// [2 heads, n_rows] float32: the gates' projections of those rows, w_gates h'.
GIBBS_EXPORT int gibbs_matrix_lstm_chunks(GIBBS_LSTM_OPERANDS, const float* gates, float* workspace, int dtype, int n_rows, int n_req, int H, int D,
                                          int V, hipStream_t stream) {
  LstmChunkArgs c{};
  if (fill(&c.a, "matrix_lstm_chunks", dtype, H, D, V, raw, ld, off_q, off_k, off_v, off_g, h, W, w_gates, b_gates, gain, cap, eps, q_scale, state,
           norm_state, slot_stride, cu, slot, out))
    return 1;
  GIBBS_REQUIRE(cu && gates && workspace && n_rows > 0 && n_req > 0 && n_req <= 65535 && gibbs_matrix_lstm_chunks_take(D, V),
                "matrix_lstm_chunks: rows=%d requests=%d, states of %d x %d", n_rows, n_req, D, V);
  const int places = ceil_div(n_rows, CHUNK) + n_req;      // (more than the requests' chunks can be)
  GIBBS_REQUIRE((long)ceil_div(V, VB) * ceil_div(D, 128) <= 65535, "matrix_lstm_chunks: states of %d x %d", D, V);
  c.n_req = n_req; c.rows = n_rows; c.gates = gates;
  c.u = workspace;
  c.un = c.u + (size_t)places * H * D * V;
  c.decay = c.un + (size_t)places * H * D;
  c.keep = c.decay + (size_t)places * H;
  c.take = c.keep + (size_t)H * n_rows;
  c.level = c.take + (size_t)H * n_rows;
  if (dtype == GIBBS_F32 ? launch_chunks<float>(c, places, stream) : launch_chunks<bf16>(c, places, stream)) return 1;
  GIBBS_LAUNCH_STATUS("matrix_lstm_chunks");
}
