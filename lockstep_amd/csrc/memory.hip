// More kernels of the mixers library: matrix memories whose gates are one number a head and token,
//
//   S_t = a_t S_(t-1) + b_t k_t v_t^T      S [N][DV] float a head, zero at a request's start
//   o_t = S_t^T q_t  (+ skip_h v_t)
//
// of which a state-space mixer (a = exp(-exp(A_log) dt), b = dt, k, v and q behind a short convolution) and the
// stabilised matrix memory with exponential gates (which also keeps n_t = a_t n_(t-1) + b_t k_t and a running
// maximum) are two choices; what surrounds them: convolutions, gates, the norms behind.
//
// Everything is computed in float whatever the compute dtype T is, on the matrix units too (products of float
// operands); T is the type of what the next matrix product reads.  A gate is kept as its logarithm (la = log a <= 0);
// sums of logarithms inside a chunk are formed in double, so a head that forgets at once and a head that hardly
// forgets are equally exact.
//
// Three ways through a request's tokens, by how many it brings:
//   one token      memory_token_kernel: convolution, gates, update and read in one launch (steps of single tokens)
//   a few tokens   memory_walk_kernel: token by token, the state in registers
//   more           chunks of 64 tokens: (1) every chunk's own contribution to the state, (2) the states in front of
//                  the chunks, one pass over the chunks, (3) every chunk's outputs from the state in front of it and
//                  the tokens inside: chunks and heads in parallel in (1) and (3).

#include "common.h"
#include "mixers_api.h"

namespace ls {

struct SeqMeta {  // one per sequence of the step (all int32), as the step's upload lays it out
  int q_off;      // first packed row
  int q_len;      // rows in this step
  int q_start;    // absolute position of the first row
  int kv_len;     // q_start + q_len
  int table_row;  // row of the block table, and the request's state slot
  int reserved[3];
};

__device__ __forceinline__ float sigmoid_m(float x) { return 1.0f / (1.0f + expf(-x)); }
__device__ __forceinline__ float silu_m(float x) { return x * sigmoid_m(x); }
__device__ __forceinline__ float softplus_m(float x) { return x > 20.0f ? x : log1pf(expf(x)); }
__device__ __forceinline__ float log_sigmoid_m(float x) { return fminf(x, 0.f) - log1pf(expf(-fabsf(x))); }

// Rows of one of q, k, v: head h of token t at p + t * ld + (h / share) * each.
struct HeadRows {
  const float* p;
  long ld;
  int each, share;
  __device__ __forceinline__ const float* at(long t, int h) const { return p + t * ld + (long)(h / share) * each; }
};

// A head's gates of a token: la = log a; b; and, for a memory with a normaliser, the floor of its denominator and the
// read-out n . q.
struct Gate {
  float la, b, floor, nq;
};

constexpr int kMemCols = 32;    // columns of a state that a workgroup of the walk takes
constexpr int kMemRowGroups = 32;
constexpr int kMemMaxRows = 256;
constexpr int kChunk = 64;      // tokens of a chunk

__device__ __forceinline__ f32x4 load4m(const float* __restrict__ p, int c, int limit, bool vec) {
  if (vec) {
    const f32x4 v = *reinterpret_cast<const f32x4*>(p + (c < limit ? c : 0));
    return c < limit ? v : f32x4{0.f, 0.f, 0.f, 0.f};
  }
  f32x4 v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < 4; ++i)
    if (c + i < limit) v[i] = p[c + i];
  return v;
}

__device__ __forceinline__ void store4m(float* __restrict__ p, int c, int limit, bool vec, const f32x4& v) {
  if (vec) {
    if (c < limit) *reinterpret_cast<f32x4*>(p + c) = v;
    return;
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
    if (c + i < limit) p[c + i] = v[i];
}

// Sum over the lanes of a wave that share lane % 8 (bits 3, 4 and 5 of the lane).
__device__ __forceinline__ float sum_by8(float v) {
  v = v + __shfl_xor(v, 8, kWave);
  v = v + __shfl_xor(v, 16, kWave);
  v = v + __shfl_xor(v, 32, kWave);
  return v;
}

// ---------------------------------------------------------------------------
// What a step of many tokens computes once, before the memory.
//
// conv_gates: raw [T][ld] float holds x | B | C (inner + 2 G N channels, at x_at) and dt (H, at dt_at).  Every channel
// passes a causal convolution y = bias + sum_a taps[a][c] in(p - (M-1) + a) (a ascending; zeros before the start) and
// silu -> conv [T][C].  Inputs before this step come from the request's ring: the input at position p lies in row p mod
// M of ring [M][C] (zeros before the start).  Gates: dt' = softplus(dt + dt_bias); la = -exp(A_log) dt', b = dt'.
// ---------------------------------------------------------------------------
constexpr int kConvTokens = 4;

__global__ __launch_bounds__(256) void conv_gates_kernel(const float* __restrict__ raw, long ld, int x_at, int dt_at, int n_tokens,
                                                         int C, int H, int M, const float* __restrict__ taps,
                                                         const float* __restrict__ bias, const float* __restrict__ a_log,
                                                         const float* __restrict__ dt_bias, const int* __restrict__ tok_seq,
                                                         const int* __restrict__ tok_pos, const SeqMeta* __restrict__ seqs,
                                                         const float* __restrict__ state, long state_stride, long ring_at,
                                                         float* __restrict__ conv, Gate* __restrict__ gates) {
  const int t0 = blockIdx.x * kConvTokens;
  if (blockIdx.y == gridDim.y - 1) {   // the gates of these tokens
    for (int i = threadIdx.x; i < kConvTokens * H; i += 256) {
      const int t = t0 + i / H, h = i % H;
      if (t >= n_tokens) break;
      const float dt = softplus_m(raw[(long)t * ld + dt_at + h] + dt_bias[h]);
      Gate g;
      g.la = -expf(a_log[h]) * dt;
      g.b = dt;
      g.floor = 1.0f;
      g.nq = 0.f;
      gates[(long)t * H + h] = g;
    }
    return;
  }
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= C) return;
  const float own_bias = bias[c];
#pragma unroll
  for (int u = 0; u < kConvTokens; ++u) {
    const int t = t0 + u;
    if (t >= n_tokens) break;
    const SeqMeta m = seqs[tok_seq[t]];
    const int pos = tok_pos[t];
    const float* ring = state + (long)m.table_row * state_stride + ring_at + c;
    const float* mine = raw + (long)(m.q_off - m.q_start) * ld + x_at + c;   // (the input at position p of this step: + p * ld)
    float y = own_bias;
    for (int a = 0; a < M; ++a) {
      const int p = pos - (M - 1) + a;
      const float* src = p >= m.q_start ? mine + (long)p * ld : ring + (long)((p + M) % M) * C;
      y = y + taps[(long)a * C + c] * *src;
    }
    conv[(long)t * C + c] = silu_m(y);
  }
}

// The last M - 1 inputs of a request go into its ring (rows p mod M), after every token of the step has read it.
__global__ __launch_bounds__(256) void conv_ring_kernel(const float* __restrict__ raw, long ld, int x_at, int C, int M,
                                                        const SeqMeta* __restrict__ seqs, float* __restrict__ state,
                                                        long state_stride, long ring_at) {
  const SeqMeta m = seqs[blockIdx.x];
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= C) return;
  float* ring = state + (long)m.table_row * state_stride + ring_at + c;
  for (int p = max(m.q_start, m.kv_len - (M - 1)); p < m.kv_len; ++p)
    ring[(long)(p % M) * C] = raw[(long)(m.q_off + p - m.q_start) * ld + x_at + c];
}

// exp_gates: raw holds the logits of the input gate (H, at i_at) and of the forget gate (H, at f_at); i = cap
// tanh((logit + i_bias) / cap), f = logsigmoid(cap tanh((logit + f_bias) / cap)).  The running maximum m_t = max(f_t +
// m_(t-1), i_t) starts at zero; la = f + m_(t-1) - m_t, b = exp(i - m_t), floor = exp(-m_t).  A wave a (request, head),
// 64 tokens at a time: m_t as a function of the maximum in front is max(F + m, M), and such pairs are composed by moves
// between lanes.  m is kept and advanced in double: where a head forgets slowly, f is far below m's last place in float,
// and what every token loses there would add up.  The state keeps m as the sum of two floats in two places a head, read at
// [q_start % 2] and left at [kv_len % 2] (a step of single tokens then never writes what it reads).
__device__ __forceinline__ void exp_gate_values(float zi, float zf, float cap, float& i, float& f) {
  i = cap * tanhf(zi / cap);
  f = log_sigmoid_m(cap * tanhf(zf / cap));
}

__device__ __forceinline__ double kept_maximum(const float* p) { return (double)p[0] + (double)p[1]; }
__device__ __forceinline__ void keep_maximum(float* p, double m) {
  p[0] = (float)m;
  p[1] = (float)(m - (double)(float)m);
}

__global__ __launch_bounds__(64) void exp_gates_kernel(const float* __restrict__ raw, long ld, int i_at, int f_at, int H,
                                                       const float* __restrict__ i_bias, const float* __restrict__ f_bias,
                                                       float cap, const SeqMeta* __restrict__ seqs, float* __restrict__ state,
                                                       long state_stride, long m_at, Gate* __restrict__ gates) {
  const int seq = blockIdx.x / H, h = blockIdx.x % H, lane = threadIdx.x;
  const SeqMeta m = seqs[seq];
  if (m.q_len <= 0) return;
  float* kept = state + (long)m.table_row * state_stride + m_at + 4 * h;
  double front = kept_maximum(kept + 2 * (m.q_start & 1));
  const float bi = i_bias[h], bf = f_bias[h];
  constexpr int AHEAD = 4;   // blocks of 64 tokens whose logits are on their way
  float zi[AHEAD], zf[AHEAD];
  auto request = [&](int t0, float& i, float& f) LS_INLINED {
    const float* row = raw + (long)(m.q_off + min(t0 + lane, m.q_len - 1)) * ld;
    i = row[i_at + h];
    f = row[f_at + h];
  };
#pragma unroll
  for (int u = 0; u < AHEAD; ++u) request(64 * u, zi[u], zf[u]);
  for (int tb = 0; tb < m.q_len; tb += 64 * AHEAD) {
#pragma unroll
    for (int u = 0; u < AHEAD; ++u) {
      const int t0 = tb + 64 * u;
      if (t0 >= m.q_len) break;
      const bool in = t0 + lane < m.q_len;
      float i, f;
      exp_gate_values(zi[u] + bi, zf[u] + bf, cap, i, f);
      request(t0 + 64 * AHEAD, zi[u], zf[u]);
      double F = in ? (double)f : 0.0, M = in ? (double)i : -1e300;   // m behind this run of tokens: max(F + m in front, M)
#pragma unroll
      for (int step = 1; step < 64; step <<= 1) {
        const double oF = __shfl_up(F, step, kWave), oM = __shfl_up(M, step, kWave);
        if (lane >= step) {
          M = fmax(F + oM, M);
          F = F + oF;
        }
      }
      const double mine = fmax(F + front, M);
      double before = __shfl_up(mine, 1, kWave);
      if (lane == 0) before = front;
      if (in) {
        Gate g;
        g.la = fminf((float)(((double)f + before) - mine), 0.f);
        g.b = expf((float)((double)i - mine));
        g.floor = expf((float)-mine);
        g.nq = 0.f;
        gates[(long)(m.q_off + t0 + lane) * H + h] = g;
      }
      front = __shfl(mine, 63, kWave);   // (lanes beyond the last token repeat its maximum: F and M are the identity there)
    }
  }
  if (lane == 0) keep_maximum(kept + 2 * (m.kv_len & 1), front);
}

// ---------------------------------------------------------------------------
// The walk: token by token.  A workgroup takes (request, head, 32 columns of the state); thread (c4 = tid % 8, group =
// tid / 8) keeps the rows group + 32 r of four neighbouring columns in registers.  A token's read-out: a thread's rows
// ascending, then its wave's eight groups by exchanges, then the waves in order.  The first block of columns also
// keeps n (NORM).  Requests with more than `longest` tokens are left to the chunks.
// ---------------------------------------------------------------------------
template <int R, bool NORM>
struct MemoryColumns {
  f32x4 S[R];
  float n[R];

  __device__ __forceinline__ void load(const float* __restrict__ s, const float* __restrict__ nv, int group, int N, int DV, int col,
                                       bool vec) {
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const int row = group + kMemRowGroups * r;
      S[r] = row < N ? load4m(s + (long)row * DV, col, DV, vec) : f32x4{0.f, 0.f, 0.f, 0.f};
      n[r] = NORM && row < N ? nv[row] : 0.f;
    }
  }
  __device__ __forceinline__ void store(float* __restrict__ s, float* __restrict__ nv, int group, int N, int DV, int col, bool vec,
                                        bool keeps_n) {
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const int row = group + kMemRowGroups * r;
      if (row < N) {
        store4m(s + (long)row * DV, col, DV, vec, S[r]);
        if (NORM && keeps_n) nv[row] = n[r];
      }
    }
  }
  // one token: the thread's part of the read-out (o) and of n . q
  __device__ __forceinline__ void step(float a, float b, const float (&kk)[R], const float (&qq)[R], const f32x4& v, f32x4& o,
                                       float& nq) {
    o = f32x4{0.f, 0.f, 0.f, 0.f};
    nq = 0.f;
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const float w = b * kk[r];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        S[r][i] = fmaf(a, S[r][i], w * v[i]);
        o[i] = fmaf(S[r][i], qq[r], o[i]);
      }
      if (NORM) {
        n[r] = fmaf(a, n[r], w);
        nq = fmaf(n[r], qq[r], nq);
      }
    }
  }
};

template <int R, bool NORM>
__global__ __launch_bounds__(256) void memory_walk_kernel(HeadRows q, HeadRows k, HeadRows v, Gate* __restrict__ gates, int H, int N,
                                                          int DV, float q_scale, const float* __restrict__ skip,
                                                          const SeqMeta* __restrict__ seqs, int longest, float* __restrict__ state,
                                                          long state_stride, int state_vec, int v_vec, float* __restrict__ out,
                                                          long ldo) {
  __shared__ float part_s[2][4][kMemCols + 1];
  const int blocks = (DV + kMemCols - 1) / kMemCols;
  const int h = blockIdx.x / blocks, cb = blockIdx.x % blocks;
  const SeqMeta m = seqs[blockIdx.y];
  if (m.q_len <= 0 || m.q_len > longest) return;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int c4 = threadIdx.x & 7, group = threadIdx.x >> 3;
  const int col = cb * kMemCols + 4 * c4;
  float* mine = state + (long)m.table_row * state_stride + (long)h * N * DV;
  float* my_n = state + (long)m.table_row * state_stride + (long)H * N * DV + (long)h * N;
  MemoryColumns<R, NORM> mem;
  mem.load(mine, my_n, group, N, DV, col, state_vec != 0);
  const float d = skip ? skip[h] : 0.f;
  float kk[R], qq[R];
  f32x4 vv;
  float la, b;
  auto request = [&](int i) LS_INLINED {
    const long t = m.q_off + i;
    const float* k_row = k.at(t, h);
    const float* q_row = q.at(t, h);
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const int row = group + kMemRowGroups * r;
      kk[r] = row < N ? k_row[row] : 0.f;
      qq[r] = row < N ? q_row[row] * q_scale : 0.f;
    }
    vv = load4m(v.at(t, h), col, DV, v_vec != 0);
    la = gates[t * H + h].la;
    b = gates[t * H + h].b;
  };
  request(0);
  for (int i = 0; i < m.q_len; ++i) {
    const f32x4 now_v = vv;
    f32x4 o;
    float nq;
    mem.step(expf(la), b, kk, qq, vv, o, nq);
    if (i + 1 < m.q_len) request(i + 1);
#pragma unroll
    for (int e = 0; e < 4; ++e) o[e] = sum_by8(o[e]);
    if (NORM) nq = sum_by8(nq);
    float(*part)[kMemCols + 1] = part_s[i & 1];
    if (lane < 8) {
#pragma unroll
      for (int e = 0; e < 4; ++e) part[w][4 * lane + e] = o[e];
      if (NORM && lane == 0) part[w][kMemCols] = nq;
    }
    __syncthreads();   // (the buffer of the token after next is written behind the next barrier: two are enough)
    const long t = m.q_off + i;
    if (threadIdx.x < 8) {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int c = col + e;
        const int at = 4 * c4 + e;
        if (c < DV)
          out[t * ldo + (long)h * DV + c] = (((part[0][at] + part[1][at]) + part[2][at]) + part[3][at]) + d * now_v[e];
      }
    }
    if (NORM && cb == 0 && threadIdx.x == 64)
      gates[t * H + h].nq = ((part[0][kMemCols] + part[1][kMemCols]) + part[2][kMemCols]) + part[3][kMemCols];
  }
  mem.store(mine, my_n, group, N, DV, col, state_vec != 0, cb == 0);
}

// ---------------------------------------------------------------------------
// A step of single tokens: everything of the memory in one launch.  Workgroups as in the walk.
// SPACE: raw holds x | B | C at x_at and dt at dt_at; the workgroup convolves its 32 columns of x and its group's B and
//   C itself (M inputs a channel), and one workgroup of those that read a channel leaves the token's input in the ring,
//   in a row that no one reads in this step.
// else: q, k, v as they are in raw (q_at, k_at, v_at), exponential gates as exp_gates_kernel forms them.
// WHOLE: a workgroup takes all columns of a head (256 threads for every 32 of them, at most 128 columns), divides the head by
// its denominator and its root mean square and multiplies it by the weight and the gate's sigmoid; normed [T][ldn] (T).
// ---------------------------------------------------------------------------
struct SpaceArgs {
  int x_at, dt_at, C, G, M;
  long ring_at;
  const float *taps, *conv_bias, *a_log, *dt_bias, *skip;
};
struct ExpArgs {
  int q_at, k_at, v_at, i_at, f_at;
  long m_at;
  float cap, q_scale;
  const float *i_bias, *f_bias;
  // WHOLE: the norm behind, weight [H * DV], the gate's logits at g_at
  const float* weight;
  int g_at;
  float eps, denom_eps;
};
constexpr int kMemWhole = 4;   // blocks of kMemCols columns that a workgroup of WHOLE takes at most

template <int R, bool SPACE, bool WHOLE, typename T>
__global__ __launch_bounds__(WHOLE ? 256 * kMemWhole : 256) void memory_token_kernel(const float* __restrict__ raw, long ld, SpaceArgs sp, ExpArgs ex,
                                                           int H, int N, int DV, const SeqMeta* __restrict__ seqs,
                                                           float* __restrict__ state, long state_stride, int state_vec,
                                                           Gate* __restrict__ gates, float* __restrict__ out, long ldo,
                                                           T* __restrict__ normed, long ldn) {
  constexpr bool NORM = !SPACE;
  constexpr int SUBS = WHOLE ? kMemWhole : 1;
  __shared__ __attribute__((aligned(16))) float v_all[SUBS][kMemCols];
  __shared__ float k_s[kMemMaxRows], q_s[kMemMaxRows], part_all[SUBS][4][kMemCols + 1], o_s[SUBS * kMemCols], nq_s;
  const int blocks = WHOLE ? 1 : (DV + kMemCols - 1) / kMemCols;
  const int sub = WHOLE ? (int)threadIdx.x >> 8 : 0, tid = threadIdx.x & 255;
  const int h = blockIdx.x / blocks, cb = WHOLE ? sub : blockIdx.x % blocks;
  float* v_s = v_all[sub];
  float(*part_s)[kMemCols + 1] = part_all[sub];
  const SeqMeta m = seqs[blockIdx.y];
  const long t = m.q_off;
  const int pos = m.q_start;
  const float* row = raw + t * ld;
  const int lane = tid & 63, w = tid >> 6;
  const int c4 = tid & 7, group = tid >> 3;
  const int col = cb * kMemCols + 4 * c4;
  float* slot = state + (long)m.table_row * state_stride;
  float* mine = slot + (long)h * N * DV;
  float* my_n = slot + (long)H * N * DV + (long)h * N;
  MemoryColumns<R, NORM> mem;
  mem.load(mine, my_n, group, N, DV, col, state_vec != 0);   // (on its way while the operands are formed)
  constexpr int PER = kMemWhole * kMemCols / 64;
  float gate_v[PER], weight_v[PER];
  if constexpr (WHOLE) {   // what the first wave applies at the end
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      const int c = min((int)threadIdx.x % 64 + 64 * j, DV - 1);
      gate_v[j] = row[ex.g_at + h * DV + c];
      weight_v[j] = ex.weight[(long)h * DV + c];
    }
  }
  float a, b, d = 0.f, floor = 1.0f;
  if constexpr (SPACE) {
    const int each = H / sp.G, g = h / each, inner = H * DV;
    const bool writes_group = cb == 0 && h == g * each;
    float* ring = slot + sp.ring_at;
    const int own_row = pos % sp.M, first_row = own_row + 1;   // (position pos - (M-1) + j lies in row (pos + 1 + j) mod M)
    for (int i = tid; i < 2 * N + kMemCols; i += 256) {
      const bool is_v = i >= 2 * N;
      const int vc = cb * kMemCols + i - 2 * N;
      if (is_v && vc >= DV) {
        v_s[i - 2 * N] = 0.f;
        continue;
      }
      const int c = is_v ? h * DV + vc : (i < N ? inner + g * N + i : inner + sp.G * N + g * N + (i - N));
      const float now = row[sp.x_at + c];
      float y = sp.conv_bias[c];
      // inputs at the positions pos - (M-1) + j: rows of the ring (zeros before the start), requested together four at a time
      for (int j0 = 0; j0 + 1 < sp.M; j0 += 4) {
        float tap[4], in[4];
#pragma unroll
        for (int u = 0; u < 4; ++u) {
          const int j = min(j0 + u, sp.M - 2);
          const int r = first_row + j;
          tap[u] = sp.taps[(long)j * sp.C + c];
          in[u] = ring[(long)(r >= sp.M ? r - sp.M : r) * sp.C + c];
        }
#pragma unroll
        for (int u = 0; u < 4; ++u)
          if (j0 + u + 1 < sp.M) y = y + tap[u] * in[u];
      }
      y = silu_m(y + sp.taps[(long)(sp.M - 1) * sp.C + c] * now);
      if (is_v) v_s[i - 2 * N] = y;
      else if (i < N) k_s[i] = y;
      else q_s[i - N] = y;
      if (is_v || writes_group) ring[(long)own_row * sp.C + c] = now;
    }
    const float dt = softplus_m(row[sp.dt_at + h] + sp.dt_bias[h]);
    a = expf(-expf(sp.a_log[h]) * dt);
    b = dt;
    d = sp.skip[h];
  } else {
    for (int i = tid + (sub ? 2 * N : 0); i < 2 * N + kMemCols; i += 256) {
      if (i < N) k_s[i] = row[ex.k_at + h * N + i];
      else if (i < 2 * N) q_s[i - N] = row[ex.q_at + h * N + i - N] * ex.q_scale;
      else v_s[i - 2 * N] = cb * kMemCols + i - 2 * N < DV ? row[ex.v_at + h * DV + cb * kMemCols + i - 2 * N] : 0.f;
    }
    float gi, gf;
    exp_gate_values(row[ex.i_at + h] + ex.i_bias[h], row[ex.f_at + h] + ex.f_bias[h], ex.cap, gi, gf);
    float* kept = slot + ex.m_at + 4 * h;
    const double before = kept_maximum(kept + 2 * (pos & 1));
    const double now = fmax((double)gf + before, (double)gi);
    if (cb == 0 && tid == 0) keep_maximum(kept + 2 * ((pos + 1) & 1), now);
    a = expf(fminf((float)(((double)gf + before) - now), 0.f));
    b = expf((float)((double)gi - now));
    floor = expf((float)-now);
  }
  __syncthreads();
  float kk[R], qq[R];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int at = group + kMemRowGroups * r;
    kk[r] = at < N ? k_s[at] : 0.f;
    qq[r] = at < N ? q_s[at] : 0.f;
  }
  const f32x4 vv = *reinterpret_cast<const f32x4*>(v_s + 4 * c4);
  f32x4 o;
  float nq;
  mem.step(a, b, kk, qq, vv, o, nq);
  mem.store(mine, my_n, group, N, DV, col, state_vec != 0, cb == 0);
#pragma unroll
  for (int e = 0; e < 4; ++e) o[e] = sum_by8(o[e]);
  if (NORM) nq = sum_by8(nq);
  if (lane < 8) {
#pragma unroll
    for (int e = 0; e < 4; ++e) part_s[w][4 * lane + e] = o[e];
    if (NORM && lane == 0) part_s[w][kMemCols] = nq;
  }
  __syncthreads();
  if constexpr (WHOLE) {
    if (tid < kMemCols) o_s[cb * kMemCols + tid] = ((part_s[0][tid] + part_s[1][tid]) + part_s[2][tid]) + part_s[3][tid];
    if (threadIdx.x == 64) nq_s = ((part_s[0][kMemCols] + part_s[1][kMemCols]) + part_s[2][kMemCols]) + part_s[3][kMemCols];
    __syncthreads();
    if (threadIdx.x >= 64) return;
    const float share = 1.0f / (fmaxf(fabsf(nq_s), floor) + ex.denom_eps);
    float v[PER], part = 0.f;   // lane i: the elements i, i + 64, ... ascending, then a butterfly
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      const int c = lane + 64 * j;
      v[j] = c < DV ? o_s[c] * share : 0.f;
      part = part + v[j] * v[j];
    }
    const float scale = 1.0f / sqrtf(wave_sum(part) / (float)DV + ex.eps);
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      const int c = lane + 64 * j;
      if (c < DV) normed[t * ldn + (long)h * DV + c] = from_f32<T>(((v[j] * scale) * weight_v[j]) * sigmoid_m(gate_v[j]));
    }
    return;
  }
  if (threadIdx.x < kMemCols) {
    const int at = threadIdx.x, c = cb * kMemCols + at;
    if (c < DV)
      out[t * ldo + (long)h * DV + c] = (((part_s[0][at] + part_s[1][at]) + part_s[2][at]) + part_s[3][at]) + d * v_s[at];
  }
  if (NORM && cb == 0 && threadIdx.x == 64) {
    gates[t * H + h].floor = floor;
    gates[t * H + h].nq = ((part_s[0][kMemCols] + part_s[1][kMemCols]) + part_s[2][kMemCols]) + part_s[3][kMemCols];
  }
}

// ---------------------------------------------------------------------------
// Chunks of 64 tokens.  items [n][2]: (request of the step, chunk); states [n][E] float, E = H N DV (+ H N with a
// normaliser), laid out like a request's state; decays [n][H].
//
// Inside a chunk L_t = la_1 + ... + la_t (double).  LDS tiles are [64][kTileRow] floats: a row of 68 floats spreads both
// the 16-byte reads along rows and the single reads down columns over all banks.
// ---------------------------------------------------------------------------
constexpr int kTileRow = 68;

// L_t of a chunk's tokens, by the first wave; tokens beyond the last add nothing and write nothing.
__device__ __forceinline__ void chunk_gates(const Gate* __restrict__ gates, long t0, int n, int H, int h, double* L_s, float* b_s) {
  if (threadIdx.x < 64) {
    const int t = threadIdx.x;
    const Gate* g = gates + (t0 + min(t, n - 1)) * H + h;
    double L = t < n ? (double)g->la : 0.0;
    b_s[t] = t < n ? g->b : 0.f;
#pragma unroll
    for (int step = 1; step < 64; step <<= 1) {
      const double o = __shfl_up(L, step, kWave);
      if (t >= step) L += o;
    }
    L_s[t] = L;
  }
}

// Copy a 64 x 64 piece of rows into an LDS tile: row r from src(r), columns c0 .. c0 + 63 below `limit`, rows below n,
// times factor(r); zeros elsewhere.
template <typename Src, typename Factor>
__device__ __forceinline__ void stage_tile(float* __restrict__ tile, Src src, int n, int c0, int limit, bool vec, Factor factor) {
  const int c = 4 * (threadIdx.x & 15);
  f32x4 got[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int r = (threadIdx.x >> 4) + 16 * j;
    got[j] = r < n ? load4m(src(r), c0 + c, limit, vec) : f32x4{0.f, 0.f, 0.f, 0.f};
  }
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int r = (threadIdx.x >> 4) + 16 * j;
    const float f = factor(r);
#pragma unroll
    for (int i = 0; i < 4; ++i) got[j][i] = got[j][i] * f;
    *reinterpret_cast<f32x4*>(tile + r * kTileRow + c) = got[j];
  }
}

// Four elements down a column of a tile: rows r .. r + 3.
__device__ __forceinline__ f32x4 tile_column(const float* tile, int r, int c) {
  return f32x4{tile[r * kTileRow + c], tile[(r + 1) * kTileRow + c], tile[(r + 2) * kTileRow + c], tile[(r + 3) * kTileRow + c]};
}

// (1) states[item] = sum_t exp(L_64 - L_t) b_t k_t v_t^T; a workgroup: 64 rows x 64 columns of one head.
__global__ __launch_bounds__(256) void memory_chunk_state_kernel(HeadRows k, HeadRows v, const Gate* __restrict__ gates, int H, int N,
                                                                 int DV, const SeqMeta* __restrict__ seqs,
                                                                 const int* __restrict__ items, float* __restrict__ states, long E,
                                                                 float* __restrict__ decays, int norm, int k_vec, int v_vec,
                                                                 int state_vec) {
  __shared__ __attribute__((aligned(16))) float k_s[64 * kTileRow], v_s[64 * kTileRow];
  __shared__ double L_s[64];
  __shared__ float b_s[64];
  const int item = blockIdx.x, h = blockIdx.y;
  const int col_blocks = (DV + 63) / 64;
  const int n0 = (blockIdx.z / col_blocks) * 64, c0 = (blockIdx.z % col_blocks) * 64;
  const SeqMeta m = seqs[items[2 * item]];
  const int first = items[2 * item + 1] * kChunk;
  const int n = min(kChunk, m.q_len - first);
  const long t0 = m.q_off + first;
  chunk_gates(gates, t0, n, H, h, L_s, b_s);
  __syncthreads();
  const double end = L_s[63];
  stage_tile(k_s, [&](int r) LS_INLINED { return k.at(t0 + r, h); }, n, n0, N, k_vec != 0,
             [&](int r) LS_INLINED { return expf((float)(end - L_s[r])) * b_s[r]; });
  stage_tile(v_s, [&](int r) LS_INLINED { return v.at(t0 + r, h); }, n, c0, DV, v_vec != 0, [](int) LS_INLINED { return 1.0f; });
  __syncthreads();
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int l16 = lane & 15, quad = lane >> 4, wr = w >> 1, wc = w & 1;
  f32x4 acc[2][2];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int ch = 0; ch < 4; ++ch) {
    f32x4 a[2], b[2];
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      a[j] = tile_column(v_s, 16 * ch + 4 * quad, wc * 32 + 16 * j + l16);
      b[j] = tile_column(k_s, 16 * ch + 4 * quad, wr * 32 + 16 * j + l16);
    }
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int j = 0; j < 2; ++j) Atom<float>::mma(acc[i][j], a[j], b[i]);
  }
  float* dst = states + (long)item * E + (long)h * N * DV;
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int row = n0 + wr * 32 + 16 * i + l16;
    if (row >= N) continue;
#pragma unroll
    for (int j = 0; j < 2; ++j) store4m(dst + (long)row * DV, c0 + wc * 32 + 16 * j + 4 * quad, DV, state_vec != 0, acc[i][j]);
  }
  if (norm && c0 == 0 && threadIdx.x < 64 && n0 + (int)threadIdx.x < N) {
    float sum = 0.f;
    for (int t = 0; t < n; ++t) sum = sum + k_s[t * kTileRow + threadIdx.x];
    states[(long)item * E + (long)H * N * DV + (long)h * N + n0 + threadIdx.x] = sum;
  }
  if (blockIdx.z == 0 && threadIdx.x == 0) decays[(long)item * H + h] = expf((float)end);
}

// (2) runs [n][4]: (request of the step, its first item, its items, 0).  The states in front of the chunks take the place
// of the chunks' contributions; the request's state moves on to behind the last chunk.  V elements a thread.
template <int V>
__global__ __launch_bounds__(256) void memory_chunk_scan_kernel(const SeqMeta* __restrict__ seqs, const int* __restrict__ runs,
                                                                float* __restrict__ states, long E, const float* __restrict__ decays,
                                                                int H, int N, int DV, float* __restrict__ state, long state_stride) {
  typedef float vec __attribute__((ext_vector_type(V)));
  const long e = ((long)blockIdx.x * 256 + threadIdx.x) * V;
  if (e >= E) return;
  const int seq = runs[4 * blockIdx.y], first = runs[4 * blockIdx.y + 1], count = runs[4 * blockIdx.y + 2];
  const long matrix = (long)N * DV;
  const int h = e < H * matrix ? (int)(e / matrix) : (int)((e - H * matrix) / N);
  float* kept = state + (long)seqs[seq].table_row * state_stride + e;
  float* at = states + (long)first * E + e;
  const float* decay = decays + (long)first * H + h;
  vec S = *reinterpret_cast<const vec*>(kept);
  constexpr int U = 8;
  for (int c0 = 0; c0 < count; c0 += U) {
    vec got[U];
    float f[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int c = min(c0 + u, count - 1);
      got[u] = *reinterpret_cast<const vec*>(at + (long)c * E);
      f[u] = decay[(long)c * H];
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (c0 + u < count) {
        *reinterpret_cast<vec*>(at + (long)(c0 + u) * E) = S;
#pragma unroll
        for (int i = 0; i < V; ++i) S[i] = fmaf(f[u], S[i], got[u][i]);
      }
  }
  *reinterpret_cast<vec*>(kept) = S;
}

// (3) o_t = exp(L_t) S_in^T q_t + sum_(s <= t) exp(L_t - L_s) b_s (q_t . k_s) v_s (+ skip v_t: on the diagonal), and
// likewise n . q without the values.  A workgroup: the 64 tokens of one chunk, one head, 64 columns; its waves 32 x 32.
__global__ __launch_bounds__(256) void memory_chunk_out_kernel(HeadRows q, HeadRows k, HeadRows v, Gate* __restrict__ gates, int H,
                                                               int N, int DV, float q_scale, const float* __restrict__ skip,
                                                               const SeqMeta* __restrict__ seqs, const int* __restrict__ items,
                                                               const float* __restrict__ states, long E, int norm, int q_vec,
                                                               int k_vec, int v_vec, int state_vec, int out_vec,
                                                               float* __restrict__ out, long ldo) {
  __shared__ __attribute__((aligned(16))) float q_s[64 * kTileRow], k_s[64 * kTileRow], s_s[64 * kTileRow];
  __shared__ double L_s[64];
  __shared__ float b_s[64], n_s[64];
  const int item = blockIdx.x, h = blockIdx.y, c0 = blockIdx.z * 64;
  const SeqMeta m = seqs[items[2 * item]];
  const int first = items[2 * item + 1] * kChunk;
  const int n = min(kChunk, m.q_len - first);
  const long t0 = m.q_off + first;
  chunk_gates(gates, t0, n, H, h, L_s, b_s);
  const float* S_in = states + (long)item * E + (long)h * N * DV;
  const float* n_in = states + (long)item * E + (long)H * N * DV + (long)h * N;
  const bool norm_here = norm != 0 && c0 == 0;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int l16 = lane & 15, quad = lane >> 4, wr = w >> 1, wc = w & 1;
  f32x4 g[2][2], o[2][2];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j) g[i][j] = o[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  float nq = 0.f;   // thread (token tid / 4, part tid % 4)
  const int my_t = threadIdx.x >> 2, my_part = threadIdx.x & 3;
  auto one = [](int) LS_INLINED { return 1.0f; };
  for (int n0 = 0; n0 < N; n0 += 64) {
    if (n0) __syncthreads();
    stage_tile(q_s, [&](int r) LS_INLINED { return q.at(t0 + r, h); }, n, n0, N, q_vec != 0, [&](int) LS_INLINED { return q_scale; });
    stage_tile(k_s, [&](int r) LS_INLINED { return k.at(t0 + r, h); }, n, n0, N, k_vec != 0, one);
    stage_tile(s_s, [&](int r) LS_INLINED { return S_in + (long)(n0 + r) * DV; }, min(64, N - n0), c0, DV, state_vec != 0, one);
    if (norm_here && threadIdx.x < 64) n_s[threadIdx.x] = n0 + (int)threadIdx.x < N ? n_in[n0 + threadIdx.x] : 0.f;
    __syncthreads();
    const int chunks = (min(64, N - n0) + 15) / 16;
    for (int ch = 0; ch < chunks; ++ch) {
      f32x4 qv[2], kv[2], sv[2];
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        qv[j] = *reinterpret_cast<const f32x4*>(q_s + (wr * 32 + 16 * j + l16) * kTileRow + 16 * ch + 4 * quad);
        kv[j] = *reinterpret_cast<const f32x4*>(k_s + (wc * 32 + 16 * j + l16) * kTileRow + 16 * ch + 4 * quad);
        sv[j] = tile_column(s_s, 16 * ch + 4 * quad, wc * 32 + 16 * j + l16);
      }
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j) {
          if (wc * 32 + 16 * j <= wr * 32 + 16 * i + 15) Atom<float>::mma(g[i][j], kv[j], qv[i]);   // (tokens of the tile's past)
          Atom<float>::mma(o[i][j], sv[j], qv[i]);
        }
    }
    if (norm_here)
      for (int i = my_part; i < 64; i += 4) nq = fmaf(q_s[my_t * kTileRow + i], n_s[i], nq);
  }
  __syncthreads();
  const float d = skip ? skip[h] : 0.f;
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int t = wr * 32 + 16 * i + l16;
    const double L = L_s[t];
    const float lead = expf((float)L);
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int s0 = wc * 32 + 16 * j + 4 * quad;
      f32x4 weight;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        o[i][j][e] = o[i][j][e] * lead;
        const int s = s0 + e;
        float x = s <= t ? expf((float)(L - L_s[s])) * b_s[s] * g[i][j][e] : 0.f;
        weight[e] = s == t ? x + d : x;
      }
      *reinterpret_cast<f32x4*>(q_s + t * kTileRow + s0) = weight;
    }
  }
  stage_tile(k_s, [&](int r) LS_INLINED { return v.at(t0 + r, h); }, n, c0, DV, v_vec != 0, one);
  __syncthreads();
  if (norm_here) {
    float sum = 0.f;
    for (int s = my_part; s < 64; s += 4) sum = sum + q_s[my_t * kTileRow + s];
    sum = fmaf(nq, expf((float)L_s[my_t]), sum);
    sum = sum + __shfl_xor(sum, 1, kWave);
    sum = sum + __shfl_xor(sum, 2, kWave);
    if (my_part == 0 && my_t < n) gates[(t0 + my_t) * H + h].nq = sum;
  }
  const int last_chunk = 2 * wr + 1;   // (the wave's tokens see the first 32 wr + 32 of the chunk at most)
  for (int ch = 0; ch <= last_chunk; ++ch) {
    f32x4 wv[2], vv[2];
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      wv[j] = *reinterpret_cast<const f32x4*>(q_s + (wr * 32 + 16 * j + l16) * kTileRow + 16 * ch + 4 * quad);
      vv[j] = tile_column(k_s, 16 * ch + 4 * quad, wc * 32 + 16 * j + l16);
    }
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int j = 0; j < 2; ++j) Atom<float>::mma(o[i][j], vv[j], wv[i]);
  }
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int t = wr * 32 + 16 * i + l16;
    if (t >= n) continue;
    float* dst = out + (t0 + t) * ldo + (long)h * DV;
#pragma unroll
    for (int j = 0; j < 2; ++j) store4m(dst, c0 + wc * 32 + 16 * j + 4 * quad, DV, out_vec != 0, o[i][j]);
  }
}

// ---------------------------------------------------------------------------
// Gate, then norm in equal parts: y [T][ldy] float times silu(z), divided by its root mean square in each of `parts`
// runs of neighbours (eps inside the root), times weight [inner]; stored as T.  A workgroup a (token, part): thread t
// adds the squares of the elements t, t + 256, ... ascending, then a butterfly over the wave and the waves in order.
// ---------------------------------------------------------------------------
// (PER: gated elements a thread keeps between the sum and the scaling; those of longer parts are formed again)
template <typename T, int PER>
__global__ __launch_bounds__(256) void gated_parts_norm_kernel(const float* __restrict__ y, long ldy, const float* __restrict__ z,
                                                               long ldz, int each, const float* __restrict__ weight, float eps,
                                                               T* __restrict__ out, long ldo) {
  __shared__ float scratch[4];
  const long t = blockIdx.x;
  const int at = blockIdx.y * each;
  const float* y_row = y + t * ldy + at;
  const float* z_row = z + t * ldz + at;
  float mine[PER], gate[PER];
  float part = 0.f;
#pragma unroll
  for (int j = 0; j < PER; ++j) {   // (addresses that are always valid: no branch between the loads)
    const int c = threadIdx.x + 256 * j;
    mine[j] = y_row[c < each ? c : 0];
    gate[j] = z_row[c < each ? c : 0];
  }
#pragma unroll
  for (int j = 0; j < PER; ++j) {
    mine[j] = (int)threadIdx.x + 256 * j < each ? mine[j] * silu_m(gate[j]) : 0.f;
    part = part + mine[j] * mine[j];
  }
  for (int c = threadIdx.x + 256 * PER; c < each; c += 256) {
    const float g = y_row[c] * silu_m(z_row[c]);
    part = part + g * g;
  }
  part = wave_sum(part);
  if ((threadIdx.x & 63) == 0) scratch[threadIdx.x >> 6] = part;
  __syncthreads();
  const float total = ((scratch[0] + scratch[1]) + scratch[2]) + scratch[3];
  const float scale = 1.0f / sqrtf(total / (float)each + eps);
  T* dst = out + t * ldo + at;
#pragma unroll
  for (int j = 0; j < PER; ++j) {
    const int c = threadIdx.x + 256 * j;
    if (c < each) dst[c] = from_f32<T>((mine[j] * scale) * weight[at + c]);
  }
  for (int c = threadIdx.x + 256 * PER; c < each; c += 256)
    dst[c] = from_f32<T>(((y_row[c] * silu_m(z_row[c])) * scale) * weight[at + c]);
}

}  // namespace ls

using namespace ls;

static bool aligned16(const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; }
// rows that move as whole vectors of four: base, row stride, head stride and length all multiples of four floats
static int rows_vec(const float* p, long ld, int each) { return aligned16(p) && ld % 4 == 0 && each % 4 == 0; }

extern "C" int ls_memory_max_rows() { return kMemMaxRows; }
extern "C" int ls_memory_chunk() { return kChunk; }
extern "C" int ls_exp_token_whole() { return kMemWhole * kMemCols; }

extern "C" int ls_conv_gates(const float* raw, long ld, int x_at, int dt_at, int n_tokens, int C, int H, int M, const float* taps,
                             const float* bias, const float* a_log, const float* dt_bias, const int* tok_seq, const int* tok_pos,
                             const void* seqs, int n_seqs, float* state, long state_stride, long ring_at, float* conv, float* gates,
                             void* stream) {
  LS_REQUIRE(n_tokens > 0 && n_seqs > 0 && C > 0 && H > 0 && M >= 1 && x_at >= 0 && dt_at >= 0 && ld >= (long)x_at + C && ld >= (long)dt_at + H,
             "conv_gates: bad sizes (%d channels, %d heads, %d taps)", C, H, M);
  LS_REQUIRE(ring_at >= 0 && state_stride >= ring_at + (long)M * C, "conv_gates: the state holds no ring of %d inputs", M);
  LS_REQUIRE(raw && taps && bias && a_log && dt_bias && tok_seq && tok_pos && seqs && state && conv && gates, "conv_gates: null operand");
  LS_REQUIRE(aligned16(gates), "conv_gates: the gates must be 16-byte aligned");
  hipStream_t s = reinterpret_cast<hipStream_t>(stream);
  const unsigned pieces = (unsigned)((C + 255) / 256);
  hipLaunchKernelGGL(conv_gates_kernel, dim3((n_tokens + kConvTokens - 1) / kConvTokens, pieces + 1), dim3(256), 0, s, raw, ld, x_at,
                     dt_at, n_tokens, C, H, M, taps, bias, a_log, dt_bias, tok_seq, tok_pos, (const SeqMeta*)seqs, state, state_stride,
                     ring_at, conv, (Gate*)gates);
  if (M > 1)
    hipLaunchKernelGGL(conv_ring_kernel, dim3(n_seqs, pieces), dim3(256), 0, s, raw, ld, x_at, C, M, (const SeqMeta*)seqs, state,
                       state_stride, ring_at);
  return check_launch("conv_gates");
}

extern "C" int ls_exp_gates(const float* raw, long ld, int i_at, int f_at, int H, const float* i_bias, const float* f_bias, float cap,
                            const void* seqs, int n_seqs, float* state, long state_stride, long m_at, float* gates, void* stream) {
  LS_REQUIRE(n_seqs > 0 && H > 0 && cap > 0.f && i_at >= 0 && f_at >= 0 && ld >= (long)i_at + H && ld >= (long)f_at + H,
             "exp_gates: bad sizes");
  LS_REQUIRE(m_at >= 0 && state_stride >= m_at + 4L * H, "exp_gates: the state holds no running maxima");
  LS_REQUIRE(raw && i_bias && f_bias && seqs && state && gates && aligned16(gates), "exp_gates: bad operands");
  hipLaunchKernelGGL(exp_gates_kernel, dim3(n_seqs * H), dim3(64), 0, reinterpret_cast<hipStream_t>(stream), raw, ld, i_at, f_at, H,
                     i_bias, f_bias, cap, (const SeqMeta*)seqs, state, state_stride, m_at, (Gate*)gates);
  return check_launch("exp_gates");
}

#define LS_BY_ROWS(CASE_)            \
  if (N <= 32) { CASE_(1) }          \
  else if (N <= 64) { CASE_(2) }     \
  else if (N <= 128) { CASE_(4) }    \
  else { CASE_(8) }

extern "C" int ls_memory_walk(const float* q, long ldq, int q_each, int q_share, const float* k, long ldk, int k_each, int k_share,
                              const float* v, long ldv, int v_each, float* gates, int H, int N, int DV, float q_scale,
                              const float* skip, int norm, const void* seqs, int n_seqs, int longest, float* state,
                              long state_stride, float* out, long ldo, void* stream) {
  LS_REQUIRE(n_seqs > 0 && n_seqs <= 65535 && H > 0 && N > 0 && N <= kMemMaxRows && DV > 0 && q_share > 0 && k_share > 0,
             "memory_walk: bad sizes (%d heads, %d rows of at most %d, %d columns)", H, N, kMemMaxRows, DV);
  LS_REQUIRE(q && k && v && gates && seqs && state && out && ldo >= (long)H * DV && q_each >= N && k_each >= N && v_each >= DV,
             "memory_walk: bad operands");
  LS_REQUIRE(state_stride >= (long)H * N * DV + (norm ? (long)H * N : 0), "memory_walk: the state is too short");
  hipStream_t s = reinterpret_cast<hipStream_t>(stream);
  const HeadRows qr{q, ldq, q_each, q_share}, kr{k, ldk, k_each, k_share}, vr{v, ldv, v_each, 1};
  const int state_vec = DV % 4 == 0 && state_stride % 4 == 0 && aligned16(state);
  const int v_vec = DV % 4 == 0 && rows_vec(v, ldv, v_each);
  const dim3 grid((unsigned)(H * ((DV + kMemCols - 1) / kMemCols)), (unsigned)n_seqs);
#define LS_WALK(R_)                                                                                                       \
  if (norm)                                                                                                               \
    hipLaunchKernelGGL((memory_walk_kernel<R_, true>), grid, dim3(256), 0, s, qr, kr, vr, (Gate*)gates, H, N, DV, q_scale, \
                       skip, (const SeqMeta*)seqs, longest, state, state_stride, state_vec, v_vec, out, ldo);             \
  else                                                                                                                    \
    hipLaunchKernelGGL((memory_walk_kernel<R_, false>), grid, dim3(256), 0, s, qr, kr, vr, (Gate*)gates, H, N, DV, q_scale, \
                       skip, (const SeqMeta*)seqs, longest, state, state_stride, state_vec, v_vec, out, ldo);
  LS_BY_ROWS(LS_WALK)
#undef LS_WALK
  return check_launch("memory_walk");
}

extern "C" int ls_space_token(const float* raw, long ld, int x_at, int dt_at, int C, int G, int M, long ring_at, const float* taps,
                              const float* conv_bias, const float* a_log, const float* dt_bias, const float* skip, int H, int N,
                              int DV, const void* seqs, int n_seqs, float* state, long state_stride, float* out, long ldo,
                              void* stream) {
  LS_REQUIRE(n_seqs > 0 && n_seqs <= 65535 && H > 0 && G > 0 && H % G == 0 && N > 0 && N <= kMemMaxRows && DV > 0 && M >= 1,
             "space_token: bad sizes (%d heads over %d groups, %d rows of at most %d, %d columns, %d taps)", H, G, N, kMemMaxRows, DV, M);
  LS_REQUIRE(C == H * DV + 2 * G * N && ld >= (long)x_at + C && ld >= (long)dt_at + H && x_at >= 0 && dt_at >= 0,
             "space_token: the projections do not fit the rows");
  LS_REQUIRE(ring_at >= (long)H * N * DV && state_stride >= ring_at + (long)M * C && ldo >= (long)H * DV, "space_token: state or output too short");
  LS_REQUIRE(raw && taps && conv_bias && a_log && dt_bias && skip && seqs && state && out, "space_token: null operand");
  hipStream_t s = reinterpret_cast<hipStream_t>(stream);
  const SpaceArgs sp{x_at, dt_at, C, G, M, ring_at, taps, conv_bias, a_log, dt_bias, skip};
  const ExpArgs ex{};
  const int state_vec = DV % 4 == 0 && state_stride % 4 == 0 && aligned16(state);
  const dim3 grid((unsigned)(H * ((DV + kMemCols - 1) / kMemCols)), (unsigned)n_seqs);
#define LS_TOKEN(R_)                                                                                                          \
  hipLaunchKernelGGL((memory_token_kernel<R_, true, false, float>), grid, dim3(256), 0, s, raw, ld, sp, ex, H, N, DV,         \
                     (const SeqMeta*)seqs, state, state_stride, state_vec, (Gate*)nullptr, out, ldo, (float*)nullptr, 0L);
  LS_BY_ROWS(LS_TOKEN)
#undef LS_TOKEN
  return check_launch("space_token");
}

extern "C" int ls_exp_token(const float* raw, long ld, int q_at, int k_at, int v_at, int i_at, int f_at, long m_at,
                            const float* i_bias, const float* f_bias, float cap, float q_scale, int H, int N, int DV,
                            const void* seqs, int n_seqs, float* state, long state_stride, float* gates, float* out, long ldo,
                            int normed_dtype, const float* weight, int g_at, float eps, float denom_eps, void* normed, long ldn,
                            void* stream) {
  // normed (or null): the head's norm and gate in the same launch (ls_exp_token_whole() columns at most); else gates, out
  LS_REQUIRE(!normed || (DV <= kMemWhole * kMemCols && weight && g_at >= 0 && ld >= (long)g_at + (long)H * DV && ldn >= (long)H * DV && eps > 0.f &&
                         (normed_dtype == kF32 || normed_dtype == kBF16)),
             "exp_token: the norm behind takes heads of up to %d columns", kMemWhole * kMemCols);
  LS_REQUIRE(n_seqs > 0 && n_seqs <= 65535 && H > 0 && N > 0 && N <= kMemMaxRows && DV > 0 && cap > 0.f,
             "exp_token: bad sizes (%d heads, %d rows of at most %d, %d columns)", H, N, kMemMaxRows, DV);
  LS_REQUIRE(q_at >= 0 && k_at >= 0 && v_at >= 0 && i_at >= 0 && f_at >= 0 && ld >= (long)q_at + (long)H * N && ld >= (long)k_at + (long)H * N &&
                 ld >= (long)v_at + (long)H * DV && ld >= (long)i_at + H && ld >= (long)f_at + H,
             "exp_token: the projections do not fit the rows");
  LS_REQUIRE(m_at >= (long)H * N * DV + (long)H * N && state_stride >= m_at + 4L * H && (normed || ldo >= (long)H * DV), "exp_token: state or output too short");
  LS_REQUIRE(raw && i_bias && f_bias && seqs && state && (normed || (gates && out)), "exp_token: null operand");
  hipStream_t s = reinterpret_cast<hipStream_t>(stream);
  const SpaceArgs sp{};
  const ExpArgs ex{q_at, k_at, v_at, i_at, f_at, m_at, cap, q_scale, i_bias, f_bias, weight, g_at, eps, denom_eps};
  const int state_vec = DV % 4 == 0 && state_stride % 4 == 0 && aligned16(state);
  const dim3 grid((unsigned)(H * ((DV + kMemCols - 1) / kMemCols)), (unsigned)n_seqs);
  const dim3 whole_grid((unsigned)H, (unsigned)n_seqs), whole_block(256 * (unsigned)((DV + kMemCols - 1) / kMemCols));
#define LS_TOKEN(R_)                                                                                                           \
  if (normed && normed_dtype == kF32)                                                                                          \
    hipLaunchKernelGGL((memory_token_kernel<R_, false, true, float>), whole_grid, whole_block, 0, s, raw, ld, sp, ex, H, N, DV, \
                       (const SeqMeta*)seqs, state, state_stride, state_vec, (Gate*)gates, out, ldo, (float*)normed, ldn);     \
  else if (normed)                                                                                                             \
    hipLaunchKernelGGL((memory_token_kernel<R_, false, true, bf16_t>), whole_grid, whole_block, 0, s, raw, ld, sp, ex, H, N, DV, \
                       (const SeqMeta*)seqs, state, state_stride, state_vec, (Gate*)gates, out, ldo, (bf16_t*)normed, ldn);    \
  else                                                                                                                         \
    hipLaunchKernelGGL((memory_token_kernel<R_, false, false, float>), grid, dim3(256), 0, s, raw, ld, sp, ex, H, N, DV,       \
                       (const SeqMeta*)seqs, state, state_stride, state_vec, (Gate*)gates, out, ldo, (float*)nullptr, 0L);
  LS_BY_ROWS(LS_TOKEN)
#undef LS_TOKEN
  return check_launch("exp_token");
}

extern "C" int ls_memory_chunks(const float* q, long ldq, int q_each, int q_share, const float* k, long ldk, int k_each, int k_share,
                                const float* v, long ldv, int v_each, float* gates, int H, int N, int DV, float q_scale,
                                const float* skip, int norm, const void* seqs, const int* items, int n_items, const int* runs,
                                int n_runs, float* states, long E, float* decays, float* state, long state_stride, float* out,
                                long ldo, void* stream) {
  LS_REQUIRE(n_items > 0 && n_runs > 0 && n_runs <= 65535 && H > 0 && H <= 65535 && N > 0 && N <= kMemMaxRows && DV > 0 && q_share > 0 && k_share > 0,
             "memory_chunks: bad sizes (%d heads, %d rows of at most %d, %d columns)", H, N, kMemMaxRows, DV);
  LS_REQUIRE(q && k && v && gates && seqs && items && runs && states && decays && state && out && ldo >= (long)H * DV &&
                 q_each >= N && k_each >= N && v_each >= DV,
             "memory_chunks: bad operands");
  LS_REQUIRE(E == (long)H * N * DV + (norm ? (long)H * N : 0) && state_stride >= E, "memory_chunks: the state is too short");
  hipStream_t s = reinterpret_cast<hipStream_t>(stream);
  const HeadRows qr{q, ldq, q_each, q_share}, kr{k, ldk, k_each, k_share}, vr{v, ldv, v_each, 1};
  const int q_vec = N % 4 == 0 && rows_vec(q, ldq, q_each), k_vec = N % 4 == 0 && rows_vec(k, ldk, k_each);
  const int v_vec = DV % 4 == 0 && rows_vec(v, ldv, v_each);
  const int state_vec = DV % 4 == 0 && E % 4 == 0 && aligned16(states);
  const int out_vec = DV % 4 == 0 && ldo % 4 == 0 && aligned16(out);
  const unsigned nz = (unsigned)((N + 63) / 64), cz = (unsigned)((DV + 63) / 64);
  hipLaunchKernelGGL(memory_chunk_state_kernel, dim3(n_items, H, nz * cz), dim3(256), 0, s, kr, vr, (const Gate*)gates, H, N, DV,
                     (const SeqMeta*)seqs, items, states, E, decays, norm, k_vec, v_vec, state_vec);
  const bool scan_vec = state_vec && N % 4 == 0 && state_stride % 4 == 0 && aligned16(state);
  if (scan_vec)
    hipLaunchKernelGGL(memory_chunk_scan_kernel<4>, dim3((unsigned)((E / 4 + 255) / 256), n_runs), dim3(256), 0, s, (const SeqMeta*)seqs,
                       runs, states, E, decays, H, N, DV, state, state_stride);
  else
    hipLaunchKernelGGL(memory_chunk_scan_kernel<1>, dim3((unsigned)((E + 255) / 256), n_runs), dim3(256), 0, s, (const SeqMeta*)seqs,
                       runs, states, E, decays, H, N, DV, state, state_stride);
  hipLaunchKernelGGL(memory_chunk_out_kernel, dim3(n_items, H, cz), dim3(256), 0, s, qr, kr, vr, (Gate*)gates, H, N, DV, q_scale, skip,
                     (const SeqMeta*)seqs, items, states, E, norm, q_vec, k_vec, v_vec, state_vec, out_vec, out, ldo);
  return check_launch("memory_chunks");
}

extern "C" int ls_gated_parts_norm(int out_dtype, const float* y, long ldy, const float* z, long ldz, int n_tokens, int inner, int parts,
                                   const float* weight, float eps, void* out, long ldo, void* stream) {
  LS_REQUIRE(n_tokens > 0 && inner > 0 && parts > 0 && parts <= 65535 && inner % parts == 0 && ldy >= inner && ldz >= inner && ldo >= inner && eps > 0.f,
             "gated_parts_norm: %d elements in %d parts", inner, parts);
  LS_REQUIRE(y && z && weight && out, "gated_parts_norm: null operand");
  LS_REQUIRE(out_dtype == kF32 || out_dtype == kBF16, "gated_parts_norm: unknown dtype %d", out_dtype);
  hipStream_t s = reinterpret_cast<hipStream_t>(stream);
  const int each = inner / parts;
#define LS_GATED(T_, PER_)                                                                                                    \
  hipLaunchKernelGGL((gated_parts_norm_kernel<T_, PER_>), dim3(n_tokens, parts), dim3(256), 0, s, y, ldy, z, ldz, each, weight, \
                     eps, (T_*)out, ldo)
#define LS_GATED_BY_SIZE(T_)             \
  if (each <= 256) LS_GATED(T_, 1);      \
  else if (each <= 1024) LS_GATED(T_, 4); \
  else if (each <= 2048) LS_GATED(T_, 8); \
  else LS_GATED(T_, 16);
  if (out_dtype == kF32) { LS_GATED_BY_SIZE(float) } else { LS_GATED_BY_SIZE(bf16_t) }
#undef LS_GATED_BY_SIZE
#undef LS_GATED
  return check_launch("gated_parts_norm");
}
