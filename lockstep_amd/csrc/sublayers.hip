// More kernels of the mixers library: the step of a residual stream whose sublayers are normalised on both sides
// (and, where asked for, replaced by an average over the results of all layers so far), a recurrence of one number a
// channel whose gates read the current token only, and the embedding with position vectors.
//
// Everything here is computed in float whatever the compute dtype T is: T is the type of what a matrix product
// reads next.  Per-row reductions have an order fixed by the row's width alone.

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

// ---------------------------------------------------------------------------
// Between two sublayers.  For a row of the residual stream X (float), in one launch:
//   y = P[0][row] + P[1][row] + ...        (the sublayer's output, left as slice sums; ascending, from +0)
//   x = X[row] + norm(y)                   (post_w null: x = X[row] + y)
//   results[keep][row] = x                 (results null: not kept)
//   x = shares[0] results[0][row] + ... + shares[keep] x      (shares null: x stays)
//   X[row] = x
//   out = norm(x)                          (T; out null: nothing)
// norm(v) = (v - m) / sqrt(mean((v - m)^2) + eps) * w (+ bias, for the last of the two; it may be null) with m the row's mean (`centred`), or 0 without it.
// With a row list the rows rows[r] are read and only `out` is written.
// Thread t of 256 owns the elements 1024 c + 4 t + {0..3}, c ascending; a sum adds them in that order, then a
// butterfly over the wave and the wave sums in wave order.  Slices and results are requested eight at a time (fewer in wide rows).
// ---------------------------------------------------------------------------
constexpr int kStepWidth = 16384;  // the widest row: 16 chunks of 1024 elements stay in registers

__device__ __forceinline__ float step_sum(float v, float* scratch /*[4], used by one sum of the launch*/) {
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0) scratch[threadIdx.x >> 6] = v;
  __syncthreads();
  return ((scratch[0] + scratch[1]) + scratch[2]) + scratch[3];
}

template <int NC>
__device__ __forceinline__ void step_norm(f32x4 (&v)[NC], const f32x4 (&w)[NC], int W, float eps, int centred, float* scratch) {
  if (centred) {
    float part = 0.f;
#pragma unroll
    for (int c = 0; c < NC; ++c)
#pragma unroll
      for (int i = 0; i < 4; ++i) part = part + v[c][i];   // (elements beyond the row are zeros)
    const float mean = step_sum(part, scratch) / (float)W;
#pragma unroll
    for (int c = 0; c < NC; ++c)
#pragma unroll
      for (int i = 0; i < 4; ++i)
        v[c][i] = 1024 * c + 4 * (int)threadIdx.x + i < W ? v[c][i] - mean : 0.f;
  }
  float part = 0.f;
#pragma unroll
  for (int c = 0; c < NC; ++c)
#pragma unroll
    for (int i = 0; i < 4; ++i) part = part + v[c][i] * v[c][i];
  const float scale = 1.0f / sqrtf(step_sum(part, scratch + 4) / (float)W + eps);
#pragma unroll
  for (int c = 0; c < NC; ++c)
#pragma unroll
    for (int i = 0; i < 4; ++i) v[c][i] = (v[c][i] * scale) * w[c][i];
}

// Four elements of a row, zeros beyond it.  VEC: whole vectors at 16-byte addresses, loaded unconditionally (from the
// row's start where the thread has none), so that a run of such loads is in flight together.
template <bool VEC>
__device__ __forceinline__ f32x4 step_load(const float* __restrict__ p, int e, int W) {
  f32x4 v = {0.f, 0.f, 0.f, 0.f};
  if (VEC) {
    const f32x4 got = *reinterpret_cast<const f32x4*>(p + (e < W ? e : 0));
    return e < W ? got : v;
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
    if (e + i < W) v[i] = p[e + i];
  return v;
}

template <bool VEC>
__device__ __forceinline__ void step_store(float* __restrict__ p, int e, int W, const f32x4& v) {
  if (VEC) {
    if (e < W) *reinterpret_cast<f32x4*>(p + e) = v;
    return;
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
    if (e + i < W) p[e + i] = v[i];
}

template <typename T, int NC, bool VEC>
__global__ __launch_bounds__(256) void residual_step_kernel(
    float* __restrict__ X, long ldx, int W, const float* __restrict__ P, int slices, long p_stride,
    const float* __restrict__ post_w, float post_eps, int post_centred, float* __restrict__ results, long r_stride, int keep,
    const float* __restrict__ shares, const float* __restrict__ weight, const float* __restrict__ bias, float eps, int centred,
    T* __restrict__ out, long ld_out, const int* __restrict__ rows) {
  constexpr int BATCH = NC <= 2 ? 8 : NC <= 4 ? 4 : NC <= 8 ? 2 : 1;
  __shared__ float scratch[16];
  const int r_out = blockIdx.x;
  const long row = rows ? rows[r_out] : r_out;
  const int e0 = 4 * (int)threadIdx.x;
  float* xrow = X + row * ldx;
  f32x4 x[NC], y[NC], acc[NC], w[NC], pw[NC];
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    x[c] = step_load<VEC>(xrow, 1024 * c + e0, W);
    y[c] = acc[c] = w[c] = pw[c] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  if (P) {
    const float* p = P + row * W;
    for (int s0 = 0; s0 < slices; s0 += BATCH) {
      f32x4 got[NC][BATCH];
#pragma unroll
      for (int u = 0; u < BATCH; ++u)
#pragma unroll
        for (int c = 0; c < NC; ++c)
          got[c][u] = step_load<VEC>(p + (long)min(s0 + u, slices - 1) * p_stride, 1024 * c + e0, W);
#pragma unroll
      for (int u = 0; u < BATCH; ++u)
        if (s0 + u < slices)
#pragma unroll
          for (int c = 0; c < NC; ++c) y[c] = y[c] + got[c][u];
    }
  }
  if (shares) {   // the results of earlier layers do not wait for this one
    const float* r = results + row * W;
    for (int j0 = 0; j0 < keep; j0 += BATCH) {
      f32x4 got[NC][BATCH];
      float a[BATCH];
#pragma unroll
      for (int u = 0; u < BATCH; ++u) {
        a[u] = shares[min(j0 + u, keep - 1)];
#pragma unroll
        for (int c = 0; c < NC; ++c)
          got[c][u] = step_load<VEC>(r + (long)min(j0 + u, keep - 1) * r_stride, 1024 * c + e0, W);
      }
#pragma unroll
      for (int u = 0; u < BATCH; ++u)
        if (j0 + u < keep)
#pragma unroll
          for (int c = 0; c < NC; ++c) acc[c] = acc[c] + a[u] * got[c][u];
    }
  }
  if (P) {
    if (post_w) {
#pragma unroll
      for (int c = 0; c < NC; ++c) pw[c] = step_load<VEC>(post_w, 1024 * c + e0, W);
      step_norm<NC>(y, pw, W, post_eps, post_centred, scratch);
    }
#pragma unroll
    for (int c = 0; c < NC; ++c) x[c] = x[c] + y[c];
  }
  if (results && !rows)
#pragma unroll
    for (int c = 0; c < NC; ++c) step_store<VEC>(results + keep * r_stride + row * W, 1024 * c + e0, W, x[c]);
  if (shares) {
    const float last = shares[keep];
#pragma unroll
    for (int c = 0; c < NC; ++c) x[c] = acc[c] + last * x[c];
  }
  if ((P || shares) && !rows)
#pragma unroll
    for (int c = 0; c < NC; ++c) step_store<VEC>(xrow, 1024 * c + e0, W, x[c]);
  if (!out) return;
#pragma unroll
  for (int c = 0; c < NC; ++c) w[c] = step_load<VEC>(weight, 1024 * c + e0, W);
  step_norm<NC>(x, w, W, eps, centred, scratch + 8);
  if (bias) {
#pragma unroll
    for (int c = 0; c < NC; ++c) x[c] = x[c] + step_load<VEC>(bias, 1024 * c + e0, W);
  }
  T* dst = out + (long)r_out * ld_out;
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int e = 1024 * c + e0;
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (e + i < W) dst[e + i] = from_f32<T>(x[c][i]);
  }
}

// ---------------------------------------------------------------------------
// A recurrence of one number a channel, whose gates read the current token only.  raw [T][ld] float holds, W channels
// each, a (at a_at), u (at u_at) and g (at g_at); biases a_b, u_b [W]:
//   z = sigmoid(a + a_b);  c = v + 1/2 where v = u + u_b >= 0, else sigmoid(v)
//   S_t = (1 - z) S_(t-1) + z c          out_t = S_t silu(g)  (T)
// state [slots][state_stride] float holds S.  (1 - z is formed as sigmoid(-(a + a_b)).)
//
// A workgroup takes one request and 16 channels, 64 runs of eight tokens at a time: a wave has four runs (16 lanes
// each).  A lane walks its run from zero, which gives the run's product of (1 - z) and its last value, so the state
// behind a run is an affine function of the state in front of it; these are composed over the wave's runs by
// moves between lanes, over the waves through LDS (every lane folds the sixteen waves' pairs itself: one barrier a
// round, two buffers), and the lane walks its run again from the state in front of it.  The operands of the next
// round are requested before the round is worked on.
// ---------------------------------------------------------------------------
template <typename T> struct Gates;
template <> struct Gates<float> {
  static __device__ __forceinline__ float sigmoid(float v) { return 1.0f / (1.0f + expf(-v)); }
};
template <> struct Gates<bf16_t> {   // the hardware's exponential and reciprocal: float32 up to the last places
  static __device__ __forceinline__ float sigmoid(float v) { return __builtin_amdgcn_rcpf(1.0f + __expf(-v)); }
};

template <typename T>
__device__ __forceinline__ void channel_gates(float a, float v, float& keep, float& write) {
  keep = Gates<T>::sigmoid(-a);
  write = Gates<T>::sigmoid(a) * (v >= 0.f ? v + 0.5f : Gates<T>::sigmoid(v));
}

// A barrier between the waves' LDS writes and reads that waits for this wave's LDS operations only: the global
// loads of the next round stay on their way across it.
__device__ __forceinline__ void round_barrier() { __asm__ volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

constexpr int kRunTokens = 8;
constexpr int kRunCols = 16;
constexpr int kRunWaves = 16;
constexpr int kRoundTokens = kRunTokens * 4 * kRunWaves;

template <typename T>
__global__ __launch_bounds__(64 * kRunWaves) void channel_recurrence_kernel(
    const float* __restrict__ raw, long ld, int a_at, int u_at, int g_at, const float* __restrict__ a_b,
    const float* __restrict__ u_b, int W, const SeqMeta* __restrict__ seqs, float* __restrict__ state, long state_stride,
    T* __restrict__ out, long ldo) {
  __shared__ float pairs[2][kRunWaves][kRunCols][2];
  const SeqMeta m = seqs[blockIdx.y];
  if (m.q_len <= 0) return;
  // neighbouring blocks of columns on one XCD (ids go round the eight of them): they share cache lines
  const int blocks = gridDim.x, id = blockIdx.x;
  const int cb = blocks % 8 == 0 ? (id % 8) * (blocks / 8) + id / 8 : id;
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6;
  const int l16 = lane & 15, sub = lane >> 4;
  const int col = cb * kRunCols + l16;
  const bool col_ok = col < W;
  const int at = col_ok ? col : 0;
  const float ab = a_b[at], ub = u_b[at];
  const float* src = raw + (long)m.q_off * ld + at;
  float* mine = state + (long)m.table_row * state_stride + at;
  float carry = *mine;
  const int run0 = (wv * 4 + sub) * kRunTokens;   // first token of the lane's run within a round
  float ra[kRunTokens], ru[kRunTokens], rg[kRunTokens];
  auto request = [&](int t0) LS_INLINED {
#pragma unroll
    for (int i = 0; i < kRunTokens; ++i) {
      const float* p = src + (long)min(t0 + run0 + i, m.q_len - 1) * ld;
      ra[i] = p[a_at];
      ru[i] = p[u_at];
      rg[i] = p[g_at];
    }
  };
  request(0);
  int set = 0;
  for (int t0 = 0; t0 < m.q_len; t0 += kRoundTokens, set ^= 1) {
    float keep[kRunTokens], write[kRunTokens], gate[kRunTokens];
#pragma unroll
    for (int i = 0; i < kRunTokens; ++i) {
      const bool in = t0 + run0 + i < m.q_len;
      channel_gates<T>(ra[i] + ab, ru[i] + ub, keep[i], write[i]);
      keep[i] = in ? keep[i] : 1.0f;
      write[i] = in ? write[i] : 0.f;
      gate[i] = rg[i];
    }
    if (t0 + kRoundTokens < m.q_len) request(t0 + kRoundTokens);
    float A = 1.0f, B = 0.f;
#pragma unroll
    for (int i = 0; i < kRunTokens; ++i) {
      A = keep[i] * A;
      B = fmaf(keep[i], B, write[i]);
    }
    // (A, B) of the runs before this one in the wave, and of the whole wave
    float eA = 1.0f, eB = 0.f, wA = 1.0f, wB = 0.f;
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      const float sA = __shfl(A, 16 * s + l16, kWave), sB = __shfl(B, 16 * s + l16, kWave);
      wB = fmaf(sA, wB, sB);
      wA = sA * wA;
      if (s < 3 && s + 1 == sub) { eA = wA; eB = wB; }
    }
    if (sub == 0) {
      pairs[set][wv][l16][0] = wA;
      pairs[set][wv][l16][1] = wB;
    }
    round_barrier();
    float front = 0.f;
#pragma unroll
    for (int s = 0; s < kRunWaves; ++s) {
      front = s == wv ? carry : front;
      carry = fmaf(pairs[set][s][l16][0], carry, pairs[set][s][l16][1]);
    }
    float S = fmaf(eA, front, eB);
#pragma unroll
    for (int i = 0; i < kRunTokens; ++i) {
      S = fmaf(keep[i], S, write[i]);
      const int t = t0 + run0 + i;
      if (t < m.q_len && col_ok)
        out[(long)(m.q_off + t) * ldo + col] = from_f32<T>(S * (gate[i] * Gates<T>::sigmoid(gate[i])));
    }
  }
  if (threadIdx.x < kRunCols && col_ok) *mine = carry;
}

// A step of single tokens: a thread a channel of a request.
template <typename T>
__global__ __launch_bounds__(64) void channel_recurrence_token_kernel(
    const float* __restrict__ raw, long ld, int a_at, int u_at, int g_at, const float* __restrict__ a_b,
    const float* __restrict__ u_b, int W, const SeqMeta* __restrict__ seqs, float* __restrict__ state, long state_stride,
    T* __restrict__ out, long ldo) {
  const int col = blockIdx.x * 64 + threadIdx.x;
  if (col >= W) return;
  const SeqMeta m = seqs[blockIdx.y];
  const float* src = raw + (long)m.q_off * ld + col;
  float* mine = state + (long)m.table_row * state_stride + col;
  const float g = src[g_at];
  float keep, write;
  channel_gates<T>(src[a_at] + a_b[col], src[u_at] + u_b[col], keep, write);
  const float S = fmaf(keep, *mine, write);
  *mine = S;
  out[(long)m.q_off * ldo + col] = from_f32<T>(S * (g * Gates<T>::sigmoid(g)));
}

// ---------------------------------------------------------------------------
// Embedding with position vectors: out[t] = table[token] * scale + v(p), v(p)[2i] = sin(p freq[i]), v(p)[2i+1] =
// cos(p freq[i]), freq [(width + 1) / 2] double.  The angle is formed and brought into (-pi, pi] in double, so its
// sine is good to float's last place at any position.
// ---------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void embed_positions_kernel(const int* __restrict__ tokens, const int* __restrict__ tok_pos,
                                                              const T* __restrict__ table, int vocab,
                                                              const double* __restrict__ freq, float* __restrict__ out,
                                                              int width, long ld_out, float scale) {
  const int t = blockIdx.x;
  const int id = tokens[t];
  const bool ok = id >= 0 && id < vocab;
  const double pos = (double)tok_pos[t];
  const T* row = table + (long)(ok ? id : 0) * width;
  float* dst = out + (long)t * ld_out;
  constexpr double kTurn = 6.283185307179586476925286766559;
  for (int i = threadIdx.x; 2 * i < width; i += 256) {
    const double angle = pos * freq[i];
    const float a = (float)(angle - kTurn * rint(angle * (1.0 / kTurn)));
    float s, c;
    sincosf(a, &s, &c);
    dst[2 * i] = ok ? to_f32(row[2 * i]) * scale + s : 0.f;
    if (2 * i + 1 < width) dst[2 * i + 1] = ok ? to_f32(row[2 * i + 1]) * scale + c : 0.f;
  }
}

}  // namespace ls

using namespace ls;

extern "C" int ls_residual_step_max_width() { return kStepWidth; }

extern "C" int ls_residual_step(int dtype, float* X, long ldx, int width, const float* P, int slices, int p_rows,
                                const float* post_w, float post_eps, int post_centred, float* results, int r_rows, int keep,
                                const float* shares, const float* weight, const float* bias, float eps, int centred, void* out, long ld_out,
                                const int* rows, int n_rows, void* stream) {
  LS_REQUIRE(n_rows > 0 && width > 0 && width <= kStepWidth && ldx >= width && X, "residual_step: rows of %d elements (at most %d)",
             width, kStepWidth);
  LS_REQUIRE(P || results || out, "residual_step: nothing to do");
  LS_REQUIRE(!P || (slices > 0 && p_rows > 0), "residual_step: bad slice sums");
  LS_REQUIRE(!post_w || (P && post_eps > 0.f), "residual_step: a norm of the sublayer's output needs its slices and eps");
  LS_REQUIRE(!results || (r_rows > 0 && keep >= 0), "residual_step: bad results");
  LS_REQUIRE(!shares || results, "residual_step: shares need results");
  LS_REQUIRE(!out || (weight && ld_out >= width && eps > 0.f), "residual_step: an output needs a weight and eps");
  LS_REQUIRE(!rows || out, "residual_step: with a row list only the output is written");
  LS_REQUIRE(dtype == kF32 || dtype == kBF16, "residual_step: unknown dtype %d", dtype);
  hipStream_t s = reinterpret_cast<hipStream_t>(stream);
  auto aligned = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  const bool vec = width % 4 == 0 && ldx % 4 == 0 && aligned(X) && aligned(P) && aligned(post_w) && aligned(results) &&
                   aligned(weight) && aligned(bias);
  const long p_stride = (long)p_rows * width, r_stride = (long)r_rows * width;
#define LS_STEP(T_, NC_, VEC_)                                                                                          \
  hipLaunchKernelGGL((residual_step_kernel<T_, NC_, VEC_>), dim3(n_rows), dim3(256), 0, s, X, ldx, width, P, slices,    \
                     p_stride, post_w, post_eps, post_centred, results, r_stride, keep, shares, weight, bias, eps, centred, \
                     (T_*)out, ld_out, rows)
#define LS_STEP_VEC(T_, NC_) \
  if (vec) LS_STEP(T_, NC_, true); else LS_STEP(T_, NC_, false)
#define LS_STEP_WIDTH(T_)                         \
  if (width <= 1024) { LS_STEP_VEC(T_, 1); }      \
  else if (width <= 2048) { LS_STEP_VEC(T_, 2); } \
  else if (width <= 4096) { LS_STEP_VEC(T_, 4); } \
  else if (width <= 8192) { LS_STEP_VEC(T_, 8); } \
  else { LS_STEP_VEC(T_, 16); }
  if (dtype == kF32) { LS_STEP_WIDTH(float) } else { LS_STEP_WIDTH(bf16_t) }
#undef LS_STEP_WIDTH
#undef LS_STEP_VEC
#undef LS_STEP
  return check_launch("residual_step");
}

extern "C" int ls_channel_recurrence(int dtype, const float* raw, long ld, int a_at, int u_at, int g_at, const float* a_b,
                                     const float* u_b, int width, const void* seqs, int n_seqs, int single_tokens,
                                     float* state, long state_stride, void* out, long ldo, void* stream) {
  LS_REQUIRE(n_seqs > 0 && width > 0 && state_stride >= width && ldo >= width, "channel_recurrence: bad sizes");
  LS_REQUIRE(a_at >= 0 && u_at >= 0 && g_at >= 0 && ld >= (long)a_at + width && ld >= (long)u_at + width && ld >= (long)g_at + width,
             "channel_recurrence: the projections do not fit the rows");
  LS_REQUIRE(raw && a_b && u_b && seqs && state && out, "channel_recurrence: null operand");
  LS_REQUIRE(n_seqs <= 65535, "channel_recurrence: %d requests in one step", n_seqs);
  LS_REQUIRE(dtype == kF32 || dtype == kBF16, "channel_recurrence: unknown dtype %d", dtype);
  hipStream_t s = reinterpret_cast<hipStream_t>(stream);
#define LS_CHANNEL(KERNEL_, T_, COLS_, THREADS_)                                                                      \
  hipLaunchKernelGGL(KERNEL_<T_>, dim3((width + COLS_ - 1) / COLS_, n_seqs), dim3(THREADS_), 0, s, raw, ld, a_at, u_at, g_at, \
                     a_b, u_b, width, (const SeqMeta*)seqs, state, state_stride, (T_*)out, ldo)
  if (single_tokens) {
    if (dtype == kF32) LS_CHANNEL(channel_recurrence_token_kernel, float, 64, 64);
    else LS_CHANNEL(channel_recurrence_token_kernel, bf16_t, 64, 64);
  } else {
    if (dtype == kF32) LS_CHANNEL(channel_recurrence_kernel, float, kRunCols, 64 * kRunWaves);
    else LS_CHANNEL(channel_recurrence_kernel, bf16_t, kRunCols, 64 * kRunWaves);
  }
#undef LS_CHANNEL
  return check_launch("channel_recurrence");
}

extern "C" int ls_embed_positions(int dtype, const int* tokens, const int* tok_pos, const void* table, int vocab,
                                  const double* freq, float* out, int n_tokens, int width, long ld_out, float scale,
                                  void* stream) {
  LS_REQUIRE(n_tokens > 0 && vocab > 0 && width > 0 && ld_out >= width, "embed_positions: bad sizes");
  LS_REQUIRE(tokens && tok_pos && table && freq && out, "embed_positions: null operand");
  hipStream_t s = reinterpret_cast<hipStream_t>(stream);
  if (dtype == kF32)
    hipLaunchKernelGGL(embed_positions_kernel<float>, dim3(n_tokens), dim3(256), 0, s, tokens, tok_pos, (const float*)table,
                       vocab, freq, out, width, ld_out, scale);
  else if (dtype == kBF16)
    hipLaunchKernelGGL(embed_positions_kernel<bf16_t>, dim3(n_tokens), dim3(256), 0, s, tokens, tok_pos, (const bf16_t*)table,
                       vocab, freq, out, width, ld_out, scale);
  else
    return fail("embed_positions: unknown dtype %d", dtype);
  return check_launch("embed_positions");
}
