// A feed-forward of many small experts of which each token uses a few (routing on the device, no
// word of it read by the host):
//
//   z[t]        = router logits of token t (float, computed by the caller's matrix product) + bias
//   chosen(t)   = the `top` experts with the largest z[t] (the lower index wins a tie), in that order
//   w[t, k]     = softmax over the chosen logits alone
//                 (scoring 1: the sigmoid of each; scoring 2: the choice is made by softmax(z) + correction, within the
//                 best groups of experts, and the weights are the chosen softmax(z) divided by their sum)
//   expert e    : y = act(W_gate[e] x, W_up[e] x),  out = W_down[e] y
//                 act(g, u) = g' sigmoid(alpha g') (u' + shift),  g' = min(g, limit),  u' = clamp(u, -limit, limit)
//                 (an infinite limit, alpha 1 and shift 0: the plain gated unit silu(g) u)
//   P[k][t]     = w[t, k] * expert chosen(t)[k] (x[t])        (float; the caller adds the slices in order)
//                 (experts from the `real`-th on have no weights: they return x[t] itself)
//
// (1) route: a wave a token picks the experts and their weights.  (2) group: the (token, choice) pairs
// are put in the order of their experts (a stable counting sort: a wave an expert counts its pairs by
// ballots, then places them; one workgroup does (1) and (2) for a step of few tokens), and every
// expert's pairs are cut into tiles of ROWS rows; the tile list has a fixed capacity that depends on the sizes only, unused
// tiles are marked.  (3) the gate and up products of every tile with the activation as epilogue; (4)
// the down products, scaled and scattered to P.  Products use the 16x16 MFMA atom with the weight
// rows as first operand (a lane ends with four consecutive output columns of one row); a row's
// contraction is one chain over ascending K from zero, so its bits do not depend on the tile it is in
// or on what else is in the step.  A weight fragment is loaded once and multiplied with all RT row
// tiles of a wave.

#include "common.h"

#include <type_traits>

namespace ls {

constexpr int kMaxTop = 16;

__device__ __forceinline__ float sigmoid_e(float x) { return 1.0f / (1.0f + expf(-x)); }

// ---------------------------------------------------------------------------
// (1) A wave a token.  Lane l holds the logits of experts l, l + 64, ...; a pick is the best of every lane's
// best (the larger value, then the lower index), found by exchanges across the wave; lane k < top keeps the
// k-th pick.  expert [T][top] int, weight [T][top] float.
// ---------------------------------------------------------------------------
constexpr int kMaxPerLane = 8;   // experts a lane holds: up to 512 experts

// scoring 0: the weights are the softmax over the chosen logits; 1: each chosen expert weighs the sigmoid of its own
// logit, and nothing is renormalised (the sigmoid grows with the logit, so the largest logits are the largest scores).
// scoring 2: scores s = softmax over all E logits; the choice goes by s + correction, among the experts of the `keep` groups
// (of `groups` equal runs of neighbours) whose largest choice score is largest; the weights are the chosen s divided by
// their sum (+ kShareEps).
constexpr float kShareEps = 1e-20f;

struct Choice {
  int scoring, groups, keep;
  const float* correction;   // [E], scoring 2
};

// A lane's (value, index) against those of the lane that a data-parallel move inside its row of sixteen names; the larger
// value stays, the lower index winning a tie (0x7fffffff: none).
__device__ __forceinline__ void keep_better(float& v, int& e, float ov, int oe) {
  const bool take = oe != 0x7fffffff && (e == 0x7fffffff || ov > v || (ov == v && oe < e));
  v = take ? ov : v;
  e = take ? oe : e;
}
template <int CTRL>
__device__ __forceinline__ void keep_better_of(float& v, int& e) {
  keep_better(v, e, __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), CTRL, 0xF, 0xF, true)),
              __builtin_amdgcn_mov_dpp(e, CTRL, 0xF, 0xF, true));
}

// A lane's entries of a vector over the experts (null: zeros).
template <int PL>
__device__ __forceinline__ void lane_entries(const float* __restrict__ of, int E, int lane, float (&mine)[PL]) {
#pragma unroll
  for (int m = 0; m < PL; ++m) mine[m] = of && lane + 64 * m < E ? of[lane + 64 * m] : 0.f;
}

// PL: experts a lane holds; bias and correction: their entries
template <int PL>
__device__ __forceinline__ void pick_top(const float* __restrict__ row, const float (&bias)[PL], const float (&correction)[PL],
                                         int E, int top, int lane, int* __restrict__ picked, float* __restrict__ share,
                                         const Choice& how) {
  float mine[PL], score[PL];
#pragma unroll
  for (int m = 0; m < PL; ++m) {
    const int e = lane + 64 * m;
    mine[m] = e < E ? row[e] + bias[m] : 0.f;
    score[m] = 0.f;
  }
  // the largest of every lane's open experts, the lower index winning a tie (0x7fffffff: none is open)
  auto largest = [&](unsigned closed, float& best_v, int& best) LS_INLINED {
    best_v = 0.f;
    best = 0x7fffffff;
#pragma unroll
    for (int m = 0; m < PL; ++m) {
      const int e = lane + 64 * m;
      if (e < E && !((closed >> m) & 1u) && (best == 0x7fffffff || mine[m] > best_v)) {
        best_v = mine[m];
        best = e;
      }
    }
    // pairs, pairs of pairs, the mirror image of the half row and of the row (after each, the lanes that met agree), then
    // the rows of sixteen
    keep_better_of<0xB1>(best_v, best);
    keep_better_of<0x4E>(best_v, best);
    keep_better_of<0x141>(best_v, best);
    keep_better_of<0x140>(best_v, best);
#pragma unroll
    for (int step = 16; step < 64; step <<= 1) keep_better(best_v, best, __shfl_xor(best_v, step, kWave), __shfl_xor(best, step, kWave));
  };
  unsigned taken = 0;
  if (how.scoring == 2) {
    float top_z;
    int at;
    largest(0u, top_z, at);
    float part = 0.f;
#pragma unroll
    for (int m = 0; m < PL; ++m) {
      score[m] = lane + 64 * m < E ? expf(mine[m] - top_z) : 0.f;
      part = part + score[m];
    }
    const float inv = 1.0f / wave_sum(part);
#pragma unroll
    for (int m = 0; m < PL; ++m) {
      score[m] = score[m] * inv;
      if (lane + 64 * m < E) mine[m] = score[m] + correction[m];
    }
    if (how.keep < how.groups) {   // the groups, best first: every pick closes its group for the next one
      const int each = E / how.groups;
      unsigned open = 0;
      for (int g = 0; g < how.keep; ++g) {
        float v;
        int best;
        largest(open, v, best);
#pragma unroll
        for (int m = 0; m < PL; ++m)
          if ((lane + 64 * m) / each == best / each) open |= 1u << m;
      }
      taken = ~open;
    }
  }
  int my_pick = 0;
  float my_value = 0.f, first = 0.f;
  for (int k = 0; k < top; ++k) {
    float best_v;
    int best;
    largest(taken, best_v, best);
    if ((best & 63) == lane) taken |= 1u << (best >> 6);
    if (k == 0) first = best_v;
    if (how.scoring == 2) {   // (the weight is the score without the correction)
      float held = 0.f;
#pragma unroll
      for (int m = 0; m < PL; ++m) held = (best >> 6) == m ? score[m] : held;
      best_v = __shfl(held, best & 63, kWave);
    }
    if (lane == k) {
      my_pick = best;
      my_value = best_v;
    }
  }
  if (how.scoring == 2) {
    const float sum = wave_sum(lane < top ? my_value : 0.f);
    if (lane < top) {
      picked[lane] = my_pick;
      share[lane] = my_value / (sum + kShareEps);
    }
    return;
  }
  const float ex = lane < top ? expf(my_value - first) : 0.f;   // (the first pick is the largest)
  const float sum = wave_sum(ex);
  if (lane < top) {
    picked[lane] = my_pick;
    share[lane] = how.scoring == 1 ? sigmoid_e(my_value) : ex / sum;
  }
}

// The experts of a token come from a table instead of a router: row token_id of table [vocab][top] names them (its
// entries differ), and every one weighs 1 / top.
__global__ __launch_bounds__(256) void route_table_kernel(const int* __restrict__ token_ids, const int* __restrict__ table,
                                                          int n_tokens, int top, int* __restrict__ expert,
                                                          float* __restrict__ weight) {
  const long pair = (long)blockIdx.x * 256 + threadIdx.x;
  if (pair >= (long)n_tokens * top) return;
  expert[pair] = table[(long)token_ids[pair / top] * top + pair % top];
  weight[pair] = 1.0f / (float)top;
}

template <int PL>
__global__ __launch_bounds__(256) void route_topk_kernel(const float* __restrict__ z, long ldz,
                                                         const float* __restrict__ bias, int n_tokens, int E, int top,
                                                         int* __restrict__ expert, float* __restrict__ weight, Choice how) {
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (t >= n_tokens) return;
  const int lane = threadIdx.x & 63;
  float own_bias[PL], own_correction[PL];
  lane_entries<PL>(bias, E, lane, own_bias);
  lane_entries<PL>(how.correction, E, lane, own_correction);
  pick_top<PL>(z + (long)t * ldz, own_bias, own_correction, E, top, lane, expert + (long)t * top, weight + (long)t * top, how);
}

// ---------------------------------------------------------------------------
// (2) order [P]: the pairs (token * top + choice) sorted by expert, stable.  tiles [cap][4]: expert (-1: unused),
// first place in order, rows, 0.  A wave an expert: it counts its pairs by ballots, adds up the counts of the
// experts before it, writes its tiles and places its pairs.  Many pairs: two launches of a wave an expert
// (count; place).  Few: one workgroup that also picks the experts, with the picks and counts in LDS.
// ---------------------------------------------------------------------------
__device__ __forceinline__ int count_pairs(const int* expert, int P, int e, int lane) {
  int n = 0;
  for (int p0 = 0; p0 < P; p0 += 256) {   // (four loads requested together)
    int got[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) got[u] = p0 + 64 * u + lane < P ? expert[p0 + 64 * u + lane] : -1;
#pragma unroll
    for (int u = 0; u < 4; ++u) n += __popcll(__ballot(got[u] == e));
  }
  return n;
}

__device__ __forceinline__ void place_pairs(const int* expert, const int* counts, int P, int E, int e, int lane,
                                            int rows_a_tile, int* __restrict__ order, int* __restrict__ tiles, int cap) {
  int base = 0, tile = 0;
  for (int j0 = 0; j0 < e; j0 += 64) {   // (sums of whole numbers: any order)
    const int c = j0 + lane < e ? counts[j0 + lane] : 0;
    int b = c, t = (c + rows_a_tile - 1) / rows_a_tile;
#pragma unroll
    for (int step = 1; step < 64; step <<= 1) {
      b += __shfl_xor(b, step, kWave);
      t += __shfl_xor(t, step, kWave);
    }
    base += b;
    tile += t;
  }
  const int n = counts[e];
  for (int i = lane; i * rows_a_tile < n; i += 64) {
    if (tile + i < cap) {
      tiles[4 * (tile + i)] = e;
      tiles[4 * (tile + i) + 1] = base + i * rows_a_tile;
      tiles[4 * (tile + i) + 2] = min(rows_a_tile, n - i * rows_a_tile);
      tiles[4 * (tile + i) + 3] = 0;
    }
  }
  if (e == E - 1) {
    const int used = tile + (n + rows_a_tile - 1) / rows_a_tile;
    for (int i = used + lane; i < cap; i += 64) {
      tiles[4 * i] = -1;
      tiles[4 * i + 1] = tiles[4 * i + 2] = tiles[4 * i + 3] = 0;
    }
  }
  int at = base;
  for (int p0 = 0; p0 < P; p0 += 256) {
    int got[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) got[u] = p0 + 64 * u + lane < P ? expert[p0 + 64 * u + lane] : -1;
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const bool mine = got[u] == e;
      const unsigned long long votes = __ballot(mine);
      if (mine) order[at + __popcll(votes & ((1ull << lane) - 1ull))] = p0 + 64 * u + lane;
      at += __popcll(votes);
    }
  }
}

__global__ __launch_bounds__(64) void route_count_kernel(const int* __restrict__ expert, int P, int* __restrict__ counts) {
  const int n = count_pairs(expert, P, blockIdx.x, threadIdx.x);
  if (threadIdx.x == 0) counts[blockIdx.x] = n;
}

__global__ __launch_bounds__(64) void route_place_kernel(const int* __restrict__ expert, const int* __restrict__ counts,
                                                         int P, int E, int rows_a_tile, int* __restrict__ order,
                                                         int* __restrict__ tiles, int cap) {
  place_pairs(expert, counts, P, E, blockIdx.x, threadIdx.x, rows_a_tile, order, tiles, cap);
}

// A barrier between LDS writes and reads that waits for this wave's LDS operations only: loads from memory (and stores
// to it) stay on their way across it.
__device__ __forceinline__ void lds_barrier() { __asm__ volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

constexpr int kSmallPairs = 512, kSmallExperts = 512;   // what the one-workgroup kernel keeps in LDS

constexpr int kProductTiles = 8;    // tiles of 16 experts whose logits the one-workgroup kernel forms itself

// PRODUCT: the logits come from up to 16 rows of x and the router's matrix [E][K] instead of z
template <int PL, typename T, bool PRODUCT>
__global__ __launch_bounds__(1024) void route_small_kernel(const float* __restrict__ z, long ldz,
                                                           const float* __restrict__ bias, int n_tokens, int E, int top,
                                                           int rows_a_tile, int* __restrict__ expert,
                                                           float* __restrict__ weight, int* __restrict__ order,
                                                           int* __restrict__ tiles, int cap,
                                                           const int* __restrict__ token_ids, const int* __restrict__ table,
                                                           Choice how, const T* __restrict__ x, long ldx,
                                                           const T* __restrict__ w_router, int K) {
  __shared__ int picks_s[kSmallPairs];
  __shared__ float share_s[kSmallPairs];
  __shared__ int counts_s[kSmallExperts];
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int P = n_tokens * top;
  float own_bias[PL], own_correction[PL];
  lane_entries<PL>(bias, E, lane, own_bias);
  lane_entries<PL>(how.correction, E, lane, own_correction);
  if constexpr (PRODUCT) {   // the logits first: z = x W^T, the column tiles and cuts of K dealt to the sixteen waves
    __shared__ f32x4 sums_s[16][64];
    __shared__ float z_s[16][16 * kProductTiles];
    constexpr int VEC = Atom<T>::VEC, KC = Atom<T>::KCHUNK, U = 8;
    const int l16 = lane & 15, quad = lane >> 4;
    const int tiles16 = (E + 15) / 16, cuts = 16 / tiles16;
    const int ct = w % tiles16, cut = w / tiles16;
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    if (cut < cuts) {
      const bool w_ok = 16 * ct + l16 < E, x_ok = l16 < n_tokens;
      const T* w_row = w_router + (long)(w_ok ? 16 * ct + l16 : 0) * K;
      const T* x_row = x + (long)(x_ok ? l16 : 0) * ldx;
      const int each = (K + KC * cuts - 1) / (KC * cuts) * KC;
      const int hi = min(K, (cut + 1) * each);
      for (int k0 = cut * each; k0 < hi; k0 += U * KC) {
        typename Atom<T>::vec_t a[U], b[U];
#pragma unroll
        for (int u = 0; u < U; ++u) {
          a[u] = load_vec<T>(w_row, 0, k0 + u * KC + VEC * quad, hi, 0, w_ok, true);
          b[u] = load_vec<T>(x_row, 0, k0 + u * KC + VEC * quad, hi, 0, x_ok, true);
        }
#pragma unroll
        for (int u = 0; u < U; ++u) Atom<T>::mma(acc, a[u], b[u]);
      }
    }
    sums_s[w][lane] = acc;
    lds_barrier();
    if (w < tiles16) {   // (the cuts in ascending order)
      f32x4 sum = sums_s[w][lane];
      for (int o = 1; o < cuts; ++o) sum = sum + sums_s[w + o * tiles16][lane];
#pragma unroll
      for (int i = 0; i < 4; ++i) z_s[l16][16 * w + 4 * quad + i] = sum[i];
    }
    lds_barrier();
    z = &z_s[0][0];
    ldz = 16 * kProductTiles;
  }
  if (table) {   // the picks are looked up, not chosen
    for (int pair = threadIdx.x; pair < P; pair += 1024) {
      picks_s[pair] = table[(long)token_ids[pair / top] * top + pair % top];
      share_s[pair] = 1.0f / (float)top;
    }
  }
  for (int t = w; t < n_tokens && !table; t += 16)
    pick_top<PL>(z + (long)t * ldz, own_bias, own_correction, E, top, lane, picks_s + t * top, share_s + t * top, how);
  lds_barrier();
  for (int pair = threadIdx.x; pair < P; pair += 1024) {
    expert[pair] = picks_s[pair];
    weight[pair] = share_s[pair];
  }
  for (int e = w; e < E; e += 16) {
    const int n = count_pairs(picks_s, P, e, lane);
    if (lane == 0) counts_s[e] = n;
  }
  lds_barrier();
  for (int e = w; e < E; e += 16) place_pairs(picks_s, counts_s, P, E, e, lane, rows_a_tile, order, tiles, cap);
}

// ---------------------------------------------------------------------------
// (3) act [P][ldy] (T) = act(x[token] W_gate[e]^T, x[token] W_up[e]^T) for the pairs of every tile, in the
// order of `order`.  w_gate, w_up [E][F][K].  A workgroup: one tile, four waves with 16 columns of F each.
// ---------------------------------------------------------------------------
// An expert that every token uses, worked on beside the routed ones in the launches of small steps: work items from `at`
// on are tiles of 16 tokens.  w_gate_up holds its rows interleaved in tiles of 16 (gate, up, gate, ...; the last tile padded
// with zeros), w_down [N][F]; the plain gated unit silu(g) u; act [n_tokens][ldy] scratch, out [n_tokens][N] float.
template <typename T>
struct SharedExpert {
  const T* w_gate_up;
  const T* w_down;
  int F, at;   // at: the routed experts' work items (0x7fffffff: there is no such expert)
  T* act;
  long ldy;
  float* out;
};

template <typename T, int RT, int KS>
__global__ __launch_bounds__(256) void experts_gate_up_kernel(const T* __restrict__ x, long ldx,
                                                              const T* __restrict__ w_gate, const T* __restrict__ w_up,
                                                              int F, int K, int top, const int* __restrict__ order,
                                                              const int* __restrict__ tiles, float limit, float alpha, float shift,
                                                              const float* __restrict__ in_weight, T* __restrict__ act, long ldy,
                                                              int real, int n_tokens, SharedExpert<T> sh) {
  // in_weight (or null): a pair's routing weight multiplies the expert's input, w * x, so both products are scaled
  // by it before the gated unit (the down product then adds the expert's output as it is)
  constexpr int VEC = Atom<T>::VEC, KC = Atom<T>::KCHUNK;
  const bool all = KS > 1 && (int)blockIdx.x >= sh.at;   // (the same for the whole workgroup)
  const int e = all ? 0 : tiles[4 * blockIdx.x];
  if (e < 0 || e >= real) return;   // (an expert that returns its input has nothing to multiply)
  const int first = all ? 16 * ((int)blockIdx.x - sh.at) : tiles[4 * blockIdx.x + 1];
  const int rows = all ? min(16, n_tokens - first) : tiles[4 * blockIdx.x + 2];
  if (all) F = sh.F;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int l16 = lane & 15, quad = lane >> 4;
  // KS 1: the four waves take 16 columns each.  KS 4 (few rows): they take a quarter of K each for the same 16
  // columns, so that all of a wave's operands are on their way at once, and their sums are added in wave order.
  const int col0 = KS == 1 ? (blockIdx.y * 4 + w) * 16 : blockIdx.y * 16;
  if (col0 >= F) return;
  const bool w_ok = all || col0 + l16 < F;
  const T* g_row = all ? sh.w_gate_up + (long)(2 * col0 + l16) * K : w_gate + ((long)e * F + (w_ok ? col0 + l16 : 0)) * K;
  const T* u_row = all ? g_row + 16L * K : w_up + ((long)e * F + (w_ok ? col0 + l16 : 0)) * K;
  const T* x_row[RT];
  bool x_ok[RT];
#pragma unroll
  for (int r = 0; r < RT; ++r) {
    x_ok[r] = 16 * r + l16 < rows;
    const int token = all ? first + l16 : (x_ok[r] ? order[first + 16 * r + l16] : 0) / top;
    x_row[r] = x + (long)(x_ok[r] ? token : 0) * ldx;
  }
  f32x4 acc_g[RT], acc_u[RT];
#pragma unroll
  for (int r = 0; r < RT; ++r) acc_g[r] = acc_u[r] = f32x4{0.f, 0.f, 0.f, 0.f};
  const bool aligned = K % VEC == 0;
  // the operands of U chunks are requested together, then multiplied in ascending order
  constexpr int U = RT == 1 ? 8 : 4;
  const int k_each = KS == 1 ? K : (K + KC * KS - 1) / (KC * KS) * KC;
  const int k_lo = KS == 1 ? 0 : w * k_each, k_hi = KS == 1 ? K : min(K, k_lo + k_each);
  for (int k0 = k_lo; k0 < k_hi; k0 += U * KC) {
    typename Atom<T>::vec_t a_g[U], a_u[U], b[U][RT];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = k0 + u * KC + VEC * quad;
      a_g[u] = load_vec<T>(g_row, 0, k, k_hi, 0, w_ok, aligned);
      a_u[u] = load_vec<T>(u_row, 0, k, k_hi, 0, w_ok, aligned);
#pragma unroll
      for (int r = 0; r < RT; ++r) b[u][r] = load_vec<T>(x_row[r], 0, k, k_hi, 0, x_ok[r], aligned);
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int r = 0; r < RT; ++r) {
        Atom<T>::mma(acc_g[r], a_g[u], b[u][r]);
        Atom<T>::mma(acc_u[r], a_u[u], b[u][r]);
      }
  }
  if constexpr (KS > 1) {
    __shared__ f32x4 sums_s[KS][2][RT][64];
#pragma unroll
    for (int r = 0; r < RT; ++r) {
      sums_s[w][0][r][lane] = acc_g[r];
      sums_s[w][1][r][lane] = acc_u[r];
    }
    __syncthreads();
    if (w != 0) return;
#pragma unroll
    for (int r = 0; r < RT; ++r)
#pragma unroll
      for (int o = 1; o < KS; ++o)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          acc_g[r][i] = acc_g[r][i] + sums_s[o][0][r][lane][i];
          acc_u[r][i] = acc_u[r][i] + sums_s[o][1][r][lane][i];
        }
  }
#pragma unroll
  for (int r = 0; r < RT; ++r) {
    if (!x_ok[r]) continue;
    T* dst = all ? sh.act + (long)(first + l16) * sh.ldy : act + (long)(first + 16 * r + l16) * ldy;
    const float wt = in_weight && !all ? in_weight[order[first + 16 * r + l16]] : 1.0f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int c = col0 + 4 * quad + i;
      if (c < F) {
        if (all) {
          dst[c] = from_f32<T>((acc_g[r][i] * sigmoid_e(acc_g[r][i])) * acc_u[r][i]);
          continue;
        }
        const float g = fminf(acc_g[r][i] * wt, limit);
        const float u = fminf(fmaxf(acc_u[r][i] * wt, -limit), limit);
        dst[c] = from_f32<T>((g * sigmoid_e(alpha * g)) * (u + shift));
      }
    }
  }
}

// A tile of an expert that returns its input: P[choice][token][c] = share * x[token][c] for the columns [c0, c1), the
// routing weight multiplying the input or the output alike.
template <typename T>
__device__ __forceinline__ void pass_input(const T* __restrict__ x, long ldx, const float* __restrict__ share, int first, int rows,
                                           int c0, int c1, int top, int n_tokens, int N, const int* __restrict__ order,
                                           float* __restrict__ P) {
  const int width = c1 - c0;
  for (int i = threadIdx.x; i < rows * width; i += 256) {
    const int pair = order[first + i / width], c = c0 + i % width;
    P[((long)(pair % top) * n_tokens + pair / top) * N + c] = share[pair] * to_f32(x[(long)(pair / top) * ldx + c]);
  }
}

// ---------------------------------------------------------------------------
// (4) P[choice][token][:] = weight[pair] * (act[place] W_down[e]^T).  w_down [E][N][F]; P [top][n_tokens][N] float.
// ---------------------------------------------------------------------------
template <typename T, int RT, int KS>
__global__ __launch_bounds__(256) void experts_down_kernel(const T* __restrict__ act, long ldy,
                                                           const T* __restrict__ w_down, int N, int F, int top,
                                                           int n_tokens, const int* __restrict__ order,
                                                           const int* __restrict__ tiles,
                                                           const float* __restrict__ weight, float* __restrict__ P,
                                                           const T* __restrict__ x, long ldx, const float* __restrict__ share,
                                                           int real, SharedExpert<T> sh) {
  constexpr int VEC = Atom<T>::VEC, KC = Atom<T>::KCHUNK;
  const bool all = KS > 1 && (int)blockIdx.x >= sh.at;
  const int e = all ? 0 : tiles[4 * blockIdx.x];
  if (e < 0) return;
  const int first = all ? 16 * ((int)blockIdx.x - sh.at) : tiles[4 * blockIdx.x + 1];
  const int rows = all ? min(16, n_tokens - first) : tiles[4 * blockIdx.x + 2];
  if (all) {
    F = sh.F;
    ldy = sh.ldy;
    act = sh.act;
    w_down = sh.w_down;
  }
  if (e >= real) {   // (the whole workgroup)
    constexpr int kCols = KS == 1 ? 64 : 16;
    pass_input<T>(x, ldx, share, first, rows, blockIdx.y * kCols, min(N, (int)(blockIdx.y + 1) * kCols), top, n_tokens, N, order, P);
    return;
  }
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int l16 = lane & 15, quad = lane >> 4;
  const int col0 = KS == 1 ? (blockIdx.y * 4 + w) * 16 : blockIdx.y * 16;
  if (col0 >= N) return;
  const bool w_ok = col0 + l16 < N;
  const T* d_row = w_down + ((long)e * N + (w_ok ? col0 + l16 : 0)) * F;
  const T* y_row[RT];
  bool y_ok[RT];
#pragma unroll
  for (int r = 0; r < RT; ++r) {
    y_ok[r] = 16 * r + l16 < rows;
    y_row[r] = act + (long)(first + (y_ok[r] ? 16 * r + l16 : 0)) * ldy;
  }
  f32x4 acc[RT];
#pragma unroll
  for (int r = 0; r < RT; ++r) acc[r] = f32x4{0.f, 0.f, 0.f, 0.f};
  const bool aligned = F % VEC == 0 && ldy % VEC == 0;
  constexpr int U = RT == 1 ? 8 : 4;
  const int k_each = KS == 1 ? F : (F + KC * KS - 1) / (KC * KS) * KC;
  const int k_lo = KS == 1 ? 0 : w * k_each, k_hi = KS == 1 ? F : min(F, k_lo + k_each);
  for (int k0 = k_lo; k0 < k_hi; k0 += U * KC) {
    typename Atom<T>::vec_t a[U], b[U][RT];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = k0 + u * KC + VEC * quad;
      a[u] = load_vec<T>(d_row, 0, k, k_hi, 0, w_ok, aligned);
#pragma unroll
      for (int r = 0; r < RT; ++r) b[u][r] = load_vec<T>(y_row[r], 0, k, k_hi, 0, y_ok[r], aligned);
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int r = 0; r < RT; ++r) Atom<T>::mma(acc[r], a[u], b[u][r]);
  }
  if constexpr (KS > 1) {
    __shared__ f32x4 sums_s[KS][RT][64];
#pragma unroll
    for (int r = 0; r < RT; ++r) sums_s[w][r][lane] = acc[r];
    __syncthreads();
    if (w != 0) return;
#pragma unroll
    for (int r = 0; r < RT; ++r)
#pragma unroll
      for (int o = 1; o < KS; ++o)
#pragma unroll
        for (int i = 0; i < 4; ++i) acc[r][i] = acc[r][i] + sums_s[o][r][lane][i];
  }
#pragma unroll
  for (int r = 0; r < RT; ++r) {
    if (!y_ok[r]) continue;
    const int pair = all ? 0 : order[first + 16 * r + l16];
    const float factor = weight && !all ? weight[pair] : 1.0f;
    float* dst = all ? sh.out + (long)(first + l16) * N : P + ((long)(pair % top) * n_tokens + pair / top) * N;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int c = col0 + 4 * quad + i;
      if (c < N) dst[c] = factor * acc[r][i];
    }
  }
}

// ---------------------------------------------------------------------------
// The same two products for tiles of 64 rows (many tokens an expert), both operands staged through LDS: a
// workgroup takes 64 rows x 64 columns, its four waves 32 x 32 each.  A stage is 128 bytes of K for every row of
// the operands (two chunks of the atom), copied from global memory into registers while the stage before it is
// multiplied, then written to the other of two LDS buffers; rows of an LDS tile are 144 bytes apart, which
// spreads the sixteen rows of a fragment read over all banks.  A row's contraction is still one chain over
// ascending chunks from zero: the same bits as the kernels above give without a cut of K.  NB: weight matrices
// that share the rows (gate and up: 2; down: 1).
// ---------------------------------------------------------------------------
constexpr int kStageBytes = 128, kLdsRow = kStageBytes + 16;

template <typename T, int NB>
struct TiledProduct {
  typedef typename Atom<T>::vec_t vec_t;
  static constexpr int VEC = Atom<T>::VEC;
  static constexpr int kStageK = kStageBytes / (int)sizeof(T);
  vec_t staged[1 + NB][2];
  f32x4 acc[NB][2][2];

  // a_row / b_row: where this thread's two pieces of a stage come from (null: zeros), for rows tid/8 and tid/8 + 32
  __device__ __forceinline__ void request(const T* const (&a_row)[2], const T* const (&b_row)[NB][2], int k0, int K) {
    const int seg = threadIdx.x & 7;
    const int k = k0 + seg * VEC;
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      staged[0][j] = (a_row[j] && k < K) ? *reinterpret_cast<const vec_t*>(a_row[j] + k) : Atom<T>::zero();
#pragma unroll
      for (int m = 0; m < NB; ++m)
        staged[1 + m][j] = (b_row[m][j] && k < K) ? *reinterpret_cast<const vec_t*>(b_row[m][j] + k) : Atom<T>::zero();
    }
  }
  __device__ __forceinline__ void store(char* lds) {
    const int row = threadIdx.x >> 3, seg = threadIdx.x & 7;
#pragma unroll
    for (int m = 0; m < 1 + NB; ++m)
#pragma unroll
      for (int j = 0; j < 2; ++j)
        *reinterpret_cast<vec_t*>(lds + ((m * 64) + row + 32 * j) * kLdsRow + seg * 16) = staged[m][j];
  }
  __device__ __forceinline__ void multiply(const char* lds) {
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
    const int l16 = lane & 15, quad = lane >> 4, wr = w >> 1, wc = w & 1;
#pragma unroll
    for (int c = 0; c < kStageBytes / 64; ++c) {
      vec_t a[2], b[NB][2];
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        a[t] = *reinterpret_cast<const vec_t*>(lds + (wr * 32 + t * 16 + l16) * kLdsRow + c * 64 + quad * 16);
#pragma unroll
        for (int m = 0; m < NB; ++m)
          b[m][t] = *reinterpret_cast<const vec_t*>(lds + ((1 + m) * 64 + wc * 32 + t * 16 + l16) * kLdsRow + c * 64 + quad * 16);
      }
#pragma unroll
      for (int m = 0; m < NB; ++m)
#pragma unroll
        for (int rt = 0; rt < 2; ++rt)
#pragma unroll
          for (int ct = 0; ct < 2; ++ct) Atom<T>::mma(acc[m][rt][ct], b[m][ct], a[rt]);
    }
  }
  __device__ __forceinline__ void run(const T* const (&a_row)[2], const T* const (&b_row)[NB][2], int K, char* lds) {
#pragma unroll
    for (int m = 0; m < NB; ++m)
#pragma unroll
      for (int rt = 0; rt < 2; ++rt)
#pragma unroll
        for (int ct = 0; ct < 2; ++ct) acc[m][rt][ct] = f32x4{0.f, 0.f, 0.f, 0.f};
    constexpr int kBuffer = (1 + NB) * 64 * kLdsRow;
    const int stages = (K + kStageK - 1) / kStageK;
    request(a_row, b_row, 0, K);
    store(lds);
    __syncthreads();
    for (int s = 0; s < stages; ++s) {
      if (s + 1 < stages) request(a_row, b_row, (s + 1) * kStageK, K);
      multiply(lds + (s & 1) * kBuffer);
      if (s + 1 < stages) store(lds + ((s + 1) & 1) * kBuffer);
      __syncthreads();
    }
  }
};

template <typename T>
__global__ __launch_bounds__(256) void experts_gate_up_tiled_kernel(const T* __restrict__ x, long ldx,
                                                                    const T* __restrict__ w_gate,
                                                                    const T* __restrict__ w_up, int F, int K, int top,
                                                                    const int* __restrict__ order,
                                                                    const int* __restrict__ tiles, float limit, float alpha,
                                                                    float shift, const float* __restrict__ in_weight,
                                                                    T* __restrict__ act, long ldy, int real) {
  __shared__ __attribute__((aligned(16))) char lds[2 * 3 * 64 * kLdsRow];
  const int e = tiles[4 * blockIdx.x];
  if (e < 0 || e >= real) return;
  const int first = tiles[4 * blockIdx.x + 1], rows = tiles[4 * blockIdx.x + 2];
  const int col0 = blockIdx.y * 64;
  const T* a_row[2];
  const T* b_row[2][2];
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    const int r = (threadIdx.x >> 3) + 32 * j;
    a_row[j] = r < rows ? x + (long)(order[first + r] / top) * ldx : nullptr;
    b_row[0][j] = col0 + r < F ? w_gate + ((long)e * F + col0 + r) * K : nullptr;
    b_row[1][j] = col0 + r < F ? w_up + ((long)e * F + col0 + r) * K : nullptr;
  }
  TiledProduct<T, 2> product;
  product.run(a_row, b_row, K, lds);
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int l16 = lane & 15, quad = lane >> 4, wr = w >> 1, wc = w & 1;
#pragma unroll
  for (int rt = 0; rt < 2; ++rt) {
    const int r = wr * 32 + rt * 16 + l16;
    if (r >= rows) continue;
    T* dst = act + (long)(first + r) * ldy;
    const float wt = in_weight ? in_weight[order[first + r]] : 1.0f;
#pragma unroll
    for (int ct = 0; ct < 2; ++ct)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int c = col0 + wc * 32 + ct * 16 + 4 * quad + i;
        if (c < F) {
          const float g = fminf(product.acc[0][rt][ct][i] * wt, limit);
          const float u = fminf(fmaxf(product.acc[1][rt][ct][i] * wt, -limit), limit);
          dst[c] = from_f32<T>((g * sigmoid_e(alpha * g)) * (u + shift));
        }
      }
  }
}

template <typename T>
__global__ __launch_bounds__(256) void experts_down_tiled_kernel(const T* __restrict__ act, long ldy,
                                                                 const T* __restrict__ w_down, int N, int F, int top,
                                                                 int n_tokens, const int* __restrict__ order,
                                                                 const int* __restrict__ tiles,
                                                                 const float* __restrict__ weight, float* __restrict__ P,
                                                                 const T* __restrict__ x, long ldx,
                                                                 const float* __restrict__ share, int real) {
  __shared__ __attribute__((aligned(16))) char lds[2 * 2 * 64 * kLdsRow];
  const int e = tiles[4 * blockIdx.x];
  if (e < 0) return;
  const int first = tiles[4 * blockIdx.x + 1], rows = tiles[4 * blockIdx.x + 2];
  const int col0 = blockIdx.y * 64;
  if (e >= real) {
    pass_input<T>(x, ldx, share, first, rows, col0, min(N, col0 + 64), top, n_tokens, N, order, P);
    return;
  }
  const T* a_row[2];
  const T* b_row[1][2];
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    const int r = (threadIdx.x >> 3) + 32 * j;
    a_row[j] = r < rows ? act + (long)(first + r) * ldy : nullptr;
    b_row[0][j] = col0 + r < N ? w_down + ((long)e * N + col0 + r) * F : nullptr;
  }
  TiledProduct<T, 1> product;
  product.run(a_row, b_row, F, lds);
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int l16 = lane & 15, quad = lane >> 4, wr = w >> 1, wc = w & 1;
#pragma unroll
  for (int rt = 0; rt < 2; ++rt) {
    const int r = wr * 32 + rt * 16 + l16;
    if (r >= rows) continue;
    const int pair = order[first + r];
    const float share = weight ? weight[pair] : 1.0f;
    float* dst = P + ((long)(pair % top) * n_tokens + pair / top) * N;
#pragma unroll
    for (int ct = 0; ct < 2; ++ct)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int c = col0 + wc * 32 + ct * 16 + 4 * quad + i;
        if (c < N) dst[c] = share * product.acc[0][rt][ct][i];
      }
  }
}

}  // namespace ls

LS_DEFINE_ERROR_API

using namespace ls;

extern "C" int ls_experts_max_top() { return kMaxTop; }

// Tiles that the pairs of n_tokens tokens can need at most, with rows_a_tile rows each.
extern "C" int ls_experts_tile_capacity(int n_tokens, int E, int top, int rows_a_tile) {
  const long pairs = (long)n_tokens * top;
  return (int)(pairs / rows_a_tile + (pairs < E ? pairs : E));
}

// z [n_tokens][ldz] float router logits, bias [E] or null -> expert, weight [n_tokens][top]; order [n_tokens * top];
// tiles [cap][4]; counts: scratch of E ints.  rows_a_tile 16, 32 or 64.
extern "C" int ls_experts_route(const float* z, long ldz, const float* bias, int n_tokens, int E, int top,
                                int rows_a_tile, int* expert, float* weight, int* order, int* tiles, int cap,
                                int* counts, int scoring, const float* correction, int groups, int keep, void* stream) {
  LS_REQUIRE(scoring >= 0 && scoring <= 2, "experts_route: scoring %d (0: softmax over the chosen, 1: sigmoid, 2: softmax over all)",
             scoring);
  LS_REQUIRE(scoring != 2 || (correction && groups > 0 && keep > 0 && keep <= groups && E % groups == 0 && top <= keep * (E / groups)),
             "experts_route: %d experts in %d groups of which %d are kept, %d a token", E, groups, keep, top);
  const Choice how{scoring, groups, keep, correction};
  LS_REQUIRE(n_tokens > 0 && E > 0 && top > 0 && top <= E && top <= kMaxTop && ldz >= E,
             "experts_route: %d tokens, %d experts, %d chosen (at most %d)", n_tokens, E, top, kMaxTop);
  LS_REQUIRE(rows_a_tile == 16 || rows_a_tile == 32 || rows_a_tile == 64, "experts_route: tiles of %d rows", rows_a_tile);
  LS_REQUIRE(z && expert && weight && order && tiles && counts, "experts_route: null operand");
  LS_REQUIRE(cap >= ls_experts_tile_capacity(n_tokens, E, top, rows_a_tile), "experts_route: %d tiles are too few", cap);
  LS_REQUIRE(E <= 64 * kMaxPerLane, "experts_route: %d experts, the routing kernel takes %d", E, 64 * kMaxPerLane);
  hipStream_t s = reinterpret_cast<hipStream_t>(stream);
  const int P = n_tokens * top;
#define LS_ROUTE(PL_)                                                                                                     \
  if (P <= kSmallPairs && E <= kSmallExperts)                                                                             \
    hipLaunchKernelGGL((route_small_kernel<PL_, float, false>), dim3(1), dim3(1024), 0, s, z, ldz, bias, n_tokens, E, top, \
                       rows_a_tile, expert, weight, order, tiles, cap, (const int*)nullptr, (const int*)nullptr, how,     \
                       (const float*)nullptr, 0L, (const float*)nullptr, 0);                                              \
  else                                                                                                                    \
    hipLaunchKernelGGL(route_topk_kernel<PL_>, dim3((n_tokens + 3) / 4), dim3(256), 0, s, z, ldz, bias, n_tokens, E, top, \
                       expert, weight, how);
  if (E <= 64) { LS_ROUTE(1) }
  else if (E <= 128) { LS_ROUTE(2) }
  else { LS_ROUTE(kMaxPerLane) }
#undef LS_ROUTE
  if (!(P <= kSmallPairs && E <= kSmallExperts)) {
    hipLaunchKernelGGL(route_count_kernel, dim3(E), dim3(64), 0, s, expert, P, counts);
    hipLaunchKernelGGL(route_place_kernel, dim3(E), dim3(64), 0, s, expert, counts, P, E, rows_a_tile, order, tiles, cap);
  }
  return check_launch("experts_route");
}

// Whether ls_experts_route_product takes a step of n_tokens tokens.
extern "C" int ls_experts_route_product_ok(int dtype, int n_tokens, int E, int top, int K) {
  return n_tokens <= 16 && E <= 16 * kProductTiles && (long)n_tokens * top <= kSmallPairs && K % (dtype == kF32 ? 4 : 8) == 0;
}

// The same with the router's product inside: x [n_tokens][ldx] and w_router [E][K] of the compute dtype instead of logits.
extern "C" int ls_experts_route_product(int dtype, const void* x, long ldx, const void* w_router, int K, const float* bias,
                                        int n_tokens, int E, int top, int rows_a_tile, int* expert, float* weight, int* order,
                                        int* tiles, int cap, int scoring, const float* correction, int groups, int keep,
                                        void* stream) {
  LS_REQUIRE(scoring >= 0 && scoring <= 2, "experts_route_product: scoring %d", scoring);
  LS_REQUIRE(scoring != 2 || (correction && groups > 0 && keep > 0 && keep <= groups && E % groups == 0 && top <= keep * (E / groups)),
             "experts_route_product: %d experts in %d groups of which %d are kept, %d a token", E, groups, keep, top);
  LS_REQUIRE(n_tokens > 0 && E > 0 && top > 0 && top <= E && top <= kMaxTop && K > 0 && ldx >= K && ls_experts_route_product_ok(dtype, n_tokens, E, top, K),
             "experts_route_product: %d tokens, %d experts, %d chosen", n_tokens, E, top);
  LS_REQUIRE(rows_a_tile == 16 || rows_a_tile == 32 || rows_a_tile == 64, "experts_route_product: tiles of %d rows", rows_a_tile);
  LS_REQUIRE(x && w_router && expert && weight && order && tiles && cap >= ls_experts_tile_capacity(n_tokens, E, top, rows_a_tile),
             "experts_route_product: bad operands");
  LS_REQUIRE(dtype == kF32 || dtype == kBF16, "experts_route_product: unknown dtype %d", dtype);
  LS_REQUIRE(reinterpret_cast<uintptr_t>(x) % 16 == 0 && reinterpret_cast<uintptr_t>(w_router) % 16 == 0 &&
                 ldx % (dtype == kF32 ? 4 : 8) == 0,
             "experts_route_product: operands must be 16-byte aligned");
  hipStream_t s = reinterpret_cast<hipStream_t>(stream);
  const Choice how{scoring, groups, keep, correction};
#define LS_ROUTE_PRODUCT(PL_, T_)                                                                                         \
  hipLaunchKernelGGL((route_small_kernel<PL_, T_, true>), dim3(1), dim3(1024), 0, s, (const float*)nullptr, 0L, bias, n_tokens, E, \
                     top, rows_a_tile, expert, weight, order, tiles, cap, (const int*)nullptr, (const int*)nullptr, how,  \
                     (const T_*)x, ldx, (const T_*)w_router, K)
  if (dtype == kF32) {
    if (E <= 64) LS_ROUTE_PRODUCT(1, float); else LS_ROUTE_PRODUCT(2, float);
  } else {
    if (E <= 64) LS_ROUTE_PRODUCT(1, bf16_t); else LS_ROUTE_PRODUCT(2, bf16_t);
  }
#undef LS_ROUTE_PRODUCT
  return check_launch("experts_route_product");
}

// The same grouping for experts that a table names: token_ids [n_tokens], table [vocab][top] with entries in [0, E).
extern "C" int ls_experts_route_table(const int* token_ids, const int* table, int n_tokens, int E, int top,
                                      int rows_a_tile, int* expert, float* weight, int* order, int* tiles, int cap,
                                      int* counts, void* stream) {
  LS_REQUIRE(n_tokens > 0 && E > 0 && top > 0 && top <= E, "experts_route_table: %d tokens, %d experts, %d a token", n_tokens, E, top);
  LS_REQUIRE(rows_a_tile == 16 || rows_a_tile == 32 || rows_a_tile == 64, "experts_route_table: tiles of %d rows", rows_a_tile);
  LS_REQUIRE(token_ids && table && expert && weight && order && tiles && counts, "experts_route_table: null operand");
  LS_REQUIRE(cap >= ls_experts_tile_capacity(n_tokens, E, top, rows_a_tile), "experts_route_table: %d tiles are too few", cap);
  hipStream_t s = reinterpret_cast<hipStream_t>(stream);
  const int P = n_tokens * top;
  if (P <= kSmallPairs && E <= kSmallExperts) {
    hipLaunchKernelGGL((route_small_kernel<1, float, false>), dim3(1), dim3(1024), 0, s, (const float*)nullptr, 0L, (const float*)nullptr,
                       n_tokens, E, top, rows_a_tile, expert, weight, order, tiles, cap, token_ids, table, Choice{0, 1, 1, nullptr},
                       (const float*)nullptr, 0L, (const float*)nullptr, 0);
  } else {
    hipLaunchKernelGGL(route_table_kernel, dim3((P + 255) / 256), dim3(256), 0, s, token_ids, table, n_tokens, top, expert,
                       weight);
    hipLaunchKernelGGL(route_count_kernel, dim3(E), dim3(64), 0, s, expert, P, counts);
    hipLaunchKernelGGL(route_place_kernel, dim3(E), dim3(64), 0, s, expert, counts, P, E, rows_a_tile, order, tiles, cap);
  }
  return check_launch("experts_route_table");
}

// x [n_tokens][ldx]; w_gate, w_up [E][F][K]; w_down [E][N][F]; act: scratch [n_tokens * top][ldy] of the compute
// dtype; P [top][n_tokens][N] float.
extern "C" int ls_experts_apply(int dtype, const void* x, long ldx, const void* w_gate, const void* w_up,
                                const void* w_down, int n_tokens, int E, int top, int K, int F, int N,
                                int rows_a_tile, const int* order, const int* tiles, int cap, const float* weight,
                                float limit, float alpha, float shift, void* act, long ldy, float* P, int weigh_input,
                                int real, const void* sh_gate_up, const void* sh_down, int sh_F, void* sh_act, long sh_ldy,
                                float* sh_out, void* stream) {
  // sh_*: an expert that every token uses, worked on in the same launches (tiles of 16 rows only; null: none)
  const bool with_shared = sh_gate_up != nullptr;
  LS_REQUIRE(!with_shared || (rows_a_tile == 16 && sh_down && sh_act && sh_out && sh_F > 0 && sh_ldy >= sh_F &&
                              reinterpret_cast<uintptr_t>(sh_gate_up) % 16 == 0 && reinterpret_cast<uintptr_t>(sh_down) % 16 == 0 &&
                              reinterpret_cast<uintptr_t>(sh_act) % 16 == 0),
             "experts_apply: a shared expert is worked on beside tiles of 16 rows, its operands 16-byte aligned");
  // weigh_input: the routing weight multiplies the expert's input instead of its output.  real: experts from this one on
  // (of the E that the tiles may name) have no weights and return their input
  LS_REQUIRE(real > 0 && real <= E && (real == E || K == N), "experts_apply: %d of %d experts with weights", real, E);
  const float* in_weight = weigh_input ? weight : nullptr;
  const float* out_weight = weigh_input ? nullptr : weight;
  LS_REQUIRE(n_tokens > 0 && E > 0 && top > 0 && K > 0 && F > 0 && N > 0 && ldx >= K && ldy >= F, "experts_apply: bad sizes");
  LS_REQUIRE(rows_a_tile == 16 || rows_a_tile == 32 || rows_a_tile == 64, "experts_apply: tiles of %d rows", rows_a_tile);
  LS_REQUIRE(x && w_gate && w_up && w_down && order && tiles && weight && act && P && cap > 0, "experts_apply: null operand");
  LS_REQUIRE(limit > 0.f, "experts_apply: the limit must be positive");
  LS_REQUIRE(dtype == kF32 || dtype == kBF16, "experts_apply: unknown dtype %d", dtype);
  const int vec = dtype == kF32 ? 4 : 8;
  LS_REQUIRE(reinterpret_cast<uintptr_t>(x) % 16 == 0 && reinterpret_cast<uintptr_t>(act) % 16 == 0 &&
                 reinterpret_cast<uintptr_t>(w_gate) % 16 == 0 && reinterpret_cast<uintptr_t>(w_up) % 16 == 0 &&
                 reinterpret_cast<uintptr_t>(w_down) % 16 == 0 && (K % vec != 0 || ldx % vec == 0),
             "experts_apply: operands must be 16-byte aligned");
  hipStream_t s = reinterpret_cast<hipStream_t>(stream);
  // tiles of 16 rows (few tokens an expert): a workgroup takes 16 columns and cuts K over its waves
  const int cols = rows_a_tile == 16 ? 16 : 64;
  const int more = with_shared ? (n_tokens + 15) / 16 : 0, widest = with_shared && sh_F > F ? sh_F : F;
  const dim3 grid_up(cap + more, (widest + cols - 1) / cols), grid_down(cap + more, (N + cols - 1) / cols);
  auto shared_of = [&](auto* of_type) {
    typedef std::remove_pointer_t<decltype(of_type)> E_;
    return SharedExpert<E_>{(const E_*)sh_gate_up, (const E_*)sh_down, sh_F, with_shared ? cap : 0x7fffffff, (E_*)sh_act, sh_ldy, sh_out};
  };
#define LS_EXPERTS(T_, RT_, KS_)                                                                                      \
  do {                                                                                                                \
    hipLaunchKernelGGL((experts_gate_up_kernel<T_, RT_, KS_>), grid_up, dim3(256), 0, s, (const T_*)x, ldx,           \
                       (const T_*)w_gate, (const T_*)w_up, F, K, top, order, tiles, limit, alpha, shift, in_weight,   \
                       (T_*)act, ldy, real, n_tokens, shared_of((T_*)nullptr));                                       \
    hipLaunchKernelGGL((experts_down_kernel<T_, RT_, KS_>), grid_down, dim3(256), 0, s, (const T_*)act, ldy,          \
                       (const T_*)w_down, N, F, top, n_tokens, order, tiles, out_weight, P, (const T_*)x, ldx, weight, real, \
                       shared_of((T_*)nullptr));                                                                      \
  } while (0)
  // tiles of 64 rows go through LDS where every row of every operand starts on a 16-byte boundary
  const bool staged = rows_a_tile == 64 && K % vec == 0 && F % vec == 0 && ldx % vec == 0 && ldy % vec == 0;
#define LS_EXPERTS_STAGED(T_)                                                                                         \
  do {                                                                                                                \
    hipLaunchKernelGGL(experts_gate_up_tiled_kernel<T_>, grid_up, dim3(256), 0, s, (const T_*)x, ldx,                 \
                       (const T_*)w_gate, (const T_*)w_up, F, K, top, order, tiles, limit, alpha, shift, in_weight,   \
                       (T_*)act, ldy, real);                                                                          \
    hipLaunchKernelGGL(experts_down_tiled_kernel<T_>, grid_down, dim3(256), 0, s, (const T_*)act, ldy,                \
                       (const T_*)w_down, N, F, top, n_tokens, order, tiles, out_weight, P, (const T_*)x, ldx, weight, real); \
  } while (0)
#define LS_EXPERTS_BY_ROWS(T_)                 \
  switch (rows_a_tile) {                       \
    case 16: LS_EXPERTS(T_, 1, 4); break;      \
    case 32: LS_EXPERTS(T_, 2, 1); break;      \
    default:                                   \
      if (staged)                              \
        LS_EXPERTS_STAGED(T_);                 \
      else                                     \
        LS_EXPERTS(T_, 4, 1);                  \
      break;                                   \
  }
  if (dtype == kF32) {
    LS_EXPERTS_BY_ROWS(float)
  } else {
    LS_EXPERTS_BY_ROWS(bf16_t)
  }
#undef LS_EXPERTS_BY_ROWS
#undef LS_EXPERTS_STAGED
#undef LS_EXPERTS
  return check_launch("experts_apply");
}
