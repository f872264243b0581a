// Routed feed-forward (mixture of experts): router, and the experts of every row's choice.
//
// Router: logits z = W_router x in float32 (W_router is kept in float32; x is read as stored),
// the `top` experts of largest logit (of equal logits the one of lower index), and their
// weights softmax(z over the chosen ones only); or (`mode` 1) the scores s = softmax(z) over all
// router outputs, the `top` outputs of largest s + correction (a learned number per output,
// null: none), and the weights s of the chosen, not renormalised.  Experts: for row r and its
// choice k with expert e and weight p,  y_r += p W_down,e (silu(W_gate,e x_r) * (W_up,e x_r)).
// `mode` 2: the scores s = sigmoid(z), the experts cut into `groups` runs of equal length of which
// the `keep` whose two best scores add up to most take part (of equal ones the one of lower
// index), the `top` largest scores among their experts, and the weights s / (sum of the
// chosen s + 1e-20) * weight_scale.
// The gated product of an expert is silu(gate) * up or the clamped swish (`ei::GateAct`).  The rows
// of another product (an expert that every row takes) may be added to the sums: `extra`.
// A router may have more outputs than there are experts: an output beyond the experts is an
// identity expert, which adds p x_r and has no matrices.
//
// Three forms of the experts.  One takes a (row, choice) pair at a time and streams the expert's
// matrices for it: any type and any sizes, matrices as stored, gate and up [E, F, W], down
// [E, W, F], stacked.  The others (bfloat16, widths that are multiples of
// 64) run every expert's pairs against its matrices as tiles on the matrix cores: for up to 64
// rows a block finds its expert's pairs itself; for more the pairs are laid out by expert on the
// device first.  Those take the matrices in operand order: tiles of 16 rows x 32 k of one
// kilobyte each, an expert's strip of 16 rows being its K / 32 tiles in a row, and inside a tile
// the piece of row r and k = 8 c .. 8 c + 7 at (c * 16 + r) * 8 elements, so that a wave's load of
// a tile is one contiguous kilobyte which holds lane l's operand at 16 l bytes.
#include "common.h"
#include <float.h>

namespace {

constexpr int kMaxTop = 64;
constexpr int kRouteMax = 8;      // experts a lane holds: up to 512 experts
constexpr int kRanked = 2;        // up to so many a lane, the choice is made by ranks

// What this wave has written to LDS, its lanes may read from here on.
__device__ __forceinline__ void wave_lds_fence() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}

// Rows [N, W] that are added to the experts' weighted sums: float32 slices or one bfloat16 tensor
// (null: none).
struct ExtraRows {
  const void* rows;
  int dtype, slices;
  size_t slice;
};

__device__ __forceinline__ float extra_at(const ExtraRows& extra, size_t at) {
  float sum = 0.f;
  if (extra.dtype == EI_F32) {
    const float* p = static_cast<const float*>(extra.rows) + at;
    for (int s = 0; s < extra.slices; ++s) sum += p[s * extra.slice];
  } else {
    sum = ei::bf16_to_f32(static_cast<const bf16_t*>(extra.rows)[at]);
  }
  return sum;
}

// The grouped choice of mode 2 by one wave: lane l holds the scores z[j] of experts l + 64 j.  A
// group that does not take part gets -1 for its experts' scores (all real ones are in [0, 1]).
// `scores` is LDS for E numbers and `group_scores` for up to E.
__device__ __forceinline__ void leave_groups_out(float (&z)[kRouteMax], float* scores,
                                                 float* group_scores, int E, int groups, int keep) {
  const int lane = threadIdx.x % EI_WAVE, size = E / groups;
#pragma unroll
  for (int j = 0; j < kRouteMax; ++j)
    if (lane + j * EI_WAVE < E) scores[lane + j * EI_WAVE] = z[j];
  wave_lds_fence();
  for (int g = lane; g < groups; g += EI_WAVE) {
    float first = 0.f, second = 0.f;            // (scores are not negative)
    for (int i = 0; i < size; ++i) {
      const float s = scores[g * size + i];
      if (s > first) { second = first; first = s; }
      else if (s > second) second = s;
    }
    group_scores[g] = first + second;
  }
  wave_lds_fence();
#pragma unroll
  for (int j = 0; j < kRouteMax; ++j) {
    const int e = lane + j * EI_WAVE;
    if (e >= E) continue;
    const int g = e / size;
    const float own = group_scores[g];
    int ahead = 0;                              // groups that come before this expert's
    for (int other = 0; other < groups; ++other) {
      const float s = group_scores[other];
      if (s > own || (s == own && other < g)) ++ahead;
    }
    if (ahead >= keep) z[j] = -1.0f;
  }
}

// A block R rows: its waves share the experts' logits out (a router row is read once for all R
// rows), wave r then chooses for row r.
template <typename TX, int R>
__global__ void __launch_bounds__(1024)
moe_route_kernel(const TX* __restrict__ x, const float* __restrict__ w_router,
                 const int32_t* __restrict__ row_seq, int32_t* __restrict__ expert,
                 float* __restrict__ weight, int N, int W, int E, int top, int mode,
                 const float* __restrict__ correction, int groups, int keep, float weight_scale) {
  __shared__ float logits[R][kRouteMax * EI_WAVE], group_scores[R][kRouteMax * EI_WAVE];
  __shared__ float ranked[R][kMaxTop];
  __shared__ int ranked_e[R][kMaxTop];
  const int wave = threadIdx.x / EI_WAVE, lane = threadIdx.x % EI_WAVE, waves = blockDim.x / EI_WAVE;
  const int row0 = blockIdx.x * R;
  const TX* x_row[R];                           // (rows beyond the last: the last row again)
#pragma unroll
  for (int r = 0; r < R; ++r) x_row[r] = x + static_cast<size_t>(min(row0 + r, N - 1)) * W;
  // (asked for now, looked at when the choice is made)
  const int own_seq = row_seq && wave < R && row0 + wave < N ? row_seq[row0 + wave] : 0;
  for (int e = wave; e < E; e += waves) {
    const float* wr = w_router + static_cast<size_t>(e) * W;
    float sum[R];
#pragma unroll
    for (int r = 0; r < R; ++r) sum[r] = 0.f;
    if (W % 4 == 0) {
#pragma unroll(R == 1 ? 8 : 4)
      for (int i = lane * 4; i < W; i += EI_WAVE * 4) {
        float wv[4];
        ei::Vec4<float>::load(wr + i, wv);
#pragma unroll
        for (int r = 0; r < R; ++r) {
          float xv[4];
          ei::Vec4<TX>::load(x_row[r] + i, xv);
          sum[r] += xv[0] * wv[0];
          sum[r] += xv[1] * wv[1];
          sum[r] += xv[2] * wv[2];
          sum[r] += xv[3] * wv[3];
        }
      }
    } else {
      for (int i = lane; i < W; i += EI_WAVE) {
#pragma unroll
        for (int r = 0; r < R; ++r) sum[r] += ei::to_f32<TX>(x_row[r][i]) * wr[i];
      }
    }
#pragma unroll
    for (int r = 0; r < R; ++r) {
      sum[r] = ei::wave_sum(sum[r]);
      if (!(sum[r] > -FLT_MAX)) sum[r] = -FLT_MAX;      // (a NaN chooses nothing ahead of a number)
      if (lane == 0) logits[r][e] = sum[r];
    }
  }
  __syncthreads();
  if (wave >= R || row0 + wave >= N) return;
  int32_t* e_out = expert + static_cast<size_t>(row0 + wave) * top;
  float* w_out = weight + static_cast<size_t>(row0 + wave) * top;
  if (own_seq < 0) {    // a padding row: no expert has anything to add
    for (int k = lane; k < top; k += EI_WAVE) { e_out[k] = 0; w_out[k] = 0.f; }
    return;
  }
  float z[kRouteMax];
#pragma unroll
  for (int j = 0; j < kRouteMax; ++j) z[j] = lane + j * EI_WAVE < E ? logits[wave][lane + j * EI_WAVE] : -FLT_MAX;
  float score[kRouteMax];                        // mode 1: the softmax over all outputs
  if (mode == 1) {
    float top_z = -FLT_MAX;
#pragma unroll
    for (int j = 0; j < kRouteMax; ++j) top_z = fmaxf(top_z, z[j]);
    top_z = ei::wave_max(top_z);
    float sum = 0.f;
#pragma unroll
    for (int j = 0; j < kRouteMax; ++j) {
      score[j] = lane + j * EI_WAVE < E ? expf(z[j] - top_z) : 0.f;
      sum += score[j];
    }
    sum = ei::wave_sum(sum);
#pragma unroll
    for (int j = 0; j < kRouteMax; ++j) {
      const int e = lane + j * EI_WAVE;
      score[j] = score[j] / sum;
      // what the choice goes by from here on
      z[j] = e < E ? score[j] + (correction ? correction[e] : 0.f) : -FLT_MAX;
    }
  }
  if (mode == 2) {
#pragma unroll
    for (int j = 0; j < kRouteMax; ++j)
      z[j] = lane + j * EI_WAVE < E ? 1.0f / (1.0f + expf(-z[j])) : -FLT_MAX;
    if (groups > 1 && keep < groups) leave_groups_out(z, logits[wave], group_scores[wave], E, groups, keep);
  }
  if (E <= kRanked * EI_WAVE) {
    // a lane finds its outputs' places in the order by comparing them with all others
    float* choice = logits[wave];
#pragma unroll
    for (int j = 0; j < kRanked; ++j)
      if (lane + j * EI_WAVE < E) choice[lane + j * EI_WAVE] = z[j];
    wave_lds_fence();
#pragma unroll
    for (int j = 0; j < kRanked; ++j) {
      const int e = lane + j * EI_WAVE;
      if (e >= E) continue;
      int rank = 0;
      for (int o = 0; o < E; ++o) {
        const float other = choice[o];
        rank += other > z[j] || (other == z[j] && o < e) ? 1 : 0;
      }
      if (rank < top) {
        ranked_e[wave][rank] = e;
        ranked[wave][rank] = mode == 1 ? score[j] : z[j];
      }
    }
    wave_lds_fence();
    const float largest = ranked[wave][0];
    float total = 0.f;
    for (int k = 0; k < top; ++k) total += mode == 2 ? ranked[wave][k] : expf(ranked[wave][k] - largest);
    if (lane < top) {
      const float mine = ranked[wave][lane];
      e_out[lane] = ranked_e[wave][lane];
      w_out[lane] = mode == 2 ? mine / (total + 1e-20f) * weight_scale
                              : mode == 1 ? mine : expf(mine - largest) / total;
    }
    return;
  }
  unsigned taken = 0;                            // bit j: this lane's expert lane + 64 j is chosen
  float total = 0.f, largest = 0.f;
  float mine = 0.f;                              // lane k keeps the k-th choice
  int mine_e = 0;
  for (int k = 0; k < top; ++k) {
    float best = -INFINITY;
    int best_e = 0x7fffffff;
#pragma unroll
    for (int j = 0; j < kRouteMax; ++j) {
      const int e = lane + j * EI_WAVE;
      if (e < E && !(taken >> j & 1u) && z[j] > best) { best = z[j]; best_e = e; }
    }
    for (int offset = EI_WAVE / 2; offset > 0; offset >>= 1) {
      const float other = __shfl_xor(best, offset, EI_WAVE);
      const int other_e = __shfl_xor(best_e, offset, EI_WAVE);
      if (other > best || (other == best && other_e < best_e)) { best = other; best_e = other_e; }
    }
    float chosen_score = 0.f;                    // mode 1: the score of the choice, from its lane
    if (best_e % EI_WAVE == lane) {
      taken |= 1u << (best_e / EI_WAVE);
      if (mode == 1) {
#pragma unroll
        for (int j = 0; j < kRouteMax; ++j)
          if (j == best_e / EI_WAVE) chosen_score = score[j];
      }
    }
    if (mode == 1) chosen_score = __shfl(chosen_score, best_e % EI_WAVE, EI_WAVE);
    if (k == 0) largest = best;
    total += mode == 2 ? best : expf(best - largest);
    if (lane == k) { mine = mode == 1 ? chosen_score : best; mine_e = best_e; }
  }
  if (lane < top) {
    e_out[lane] = mine_e;
    w_out[lane] = mode == 2 ? mine / (total + 1e-20f) * weight_scale
                            : mode == 1 ? mine : expf(mine - largest) / total;
  }
}

// act [N * top, F] = silu(W_gate,e x) * (W_up,e x) for every (row, choice).  A block a pair and
// a strip of 16 outputs; a wave takes four outputs at a time.
template <typename T>
__global__ void __launch_bounds__(256)
moe_gate_up_kernel(const T* __restrict__ x, const T* __restrict__ w_gate, const T* __restrict__ w_up,
                   const int32_t* __restrict__ expert, const float* __restrict__ weight,
                   T* __restrict__ act, int W, int F, int top, int E, ei::GateAct how) {
  const int pair = blockIdx.x;
  if (weight[pair] == 0.f) return;              // a padding row's choice
  const int row = pair / top, e = expert[pair];
  if (e >= E) return;                           // an identity expert has no product
  const int wave = threadIdx.x / EI_WAVE, lane = threadIdx.x % EI_WAVE;
  const int f0 = blockIdx.y * 16 + wave * 4;
  if (f0 >= F) return;
  const T* xr = x + static_cast<size_t>(row) * W;
  const T* g = w_gate + (static_cast<size_t>(e) * F + f0) * W;
  const T* u = w_up + (static_cast<size_t>(e) * F + f0) * W;
  const int nf = min(4, F - f0);
  float sg[4] = {0.f, 0.f, 0.f, 0.f}, su[4] = {0.f, 0.f, 0.f, 0.f};
  if (W % 8 == 0) {
    for (int i = lane * 8; i < W; i += EI_WAVE * 8) {
      float xv[8];
      ei::VecN<T, 8>::load(xr + i, xv);
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        if (q < nf) {
          float a[8], b[8];
          ei::VecN<T, 8>::load(g + static_cast<size_t>(q) * W + i, a);
          ei::VecN<T, 8>::load(u + static_cast<size_t>(q) * W + i, b);
#pragma unroll
          for (int v = 0; v < 8; ++v) { sg[q] += a[v] * xv[v]; su[q] += b[v] * xv[v]; }
        }
      }
    }
  } else {
    for (int i = lane; i < W; i += EI_WAVE) {
      const float xv = ei::to_f32<T>(xr[i]);
      for (int q = 0; q < nf; ++q) {
        sg[q] += ei::to_f32<T>(g[static_cast<size_t>(q) * W + i]) * xv;
        su[q] += ei::to_f32<T>(u[static_cast<size_t>(q) * W + i]) * xv;
      }
    }
  }
#pragma unroll
  for (int q = 0; q < 4; ++q) {
    const float gate = ei::wave_sum(sg[q]), up = ei::wave_sum(su[q]);
    if (lane == 0 && q < nf)
      act[static_cast<size_t>(pair) * F + f0 + q] = ei::from_f32<T>(ei::gated_product<T>(gate, up, how));
  }
}

// out [N, W] float32 = sum over a row's choices of weight * W_down,e act.  A block a row and a
// strip of 16 columns; a wave takes four columns at a time.
template <typename T>
__global__ void __launch_bounds__(256)
moe_down_kernel(const T* __restrict__ act, const T* __restrict__ w_down,
                const int32_t* __restrict__ expert, const float* __restrict__ weight,
                float* __restrict__ out, int W, int F, int top, int E, const T* __restrict__ x,
                ExtraRows extra) {
  const int row = blockIdx.x;
  const int wave = threadIdx.x / EI_WAVE, lane = threadIdx.x % EI_WAVE;
  const int c0 = blockIdx.y * 16 + wave * 4;
  if (c0 >= W) return;
  const int nc = min(4, W - c0);
  float total[4] = {0.f, 0.f, 0.f, 0.f};
  for (int k = 0; k < top; ++k) {
    const int pair = row * top + k;
    const float p = weight[pair];
    if (p == 0.f) continue;
    if (expert[pair] >= E) {                    // an identity expert: the row itself
      for (int q = 0; q < nc; ++q)
        total[q] += p * ei::to_f32<T>(x[static_cast<size_t>(row) * W + c0 + q]);
      continue;
    }
    const T* a = act + static_cast<size_t>(pair) * F;
    const T* d = w_down + (static_cast<size_t>(expert[pair]) * W + c0) * F;
    float s[4] = {0.f, 0.f, 0.f, 0.f};
    if (F % 8 == 0) {
      for (int i = lane * 8; i < F; i += EI_WAVE * 8) {
        float av[8];
        ei::VecN<T, 8>::load(a + i, av);
#pragma unroll
        for (int q = 0; q < 4; ++q) {
          if (q < nc) {
            float dv[8];
            ei::VecN<T, 8>::load(d + static_cast<size_t>(q) * F + i, dv);
#pragma unroll
            for (int v = 0; v < 8; ++v) s[q] += dv[v] * av[v];
          }
        }
      }
    } else {
      for (int i = lane; i < F; i += EI_WAVE) {
        const float av = ei::to_f32<T>(a[i]);
        for (int q = 0; q < nc; ++q) s[q] += ei::to_f32<T>(d[static_cast<size_t>(q) * F + i]) * av;
      }
    }
#pragma unroll
    for (int q = 0; q < 4; ++q) total[q] += p * ei::wave_sum(s[q]);
  }
  if (lane < nc) {
    float sum = lane == 0 ? total[0] : lane == 1 ? total[1] : lane == 2 ? total[2] : total[3];
    const size_t at = static_cast<size_t>(row) * W + c0 + lane;
    if (extra.rows) sum += extra_at(extra, at);
    out[at] = sum;
  }
}


// ---------------------------------------------------------------------------------------
// The experts as grouped matrix products on the matrix cores (bfloat16, K a multiple of 64).
//
// moe_group: the (row, choice) pairs counted and laid out by expert: `sorted` [P] holds the
// pairs of expert 0, then those of expert 1, ...; `place` [P] is where a pair went (-1: a pair
// of weight 0, which is left out; -2: a pair of an identity expert, an output of the router
// beyond the E experts); `starts` [E + 1] are the experts' first places.  A block an expert: it
// counts its own pairs and those of the experts before it, then lays its own out, in an order
// that depends on the pairs alone.
__global__ void __launch_bounds__(1024)
moe_group_kernel(const int32_t* __restrict__ expert, const float* __restrict__ weight,
                 int32_t* __restrict__ sorted, int32_t* __restrict__ place,
                 int32_t* __restrict__ starts, int P, int E) {
  constexpr int WAVES = 16, U = 8;
  __shared__ int counts[2][WAVES];
  const int e = blockIdx.x;
  const int wave = threadIdx.x / EI_WAVE, lane = threadIdx.x % EI_WAVE;
  int before = 0, own = 0;
  for (int p0 = threadIdx.x; p0 < P; p0 += 1024 * U) {
    int x[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int p = p0 + u * 1024;
      x[u] = p < P && weight[p] != 0.f ? expert[p] : E;
      if (e == 0 && p < P) {                       // (once: the pairs that are left out)
        if (weight[p] == 0.f) place[p] = -1;
        else if (x[u] >= E) place[p] = -2;
      }
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      before += x[u] < e ? 1 : 0;
      own += x[u] == e ? 1 : 0;
    }
  }
#pragma unroll
  for (int offset = 1; offset < EI_WAVE; offset <<= 1) {
    before += __shfl_xor(before, offset, EI_WAVE);
    own += __shfl_xor(own, offset, EI_WAVE);
  }
  if (lane == 0) {
    counts[0][wave] = before;
    counts[1][wave] = own;
  }
  __syncthreads();
  before = own = 0;
#pragma unroll
  for (int w = 0; w < WAVES; ++w) {
    before += counts[0][w];
    own += counts[1][w];
  }
  if (threadIdx.x == 0) {
    starts[e] = before;
    if (e == E - 1) starts[E] = before + own;
  }
  int at = before;
  for (int p0 = 0; p0 < P && at < before + own; p0 += 1024 * U) {
    unsigned long long mine[U];
    int here = 0;
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int p = p0 + u * 1024 + threadIdx.x;
      mine[u] = __ballot(p < P && expert[p] == e && weight[p] != 0.f);
      here += __popcll(mine[u]);
    }
    __syncthreads();                               // the counts before have been read
    if (lane == 0) counts[0][wave] = here;
    __syncthreads();
    int q = at, total = 0;
#pragma unroll
    for (int w = 0; w < WAVES; ++w) {
      if (w < wave) q += counts[0][w];
      total += counts[0][w];
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      if (mine[u] >> lane & 1ull) {
        const int p = p0 + u * 1024 + threadIdx.x;
        const int to = q + __popcll(mine[u] & ((1ull << lane) - 1ull));
        sorted[to] = p;
        place[p] = to;
      }
      q += __popcll(mine[u]);
    }
    at += total;
  }
}

typedef __bf16 moe_bf16x8 __attribute__((ext_vector_type(8)));
typedef float moe_f32x4 __attribute__((ext_vector_type(4)));

constexpr int kTileN = 64, kTileK = 64;      // (kTileK: the least K-tile; K must be a multiple)

// The tile `t` of TM places: its expert and its first place within the expert's span, or -1
// beyond the last tile.  Every wave works it out for itself, an expert a lane.
__device__ __forceinline__ int find_tile(const int32_t* __restrict__ starts, int E, int TM, int t,
                                         int& m0) {
  const int lane = threadIdx.x % EI_WAVE;
  for (int base = 0; base < E; base += EI_WAVE) {
    const int e = base + lane;
    const int tiles = e < E ? (starts[e + 1] - starts[e] + TM - 1) / TM : 0;
    int upto = tiles;                             // tiles of this and of the lanes before
#pragma unroll
    for (int offset = 1; offset < EI_WAVE; offset <<= 1) {
      const int other = __shfl_up(upto, offset, EI_WAVE);
      if (lane >= offset) upto += other;
    }
    const int total = __builtin_amdgcn_readfirstlane(__shfl(upto, EI_WAVE - 1, EI_WAVE));
    if (t < total) {
      const int found = __ffsll(static_cast<unsigned long long>(__ballot(upto > t))) - 1;
      m0 = __builtin_amdgcn_readfirstlane((t - __shfl(upto - tiles, found, EI_WAVE)) * TM);
      return __builtin_amdgcn_readfirstlane(base + found);
    }
    t -= total;
  }
  m0 = 0;
  return -1;
}

// One tile of MB * 16 places of one expert against 64 rows of its matrix (GATED: of its gate
// and of its up matrix).  GATED: the rows of `a` are gathered (row = pair / top) and
// silu(gate) * up goes to `out_act` [P, N] at the pairs' places; else the rows of `a` are the
// places themselves and the float32 products go to `out_sum` [P, N].  A wave owns 16 rows of
// the matrix, which it reads from global memory straight into operand registers one K-tile
// ahead; the places' rows travel through LDS (16-byte chunks stored at chunk ^ row % 8).  KT is
// the K-tile: 64 for the large tiles of prompts, 256 for the small ones of decoding, where a
// wave has little to multiply and lives on how many loads of the matrix it keeps in flight.
template <int MB, bool GATED, int KT>
__global__ void __launch_bounds__(256)
moe_gemm_kernel(const bf16_t* __restrict__ a, const int32_t* __restrict__ sorted,
                const int32_t* __restrict__ starts, const bf16_t* __restrict__ w1,
                const bf16_t* __restrict__ w2, bf16_t* __restrict__ out_act,
                float* __restrict__ out_sum, int E, int N, int K, int top, ei::GateAct how) {
  constexpr int TM = MB * 16;
  constexpr int PER_THREAD = TM * (KT / 8) / 256 > 0 ? TM * (KT / 8) / 256 : 1;
  __shared__ __attribute__((aligned(16))) bf16_t xs[TM * KT];
  int m0;
  const int e = find_tile(starts, E, TM, blockIdx.x, m0);      // which expert's tile this block is
  if (e < 0) return;
  const int first = starts[e] + m0;                           // the tile's first place
  const int valid = min(TM, starts[e + 1] - first);           // places of the tile that exist
  const int wave = threadIdx.x / EI_WAVE, lane = threadIdx.x % EI_WAVE;
  const int r16 = lane % 16, quarter = lane / 16;
  const int n_wave = blockIdx.y * kTileN + wave * 16;         // the wave's first matrix row
  const size_t strip = (static_cast<size_t>(e) * (N / 16) + n_wave / 16) * (K / 32);   // (N is a multiple of 64)
  const bf16_t* w1_strip = w1 + strip * 512 + lane * 8;
  const bf16_t* w2_strip = GATED ? w2 + strip * 512 + lane * 8 : nullptr;
  // the chunks of the places' rows that this thread carries into LDS
  const bf16_t* src[PER_THREAD];
  int dst[PER_THREAD];
#pragma unroll
  for (int i = 0; i < PER_THREAD; ++i) {
    const int index = threadIdx.x + i * 256;
    const int row = index / (KT / 8), chunk = index % (KT / 8);
    const int at = first + min(row, valid - 1);               // (clamped: such rows are not stored)
    const size_t source_row = GATED ? static_cast<size_t>(sorted[at] / top) : static_cast<size_t>(at);
    src[i] = a + source_row * K + chunk * 8;
    dst[i] = row * KT + ((chunk ^ (row % 8)) * 8);
  }
  const bool carries = threadIdx.x < TM * (KT / 8);      // (tiles of fewer chunks than threads)
  moe_f32x4 acc1[MB], acc2[GATED ? MB : 1];
#pragma unroll
  for (int mb = 0; mb < MB; ++mb) {
    acc1[mb] = moe_f32x4{0.f, 0.f, 0.f, 0.f};
    if (GATED) acc2[mb] = moe_f32x4{0.f, 0.f, 0.f, 0.f};
  }
  uint4 x_next[PER_THREAD];
  constexpr int STEPS = KT / 32;
  moe_bf16x8 wa[STEPS], wb[GATED ? STEPS : 1], wa_next[STEPS], wb_next[GATED ? STEPS : 1];
  auto fetch = [&](int k0) {
#pragma unroll
    for (int i = 0; i < PER_THREAD; ++i)
      if (carries) x_next[i] = *reinterpret_cast<const uint4*>(src[i] + k0);
#pragma unroll
    for (int s = 0; s < STEPS; ++s) {
      wa_next[s] = *reinterpret_cast<const moe_bf16x8*>(w1_strip + (k0 / 32 + s) * 512);
      if (GATED) wb_next[s] = *reinterpret_cast<const moe_bf16x8*>(w2_strip + (k0 / 32 + s) * 512);
    }
  };
  fetch(0);
  for (int k0 = 0; k0 < K; k0 += KT) {
    __syncthreads();                       // everybody has read the tile before
#pragma unroll
    for (int i = 0; i < PER_THREAD; ++i)
      if (carries) *reinterpret_cast<uint4*>(&xs[dst[i]]) = x_next[i];
#pragma unroll
    for (int s = 0; s < STEPS; ++s) {
      wa[s] = wa_next[s];
      if (GATED) wb[s] = wb_next[s];
    }
    __syncthreads();
    if (k0 + KT < K) fetch(k0 + KT);
#pragma unroll
    for (int s = 0; s < STEPS; ++s) {
#pragma unroll
      for (int mb = 0; mb < MB; ++mb) {
        const int row = mb * 16 + r16, chunk = s * 4 + quarter;
        const moe_bf16x8 xf = *reinterpret_cast<const moe_bf16x8*>(
            &xs[row * KT + ((chunk ^ (row % 8)) * 8)]);
        acc1[mb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wa[s], xf, acc1[mb], 0, 0, 0);
        if (GATED) acc2[mb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wb[s], xf, acc2[mb], 0, 0, 0);
      }
    }
  }
  // lane (r16, quarter) holds, of place mb * 16 + r16, the matrix rows n_wave + 4 quarter + i
#pragma unroll
  for (int mb = 0; mb < MB; ++mb) {
    const int row = mb * 16 + r16;
    if (row >= valid) continue;
    const size_t at = static_cast<size_t>(first + row) * N;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int n = n_wave + 4 * quarter + i;
      if (n >= N) continue;
      if (GATED) {
        out_act[at + n] = ei::f32_to_bf16(ei::gated_product<bf16_t>(acc1[mb][i], acc2[mb][i], how));
      } else {
        out_sum[at + n] = acc1[mb][i];
      }
    }
  }
}

// The experts of up to MB * 16 rows: a block an expert and STRIPS strips of 16 rows of its matrix
// (GATED: of its gate and of its up matrix).  The block finds the pairs that chose its expert
// itself, in the order of the pairs (padding rows left out); KS waves share a strip's K out and
// meet in LDS.  Both operands come from memory straight into operand registers, U steps of 32 at a
// time.  GATED: the
// gated products go to out_act [pairs, N] at the pairs' own places; else the products times the
// pairs' weights go to out_sum [top, rows, N], slice = the choice; the blocks of "expert" E, where
// there are such, write the identity experts' slices, weight times the row itself.
template <int MB, bool GATED, int STRIPS, int KS, int U>
__global__ void __launch_bounds__(STRIPS * KS * EI_WAVE)
moe_few_kernel(const bf16_t* __restrict__ a, const int32_t* __restrict__ expert,
               const float* __restrict__ weight, const int32_t* __restrict__ row_seq,
               const bf16_t* __restrict__ w1, const bf16_t* __restrict__ w2,
               bf16_t* __restrict__ out_act, float* __restrict__ out_sum, int rows, int N, int K,
               int top, int E, const bf16_t* __restrict__ x, ei::GateAct how) {
  constexpr int G = GATED ? 2 : 1, WAVES = STRIPS * KS;
  __shared__ int places[MB * 16];
  __shared__ int wave_counts[WAVES];
  __shared__ float red[WAVES][MB][G][4][EI_WAVE];
  const int e = blockIdx.y, n0 = blockIdx.x * (STRIPS * 16), pairs = rows * top;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / EI_WAVE), lane = threadIdx.x % EI_WAVE;
  if (!GATED && e == E) {
    for (int o = threadIdx.x; o < pairs * STRIPS * 16; o += WAVES * EI_WAVE) {
      const int p = o / (STRIPS * 16), row = p / top, n = n0 + o % (STRIPS * 16);
      if (expert[p] >= E && !(row_seq && row_seq[row] < 0))
        out_sum[(static_cast<size_t>(p % top) * rows + row) * N + n] =
            weight[p] * ei::bf16_to_f32(x[static_cast<size_t>(row) * N + n]);
    }
    return;
  }
  const int n_strip = wave / KS, slice = wave % KS;
  const size_t strip = (static_cast<size_t>(e) * (N / 16) + n0 / 16 + n_strip) * (K / 32);
  const bf16_t* w1_strip = w1 + strip * 512 + lane * 8;
  const bf16_t* w2_strip = GATED ? w2 + strip * 512 + lane * 8 : nullptr;
  const int steps = K / 32, per = (steps + KS - 1) / KS;
  const int s_begin = slice * per, s_end = min(steps, (slice + 1) * per);
  int count = 0;
  for (int base = 0; base < pairs; base += WAVES * EI_WAVE) {
    const int p = base + threadIdx.x;
    const bool mine = p < pairs && expert[p] == e && !(row_seq && row_seq[p / top] < 0);
    const unsigned long long mask = __ballot(mine);
    if (lane == 0) wave_counts[wave] = __popcll(mask);
    __syncthreads();
    int before = count, total = 0;
#pragma unroll
    for (int w = 0; w < WAVES; ++w) {
      if (w < wave) before += wave_counts[w];
      total += wave_counts[w];
    }
    const int at = before + __popcll(mask & ((1ull << lane) - 1ull));
    if (mine && at < MB * 16) places[at] = p;    // (a row chooses an expert once at most)
    count += total;
    __syncthreads();
  }
  count = min(__builtin_amdgcn_readfirstlane(count), MB * 16);
  if (count == 0) return;
  const int r16 = lane % 16, quarter = lane / 16;
  const bf16_t* x_row[MB];
#pragma unroll
  for (int mb = 0; mb < MB; ++mb) {
    const int p = places[min(mb * 16 + r16, count - 1)];      // (clamped: such rows are not stored)
    x_row[mb] = a + static_cast<size_t>(GATED ? p / top : p) * K + quarter * 8;
  }
  moe_f32x4 acc[MB][G];
#pragma unroll
  for (int mb = 0; mb < MB; ++mb)
#pragma unroll
    for (int g = 0; g < G; ++g) acc[mb][g] = moe_f32x4{0.f, 0.f, 0.f, 0.f};
  for (int s0 = s_begin; s0 < s_end; s0 += U) {
    moe_bf16x8 wa[U], wb[GATED ? U : 1], xf[U][MB];
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (s0 + u < s_end) {
        wa[u] = *reinterpret_cast<const moe_bf16x8*>(w1_strip + (s0 + u) * 512);
        if (GATED) wb[u] = *reinterpret_cast<const moe_bf16x8*>(w2_strip + (s0 + u) * 512);
#pragma unroll
        for (int mb = 0; mb < MB; ++mb)
          if (mb * 16 < count) xf[u][mb] = *reinterpret_cast<const moe_bf16x8*>(x_row[mb] + (s0 + u) * 32);
      }
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (s0 + u < s_end) {
#pragma unroll
        for (int mb = 0; mb < MB; ++mb)
          if (mb * 16 < count) {
            acc[mb][0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wa[u], xf[u][mb], acc[mb][0], 0, 0, 0);
            if (GATED)
              acc[mb][G - 1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wb[u], xf[u][mb], acc[mb][G - 1], 0, 0, 0);
          }
      }
  }
#pragma unroll
  for (int mb = 0; mb < MB; ++mb)
#pragma unroll
    for (int g = 0; g < G; ++g)
#pragma unroll
      for (int i = 0; i < 4; ++i) red[wave][mb][g][i][lane] = acc[mb][g][i];
  __syncthreads();
  // lane (r16, quarter) of a wave held, of place mb * 16 + r16, the matrix rows n0 + 4 quarter + i
  for (int o = threadIdx.x; o < count * STRIPS * 16; o += WAVES * EI_WAVE) {
    const int index = o / (STRIPS * 16), n = o % (STRIPS * 16);
    const int mb = index / 16, from = index % 16 + 16 * (n % 16 / 4), i = n % 4, first = n / 16 * KS;
    float sum[G];
#pragma unroll
    for (int g = 0; g < G; ++g) {
      sum[g] = 0.f;
#pragma unroll
      for (int w = 0; w < KS; ++w) sum[g] += red[first + w][mb][g][i][from];
    }
    const int p = places[index];
    if (GATED)
      out_act[static_cast<size_t>(p) * N + n0 + n] =
          ei::f32_to_bf16(ei::gated_product<bf16_t>(sum[0], sum[G - 1], how));
    else
      out_sum[(static_cast<size_t>(p % top) * rows + p / top) * N + n0 + n] = weight[p] * sum[0];
  }
}

// The experts of a prompt: tiles of 128 places of one expert against 128 rows of its matrix
// (GATED: 64 of its gate and the same 64 of its up matrix) on 32x32x16 products.  A block of four
// waves, two by two; a wave holds 64 places against 64 matrix rows (GATED: 32 of each matrix, so
// that a lane ends up with the gate and the up sum of the same element).  K goes by in tiles of 64
// through two LDS buffers for both operands, moved from global memory straight into LDS (a wave
// load is a kilobyte, lane l's 16 bytes at place l of it): tile k + 1 is asked for right after the
// barrier that frees its buffer and arrives while tile k is multiplied; a second block on the
// compute unit covers the rest of the wait.  The matrix comes in operand order; of the places' rows
// the 16-byte pieces are exchanged among themselves (piece ^ (row / 2) % 8), so that 16 rows read
// at one place of a row meet every bank once, and a lane fetches the piece that belongs at its
// place.
// Blocks are dealt to the 8 XCDs round robin; block ids are laid out so that an XCD works on
// `group` tiles of places at a time against all rows of the matrix, whose operands its L2 then
// holds.
constexpr int kBig = 128, kBigK = 64;
typedef float moe_f32x16 __attribute__((ext_vector_type(16)));

template <bool GATED>
__global__ void __launch_bounds__(256, 2)
moe_tile_kernel(const bf16_t* __restrict__ a, const int32_t* __restrict__ sorted,
                const int32_t* __restrict__ starts, const bf16_t* __restrict__ w1,
                const bf16_t* __restrict__ w2, bf16_t* __restrict__ out_act,
                float* __restrict__ out_sum, int E, int N, int K, int top, int n_tiles,
                int place_tiles, int group, ei::GateAct how) {
  __shared__ __attribute__((aligned(1024))) bf16_t lds[2][2][kBig * kBigK];   // [buffer][operand]
  const int xcd = blockIdx.x & 7, slot = blockIdx.x >> 3;
  const int per_group = group * n_tiles, rest = slot % per_group;
  const int tile = (slot / per_group * 8 + xcd) * group + rest % group, n_tile = rest / group;
  if (tile >= place_tiles) return;
  int m0;
  const int e = find_tile(starts, E, kBig, tile, m0);
  if (e < 0) return;
  const int first = starts[e] + m0;                           // the tile's first place
  const int valid = min(kBig, starts[e + 1] - first);         // places of the tile that exist
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / EI_WAVE), lane = threadIdx.x % EI_WAVE;
  const int l32 = lane & 31, half = lane >> 5, wm = wave >> 1, wn = wave & 1;
  constexpr int LOADS = kBig * kBigK * 2 / 1024 / 4;          // wave loads of an operand's tile a wave
  const bf16_t* from_a[LOADS];
  const bf16_t* from_b[LOADS];
#pragma unroll
  for (int i = 0; i < LOADS; ++i) {
    const int row = (wave * LOADS + i) * 8 + lane / 8, piece = (lane % 8) ^ ((row >> 1) & 7);
    const int at = first + min(row, valid - 1);               // (clamped: such rows are not stored)
    const size_t source = GATED ? static_cast<size_t>(sorted[at] / top) : static_cast<size_t>(at);
    from_a[i] = a + source * K + piece * 8;
    // (a wave load of the matrix is one of its tiles: strip `load / 2` of the block's eight, the
    // first or the second 32 of K)
    const int load = wave * LOADS + i, strip = load / 2;
    const bf16_t* matrix = GATED && strip >= 4 ? w2 : w1;
    const int n_strip = GATED ? n_tile * 4 + strip % 4 : n_tile * 8 + strip;
    from_b[i] = matrix + ((static_cast<size_t>(e) * (N / 16) + min(n_strip, N / 16 - 1)) * (K / 32) +
                          load % 2) * 512 + lane * 8;
  }
  auto fetch = [&](int k0, int buffer) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < LOADS; ++i) {
      const int at = (wave * LOADS + i) * 512;
      __builtin_amdgcn_global_load_lds(
          (const __attribute__((address_space(1))) void*)(from_a[i] + k0),
          (__attribute__((address_space(3))) void*)(&lds[buffer][0][at]), 16, 0, 0);
      __builtin_amdgcn_global_load_lds(
          (const __attribute__((address_space(1))) void*)(from_b[i] + k0 * 16),
          (__attribute__((address_space(3))) void*)(&lds[buffer][1][at]), 16, 0, 0);
    }
  };
  int read_a[2], read_b[2], piece_at[4];
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    read_a[j] = (wm * 64 + j * 32 + l32) * kBigK;
    const int row_b = GATED ? j * 64 + wn * 32 + l32 : wn * 64 + j * 32 + l32;
    read_b[j] = row_b / 16 * 1024 + row_b % 16 * 8 + half * 128;
  }
#pragma unroll
  for (int s = 0; s < 4; ++s) piece_at[s] = ((2 * s + half) ^ ((l32 >> 1) & 7)) * 8;
  moe_f32x16 acc[2][2];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int v = 0; v < 16; ++v) acc[i][j][v] = 0.f;
  fetch(0, 0);
  const int k_tiles = K / kBigK;
  for (int kt = 0; kt < k_tiles; ++kt) {
    const int buffer = kt & 1;
    // this tile has arrived (every wave waits for its own loads), the other buffer is free
    __builtin_amdgcn_s_waitcnt(0x0F70);
    __syncthreads();
    if (kt + 1 < k_tiles) fetch((kt + 1) * kBigK, buffer ^ 1);
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      moe_bf16x8 fa[2], fb[2];
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        fa[j] = *reinterpret_cast<const moe_bf16x8*>(&lds[buffer][0][read_a[j] + piece_at[s]]);
        fb[j] = *reinterpret_cast<const moe_bf16x8*>(&lds[buffer][1][read_b[j] + s / 2 * 512 + s % 2 * 256]);
      }
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j)
          acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(fa[i], fb[j], acc[i][j], 0, 0, 0);
    }
  }
  // lane (matrix row l32, half) holds the places 8 (v / 4) + 4 half + v % 4 of a block of 32
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int v = 0; v < 16; ++v) {
      const int row = wm * 64 + i * 32 + 8 * (v / 4) + 4 * half + v % 4;
      if (row >= valid) continue;
      const size_t at = static_cast<size_t>(first + row) * N;
      if (GATED) {
        out_act[at + n_tile * (kBig / 2) + wn * 32 + l32] =
            ei::f32_to_bf16(ei::gated_product<bf16_t>(acc[i][0][v], acc[i][1][v], how));
      } else {
#pragma unroll
        for (int j = 0; j < 2; ++j) {
          const int n = n_tile * kBig + wn * 64 + j * 32 + l32;
          if (n < N) out_sum[at + n] = acc[i][j][v];
        }
      }
    }
}

template <bool GATED>
void launch_tiles(const bf16_t* a, const int32_t* sorted, const int32_t* starts, const bf16_t* w1,
                  const bf16_t* w2, bf16_t* act, float* sums, int P, int E, int N, int K, int top,
                  const ei::GateAct& how, hipStream_t stream) {
  const int n_tiles = (N + (GATED ? kBig / 2 : kBig) - 1) / (GATED ? kBig / 2 : kBig);
  const int place_tiles = P / kBig + E;             // at most: whole tiles and one rest an expert
  const int group = place_tiles >= 128 ? 4 : 2;
  const int groups = (place_tiles + group - 1) / group;
  const unsigned blocks = static_cast<unsigned>((groups + 7) / 8 * 8) * group * n_tiles;
  moe_tile_kernel<GATED><<<blocks, 256, 0, stream>>>(a, sorted, starts, w1, w2, act, sums, E, N, K,
                                                     top, n_tiles, place_tiles, group, how);
}

// out [rows, W] = sum over a row's choices of weight * the choice's product row, four columns a
// thread.
__global__ void moe_combine_kernel(const float* __restrict__ sums, const int32_t* __restrict__ place,
                                   const float* __restrict__ weight, float* __restrict__ out,
                                   int W, int top, size_t total, const bf16_t* __restrict__ x,
                                   ExtraRows extra) {
  const size_t start = (static_cast<size_t>(blockIdx.x) * blockDim.x + threadIdx.x) * 4;
  const size_t step = static_cast<size_t>(gridDim.x) * blockDim.x * 4;
  for (size_t idx = start; idx < total; idx += step) {
    const size_t row = idx / W, col = idx % W;
    float sum[4] = {0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < top; k0 += 4) {
      int q[4];
      float p[4], v[4][4];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        q[u] = k0 + u < top ? place[row * top + k0 + u] : -1;
        p[u] = k0 + u < top ? weight[row * top + k0 + u] : 0.f;
      }
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        v[u][0] = v[u][1] = v[u][2] = v[u][3] = 0.f;
        if (q[u] >= 0) ei::Vec4<float>::load(sums + static_cast<size_t>(q[u]) * W + col, v[u]);
        else if (q[u] == -2) ei::Vec4<bf16_t>::load(x + idx, v[u]);            // identity
      }
#pragma unroll
      for (int u = 0; u < 4; ++u)
#pragma unroll
        for (int i = 0; i < 4; ++i) sum[i] += p[u] * v[u][i];
    }
    if (extra.rows) {
      float more[4];
      if (extra.dtype == EI_F32) {
        const float* from = static_cast<const float*>(extra.rows) + idx;
        for (int s = 0; s < extra.slices; ++s) {
          ei::Vec4<float>::load(from + s * extra.slice, more);
#pragma unroll
          for (int i = 0; i < 4; ++i) sum[i] += more[i];
        }
      } else {
        ei::Vec4<bf16_t>::load(static_cast<const bf16_t*>(extra.rows) + idx, more);
#pragma unroll
        for (int i = 0; i < 4; ++i) sum[i] += more[i];
      }
    }
    ei::Vec4<float>::store(out + idx, sum);
  }
}

bool known_act(int kind) { return kind >= 0 && kind <= 2; }

bool extra_fits(const void* rows, int dtype, int slices, long long slice) {
  return !rows || (slices >= 1 && slice >= 0 && (dtype == EI_F32 || (dtype == EI_BF16 && slices == 1)));
}

}  // namespace

extern "C" int ei_moe_route(const void* x, int x_dtype, const float* w_router, const int32_t* row_seq,
                            int32_t* expert, float* weight, int N, int W, int E, int top,
                            int mode, const float* correction, int groups, int keep,
                            float weight_scale, hipStream_t stream) {
  EI_REQUIRE(x && w_router && expert && weight && N > 0 && W > 0, "moe_route: bad arguments");
  EI_REQUIRE(E >= 1 && E <= kRouteMax * EI_WAVE && top >= 1 && top <= E && top <= kMaxTop,
             "moe_route: up to 512 experts, of which 1 to 64 are chosen");
  EI_REQUIRE(mode >= 0 && mode <= 2, "moe_route: unknown mode");
  EI_REQUIRE(groups >= 1 && E % groups == 0 && keep >= 1 && keep <= groups && (groups == 1 || mode == 2) &&
                 top <= E / groups * keep,
             "moe_route: equal groups of experts, enough of them kept for the choice");
  // few rows: a block of up to 16 waves a row, an expert a wave where there are as many; many rows:
  // four rows a block, which read the router's matrix together
#define EI_ROUTE(TX)                                                                           \
  do {                                                                                         \
    const TX* xx = static_cast<const TX*>(x);                                                  \
    if (N >= 512)                                                                              \
      moe_route_kernel<TX, 4><<<(N + 3) / 4, EI_WAVE * (E >= 8 ? 8 : 4), 0, stream>>>(         \
          xx, w_router, row_seq, expert, weight, N, W, E, top, mode, correction, groups, keep, \
          weight_scale);                                                                       \
    else                                                                                       \
      moe_route_kernel<TX, 1><<<N, EI_WAVE * (E >= 16 ? 16 : E >= 8 ? 8 : 4), 0, stream>>>(    \
          xx, w_router, row_seq, expert, weight, N, W, E, top, mode, correction, groups, keep, \
          weight_scale);                                                                       \
  } while (0)
  if (x_dtype == EI_F32) EI_ROUTE(float);
  else if (x_dtype == EI_BF16) EI_ROUTE(bf16_t);
  else EI_REQUIRE(false, "moe_route: unknown dtype");
#undef EI_ROUTE
  EI_LAUNCH_CHECK();
}

extern "C" int ei_moe_experts(const void* x, const void* w_gate, const void* w_up, const void* w_down,
                              int dtype, const int32_t* expert, const float* weight, void* act,
                              float* out, int N, int W, int F, int E, int top, int act_kind,
                              float limit, float alpha, const void* extra_rows, int extra_dtype,
                              int extra_slices, long long extra_slice, hipStream_t stream) {
  EI_REQUIRE(x && w_gate && w_up && w_down && expert && weight && act && out, "moe_experts: null pointer");
  EI_REQUIRE(known_act(act_kind), "moe_experts: unknown activation");
  EI_REQUIRE(extra_fits(extra_rows, extra_dtype, extra_slices, extra_slice),
             "moe_experts: the rows to add have the wrong type");
  const ei::GateAct how{act_kind, limit, alpha};
  const ExtraRows extra{extra_rows, extra_dtype, extra_slices, static_cast<size_t>(extra_slice)};
  EI_REQUIRE(N > 0 && W > 0 && F > 0 && top >= 1, "moe_experts: sizes must be positive");
  EI_REQUIRE(static_cast<long long>(N) * top <= 0x7fffffffLL && (F + 15) / 16 <= 65535 &&
                 (W + 15) / 16 <= 65535, "moe_experts: too large for one launch");
  const dim3 grid_up(N * top, (F + 15) / 16), grid_down(N, (W + 15) / 16);
#define EI_MOE(T)                                                                              \
  do {                                                                                         \
    moe_gate_up_kernel<T><<<grid_up, 256, 0, stream>>>(                                        \
        static_cast<const T*>(x), static_cast<const T*>(w_gate), static_cast<const T*>(w_up),  \
        expert, weight, static_cast<T*>(act), W, F, top, E, how);                              \
    moe_down_kernel<T><<<grid_down, 256, 0, stream>>>(                                         \
        static_cast<const T*>(act), static_cast<const T*>(w_down), expert, weight, out, W, F, top, \
        E, static_cast<const T*>(x), extra);                                                   \
  } while (0)
  if (dtype == EI_F32) EI_MOE(float);
  else if (dtype == EI_BF16) EI_MOE(bf16_t);
  else EI_REQUIRE(false, "moe_experts: unknown dtype");
#undef EI_MOE
  EI_LAUNCH_CHECK();
}

// Whether `ei_moe_experts_grouped` takes these sizes.
extern "C" int ei_moe_grouped_supported(int dtype, int W, int F, int E) {
  return dtype == EI_BF16 && W % kTileK == 0 && F % kTileK == 0 && E <= kRouteMax * EI_WAVE ? 1 : 0;
}

// The experts as grouped products.  Scratch: sorted, place [P] and starts [E + 1] int32,
// act [P, F] bfloat16, sums [P, W] float32, with P = N * top.
extern "C" int ei_moe_experts_grouped(const void* x, const void* w_gate, const void* w_up,
                                      const void* w_down, const int32_t* expert, const float* weight,
                                      int32_t* sorted, int32_t* place, int32_t* starts, void* act,
                                      float* sums, float* out, int N, int W, int F, int E, int top,
                                      int act_kind, float limit, float alpha,
                                      const void* extra_rows, int extra_dtype, int extra_slices,
                                      long long extra_slice, hipStream_t stream) {
  EI_REQUIRE(known_act(act_kind), "moe_experts_grouped: unknown activation");
  EI_REQUIRE(extra_fits(extra_rows, extra_dtype, extra_slices, extra_slice),
             "moe_experts_grouped: the rows to add have the wrong type");
  const ei::GateAct how{act_kind, limit, alpha};
  const ExtraRows extra{extra_rows, extra_dtype, extra_slices, static_cast<size_t>(extra_slice)};
  EI_REQUIRE(x && w_gate && w_up && w_down && expert && weight && sorted && place && starts && act &&
                 sums && out, "moe_experts_grouped: null pointer");
  EI_REQUIRE(N > 0 && top >= 1 && E >= 1 && ei_moe_grouped_supported(EI_BF16, W, F, E),
             "moe_experts_grouped: sizes it does not take");
  const long long pairs = static_cast<long long>(N) * top;
  EI_REQUIRE(pairs <= 0x3fffffffLL, "moe_experts_grouped: too many rows for one launch");
  const int P = static_cast<int>(pairs);
  moe_group_kernel<<<E, 1024, 0, stream>>>(expert, weight, sorted, place, starts, P, E);
  const bf16_t* xb = static_cast<const bf16_t*>(x);
  const bf16_t* g = static_cast<const bf16_t*>(w_gate);
  const bf16_t* u = static_cast<const bf16_t*>(w_up);
  const bf16_t* d = static_cast<const bf16_t*>(w_down);
  bf16_t* ab = static_cast<bf16_t*>(act);
  // tiles of 32 places while an expert has few (decoding), of 128 for prompts
  if (P <= 32 * E) {
    const unsigned tiles = static_cast<unsigned>((P + 31) / 32 + E);
    const dim3 grid_up(tiles, (F + kTileN - 1) / kTileN), grid_down(tiles, (W + kTileN - 1) / kTileN);
    // (the long K-tile where few experts are at work and their waves cannot fill the chip:
    // measured at 2, 16 and 128 pairs over 8 experts of 2,816 x 2,048)
    const bool few = P <= 4;
    if (few && W % 256 == 0)
      moe_gemm_kernel<2, true, 256><<<grid_up, 256, 0, stream>>>(xb, sorted, starts, g, u, ab, nullptr, E, F, W, top, how);
    else
      moe_gemm_kernel<2, true, 64><<<grid_up, 256, 0, stream>>>(xb, sorted, starts, g, u, ab, nullptr, E, F, W, top, how);
    if (few && F % 256 == 0)
      moe_gemm_kernel<2, false, 256><<<grid_down, 256, 0, stream>>>(ab, sorted, starts, d, nullptr, nullptr, sums, E, W, F, top, how);
    else
      moe_gemm_kernel<2, false, 64><<<grid_down, 256, 0, stream>>>(ab, sorted, starts, d, nullptr, nullptr, sums, E, W, F, top, how);
  } else {
    launch_tiles<true>(xb, sorted, starts, g, u, ab, nullptr, P, E, F, W, top, how, stream);
    launch_tiles<false>(ab, sorted, starts, d, nullptr, nullptr, sums, P, E, W, F, top, how, stream);
  }
  const size_t total = static_cast<size_t>(N) * W;
  size_t blocks = (total / 4 + 255) / 256;
  if (blocks > static_cast<size_t>(ei_compute_units()) * 16) blocks = static_cast<size_t>(ei_compute_units()) * 16;
  moe_combine_kernel<<<static_cast<unsigned>(blocks), 256, 0, stream>>>(sums, place, weight, out, W, top, total, xb, extra);
  EI_LAUNCH_CHECK();
}

// Most rows that `ei_moe_experts_few` takes.
extern "C" int ei_moe_few_rows() { return 64; }

// The experts of at most 64 rows: act [N * top, F] bfloat16 is scratch; slice k of out [top, N, W]
// float32 receives every row's k-th choice's product row times its weight (a padding row, row_seq
// < 0, is not written).  A row chooses an output of the router once at most; outputs from E on are
// identity experts, which there are `identity` of.
extern "C" int ei_moe_experts_few(const void* x, const void* w_gate, const void* w_up,
                                  const void* w_down, const int32_t* expert, const float* weight,
                                  const int32_t* row_seq, void* act, float* out, int N, int W, int F,
                                  int E, int top, int identity, int act_kind, float limit,
                                  float alpha, hipStream_t stream) {
  EI_REQUIRE(x && w_gate && w_up && w_down && expert && weight && act && out && identity >= 0,
             "moe_experts_few: null pointer");
  EI_REQUIRE(N > 0 && N <= ei_moe_few_rows() && top >= 1 && E >= 1 && E < 65535 &&
                 ei_moe_grouped_supported(EI_BF16, W, F, E),
             "moe_experts_few: sizes it does not take");
  EI_REQUIRE(known_act(act_kind), "moe_experts_few: unknown activation");
  const ei::GateAct how{act_kind, limit, alpha};
  const bf16_t* xb = static_cast<const bf16_t*>(x);
  const bf16_t* g = static_cast<const bf16_t*>(w_gate);
  const bf16_t* u = static_cast<const bf16_t*>(w_up);
  const bf16_t* d = static_cast<const bf16_t*>(w_down);
  bf16_t* ab = static_cast<bf16_t*>(act);
  const int down_experts = E + (identity > 0 ? 1 : 0);
#define EI_FEW(MB, GATED, STRIPS, KS, U, EXPERTS, A, W1, W2, ACT, OUT, ROWS, COLS)             \
  moe_few_kernel<MB, GATED, STRIPS, KS, U>                                                     \
      <<<dim3(ROWS / (STRIPS * 16), EXPERTS), STRIPS * KS * EI_WAVE, 0, stream>>>(             \
          A, expert, weight, row_seq, W1, W2, ACT, OUT, N, ROWS, COLS, top, E, xb, how)
  if (N <= 16) {
    EI_FEW(1, true, 1, 8, 8, E, xb, g, u, ab, nullptr, F, W);
    EI_FEW(1, false, 1, 8, 8, down_experts, ab, d, nullptr, nullptr, out, W, F);
  } else if (N <= 32) {
    EI_FEW(2, true, 1, 8, 8, E, xb, g, u, ab, nullptr, F, W);
    EI_FEW(2, false, 1, 8, 8, down_experts, ab, d, nullptr, nullptr, out, W, F);
  } else {
    EI_FEW(4, true, 1, 8, 4, E, xb, g, u, ab, nullptr, F, W);
    EI_FEW(4, false, 4, 2, 6, down_experts, ab, d, nullptr, nullptr, out, W, F);
  }
#undef EI_FEW
  EI_LAUNCH_CHECK();
}
