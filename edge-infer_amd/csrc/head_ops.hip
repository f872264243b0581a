// Per-head operations around attention over a compressed (latent) cache, and the mixing of
// queries over heads.  All sums, norms, angles and rotations are float32; inputs may be the
// float32 slices of a sliced product (they are added in slice order while they are read).
//
//   latent_down_store  one row of a fused down-projection [queries' latent | keys' latent |
//                      rotated key part | gate logits]: RMS norm of the two latents, the
//                      queries' latent out in the storage type, the keys' latent and the
//                      rotated key part into the row's cache page (one row of
//                      kv_rank + rot_dim elements a position), the gate logits out as float32;
//                      where the queries lie in the same projection, their rotated parts as well
//   head_matmul        Y[n, h, :] = X[n, h, :] . M[h] for one matrix [in, out] a head; the result
//                      may be multiplied by the sigmoid of a gate an element, and X may be the merge of
//                      the slices that attention over a cut key range has left
//   heads_to_rows      rows of heads out of a product made head by head ([heads, N, J]): gated, or
//                      with every head's rotated part behind it
//   rotate_pairs       neighbouring elements (2i, 2i + 1) of a part of every head turn by
//                      position * frequency[i]
//   mix_heads          queries mixed over heads with a matrix T [heads, heads], kept apart by
//                      the kv head they meet: out[n, h, c, :] = sum over heads g of kv head c of
//                      T[h, g] q[n, g, :]
#include "common.h"
#include "few_rows.h"

namespace {

template <typename TI>
__device__ __forceinline__ float sliced(const TI* p, int nsplit, size_t split_stride) {
  float x = 0.f;
  for (int s = 0; s < nsplit; ++s) x += ei::to_f32<TI>(p[s * split_stride]);
  return x;
}

__device__ __forceinline__ float opened(float z) { return 1.0f / (1.0f + expf(-z)); }

template <typename TI, typename TO, typename TF>
__global__ void latent_down_store_kernel(
    const TI* __restrict__ proj, int nsplit, size_t split_stride, size_t row_stride, int P,
    const float* __restrict__ q_norm_w, const float* __restrict__ c_norm_w, float eps,
    const TF* __restrict__ freq, float turn_scale, const int32_t* __restrict__ row_pos,
    const int32_t* __restrict__ row_seq, const int32_t* __restrict__ page_table, int table_width,
    TO* __restrict__ q_latent, TO* __restrict__ k_pages, float* __restrict__ gate_out, int q_rank,
    int kv_rank, int rot_dim, int n_gate, int write_cache, const TI* __restrict__ turns, int heads,
    int turn_head, TO* __restrict__ turned, size_t turned_row, int turned_head) {
  extern __shared__ float row_values[];      // [P]
  __shared__ float scratch[16];
  const int row = blockIdx.x;
  const int seq = row_seq[row];
  if (seq < 0) return;                       // a padding row of a fixed-size batch
  const int pos = row_pos[row];
  const TI* src = proj + static_cast<size_t>(row) * row_stride;
  float sum_q = 0.f, sum_c = 0.f;
  for (int i = threadIdx.x; i < P; i += blockDim.x) {
    const float x = sliced<TI>(src + i, nsplit, split_stride);
    row_values[i] = x;
    if (i < q_rank) sum_q += x * x;
    else if (i < q_rank + kv_rank) sum_c += x * x;
  }
  if (turns) {                               // the queries' rotated parts, in the same launch
    const TI* from = turns + static_cast<size_t>(row) * row_stride;
    TO* to = turned + static_cast<size_t>(row) * turned_row;
    const int half = rot_dim / 2;
    for (int idx = threadIdx.x; idx < heads * half; idx += blockDim.x) {
      const int h = idx / half, i = idx % half;
      const float u = sliced<TI>(from + h * turn_head + 2 * i, nsplit, split_stride);
      const float v = sliced<TI>(from + h * turn_head + 2 * i + 1, nsplit, split_stride);
      float sn, cs;
      ei::turn_at<TO>(pos, freq[i], sn, cs);
      cs *= turn_scale;
      sn *= turn_scale;
      TO* dst = to + h * turned_head + 2 * i;
      dst[0] = ei::from_f32<TO>(u * cs - v * sn);
      dst[1] = ei::from_f32<TO>(v * cs + u * sn);
    }
  }
  if (P == 0) return;                        // a layer that only reads another layer's cache
  float inv_q = 1.0f;
  if (q_rank > 0)
    inv_q = 1.0f / sqrtf(ei::block_sum(sum_q, scratch) / static_cast<float>(q_rank) + eps);
  float inv_c = 1.0f;
  if (kv_rank > 0)
    inv_c = 1.0f / sqrtf(ei::block_sum(sum_c, scratch) / static_cast<float>(kv_rank) + eps);
  for (int i = threadIdx.x; i < q_rank; i += blockDim.x)
    q_latent[static_cast<size_t>(row) * q_rank + i] =
        ei::from_f32<TO>((row_values[i] * inv_q) * q_norm_w[i]);
  for (int h = threadIdx.x; h < n_gate; h += blockDim.x)
    gate_out[static_cast<size_t>(row) * n_gate + h] = row_values[q_rank + kv_rank + rot_dim + h];
  if (!write_cache) return;
  const int page = page_table[static_cast<size_t>(seq) * table_width + pos / EI_PAGE];
  if (page < 0) return;
  const int width = kv_rank + rot_dim;
  TO* dst = k_pages + (static_cast<size_t>(page) * EI_PAGE + pos % EI_PAGE) * width;
  for (int i = threadIdx.x; i < kv_rank; i += blockDim.x)
    dst[i] = ei::from_f32<TO>((row_values[q_rank + i] * inv_c) * c_norm_w[i]);
  const float* turn = row_values + q_rank + kv_rank;
  for (int i = threadIdx.x; i < rot_dim / 2; i += blockDim.x) {
    float sn, cs;
    ei::turn_at<TO>(pos, freq[i], sn, cs);
    cs *= turn_scale;
    sn *= turn_scale;
    const float u = turn[2 * i], v = turn[2 * i + 1];
    dst[kv_rank + 2 * i] = ei::from_f32<TO>(u * cs - v * sn);
    dst[kv_rank + 2 * i + 1] = ei::from_f32<TO>(v * cs + u * sn);
  }
}

constexpr int kMaxSlices = 64;

// What stands for x where attention has left a row's output in slices of the key range: unnormalised
// sums part_o [N, heads, slices, K], and per slice a maximum and a sum of weights part_ml [.., 2].
struct Slices {
  const float* part_o;
  const float* part_ml;
  int n;
};

// Block: head blockIdx.y, rows blockIdx.x * R .., output columns blockIdx.z * 64 + t % 64.
template <typename TI, typename TW, typename TO, typename TG, int R, int PARTS>
__global__ void __launch_bounds__(ei::kFewCols * PARTS)
head_matmul_kernel(const TI* __restrict__ x, int nsplit, size_t split_stride, long long x_row,
                   int x_head, int x_first, const TW* __restrict__ m, TO* __restrict__ y,
                   long long y_row, int y_head, int y_first, int N, int K, int J,
                   const TG* __restrict__ gate, int gate_slices, size_t gate_stride, size_t gate_row,
                   Slices slices) {
  __shared__ ei::FewRows<R, PARTS> few;
  __shared__ float weight[R][kMaxSlices];
  const int h = blockIdx.y, heads = gridDim.y;
  const int row0 = blockIdx.x * R;
  const int col = threadIdx.x % ei::kFewCols;
  const int j = blockIdx.z * ei::kFewCols + col;
  const TW* mh = m + static_cast<size_t>(h) * K * J;
  if (slices.part_o) {
    // a wave a row: what each slice of it counts for, over the sum of all
    const int lane = threadIdx.x % EI_WAVE;
    for (int r = threadIdx.x / EI_WAVE; r < R; r += PARTS) {
      if (row0 + r >= N) break;
      const float* ml = slices.part_ml +
                        (static_cast<size_t>(row0 + r) * heads + h) * slices.n * 2;
      const bool mine = lane < slices.n;
      const float m_own = mine ? ml[2 * lane] : -1.0e30f, l_own = mine ? ml[2 * lane + 1] : 0.f;
      const float m_all = ei::wave_max(m_own);
      const float f = mine ? expf(m_own - m_all) : 0.f;
      const float l = ei::wave_sum(l_own * f);
      weight[r][lane] = l > 0.f ? f / l : 0.f;
    }
    __syncthreads();
    few.product(mh, J, K, j, J - 1, [&](int r, int k) {
      if (row0 + r >= N) return 0.f;
      const float* po = slices.part_o +
                        (static_cast<size_t>(row0 + r) * heads + h) * slices.n * K + k;
      float v = 0.f;
      for (int s0 = 0; s0 < slices.n; s0 += 8) {            // eight slices per trip to memory
        float p[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) p[u] = s0 + u < slices.n ? po[static_cast<size_t>(s0 + u) * K] : 0.f;
#pragma unroll
        for (int u = 0; u < 8; ++u)
          if (s0 + u < slices.n) v = fmaf(p[u], weight[r][s0 + u], v);
      }
      return v;
    });
  } else {
    few.product(mh, J, K, j, J - 1, [&](int r, int k) {
      return row0 + r < N ? sliced<TI>(x + static_cast<size_t>(row0 + r) * x_row + h * x_head + x_first + k,
                                       nsplit, split_stride)
                          : 0.f;
    });
  }
  if (j >= J) return;
  for (int r = threadIdx.x / ei::kFewCols; r < R && row0 + r < N; r += PARTS) {
    float total = few.total(r, col);
    if (gate)      // (element j of head h has column h J + j)
      total *= opened(sliced<TG>(gate + (row0 + r) * gate_row + static_cast<size_t>(h) * J + j,
                                 gate_slices, gate_stride));
    y[static_cast<size_t>(row0 + r) * y_row + h * y_head + y_first + j] = ei::from_f32<TO>(total);
  }
}

template <typename TI, typename TO, typename TF>
__global__ void rotate_pairs_kernel(const TI* __restrict__ x, int nsplit, size_t split_stride,
                                    long long x_row, int x_head, int x_first,
                                    const TF* __restrict__ freq, float turn_scale,
                                    const int32_t* __restrict__ row_pos, TO* __restrict__ y,
                                    long long y_row, int y_head, int y_first, int heads, int half,
                                    size_t total) {
  const size_t start = static_cast<size_t>(blockIdx.x) * blockDim.x + threadIdx.x;
  const size_t step = static_cast<size_t>(gridDim.x) * blockDim.x;
  for (size_t idx = start; idx < total; idx += step) {
    const int i = static_cast<int>(idx % half);
    const int h = static_cast<int>((idx / half) % heads);
    const size_t row = idx / (static_cast<size_t>(half) * heads);
    const TI* src = x + row * x_row + h * x_head + x_first + 2 * i;
    const float u = sliced<TI>(src, nsplit, split_stride);
    const float v = sliced<TI>(src + 1, nsplit, split_stride);
    float sn, cs;
    ei::turn_at<TO>(row_pos[row], freq[i], sn, cs);
    cs *= turn_scale;
    sn *= turn_scale;
    TO* dst = y + row * y_row + h * y_head + y_first + 2 * i;
    dst[0] = ei::from_f32<TO>(u * cs - v * sn);
    dst[1] = ei::from_f32<TO>(v * cs + u * sn);
  }
}

// made [heads, N, J] -> y[n, h * y_head + 0..J), times the sigmoid of gate[n, h J + j] where there is
// a gate; with `turns`, the R elements of every head that follow its J are the rotated part of the
// same head, element pairs (2 i, 2 i + 1) of turns[n, h * turn_head + ..].  A thread makes two
// neighbouring elements (V = 2) or eight.
template <typename T, int V>
__global__ void heads_to_rows_kernel(const T* __restrict__ made, T* __restrict__ y, size_t y_row,
                                     int y_head, int heads, int J, size_t N,
                                     const T* __restrict__ gate, size_t gate_row,
                                     const T* __restrict__ turns, size_t turns_row, int turn_head,
                                     int R, const double* __restrict__ freq, float turn_scale,
                                     const int32_t* __restrict__ row_pos, size_t total) {
  const size_t start = static_cast<size_t>(blockIdx.x) * blockDim.x + threadIdx.x;
  const size_t step = static_cast<size_t>(gridDim.x) * blockDim.x;
  const int pieces = (J + R) / V;
  for (size_t idx = start; idx < total; idx += step) {
    const int at = static_cast<int>(idx % pieces) * V;
    const int h = static_cast<int>(idx / pieces % heads);
    const size_t n = idx / (static_cast<size_t>(pieces) * heads);
    float x[V];
    if (at < J) {
      const T* src = made + (static_cast<size_t>(h) * N + n) * J + at;
      if constexpr (V == 8) ei::VecN<T, 8>::load(src, x);
      else
#pragma unroll
        for (int e = 0; e < V; ++e) x[e] = ei::to_f32<T>(src[e]);
      if (gate) {
        const T* g = gate + n * gate_row + static_cast<size_t>(h) * J + at;
        float z[V];
        if constexpr (V == 8) ei::VecN<T, 8>::load(g, z);
        else
#pragma unroll
          for (int e = 0; e < V; ++e) z[e] = ei::to_f32<T>(g[e]);
#pragma unroll
        for (int e = 0; e < V; ++e) x[e] *= opened(z[e]);
      }
    } else {
      const T* src = turns + n * turns_row + static_cast<size_t>(h) * turn_head + at - J;
      float z[V];
      if constexpr (V == 8) ei::VecN<T, 8>::load(src, z);
      else
#pragma unroll
        for (int e = 0; e < V; ++e) z[e] = ei::to_f32<T>(src[e]);
      const int pos = row_pos[n];
#pragma unroll
      for (int e = 0; e < V; e += 2) {
        float sn, cs;
        ei::turn_at<T>(pos, freq[(at - J + e) / 2], sn, cs);
        cs *= turn_scale;
        sn *= turn_scale;
        x[e] = z[e] * cs - z[e + 1] * sn;
        x[e + 1] = z[e + 1] * cs + z[e] * sn;
      }
    }
    T* dst = y + n * y_row + static_cast<size_t>(h) * y_head + at;
    if constexpr (V == 8) ei::VecN<T, 8>::store(dst, x);
    else
#pragma unroll
      for (int e = 0; e < V; ++e) dst[e] = ei::from_f32<T>(x[e]);
  }
}

template <typename T>
__global__ void mix_heads_kernel(const T* __restrict__ q, const float* __restrict__ talk,
                                 T* __restrict__ out, int heads, int kv_heads, int D,
                                 size_t total) {
  const size_t start = static_cast<size_t>(blockIdx.x) * blockDim.x + threadIdx.x;
  const size_t step = static_cast<size_t>(gridDim.x) * blockDim.x;
  const int share = heads / kv_heads;
  for (size_t idx = start; idx < total; idx += step) {
    const int d = static_cast<int>(idx % D);
    const int c = static_cast<int>((idx / D) % kv_heads);
    const int h = static_cast<int>((idx / (static_cast<size_t>(D) * kv_heads)) % heads);
    const size_t row = idx / (static_cast<size_t>(D) * kv_heads * heads);
    const T* src = q + (row * heads + static_cast<size_t>(c) * share) * D + d;
    const float* t = talk + static_cast<size_t>(h) * heads + c * share;
    float sum = 0.f;
    for (int g = 0; g < share; ++g) sum += t[g] * ei::to_f32<T>(src[static_cast<size_t>(g) * D]);
    out[idx] = ei::from_f32<T>(sum);
  }
}

// The same for head sizes that are a multiple of 8: a thread makes 8 neighbouring elements
// (16-byte accesses in bfloat16).
template <typename T>
__global__ void mix_heads_vec_kernel(const T* __restrict__ q, const float* __restrict__ talk,
                                     T* __restrict__ out, int heads, int kv_heads, int D,
                                     size_t total_octets) {
  const size_t start = static_cast<size_t>(blockIdx.x) * blockDim.x + threadIdx.x;
  const size_t step = static_cast<size_t>(gridDim.x) * blockDim.x;
  const int share = heads / kv_heads;
  const int octets = D / 8;
  for (size_t idx = start; idx < total_octets; idx += step) {
    const int d = static_cast<int>(idx % octets) * 8;
    const int c = static_cast<int>((idx / octets) % kv_heads);
    const int h = static_cast<int>((idx / (static_cast<size_t>(octets) * kv_heads)) % heads);
    const size_t row = idx / (static_cast<size_t>(octets) * kv_heads * heads);
    const T* src = q + (row * heads + static_cast<size_t>(c) * share) * D + d;
    const float* t = talk + static_cast<size_t>(h) * heads + c * share;
    float sum[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) sum[e] = 0.f;
    for (int g = 0; g < share; ++g) {
      float x[8];
      ei::VecN<T, 8>::load(src + static_cast<size_t>(g) * D, x);
      const float w = t[g];
#pragma unroll
      for (int e = 0; e < 8; ++e) sum[e] += w * x[e];
    }
    ei::VecN<T, 8>::store(out + idx * 8, sum);
  }
}

inline unsigned capped_blocks(size_t n, int threads) {
  size_t blocks = (n + threads - 1) / threads;
  const size_t most = static_cast<size_t>(ei_compute_units()) * 16;
  return static_cast<unsigned>(blocks > most ? most : (blocks < 1 ? 1 : blocks));
}

}  // namespace

// proj: [nsplit][N, row_stride], rows that begin with q_rank + kv_rank + rot_dim + n_gate columns
// (q_rank 0: the queries have no latent; kv_rank 0: the layer caches nothing, and rot_dim then
// only serves the queries); k_pages: [pages, 1, 64, kv_rank + rot_dim].  freq: [rot_dim / 2] of
// float32 or (freq_double) float64; turn_scale multiplies cosine and sine.  turns (or null): the
// first rotated query element in the first row of the same projection, heads turn_head apart;
// turned: where the first one goes, rows turned_row and heads turned_head apart.
extern "C" int ei_latent_down_store(const void* proj, int in_dtype, int nsplit,
                                    long long split_stride, long long row_stride,
                                    const float* q_norm_w,
                                    const float* c_norm_w, float eps, const void* freq,
                                    int freq_double, float turn_scale,
                                    const int32_t* row_pos, const int32_t* row_seq,
                                    const int32_t* page_table, int table_width, void* q_latent,
                                    void* k_pages, float* gate_out, int out_dtype, int N, int q_rank,
                                    int kv_rank, int rot_dim, int n_gate, int write_cache,
                                    const void* turns, int heads, int turn_head, void* turned,
                                    long long turned_row, int turned_head, hipStream_t stream) {
  EI_REQUIRE(N > 0 && q_rank >= 0 && kv_rank >= 0 && rot_dim >= 0 && rot_dim % 2 == 0 && n_gate >= 0,
             "latent_down_store: bad sizes");
  EI_REQUIRE(proj && row_pos && row_seq && nsplit >= 1 && (q_rank == 0 || (q_norm_w && q_latent)) &&
                 (kv_rank == 0 || c_norm_w),
             "latent_down_store: null pointer");
  EI_REQUIRE(rot_dim == 0 || freq, "latent_down_store: a rotation needs its frequencies");
  EI_REQUIRE(n_gate == 0 || gate_out, "latent_down_store: gate logits need a place");
  EI_REQUIRE(!write_cache || (k_pages && page_table && table_width > 0 && kv_rank > 0),
             "latent_down_store: the cache is missing");
  EI_REQUIRE(!turns || (turned && heads > 0 && rot_dim > 0 && turn_head >= rot_dim &&
                        turned_head >= rot_dim &&
                        static_cast<long long>(heads - 1) * turned_head + rot_dim <= turned_row),
             "latent_down_store: the queries' rotated parts do not fit their rows");
  const int P = kv_rank == 0 ? q_rank + n_gate : q_rank + kv_rank + rot_dim + n_gate;
  EI_REQUIRE(kv_rank > 0 || (q_rank == 0 && n_gate == 0),
             "latent_down_store: without a latent the queries' rotated parts are all there is");
  EI_REQUIRE(row_stride >= P, "latent_down_store: rows narrower than their parts");
  const size_t lds = static_cast<size_t>(P) * sizeof(float);
  EI_REQUIRE(lds <= 60 * 1024, "latent_down_store: row too wide");
  // few rows: up to 1024 threads a row, so that a row's loads are in flight together
  const int work = P > heads * rot_dim / 2 ? P : heads * rot_dim / 2;
  const int threads = N <= 64 ? (work >= 768 ? 1024 : 512) : 256;
  const size_t ss = static_cast<size_t>(split_stride), rs = static_cast<size_t>(row_stride);
#define EI_LDS_CASE_F(TI, TO, TF)                                                               \
  latent_down_store_kernel<TI, TO, TF><<<N, threads, lds, stream>>>(                            \
      static_cast<const TI*>(proj), nsplit, ss, rs, P, q_norm_w, c_norm_w, eps,                 \
      static_cast<const TF*>(freq), turn_scale, row_pos, row_seq, page_table, table_width,      \
      static_cast<TO*>(q_latent), static_cast<TO*>(k_pages), gate_out, q_rank, kv_rank, rot_dim, \
      n_gate, write_cache, static_cast<const TI*>(turns), heads, turn_head,                     \
      static_cast<TO*>(turned), static_cast<size_t>(turned_row), turned_head)
#define EI_LDS_CASE(TI, TO)                         \
  do {                                              \
    if (freq_double) EI_LDS_CASE_F(TI, TO, double); \
    else EI_LDS_CASE_F(TI, TO, float);              \
  } while (0)
  if (in_dtype == EI_F32 && out_dtype == EI_F32) EI_LDS_CASE(float, float);
  else if (in_dtype == EI_F32 && out_dtype == EI_BF16) EI_LDS_CASE(float, bf16_t);
  else if (in_dtype == EI_BF16 && out_dtype == EI_BF16) EI_LDS_CASE(bf16_t, bf16_t);
  else EI_REQUIRE(false, "latent_down_store: unsupported dtype combination");
#undef EI_LDS_CASE
#undef EI_LDS_CASE_F
  EI_LAUNCH_CHECK();
}

// x: [nsplit][N, x_row] read at x_head * h + x_first + 0..K; m: [heads, K, J] of the storage
// type; y: [N, y_row] written at y_head * h + y_first + 0..J.  gate (or null): gate_slices slices
// of rows gate_row apart; element j of head h is multiplied by the sigmoid of column h J + j.
// n_slices > 0: x is not read, the rows come from part_o [N, heads, n_slices, K] and part_ml [N,
// heads, n_slices, 2] as a sliced attention kernel leaves them.
extern "C" int ei_head_matmul(const void* x, int x_dtype, int nsplit, long long split_stride,
                              long long x_row, int x_head, int x_first, const void* m,
                              int m_dtype, void* y, int y_dtype, long long y_row, int y_head,
                              int y_first, int N, int heads, int K, int J, const void* gate,
                              int gate_dtype, int gate_slices, long long gate_stride,
                              long long gate_row, const float* part_o, const float* part_ml,
                              int n_slices, hipStream_t stream) {
  EI_REQUIRE(!gate || (gate_slices >= 1 && gate_row >= static_cast<long long>(heads) * J &&
                       (gate_dtype == EI_F32 || gate_dtype == EI_BF16)),
             "head_matmul: a gate's row holds one column an element");
  EI_REQUIRE(N > 0 && heads > 0 && K > 0 && J > 0, "head_matmul: bad sizes");
  EI_REQUIRE(m && y, "head_matmul: null pointer");
  EI_REQUIRE(n_slices >= 0 && n_slices <= kMaxSlices && (n_slices == 0 || (part_o && part_ml)),
             "head_matmul: at most 64 slices, with their sums and weights");
  EI_REQUIRE(n_slices > 0 || (x && nsplit >= 1 && x_first >= 0 &&
                              static_cast<long long>(heads - 1) * x_head + x_first + K <= x_row),
             "head_matmul: a head's part lies outside its row of x");
  EI_REQUIRE(y_first >= 0 && static_cast<long long>(heads - 1) * y_head + y_first + J <= y_row,
             "head_matmul: a head's part lies outside its row of y");
  const int col_blocks = (J + ei::kFewCols - 1) / ei::kFewCols;
  EI_REQUIRE(heads <= 65535 && col_blocks <= 65535, "head_matmul: too many heads or columns");
  const Slices slices{n_slices > 0 ? part_o : nullptr, part_ml, n_slices};
  if (n_slices > 0) x_dtype = m_dtype;
  const size_t ss = static_cast<size_t>(split_stride);
  // rows a block takes: all of a decode step's few, more where weights are used by many rows
  const int rows = N == 1 ? 1 : (N <= 64 ? 8 : 16);
  const bool deep = K > 4 * ei::kFewK && rows < 16;        // 16 threads a column instead of 4
  const dim3 grid((N + rows - 1) / rows, heads, col_blocks);
#define EI_HM_RP(TI, TW, TO, TG, RR, PP)                                                          \
  head_matmul_kernel<TI, TW, TO, TG, RR, PP><<<grid, ei::kFewCols * PP, 0, stream>>>(             \
      static_cast<const TI*>(x), nsplit, ss, x_row, x_head, x_first, static_cast<const TW*>(m),   \
      static_cast<TO*>(y), y_row, y_head, y_first, N, K, J, static_cast<const TG*>(gate),         \
      gate_slices, static_cast<size_t>(gate_stride), static_cast<size_t>(gate_row), slices)
#define EI_HM_CASE_G(TI, TW, TO, TG)                              \
  do {                                                            \
    if (rows == 1 && deep) EI_HM_RP(TI, TW, TO, TG, 1, 16);       \
    else if (rows == 1) EI_HM_RP(TI, TW, TO, TG, 1, 4);           \
    else if (rows == 8 && deep) EI_HM_RP(TI, TW, TO, TG, 8, 16);  \
    else if (rows == 8) EI_HM_RP(TI, TW, TO, TG, 8, 4);           \
    else EI_HM_RP(TI, TW, TO, TG, 16, 4);                         \
  } while (0)
#define EI_HM_CASE(TI, TW, TO)                                          \
  do {                                                                  \
    if (gate && gate_dtype == EI_BF16) EI_HM_CASE_G(TI, TW, TO, bf16_t); \
    else EI_HM_CASE_G(TI, TW, TO, float);                               \
  } while (0)
  if (x_dtype == EI_F32 && m_dtype == EI_F32 && y_dtype == EI_F32) EI_HM_CASE(float, float, float);
  else if (x_dtype == EI_F32 && m_dtype == EI_BF16 && y_dtype == EI_BF16) EI_HM_CASE(float, bf16_t, bf16_t);
  else if (x_dtype == EI_BF16 && m_dtype == EI_BF16 && y_dtype == EI_BF16) EI_HM_CASE(bf16_t, bf16_t, bf16_t);
  else EI_REQUIRE(false, "head_matmul: unsupported dtype combination");
#undef EI_HM_CASE
#undef EI_HM_CASE_G
#undef EI_HM_RP
  EI_LAUNCH_CHECK();
}

extern "C" int ei_rotate_pairs(const void* x, int x_dtype, int nsplit, long long split_stride,
                               long long x_row, int x_head, int x_first, const void* freq,
                               int freq_double, float turn_scale,
                               const int32_t* row_pos, void* y, int y_dtype, long long y_row,
                               int y_head, int y_first, int N, int heads, int rot_dim,
                               hipStream_t stream) {
  EI_REQUIRE(N > 0 && heads > 0 && rot_dim > 0 && rot_dim % 2 == 0 && nsplit >= 1,
             "rotate_pairs: bad sizes");
  EI_REQUIRE(x && y && freq && row_pos, "rotate_pairs: null pointer");
  EI_REQUIRE(x_first >= 0 && y_first >= 0 &&
                 static_cast<long long>(heads - 1) * x_head + x_first + rot_dim <= x_row &&
                 static_cast<long long>(heads - 1) * y_head + y_first + rot_dim <= y_row,
             "rotate_pairs: a head's part lies outside its row");
  const int half = rot_dim / 2;
  const size_t total = static_cast<size_t>(N) * heads * half;
  const size_t ss = static_cast<size_t>(split_stride);
  const unsigned blocks = capped_blocks(total, 256);
#define EI_RP_CASE_F(TI, TO, TF)                                                               \
  rotate_pairs_kernel<TI, TO, TF><<<blocks, 256, 0, stream>>>(                                 \
      static_cast<const TI*>(x), nsplit, ss, x_row, x_head, x_first,                           \
      static_cast<const TF*>(freq), turn_scale, row_pos, static_cast<TO*>(y), y_row, y_head,   \
      y_first, heads, half, total)
#define EI_RP_CASE(TI, TO)                         \
  do {                                             \
    if (freq_double) EI_RP_CASE_F(TI, TO, double); \
    else EI_RP_CASE_F(TI, TO, float);              \
  } while (0)
  if (x_dtype == EI_F32 && y_dtype == EI_F32) EI_RP_CASE(float, float);
  else if (x_dtype == EI_F32 && y_dtype == EI_BF16) EI_RP_CASE(float, bf16_t);
  else if (x_dtype == EI_BF16 && y_dtype == EI_BF16) EI_RP_CASE(bf16_t, bf16_t);
  else EI_REQUIRE(false, "rotate_pairs: unsupported dtype combination");
#undef EI_RP_CASE
#undef EI_RP_CASE_F
  EI_LAUNCH_CHECK();
}

// made: [heads, N, J] of `dtype`; y: rows y_row, heads y_head elements apart.  gate (or null): rows
// gate_row apart, one column an element [heads * J].  turns (or null): every head's rotated part of
// R elements follows its J in y, made from turns (rows turns_row, heads turn_head apart) with
// float64 frequencies [R / 2]; J, R even.
extern "C" int ei_heads_to_rows(const void* made, int dtype, void* y, long long y_row, int y_head,
                                int N, int heads, int J, const void* gate, long long gate_row,
                                const void* turns, long long turns_row, int turn_head, int R,
                                const double* freq, float turn_scale, const int32_t* row_pos,
                                hipStream_t stream) {
  if (!turns) R = 0;
  EI_REQUIRE(made && y && N > 0 && heads > 0 && J > 0 && R >= 0 && J % 2 == 0 && R % 2 == 0,
             "heads_to_rows: bad sizes");
  EI_REQUIRE(y_head >= J + R && static_cast<long long>(heads - 1) * y_head + J + R <= y_row,
             "heads_to_rows: a head's part lies outside its row");
  EI_REQUIRE(!gate || gate_row >= static_cast<long long>(heads) * J,
             "heads_to_rows: a gate's row holds one column an element");
  EI_REQUIRE(!turns || (R > 0 && freq && row_pos && turn_head >= R &&
                        static_cast<long long>(heads - 1) * turn_head + R <= turns_row),
             "heads_to_rows: the rotated parts lie outside their rows");
  const auto aligned16 = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  const bool vec = J % 8 == 0 && R % 8 == 0 && y_row % 8 == 0 && y_head % 8 == 0 && aligned16(made) &&
                   aligned16(y) && (!gate || (gate_row % 8 == 0 && aligned16(gate))) &&
                   (!turns || (turns_row % 8 == 0 && turn_head % 8 == 0 && aligned16(turns)));
  const size_t total = static_cast<size_t>(N) * heads * ((J + R) / (vec ? 8 : 2));
  const unsigned blocks = capped_blocks(total, 256);
#define EI_HR_CASE(T, V)                                                                          \
  heads_to_rows_kernel<T, V><<<blocks, 256, 0, stream>>>(                                         \
      static_cast<const T*>(made), static_cast<T*>(y), static_cast<size_t>(y_row), y_head, heads, \
      J, static_cast<size_t>(N), static_cast<const T*>(gate), static_cast<size_t>(gate_row),      \
      static_cast<const T*>(turns), static_cast<size_t>(turns_row), turn_head, R, freq,           \
      turn_scale, row_pos, total)
  if (dtype == EI_F32) {
    if (vec) EI_HR_CASE(float, 8);
    else EI_HR_CASE(float, 2);
  } else if (dtype == EI_BF16) {
    if (vec) EI_HR_CASE(bf16_t, 8);
    else EI_HR_CASE(bf16_t, 2);
  } else {
    EI_REQUIRE(false, "heads_to_rows: unknown dtype");
  }
#undef EI_HR_CASE
  EI_LAUNCH_CHECK();
}

// q: [N, heads, D]; talk: float32 [heads, heads]; out: [N, heads, kv_heads, D].
extern "C" int ei_mix_heads(const void* q, int dtype, const float* talk, void* out, int N,
                            int heads, int kv_heads, int D, hipStream_t stream) {
  EI_REQUIRE(N > 0 && heads > 0 && kv_heads > 0 && D > 0 && heads % kv_heads == 0,
             "mix_heads: bad sizes");
  EI_REQUIRE(q && talk && out, "mix_heads: null pointer");
  const size_t total = static_cast<size_t>(N) * heads * kv_heads * D;
  if (D % 8 == 0) {
    const size_t octets = total / 8;
    const unsigned vblocks = capped_blocks(octets, 256);
    if (dtype == EI_F32)
      mix_heads_vec_kernel<float><<<vblocks, 256, 0, stream>>>(
          static_cast<const float*>(q), talk, static_cast<float*>(out), heads, kv_heads, D, octets);
    else if (dtype == EI_BF16)
      mix_heads_vec_kernel<bf16_t><<<vblocks, 256, 0, stream>>>(
          static_cast<const bf16_t*>(q), talk, static_cast<bf16_t*>(out), heads, kv_heads, D, octets);
    else
      EI_REQUIRE(false, "mix_heads: unknown dtype");
    EI_LAUNCH_CHECK();
  }
  const unsigned blocks = capped_blocks(total, 256);
  if (dtype == EI_F32)
    mix_heads_kernel<float><<<blocks, 256, 0, stream>>>(
        static_cast<const float*>(q), talk, static_cast<float*>(out), heads, kv_heads, D, total);
  else if (dtype == EI_BF16)
    mix_heads_kernel<bf16_t><<<blocks, 256, 0, stream>>>(
        static_cast<const bf16_t*>(q), talk, static_cast<bf16_t*>(out), heads, kv_heads, D, total);
  else
    EI_REQUIRE(false, "mix_heads: unknown dtype");
  EI_LAUNCH_CHECK();
}
