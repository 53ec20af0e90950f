// Attention to cached latents. The cache holds, per token, one row of W numbers: the normed latent (`rank`), the rotated
// key part that all heads share (`rot_dim`), zeros up to W (a multiple of 32); pages are [64][W]. With a head's matrices
// from the latent to its plain key and its value (U_k [dim, rank], U_v [vdim, rank]),
//
//   score = (q_plain . U_k c + q_rot . k_rot) * scale = ([U_k^T q_plain | q_rot] . [c | k_rot]) * scale
//   out   = sum_j p_j U_v c_j = U_v (sum_j p_j c_j)
//
// so every head attends to the same rows: the query is taken to the latent's side first, the weighted sum of latents
// back to the value's side afterwards. Scores, softmax and both norms are float arithmetic in both precisions.
#include "common.h"

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(8))) uint16_t u16x8;
#define MFMA16(a, b, c) __builtin_amdgcn_mfma_f32_16x16x32_bf16((a), (b), (c), 0, 0, 0)

#define MLA_MAX_WIDTH 960          // features of a cached row; half a page and a tile of queries wait in LDS

// ---------------------------------------------------------------------------------------------------
// What a step's rows bring: `src` holds, per row, the queries' latent | the keys' latent | the key part to be rotated (the
// float partial sums of a split product, or the activation dtype). c_q = rms(.) * w_q; c = rms(.) * w_kv goes to the
// row's place in its page (and to c_out when asked for), the key part after it, turned by pairs (feature 2i with 2i + 1)
// of its first `rot` features. rank = 0: only the queries' latent. A workgroup a row; the row waits in LDS.
template <typename T, typename D>
__global__ __launch_bounds__(256) void latent_rows_in_kernel(
    const D* __restrict__ src, int64_t stride, int n_partials, int64_t partial_stride, const float* __restrict__ w_q,
    T* __restrict__ c_q, int q_rank, const float* __restrict__ w_kv, T* __restrict__ c_out, int rank, int rot_dim,
    const float* __restrict__ cos_t, const float* __restrict__ sin_t, int rot, int pairs, float eps,
    const int* __restrict__ row_slot, const int* __restrict__ row_pos, T* __restrict__ pages,
    const int* __restrict__ page_table, int max_pages, int width, int write_kv) {
  extern __shared__ float held[];
  __shared__ float scratch[16];
  const int64_t row = blockIdx.x;
  const int total = q_rank + (rank ? rank + rot_dim : 0);
  float sq = 0.f, sk = 0.f;
  for (int i = threadIdx.x; i < total; i += blockDim.x) {
    float v = 0.f;
    int p = 0;
    for (; p + 4 <= n_partials; p += 4) {                            // four loads in flight; added in the order 0, 1, ...
      float t[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) t[u] = load_as_float(src + (p + u) * partial_stride + row * stride + i);
#pragma unroll
      for (int u = 0; u < 4; ++u) v += t[u];
    }
    for (; p < n_partials; ++p) v += load_as_float(src + p * partial_stride + row * stride + i);
    held[i] = v;
    if (i < q_rank) sq += v * v;
    else if (i < q_rank + rank) sk += v * v;
  }
  sq = block_sum(sq, scratch);
  const float rq = rsqrtf(sq / (float)q_rank + eps);
  for (int i = threadIdx.x; i < q_rank; i += blockDim.x) store_from_float(c_q + row * q_rank + i, held[i] * rq * w_q[i]);
  if (rank == 0) return;
  sk = block_sum(sk, scratch);
  const float rk = rsqrtf(sk / (float)rank + eps);
  const int slot = row_slot[row], pos = row_pos[row];
  const int page = (slot >= 0 && write_kv) ? page_of(page_table, max_pages, slot, pos) : -1;
  T* dst = pages + ((int64_t)(page < 0 ? 0 : page) * PAGE_TOKENS + pos % PAGE_TOKENS) * width;
  const float* lat = held + q_rank;
  for (int i = threadIdx.x; i < rank; i += blockDim.x) {
    const float v = lat[i] * rk * w_kv[i];
    if (c_out != nullptr) store_from_float(c_out + row * rank + i, v);
    if (page >= 0) store_from_float(dst + i, v);
  }
  if (page < 0) return;
  const float* key = lat + rank;
  const int half = rot / 2;
  for (int i = threadIdx.x; i < rot_dim; i += blockDim.x) {
    float v = key[i];
    if (i < rot) {
      const int f = pairs ? i / 2 : i % half;
      const bool low = pairs ? i % 2 == 0 : i < half;
      const float other = key[pairs ? i ^ 1 : (low ? i + half : i - half)];
      const float c = cos_t[(int64_t)pos * half + f], s = sin_t[(int64_t)pos * half + f];
      v = low ? v * c - other * s : v * c + other * s;
    }
    store_from_float(dst + rank + i, v);
  }
}

DRYFT_API int dryft_latent_rows_in(const void* src, int kind, int64_t stride, int n_partials, int64_t partial_stride,
                                   const float* w_q, void* c_q, int q_rank, const float* w_kv, void* c_out, int rank,
                                   int rot_dim, const float* cos_t, const float* sin_t, int rot, int pairs, float eps,
                                   const int* row_slot, const int* row_pos, void* pages, const int* page_table,
                                   int max_pages, int width, int write_kv, int n_rows, int is_f32, hipStream_t stream) {
  if (n_rows <= 0) return 0;
  if (q_rank <= 0 || rank < 0 || rot_dim < 0 || rot < 0 || rot % 2 || rot > rot_dim || rank + rot_dim > width) return -1;
  const size_t lds = (size_t)(q_rank + rank + rot_dim) * sizeof(float);
  if (lds > 64 * 1024) return -1;
#define LR(TT, DD)                                                                                                   \
  hipLaunchKernelGGL((latent_rows_in_kernel<TT, DD>), dim3(n_rows), dim3(256), lds, stream, (const DD*)src, stride,    \
                     n_partials, partial_stride, w_q, (TT*)c_q, q_rank, w_kv, (TT*)c_out, rank, rot_dim, cos_t, sin_t, \
                     rot, pairs, eps, row_slot, row_pos, (TT*)pages, page_table, max_pages, width, write_kv)
  if (is_f32) LR(float, float);
  else if (kind == 2) LR(bf16_t, float);
  else LR(bf16_t, bf16_t);
#undef LR
  return DRYFT_LAUNCH_CHECK();
}

// ---------------------------------------------------------------------------------------------------
// A matrix per head: y[row, y_col + h y_head + n] = sum_k x[row, x_col + h x_head + k] M[h][n][k], n < N, k < K; M is
// [heads][N padded to 16][K padded to 32] with zeros behind. With `rot_dim` > 0 one more block of the grid's last
// dimension takes what lies after the head's K features, x[.. K + i], to y[.. N + i], its first `rot` features turned (by
// pairs, or over halves) at the row's position, and zeros up to y_head: the queries of the kernels below.
// Float32: plain multiply-adds. bfloat16: the matrix cores, a wave 16 outputs by 16 rows, M as the first operand.
template <typename T>
__device__ __forceinline__ void turn_tail(const T* __restrict__ x, int64_t x_stride, int x_col, int x_head, int K,
                                          T* __restrict__ y, int64_t y_stride, int y_head, int N, int rows, int row0,
                                          int head, int rot_dim, const float* __restrict__ cos_t,
                                          const float* __restrict__ sin_t, int rot, int pairs,
                                          const int* __restrict__ row_pos) {
  const int tail = y_head - N, half = rot / 2;
  for (int e = threadIdx.x; e < 16 * tail; e += blockDim.x) {
    const int row = row0 + e / tail, i = e % tail;
    if (row >= rows) continue;
    const T* src = x + row * x_stride + x_col + (int64_t)head * x_head + K;
    float v = i < rot_dim ? load_as_float(src + i) : 0.f;
    if (i < rot) {
      const int f = pairs ? i / 2 : i % half;
      const bool low = pairs ? i % 2 == 0 : i < half;
      const float other = load_as_float(src + (pairs ? i ^ 1 : (low ? i + half : i - half)));
      const int64_t pos = row_pos[row];
      const float c = cos_t[pos * half + f], s = sin_t[pos * half + f];
      v = low ? v * c - other * s : v * c + other * s;
    }
    store_from_float(y + row * y_stride + (int64_t)head * y_head + N + i, v);
  }
}

__global__ __launch_bounds__(256) void head_product_kernel(
    const bf16_t* __restrict__ x, int64_t x_stride, int x_col, int x_head, const bf16_t* __restrict__ m, int K, int Kp, int N,
    int Np, bf16_t* __restrict__ y, int64_t y_stride, int y_head, int rows, int vec, int rot_dim,
    const float* __restrict__ cos_t, const float* __restrict__ sin_t, int rot, int pairs, const int* __restrict__ row_pos) {
  const int row0 = blockIdx.x * 16, head = blockIdx.y, n_groups = (Np + 63) / 64;
  if ((int)blockIdx.z == n_groups) {
    turn_tail(x, x_stride, x_col, x_head, K, y, y_stride, y_head, N, rows, row0, head, rot_dim, cos_t, sin_t, rot, pairs,
              row_pos);
    return;
  }
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE, g = lane / 16, c = lane % 16;
  const int n0 = blockIdx.z * 64 + wave * 16;
  if (n0 >= Np) return;
  const int row = min(row0 + c, rows - 1);
  const bf16_t* xr = x + row * x_stride + x_col + (int64_t)head * x_head;
  const bf16_t* mr = m + ((int64_t)head * Np + n0 + c) * Kp + 8 * g;
  vf4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 8
  for (int k0 = 0; k0 < Kp; k0 += 32) {
    const int k = k0 + 8 * g;
    const bf16x8 a = *(const bf16x8*)(mr + k0);
    u16x8 b;
    if (vec) {
      b = k < K ? *(const u16x8*)(xr + k) : u16x8{0, 0, 0, 0, 0, 0, 0, 0};
    } else {
#pragma unroll
      for (int j = 0; j < 8; ++j) b[j] = k + j < K ? xr[k + j].bits : 0;
    }
    acc = MFMA16(a, __builtin_bit_cast(bf16x8, b), acc);
  }
  if (row0 + c >= rows) return;
  bf16_t* out = y + (row0 + c) * y_stride + (int64_t)head * y_head + n0 + 4 * g;
#pragma unroll
  for (int r = 0; r < 4; ++r)
    if (n0 + 4 * g + r < N) out[r] = float_to_bf16(acc[r]);
}

__global__ __launch_bounds__(256) void head_product_f32_kernel(
    const float* __restrict__ x, int64_t x_stride, int x_col, int x_head, const float* __restrict__ m, int K, int Kp, int N,
    int Np, float* __restrict__ y, int64_t y_stride, int y_head, int rows, int rot_dim, const float* __restrict__ cos_t,
    const float* __restrict__ sin_t, int rot, int pairs, const int* __restrict__ row_pos) {
  const int row0 = blockIdx.x * 16, head = blockIdx.y, n_groups = (Np + 63) / 64;
  if ((int)blockIdx.z == n_groups) {
    turn_tail(x, x_stride, x_col, x_head, K, y, y_stride, y_head, N, rows, row0, head, rot_dim, cos_t, sin_t, rot, pairs,
              row_pos);
    return;
  }
  for (int e = threadIdx.x; e < 16 * 64; e += 256) {
    const int row = row0 + e / 64, n = blockIdx.z * 64 + e % 64;
    if (row >= rows || n >= N) continue;
    const float* xr = x + row * x_stride + x_col + (int64_t)head * x_head;
    const float* mr = m + ((int64_t)head * Np + n) * Kp;
    float acc = 0.f;
    for (int k = 0; k < K; ++k) acc += xr[k] * mr[k];
    y[row * y_stride + (int64_t)head * y_head + n] = acc;
  }
}

DRYFT_API int dryft_head_product(const void* x, int64_t x_stride, int x_col, int x_head, const void* m, int K, int Kp, int N,
                                 int Np, void* y, int64_t y_stride, int y_head, int rows, int heads, int rot_dim,
                                 const float* cos_t, const float* sin_t, int rot, int pairs, const int* row_pos, int is_f32,
                                 hipStream_t stream) {
  if (rows <= 0) return 0;
  if (heads <= 0 || K <= 0 || N <= 0 || K > Kp || Kp % 32 || N > Np || Np % 16 || y_head < N) return -1;
  if (rot < 0 || rot % 2 || rot > rot_dim || (rot_dim > 0 && N + rot_dim > y_head)) return -1;
  const dim3 grid((rows + 15) / 16, heads, (Np + 63) / 64 + (rot_dim > 0 ? 1 : 0));
  if (is_f32) {
    hipLaunchKernelGGL(head_product_f32_kernel, grid, dim3(256), 0, stream, (const float*)x, x_stride, x_col, x_head,
                       (const float*)m, K, Kp, N, Np, (float*)y, y_stride, y_head, rows, rot_dim, cos_t, sin_t, rot, pairs,
                       row_pos);
  } else {
    const int vec = K % 8 == 0 && x_col % 8 == 0 && x_head % 8 == 0 && x_stride % 8 == 0 && ((uintptr_t)x & 15) == 0;
    hipLaunchKernelGGL(head_product_kernel, grid, dim3(256), 0, stream, (const bf16_t*)x, x_stride, x_col, x_head,
                       (const bf16_t*)m, K, Kp, N, Np, (bf16_t*)y, y_stride, y_head, rows, vec, rot_dim, cos_t, sin_t, rot,
                       pairs, row_pos);
  }
  return DRYFT_LAUNCH_CHECK();
}

// ---------------------------------------------------------------------------------------------------
// bfloat16: a workgroup takes a tile of up to 16 (row, head) pairs of one sequence (all heads of one row, or several
// rows' where a row has few) and one run of the sequence's half pages (32 positions). The pairs are the 16 columns of both
// products. S^T = K Q^T: a wave takes 16 of the 32 positions and half of the features, and leaves its part of the scores
// in LDS, from where every lane takes the scores of exactly the 8 positions that it contributes to the second product,
// O^T = C^T P^T, whose features the waves deal out among themselves. Half a page lies in LDS row by row; the second
// product's first operand gathers 8 positions of a feature from it. The next half page's loads are in flight
// meanwhile. Each run leaves its maximum, sum and weighted sum of latents (float); `latent_combine` joins them in order.
#define LATENT_KEYS 32

// NT: feature tiles of 16 a wave owns at most; NL: 16-byte pieces of half a page a thread brings in at most
template <int NT, int NL>
__global__ __launch_bounds__(256) void latent_split_kernel(
    const bf16_t* __restrict__ q, const bf16_t* __restrict__ pages, const int* __restrict__ page_table, int max_pages,
    const int* __restrict__ seq_slot, const int* __restrict__ cu_rows, const int* __restrict__ q_len,
    const int* __restrict__ seq_start, const int* __restrict__ tile_cu, int n_seqs, int H, int width, int rank, float scale,
    float* __restrict__ part_o, float* __restrict__ part_ml, int splits) {
  extern __shared__ __attribute__((aligned(16))) char lds_raw[];
  const int ws = width + 8;
  vf4* s_part = (vf4*)lds_raw;                           // [4 waves][64 lanes]
  bf16_t* page_s = (bf16_t*)(s_part + 256);              // [32][ws]
  bf16_t* q_s = page_s + LATENT_KEYS * ws;               // [16][ws]
  if ((int)blockIdx.x >= tile_cu[n_seqs]) return;
  int seq = 0;
  while (tile_cu[seq + 1] <= (int)blockIdx.x) ++seq;
  const int slot = seq_slot[seq];
  if (slot < 0) return;
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid % WAVE, g = lane / 16, c = lane % 16;
  const int hc = H < 16 ? H : 16, rt = 16 / hc, h0 = blockIdx.y * 16;
  const int r0 = ((int)blockIdx.x - tile_cu[seq]) * rt, rows_here = q_len[seq], start = seq_start[seq];
  const int64_t row_base = cu_rows[seq];
  const int my_row = r0 + c / hc, my_head = h0 + c % hc;             // the pair of the lane's column
  const bool live = c / hc < rt && my_row < rows_here && my_head < H;
  const int my_pos = start + my_row;
  const int last_pos = start + min(r0 + rt, rows_here) - 1;
  const int n_halves = last_pos / LATENT_KEYS + 1, per = (n_halves + splits - 1) / splits;
  const int begin = blockIdx.z * per, end = min(n_halves, begin + per);
  const int chunks = width / 8, pieces = LATENT_KEYS * chunks;
  vu4 next[NL];
  int page_ok = 0;
  auto fetch = [&](int half) {                                       // rows of a page lie end to end
    const int page = page_table[(int64_t)slot * max_pages + half / 2];
    page_ok = page >= 0;
    const vu4* src = (const vu4*)(pages + ((int64_t)(page < 0 ? 0 : page) * PAGE_TOKENS + half % 2 * LATENT_KEYS) * width);
#pragma unroll
    for (int u = 0; u < NL; ++u) next[u] = src[min(tid + 256 * u, pieces - 1)];
  };
  if (begin < end) fetch(begin);
  for (int e = tid; e < 16 * chunks; e += 256) {                     // the tile's queries, zeros for columns without a pair
    const int col = e / chunks, k = (e % chunks) * 8;
    const int row = r0 + col / hc, head = h0 + col % hc;
    vu4 v = {0, 0, 0, 0};
    if (col / hc < rt && row < rows_here && head < H) v = *(const vu4*)(q + ((row_base + row) * H + head) * width + k);
    *(vu4*)(q_s + col * ws + k) = v;
  }
  vf4 O[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) O[t] = vf4{0.f, 0.f, 0.f, 0.f};
  const int blocks = width / 32, k_from = wave < 2 ? 0 : blocks / 2, k_to = wave < 2 ? blocks / 2 : blocks;
  const bf16_t* k_row = page_s + (16 * (wave & 1) + c) * ws + 8 * g;
  const bf16_t* q_row = q_s + c * ws + 8 * g;
  float m = -INFINITY, l = 0.f;
  for (int half = begin; half < end; ++half) {
    __syncthreads();                                                 // the half page before has been read
#pragma unroll
    for (int u = 0; u < NL; ++u) {
      const int e = tid + 256 * u;
      if (e < pieces) *(vu4*)(page_s + (e / chunks) * ws + (e % chunks) * 8) = next[u];
    }
    const bool seen = page_ok != 0;
    __syncthreads();
    if (half + 1 < end) fetch(half + 1);
    vf4 part = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int k = k_from; k < k_to; ++k) part = MFMA16(*(const bf16x8*)(k_row + 32 * k), *(const bf16x8*)(q_row + 32 * k), part);
    s_part[wave * WAVE + lane] = part;
    __syncthreads();
    // positions 8g .. 8g + 7 of the half page: of 16-position tile g / 2, held by its lane groups 2 (g % 2) and the next
    float s[8], top = -INFINITY;
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int at = (g / 2) * WAVE + (2 * (g % 2) + i) * 16 + c;
      const vf4 lo = s_part[at], hi = s_part[2 * WAVE + at];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int pos = half * LATENT_KEYS + 8 * g + 4 * i + r;
        s[4 * i + r] = (live && seen && pos <= my_pos) ? (lo[r] + hi[r]) * scale : -INFINITY;
        top = fmaxf(top, s[4 * i + r]);
      }
    }
    top = fmaxf(top, __shfl_xor(top, 16, WAVE));
    top = fmaxf(top, __shfl_xor(top, 32, WAVE));
    const float m_new = fmaxf(m, top);
    const float base = m_new == -INFINITY ? 0.f : m_new;             // a column that has seen no key yet keeps weight 0
    const float alpha = expf(m - base);
    m = m_new;
    float sum = 0.f;
    u16x8 pb;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const bf16_t p = float_to_bf16(expf(s[e] - base));
      sum += bf16_to_float(p);
      pb[e] = p.bits;
    }
    l = l * alpha + sum;
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const int f = 16 * (wave + 4 * t) + c;                         // the lane's feature as a row of the first operand
      if (16 * (wave + 4 * t) < rank) {
#pragma unroll
        for (int r = 0; r < 4; ++r) O[t][r] *= alpha;
        u16x8 a;
#pragma unroll
        for (int e = 0; e < 8; ++e) a[e] = page_s[(8 * g + e) * ws + f].bits;
        O[t] = MFMA16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, pb), O[t]);
      }
    }
  }
  l += __shfl_xor(l, 16, WAVE);
  l += __shfl_xor(l, 32, WAVE);
  if (!live) return;
  const int64_t at = (((row_base + my_row) * H + my_head) * splits + blockIdx.z);
  if (wave == 0 && g == 0) { part_ml[2 * at] = m; part_ml[2 * at + 1] = l; }
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const int f = 16 * (wave + 4 * t) + 4 * g;
    if (rank % 4 == 0) {
      if (f < rank) *(vf4*)(part_o + at * rank + f) = O[t];
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (f + r < rank) part_o[at * rank + f + r] = O[t][r];
    }
  }
}

// The runs of a (row, head) joined in order; rows of sequences that sit out give zeros. Thread tid holds four features
// (V = 4) or one; groups of threads take every `groups`-th run and are added up in order through LDS.
#define LATENT_MAX_SPLITS 64

template <int V>
__global__ __launch_bounds__(256) void latent_combine_kernel(const float* __restrict__ part_o, const float* __restrict__ part_ml,
                                                             const int* __restrict__ row_slot, bf16_t* __restrict__ out,
                                                             int H, int rank, int splits) {
  __shared__ float weight[LATENT_MAX_SPLITS], sums[256 * V];
  const int64_t at = (int64_t)blockIdx.x * H + blockIdx.y;
  const int tid = threadIdx.x, per = rank / V;                       // threads that hold a run's features
  if (row_slot[blockIdx.x] < 0) {
    for (int f = tid; f < rank; f += 256) out[at * rank + f] = float_to_bf16(0.f);
    return;
  }
  if (tid < WAVE) {
    float m = -INFINITY, l = 0.f;
    if (tid < splits) { m = part_ml[2 * (at * splits + tid)]; l = part_ml[2 * (at * splits + tid) + 1]; }
    const float top = wave_max(m), w = expf(m - top);                // some run holds a key: top is finite
    const float total = wave_sum(l * w);
    weight[tid] = w / total;
  }
  __syncthreads();
  const int groups = per < 256 ? 256 / per : 1;
  for (int p0 = 0; p0 < per; p0 += 256) {
    const int group = groups > 1 ? tid / per : 0, p = groups > 1 ? tid % per : p0 + tid;
    float o[V];
#pragma unroll
    for (int j = 0; j < V; ++j) o[j] = 0.f;
    if (group < groups && p < per) {
      const float* src = part_o + at * splits * rank + (int64_t)p * V;
      for (int s0 = group; s0 < splits; s0 += 8 * groups) {
        float x[8][V];
#pragma unroll
        for (int u = 0; u < 8; ++u) {
          const int s = s0 + u * groups;
          if constexpr (V == 4) {
            const vf4 t = s < splits ? *(const vf4*)(src + (int64_t)s * rank) : vf4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int j = 0; j < 4; ++j) x[u][j] = t[j];
          } else {
            x[u][0] = s < splits ? src[(int64_t)s * rank] : 0.f;
          }
        }
#pragma unroll
        for (int u = 0; u < 8; ++u) {
          const float w = s0 + u * groups < splits ? weight[s0 + u * groups] : 0.f;
#pragma unroll
          for (int j = 0; j < V; ++j) o[j] += w * x[u][j];
        }
      }
    }
    if (groups == 1) {
      if (p < per)
#pragma unroll
        for (int j = 0; j < V; ++j) out[at * rank + p * V + j] = float_to_bf16(o[j]);
      continue;
    }
    if (group < groups)
#pragma unroll
      for (int j = 0; j < V; ++j) sums[(group * per + p) * V + j] = o[j];
    __syncthreads();
    for (int f = tid; f < rank; f += 256) {
      float sum = 0.f;
      for (int q = 0; q < groups; ++q) sum += sums[q * rank + f];
      out[at * rank + f] = float_to_bf16(sum);
    }
  }
}

DRYFT_API int dryft_latent_split(const void* q, const void* pages, const int* page_table, int max_pages,
                                 const int* seq_slot, const int* cu_rows, const int* q_len, const int* seq_start,
                                 const int* tile_cu, int n_seqs, int max_tiles, const int* row_slot, int n_rows, int H,
                                 int width, int rank, float scale, float* part_o, float* part_ml, int splits, void* out,
                                 hipStream_t stream) {
  if (n_rows <= 0) return 0;
  if (H <= 0 || width % 32 || width > MLA_MAX_WIDTH || rank <= 0 || rank > width || splits <= 0 ||
      splits > LATENT_MAX_SPLITS)
    return -1;
  const size_t lds = (size_t)(LATENT_KEYS + 16) * (width + 8) * sizeof(bf16_t) + 256 * sizeof(vf4);
  if (max_tiles > 0) {
    const dim3 grid(max_tiles, (H + 15) / 16, splits);
#define LS(NN, LL)                                                                                                   \
  {                                                                                                                  \
    if (lds > 64 * 1024 && hipFuncSetAttribute((const void*)latent_split_kernel<NN, LL>,                             \
                                               hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess)  \
      return -2;                                                                                                     \
    hipLaunchKernelGGL((latent_split_kernel<NN, LL>), grid, dim3(256), lds, stream, (const bf16_t*)q,                \
                       (const bf16_t*)pages, page_table, max_pages, seq_slot, cu_rows, q_len, seq_start, tile_cu,    \
                       n_seqs, H, width, rank, scale, part_o, part_ml, splits);                                      \
  }
#define LSW(NN) if (width <= 256) LS(NN, 4) else if (width <= 576) LS(NN, 9) else LS(NN, 15)
    if (rank <= 64) { LSW(1) }
    else if (rank <= 128) { LSW(2) }
    else if (rank <= 256) { LSW(4) }
    else if (rank <= 512) { LSW(8) }
    else { LS(15, 15) }
#undef LSW
#undef LS
    const int rc = DRYFT_LAUNCH_CHECK();
    if (rc) return rc;
  }
  if (rank % 4 == 0)
    hipLaunchKernelGGL(latent_combine_kernel<4>, dim3(n_rows, H), dim3(256), 0, stream, part_o, part_ml, row_slot,
                       (bf16_t*)out, H, rank, splits);
  else
    hipLaunchKernelGGL(latent_combine_kernel<1>, dim3(n_rows, H), dim3(256), 0, stream, part_o, part_ml, row_slot,
                       (bf16_t*)out, H, rank, splits);
  return DRYFT_LAUNCH_CHECK();
}

// ---------------------------------------------------------------------------------------------------
// Float32: one workgroup per (row, head), plain arithmetic; 256 keys at a time, a thread a key, then a thread a feature.
__global__ __launch_bounds__(256) void latent_attend_f32_kernel(const float* __restrict__ q, const float* __restrict__ pages,
                                                                const int* __restrict__ page_table, int max_pages,
                                                                const int* __restrict__ row_slot,
                                                                const int* __restrict__ row_pos, float* __restrict__ out,
                                                                int H, int width, int rank, float scale) {
  __shared__ __attribute__((aligned(16))) float qs[MLA_MAX_WIDTH];
  __shared__ float ps[256];
  __shared__ int held_pages[4];
  __shared__ float scratch[16];
  const int64_t row = blockIdx.x, at = row * H + blockIdx.y;
  const int tid = threadIdx.x, slot = row_slot[row], pos = row_pos[row];
  if (slot < 0) {
    for (int f = tid; f < rank; f += 256) out[at * rank + f] = 0.f;
    return;
  }
  for (int i = tid; i < width; i += 256) qs[i] = q[at * width + i];
  float m = -INFINITY, l = 0.f, acc[4] = {0.f, 0.f, 0.f, 0.f};
  for (int c0 = 0; c0 <= pos; c0 += 256) {
    __syncthreads();
    if (tid < 4) held_pages[tid] = c0 + 64 * tid <= pos ? page_of(page_table, max_pages, slot, c0 + 64 * tid) : -1;
    __syncthreads();
    const int j = c0 + tid, page = held_pages[tid / 64];
    const bool seen = j <= pos && page >= 0;
    float s = -INFINITY;
    if (seen) {
      const float* k = pages + ((int64_t)page * PAGE_TOKENS + tid % 64) * width;
      float d = 0.f;
      for (int i = 0; i < width; i += 4) {
        const vf4 k4 = *(const vf4*)(k + i), q4 = *(const vf4*)(qs + i);
#pragma unroll
        for (int u = 0; u < 4; ++u) d += k4[u] * q4[u];
      }
      s = d * scale;
    }
    const float m_new = fmaxf(m, block_max(s, scratch)), alpha = expf(m - m_new);      // every run holds a key the row sees
    const float p = seen ? expf(s - m_new) : 0.f;
    l = l * alpha + block_sum(p, scratch);
    ps[tid] = p;
    __syncthreads();
    const int n = min(256, pos - c0 + 1);
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int f = tid + 256 * u;
      if (f >= rank) continue;
      float a = acc[u] * alpha;
      for (int jj = 0; jj < n; ++jj) {
        const int pg = held_pages[jj / 64];
        if (pg >= 0) a += ps[jj] * pages[((int64_t)pg * PAGE_TOKENS + jj % 64) * width + f];
      }
      acc[u] = a;
    }
    m = m_new;
  }
#pragma unroll
  for (int u = 0; u < 4; ++u)
    if (tid + 256 * u < rank) out[at * rank + tid + 256 * u] = acc[u] / l;
}

DRYFT_API int dryft_latent_attend_f32(const void* q, const void* pages, const int* page_table, int max_pages,
                                      const int* row_slot, const int* row_pos, void* out, int n_rows, int H, int width,
                                      int rank, float scale, hipStream_t stream) {
  if (n_rows <= 0) return 0;
  if (H <= 0 || width % 32 || width > MLA_MAX_WIDTH || rank <= 0 || rank > width) return -1;
  hipLaunchKernelGGL(latent_attend_f32_kernel, dim3(n_rows, H), dim3(256), 0, stream, (const float*)q, (const float*)pages,
                     page_table, max_pages, row_slot, row_pos, (float*)out, H, width, rank, scale);
  return DRYFT_LAUNCH_CHECK();
}
