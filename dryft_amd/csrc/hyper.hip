// Several copies of a float32 residual stream (hyper-connections): one launch mixes the copies, lets the last
// sublayer's output enter them, writes them back, and forms the weighted sum that the next sublayer reads,
// normed. Per row and column c, with n copies x_1..x_n and the output y of the sublayer before:
//
//   x'_t = sum_s mix[s][t] x_s + write[t] y          (all copies from the old ones; skipped when there is no y)
//   u    = sum_t read[t] x'_t                          (read == null: the plain sum)
//   h    = u / sqrt(mean_c(u^2) + eps) * weight        (or u itself, float32, when not normed)
//   h    = (u - mean_c(u)) / sqrt(mean_c((u - mean_c(u))^2) + eps) * weight + bias     (centred; the bias is optional)
//
// x is the copies [n, rows, width] in float32, or a single [rows, width] in the activation dtype that every
// copy equals (the embedding's output when the stream starts). y is a tensor in the activation dtype or float32
// partial sums over K of the product that made it, added up here in order. Statistics are float.
#include "common.h"

#define HYPER_MAX 8

template <typename T, int N>
__global__ __launch_bounds__(1024) void hyper_norm_kernel(const void* __restrict__ x_in, int x_is_copies,
                                                         const void* __restrict__ delta, int delta_kind, int n_partials,
                                                         int64_t partial_stride, const float* __restrict__ mix,
                                                         const float* __restrict__ write_w,
                                                         const float* __restrict__ read_w,
                                                         const float* __restrict__ weight,
                                                         const float* __restrict__ bias, float* __restrict__ x_out,
                                                         void* __restrict__ y_out, int normed, int centred, int rows,
                                                         int width, float eps) {
  extern __shared__ float u_row[];          // [width]
  __shared__ float scratch[16];
  const int64_t row = blockIdx.x;
  const int64_t plane = (int64_t)rows * width;
  float m[N][N], wr[N], rd[N];
#pragma unroll
  for (int s = 0; s < N; ++s) {
    wr[s] = delta_kind ? write_w[s] : 0.f;
    rd[s] = read_w ? read_w[s] : 1.f;
#pragma unroll
    for (int t = 0; t < N; ++t) m[s][t] = delta_kind ? mix[s * N + t] : (s == t ? 1.f : 0.f);
  }
  float ss = 0.f, su = 0.f;
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    const int64_t at = row * width + c;
    float x[N];
    if (x_is_copies) {
#pragma unroll
      for (int s = 0; s < N; ++s) x[s] = ((const float*)x_in)[s * plane + at];
    } else {
      const float v = load_as_float((const T*)x_in + at);
#pragma unroll
      for (int s = 0; s < N; ++s) x[s] = v;
    }
    float y = 0.f;
    if (delta_kind == 1) {
      y = load_as_float((const T*)delta + at);
    } else if (delta_kind == 2) {
      for (int p = 0; p < n_partials; ++p) y += ((const float*)delta)[p * partial_stride + at];
      y = rounded_as<T>(y);                 // what the product would have stored in the activation dtype
    }
    float u = 0.f;
    float nx[N];
#pragma unroll
    for (int t = 0; t < N; ++t) {
      float a = 0.f;
      if (delta_kind) {
#pragma unroll
        for (int s = 0; s < N; ++s) a += m[s][t] * x[s];
        a += wr[t] * y;
      } else {
        a = x[t];
      }
      nx[t] = a;
      u += rd[t] * a;
    }
    if (x_out) {
#pragma unroll
      for (int t = 0; t < N; ++t) x_out[t * plane + at] = nx[t];
    }
    u_row[c] = u;
    ss += u * u;
    su += u;
  }
  if (!y_out) return;
  if (!normed) {
    for (int c = threadIdx.x; c < width; c += blockDim.x) ((float*)y_out)[row * width + c] = u_row[c];
    return;
  }
  float mean = 0.f;
  if (centred) {                              // a thread reads back only the columns it wrote itself
    mean = block_sum(su, scratch) / (float)width;
    ss = 0.f;
    for (int c = threadIdx.x; c < width; c += blockDim.x) { const float d = u_row[c] - mean; ss += d * d; }
  }
  ss = block_sum(ss, scratch);
  const float r = 1.f / sqrtf(ss / (float)width + eps);
  for (int c = threadIdx.x; c < width; c += blockDim.x)
    store_from_float((T*)y_out + row * width + c, (u_row[c] - mean) * r * weight[c] + (bias ? bias[c] : 0.f));
}

// The same for widths that are a multiple of 4 and 16-byte aligned operands: a thread takes R runs of 4 neighbouring
// columns, moves them with 16-byte loads and stores (8 bytes in the 16-bit dtype), asks for four partial sums at a time,
// and keeps the weighted sum in registers between the passes.
template <typename T>
__device__ __forceinline__ vf4 load4_as_float(const T* p);
template <>
__device__ __forceinline__ vf4 load4_as_float<float>(const float* p) { return *(const vf4*)p; }
template <>
__device__ __forceinline__ vf4 load4_as_float<bf16_t>(const bf16_t* p) {
  const uint2 a = *(const uint2*)p;
  return vf4{__uint_as_float(a.x << 16), __uint_as_float(a.x & 0xffff0000u), __uint_as_float(a.y << 16),
             __uint_as_float(a.y & 0xffff0000u)};
}
__device__ __forceinline__ void store4_from_float(float* p, vf4 v) { *(vf4*)p = v; }
__device__ __forceinline__ void store4_from_float(bf16_t* p, vf4 v) {
  uint2 a;
  a.x = (uint32_t)float_to_bf16(v[0]).bits | ((uint32_t)float_to_bf16(v[1]).bits << 16);
  a.y = (uint32_t)float_to_bf16(v[2]).bits | ((uint32_t)float_to_bf16(v[3]).bits << 16);
  *(uint2*)p = a;
}

template <typename T, int N, int R>
__global__ __launch_bounds__(1024) void hyper_norm_vec_kernel(const void* __restrict__ x_in, int x_is_copies,
                                                             const void* __restrict__ delta, int delta_kind,
                                                             int n_partials, int64_t partial_stride,
                                                             const float* __restrict__ mix,
                                                             const float* __restrict__ write_w,
                                                             const float* __restrict__ read_w,
                                                             const float* __restrict__ weight,
                                                             const float* __restrict__ bias, float* __restrict__ x_out,
                                                             void* __restrict__ y_out, int normed, int centred, int rows,
                                                             int width, float eps) {
  __shared__ float scratch[16];
  const int64_t row = blockIdx.x;
  const int64_t plane = (int64_t)rows * width;
  const vf4 zero = {0.f, 0.f, 0.f, 0.f};
  vf4 u[R];
  float ss = 0.f, su = 0.f;
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int c = 4 * ((int)threadIdx.x + r * (int)blockDim.x);
    u[r] = zero;
    if (c >= width) continue;
    const int64_t at = row * width + c;
    vf4 x[N];
    if (x_is_copies) {
#pragma unroll
      for (int s = 0; s < N; ++s) x[s] = *(const vf4*)((const float*)x_in + s * plane + at);
    } else {
      const vf4 v = load4_as_float((const T*)x_in + at);
#pragma unroll
      for (int s = 0; s < N; ++s) x[s] = v;
    }
    vf4 y = zero;
    if (delta_kind == 1) {
      y = load4_as_float((const T*)delta + at);
    } else if (delta_kind == 2) {
      const float* part = (const float*)delta + at;
      int p = 0;
      for (; p + 4 <= n_partials; p += 4) {                   // four loads in flight; added in the order 0, 1, ...
        vf4 t[4];
#pragma unroll
        for (int q = 0; q < 4; ++q) t[q] = *(const vf4*)(part + (p + q) * partial_stride);
#pragma unroll
        for (int q = 0; q < 4; ++q) y += t[q];
      }
      for (; p < n_partials; ++p) y += *(const vf4*)(part + p * partial_stride);
#pragma unroll
      for (int j = 0; j < 4; ++j) y[j] = rounded_as<T>(y[j]);
    }
#pragma unroll
    for (int t = 0; t < N; ++t) {
      vf4 a = x[t];
      if (delta_kind) {
        a = zero;
#pragma unroll
        for (int s = 0; s < N; ++s) a += mix[s * N + t] * x[s];
        a += write_w[t] * y;
      }
      u[r] += (read_w ? read_w[t] : 1.f) * a;
      if (x_out) *(vf4*)(x_out + t * plane + at) = a;
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) { ss += u[r][j] * u[r][j]; su += u[r][j]; }
  }
  if (!y_out) return;
  if (!normed) {
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const int c = 4 * ((int)threadIdx.x + r * (int)blockDim.x);
      if (c < width) *(vf4*)((float*)y_out + row * width + c) = u[r];
    }
    return;
  }
  float mean = 0.f;
  if (centred) {
    mean = block_sum(su, scratch) / (float)width;
    ss = 0.f;
#pragma unroll
    for (int r = 0; r < R; ++r)
      if (4 * ((int)threadIdx.x + r * (int)blockDim.x) < width) {
#pragma unroll
        for (int j = 0; j < 4; ++j) ss += (u[r][j] - mean) * (u[r][j] - mean);
      }
  }
  ss = block_sum(ss, scratch);
  const float inv = 1.f / sqrtf(ss / (float)width + eps);
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int c = 4 * ((int)threadIdx.x + r * (int)blockDim.x);
    if (c >= width) continue;
    vf4 v = (u[r] - mean) * inv * *(const vf4*)(weight + c);
    if (bias) v += *(const vf4*)(bias + c);
    store4_from_float((T*)y_out + row * width + c, v);
  }
}

template <typename T, int R>
static int launch_hyper_vec(int n, int threads, hipStream_t stream, const void* x, int x_is_copies, const void* delta,
                            int delta_kind, int n_partials, int64_t partial_stride, const float* mix,
                            const float* write_w, const float* read_w, const float* weight, const float* bias,
                            float* x_out, void* y, int normed, int centred, int rows, int width, float eps) {
#define HYPER_VEC(N)                                                                                               \
  case N:                                                                                                          \
    hipLaunchKernelGGL((hyper_norm_vec_kernel<T, N, R>), dim3(rows), dim3(threads), 0, stream, x, x_is_copies, delta, \
                       delta_kind, n_partials, partial_stride, mix, write_w, read_w, weight, bias, x_out, y, normed,  \
                       centred, rows, width, eps);                                                                 \
    break;
  switch (n) {
    HYPER_VEC(1) HYPER_VEC(2) HYPER_VEC(3) HYPER_VEC(4) HYPER_VEC(5) HYPER_VEC(6) HYPER_VEC(7) HYPER_VEC(8)
    default: return -1;
  }
#undef HYPER_VEC
  return DRYFT_LAUNCH_CHECK();
}

template <typename T>
static int launch_hyper(int n, dim3 grid, dim3 block, size_t lds, hipStream_t stream, const void* x, int x_is_copies,
                        const void* delta, int delta_kind, int n_partials, int64_t partial_stride, const float* mix,
                        const float* write_w, const float* read_w, const float* weight, const float* bias, float* x_out,
                        void* y, int normed, int centred, int rows, int width, float eps) {
#define HYPER_CASE(N)                                                                                              \
  case N:                                                                                                          \
    hipLaunchKernelGGL((hyper_norm_kernel<T, N>), grid, block, lds, stream, x, x_is_copies, delta, delta_kind,     \
                       n_partials, partial_stride, mix, write_w, read_w, weight, bias, x_out, y, normed, centred, rows, \
                       width, eps);                                                                                \
    break;
  switch (n) {
    HYPER_CASE(1) HYPER_CASE(2) HYPER_CASE(3) HYPER_CASE(4) HYPER_CASE(5) HYPER_CASE(6) HYPER_CASE(7) HYPER_CASE(8)
    default: return -1;
  }
#undef HYPER_CASE
  return DRYFT_LAUNCH_CHECK();
}

DRYFT_API int dryft_hyper_max_streams() { return HYPER_MAX; }

DRYFT_API int dryft_hyper_norm(const void* x, int x_is_copies, int n, const void* delta, int delta_kind, int n_partials,
                               int64_t partial_stride, const float* mix, const float* write_w, const float* read_w,
                               const float* weight, const float* bias, float* x_out, void* y, int normed, int centred,
                               int rows, int width, float eps, int is_f32, hipStream_t stream) {
  if (rows <= 0) return 0;
  if (n < 1 || n > HYPER_MAX || width <= 0 || width > 16384) return -1;
  if (delta_kind && (mix == nullptr || write_w == nullptr)) return -1;
  if (y && normed && weight == nullptr) return -1;
  const uintptr_t all = (uintptr_t)x | (uintptr_t)delta | (uintptr_t)weight | (uintptr_t)bias | (uintptr_t)x_out | (uintptr_t)y;
  if (width % 4 == 0 && width <= 8192 && (all & 15) == 0 && partial_stride % 4 == 0) {
    const int quads = width / 4;
    // few rows: a run a thread, so that a row's loads are all in flight at once; many: fuller threads in fewer waves
    const int want = rows <= 128 || quads <= 256 ? quads : (quads + 1) / 2;
    const int threads = want <= 64 ? 64 : (want < 1024 ? (want + 63) / 64 * 64 : 1024);
#define HYPER_V(TT, RR)                                                                                            \
  return launch_hyper_vec<TT, RR>(n, threads, stream, x, x_is_copies, delta, delta_kind, n_partials, partial_stride, mix, \
                                  write_w, read_w, weight, bias, x_out, y, normed, centred, rows, width, eps)
    if (quads <= threads) {
      if (is_f32) HYPER_V(float, 1);
      HYPER_V(bf16_t, 1);
    }
    if (is_f32) HYPER_V(float, 2);                            // 1,024 threads take up to 8,192 columns in two runs
    HYPER_V(bf16_t, 2);
#undef HYPER_V
  }
  // few rows: more threads a row, so that a row's loads are all in flight at once
  dim3 grid(rows), block(rows <= 128 && width >= 1024 ? 1024 : 256);
  const size_t lds = (size_t)width * sizeof(float);
  if (is_f32)
    return launch_hyper<float>(n, grid, block, lds, stream, x, x_is_copies, delta, delta_kind, n_partials,
                               partial_stride, mix, write_w, read_w, weight, bias, x_out, y, normed, centred, rows, width,
                               eps);
  return launch_hyper<bf16_t>(n, grid, block, lds, stream, x, x_is_copies, delta, delta_kind, n_partials,
                              partial_stride, mix, write_w, read_w, weight, bias, x_out, y, normed, centred, rows, width,
                              eps);
}
