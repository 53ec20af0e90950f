// Linear attention with a matrix state per head: a decay per key channel and token, or a fixed one per head.
//
//   S_t = diag(alpha_t) S_(t-1) + k_t v_t^T,    o_t = S_t^T q_t        (S is D x Dv per head)
//
// q, k and v arrive in the activation dtype as runs of columns of one projection; q and k may be turned by a rotation
// over halves on their way in (float32 tables) and are multiplied by a number each. Everything from there on is float
// arithmetic in both precisions: the rotated q and k, the decays, the state (float32 in the state store), the sums.
// The decays come as natural logarithms, ld[row, head, channel] or ld_head[head].
//
// Two kernels. `linattn_token` serves steps of one row a sequence: the state passes through the registers of one
// workgroup per (sequence, head), which also norms and gates the read-out. `linattn_chunk` serves everything else,
// sixteen tokens at a time on the matrix cores in full 32-bit precision (v_mfma_f32_16x16x4_f32). With b_t the sum of
// the logarithms of a chunk's first t decays (per channel) and S the state before the chunk,
//
//   o_t  = (q_t e^(b_t))^T S + sum_(s <= t) a_st v_s,   a_st = sum_i k_si e^(-b_si) q_ti e^(b_ti)
//   S'   = diag(e^(b_16)) S + sum_s (k_s e^(b_16 - b_s)) v_s^T
//
// where only e^(-b_s) can grow. A chunk in which some channel's b_16 lies below LIN_STRONG forms its a_st pair by pair
// with e^(b_t - b_s) instead (at most 1), so that no decay, however strong, leaves the range of a float.
#include "common.h"

#define LIN_CHUNK 16
#define LIN_MAX_DIM 256
#define LIN_STRONG (-86.f)               // in powers of two, as all logarithms inside the chunk kernel
#define LIN_LOG2E 1.4426950408889634f

// Feature i of a head turned by the row's position: feature i of the first `rot` with feature i + rot/2.
template <typename T>
__device__ __forceinline__ float turned(const T* head, int i, int rot, const float* __restrict__ cos_t,
                                        const float* __restrict__ sin_t, int64_t pos) {
  const float x = load_as_float(head + i);
  if (i >= rot) return x;
  const int half = rot / 2, f = i < half ? i : i - half;
  const float other = load_as_float(head + (i < half ? i + half : i - half));
  const float c = cos_t[pos * half + f], s = sin_t[pos * half + f];
  return i < half ? x * c - other * s : x * c + other * s;
}

// ---------------------------------------------------------------------------------------------------
// Token by token. A workgroup takes one (sequence, head). A thread keeps V neighbouring columns of the state rows
// rg, rg + RG, ... (NR of them at most); RG row groups of C column groups. Per token the partial read-outs are added
// up over the row groups through LDS, then
//
//   out = o / sqrt(mean(o^2) + eps) * weight * silu(gate)          (weight optional, one for all heads)
template <typename T, int V, int NR>
__global__ __launch_bounds__(1024) void linattn_token_kernel(
    const T* __restrict__ proj, int64_t stride, int q_col, int k_col, int v_col, int g_col, float q_scale, float k_scale,
    const float* __restrict__ cos_t, const float* __restrict__ sin_t, int rot, const int* __restrict__ row_pos,
    const float* __restrict__ ld, const float* __restrict__ head_decay, const int* __restrict__ seq_slot,
    const int* __restrict__ cu_rows, const int* __restrict__ q_len, float* __restrict__ state,
    const float* __restrict__ weight, float eps, T* __restrict__ out, int H, int D, int Dv, int write_state, int C, int RG) {
  __shared__ float sq[LIN_MAX_DIM], sk[LIN_MAX_DIM], sa[LIN_MAX_DIM];
  __shared__ __attribute__((aligned(16))) float sv[LIN_MAX_DIM], red[4096];
  __shared__ float scratch[16];
  const int seq = blockIdx.x, head = blockIdx.y, tid = threadIdx.x;
  const int slot = seq_slot[seq], n = q_len[seq];
  const int64_t first = cu_rows[seq];
  if (slot < 0) {                      // a sequence that sits out: its rows of the output hold zeros
    for (int e = tid; e < n * Dv; e += blockDim.x) store_from_float(out + ((first + e / Dv) * H + head) * Dv + e % Dv, 0.f);
    return;
  }
  const int rg = tid / C, c = tid % C;
  const bool mine = rg < RG;
  float* at = state + (((int64_t)slot * H + head) * D + rg) * Dv + c * V;
  float S[NR][V];
#pragma unroll
  for (int j = 0; j < NR; ++j) {
    const bool in = mine && rg + j * RG < D;
    if constexpr (V == 4) {
      const vf4 x = in ? *(const vf4*)(at + (int64_t)j * RG * Dv) : vf4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int u = 0; u < 4; ++u) S[j][u] = x[u];
    } else {
      S[j][0] = in ? at[(int64_t)j * RG * Dv] : 0.f;
    }
  }
  for (int t = 0; t < n; ++t) {
    const int64_t row = first + t;
    const T* p = proj + row * stride;
    __syncthreads();                   // the token before has been read
    for (int i = tid; i < D; i += blockDim.x) {
      const int64_t pos = rot ? row_pos[row] : 0;
      sq[i] = turned(p + q_col + head * D, i, rot, cos_t, sin_t, pos) * q_scale;
      sk[i] = turned(p + k_col + head * D, i, rot, cos_t, sin_t, pos) * k_scale;
      sa[i] = ld != nullptr ? expf(ld[(row * H + head) * D + i]) : head_decay[head];
    }
    for (int i = tid; i < Dv; i += blockDim.x) sv[i] = load_as_float(p + v_col + head * Dv + i);
    __syncthreads();
    if (mine) {
      float acc[V], v[V];
#pragma unroll
      for (int u = 0; u < V; ++u) { acc[u] = 0.f; v[u] = sv[c * V + u]; }
#pragma unroll
      for (int j = 0; j < NR; ++j) {
        const int r = rg + j * RG;
        if (r < D) {
          const float a = sa[r], k = sk[r], q = sq[r];
#pragma unroll
          for (int u = 0; u < V; ++u) {
            S[j][u] = a * S[j][u] + k * v[u];
            acc[u] += q * S[j][u];
          }
        }
      }
#pragma unroll
      for (int u = 0; u < V; ++u) red[rg * Dv + c * V + u] = acc[u];
    }
    __syncthreads();
    float o = 0.f;
    if (tid < Dv)
      for (int r = 0; r < RG; ++r) o += red[r * Dv + tid];
    const float inv = 1.f / sqrtf(block_sum(o * o, scratch) / (float)Dv + eps);
    if (tid < Dv) {
      const float g = load_as_float(p + g_col + head * Dv + tid);
      store_from_float(out + (row * H + head) * Dv + tid,
                       o * inv * (weight != nullptr ? weight[tid] : 1.f) * (g / (1.f + expf(-g))));
    }
  }
  if (!write_state || !mine) return;
#pragma unroll
  for (int j = 0; j < NR; ++j) {
    if (rg + j * RG < D) {
      if constexpr (V == 4) *(vf4*)(at + (int64_t)j * RG * Dv) = vf4{S[j][0], S[j][1], S[j][2], S[j][3]};
      else at[(int64_t)j * RG * Dv] = S[j][0];
    }
  }
}

// ---------------------------------------------------------------------------------------------------
// Sixteen tokens at a time. A workgroup of four waves takes 64 value columns of one (sequence or segment, head), a wave
// 16 of them. A wave keeps its columns of the state as accumulator tiles of 16 channels (lane (g, c) = (lane / 16,
// lane % 16) holds channels 4g .. 4g + 3 of column c), which serve as they are as the second operand of the read-out's
// product: the four steps of a tile's contraction take channels 4g + j, j = 0 .. 3, so that lane group g always
// contributes the channels it holds, and the first operand's four values of a lane are one 16-byte read. The scores
// of the chunk's pairs come out of their product the same way round that the second product takes them. A chunk's
// operands are formed by all threads (a thread has one channel and TT tokens) into one of two LDS buffers, while the next
// chunk's loads are in flight; one barrier a chunk.
//
// Long prompts are cut into segments of `seg_rows` rows that run side by side (MODE 1, then the carry kernel, then
// MODE 2; MODE 0 walks a whole sequence): the recurrence is linear in the state, so a segment's effect is S_out =
// diag(P) S_in + L with P the product of its decays and L the state it reaches from zero. MODE 1 computes L and P of
// every segment but a sequence's last; MODE 2 starts every segment from the state that enters it and writes its
// read-outs, and a sequence's last segment writes the state back. Segment x of the step belongs to the sequence s with
// seg_cu[s] <= x < seg_cu[s + 1] (a sequence that sits out has none).
#define LIN_KT (LIN_CHUNK + 4)           // floats a channel of k~ takes in LDS

template <int DP> constexpr int lin_buffer_floats() { return 2 * LIN_CHUNK * (DP + 4) + DP * LIN_KT + DP; }

template <typename T, int DP, int MODE, bool ROT, bool CHAN>
__global__ __launch_bounds__(256) void linattn_chunk_kernel(
    const T* __restrict__ proj, int64_t stride, int q_col, int k_col, int v_col, float q_scale, float k_scale,
    const float* __restrict__ cos_t, const float* __restrict__ sin_t, int rot, const int* __restrict__ row_pos,
    const float* __restrict__ ld, const float* __restrict__ ld_head, const int* __restrict__ seq_slot,
    const int* __restrict__ cu_rows, const int* __restrict__ q_len, float* __restrict__ state, float* __restrict__ o_raw,
    int H, int D, int Dv, int write_state, const int* __restrict__ seg_cu, int n_seqs, int seg_rows,
    float* __restrict__ seg_state, float* __restrict__ seg_decay) {
  constexpr int TPC = 256 / DP, TT = LIN_CHUNK / TPC, TILES = DP / 16, LD = DP + 4;
  extern __shared__ __attribute__((aligned(16))) float lds[];      // two buffers of q~ | k^ | k~ transposed | e^(b_16)
  __shared__ int strong[3];
  int seq = blockIdx.x, seg = 0, n_segs = 1;
  if (MODE != 0) {
    if ((int)blockIdx.x >= seg_cu[n_seqs]) return;
    seq = 0;
    while (seg_cu[seq + 1] <= (int)blockIdx.x) ++seq;
    seg = blockIdx.x - seg_cu[seq];
    n_segs = seg_cu[seq + 1] - seg_cu[seq];
    if (MODE == 1 && seg == n_segs - 1) return;                     // nobody needs the last segment's summary
  }
  const int head = blockIdx.y, tid = threadIdx.x, wave = tid / WAVE, lane = tid % WAVE, g = lane / 16, c = lane % 16;
  const int col = blockIdx.z * 64 + 16 * wave + c;                  // the lane's value column
  const bool busy = (int)blockIdx.z * 64 + 16 * wave < Dv;          // the wave has columns of its own
  const int slot = seq_slot[seq];
  const int64_t first = cu_rows[seq] + (MODE == 0 ? 0 : seg * seg_rows);
  const int n = MODE == 0 ? q_len[seq] : min(seg_rows, q_len[seq] - seg * seg_rows);
  if (slot < 0) {                       // a sequence that sits out: its rows of the read-out hold zeros
    for (int e = tid; e < n * 64; e += 256)
      if ((int)blockIdx.z * 64 + e % 64 < Dv)
        o_raw[((first + e / 64) * H + head) * Dv + blockIdx.z * 64 + e % 64] = 0.f;
    return;
  }
  if (n <= 0) return;
  float* s_mine = state + ((int64_t)slot * H + head) * D * Dv;
  float* s_seg = MODE == 0 ? nullptr : seg_state + ((int64_t)blockIdx.x * H + head) * D * Dv;
  const float* s_from = MODE == 2 ? s_seg : s_mine;
  vf4 S[TILES];
#pragma unroll
  for (int m = 0; m < TILES; ++m)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 16 * m + 4 * g + r;
      S[m][r] = (MODE != 1 && i < D && col < Dv) ? s_from[(int64_t)i * Dv + col] : 0.f;
    }
  const int ch = tid % DP, part = tid / DP;                         // the thread's channel, its run of TT tokens
  const float hl = CHAN ? 0.f : ld_head[head] * LIN_LOG2E;
  const int half = rot / 2, twin = ch < half ? ch + half : ch - half, freq = ch < half ? ch : ch - half;
  const bool turns = ROT && ch < rot;
  const float sign = ch < half ? -1.f : 1.f;
  // What a chunk brings stays as it was loaded until it is used (a conversion here would wait for the loads), and every
  // load goes to a place that exists: a token beyond the last reads the last, a channel beyond D the last.
  const int chc = min(ch, D - 1), twc = turns ? twin : chc, frc = turns ? freq : 0, vcc = min(col, Dv - 1);
  const int step = (int)stride, wide = H * D;
  const T* base = proj + first * stride;
  const int64_t pos0 = ROT ? row_pos[first] : 0;                    // a sequence's rows stand at consecutive positions
  T fq[TT], fk[TT], fq2[TT], fk2[TT], fv[4];
  float fc[TT], fs[TT], fl[LIN_CHUNK];
  auto fetch = [&](int t0) {
    const int last = n - 1 - t0;
    const T* qc = base + (int64_t)t0 * stride + q_col + head * D;
    const T* kc = base + (int64_t)t0 * stride + k_col + head * D;
    const T* vc = base + (int64_t)t0 * stride + v_col + head * Dv;
    const float* cc = cos_t + (pos0 + t0) * half;
    const float* sc = sin_t + (pos0 + t0) * half;
#pragma unroll
    for (int u = 0; u < TT; ++u) {
      const int t = min(part * TT + u, last);
      if (MODE != 1) fq[u] = qc[t * step + chc];
      fk[u] = kc[t * step + chc];
      if (ROT) {
        if (MODE != 1) fq2[u] = qc[t * step + twc];
        fk2[u] = kc[t * step + twc];
        fc[u] = cc[t * half + frc];
        fs[u] = sc[t * half + frc];
      }
    }
    if (CHAN) {
      const float* lc = ld + (first + t0) * wide + head * D;
#pragma unroll
      for (int t = 0; t < LIN_CHUNK; ++t) fl[t] = lc[min(t, last) * wide + chc];
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) fv[j] = vc[min(4 * g + j, last) * step + vcc];
  };
  float total = 0.f;
  fetch(0);
  if (tid < 3) strong[tid] = 0;
  __syncthreads();
  for (int t0 = 0, turn = 0, flag = 0; t0 < n; t0 += LIN_CHUNK, turn ^= 1, flag = flag == 2 ? 0 : flag + 1) {
    float* Qt = lds + turn * lin_buffer_floats<DP>();               // [16][LD]
    float* Kh = Qt + LIN_CHUNK * LD;                                // [16][LD]
    float* Kt = Kh + LIN_CHUNK * LD;                                // [DP][LIN_KT]
    float* eb = Kt + DP * LIN_KT;                                   // [DP]
    const int left = n - t0;                                        // tokens of the sequence from here on
    {
      float own[TT], run = 0.f;
#pragma unroll
      for (int t = 0; t < LIN_CHUNK; ++t) {
        if (t < left) run += CHAN ? fl[t] * LIN_LOG2E : hl;
        if (t / TT == part) own[t % TT] = run;
      }
      const float grow = __builtin_amdgcn_exp2f(-run);              // k^ = k~ e^(-b_16)
      float kt[TT];
#pragma unroll
      for (int u = 0; u < TT; ++u) {
        const int t = part * TT + u;
        const bool in = t < left && ch < D;
        float k = load_as_float(&fk[u]);
        if (ROT && turns) k = k * fc[u] + load_as_float(&fk2[u]) * (sign * fs[u]);
        kt[u] = in ? k * k_scale * __builtin_amdgcn_exp2f(run - own[u]) : 0.f;
        if (MODE != 1) {
          float q = load_as_float(&fq[u]);
          if (ROT && turns) q = q * fc[u] + load_as_float(&fq2[u]) * (sign * fs[u]);
          Qt[t * LD + ch] = in ? q * q_scale * __builtin_amdgcn_exp2f(own[u]) : 0.f;
          Kh[t * LD + ch] = kt[u] * grow;
        }
      }
      if constexpr (TT % 4 == 0) {
#pragma unroll
        for (int u = 0; u < TT; u += 4)
          *(vf4*)(Kt + ch * LIN_KT + part * TT + u) = vf4{kt[u], kt[u + 1], kt[u + 2], kt[u + 3]};
      } else {
#pragma unroll
        for (int u = 0; u < TT; ++u) Kt[ch * LIN_KT + part * TT + u] = kt[u];
      }
      if (part == 0) eb[ch] = __builtin_amdgcn_exp2f(run);
      if (MODE == 1) total += run;
      if (MODE != 1 && ch < D && run < LIN_STRONG) strong[flag] = 1;
    }
    vf4 v;
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = 4 * g + j < left && col < Dv ? load_as_float(&fv[j]) : 0.f;
    __syncthreads();
    if (tid == 0) strong[flag == 0 ? 2 : flag - 1] = 0;             // read by everyone before this barrier, set after the next
    if (t0 + LIN_CHUNK < n) fetch(t0 + LIN_CHUNK);
    if (!busy) continue;
    if (MODE != 1) {
      vf4 o = {0.f, 0.f, 0.f, 0.f}, a = {0.f, 0.f, 0.f, 0.f};       // a[r]: the score of token s = 4g + r for token t = c
      const bool pairwise = strong[flag] != 0;
#pragma unroll
      for (int m = 0; m < TILES; ++m) {
        const vf4 q4 = *(const vf4*)(Qt + c * LD + 16 * m + 4 * g);
        const vf4 k4 = *(const vf4*)(Kh + c * LD + 16 * m + 4 * g);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          o = __builtin_amdgcn_mfma_f32_16x16x4f32(q4[j], S[m][j], o, 0, 0, 0);
          a = __builtin_amdgcn_mfma_f32_16x16x4f32(k4[j], q4[j], a, 0, 0, 0);
        }
      }
      // The scores leave the matrix cores before the branch: the compiler does not keep the distance that a read of their
      // last register needs when the read comes right behind a taken branch.
      asm volatile("s_nop 15" : "+v"(a));
      if (pairwise) {
        a = vf4{0.f, 0.f, 0.f, 0.f};
        if (t0 + c < n) {
          const T* pq = proj + (first + t0 + c) * stride + head * D;
          const int64_t pos = ROT ? row_pos[first + t0] : 0;
          for (int i = 0; i < D; ++i) {
            float run = 0.f, bt = 0.f, bs[4] = {0.f, 0.f, 0.f, 0.f};
            for (int t = 0; t <= c; ++t) {
              run += CHAN ? ld[((first + t0 + t) * H + head) * D + i] * LIN_LOG2E : hl;
#pragma unroll
              for (int r = 0; r < 4; ++r)
                if (t == 4 * g + r) bs[r] = run;
            }
            bt = run;
            const float q = turned(pq + q_col, i, rot, cos_t, sin_t, pos + c) * q_scale;
#pragma unroll
            for (int r = 0; r < 4; ++r)
              if (4 * g + r <= c) {
                const T* pk = proj + (first + t0 + 4 * g + r) * stride + head * D;
                a[r] += q * turned(pk + k_col, i, rot, cos_t, sin_t, pos + 4 * g + r) * k_scale * __builtin_amdgcn_exp2f(bt - bs[r]);
              }
          }
        }
      }
#pragma unroll
      for (int j = 0; j < 4; ++j)
        o = __builtin_amdgcn_mfma_f32_16x16x4f32(4 * g + j <= c ? a[j] : 0.f, v[j], o, 0, 0, 0);
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (t0 + 4 * g + r < n && col < Dv) o_raw[((first + t0 + 4 * g + r) * H + head) * Dv + col] = o[r];
    }
#pragma unroll
    for (int m = 0; m < TILES; ++m) {
      const vf4 e4 = *(const vf4*)(eb + 16 * m + 4 * g);
      const vf4 k4 = *(const vf4*)(Kt + (16 * m + c) * LIN_KT + 4 * g);
#pragma unroll
      for (int r = 0; r < 4; ++r) S[m][r] *= e4[r];
#pragma unroll
      for (int j = 0; j < 4; ++j) S[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(k4[j], v[j], S[m], 0, 0, 0);
    }
  }
  if (MODE == 1 && blockIdx.z == 0 && part == 0 && ch < D)
    seg_decay[((int64_t)blockIdx.x * H + head) * D + ch] = __builtin_amdgcn_exp2f(total);
  if (MODE == 2 && seg != n_segs - 1) return;                       // the last segment leaves the sequence's state
  if (MODE != 1 && !write_state) return;
  float* s_to = MODE == 1 ? s_seg : s_mine;
#pragma unroll
  for (int m = 0; m < TILES; ++m)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 16 * m + 4 * g + r;
      if (i < D && col < Dv) s_to[(int64_t)i * Dv + col] = S[m][r];
    }
}

// The state that enters each segment of a sequence: S_in[0] is the sequence's own state, S_in[s + 1] = diag(P[s]) S_in[s]
// + L[s]. A thread an entry of the state; `seg_state` holds L when the kernel starts and S_in when it ends.
__global__ __launch_bounds__(256) void linattn_carry_kernel(const int* __restrict__ seq_slot, const int* __restrict__ seg_cu,
                                                            const float* __restrict__ state, float* __restrict__ seg_state,
                                                            const float* __restrict__ seg_decay, int H, int D, int Dv) {
  const int seq = blockIdx.x, head = blockIdx.y, e = blockIdx.z * 256 + threadIdx.x;
  const int x0 = seg_cu[seq], n_segs = seg_cu[seq + 1] - x0, slot = seq_slot[seq];
  const int entries = D * Dv;
  if (slot < 0 || e >= entries) return;
  float held = state[((int64_t)slot * H + head) * entries + e];
  const int i = e / Dv;
  float next = n_segs > 1 ? seg_state[((int64_t)x0 * H + head) * entries + e] : 0.f;
  for (int s = 0; s < n_segs; ++s) {
    float* at = seg_state + ((int64_t)(x0 + s) * H + head) * entries + e;
    const float local = next;
    if (s + 2 < n_segs) next = at[(int64_t)H * entries];             // the next segment's, on its way meanwhile
    *at = held;
    if (s + 1 < n_segs) held = seg_decay[((int64_t)(x0 + s) * H + head) * D + i] * held + local;
  }
}

DRYFT_API int dryft_linattn_max_dim() { return LIN_MAX_DIM; }

DRYFT_API int dryft_linattn_token(const void* proj, int64_t stride, int q_col, int k_col, int v_col, int g_col,
                                  float q_scale, float k_scale, const float* cos_t, const float* sin_t, int rot,
                                  const int* row_pos, const float* ld, const float* head_decay, const int* seq_slot,
                                  const int* cu_rows, const int* q_len, int n_seqs, float* state, const float* weight,
                                  float eps, void* out, int H, int D, int Dv, int write_state, int is_f32,
                                  hipStream_t stream) {
  if (n_seqs <= 0) return 0;
  if (H <= 0 || D <= 0 || Dv <= 0 || D > LIN_MAX_DIM || Dv > LIN_MAX_DIM || rot < 0 || rot % 2 || rot > D) return -1;
  if ((ld == nullptr) == (head_decay == nullptr)) return -1;
  const int V = Dv % 4 == 0 && ((uintptr_t)state & 15) == 0 ? 4 : 1;
  const int C = Dv / V;
  int RG = 1024 / C;
  if (RG > D) RG = D;
  if (RG * Dv > 4096) RG = 4096 / Dv;
  int threads = (RG * C + WAVE - 1) / WAVE * WAVE;
  if (threads < 256) threads = 256;
  const int rows = (D + RG - 1) / RG;
#define LT(TT, VV, NN)                                                                                               \
  hipLaunchKernelGGL((linattn_token_kernel<TT, VV, NN>), dim3(n_seqs, H), dim3(threads), 0, stream, (const TT*)proj, \
                     stride, q_col, k_col, v_col, g_col, q_scale, k_scale, cos_t, sin_t, rot, row_pos, ld, head_decay, \
                     seq_slot, cu_rows, q_len, state, weight, eps, (TT*)out, H, D, Dv, write_state, C, RG)
#define LTV(TT)                                                                                                      \
  if (V == 4) {                                                                                                      \
    if (rows <= 4) { LT(TT, 4, 4); }                                                                                 \
    else if (rows <= 8) { LT(TT, 4, 8); }                                                                            \
    else if (rows <= 16) { LT(TT, 4, 16); }                                                                          \
    else { return -1; }                                                                                              \
  } else {                                                                                                           \
    if (rows <= 8) { LT(TT, 1, 8); }                                                                                 \
    else if (rows <= 64) { LT(TT, 1, 64); }                                                                          \
    else { return -1; }                                                                                              \
  }
  if (is_f32) { LTV(float) } else { LTV(bf16_t) }
#undef LTV
#undef LT
  return DRYFT_LAUNCH_CHECK();
}

template <typename T, int DP, int MODE, bool ROT, bool CHAN>
static int launch_chunk(hipStream_t stream, const void* proj, int64_t stride, int q_col, int k_col, int v_col,
                        float q_scale, float k_scale, const float* cos_t, const float* sin_t, int rot, const int* row_pos,
                        const float* ld, const float* ld_head, const int* seq_slot, const int* cu_rows, const int* q_len,
                        int n_seqs, float* state, float* o_raw, int H, int D, int Dv, int write_state, const int* seg_cu,
                        int max_segs, int seg_rows, float* seg_state, float* seg_decay) {
  auto kernel = linattn_chunk_kernel<T, DP, MODE, ROT, CHAN>;
  const size_t bytes = 2 * sizeof(float) * lin_buffer_floats<DP>();
  if (bytes > 64 * 1024 &&
      hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes) != hipSuccess)
    return -2;
  hipLaunchKernelGGL(kernel, dim3(MODE == 0 ? n_seqs : max_segs, H, (Dv + 63) / 64), dim3(256), bytes, stream,
                     (const T*)proj, stride, q_col, k_col, v_col, q_scale, k_scale, cos_t, sin_t, rot, row_pos, ld, ld_head,
                     seq_slot, cu_rows, q_len, state, o_raw, H, D, Dv, write_state, seg_cu, n_seqs, seg_rows, seg_state,
                     seg_decay);
  return DRYFT_LAUNCH_CHECK();
}

DRYFT_API int dryft_linattn_chunk(const void* proj, int64_t stride, int q_col, int k_col, int v_col, float q_scale,
                                  float k_scale, const float* cos_t, const float* sin_t, int rot, const int* row_pos,
                                  const float* ld, const float* ld_head, const int* seq_slot, const int* cu_rows,
                                  const int* q_len, int n_seqs, float* state, float* o_raw, int H, int D, int Dv,
                                  int write_state, const int* seg_cu, int max_segs, int seg_rows, float* seg_state,
                                  float* seg_decay, int is_f32, hipStream_t stream) {
  if (n_seqs <= 0) return 0;
  if (H <= 0 || H > 65535 || D <= 0 || Dv <= 0 || D > LIN_MAX_DIM || Dv > LIN_MAX_DIM || rot < 0 || rot % 2 || rot > D)
    return -1;
  if ((ld == nullptr) == (ld_head == nullptr)) return -1;
  const bool cut = seg_cu != nullptr;
  if (cut && max_segs <= 0) return 0;
  if (cut && (seg_rows <= 0 || seg_state == nullptr || seg_decay == nullptr || !write_state)) return -1;
#define LC(TT, DD, M, R, CH)                                                                                         \
  launch_chunk<TT, DD, M, R, CH>(stream, proj, stride, q_col, k_col, v_col, q_scale, k_scale, cos_t, sin_t, rot, row_pos, \
                                 ld, ld_head, seq_slot, cu_rows, q_len, n_seqs, state, o_raw, H, D, Dv, write_state,    \
                                 seg_cu, max_segs, seg_rows, seg_state, seg_decay)
#define LC_FORM(TT, DD, M)                                                                                           \
  (rot ? (ld ? LC(TT, DD, M, true, true) : LC(TT, DD, M, true, false))                                               \
       : (ld ? LC(TT, DD, M, false, true) : LC(TT, DD, M, false, false)))
#define LC_SIZE(TT, M)                                                                                               \
  (D <= 16 ? LC_FORM(TT, 16, M) : D <= 32 ? LC_FORM(TT, 32, M) : D <= 64 ? LC_FORM(TT, 64, M)                        \
   : D <= 128 ? LC_FORM(TT, 128, M) : LC_FORM(TT, 256, M))
#define LC_RUN(M) (is_f32 ? LC_SIZE(float, M) : LC_SIZE(bf16_t, M))
  if (!cut) return LC_RUN(0);
  int rc = LC_RUN(1);
  if (rc) return rc;
  hipLaunchKernelGGL(linattn_carry_kernel, dim3(n_seqs, H, (D * Dv + 255) / 256), dim3(256), 0, stream, seq_slot, seg_cu,
                     state, seg_state, seg_decay, H, D, Dv);
  rc = DRYFT_LAUNCH_CHECK();
  if (rc) return rc;
  return LC_RUN(2);
#undef LC_RUN
#undef LC_SIZE
#undef LC_FORM
#undef LC
}
