// Queries and keys that pass a short causal convolution on their way from the projection to the cache.  A token's row of
// the joined projection is [q: Hq * dim | k: Hkv * dim | g: Hq (where there is a gate)]; with u = row + bias for q and k,
//
//   y_t[d]  = sum_(lag = 0 .. taps - 1) w[taps - 1 - lag][d] u_(t - lag)[d]     each channel of q and k; u before a sequence is 0
//   value   = y of the key heads
//   q, k    = y / sqrt(mean(y^2) + eps) * weight                               over the whole projection of q, and of k
//   q, k    turned by position * inv_freq[pair] (adjacent pairs; a frequency of 0 leaves its pair alone)
//   gate    = sigmoid(g)                                                       one number a query head
//
// Keys and values go into the paged cache (layout: top of rope_kv.hip), queries to q_out [T][Hq][head_dim], gates to
// gate_out [T][Hq]; heads are padded with zeros from `dim` to `head_dim` elements.  The last taps - 1 values of u are a
// sequence's state (float32 [taps - 1][channels], oldest first, zero when the request is admitted).  The main kernel only
// reads it, and the state kernel replaces it afterwards, in the same stream; in a step of single tokens (a decode step) the token's
// block is the state's only reader and moves it itself.  Rows are of type TS, or float32 partial sums of a split K that are
// added in order.  float32 arithmetic; the sum over the taps runs from the oldest to the newest.
//
// A block takes up to CONVQK_TOKENS consecutive tokens: a thread keeps a channel's weights and its last inputs in registers
// while it goes down the tokens, and y stays in LDS for the norms and the rotation.
#include "common.h"

CWM_DEFINE_ERROR_API

#define CONVQK_THREADS 1024  // at most
#define CONVQK_MAX_TAPS 16
#define CONVQK_MAX_HEAD 256
#define CONVQK_TOKENS 4
#define CONVQK_MAX_LDS (60 * 1024)  // bytes of y

extern "C" int cwm_conv_qk_max_taps() { return CONVQK_MAX_TAPS; }
extern "C" int cwm_conv_qk_max_channels() { return CONVQK_MAX_LDS / 4; }

template <typename TS>
__device__ __forceinline__ float convqk_input(const TS* __restrict__ src, long stride, int n_partials, long partial_stride, long t, int d) {
  float v = 0.f;
  for (int p = 0; p < n_partials; ++p) v += Elem<TS>::load(src + (size_t)p * partial_stride + (size_t)t * stride + d);
  return v;
}

// W consecutive elements (1 or 4) of a float32 vector, and of a row of the projection
template <int W>
__device__ __forceinline__ void convqk_floats(const float* __restrict__ p, float (&v)[W]) {
  if constexpr (W == 4) {
    const float4 x = *(const float4*)p;
    v[0] = x.x, v[1] = x.y, v[2] = x.z, v[3] = x.w;
  } else {
    v[0] = *p;
  }
}
template <typename TS, int W>
__device__ __forceinline__ void convqk_row(const TS* __restrict__ src, long stride, int n_partials, long partial_stride, long t, int d, float (&v)[W]) {
  const TS* row = src + (size_t)t * stride + d;
  if constexpr (W == 1) {
    v[0] = convqk_input(src, stride, n_partials, partial_stride, t, d);
  } else if constexpr (sizeof(TS) == 2) {
    const uint2 x = *(const uint2*)row;  // partial sums are float32: one row here
    v[0] = __uint_as_float(x.x << 16), v[1] = __uint_as_float(x.x & 0xffff0000u);
    v[2] = __uint_as_float(x.y << 16), v[3] = __uint_as_float(x.y & 0xffff0000u);
  } else {
    v[0] = v[1] = v[2] = v[3] = 0.f;
    for (int p = 0; p < n_partials; p += 4) {
      // four partial sums in flight at a time; what lies past the last is the last again, times zero
      float4 z[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) z[u] = *(const float4*)(row + (size_t)min(p + u, n_partials - 1) * partial_stride);
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const float keep = p + u < n_partials ? 1.f : 0.f;
        v[0] = fmaf(keep, z[u].x, v[0]), v[1] = fmaf(keep, z[u].y, v[1]), v[2] = fmaf(keep, z[u].z, v[2]), v[3] = fmaf(keep, z[u].w, v[3]);
      }
    }
  }
}

// MAXT: room for that many taps in registers (taps <= MAXT); TB: tokens a block; W: channels a thread takes at a time (4:
// sizes are multiples of 4 and rows start at multiples of four elements)
template <typename TS, typename TO, int MAXT, int TB, int W>
__global__ void __launch_bounds__(CONVQK_THREADS)
conv_qk_kernel(const TS* __restrict__ src, long src_stride, int n_partials, long partial_stride, const float* __restrict__ bias,
               const float* __restrict__ taps_w, int taps, float* __restrict__ state, long state_ld, const int* __restrict__ slots,
               const int* __restrict__ cu_q, const int* __restrict__ seq_of_token, int n_slots, bool moves_state, TO* __restrict__ q_out,
               float* __restrict__ gate_out, const float* __restrict__ q_weight, const float* __restrict__ k_weight, float eps,
               const int* __restrict__ positions, const float* __restrict__ inv_freq, TO* __restrict__ cache,
               const int* __restrict__ block_table, int table_width, int page_size, int num_pages, int n_tokens, int n_q_heads,
               int n_kv_heads, int dim, int head_dim) {
  extern __shared__ __attribute__((aligned(16))) float y_all[];  // [TB][channels]
  __shared__ float cs[TB][CONVQK_MAX_HEAD];
  __shared__ float sums[2 * TB][CONVQK_THREADS / CWM_WAVE];
  const int t0 = blockIdx.x * TB;
  const int n = min(TB, n_tokens - t0);
  const int q_width = n_q_heads * dim, channels = q_width + n_kv_heads * dim;
  const int half = head_dim / 2;
  int seq_of[TB], start_of[TB], pos_of[TB], page_of[TB];
  float* state_of[TB];
#pragma unroll
  for (int k = 0; k < TB; ++k) {
    const int t = min(t0 + k, n_tokens - 1);
    seq_of[k] = seq_of_token[t];
    pos_of[k] = positions[t];
    start_of[k] = cu_q[seq_of[k]];
    const int slot = slots[seq_of[k]];
    state_of[k] = state && slot >= 0 && slot < n_slots ? state + (size_t)slot * state_ld : nullptr;
    const int lp = pos_of[k] / page_size;
    page_of[k] = lp < table_width ? block_table[(size_t)seq_of[k] * table_width + lp] : -1;
  }
  for (int i = threadIdx.x; i < n * half; i += blockDim.x) {
    const int k = i / half, pair = i - k * half;
    float c = 1.f, s = 0.f;
    const float f = inv_freq ? inv_freq[pair] : 0.f;
    if (f != 0.f) sincos_turn(positions[t0 + k], f, &s, &c);
    cs[k][2 * pair] = c;
    cs[k][2 * pair + 1] = s;
  }
  // ---- the convolutions, W channels a thread at a time ----------------------------------------------------------- //
  float sq[TB], sk[TB];
#pragma unroll
  for (int k = 0; k < TB; ++k) sq[k] = sk[k] = 0.f;
  for (int d = W * threadIdx.x; d < channels; d += W * blockDim.x) {
    float w[MAXT][W], u[MAXT][W], b[W];  // u[j] meets tap j; the newest input is u[taps - 1]
#pragma unroll
    for (int j = 0; j < MAXT; ++j) {
#pragma unroll
      for (int i = 0; i < W; ++i) w[j][i] = u[j][i] = 0.f;
      if (j < taps) convqk_floats<W>(taps_w + (size_t)j * channels + d, w[j]);
    }
#pragma unroll
    for (int i = 0; i < W; ++i) b[i] = 0.f;
    if (bias) convqk_floats<W>(bias + d, b);
#pragma unroll
    for (int k = 0; k < TB; ++k) {
      if (k >= n) continue;
      const int t = t0 + k;
      if (k == 0 || seq_of[k] != seq_of[k == 0 ? 0 : k - 1]) {
        // the block's first token of this sequence: the inputs before it come from the step's rows or from the state
#pragma unroll
        for (int j = 0; j < MAXT - 1; ++j) {
          if (j >= taps - 1) continue;
          const int s = t - (taps - 1) + j;
          if (s >= start_of[k]) {
            convqk_row<TS, W>(src, src_stride, n_partials, partial_stride, s, d, u[j]);
#pragma unroll
            for (int i = 0; i < W; ++i) u[j][i] += b[i];
          } else if (state_of[k]) {
            convqk_floats<W>(state_of[k] + (size_t)(taps - 1 + (s - start_of[k])) * channels + d, u[j]);
          } else {
#pragma unroll
            for (int i = 0; i < W; ++i) u[j][i] = 0.f;
          }
        }
      } else {
#pragma unroll
        for (int j = 0; j < MAXT - 1; ++j)
#pragma unroll
          for (int i = 0; i < W; ++i) u[j][i] = u[j + 1][i];
      }
      float own[W], acc[W];
      convqk_row<TS, W>(src, src_stride, n_partials, partial_stride, t, d, own);
#pragma unroll
      for (int i = 0; i < W; ++i) acc[i] = 0.f;
#pragma unroll
      for (int j = 0; j < MAXT; ++j)
#pragma unroll
        for (int i = 0; i < W; ++i) {
          if (j == taps - 1) u[j][i] = own[i] + b[i];
          if (j < taps) acc[i] = fmaf(w[j][i], u[j][i], acc[i]);
        }
      if (moves_state && state_of[k]) {
#pragma unroll
        for (int j = 1; j < MAXT; ++j)
          if (j < taps)
#pragma unroll
            for (int i = 0; i < W; ++i) state_of[k][(size_t)(j - 1) * channels + d + i] = u[j][i];
      }
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < W; ++i) {
        y_all[(size_t)k * channels + d + i] = acc[i];
        ss += acc[i] * acc[i];
      }
      if (d < q_width)
        sq[k] += ss;
      else
        sk[k] += ss;
    }
  }
  // ---- the root mean squares of a token's queries and keys ------------------------------------------------------ //
  const int lane = threadIdx.x & (CWM_WAVE - 1), wave = threadIdx.x / CWM_WAVE, waves = blockDim.x / CWM_WAVE;
#pragma unroll
  for (int k = 0; k < TB; ++k) {
    const float a = wave_sum(sq[k]), c = wave_sum(sk[k]);
    if (lane == 0) {
      sums[2 * k][wave] = a;
      sums[2 * k + 1][wave] = c;
    }
  }
  __syncthreads();
#pragma unroll
  for (int k = 0; k < TB; ++k) {
    if (k >= n) continue;
    float tq = 0.f, tk = 0.f;
    for (int w2 = 0; w2 < waves; ++w2) {
      tq += sums[2 * k][w2];
      tk += sums[2 * k + 1][w2];
    }
    const float q_rstd = 1.0f / sqrtf(tq / (float)q_width + eps), k_rstd = 1.0f / sqrtf(tk / (float)(channels - q_width) + eps);
    const int t = t0 + k;
    const float* y = y_all + (size_t)k * channels;
    const int slot = pos_of[k] % page_size;
    TO* kdst = nullptr;
    TO* vdst = nullptr;
    if (page_of[k] >= 0 && page_of[k] < num_pages) {
      const size_t plane = (size_t)n_kv_heads * page_size * head_dim;
      kdst = cache + (size_t)page_of[k] * 2 * plane;
      vdst = kdst + plane;
    }
    const int v_block = (page_size % 8 == 0) ? 8 : page_size;
    // a head's pairs; of a key head also its values, which are y as it is
    for (int e = threadIdx.x; e < (n_q_heads + n_kv_heads) * half; e += blockDim.x) {
      const int hh = e / half, i = e - hh * half;
      const bool is_key = hh >= n_q_heads;
      const int head = is_key ? hh - n_q_heads : hh;
      const float yr = 2 * i < dim ? y[hh * dim + 2 * i] : 0.f, yi = 2 * i + 1 < dim ? y[hh * dim + 2 * i + 1] : 0.f;
      const float* weight = is_key ? k_weight : q_weight;
      float re = yr, im = yi;
      if (weight) {
        const float rstd = is_key ? k_rstd : q_rstd;
        re *= rstd * (2 * i < dim ? weight[head * dim + 2 * i] : 0.f);
        im *= rstd * (2 * i + 1 < dim ? weight[head * dim + 2 * i + 1] : 0.f);
      }
      const float c = cs[k][2 * i], s = cs[k][2 * i + 1];
      TO* dst = nullptr;
      if (!is_key)
        dst = q_out + ((size_t)t * n_q_heads + head) * head_dim;
      else if (kdst)
        dst = kdst + ((size_t)head * page_size + slot) * head_dim;
      if (dst) {
        if constexpr (sizeof(TO) == 2) {
          *(uint32_t*)(dst + 2 * i) = pack2_bf16(re * c - im * s, im * c + re * s);
        } else {
          Elem<TO>::store(dst + 2 * i, re * c - im * s);
          Elem<TO>::store(dst + 2 * i + 1, im * c + re * s);
        }
      }
      if (is_key && vdst) {
        TO* v = vdst + (size_t)head * head_dim * page_size + ((size_t)(slot / v_block) * head_dim + 2 * i) * v_block + slot % v_block;
        Elem<TO>::store(v, yr);
        Elem<TO>::store(v + v_block, yi);
      }
    }
    if (gate_out)
      for (int h = threadIdx.x; h < n_q_heads; h += blockDim.x)
        gate_out[(size_t)t * n_q_heads + h] = 1.0f / (1.0f + expf(-convqk_input(src, src_stride, n_partials, partial_stride, t, channels + h)));
  }
}

// A sequence's new state: row r is the portion's input n - (taps - 1) + r, or, before the portion, row r + n of the old
// state (rows are written in rising order, each after the higher row it may come from has been read).
template <typename TS>
__global__ void __launch_bounds__(256)
conv_qk_state_kernel(const TS* __restrict__ src, long src_stride, int n_partials, long partial_stride, const float* __restrict__ bias,
                     float* __restrict__ state, long state_ld, const int* __restrict__ slots, const int* __restrict__ cu_q, int n_slots,
                     int channels, int taps) {
  const int b = blockIdx.x;
  const int d = blockIdx.y * 256 + threadIdx.x;
  if (d >= channels) return;
  const int slot = slots[b];
  if (slot < 0 || slot >= n_slots) return;
  float* srow = state + (size_t)slot * state_ld;
  const int start = cu_q[b], n = cu_q[b + 1] - start;
  for (int r = 0; r < taps - 1; ++r) {
    const int rel = n - (taps - 1) + r;
    float v;
    if (rel >= 0)
      v = convqk_input(src, src_stride, n_partials, partial_stride, start + rel, d) + (bias ? bias[d] : 0.f);
    else
      v = srow[(size_t)(r + n) * channels + d];
    srow[(size_t)r * channels + d] = v;
  }
}

// src: [n_tokens][src_stride] of src_dtype or n_partials float32 slabs.  bias: float32 [channels] or null.  taps_w: float32
// [taps][channels], a row a tap, the last row the current token's.  state: float32 [n_slots][state_ld], null where taps ==
// 1.  write_state 1: replaced by a second launch; 2: every portion of the step is one token long, and the first launch
// moves the state itself.  q_weight [Hq * dim], k_weight [Hkv * dim]: float32 or null (no norm).  gate_out: float32
// [n_tokens][Hq] or null (the rows then hold no gate).
extern "C" int cwm_conv_qk(const void* src, int src_dtype, long src_stride, int n_partials, long partial_stride, const float* bias,
                           const float* taps_w, int taps, float* state, long state_ld, const int* slots, const int* cu_q,
                           const int* seq_of_token, int n_slots, int n_seqs, int write_state, void* q_out, int out_dtype, float* gate_out,
                           const float* q_weight, const float* k_weight, float eps, const int* positions, const float* inv_freq,
                           void* cache, const int* block_table, int table_width, int page_size, int num_pages, int n_tokens, int n_q_heads,
                           int n_kv_heads, int dim, int head_dim, hipStream_t stream) {
  CWM_REQUIRE(n_tokens >= 0 && n_seqs >= 0 && n_partials >= 1 && n_q_heads >= 1 && n_kv_heads >= 1 && dim >= 1, "conv_qk: bad sizes");
  CWM_REQUIRE(n_partials == 1 || src_dtype == CWM_F32, "conv_qk: partial sums must be float32");
  CWM_REQUIRE(taps >= 1 && taps <= CONVQK_MAX_TAPS, "conv_qk: %d taps are outside 1..%d", taps, CONVQK_MAX_TAPS);
  CWM_REQUIRE(head_dim % 2 == 0 && head_dim >= dim && head_dim <= CONVQK_MAX_HEAD, "conv_qk: heads of %d do not fit an even cached head of %d, at most %d", dim,
              head_dim, CONVQK_MAX_HEAD);
  const int channels = (n_q_heads + n_kv_heads) * dim;
  CWM_REQUIRE((long)channels * 4 <= CONVQK_MAX_LDS, "conv_qk: %d channels, the kernel takes up to %d", channels, CONVQK_MAX_LDS / 4);
  CWM_REQUIRE(src && taps_w && slots && cu_q && seq_of_token && q_out && positions && cache && block_table, "conv_qk: arguments missing");
  CWM_REQUIRE(taps == 1 || (state && state_ld >= (long)(taps - 1) * channels), "conv_qk: the state does not hold %d rows of %d", taps - 1, channels);
  CWM_REQUIRE(page_size > 0 && num_pages > 0 && table_width > 0, "conv_qk: bad cache geometry");
  CWM_REQUIRE(eps > 0.f || (!q_weight && !k_weight), "conv_qk: eps must be positive");
  CWM_REQUIRE(write_state == 1 || write_state == 2, "conv_qk: unknown way to move the state");
  if (n_tokens == 0) return 0;
  const bool moves = write_state == 2 && taps > 1;
  // a block walks down several tokens where there are many of them and their rows fit
  const int tb = n_tokens >= 1024 && taps <= 4 && (long)CONVQK_TOKENS * channels * 4 <= CONVQK_MAX_LDS ? CONVQK_TOKENS : 1;
  const size_t lds = (size_t)tb * channels * sizeof(float);
  const uintptr_t row_bytes = src_dtype == CWM_F32 ? 16 : 8;
  const bool vec = taps <= 4 && (n_q_heads * dim) % 4 == 0 && channels % 4 == 0 && src_stride % 4 == 0 && partial_stride % 4 == 0 && state_ld % 4 == 0 &&
                   ((uintptr_t)src % row_bytes) == 0 && ((uintptr_t)bias % 16) == 0 && ((uintptr_t)taps_w % 16) == 0 && ((uintptr_t)state % 16) == 0;
  int threads = ((vec ? channels / 4 : channels) + CWM_WAVE - 1) / CWM_WAVE * CWM_WAVE;
  if (threads < 256) threads = 256;
  if (threads > CONVQK_THREADS) threads = CONVQK_THREADS;
#define CWM_CONVQK_GO(TS, TO, MAXT, TB, W)                                                                                              \
  hipLaunchKernelGGL((conv_qk_kernel<TS, TO, MAXT, TB, W>), dim3((n_tokens + TB - 1) / TB), dim3(threads), lds, stream,                 \
                     (const TS*)src, src_stride, n_partials, partial_stride, bias, taps_w, taps, state, state_ld, slots, cu_q,          \
                     seq_of_token, n_slots, moves, (TO*)q_out, gate_out, q_weight, k_weight, eps, positions, inv_freq, (TO*)cache,      \
                     block_table, table_width, page_size, num_pages, n_tokens, n_q_heads, n_kv_heads, dim, head_dim)
#define CWM_CONVQK(TS, TO)                                                                                                              \
  do {                                                                                                                                  \
    if (taps > 4) CWM_CONVQK_GO(TS, TO, CONVQK_MAX_TAPS, 1, 1);                                                                         \
    else if (tb == 1 && vec) CWM_CONVQK_GO(TS, TO, 4, 1, 4);                                                                            \
    else if (tb == 1) CWM_CONVQK_GO(TS, TO, 4, 1, 1);                                                                                   \
    else if (vec) CWM_CONVQK_GO(TS, TO, 4, CONVQK_TOKENS, 4);                                                                           \
    else CWM_CONVQK_GO(TS, TO, 4, CONVQK_TOKENS, 1);                                                                                    \
    if (write_state == 1 && taps > 1)                                                                                                   \
      hipLaunchKernelGGL((conv_qk_state_kernel<TS>), dim3(n_seqs, (channels + 255) / 256), dim3(256), 0, stream, (const TS*)src, src_stride, \
                         n_partials, partial_stride, bias, state, state_ld, slots, cu_q, n_slots, channels, taps);                     \
  } while (0)
  switch ((src_dtype << 1) | out_dtype) {
    case 0: CWM_CONVQK(float, float); break;
    case 1: CWM_CONVQK(float, bf16_t); break;
    case 3: CWM_CONVQK(bf16_t, bf16_t); break;
    default: return cwm_fail("conv_qk: source type %d with cache type %d is not built", src_dtype, out_dtype);
  }
#undef CWM_CONVQK
#undef CWM_CONVQK_GO
  return cwm_launch_status("conv_qk");
}
