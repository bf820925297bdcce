// minGRU: every element of a state is an average over time whose weight depends on the token alone, not on the state:
//
//   z_t = sigmoid(a_t + b_z),   c_t = g(u_t + b_x)        a, u: projections of the token;  g(u) = u + 1/2 for u >= 0,
//   S_t = (1 - z_t) S_(t-1) + z_t c_t                     sigmoid(u) for u < 0
//   out_t = S_t * silu(y_t)                               y: a third projection
//
// S is float32, `width` values in the sequence's slot from one step to the next.  z and 1 - z are both
// formed from exp(-|.|), so neither loses digits where the gate is nearly shut or nearly open.
//
// `min_gru_walk_kernel`: a thread owns CH neighbouring elements and walks tokens one by one.
//   MODE 0: a block a (elements, sequence), over the sequence's tokens of the step, from its slot and back to it.
//   MODE 1: a block a (elements, segment of a sequence): the segment's product of (1 - z) and its state from zero (the
//           last segment's entry receives what the sequence's slot holds instead).
//   MODE 2: a block a (elements, segment): the segment's start is carried across the segments before it (their sums
//           and products, read by this block itself: a few dozen at most), then it walks with results; a sequence's
//           last segment leaves the state in the slot.
// A step without a long portion is MODE 0 in one launch, and gives the same bits however a sequence is cut; a step
// with one runs MODE 1 and MODE 2, which differ from the walk by float32 rounding.
#include "common.h"

CWM_DEFINE_ERROR_API

#define MGRU_THREADS 128

template <typename T, int CH> struct Cols;
template <typename T> struct Cols<T, 1> {
  static __device__ __forceinline__ void load(const T* p, float (&v)[1]) { v[0] = Elem<T>::load(p); }
  static __device__ __forceinline__ void store(T* p, const float (&v)[1]) { Elem<T>::store(p, v[0]); }
};
template <> struct Cols<float, 2> {
  static __device__ __forceinline__ void load(const float* p, float (&v)[2]) {
    const float2 x = *(const float2*)p;
    v[0] = x.x, v[1] = x.y;
  }
  static __device__ __forceinline__ void store(float* p, const float (&v)[2]) { *(float2*)p = make_float2(v[0], v[1]); }
};
template <> struct Cols<bf16_t, 2> {
  static __device__ __forceinline__ void load(const bf16_t* p, float (&v)[2]) {
    const uint32_t x = *(const uint32_t*)p;
    v[0] = __uint_as_float(x << 16), v[1] = __uint_as_float(x & 0xffff0000u);
  }
  static __device__ __forceinline__ void store(bf16_t* p, const float (&v)[2]) { *(uint32_t*)p = pack2_bf16(v[0], v[1]); }
};

// FAST: the hardware's exponential and reciprocal, each within a unit in the last place of float32 or so (results that
// are stored in bfloat16); else the library's.
template <bool FAST>
__device__ __forceinline__ float exp_of(float x) {
  return FAST ? __builtin_amdgcn_exp2f(x * 1.4426950408889634f) : expf(x);
}
template <bool FAST>
__device__ __forceinline__ float inverse_of(float x) {
  return FAST ? __builtin_amdgcn_rcpf(x) : 1.0f / x;
}

// sigmoid(v) and 1 - sigmoid(v)
template <bool FAST>
__device__ __forceinline__ void gate_pair(float v, float& open, float& keep) {
  const float e = exp_of<FAST>(-fabsf(v));
  const float inv = inverse_of<FAST>(1.0f + e);
  open = v >= 0.f ? inv : e * inv;
  keep = v >= 0.f ? e * inv : inv;
}

template <bool FAST>
__device__ __forceinline__ float candidate_of(float u) {
  return u >= 0.f ? u + 0.5f : inverse_of<FAST>(1.0f + exp_of<FAST>(-u));
}

// segments: int32 [n][6]: sequence, first token, end token, number of the segment in its sequence, the sequence's first
// entry of the scratch, segments of the sequence.  seg_sum, seg_keep: float32 [n][width].
template <typename TS, typename TO, int CH, int MODE>
__global__ void __launch_bounds__(MGRU_THREADS)
min_gru_walk_kernel(const TS* __restrict__ proj, long ld, int n_partials, long partial_stride, const float* __restrict__ z_bias,
                    const float* __restrict__ x_bias, TO* __restrict__ out, float* __restrict__ state, long state_ld,
                    const int* __restrict__ slots, const int* __restrict__ cu_q, int n_slots, int width,
                    const int* __restrict__ segments, float* __restrict__ seg_sum, float* __restrict__ seg_keep) {
  constexpr bool FAST = sizeof(TO) == 2;
  constexpr int AHEAD = MODE == 0 ? 2 : 8;  // tokens whose loads are in flight together, while those before are worked on
  const int c0 = CH * (blockIdx.x * MGRU_THREADS + threadIdx.x);
  if (c0 >= width) return;
  int b, t0, t1, number = 0, base = 0;
  bool last = true;
  if constexpr (MODE == 0) {
    b = blockIdx.y, t0 = cu_q[b], t1 = cu_q[b + 1];
  } else {
    const int* sg = segments + 6 * blockIdx.y;
    b = sg[0], t0 = sg[1], t1 = sg[2], number = sg[3], base = sg[4], last = number == sg[5] - 1;
  }
  const int slot = slots[b];
  if (slot < 0 || slot >= n_slots) return;
  float* st = state + (size_t)slot * state_ld + c0;
  if (MODE == 1 && last) {  // nothing comes after it: its entry hands on what the sequence started from
#pragma unroll
    for (int i = 0; i < CH; ++i) seg_sum[(size_t)(base + number) * width + c0 + i] = st[i];
    return;
  }
  float S[CH], K[CH], bz[CH], bx[CH];
#pragma unroll
  for (int i = 0; i < CH; ++i) {
    bz[i] = z_bias[c0 + i], bx[i] = x_bias[c0 + i];
    S[i] = MODE == 0 ? st[i] : 0.f;
    K[i] = 1.f;
  }
  if constexpr (MODE == 2) {
    // the slot itself may already be the last segment's: what it held lies in that segment's entry
    const size_t held = (size_t)(base + segments[6 * blockIdx.y + 5] - 1) * width + c0;
#pragma unroll
    for (int i = 0; i < CH; ++i) S[i] = seg_sum[held + i];
    for (int s = 0; s < number; s += 16) {  // sixteen segments' loads in flight
      float keep[16][CH], add[16][CH];
#pragma unroll
      for (int a = 0; a < 16; ++a) {
        const size_t at = (size_t)(base + min(s + a, number - 1)) * width + c0;
        Cols<float, CH>::load(seg_keep + at, keep[a]);
        Cols<float, CH>::load(seg_sum + at, add[a]);
      }
#pragma unroll
      for (int a = 0; a < 16; ++a)
#pragma unroll
        for (int i = 0; i < CH; ++i) S[i] = s + a < number ? fmaf(keep[a][i], S[i], add[a][i]) : S[i];
    }
  }
  auto fetch = [&](int t, int part, float (&v)[CH]) {
    const TS* p = proj + (size_t)t * ld + (size_t)part * width + c0;
    Cols<TS, CH>::load(p, v);
    for (int q = 1; q < n_partials; ++q) {
      float more[CH];
      Cols<TS, CH>::load(p + (size_t)q * partial_stride, more);
#pragma unroll
      for (int i = 0; i < CH; ++i) v[i] += more[i];
    }
  };
  float z[AHEAD][CH], x[AHEAD][CH], y[AHEAD][CH];
  auto fetch_from = [&](int t) {
#pragma unroll
    for (int a = 0; a < AHEAD; ++a) {
      const int tt = min(t + a, t1 - 1);  // past the last token: that one again, not used
      fetch(tt, 0, z[a]);
      fetch(tt, 1, x[a]);
      if constexpr (MODE != 1) fetch(tt, 2, y[a]);
    }
  };
  fetch_from(t0);
  for (int t = t0; t < t1; t += AHEAD) {
    // what does not depend on the state, then the next tokens' loads, then the chain through the state
    float keep[AHEAD][CH], add[AHEAD][CH], shown[AHEAD][CH];
#pragma unroll
    for (int a = 0; a < AHEAD; ++a)
#pragma unroll
      for (int i = 0; i < CH; ++i) {
        float open;
        gate_pair<FAST>(z[a][i] + bz[i], open, keep[a][i]);
        add[a][i] = open * candidate_of<FAST>(x[a][i] + bx[i]);
        if constexpr (MODE != 1) shown[a][i] = y[a][i] * inverse_of<FAST>(1.0f + exp_of<FAST>(-y[a][i]));
      }
    if (t + AHEAD < t1) fetch_from(t + AHEAD);
#pragma unroll
    for (int a = 0; a < AHEAD; ++a) {
      if (t + a < t1) {
        float o[CH];
#pragma unroll
        for (int i = 0; i < CH; ++i) {
          S[i] = fmaf(keep[a][i], S[i], add[a][i]);
          if constexpr (MODE == 1) K[i] *= keep[a][i];
          if constexpr (MODE != 1) o[i] = S[i] * shown[a][i];
        }
        if constexpr (MODE != 1) Cols<TO, CH>::store(out + (size_t)(t + a) * width + c0, o);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < CH; ++i) {
    if constexpr (MODE == 1) {
      seg_sum[(size_t)(base + number) * width + c0 + i] = S[i];
      seg_keep[(size_t)(base + number) * width + c0 + i] = K[i];
    } else {
      if (MODE == 0 || last) st[i] = S[i];
    }
  }
}


// proj: [n_tokens][ld] of src_dtype with z, x and gate columns (width each) leading a row, or n_partials float32 slabs
// partial_stride apart.  z_bias, x_bias: float32 [width].  out: contiguous [n_tokens][width].  state: float32 [n_slots]
// [state_ld], width <= state_ld; slots: int32 [n_seqs]; cu_q: int32 [n_seqs + 1].  segments (or null: every sequence is
// walked whole): int32 [n_segments][6] as above, all segments of the step; seg_sum, seg_keep: float32 [n_segments][width].
extern "C" int cwm_min_gru(const void* proj, int src_dtype, long ld, int n_partials, long partial_stride, const float* z_bias,
                           const float* x_bias, void* out, int out_dtype, float* state, long state_ld, const int* slots,
                           const int* cu_q, int n_slots, int n_tokens, int n_seqs, int width, const int* segments,
                           int n_segments, float* seg_sum, float* seg_keep, hipStream_t stream) {
  CWM_REQUIRE(n_tokens >= 0 && n_seqs >= 0 && width >= 1 && state_ld >= width, "min_gru: bad sizes");
  CWM_REQUIRE(proj && z_bias && x_bias && out && state && slots && cu_q, "min_gru: arguments missing");
  CWM_REQUIRE(n_partials >= 1 && (n_partials == 1 || src_dtype == CWM_F32), "min_gru: partial sums must be float32");
  CWM_REQUIRE(n_seqs <= 65535 && n_segments <= 65535, "min_gru: too many sequences or segments for one launch");
  CWM_REQUIRE(!segments || (n_segments >= 1 && seg_sum && seg_keep), "min_gru: segments need their scratch");
  if (n_tokens == 0 || n_seqs == 0) return 0;
  const int src_bytes = src_dtype == CWM_F32 ? 4 : 2;
  const bool two = width % 2 == 0 && ld % 2 == 0 && partial_stride % 2 == 0 && ((uintptr_t)proj % (2 * src_bytes)) == 0 &&
                   ((uintptr_t)out % (2 * (out_dtype == CWM_F32 ? 4 : 2))) == 0;
  const unsigned gx = (unsigned)((width + (two ? 2 : 1) * MGRU_THREADS - 1) / ((two ? 2 : 1) * MGRU_THREADS));
#define CWM_MGRU_GO(TS, TO, CH, MODE, COUNT)                                                                               \
  hipLaunchKernelGGL((min_gru_walk_kernel<TS, TO, CH, MODE>), dim3(gx, COUNT), dim3(MGRU_THREADS), 0, stream, (const TS*)proj, \
                     ld, n_partials, partial_stride, z_bias, x_bias, (TO*)out, state, state_ld, slots, cu_q, n_slots, width,  \
                     segments, seg_sum, seg_keep)
#define CWM_MGRU_CH(TS, TO, CH)                    \
  do {                                             \
    if (segments) {                                \
      CWM_MGRU_GO(TS, TO, CH, 1, n_segments);      \
      CWM_MGRU_GO(TS, TO, CH, 2, n_segments);      \
    } else {                                       \
      CWM_MGRU_GO(TS, TO, CH, 0, n_seqs);          \
    }                                              \
  } while (0)
#define CWM_MGRU(TS, TO)                           \
  do {                                             \
    if (two)                                       \
      CWM_MGRU_CH(TS, TO, 2);                      \
    else                                           \
      CWM_MGRU_CH(TS, TO, 1);                      \
  } while (0)
  switch ((src_dtype << 1) | out_dtype) {
    case 0: CWM_MGRU(float, float); break;
    case 1: CWM_MGRU(float, bf16_t); break;
    case 3: CWM_MGRU(bf16_t, bf16_t); break;
    default: return cwm_fail("min_gru: a projection of type %d with results of type %d is not built", src_dtype, out_dtype);
  }
#undef CWM_MGRU
#undef CWM_MGRU_CH
#undef CWM_MGRU_GO
  return cwm_launch_status("min_gru");
}
