// Several blends of a token's row with the row before it, out of one pass:
//
//   out_s[t] = h_t + (h_(t-1) - h_t) * mu_s          s = 0 .. n_mixes - 1, element by element
//
// with zeros before a sequence's first token.  The last h of a sequence is its state (float32, `dim` values from
// `state_offset` on in the sequence's slot), so that a portion's first token finds what the step before left.  The
// block of a portion's first token is the only one that touches the state: each of its threads reads the elements it
// owns and then leaves the portion's last row there.  float32 arithmetic.
#include "common.h"

CWM_DEFINE_ERROR_API

#define TMIX_THREADS 256
#define TMIX_MAX 8

extern "C" int cwm_token_mix_max() { return TMIX_MAX; }

template <typename T, int W> struct Some;
template <typename T> struct Some<T, 1> {
  static __device__ __forceinline__ void load(const T* p, float (&v)[1]) { v[0] = Elem<T>::load(p); }
  static __device__ __forceinline__ void store(T* p, const float (&v)[1]) { Elem<T>::store(p, v[0]); }
};
template <> struct Some<float, 4> {
  static __device__ __forceinline__ void load(const float* p, float (&v)[4]) {
    const float4 x = *(const float4*)p;
    v[0] = x.x, v[1] = x.y, v[2] = x.z, v[3] = x.w;
  }
  static __device__ __forceinline__ void store(float* p, const float (&v)[4]) { *(float4*)p = make_float4(v[0], v[1], v[2], v[3]); }
};
template <> struct Some<bf16_t, 4> {
  static __device__ __forceinline__ void load(const bf16_t* p, float (&v)[4]) {
    const uint2 x = *(const uint2*)p;
    v[0] = __uint_as_float(x.x << 16), v[1] = __uint_as_float(x.x & 0xffff0000u);
    v[2] = __uint_as_float(x.y << 16), v[3] = __uint_as_float(x.y & 0xffff0000u);
  }
  static __device__ __forceinline__ void store(bf16_t* p, const float (&v)[4]) {
    uint2 x;
    x.x = pack2_bf16(v[0], v[1]);
    x.y = pack2_bf16(v[2], v[3]);
    *(uint2*)p = x;
  }
};

template <typename T, int W>
__global__ void __launch_bounds__(TMIX_THREADS)
token_mix_kernel(const T* __restrict__ h, const float* __restrict__ mu, int n_mixes, T* __restrict__ out, long mix_stride,
                 float* state, long state_ld, long state_offset, const int* __restrict__ slots, const int* __restrict__ cu_q,
                 const int* __restrict__ seq_of_token, int n_slots, int dim) {
  const int t = blockIdx.x;
  const int d = W * (blockIdx.y * TMIX_THREADS + threadIdx.x);
  if (d >= dim) return;
  const int b = seq_of_token[t];
  float x[W], prev[W];
  Some<T, W>::load(h + (size_t)t * dim + d, x);
  if (t == cu_q[b]) {
    const int slot = slots[b];
    if (slot >= 0 && slot < n_slots) {
      float* srow = state + (size_t)slot * state_ld + state_offset + d;
      float last[W];
      Some<T, W>::load(h + (size_t)(cu_q[b + 1] - 1) * dim + d, last);
#pragma unroll
      for (int i = 0; i < W; ++i) prev[i] = srow[i];
#pragma unroll
      for (int i = 0; i < W; ++i) srow[i] = last[i];
    } else {
#pragma unroll
      for (int i = 0; i < W; ++i) prev[i] = 0.f;
    }
  } else {
    Some<T, W>::load(h + (size_t)(t - 1) * dim + d, prev);
  }
  for (int s = 0; s < n_mixes; ++s) {
    float m[W], o[W];
    Some<float, W>::load(mu + (size_t)s * dim + d, m);
#pragma unroll
    for (int i = 0; i < W; ++i) o[i] = fmaf(prev[i] - x[i], m[i], x[i]);
    Some<T, W>::store(out + (size_t)s * mix_stride + (size_t)t * dim + d, o);
  }
}

// h: contiguous [n_tokens][dim] of `dtype`; mu: float32 [n_mixes][dim]; out: n_mixes tensors [n_tokens][dim] of `dtype`,
// mix_stride elements apart; state: float32 [n_slots][state_ld]; slots: int32 [n_seqs]; cu_q: int32 [n_seqs + 1];
// seq_of_token: int32 [n_tokens].
extern "C" int cwm_token_mix(const void* h, int dtype, const float* mu, int n_mixes, void* out, long mix_stride, float* state,
                             long state_ld, long state_offset, const int* slots, const int* cu_q, const int* seq_of_token,
                             int n_slots, int n_tokens, int dim, hipStream_t stream) {
  CWM_REQUIRE(h && mu && out && state && slots && cu_q && seq_of_token, "token_mix: arguments missing");
  CWM_REQUIRE(n_tokens >= 0 && dim >= 1 && n_mixes >= 1 && n_mixes <= TMIX_MAX && n_slots > 0, "token_mix: bad sizes");
  CWM_REQUIRE(state_offset >= 0 && state_offset + dim <= state_ld, "token_mix: the state's row does not hold %d values from %ld on", dim, state_offset);
  CWM_REQUIRE(mix_stride >= (long)n_tokens * dim, "token_mix: the results overlap");
  if (n_tokens == 0) return 0;
  const int bytes = dtype == CWM_F32 ? 4 : 2;
  const bool vec = dim % 4 == 0 && mix_stride % 4 == 0 && ((uintptr_t)h % (4 * bytes)) == 0 && ((uintptr_t)out % (4 * bytes)) == 0 &&
                   ((uintptr_t)mu % 16) == 0;
  const int per = (vec ? 4 : 1) * TMIX_THREADS;
  const dim3 grid(n_tokens, (dim + per - 1) / per);
#define CWM_TMIX(T, W)                                                                                                     \
  hipLaunchKernelGGL((token_mix_kernel<T, W>), grid, dim3(TMIX_THREADS), 0, stream, (const T*)h, mu, n_mixes, (T*)out,       \
                     mix_stride, state, state_ld, state_offset, slots, cu_q, seq_of_token, n_slots, dim)
  if (dtype == CWM_F32) {
    if (vec) CWM_TMIX(float, 4); else CWM_TMIX(float, 1);
  } else if (dtype == CWM_BF16) {
    if (vec) CWM_TMIX(bf16_t, 4); else CWM_TMIX(bf16_t, 1);
  } else {
    return cwm_fail("token_mix: unknown element type %d", dtype);
  }
#undef CWM_TMIX
  return cwm_launch_status("token_mix");
}
