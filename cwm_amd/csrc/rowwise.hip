// Row-wise kernels of the decoder: token embedding gather, residual-add fused with
// RMSNorm, and SiLU(gate) * up.  All arithmetic is float32; storage types are
// chosen per argument (float32 or bfloat16).
//
// Formulas: embedding cwm/fastgen/forward.py:543-546; RMSNorm
// cwm/fastgen/kernels/rmsnorm.py:34-61; SiLU * up cwm/fastgen/forward.py:781.
#include "common.h"

CWM_DEFINE_ERROR_API

// ---- embedding: out[t, :] = scale * table[token[t], :] as float32 -------------- //
// (scale is 1 for the architecture of the reference; others multiply the embedding)
template <typename TW>
__global__ void embedding_kernel(float* __restrict__ out, const TW* __restrict__ table,
                                 const int* __restrict__ tokens, int dim, int vocab, float scale) {
  const int t = blockIdx.x;
  const int tok = tokens[t];
  float* dst = out + (size_t)t * dim;
  if (tok < 0 || tok >= vocab) {  // the host checks ids; never read outside the table
    for (int i = threadIdx.x; i < dim; i += blockDim.x) dst[i] = __uint_as_float(0x7fc00000u);
    return;
  }
  const TW* src = table + (size_t)tok * dim;
  for (int i = threadIdx.x; i < dim; i += blockDim.x) dst[i] = scale * Elem<TW>::load(src + i);
}

extern "C" int cwm_embedding(void* out, const void* table, int table_dtype, const int* tokens,
                             int n_tokens, int dim, int vocab, float scale, hipStream_t stream) {
  CWM_REQUIRE(n_tokens >= 0 && dim > 0 && vocab > 0, "embedding: bad sizes T=%d D=%d V=%d", n_tokens, dim, vocab);
  if (n_tokens == 0) return 0;
  const int threads = dim >= 1024 ? 256 : (dim >= 256 ? 128 : 64);
  if (table_dtype == CWM_F32)
    hipLaunchKernelGGL(embedding_kernel<float>, dim3(n_tokens), dim3(threads), 0, stream, (float*)out,
                       (const float*)table, tokens, dim, vocab, scale);
  else if (table_dtype == CWM_BF16)
    hipLaunchKernelGGL(embedding_kernel<bf16_t>, dim3(n_tokens), dim3(threads), 0, stream, (float*)out,
                       (const bf16_t*)table, tokens, dim, vocab, scale);
  else
    return cwm_fail("embedding: unknown table dtype %d", table_dtype);
  return cwm_launch_status("embedding");
}

// out[t, :] = scale * table[token[t], :] + s(positions[t]), the sinusoidal position vector s(p)[2i] = sin(p f_i),
// s(p)[2i + 1] = cos(p f_i).  `turns` holds f_i / (2 pi) in float64 (one value a pair): the angle in turns is reduced to
// [-1/2, 1/2] in float64, so that a far position costs no digits of it.
template <typename TW>
__global__ void embedding_sinusoid_kernel(float* __restrict__ out, const TW* __restrict__ table, const int* __restrict__ tokens,
                                          const int* __restrict__ positions, const double* __restrict__ turns, int dim, int vocab,
                                          float scale) {
  const int t = blockIdx.x;
  const int tok = tokens[t];
  const bool known = tok >= 0 && tok < vocab;
  const double p = (double)positions[t];
  float* dst = out + (size_t)t * dim;
  const TW* src = table + (size_t)(known ? tok : 0) * dim;
  for (int i = blockIdx.y * blockDim.x + threadIdx.x; 2 * i < dim; i += gridDim.y * blockDim.x) {
    const double a = p * turns[i];
    float s, c;
    sincosf((float)(a - rint(a)) * 6.283185307179586f, &s, &c);
    dst[2 * i] = known ? fmaf(scale, Elem<TW>::load(src + 2 * i), s) : __uint_as_float(0x7fc00000u);
    if (2 * i + 1 < dim) dst[2 * i + 1] = known ? fmaf(scale, Elem<TW>::load(src + 2 * i + 1), c) : __uint_as_float(0x7fc00000u);
  }
}

extern "C" int cwm_embedding_sinusoid(void* out, const void* table, int table_dtype, const int* tokens, const int* positions,
                                      const double* turns, int n_tokens, int dim, int vocab, float scale, hipStream_t stream) {
  CWM_REQUIRE(n_tokens >= 0 && dim > 0 && vocab > 0, "embedding_sinusoid: bad sizes T=%d D=%d V=%d", n_tokens, dim, vocab);
  CWM_REQUIRE(out && table && tokens && positions && turns, "embedding_sinusoid: arguments missing");
  if (n_tokens == 0) return 0;
  const int pairs = (dim + 1) / 2;
  const int threads = pairs >= 256 ? 256 : (pairs >= 128 ? 128 : 64);
  const dim3 grid(n_tokens, n_tokens >= 512 ? 1 : (pairs + threads - 1) / threads);
  if (table_dtype == CWM_F32)
    hipLaunchKernelGGL(embedding_sinusoid_kernel<float>, grid, dim3(threads), 0, stream, (float*)out, (const float*)table, tokens,
                       positions, turns, dim, vocab, scale);
  else if (table_dtype == CWM_BF16)
    hipLaunchKernelGGL(embedding_sinusoid_kernel<bf16_t>, grid, dim3(threads), 0, stream, (float*)out, (const bf16_t*)table, tokens,
                       positions, turns, dim, vocab, scale);
  else
    return cwm_fail("embedding_sinusoid: unknown table dtype %d", table_dtype);
  return cwm_launch_status("embedding_sinusoid");
}

// ---- h += delta (float32), out = h * rsqrt(mean(h^2) + eps) * w ---------------- //
// One block per output row.  With `rows`, output row r is computed from source row
// rows[r] and h is not modified.
template <typename TD, typename TW, typename TO>
__global__ void add_rmsnorm_kernel(float* __restrict__ h, const TD* __restrict__ delta, int n_partials,
                                   long partial_stride, const TW* __restrict__ weight, TO* __restrict__ out,
                                   const int* __restrict__ rows, int dim, float eps) {
  __shared__ float scratch[16];
  const int r = blockIdx.x;
  const int src = rows ? rows[r] : r;
  float* hrow = h + (size_t)src * dim;
  const TD* drow = delta ? delta + (size_t)src * dim : nullptr;
  const bool write_back = (delta != nullptr) && (rows == nullptr);
  float ss = 0.f;
  for (int i = threadIdx.x; i < dim; i += blockDim.x) {
    float v = hrow[i];
    if (drow) {
      for (int p = 0; p < n_partials; ++p) v += Elem<TD>::load(drow + (size_t)p * partial_stride + i);
      if (write_back) hrow[i] = v;
    }
    ss += v * v;
  }
  ss = block_sum(ss, scratch);
  const float rstd = 1.0f / sqrtf(ss / (float)dim + eps);
  TO* orow = out + (size_t)r * dim;
  for (int i = threadIdx.x; i < dim; i += blockDim.x) {
    float v = hrow[i];
    if (drow && !write_back)
      for (int p = 0; p < n_partials; ++p) v += Elem<TD>::load(drow + (size_t)p * partial_stride + i);
    Elem<TO>::store(orow + i, v * rstd * Elem<TW>::load(weight + i));
  }
}

// The same for rows that fit in registers (dim % 4 == 0, dim <= 4 * CHUNKS * threads):
// every load of a row is issued at once, the row is read once and never re-read.
template <typename T> struct Vec4;
template <> struct Vec4<float> {
  static __device__ __forceinline__ void load(const float* p, float (&v)[4]) {
    const float4 x = *(const float4*)p;
    v[0] = x.x; v[1] = x.y; v[2] = x.z; v[3] = x.w;
  }
  static __device__ __forceinline__ void store(float* p, const float (&v)[4]) { *(float4*)p = make_float4(v[0], v[1], v[2], v[3]); }
};
template <> struct Vec4<bf16_t> {
  static __device__ __forceinline__ void load(const bf16_t* p, float (&v)[4]) {
    const uint2 x = *(const uint2*)p;
    v[0] = __uint_as_float(x.x << 16); v[1] = __uint_as_float(x.x & 0xffff0000u);
    v[2] = __uint_as_float(x.y << 16); v[3] = __uint_as_float(x.y & 0xffff0000u);
  }
  static __device__ __forceinline__ void store(bf16_t* p, const float (&v)[4]) {
    uint2 x;
    x.x = (uint32_t)f32_to_bf16(v[0]) | ((uint32_t)f32_to_bf16(v[1]) << 16);
    x.y = (uint32_t)f32_to_bf16(v[2]) | ((uint32_t)f32_to_bf16(v[3]) << 16);
    *(uint2*)p = x;
  }
};

template <typename TD, typename TW, typename TO, int CHUNKS>
__global__ void add_rmsnorm_regs_kernel(float* __restrict__ h, const TD* __restrict__ delta, int n_partials,
                                        long partial_stride, const TW* __restrict__ weight, TO* __restrict__ out,
                                        const int* __restrict__ rows, int dim, float eps) {
  __shared__ float scratch[16];
  const int r = blockIdx.x;
  const int src = rows ? rows[r] : r;
  float* hrow = h + (size_t)src * dim;
  const TD* drow = delta ? delta + (size_t)src * dim : nullptr;
  const bool write_back = (delta != nullptr) && (rows == nullptr);
  const int n_chunks = dim >> 2;
  float v[CHUNKS][4], w[CHUNKS][4];
#pragma unroll
  for (int c = 0; c < CHUNKS; ++c) {
    const int chunk = threadIdx.x + c * blockDim.x;
    if (chunk < n_chunks) {
      Vec4<float>::load(hrow + 4 * chunk, v[c]);
      Vec4<TW>::load(weight + 4 * chunk, w[c]);
      if (drow) {
        // four partial sums in flight at a time (a fifth would wait for the first otherwise); what lies
        // past the last one is loaded again from the last and not added; the order of the sum stays p = 0, 1, ...
        if (n_partials == 1) {
          float d[4];
          Vec4<TD>::load(drow + 4 * chunk, d);
#pragma unroll
          for (int i = 0; i < 4; ++i) v[c][i] += d[i];
        } else
        for (int p = 0; p < n_partials; p += 4) {
          float d[4][4];
#pragma unroll
          for (int u = 0; u < 4; ++u) Vec4<TD>::load(drow + (size_t)min(p + u, n_partials - 1) * partial_stride + 4 * chunk, d[u]);
#pragma unroll
          for (int u = 0; u < 4; ++u) {
            const float keep = p + u < n_partials ? 1.0f : 0.0f;
#pragma unroll
            for (int i = 0; i < 4; ++i) v[c][i] += keep * d[u][i];
          }
        }
      }
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i) v[c][i] = w[c][i] = 0.f;
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < CHUNKS; ++c) {
    const int chunk = threadIdx.x + c * blockDim.x;
    if (write_back && chunk < n_chunks) Vec4<float>::store(hrow + 4 * chunk, v[c]);
#pragma unroll
    for (int i = 0; i < 4; ++i) ss += v[c][i] * v[c][i];
  }
  ss = block_sum(ss, scratch);
  const float rstd = 1.0f / sqrtf(ss / (float)dim + eps);
  TO* orow = out + (size_t)r * dim;
#pragma unroll
  for (int c = 0; c < CHUNKS; ++c) {
    const int chunk = threadIdx.x + c * blockDim.x;
    if (chunk < n_chunks) {
      float y[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) y[i] = v[c][i] * rstd * w[c][i];
      Vec4<TO>::store(orow + 4 * chunk, y);
    }
  }
}

template <typename TD, typename TW, typename TO>
static void launch_add_rmsnorm(void* h, const void* delta, int n_partials, long partial_stride, const void* w, void* out,
                               const int* rows, int n_out, int dim, float eps, hipStream_t stream) {
  const int n_chunks = dim / 4;
  if (dim % 4 == 0 && n_chunks <= 4 * 512) {
    // all pointers are rows of contiguous tensors whose row length is a multiple of 4: 16-byte aligned loads
    int threads = 64;
    while (threads < 512 && threads * 4 < n_chunks) threads *= 2;
    const int chunks = (n_chunks + threads - 1) / threads;
    auto go = [&](auto kernel) {
      hipLaunchKernelGGL(kernel, dim3(n_out), dim3(threads), 0, stream, (float*)h, (const TD*)delta, n_partials,
                         partial_stride, (const TW*)w, (TO*)out, rows, dim, eps);
    };
    if (chunks <= 1) go(add_rmsnorm_regs_kernel<TD, TW, TO, 1>);
    else if (chunks <= 2) go(add_rmsnorm_regs_kernel<TD, TW, TO, 2>);
    else if (chunks <= 3) go(add_rmsnorm_regs_kernel<TD, TW, TO, 3>);
    else go(add_rmsnorm_regs_kernel<TD, TW, TO, 4>);
    return;
  }
  const int threads = dim >= 2048 ? 512 : (dim >= 512 ? 256 : (dim >= 128 ? 128 : 64));
  hipLaunchKernelGGL((add_rmsnorm_kernel<TD, TW, TO>), dim3(n_out), dim3(threads), 0, stream, (float*)h,
                     (const TD*)delta, n_partials, partial_stride, (const TW*)w, (TO*)out, rows, dim, eps);
}

extern "C" int cwm_add_rmsnorm(void* h, const void* delta, int delta_dtype, int n_partials, long partial_stride,
                               const void* weight, int weight_dtype, void* out, int out_dtype, const int* rows,
                               int n_out, int dim, float eps, hipStream_t stream) {
  CWM_REQUIRE(n_out >= 0 && dim > 0, "add_rmsnorm: bad sizes rows=%d D=%d", n_out, dim);
  CWM_REQUIRE(n_partials >= 1 && (n_partials == 1 || delta_dtype == CWM_F32), "add_rmsnorm: partial sums must be float32");
  CWM_REQUIRE(eps > 0.f, "add_rmsnorm: eps must be positive");
  if (n_out == 0) return 0;
  if (!delta) delta_dtype = CWM_F32;
  const int key = (delta_dtype << 2) | (weight_dtype << 1) | out_dtype;
  switch (key) {
    case 0: launch_add_rmsnorm<float, float, float>(h, delta, n_partials, partial_stride, weight, out, rows, n_out, dim, eps, stream); break;
    case 1: launch_add_rmsnorm<float, float, bf16_t>(h, delta, n_partials, partial_stride, weight, out, rows, n_out, dim, eps, stream); break;
    case 2: launch_add_rmsnorm<float, bf16_t, float>(h, delta, n_partials, partial_stride, weight, out, rows, n_out, dim, eps, stream); break;
    case 3: launch_add_rmsnorm<float, bf16_t, bf16_t>(h, delta, n_partials, partial_stride, weight, out, rows, n_out, dim, eps, stream); break;
    case 4: launch_add_rmsnorm<bf16_t, float, float>(h, delta, n_partials, partial_stride, weight, out, rows, n_out, dim, eps, stream); break;
    case 5: launch_add_rmsnorm<bf16_t, float, bf16_t>(h, delta, n_partials, partial_stride, weight, out, rows, n_out, dim, eps, stream); break;
    case 6: launch_add_rmsnorm<bf16_t, bf16_t, float>(h, delta, n_partials, partial_stride, weight, out, rows, n_out, dim, eps, stream); break;
    case 7: launch_add_rmsnorm<bf16_t, bf16_t, bf16_t>(h, delta, n_partials, partial_stride, weight, out, rows, n_out, dim, eps, stream); break;
    default: return cwm_fail("add_rmsnorm: unknown dtypes delta=%d weight=%d out=%d", delta_dtype, weight_dtype, out_dtype);
  }
  return cwm_launch_status("add_rmsnorm");
}

// ---- out[t, f] = silu(gate[t, f]) * up[t, f] ------------------------------------ //
// Row t of x holds 2F values: gate[f] at f and up[f] at F + f, or, with `grouped`, gate and up
// in alternating groups of 8 (gate[f] at 16 * (f / 8) + f % 8, up[f] 8 further), the order in
// which a product with row-interleaved gate/up weights delivers them.
template <typename T>
__global__ void silu_mul_kernel(T* __restrict__ out, const T* __restrict__ x, int hidden, size_t total, int grouped) {
  size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  const size_t stride = (size_t)gridDim.x * blockDim.x;
  for (; idx < total; idx += stride) {
    const size_t t = idx / hidden;
    const int f = (int)(idx - t * hidden);
    const T* row = x + t * 2 * (size_t)hidden;
    const int at = grouped ? 16 * (f >> 3) + (f & 7) : f;
    const float g = Elem<T>::load(row + at);
    const float u = Elem<T>::load(row + at + (grouped ? 8 : hidden));
    const float s = g / (1.0f + expf(-g));
    Elem<T>::store(out + idx, s * u);
  }
}

// eight bfloat16 pairs per thread, 16-byte loads and stores (hidden % 8 == 0)
__global__ void silu_mul_bf16x8_kernel(bf16_t* __restrict__ out, const bf16_t* __restrict__ x, int hidden8, size_t total8,
                                       int grouped) {
  size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  const size_t stride = (size_t)gridDim.x * blockDim.x;
  for (; idx < total8; idx += stride) {
    const size_t t = idx / hidden8;
    const int f8 = (int)(idx - t * hidden8);
    const bf16_t* row = x + t * 16 * (size_t)hidden8;
    const uint4 g = *(const uint4*)(row + (grouped ? 16 : 8) * f8);
    const uint4 u = *(const uint4*)(row + (grouped ? 16 * f8 + 8 : 8 * (size_t)hidden8 + 8 * f8));
    const uint32_t gi[4] = {g.x, g.y, g.z, g.w};
    const uint32_t ui[4] = {u.x, u.y, u.z, u.w};
    uint32_t o[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float g0 = __uint_as_float(gi[i] << 16), g1 = __uint_as_float(gi[i] & 0xffff0000u);
      const float u0 = __uint_as_float(ui[i] << 16), u1 = __uint_as_float(ui[i] & 0xffff0000u);
      const float s0 = g0 / (1.0f + expf(-g0));
      const float s1 = g1 / (1.0f + expf(-g1));
      o[i] = (uint32_t)f32_to_bf16(s0 * u0) | ((uint32_t)f32_to_bf16(s1 * u1) << 16);
    }
    *(uint4*)(out + 8 * idx) = make_uint4(o[0], o[1], o[2], o[3]);
  }
}

// The same from float32 partial sums x[p][t][2F] of a product whose K was split: the partials are
// added in order p = 0, 1, ..., the sums rounded to the output type (as the product would have
// stored them), then silu(gate) * up.  Four columns per thread (hidden % 4 == 0).
template <typename T>
__global__ void silu_mul_partials_kernel(T* __restrict__ out, const float* __restrict__ x, int n_partials, size_t part_stride,
                                         int hidden4, size_t total4, int grouped) {
  size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  const size_t stride = (size_t)gridDim.x * blockDim.x;
  for (; idx < total4; idx += stride) {
    const size_t t = idx / hidden4;
    const int f4 = (int)(idx - t * hidden4);
    const float* row = x + t * 8 * (size_t)hidden4 + (grouped ? 16 * (f4 >> 1) + 4 * (f4 & 1) : 4 * f4);
    const size_t to_up = grouped ? 8 : 4 * (size_t)hidden4;
    float4 g = make_float4(0.f, 0.f, 0.f, 0.f), u = g;
    for (int p = 0; p < n_partials; ++p) {
      const float4 gp = *(const float4*)(row + p * part_stride);
      const float4 up = *(const float4*)(row + p * part_stride + to_up);
      g.x += gp.x; g.y += gp.y; g.z += gp.z; g.w += gp.w;
      u.x += up.x; u.y += up.y; u.z += up.z; u.w += up.w;
    }
    const float gs[4] = {g.x, g.y, g.z, g.w};
    const float us[4] = {u.x, u.y, u.z, u.w};
    T* o = out + 4 * idx;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      T gr, ur;
      Elem<T>::store(&gr, gs[i]);
      Elem<T>::store(&ur, us[i]);
      const float gv = Elem<T>::load(&gr), uv = Elem<T>::load(&ur);
      Elem<T>::store(o + i, gv / (1.0f + expf(-gv)) * uv);
    }
  }
}

extern "C" int cwm_silu_mul_partials(void* out, int out_dtype, const void* partials, int n_partials, int n_tokens, int hidden,
                                     int grouped, hipStream_t stream) {
  CWM_REQUIRE(!grouped || hidden % 8 == 0, "silu_mul_partials: groups of 8 need F=%d to be a multiple of 8", hidden);
  CWM_REQUIRE(n_tokens >= 0 && hidden > 0 && n_partials > 0, "silu_mul_partials: bad sizes P=%d T=%d F=%d", n_partials,
              n_tokens, hidden);
  CWM_REQUIRE(hidden % 4 == 0 && ((uintptr_t)partials % 16) == 0, "silu_mul_partials: F=%d must be a multiple of 4 and the "
              "partial sums 16-byte aligned", hidden);
  if (n_tokens == 0) return 0;
  const size_t total4 = (size_t)n_tokens * (hidden / 4);
  const size_t part_stride = (size_t)n_tokens * 2 * hidden;
  const int threads = 256;
  size_t blocks = (total4 + threads - 1) / threads;
  if (blocks > 16384) blocks = 16384;
  if (out_dtype == CWM_F32)
    hipLaunchKernelGGL(silu_mul_partials_kernel<float>, dim3((unsigned)blocks), dim3(threads), 0, stream, (float*)out,
                       (const float*)partials, n_partials, part_stride, hidden / 4, total4, grouped);
  else if (out_dtype == CWM_BF16)
    hipLaunchKernelGGL(silu_mul_partials_kernel<bf16_t>, dim3((unsigned)blocks), dim3(threads), 0, stream, (bf16_t*)out,
                       (const float*)partials, n_partials, part_stride, hidden / 4, total4, grouped);
  else
    return cwm_fail("silu_mul_partials: unknown dtype %d", out_dtype);
  return cwm_launch_status("silu_mul_partials");
}

extern "C" int cwm_silu_mul(void* out, const void* x, int dtype, int n_tokens, int hidden, int grouped, hipStream_t stream) {
  CWM_REQUIRE(n_tokens >= 0 && hidden > 0, "silu_mul: bad sizes T=%d F=%d", n_tokens, hidden);
  CWM_REQUIRE(!grouped || hidden % 8 == 0, "silu_mul: groups of 8 need F=%d to be a multiple of 8", hidden);
  if (n_tokens == 0) return 0;
  const size_t total = (size_t)n_tokens * hidden;
  const int threads = 256;
  if (dtype == CWM_BF16 && hidden % 8 == 0 && ((uintptr_t)x % 16) == 0 && ((uintptr_t)out % 16) == 0) {
    const size_t total8 = total / 8;
    size_t blocks = (total8 + threads - 1) / threads;
    if (blocks > 16384) blocks = 16384;
    hipLaunchKernelGGL(silu_mul_bf16x8_kernel, dim3((unsigned)blocks), dim3(threads), 0, stream, (bf16_t*)out,
                       (const bf16_t*)x, hidden / 8, total8, grouped);
    return cwm_launch_status("silu_mul");
  }
  size_t blocks = (total + threads - 1) / threads;
  if (blocks > 65536) blocks = 65536;
  if (dtype == CWM_F32)
    hipLaunchKernelGGL(silu_mul_kernel<float>, dim3((unsigned)blocks), dim3(threads), 0, stream, (float*)out,
                       (const float*)x, hidden, total, grouped);
  else if (dtype == CWM_BF16)
    hipLaunchKernelGGL(silu_mul_kernel<bf16_t>, dim3((unsigned)blocks), dim3(threads), 0, stream, (bf16_t*)out,
                       (const bf16_t*)x, hidden, total, grouped);
  else
    return cwm_fail("silu_mul: unknown dtype %d", dtype);
  return cwm_launch_status("silu_mul");
}

// ---- out = sum over p of partials[p] (float32, in order) ----------------------- //
template <typename TO>
__global__ void sum_partials_kernel(TO* __restrict__ out, const float* __restrict__ partials, int n_partials, long count) {
  long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
  const long stride = (long)gridDim.x * blockDim.x;
  for (; i < count; i += stride) {
    float v = 0.f;
    for (int p = 0; p < n_partials; ++p) v += partials[(size_t)p * count + i];
    Elem<TO>::store(out + i, v);
  }
}

extern "C" int cwm_sum_partials(void* out, int out_dtype, const float* partials, int n_partials, long count,
                                hipStream_t stream) {
  CWM_REQUIRE(n_partials >= 1 && count >= 0, "sum_partials: bad sizes");
  if (count == 0) return 0;
  long blocks = (count + 255) / 256;
  if (blocks > 4096) blocks = 4096;
  if (out_dtype == CWM_F32)
    hipLaunchKernelGGL(sum_partials_kernel<float>, dim3((unsigned)blocks), dim3(256), 0, stream, (float*)out, partials,
                       n_partials, count);
  else if (out_dtype == CWM_BF16)
    hipLaunchKernelGGL(sum_partials_kernel<bf16_t>, dim3((unsigned)blocks), dim3(256), 0, stream, (bf16_t*)out, partials,
                       n_partials, count);
  else
    return cwm_fail("sum_partials: unknown dtype %d", out_dtype);
  return cwm_launch_status("sum_partials");
}

// ---- out = act(sum over p of x[p]) ------------------------------------------------ //
// The activation between the two products of a feed-forward without a gate: `x` is [count] values of type TX, or
// n_partials float32 slabs `count` apart that are added in order first; float32 arithmetic, rounded once.
// kind 0: the square of relu; 1: relu; 2: gelu (tanh form); 3: silu; 4: gelu (erf form); 5: tanh.
#define CWM_ACT_KINDS 6
__device__ __forceinline__ float act_value(float z, int kind) {
  switch (kind) {
    case 0: {
      const float r = fmaxf(z, 0.f);
      return r * r;
    }
    case 1:
      return fmaxf(z, 0.f);
    case 2:
      return 0.5f * z * (1.f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
    case 4:
      return 0.5f * z * (1.f + erff(z * 0.7071067811865476f));
    case 5:
      return tanhf(z);
    default:
      return z / (1.f + expf(-z));
  }
}

template <typename TX, typename TO>
__global__ void act_rows_kernel(TO* __restrict__ out, const TX* __restrict__ x, int n_partials, long count, int kind) {
  long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
  const long stride = (long)gridDim.x * blockDim.x;
  for (; i < count; i += stride) {
    float v = 0.f;
    for (int p = 0; p < n_partials; ++p) v += Elem<TX>::load(x + (size_t)p * count + i);
    Elem<TO>::store(out + i, act_value(v, kind));
  }
}

extern "C" int cwm_act_rows(void* out, int out_dtype, const void* x, int x_dtype, int n_partials, long count, int kind,
                            hipStream_t stream) {
  CWM_REQUIRE(n_partials >= 1 && count >= 0, "act_rows: bad sizes");
  CWM_REQUIRE(n_partials == 1 || x_dtype == CWM_F32, "act_rows: partial sums must be float32");
  CWM_REQUIRE(kind >= 0 && kind < CWM_ACT_KINDS, "act_rows: unknown activation %d", kind);
  if (count == 0) return 0;
  long blocks = (count + 255) / 256;
  if (blocks > 8192) blocks = 8192;
  const int key = (x_dtype << 1) | out_dtype;
#define CWM_ACT_LAUNCH(TX, TO)                                                                                        \
  hipLaunchKernelGGL((act_rows_kernel<TX, TO>), dim3((unsigned)blocks), dim3(256), 0, stream, (TO*)out, (const TX*)x, \
                     n_partials, count, kind)
  switch (key) {
    case 0: CWM_ACT_LAUNCH(float, float); break;
    case 1: CWM_ACT_LAUNCH(float, bf16_t); break;
    case 2: CWM_ACT_LAUNCH(bf16_t, float); break;
    case 3: CWM_ACT_LAUNCH(bf16_t, bf16_t); break;
    default: return cwm_fail("act_rows: unknown dtypes x=%d out=%d", x_dtype, out_dtype);
  }
#undef CWM_ACT_LAUNCH
  return cwm_launch_status("act_rows");
}

// ---- out = gated(sum over p of x[p]) ------------------------------------------------ //
// What a gated feed-forward makes of its joined gate/up product: `x` is [T, 2 F (+ extra)] of type TX, a row's gate
// values first, then its up values (or n_partials float32 slabs that are added in order first); out [T, F].
// kind 0: silu(g) * u.  kind 1: g' * sigmoid(alpha * g') * (u' + 1) with g' = min(g, limit), u' = clamp(u, -limit,
// limit).  kind 2: gelu(g) * u, the tanh form of gelu.  With `row_gate_col` >= 0 the row is also multiplied by the sigmoid of that column of x (one more output
// of the same product: a gate on the whole row).  float32 arithmetic, rounded once.
__device__ __forceinline__ float gated_pair(float g, float u, int kind, float alpha, float limit) {
  if (kind == 1) {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    return g / (1.f + expf(-alpha * g)) * (u + 1.f);
  }
  if (kind == 2) return act_value(g, 2) * u;
  return g / (1.f + expf(-g)) * u;
}

template <typename TX, typename TO>
__global__ void gated_act_rows_kernel(TO* __restrict__ out, const TX* __restrict__ x, long x_ld, int n_partials,
                                      long partial_stride, int n_rows, int hidden, int row_gate_col, int kind, float alpha,
                                      float limit) {
  const long count = (long)n_rows * hidden;
  long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
  const long stride = (long)gridDim.x * blockDim.x;
  for (; i < count; i += stride) {
    const long t = i / hidden;
    const int f = (int)(i - t * hidden);
    const TX* row = x + (size_t)t * x_ld;
    float g = 0.f, u = 0.f, r = 0.f;
    for (int p = 0; p < n_partials; ++p) {
      g += Elem<TX>::load(row + (size_t)p * partial_stride + f);
      u += Elem<TX>::load(row + (size_t)p * partial_stride + hidden + f);
      if (row_gate_col >= 0) r += Elem<TX>::load(row + (size_t)p * partial_stride + row_gate_col);
    }
    float v = gated_pair(g, u, kind, alpha, limit);
    if (row_gate_col >= 0) v *= 1.f / (1.f + expf(-r));
    Elem<TO>::store(out + i, v);
  }
}

extern "C" int cwm_gated_act_rows(void* out, int out_dtype, const void* x, int x_dtype, long x_ld, int n_partials,
                                  long partial_stride, int n_rows, int hidden, int row_gate_col, int kind, float alpha,
                                  float limit, hipStream_t stream) {
  CWM_REQUIRE(n_partials >= 1 && n_rows >= 0 && hidden >= 1, "gated_act_rows: bad sizes");
  CWM_REQUIRE(n_partials == 1 || x_dtype == CWM_F32, "gated_act_rows: partial sums must be float32");
  CWM_REQUIRE(kind >= 0 && kind <= 2, "gated_act_rows: unknown gated activation %d", kind);
  CWM_REQUIRE(kind != 1 || limit > 0.f, "gated_act_rows: the clamped form needs a positive limit");
  if (n_rows == 0) return 0;
  long blocks = ((long)n_rows * hidden + 255) / 256;
  if (blocks > 8192) blocks = 8192;
  const int key = (x_dtype << 1) | out_dtype;
#define CWM_GACT_LAUNCH(TX, TO)                                                                                         \
  hipLaunchKernelGGL((gated_act_rows_kernel<TX, TO>), dim3((unsigned)blocks), dim3(256), 0, stream, (TO*)out, (const TX*)x, \
                     x_ld, n_partials, partial_stride, n_rows, hidden, row_gate_col, kind, alpha, limit)
  switch (key) {
    case 0: CWM_GACT_LAUNCH(float, float); break;
    case 1: CWM_GACT_LAUNCH(float, bf16_t); break;
    case 2: CWM_GACT_LAUNCH(bf16_t, float); break;
    case 3: CWM_GACT_LAUNCH(bf16_t, bf16_t); break;
    default: return cwm_fail("gated_act_rows: unknown dtypes x=%d out=%d", x_dtype, out_dtype);
  }
#undef CWM_GACT_LAUNCH
  return cwm_launch_status("gated_act_rows");
}
