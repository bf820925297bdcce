// The sum of several sublayers' results, each normalised over the row first, joined to the residual, and the norm that
// reads the residual next, in one pass:
//
//   x   <- x + sum_a c_a y_a / sqrt(mean(y_a^2) + eps_a) * w_a        in the order of the addends
//   out  = x / sqrt(mean(x^2) + eps) * w
//
// An addend y_a is a [T, D] tensor (rows may lie apart), float32 partial sums [P, T, D] of a product whose K was
// split, added in order, or a token's weighted sum of float32 rows, y_a[t] = sum_k c[t][k] rows[index[t][k]] in the order
// of k (what routed experts leave: an index below 0 names no row).  float32 arithmetic.  One block a row.  With `rows` only those rows are read and the residual
// is left as it was.  Rows of up to 8,192 elements (a multiple of 4) with up to two addends stay in registers; others
// are read again for every pass.
#include "common.h"

CWM_DEFINE_ERROR_API

#define NSUM_MAX 4

struct NsumAddend {
  const void* ptr;
  const float* weight;  // [dim]
  long ld;              // elements between rows
  long partial_stride;  // elements between partial sums
  int n_partials;
  int dtype;
  float scale;
  const int* row_index;  // [T][n_partials]: the rows of a weighted sum; null for the other two kinds
  const float* row_weight;
};

struct NsumAddends {
  NsumAddend a[NSUM_MAX];
  int n;
  float eps;
};

extern "C" int cwm_normed_sum_max_addends() { return NSUM_MAX; }

__device__ __forceinline__ void nsum_load4(const void* p, int dtype, size_t e, float (&v)[4]) {
  if (dtype == CWM_F32) {
    const float4 x = *(const float4*)((const float*)p + e);
    v[0] = x.x, v[1] = x.y, v[2] = x.z, v[3] = x.w;
  } else {
    const uint2 x = *(const uint2*)((const bf16_t*)p + e);
    v[0] = __uint_as_float(x.x << 16), v[1] = __uint_as_float(x.x & 0xffff0000u);
    v[2] = __uint_as_float(x.y << 16), v[3] = __uint_as_float(x.y & 0xffff0000u);
  }
}

__device__ __forceinline__ float nsum_value(const NsumAddend& ad, size_t t, int e) {
  float y = 0.f;
  if (ad.row_index) {
    for (int k = 0; k < ad.n_partials; ++k) {
      const int row = ad.row_index[t * ad.n_partials + k];
      if (row >= 0) y += ad.row_weight[t * ad.n_partials + k] * ((const float*)ad.ptr)[(size_t)row * ad.ld + e];
    }
    return y;
  }
  for (int p = 0; p < ad.n_partials; ++p) {
    const size_t at = (size_t)p * ad.partial_stride + t * ad.ld + e;
    y += ad.dtype == CWM_F32 ? ((const float*)ad.ptr)[at] : bf16_to_f32(((const bf16_t*)ad.ptr)[at]);
  }
  return y;
}

// the sums of N values over the block, in a fixed order; `scratch` holds N * 16 floats
template <int N>
__device__ __forceinline__ void block_sums(float (&v)[N], float* scratch) {
  const int lane = threadIdx.x & (CWM_WAVE - 1), wave = threadIdx.x / CWM_WAVE, waves = blockDim.x / CWM_WAVE;
#pragma unroll
  for (int a = 0; a < N; ++a) v[a] = wave_sum(v[a]);
  __syncthreads();
  if (lane == 0)
#pragma unroll
    for (int a = 0; a < N; ++a) scratch[16 * a + wave] = v[a];
  __syncthreads();
#pragma unroll
  for (int a = 0; a < N; ++a) {
    float total = 0.f;
    for (int w = 0; w < waves; ++w) total += scratch[16 * a + w];
    v[a] = total;
  }
}

template <typename TO, int N, int CHUNKS>
__global__ void normed_sum_regs_kernel(float* __restrict__ h, NsumAddends ad, const float* __restrict__ weight, TO* __restrict__ out,
                                       const int* __restrict__ rows, int dim, float eps) {
  __shared__ float scratch[16 * N];
  const int r = blockIdx.x;
  const size_t t = rows ? (size_t)rows[r] : (size_t)r;
  const int n_chunks = dim >> 2;
  float* hrow = h + t * dim;
  float x[CHUNKS][4], y[N][CHUNKS][4];
  float sq[N];
#pragma unroll
  for (int c = 0; c < CHUNKS; ++c) {
    const int chunk = threadIdx.x + c * blockDim.x;
#pragma unroll
    for (int i = 0; i < 4; ++i) x[c][i] = 0.f;
    if (chunk < n_chunks) nsum_load4(hrow, CWM_F32, 4 * chunk, x[c]);
#pragma unroll
    for (int a = 0; a < N; ++a) {
#pragma unroll
      for (int i = 0; i < 4; ++i) y[a][c][i] = 0.f;
      if (chunk < n_chunks) {
        if (ad.a[a].row_index) {
          // four rows in flight at a time; what lies past the last, or names no row, is some row times zero
          const int top = ad.a[a].n_partials;
          for (int k = 0; k < top; k += 4) {
            float z[4][4], keep[4];
#pragma unroll
            for (int u = 0; u < 4; ++u) {
              const size_t at = t * top + min(k + u, top - 1);
              const int row = ad.a[a].row_index[at];
              keep[u] = k + u < top && row >= 0 ? ad.a[a].row_weight[at] : 0.f;
              nsum_load4(ad.a[a].ptr, CWM_F32, (size_t)max(row, 0) * ad.a[a].ld + 4 * chunk, z[u]);
              if (keep[u] == 0.f) z[u][0] = z[u][1] = z[u][2] = z[u][3] = 0.f;
            }
#pragma unroll
            for (int u = 0; u < 4; ++u)
#pragma unroll
              for (int i = 0; i < 4; ++i) y[a][c][i] = fmaf(keep[u], z[u][i], y[a][c][i]);
          }
        } else if (ad.a[a].n_partials == 1) {
          nsum_load4(ad.a[a].ptr, ad.a[a].dtype, t * ad.a[a].ld + 4 * chunk, y[a][c]);
        } else {
          // four partial sums in flight at a time; what lies past the last is the last again, times zero
          for (int p = 0; p < ad.a[a].n_partials; p += 4) {
            float z[4][4];
#pragma unroll
            for (int u = 0; u < 4; ++u)
              nsum_load4(ad.a[a].ptr, CWM_F32, (size_t)min(p + u, ad.a[a].n_partials - 1) * ad.a[a].partial_stride + t * ad.a[a].ld + 4 * chunk, z[u]);
#pragma unroll
            for (int u = 0; u < 4; ++u) {
              const float keep = p + u < ad.a[a].n_partials ? 1.0f : 0.0f;
#pragma unroll
              for (int i = 0; i < 4; ++i) y[a][c][i] = fmaf(keep, z[u][i], y[a][c][i]);
            }
          }
        }
      }
    }
  }
#pragma unroll
  for (int a = 0; a < N; ++a) {
    sq[a] = 0.f;
#pragma unroll
    for (int c = 0; c < CHUNKS; ++c) sq[a] += (y[a][c][0] * y[a][c][0] + y[a][c][1] * y[a][c][1]) + (y[a][c][2] * y[a][c][2] + y[a][c][3] * y[a][c][3]);
  }
  block_sums<N>(sq, scratch);
  float ss[1] = {0.f};
#pragma unroll
  for (int c = 0; c < CHUNKS; ++c) {
    const int chunk = threadIdx.x + c * blockDim.x;
    if (chunk < n_chunks) {
#pragma unroll
      for (int a = 0; a < N; ++a) {
        const float f = ad.a[a].scale / sqrtf(sq[a] / (float)dim + ad.eps);
        const float4 w = *(const float4*)(ad.a[a].weight + 4 * chunk);
        x[c][0] = fmaf(y[a][c][0] * f, w.x, x[c][0]), x[c][1] = fmaf(y[a][c][1] * f, w.y, x[c][1]);
        x[c][2] = fmaf(y[a][c][2] * f, w.z, x[c][2]), x[c][3] = fmaf(y[a][c][3] * f, w.w, x[c][3]);
      }
      if (!rows) *(float4*)(hrow + 4 * chunk) = make_float4(x[c][0], x[c][1], x[c][2], x[c][3]);
      ss[0] += (x[c][0] * x[c][0] + x[c][1] * x[c][1]) + (x[c][2] * x[c][2] + x[c][3] * x[c][3]);
    }
  }
  block_sums<1>(ss, scratch);
  const float rstd = 1.0f / sqrtf(ss[0] / (float)dim + eps);
  TO* orow = out + (size_t)r * dim;
#pragma unroll
  for (int c = 0; c < CHUNKS; ++c) {
    const int chunk = threadIdx.x + c * blockDim.x;
    if (chunk < n_chunks) {
      const float4 w = *(const float4*)(weight + 4 * chunk);
      const float o[4] = {x[c][0] * rstd * w.x, x[c][1] * rstd * w.y, x[c][2] * rstd * w.z, x[c][3] * rstd * w.w};
      if constexpr (sizeof(TO) == 4) {
        *(float4*)(orow + 4 * chunk) = make_float4(o[0], o[1], o[2], o[3]);
      } else {
        uint2 v;
        v.x = pack2_bf16(o[0], o[1]);
        v.y = pack2_bf16(o[2], o[3]);
        *(uint2*)(orow + 4 * chunk) = v;
      }
    }
  }
}

template <typename TO>
__global__ void normed_sum_kernel(float* __restrict__ h, NsumAddends ad, const float* __restrict__ weight, TO* __restrict__ out,
                                  const int* __restrict__ rows, int dim, float eps) {
  __shared__ float scratch[16 * NSUM_MAX];
  const int r = blockIdx.x;
  const size_t t = rows ? (size_t)rows[r] : (size_t)r;
  float* hrow = h + t * dim;
  float sq[NSUM_MAX];
#pragma unroll
  for (int a = 0; a < NSUM_MAX; ++a) {
    sq[a] = 0.f;
    if (a < ad.n)
      for (int e = threadIdx.x; e < dim; e += blockDim.x) {
        const float y = nsum_value(ad.a[a], t, e);
        sq[a] += y * y;
      }
  }
  block_sums<NSUM_MAX>(sq, scratch);
#pragma unroll
  for (int a = 0; a < NSUM_MAX; ++a) sq[a] = a < ad.n ? ad.a[a].scale / sqrtf(sq[a] / (float)dim + ad.eps) : 0.f;
  auto summed = [&](int e) {
    float x = hrow[e];
#pragma unroll
    for (int a = 0; a < NSUM_MAX; ++a)
      if (a < ad.n) x = fmaf(nsum_value(ad.a[a], t, e) * sq[a], ad.a[a].weight[e], x);
    return x;
  };
  float ss[1] = {0.f};
  for (int e = threadIdx.x; e < dim; e += blockDim.x) {
    const float x = summed(e);
    if (!rows) hrow[e] = x;
    ss[0] += x * x;
  }
  block_sums<1>(ss, scratch);
  const float rstd = 1.0f / sqrtf(ss[0] / (float)dim + eps);
  // the thread that wrote an element of the residual is the one that reads it back
  for (int e = threadIdx.x; e < dim; e += blockDim.x) Elem<TO>::store(out + (size_t)r * dim + e, (rows ? summed(e) : hrow[e]) * rstd * weight[e]);
}

// row_index[a], row_weight[a]: null, or the addend is a weighted sum of rows of ptrs[a] (float32), n_partials[a] of them a token.
// h: float32 [T, dim], changed in place unless `rows` chooses rows.  Addend a: ptrs[a] of dtypes[a], rows lds[a] elements
// apart, n_partials[a] slabs partial_strides[a] elements apart, normalised with `addend_eps`, times weights[a] (float32
// [dim]) and scales[a].  weight: float32 [dim]; out: [n_out, dim] of out_dtype.
extern "C" int cwm_normed_sum(float* h, int n_addends, const void* const* ptrs, const int* dtypes, const long* lds,
                              const int* n_partials, const long* partial_strides, const float* scales, const void* const* weights,
                              const void* const* row_index, const void* const* row_weight, float addend_eps, const float* weight,
                              float eps, void* out, int out_dtype, const int* rows,
                              int n_out, int dim, hipStream_t stream) {
  CWM_REQUIRE(n_out >= 0 && dim >= 1, "normed_sum: bad sizes");
  CWM_REQUIRE(n_addends >= 1 && n_addends <= NSUM_MAX, "normed_sum: %d addends are outside 1..%d", n_addends, NSUM_MAX);
  CWM_REQUIRE(h && weight && out, "normed_sum: arguments missing");
  CWM_REQUIRE(eps > 0.f && addend_eps > 0.f, "normed_sum: eps must be positive");
  if (n_out == 0) return 0;
  NsumAddends ad;
  ad.n = n_addends;
  ad.eps = addend_eps;
  const int out_bytes = out_dtype == CWM_F32 ? 4 : 2;
  bool vec = dim % 4 == 0 && ((uintptr_t)h % 16) == 0 && ((uintptr_t)weight % 16) == 0 && ((uintptr_t)out % (4 * out_bytes)) == 0;
  for (int a = 0; a < n_addends; ++a) {
    CWM_REQUIRE(ptrs[a] && weights[a] && n_partials[a] >= 1, "normed_sum: addend %d is empty", a);
    CWM_REQUIRE(n_partials[a] == 1 || dtypes[a] == CWM_F32, "normed_sum: partial sums must be float32");
    ad.a[a] = NsumAddend{ptrs[a], (const float*)weights[a], lds[a], partial_strides[a], n_partials[a], dtypes[a], scales[a],
                         (const int*)row_index[a], (const float*)row_weight[a]};
    CWM_REQUIRE((row_index[a] == nullptr) == (row_weight[a] == nullptr) && (!row_index[a] || dtypes[a] == CWM_F32),
                "normed_sum: a weighted sum of rows has indices, weights and float32 rows");
    const int bytes = dtypes[a] == CWM_F32 ? 4 : 2;
    vec = vec && lds[a] % 4 == 0 && partial_strides[a] % 4 == 0 && ((uintptr_t)ptrs[a] % (4 * bytes)) == 0 && ((uintptr_t)weights[a] % 16) == 0;
  }
  const int n_chunks = dim / 4;
  int threads = 64;
  while (threads < 512 && threads * 2 < n_chunks) threads *= 2;
  const int chunks = (n_chunks + threads - 1) / threads;
#define CWM_NSUM_REGS(TO, N, C) \
  hipLaunchKernelGGL((normed_sum_regs_kernel<TO, N, C>), dim3(n_out), dim3(threads), 0, stream, h, ad, weight, (TO*)out, rows, dim, eps)
#define CWM_NSUM_N(TO, N)                              \
  do {                                                 \
    if (chunks <= 1) CWM_NSUM_REGS(TO, N, 1);          \
    else if (chunks <= 2) CWM_NSUM_REGS(TO, N, 2);     \
    else CWM_NSUM_REGS(TO, N, 4);                      \
  } while (0)
#define CWM_NSUM(TO)                                                                                                        \
  do {                                                                                                                      \
    if (vec && chunks <= 4 && n_addends == 1) CWM_NSUM_N(TO, 1);                                                             \
    else if (vec && chunks <= 4 && n_addends == 2) CWM_NSUM_N(TO, 2);                                                        \
    else hipLaunchKernelGGL((normed_sum_kernel<TO>), dim3(n_out), dim3(256), 0, stream, h, ad, weight, (TO*)out, rows, dim, eps); \
  } while (0)
  if (out_dtype == CWM_F32) CWM_NSUM(float);
  else if (out_dtype == CWM_BF16) CWM_NSUM(bf16_t);
  else return cwm_fail("normed_sum: unknown output type %d", out_dtype);
#undef CWM_NSUM
#undef CWM_NSUM_N
#undef CWM_NSUM_REGS
  return cwm_launch_status("normed_sum");
}
