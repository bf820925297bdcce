// What attention through a cached latent makes of its projections, in one pass over a token's row:
//
//   cached row   [ rot(k') | c | 0 ]    c = rms(c') * w over `rank` elements (eps inside the root), k' the `lead` rotated
//                                       elements that all heads share, zeros up to `row` elements; written as the token's
//                                       key and as its value into the paged cache (one key/value head of size `row`)
//   queries      ask[t][h][0 .. lead)   = rot(r_h), the rotated part of head h; the rest of ask[t][h] is filled by the product
//                                       of the head's unrotated part with its own matrix
//                rest[t][h][0 .. n)     = the unrotated part, where the caller wants it (partial sums have to be added
//                                       somewhere; a plain projection is read by the product where it lies)
//
// Sources: rows [k' | c'] and rows of heads [r_h | n_h], each [T][stride] of type TS or float32 partial sums of a split K
// that are added in order; they may be parts of one joined product.  Rotation of adjacent pairs by position *
// inv_freq[pair] (a frequency of 0 leaves its pair alone).  float32 arithmetic.  The blocks of a token (gridDim.y of
// them) share its heads; the first one also makes the cached row.  Cache layout: top of rope_kv.hip.
#include "common.h"

CWM_DEFINE_ERROR_API

#define LATENT_MAX_ROW 1024
#define LATENT_THREADS 256

template <typename TS, typename TO>
__global__ void __launch_bounds__(LATENT_THREADS)
latent_rows_kernel(const TS* __restrict__ q_src, long q_stride, int q_partials, long q_partial_stride, const TS* __restrict__ kv_src,
                   long kv_stride, int kv_partials, long kv_partial_stride, const float* __restrict__ weight, float eps,
                   const int* __restrict__ positions, const int* __restrict__ seq_of_token, const float* __restrict__ inv_freq,
                   TO* __restrict__ ask, TO* __restrict__ rest, TO* __restrict__ cache, const int* __restrict__ block_table,
                   int table_width, int page_size, int num_pages, int n_heads, int lead, int n_rest, int rank, int row) {
  __shared__ float scratch[16];
  __shared__ float cs[LATENT_MAX_ROW];  // cos, sin of each pair of the leading elements
  const int t = blockIdx.x;
  const int pos = positions[t];
  for (int i = threadIdx.x; 2 * i < lead; i += blockDim.x) {
    float c = 1.f, s = 0.f;
    const float f = inv_freq ? inv_freq[i] : 0.f;
    if (f != 0.f) sincos_turn(pos, f, &s, &c);
    cs[2 * i] = c;
    cs[2 * i + 1] = s;
  }
  __syncthreads();
  if (kv_src && blockIdx.y == 0) {
    const TS* src = kv_src + (size_t)t * kv_stride;
    auto value = [&](int e) {
      float v = 0.f;
      for (int p = 0; p < kv_partials; ++p) v += Elem<TS>::load(src + (size_t)p * kv_partial_stride + e);
      return v;
    };
    float ss = 0.f;
    for (int e = threadIdx.x; e < rank; e += blockDim.x) {
      const float v = value(lead + e);
      ss += v * v;
    }
    const float rstd = 1.0f / sqrtf(block_sum(ss, scratch) / (float)rank + eps);
    const int lp = pos / page_size;
    const int slot = pos - lp * page_size;
    const int page = lp < table_width ? block_table[(size_t)seq_of_token[t] * table_width + lp] : -1;
    if (page >= 0 && page < num_pages) {
      const size_t plane = (size_t)page_size * row;
      const int v_block = (page_size % 8 == 0) ? 8 : page_size;
      TO* kdst = cache + (size_t)page * 2 * plane + (size_t)slot * row;
      TO* vdst = cache + (size_t)page * 2 * plane + plane + (size_t)(slot / v_block) * row * v_block + slot % v_block;
      for (int e = threadIdx.x; e < row; e += blockDim.x) {
        float v = 0.f;
        if (e < lead) {
          const float re = value(e & ~1), im = value(e | 1);
          const float c = cs[e & ~1], s = cs[e | 1];
          v = (e & 1) ? im * c + re * s : re * c - im * s;
        } else if (e < lead + rank) {
          v = value(e) * rstd * weight[e - lead];
        }
        Elem<TO>::store(kdst + e, v);
        Elem<TO>::store(vdst + (size_t)e * v_block, v);
      }
    }
  }
  // the heads: pairs of the rotated part, then (where it is wanted) the unrotated part
  const TS* src = q_src + (size_t)t * q_stride;
  const int width = lead + n_rest;
  auto value = [&](int e) {
    float v = 0.f;
    for (int p = 0; p < q_partials; ++p) v += Elem<TS>::load(src + (size_t)p * q_partial_stride + e);
    return v;
  };
  const int first = blockIdx.y * blockDim.x + threadIdx.x, step = gridDim.y * blockDim.x;
  const int half = lead / 2;
  for (int e = first; e < n_heads * half; e += step) {
    const int h = e / half, i = e - h * half;
    const float re = value(h * width + 2 * i), im = value(h * width + 2 * i + 1);
    const float c = cs[2 * i], s = cs[2 * i + 1];
    TO* dst = ask + ((size_t)t * n_heads + h) * row + 2 * i;
    Elem<TO>::store(dst, re * c - im * s);
    Elem<TO>::store(dst + 1, im * c + re * s);
  }
  if (rest)
    for (int e = first; e < n_heads * n_rest; e += step) {
      const int h = e / n_rest, d = e - h * n_rest;
      Elem<TO>::store(rest + (size_t)t * n_heads * n_rest + e, value(h * width + lead + d));
    }
}

// q_src: rows of n_heads * (lead + n_rest) elements of src_dtype, q_stride apart (or q_partials float32 slabs).  kv_src:
// rows of lead + rank elements, or null where another layer has written the cache; weight: float32 [rank].  ask:
// [T][n_heads][row]; rest: [T][n_heads][n_rest] or null.  cache: [pages][2][page_size * row].
extern "C" int cwm_latent_rows(const void* q_src, long q_stride, int q_partials, long q_partial_stride, const void* kv_src, long kv_stride,
                               int kv_partials, long kv_partial_stride, int src_dtype, const float* weight, float eps, const int* positions,
                               const int* seq_of_token, const float* inv_freq, void* ask, void* rest, int out_dtype, void* cache,
                               const int* block_table, int table_width, int page_size, int num_pages, int n_tokens, int n_heads, int lead,
                               int n_rest, int rank, int row, hipStream_t stream) {
  CWM_REQUIRE(n_tokens >= 0 && n_heads >= 1 && lead >= 0 && lead % 2 == 0 && n_rest >= 1 && rank >= 1, "latent_rows: bad sizes");
  CWM_REQUIRE(row >= lead + rank && row <= LATENT_MAX_ROW, "latent_rows: a cached row of %d elements does not hold %d + %d, or is more than %d", row,
              lead, rank, LATENT_MAX_ROW);
  CWM_REQUIRE(q_src && ask && positions && q_partials >= 1 && kv_partials >= 1, "latent_rows: arguments missing");
  CWM_REQUIRE((q_partials == 1 && kv_partials == 1) || src_dtype == CWM_F32, "latent_rows: partial sums must be float32");
  if (kv_src) {
    CWM_REQUIRE(weight && cache && block_table && seq_of_token && eps > 0.f, "latent_rows: a cached row needs its norm and a block table");
    CWM_REQUIRE(page_size > 0 && num_pages > 0 && table_width > 0, "latent_rows: bad cache geometry");
  }
  if (n_tokens == 0) return 0;
  // few tokens: several blocks a token, so that a decode step's rows are not left to as many blocks
  const int per_token = (n_heads * (rest ? lead / 2 + n_rest : lead / 2) + LATENT_THREADS - 1) / LATENT_THREADS;
  const int gy = n_tokens >= 512 ? 1 : (per_token < 1 ? 1 : (per_token > 16 ? 16 : per_token));
#define CWM_LATENT(TS, TO)                                                                                                            \
  hipLaunchKernelGGL((latent_rows_kernel<TS, TO>), dim3(n_tokens, gy), dim3(LATENT_THREADS), 0, stream, (const TS*)q_src, q_stride,    \
                     q_partials, q_partial_stride, (const TS*)kv_src, kv_stride, kv_partials, kv_partial_stride, weight, eps,          \
                     positions, seq_of_token, inv_freq, (TO*)ask, (TO*)rest, (TO*)cache, block_table, table_width, page_size,          \
                     num_pages, n_heads, lead, n_rest, rank, row)
  switch ((src_dtype << 1) | out_dtype) {
    case 0: CWM_LATENT(float, float); break;
    case 1: CWM_LATENT(float, bf16_t); break;
    case 3: CWM_LATENT(bf16_t, bf16_t); break;
    default: return cwm_fail("latent_rows: source type %d with cache type %d is not built", src_dtype, out_dtype);
  }
#undef CWM_LATENT
  return cwm_launch_status("latent_rows");
}
