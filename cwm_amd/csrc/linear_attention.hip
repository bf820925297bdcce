// Linear attention with a matrix state per head that decays channel by channel, in two forms (KIND).
//
// KIND_GLA, gated linear attention:
//   alpha_t = sigmoid(z_t)^(1 / tau)                     one decay a key channel (z: float32 logits, heads x dim)
//   S_t     = diag(alpha_t) S_(t-1) + k_t v_t^T          S: dim x vdim, float32, carried from token to token
//   o_t     = S_t^T (q_scale q_t)
//   out_t   = o_t / sqrt(mean(o_t^2) + eps) * w * silu(g_t)     per head over vdim; w of vdim values for all heads
// KIND_WKV, the current token's value counted with a weight of its own instead of from the state:
//   alpha_t = exp(-exp(z_t))
//   o_t     = S_(t-1)^T q_t + (sum_d q_t[d] u[d] k_t[d]) v_t        u: one weight a key channel (the bonus)
//   S_t     = diag(alpha_t) S_(t-1) + k_t v_t^T
//   out_t   as above, with a weight of heads x vdim values
//
// Three ways through a step's tokens:
//
// `gla_walk_kernel`, MODE 0: a block a (tile of value columns, head, sequence) walks the sequence's tokens one by one,
// from the state that the step before left in the sequence's slot, and leaves the new state there.  A thread holds up
// to 32 rows of one column of S in registers; `split` neighbouring lanes share a column (a run of consecutive rows each,
// a multiple of four, read from LDS sixteen bytes at a time) and add their parts of o_t by shuffles.  q, k, the decays
// and v of 16 (or 8) tokens are staged in LDS at a time, in float32, the decays computed once a (token, channel).  The
// same tokens give the same bits however they are cut into steps.  The state of a (head, tile) lies in memory in the
// order its threads hold it (row r of thread i at [r][i]), so it is read and written in whole lines.
//
// Segments side by side: a step with long portions cuts them into segments and runs three launches: every segment but a
// sequence's last from a zero state, leaving its own sum and the product of its decays (MODE 1); `gla_carry_kernel`,
// which carries the states across a sequence's segments, start_(s+1) = decay_s * start_s + sum_s; and every segment from
// its true start with its results (MODE 2).  That differs from the walk by float32 rounding only.
//
// `gla_block_kernel` is MODE 1 and MODE 2 on the matrix cores (float32 operands and sums), 16 tokens at a time: with
// w the decays, P_t their products from the block's first token to t, and Q_s those after s to the block's last,
//   o_t  = (q_t P)^T S + sum_(s <= t) a_ts v_s,     a_ts = sum_d q_t[d] k_s[d] w_(s+1)[d] .. w_t[d]
//   S   <- diag(w_1 .. w_16) S + sum_s (k_s Q_s) v_s^T
// (KIND_WKV: products up to t - 1, and a_tt = sum_d q_t u k_t).  Every factor is a product of decays, at most one: no
// logarithm and no quotient of decays, which might overflow, is formed.  The state stays in the accumulators of the matrix
// instruction (16 columns a wavefront, or 32), in the order that makes it the next product's operand as it is.
// `gla_walk_kernel` has these two modes as well, for heads of more than GLA_BLOCK_DIM rows.
//
// The norm of every head's o_t, its weight and the gate are done where a block holds a head's columns of a token together;
// else by `gla_out_kernel`, a wavefront a (token, head).
#include "common.h"

CWM_DEFINE_ERROR_API

#define GLA_THREADS 256
#define GLA_ROWS 32        // rows of a column that one thread holds at most
#define GLA_MAX_DIM 256    // = GLA_ROWS * 8 lanes a column
#define GLA_CHUNK 16       // tokens staged at a time (8 where the rows are long)

extern "C" int cwm_gla_max_dim() { return GLA_MAX_DIM; }

#define GLA_BLOCK_DIM 128  // rows of a head that gla_block_kernel takes at most

extern "C" int cwm_gla_block_dim() { return GLA_BLOCK_DIM; }

// lanes that share a column of the state: the fewest (1, 2, 4, 8) that leave a lane at most GLA_ROWS rows, and more of
// them where a block would otherwise have twice the columns that a head has
static inline int gla_split(int dim, int vdim) {
  int split = 1;
  while (split < 8 && ((dim + split - 1) / split > GLA_ROWS || GLA_THREADS / split / 2 >= vdim)) split *= 2;
  return split;
}
// rows of a column that a lane holds: a multiple of 4
__host__ __device__ static inline int gla_rows(int dim, int split) { return ((dim + split - 1) / split + 3) / 4 * 4; }
extern "C" int cwm_gla_split(int dim, int vdim) { return gla_split(dim, vdim); }
// float32 elements of a request's state
extern "C" long cwm_gla_state_elems(int heads, int dim, int vdim) {
  const int split = gla_split(dim, vdim), rows = gla_rows(dim, split), cols = GLA_THREADS / split;
  return (long)heads * ((vdim + cols - 1) / cols) * rows * GLA_THREADS;
}

#define KIND_GLA 0
#define KIND_WKV 1

// One head's results of one token by one wavefront: o over its root mean square, times weight, times silu(gate).
template <typename T>
__device__ __forceinline__ void gla_finish(const float* o, const T* __restrict__ gate, const float* __restrict__ weight,
                                           T* __restrict__ out, int vdim, float eps) {
  const int lane = threadIdx.x & (CWM_WAVE - 1);
  float sq = 0.f;
  for (int e = lane; e < vdim; e += CWM_WAVE) sq += o[e] * o[e];
  const float rstd = 1.0f / sqrtf(wave_sum(sq) / (float)vdim + eps);
  for (int e = lane; e < vdim; e += CWM_WAVE) {
    const float g = Elem<T>::load(gate + e);
    Elem<T>::store(out + e, o[e] * rstd * weight[e] * (g / (1.0f + expf(-g))));
  }
}

template <int KIND>
__device__ __forceinline__ float gla_decay(float z, float inv_tau) {
  if constexpr (KIND == KIND_WKV) return expf(-expf(z));
  // sigmoid(z)^(1 / tau) = exp(-softplus(-z) / tau), with softplus(x) = max(x, 0) + log1p(exp(-|x|))
  const float sp = fmaxf(-z, 0.f) + log1pf(expf(-fabsf(z)));
  return expf(-sp * inv_tau);
}

// segments: int32 [n][6]: sequence, first token, end token, number of the segment in its sequence, the sequence's first
// entry of the scratch states, segments of the sequence.
// MODE 0: a block a (tile, head, sequence) walks the sequence's tokens from the state in its slot and leaves the new one.
// MODE 1: a block a (tile, head, segment) walks from zero without results and leaves the segment's sum and decay product.
// MODE 2: a block a (tile, head, segment) walks from seg_start with results; a sequence's last segment writes the slot.
template <typename T, int MODE, int KIND>
__global__ void __launch_bounds__(GLA_THREADS)
gla_walk_kernel(const T* __restrict__ q, const T* __restrict__ k, const T* __restrict__ v_in, const T* __restrict__ gate,
                long proj_ld, const float* __restrict__ weight, int weight_stride, T* __restrict__ out, float eps,
                const float* __restrict__ bonus, const float* __restrict__ z, long z_ld, float* __restrict__ o_raw,
                float* __restrict__ state, long state_ld, const int* __restrict__ slots, const int* __restrict__ cu_q,
                int n_slots, int heads, int dim, int vdim, int split, int chunk, float inv_tau, float q_scale,
                const int* __restrict__ segments, float* __restrict__ seg_local, float* __restrict__ seg_decay,
                const float* __restrict__ seg_start, long seg_ld) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int vt = blockIdx.x, h = blockIdx.y;
  const int cols = GLA_THREADS / split, rows = gla_rows(dim, split), dpad = split * rows;
  const int col = threadIdx.x / split, part = threadIdx.x % split;
  const int e = vt * cols + col;  // this thread's value column
  const bool live = e < vdim;
  float* qs = lds;                  // [chunk][dpad]: rows beyond dim hold zeros (a zero key and query leave their rows of S at zero)
  float* ks = qs + chunk * dpad;    // [chunk][dpad]
  float* as = ks + chunk * dpad;    // [chunk][dpad]
  float* vs = as + chunk * dpad;    // [chunk][cols]
  float* cs = vs + chunk * cols;    // [chunk]: the share of a token's own value (KIND_WKV)
  float* os = cs + chunk;           // [chunk][cols]: the results, where one tile holds all of a head's columns
  int b, t0, t1, seg = 0;
  bool last = true;
  if constexpr (MODE == 0) {
    b = blockIdx.z, t0 = cu_q[b], t1 = cu_q[b + 1];
  } else {
    const int* sg = segments + 6 * blockIdx.z;
    b = sg[0], t0 = sg[1], t1 = sg[2], seg = sg[4] + sg[3], last = sg[3] == sg[5] - 1;
    if (MODE == 1 && last) return;  // nothing comes after it
  }
  const int slot = slots[b];
  if (slot < 0 || slot >= n_slots) return;
  const int n_vt = gridDim.x;
  const size_t tile_at = ((size_t)h * n_vt + vt) * rows * GLA_THREADS + threadIdx.x;
  float* st = state + (size_t)slot * state_ld + tile_at;
  float S[GLA_ROWS];
  float P[MODE == 1 ? GLA_ROWS : 1];
#pragma unroll
  for (int r = 0; r < GLA_ROWS; ++r) {
    if constexpr (MODE == 0) S[r] = r < rows ? st[(size_t)r * GLA_THREADS] : 0.f;
    if constexpr (MODE == 1) S[r] = 0.f, P[r] = 1.f;
    if constexpr (MODE == 2) S[r] = r < rows ? seg_start[(size_t)seg * seg_ld + tile_at + (size_t)r * GLA_THREADS] : 0.f;
  }
  for (int c0 = t0; c0 < t1; c0 += chunk) {
    const int n = min(chunk, t1 - c0);
    __syncthreads();  // the chunk before has been walked
    for (int i = threadIdx.x; i < n * dpad; i += GLA_THREADS) {
      const int tt = i / dpad, d = i - tt * dpad;
      const size_t at = (size_t)(c0 + tt) * proj_ld + h * dim + d;
      const bool real = d < dim;
      if constexpr (MODE != 1) qs[i] = real ? Elem<T>::load(q + at) * q_scale : 0.f;
      ks[i] = real ? Elem<T>::load(k + at) : 0.f;
      as[i] = real ? gla_decay<KIND>(z[(size_t)(c0 + tt) * z_ld + h * dim + d], inv_tau) : 0.f;
    }
    for (int i = threadIdx.x; i < n * cols; i += GLA_THREADS) {
      const int tt = i / cols, cc = i - tt * cols;
      const int ee = vt * cols + cc;
      vs[i] = ee < vdim ? Elem<T>::load(v_in + (size_t)(c0 + tt) * proj_ld + h * vdim + ee) : 0.f;
    }
    __syncthreads();
    if constexpr (KIND == KIND_WKV && MODE != 1) {  // 16 lanes a token
      const int tt = threadIdx.x >> 4;
      float c = 0.f;
      if (tt < n)
        for (int d = threadIdx.x & 15; d < dim; d += 16) c = fmaf(qs[tt * dpad + d] * ks[tt * dpad + d], bonus[h * dim + d], c);
#pragma unroll
      for (int off = 1; off < 16; off *= 2) c += __shfl_xor(c, off, CWM_WAVE);
      if ((threadIdx.x & 15) == 0 && tt < n) cs[tt] = c;
      __syncthreads();
    }
    for (int tt = 0; tt < n; ++tt) {
      const float v = vs[tt * cols + col];
      const float* qrow = qs + tt * dpad;
      const float* krow = ks + tt * dpad;
      const float* arow = as + tt * dpad;
      float o = (KIND == KIND_WKV && MODE != 1 && part == 0) ? cs[tt] * v : 0.f;
      const int d0 = part * rows;  // this lane's rows: d0 .. d0 + rows - 1 (rows is a multiple of 4; LDS rows are padded to it)
#pragma unroll
      for (int r = 0; r < GLA_ROWS; r += 4) {
        if (r < rows) {
          const float4 a4 = *(const float4*)(arow + d0 + r);
          const float4 k4 = *(const float4*)(krow + d0 + r);
          if constexpr (KIND == KIND_WKV && MODE != 1) {  // from the state before this token
            const float4 q4 = *(const float4*)(qrow + d0 + r);
            o = fmaf(S[r], q4.x, o), o = fmaf(S[r + 1], q4.y, o), o = fmaf(S[r + 2], q4.z, o), o = fmaf(S[r + 3], q4.w, o);
          }
          S[r] = fmaf(a4.x, S[r], k4.x * v), S[r + 1] = fmaf(a4.y, S[r + 1], k4.y * v);
          S[r + 2] = fmaf(a4.z, S[r + 2], k4.z * v), S[r + 3] = fmaf(a4.w, S[r + 3], k4.w * v);
          if constexpr (MODE == 1) P[r] *= a4.x, P[r + 1] *= a4.y, P[r + 2] *= a4.z, P[r + 3] *= a4.w;
          if constexpr (KIND == KIND_GLA && MODE != 1) {
            const float4 q4 = *(const float4*)(qrow + d0 + r);
            o = fmaf(S[r], q4.x, o), o = fmaf(S[r + 1], q4.y, o), o = fmaf(S[r + 2], q4.z, o), o = fmaf(S[r + 3], q4.w, o);
          }
        }
      }
      if constexpr (MODE != 1) {
        for (int off = 1; off < split; off *= 2) o += __shfl_xor(o, off, CWM_WAVE);
        if (part == 0 && live) {
          if (n_vt == 1)
            os[tt * cols + col] = o;
          else
            o_raw[(size_t)(c0 + tt) * heads * vdim + h * vdim + e] = o;
        }
      }
    }
    if constexpr (MODE != 1) {
      if (n_vt == 1) {
        __syncthreads();
        for (int tt = threadIdx.x / CWM_WAVE; tt < n; tt += GLA_THREADS / CWM_WAVE)
          gla_finish(os + tt * cols, gate + (size_t)(c0 + tt) * proj_ld + h * vdim, weight + h * weight_stride,
                     out + ((size_t)(c0 + tt) * heads + h) * vdim, vdim, eps);
      }
    }
  }
#pragma unroll
  for (int r = 0; r < GLA_ROWS; ++r) {
    if (r >= rows) continue;
    if constexpr (MODE == 1) {
      seg_local[(size_t)seg * seg_ld + tile_at + (size_t)r * GLA_THREADS] = S[r];
      if (vt == 0 && col == 0 && part * rows + r < dim) seg_decay[(size_t)seg * heads * dim + h * dim + part * rows + r] = P[r];
    } else {
      if (last) st[(size_t)r * GLA_THREADS] = S[r];
    }
  }
}

// sum over the 16 lanes of a row of the wavefront, in every one of them (row rotations of the vector unit's operands)
__device__ __forceinline__ float row16_sum(float x) {
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x128, 0xf, 0xf, false));  // row_ror:8
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x124, 0xf, 0xf, false));  // row_ror:4
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x122, 0xf, 0xf, false));  // row_ror:2
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x121, 0xf, 0xf, false));  // row_ror:1
  return x;
}

// four consecutive bfloat16 values of a row, zeros from `limit` on
__device__ __forceinline__ uint2 load4_bf16(const bf16_t* row, int at, int limit, bool vec) {
  uint2 x = make_uint2(0u, 0u);
  if (vec) {
    if (at < limit) x = *(const uint2*)(row + at);
  } else {
    uint32_t h[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) h[i] = at + i < limit ? row[at + i] : 0u;
    x.x = h[0] | (h[1] << 16), x.y = h[2] | (h[3] << 16);
  }
  return x;
}

__device__ __forceinline__ void unpack4_bf16(uint2 x, float (&v)[4]) {
  v[0] = __uint_as_float(x.x << 16), v[1] = __uint_as_float(x.x & 0xffff0000u);
  v[2] = __uint_as_float(x.y << 16), v[3] = __uint_as_float(x.y & 0xffff0000u);
}

// A block of four wavefronts a (64 * EC value columns, head, segment); wavefront w owns columns 16 EC w .. of them.
// CS: channels of a token that a thread stages (16 threads a token): heads of up to 16 CS rows.  `segments` as above.
// Matrix-core layout (v_mfma_f32_16x16x4_f32, lane = 16 g + m): A holds element [m][k = g], B [k = g][m], the result
// rows 4 g + i (i = 0 .. 3) of column m.  Which four of the summed-over indices an instruction takes as its k is free as
// long as A and B agree: with k = 4 g + i the accumulator register i of a tile of S is B as it stands.
template <int MODE, int KIND, int CS, int EC>
__global__ void __launch_bounds__(GLA_THREADS)
gla_block_kernel(const bf16_t* __restrict__ q, const bf16_t* __restrict__ k, const bf16_t* __restrict__ v,
                 const bf16_t* __restrict__ gate, long proj_ld, const float* __restrict__ bonus, const float* __restrict__ z,
                 long z_ld, const float* __restrict__ weight, int weight_stride, float eps, float* __restrict__ o_raw,
                 bf16_t* __restrict__ out, float* __restrict__ state, long state_ld, const int* __restrict__ slots, int n_slots,
                 int heads, int dim, int vdim, int split, float inv_tau, float q_scale, bool vec, const int* __restrict__ segments,
                 float* __restrict__ seg_local, float* __restrict__ seg_decay, const float* __restrict__ seg_start, long seg_ld) {
  constexpr int DP = 16 * CS, LD = DP + 4, DT = DP / 16, VC = 64 * EC, VLD = VC + 4;
  __shared__ __attribute__((aligned(16))) float Qs[MODE == 2 ? 16 : 1][LD], Ks[16][LD], Ws[16][LD];
  __shared__ __attribute__((aligned(16))) float Qp[MODE == 2 ? 16 : 1][LD], Kq[16][LD], dec[DP];
  __shared__ __attribute__((aligned(16))) float Vs[16][VLD], As[MODE == 2 ? 16 : 1][20];
  __shared__ float sq_part[MODE == 2 ? 4 : 1][16];
  const int tid = threadIdx.x, lane = tid & 63, m = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.y, e0 = blockIdx.x * VC;
  const bool whole_head = gridDim.x == 1;
  const int* sg = segments + 6 * blockIdx.z;
  const int b = sg[0], t0 = sg[1], t1 = sg[2], seg = sg[4] + sg[3];
  const bool last = sg[3] == sg[5] - 1, alone = sg[5] == 1;
  if (MODE == 1 && last) return;  // nothing comes after it
  const int slot = slots[b];
  if (slot < 0 || slot >= n_slots) return;

  // the state's place in memory (the walking kernel's order)
  const int cols = GLA_THREADS / split, rows = gla_rows(dim, split), n_vt = (vdim + cols - 1) / cols;
  auto state_at = [&](int d, int e) -> long {  // -1: a row or column that the state does not have
    if (d >= split * rows || e >= n_vt * cols) return -1;
    const int vt = e / cols, col = e - vt * cols, part = d / rows, r = d - part * rows;
    return (((long)h * n_vt + vt) * rows + r) * GLA_THREADS + col * split + part;
  };
  float* home = state + (size_t)slot * state_ld;
  float4v S[DT][EC];
#pragma unroll
  for (int dt = 0; dt < DT; ++dt)
#pragma unroll
    for (int ec = 0; ec < EC; ++ec)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        S[dt][ec][i] = 0.f;
        if constexpr (MODE == 2) {
          const long at = state_at(16 * dt + 4 * g + i, e0 + 16 * (EC * wave + ec) + m);
          if (at >= 0) S[dt][ec][i] = alone ? home[at] : seg_start[(size_t)seg * seg_ld + at];
        }
      }
  // the upper triangle of the block's scores is zero and stays so
  if constexpr (MODE == 2) As[tid >> 4][tid & 15] = 0.f;

  // staging: thread (token ts, slice sl) takes CS channels and 4 EC value columns of its token
  const int ts = tid >> 4, sl = tid & 15;
  uint2 rq[CS / 4], rk[CS / 4], rv[EC];
  float rz[CS];
  float u[CS];
#pragma unroll
  for (int i = 0; i < CS; ++i) u[i] = (KIND == KIND_WKV && MODE == 2 && sl * CS + i < dim) ? bonus[h * dim + sl * CS + i] : 1.f;
  auto fetch = [&](int c0) {
    const bool there = c0 + ts < t1;
    const size_t row = (size_t)(there ? c0 + ts : t0) * proj_ld;
    const float* zr = z + (size_t)(there ? c0 + ts : t0) * z_ld + h * dim;
#pragma unroll
    for (int i = 0; i < CS / 4; ++i) {
      const int c = sl * CS + 4 * i, limit = there ? dim : 0;
      if constexpr (MODE == 2) rq[i] = load4_bf16(q + row + h * dim, c, limit, vec);
      rk[i] = load4_bf16(k + row + h * dim, c, limit, vec);
#pragma unroll
      for (int x = 0; x < 4; ++x) rz[4 * i + x] = c + x < limit ? zr[c + x] : 0.f;
    }
#pragma unroll
    for (int i = 0; i < EC; ++i) rv[i] = load4_bf16(v + row + h * vdim, e0 + 4 * (EC * sl + i), there ? vdim : 0, vec);
  };
  float product = 1.f;  // MODE 1: of the segment's decays, in the thread that forms a channel's products
  fetch(t0);
  for (int c0 = t0; c0 < t1; c0 += 16) {
    const int n = min(16, t1 - c0);
    __syncthreads();  // the block of tokens before is done with
#pragma unroll
    for (int i = 0; i < CS / 4; ++i) {
      float kk[4], ww[4];
      const int c = sl * CS + 4 * i;
      unpack4_bf16(rk[i], kk);
#pragma unroll
      for (int x = 0; x < 4; ++x) ww[x] = (ts < n && c + x < dim) ? gla_decay<KIND>(rz[4 * i + x], inv_tau) : 1.f;
      *(float4*)&Ks[ts][c] = make_float4(kk[0], kk[1], kk[2], kk[3]);
      *(float4*)&Ws[ts][c] = make_float4(ww[0], ww[1], ww[2], ww[3]);
      if constexpr (MODE == 2) {
        float qq[4];
        unpack4_bf16(rq[i], qq);
        *(float4*)&Qs[ts][c] = make_float4(qq[0] * q_scale, qq[1] * q_scale, qq[2] * q_scale, qq[3] * q_scale);
      }
    }
#pragma unroll
    for (int i = 0; i < EC; ++i) {
      float vv[4];
      unpack4_bf16(rv[i], vv);
      *(float4*)&Vs[ts][4 * (EC * sl + i)] = make_float4(vv[0], vv[1], vv[2], vv[3]);
    }
    __syncthreads();
    if (c0 + 16 < t1) fetch(c0 + 16);  // in flight while this block of tokens is worked on
    bf16_t gt[4][EC];
    if constexpr (MODE == 2) {
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int ec = 0; ec < EC; ++ec) {
          const int t = 4 * g + i, e = e0 + 16 * (EC * wave + ec) + m;
          gt[i][ec] = (whole_head && t < n && e < vdim) ? gate[(size_t)(c0 + t) * proj_ld + h * vdim + e] : (bf16_t)0;
        }
    }
    // ---- products of decays: queries from the block's start (threads of the last wavefronts), keys to its end ------- //
    for (int job = GLA_THREADS - 1 - tid; job < 2 * DP; job += GLA_THREADS) {
      const int c = job & (DP - 1);
      float w[16], x[16];
      if (job < DP) {
#pragma unroll
        for (int t = 0; t < 16; ++t) w[t] = Ws[t][c], x[t] = Ks[t][c];
        float p = 1.f;
#pragma unroll
        for (int t = 15; t >= 0; --t) {
          Kq[t][c] = x[t] * p;
          p *= w[t];
        }
        dec[c] = p;
        if constexpr (MODE == 1) product *= p;
      } else if constexpr (MODE == 2) {
#pragma unroll
        for (int t = 0; t < 16; ++t) w[t] = Ws[t][c], x[t] = Qs[t][c];
        float p = 1.f;
#pragma unroll
        for (int t = 0; t < 16; ++t) {
          if constexpr (KIND == KIND_GLA) p *= w[t];
          Qp[t][c] = x[t] * p;
          if constexpr (KIND == KIND_WKV) p *= w[t];
        }
      }
    }
    // ---- scores within the block: key ts against the queries from its own token on, CS channels a lane ------------- //
    if constexpr (MODE == 2) {
      float p[CS];
      float own = 0.f;
#pragma unroll
      for (int i = 0; i < CS; i += 4) {
        const float4 kk = *(const float4*)&Ks[ts][sl * CS + i], qq = *(const float4*)&Qs[ts][sl * CS + i];
        p[i] = kk.x, p[i + 1] = kk.y, p[i + 2] = kk.z, p[i + 3] = kk.w;
        own = fmaf(qq.x * kk.x, u[i], own), own = fmaf(qq.y * kk.y, u[i + 1], own);
        own = fmaf(qq.z * kk.z, u[i + 2], own), own = fmaf(qq.w * kk.w, u[i + 3], own);
      }
      own = row16_sum(own);
      if (sl == 0) As[ts][ts] = own;
      const int most = 15 - 4 * wave;  // the wavefront's first key has the most queries after it
      for (int after = 1; after <= most; ++after) {
        const int t = ts + after, tr = min(t, 15);
        float dot = 0.f;
#pragma unroll
        for (int i = 0; i < CS; i += 4) {
          const float4 w = *(const float4*)&Ws[tr][sl * CS + i], qq = *(const float4*)&Qs[tr][sl * CS + i];
          if constexpr (KIND == KIND_GLA) p[i] *= w.x, p[i + 1] *= w.y, p[i + 2] *= w.z, p[i + 3] *= w.w;
          dot = fmaf(qq.x, p[i], dot), dot = fmaf(qq.y, p[i + 1], dot), dot = fmaf(qq.z, p[i + 2], dot), dot = fmaf(qq.w, p[i + 3], dot);
          if constexpr (KIND == KIND_WKV) p[i] *= w.x, p[i + 1] *= w.y, p[i + 2] *= w.z, p[i + 3] *= w.w;
        }
        dot = row16_sum(dot);
        if (sl == 0 && t < 16) As[t][ts] = dot;
      }
    }
    __syncthreads();
    // ---- results from the state and from the block's own tokens, then the state -------------------------------------- //
    float vb[EC][4];
#pragma unroll
    for (int ec = 0; ec < EC; ++ec)
#pragma unroll
      for (int i = 0; i < 4; ++i) vb[ec][i] = Vs[4 * g + i][16 * (EC * wave + ec) + m];
    float4v o[EC];
    if constexpr (MODE == 2) {
#pragma unroll
      for (int ec = 0; ec < EC; ++ec) o[ec] = (float4v){0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int dt = 0; dt < DT; ++dt) {
        const float4v a = *(const float4v*)&Qp[m][16 * dt + 4 * g];
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
          for (int ec = 0; ec < EC; ++ec) o[ec] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], S[dt][ec][i], o[ec], 0, 0, 0);
      }
      const float4v a = *(const float4v*)&As[m][4 * g];
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int ec = 0; ec < EC; ++ec) o[ec] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], vb[ec][i], o[ec], 0, 0, 0);
    }
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      const float4v f = *(const float4v*)&dec[16 * dt + 4 * g];
#pragma unroll
      for (int ec = 0; ec < EC; ++ec)
#pragma unroll
        for (int i = 0; i < 4; ++i) S[dt][ec][i] *= f[i];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float a = Kq[4 * g + i][16 * dt + m];
#pragma unroll
        for (int ec = 0; ec < EC; ++ec) S[dt][ec] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, vb[ec][i], S[dt][ec], 0, 0, 0);
      }
    }
    if constexpr (MODE == 2) {
      if (whole_head) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          float sq = 0.f;
#pragma unroll
          for (int ec = 0; ec < EC; ++ec) sq = fmaf(o[ec][i], o[ec][i], sq);  // columns past the head's are zero
          sq = row16_sum(sq);
          if (m == 0) sq_part[wave][4 * g + i] = sq;
        }
        __syncthreads();
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = 4 * g + i;
        const float sq = whole_head ? (sq_part[0][t] + sq_part[1][t]) + (sq_part[2][t] + sq_part[3][t]) : 0.f;
        const float rstd = 1.0f / sqrtf(sq / (float)vdim + eps);
#pragma unroll
        for (int ec = 0; ec < EC; ++ec) {
          const int e = e0 + 16 * (EC * wave + ec) + m;
          if (t < n && e < vdim) {
            const size_t at = ((size_t)(c0 + t) * heads + h) * vdim + e;
            if (whole_head) {
              const float gv = bf16_to_f32(gt[i][ec]);
              out[at] = f32_to_bf16(o[ec][i] * rstd * weight[h * weight_stride + e] * (gv / (1.0f + expf(-gv))));
            } else {
              o_raw[at] = o[ec][i];
            }
          }
        }
      }
    }
  }
  if (MODE == 1 || last) {
#pragma unroll
    for (int dt = 0; dt < DT; ++dt)
#pragma unroll
      for (int ec = 0; ec < EC; ++ec)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const long at = state_at(16 * dt + 4 * g + i, e0 + 16 * (EC * wave + ec) + m);
          if (at < 0) continue;
          if constexpr (MODE == 1)
            seg_local[(size_t)seg * seg_ld + at] = S[dt][ec][i];
          else
            home[at] = S[dt][ec][i];
        }
  }
  if constexpr (MODE == 1) {
    const int c = GLA_THREADS - 1 - tid;
    if (blockIdx.x == 0 && c < dim) seg_decay[(size_t)seg * heads * dim + h * dim + c] = product;
  }
}

// The states at the segments' starts: a thread an element of a sequence's state walks the sequence's segments in order.
__global__ void __launch_bounds__(GLA_THREADS)
gla_carry_kernel(const int* __restrict__ segments, const float* __restrict__ state, long state_ld, const int* __restrict__ slots,
                 int n_slots, int heads, int dim, int split, int n_vt, const float* __restrict__ seg_local,
                 const float* __restrict__ seg_decay, float* __restrict__ seg_start, long seg_ld, long elems) {
  const int* sg = segments + 6 * blockIdx.y;
  if (sg[3] != 0) return;  // the sequence's first segment stands for all of them
  const long i = (long)blockIdx.x * GLA_THREADS + threadIdx.x;
  if (i >= elems) return;
  const int rows = gla_rows(dim, split);
  const long line = i / GLA_THREADS;  // [head][tile][row]
  const int h = (int)(line / (n_vt * rows)), d = ((int)(i % GLA_THREADS) % split) * rows + (int)(line % rows);
  const float* dp = seg_decay + h * dim + min(d, dim - 1);  // rows past the head's hold zeros, which stay
  const int slot = slots[sg[0]], first = sg[4], count = sg[5];
  float cur = (slot >= 0 && slot < n_slots) ? state[(size_t)slot * state_ld + i] : 0.f;
  for (int s = 0; s < count; s += 8) {
    float add[8], keep[8];
#pragma unroll
    for (int a = 0; a < 8; ++a) {  // the last segment has neither sum nor decays: what lies past the others is not used
      const size_t seg = first + min(s + a, max(count - 2, 0));
      add[a] = seg_local[seg * seg_ld + i], keep[a] = dp[seg * heads * dim];
    }
#pragma unroll
    for (int a = 0; a < 8; ++a) {
      if (s + a < count) seg_start[(size_t)(first + s + a) * seg_ld + i] = cur;
      cur = fmaf(keep[a], cur, add[a]);
    }
  }
}

template <typename T>
__global__ void __launch_bounds__(CWM_WAVE)
gla_out_kernel(const float* __restrict__ o_raw, const T* __restrict__ gate, long gate_ld, const float* __restrict__ weight,
               int weight_stride, T* __restrict__ out, int heads, int vdim, float eps) {
  const int t = blockIdx.x / heads, h = blockIdx.x - t * heads;
  gla_finish(o_raw + ((size_t)t * heads + h) * vdim, gate + (size_t)t * gate_ld + h * vdim, weight + h * weight_stride,
             out + ((size_t)t * heads + h) * vdim, vdim, eps);
}

// q, k ([T][heads * dim]) and v, gate ([T][heads * vdim]) of `dtype`, rows proj_ld elements apart.  bonus: null
// (KIND_GLA: decays sigmoid(z)^(1 / tau)), or float32 [heads * dim] (KIND_WKV: decays exp(-exp(z)), tau is not read).  z:
// float32 [T, heads * dim], rows z_ld apart.  weight: float32, head h's vdim values from h * weight_stride on.  state: float32
// [n_slots, state_ld] with cwm_gla_state_elems(...) <= state_ld elements a request; slots: int32 [n_seqs]; cu_q: int32
// [n_seqs + 1].  o_raw: float32 [T, heads * vdim] scratch.  out: [T, heads * vdim] of `dtype`.  segments (or null: every
// sequence is walked by one block a tile): int32 [n_segments][6] as above, all segments of the step in the order of the
// sequences; seg_local, seg_start: float32 [n_segments][seg_ld] scratch, seg_decay: float32 [n_segments][heads * dim]
// (all three null where every sequence is one segment).  Segments with bfloat16 and heads of up to GLA_BLOCK_DIM rows run
// on the matrix cores.
extern "C" int cwm_gated_linear_attention(const void* q, const void* k, const void* v, const void* gate, long proj_ld, int dtype,
                                          const float* bonus, const float* z, long z_ld, const float* weight,
                                          int weight_stride, float* o_raw, void* out, float* state, long state_ld,
                                          const int* slots, const int* cu_q, int n_slots, int n_tokens, int n_seqs, int heads,
                                          int dim, int vdim, float tau, float eps, float q_scale, const int* segments,
                                          int n_segments, float* seg_local, float* seg_decay, float* seg_start, long seg_ld,
                                          hipStream_t stream) {
  CWM_REQUIRE(n_tokens >= 0 && n_seqs >= 0 && heads >= 1 && vdim >= 1, "gated_linear_attention: bad sizes");
  CWM_REQUIRE(dim >= 1 && dim <= GLA_MAX_DIM, "gated_linear_attention: heads of %d rows are outside 1..%d", dim, GLA_MAX_DIM);
  CWM_REQUIRE((bonus || tau > 0.f) && eps > 0.f, "gated_linear_attention: tau and eps must be positive");
  CWM_REQUIRE(q && k && v && gate && z && weight && o_raw && out && state && slots && cu_q, "gated_linear_attention: arguments missing");
  CWM_REQUIRE(state_ld >= cwm_gla_state_elems(heads, dim, vdim), "gated_linear_attention: a state row of %ld elements is too short", state_ld);
  CWM_REQUIRE(n_seqs <= 65535 && heads <= 65535 && n_segments <= 65535, "gated_linear_attention: too many sequences, segments or heads for one launch");
  const bool several = seg_local != nullptr;
  CWM_REQUIRE(!segments || n_segments >= 1, "gated_linear_attention: an empty list of segments");
  CWM_REQUIRE(!several || (segments && seg_decay && seg_start && seg_ld >= cwm_gla_state_elems(heads, dim, vdim)),
              "gated_linear_attention: segments need their scratch states");
  if (n_tokens == 0 || n_seqs == 0) return 0;
  const int split = gla_split(dim, vdim), cols = GLA_THREADS / split, n_vt = (vdim + cols - 1) / cols;
  const int dpad = split * gla_rows(dim, split);
  const long elems = cwm_gla_state_elems(heads, dim, vdim);
  const float inv_tau = bonus ? 1.0f : 1.0f / tau;
  const bool on_matrix_cores = segments && dtype == CWM_BF16 && dim <= GLA_BLOCK_DIM;
  CWM_REQUIRE(on_matrix_cores || !segments || several, "gated_linear_attention: segments need their scratch states");
  auto carry = [&] {
    hipLaunchKernelGGL(gla_carry_kernel, dim3((unsigned)((elems + GLA_THREADS - 1) / GLA_THREADS), n_segments), dim3(GLA_THREADS), 0,
                       stream, segments, state, state_ld, slots, n_slots, heads, dim, split, n_vt, seg_local, seg_decay, seg_start,
                       seg_ld, elems);
  };
  int tiles = n_vt;  // blocks that share a head's columns
  if (on_matrix_cores) {
    const int ec = vdim <= 64 ? 1 : 2;
    tiles = (vdim + 64 * ec - 1) / (64 * ec);
    const bool vec = dim % 4 == 0 && vdim % 4 == 0 && proj_ld % 4 == 0 &&
                     (((uintptr_t)q | (uintptr_t)k | (uintptr_t)v) % 8) == 0;
    const dim3 grid(tiles, heads, n_segments);
#define CWM_GLA_BLOCK(MODE, KIND, CS, EC)                                                                                   \
  hipLaunchKernelGGL((gla_block_kernel<MODE, KIND, CS, EC>), grid, dim3(GLA_THREADS), 0, stream, (const bf16_t*)q,            \
                     (const bf16_t*)k, (const bf16_t*)v, (const bf16_t*)gate, proj_ld, bonus, z, z_ld, weight, weight_stride,  \
                     eps, o_raw, (bf16_t*)out, state, state_ld, slots, n_slots, heads, dim, vdim, split, inv_tau, q_scale, vec, \
                     segments, seg_local, seg_decay, seg_start, seg_ld)
#define CWM_GLA_BLOCK_EC(MODE, KIND, CS)          \
  do {                                            \
    if (ec == 1)                                  \
      CWM_GLA_BLOCK(MODE, KIND, CS, 1);           \
    else                                          \
      CWM_GLA_BLOCK(MODE, KIND, CS, 2);           \
  } while (0)
#define CWM_GLA_BLOCK_CS(MODE, KIND)              \
  do {                                            \
    if (dim <= 64)                                \
      CWM_GLA_BLOCK_EC(MODE, KIND, 4);            \
    else                                          \
      CWM_GLA_BLOCK_EC(MODE, KIND, 8);            \
  } while (0)
#define CWM_GLA_BLOCK_KIND(MODE)                  \
  do {                                            \
    if (bonus)                                    \
      CWM_GLA_BLOCK_CS(MODE, KIND_WKV);           \
    else                                          \
      CWM_GLA_BLOCK_CS(MODE, KIND_GLA);           \
  } while (0)
    if (several) {
      CWM_GLA_BLOCK_KIND(1);
      carry();
    }
    CWM_GLA_BLOCK_KIND(2);
#undef CWM_GLA_BLOCK_KIND
#undef CWM_GLA_BLOCK_CS
#undef CWM_GLA_BLOCK_EC
#undef CWM_GLA_BLOCK
    const int status = cwm_launch_status("gated_linear_attention (blocks)");
    if (status) return status;
  } else {
    int chunk = GLA_CHUNK;
    while (chunk > 1 && sizeof(float) * (size_t)chunk * (3 * dpad + 2 * cols + 1) > 49152) chunk /= 2;
    const size_t lds = sizeof(float) * (size_t)chunk * (3 * dpad + 2 * cols + 1);
    const dim3 grid(n_vt, heads, n_seqs), grid_seg(n_vt, heads, segments ? n_segments : 1);
#define CWM_GLA_WALK(T, MODE, KIND, GRID)                                                                                   \
  hipLaunchKernelGGL((gla_walk_kernel<T, MODE, KIND>), GRID, dim3(GLA_THREADS), lds, stream, (const T*)q, (const T*)k,         \
                     (const T*)v, (const T*)gate, proj_ld, weight, weight_stride, (T*)out, eps, bonus, z, z_ld, o_raw, state,   \
                     state_ld, slots, cu_q, n_slots, heads, dim, vdim, split, chunk, inv_tau, q_scale, segments, seg_local,     \
                     seg_decay, seg_start, seg_ld)
#define CWM_GLA_KIND(T, KIND)                     \
  do {                                            \
    if (segments) {                               \
      CWM_GLA_WALK(T, 1, KIND, grid_seg);         \
      carry();                                    \
      CWM_GLA_WALK(T, 2, KIND, grid_seg);         \
    } else {                                      \
      CWM_GLA_WALK(T, 0, KIND, grid);             \
    }                                             \
  } while (0)
#define CWM_GLA(T)                  \
  do {                              \
    if (bonus)                      \
      CWM_GLA_KIND(T, KIND_WKV);    \
    else                            \
      CWM_GLA_KIND(T, KIND_GLA);    \
  } while (0)
    if (dtype == CWM_F32) CWM_GLA(float);
    else if (dtype == CWM_BF16) CWM_GLA(bf16_t);
    else return cwm_fail("gated_linear_attention: unknown element type %d", dtype);
#undef CWM_GLA
#undef CWM_GLA_KIND
#undef CWM_GLA_WALK
    const int status = cwm_launch_status("gated_linear_attention");
    if (status) return status;
  }
  if (tiles > 1) {
    if (dtype == CWM_F32)
      hipLaunchKernelGGL((gla_out_kernel<float>), dim3(n_tokens * heads), dim3(CWM_WAVE), 0, stream, o_raw, (const float*)gate,
                         proj_ld, weight, weight_stride, (float*)out, heads, vdim, eps);
    else
      hipLaunchKernelGGL((gla_out_kernel<bf16_t>), dim3(n_tokens * heads), dim3(CWM_WAVE), 0, stream, o_raw, (const bf16_t*)gate,
                         proj_ld, weight, weight_stride, (bf16_t*)out, heads, vdim, eps);
  }
  return cwm_launch_status("gated_linear_attention (results)");
}

// ---- a decode step of the form with a bonus, from the projections' sums to the gated result -------------------------- //
// One token a sequence; a block a (head, sequence).  sums: the product's float32 partial sums, a row [r | k | v | g | low],
// heads * dim values of the first four and `rank` of the last.  The decay's logits are z = w2 tanh(low) + w0, its second
// matrix (bfloat16) read beside the state; then the recurrence as in the walk (the state lies as the walk keeps it), the
// norm of the head's result, its weight and the gate.  All sums float32.
__device__ __forceinline__ float partial_sum(const float* p, int n_partials, long stride) {
  if (n_partials == 1) return *p;
  float total = 0.f;
  for (int q = 0; q < n_partials; q += 4) {  // four in flight, added in their order; past the last: that one times zero
    float x[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) x[u] = p[(size_t)min(q + u, n_partials - 1) * stride];
#pragma unroll
    for (int u = 0; u < 4; ++u) total = fmaf(q + u < n_partials ? 1.0f : 0.0f, x[u], total);
  }
  return total;
}

__global__ void __launch_bounds__(GLA_THREADS)
wkv_token_kernel(const float* __restrict__ sums, long ld, int n_partials, long partial_stride, const bf16_t* __restrict__ w2,
                 int rank, const float* __restrict__ w0, const float* __restrict__ bonus, const float* __restrict__ weight,
                 float eps, bf16_t* __restrict__ out, float* __restrict__ state, long state_ld, const int* __restrict__ slots,
                 int n_slots, int heads, int dim, int split) {
  __shared__ __attribute__((aligned(16))) float qs[GLA_MAX_DIM], ks[GLA_MAX_DIM], uk[GLA_MAX_DIM], as[GLA_MAX_DIM];
  __shared__ float vs[GLA_MAX_DIM], gs[GLA_MAX_DIM], os[GLA_MAX_DIM];
  extern __shared__ float low[];  // [rank]
  const int h = blockIdx.x, t = blockIdx.y, tid = threadIdx.x;
  const int cols = GLA_THREADS / split, rows = gla_rows(dim, split), dpad = split * rows, n_vt = (dim + cols - 1) / cols;
  const int col = tid / split, part = tid % split;
  const int inner = heads * dim;
  const int slot = slots[t];
  if (slot < 0 || slot >= n_slots) return;
  float* st = state + (size_t)slot * state_ld + (size_t)h * n_vt * rows * GLA_THREADS + tid;
  // the first tile's state and the thread's share of w2 are in flight while the projections are added up
  float S[GLA_ROWS];
#pragma unroll
  for (int r = 0; r < GLA_ROWS; ++r) S[r] = r < rows ? st[(size_t)r * GLA_THREADS] : 0.f;
  int lanes = 1;  // threads that share a channel's logit
  while (lanes < 8 && 2 * lanes * dim <= GLA_THREADS) lanes *= 2;
  const int share = rank / lanes, chan = tid / lanes, piece = tid - chan * lanes;
  const bool vec = share * lanes == rank && share % 8 == 0 && share <= 32 && ((uintptr_t)w2 % 16) == 0;
  uint4 w2r[4];
#pragma unroll
  for (int i = 0; i < 4; ++i)
    w2r[i] = (vec && chan < dim && 8 * i < share) ? *(const uint4*)(w2 + (size_t)(h * dim + chan) * rank + piece * share + 8 * i) : make_uint4(0, 0, 0, 0);
  // and so are what the later stages read of the weights: no stage then waits for memory of its own
  const float w0r = chan < dim ? w0[h * dim + chan] : 0.f;
  float wr[GLA_MAX_DIM / CWM_WAVE];
#pragma unroll
  for (int i = 0; i < GLA_MAX_DIM / CWM_WAVE; ++i) {
    const int e = tid + CWM_WAVE * i;
    wr[i] = (tid < CWM_WAVE && e < dim) ? weight[h * dim + e] : 0.f;
  }
  const float* row = sums + (size_t)t * ld;
  for (int d = tid; d < dpad; d += GLA_THREADS) {
    const bool real = d < dim;
    const int c = h * dim + d;
    const float kk = real ? partial_sum(row + inner + c, n_partials, partial_stride) : 0.f;
    qs[d] = real ? partial_sum(row + c, n_partials, partial_stride) : 0.f;
    ks[d] = kk;
    uk[d] = real ? kk * bonus[c] : 0.f;
    as[d] = 0.f;
    if (real) {
      vs[d] = partial_sum(row + 2 * inner + c, n_partials, partial_stride);
      gs[d] = partial_sum(row + 3 * inner + c, n_partials, partial_stride);
    }
  }
  for (int j = tid; j < rank; j += GLA_THREADS) low[j] = tanhf(partial_sum(row + 4 * inner + j, n_partials, partial_stride));
  __syncthreads();
  for (int c = chan; c < dim; c += GLA_THREADS / lanes) {
    float z = 0.f;
    if (vec) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        if (8 * i < share) {
          const uint4 w = c == chan ? w2r[i] : *(const uint4*)(w2 + (size_t)(h * dim + c) * rank + piece * share + 8 * i);
          const uint32_t ws[4] = {w.x, w.y, w.z, w.w};
          const float* l = low + piece * share + 8 * i;
#pragma unroll
          for (int x = 0; x < 4; ++x) {
            z = fmaf(__uint_as_float(ws[x] << 16), l[2 * x], z);
            z = fmaf(__uint_as_float(ws[x] & 0xffff0000u), l[2 * x + 1], z);
          }
        }
      }
    } else {
      for (int j = piece; j < rank; j += lanes) z = fmaf(bf16_to_f32(w2[(size_t)(h * dim + c) * rank + j]), low[j], z);
    }
    for (int off = 1; off < lanes; off *= 2) z += __shfl_xor(z, off, CWM_WAVE);
    if (piece == 0) as[c] = gla_decay<KIND_WKV>(z + (c == chan ? w0r : w0[h * dim + c]), 1.0f);
  }
  __syncthreads();
  const int d0 = part * rows;
  for (int vt = 0; vt < n_vt; ++vt) {
    float* tile = st + (size_t)vt * rows * GLA_THREADS;
    if (vt > 0) {
#pragma unroll
      for (int r = 0; r < GLA_ROWS; ++r) S[r] = r < rows ? tile[(size_t)r * GLA_THREADS] : 0.f;
    }
    const int e = vt * cols + col;
    const float v = e < dim ? vs[e] : 0.f;
    float o = 0.f;
#pragma unroll
    for (int r = 0; r < GLA_ROWS; r += 4) {
      if (r < rows) {
        const float4 q4 = *(const float4*)(qs + d0 + r), k4 = *(const float4*)(ks + d0 + r);
        const float4 u4 = *(const float4*)(uk + d0 + r), a4 = *(const float4*)(as + d0 + r);
        o = fmaf(fmaf(u4.x, v, S[r]), q4.x, o), o = fmaf(fmaf(u4.y, v, S[r + 1]), q4.y, o);
        o = fmaf(fmaf(u4.z, v, S[r + 2]), q4.z, o), o = fmaf(fmaf(u4.w, v, S[r + 3]), q4.w, o);
        tile[(size_t)r * GLA_THREADS] = fmaf(a4.x, S[r], k4.x * v);
        tile[(size_t)(r + 1) * GLA_THREADS] = fmaf(a4.y, S[r + 1], k4.y * v);
        tile[(size_t)(r + 2) * GLA_THREADS] = fmaf(a4.z, S[r + 2], k4.z * v);
        tile[(size_t)(r + 3) * GLA_THREADS] = fmaf(a4.w, S[r + 3], k4.w * v);
      }
    }
    for (int off = 1; off < split; off *= 2) o += __shfl_xor(o, off, CWM_WAVE);
    if (part == 0 && e < dim) os[e] = o;
  }
  __syncthreads();
  if (tid >= CWM_WAVE) return;
  float sq = 0.f;
  for (int e = tid; e < dim; e += CWM_WAVE) sq += os[e] * os[e];
  const float rstd = 1.0f / sqrtf(wave_sum(sq) / (float)dim + eps);
#pragma unroll
  for (int i = 0; i < GLA_MAX_DIM / CWM_WAVE; ++i) {
    const int e = tid + CWM_WAVE * i;
    if (e < dim) {
      const float g = gs[e];
      out[(size_t)t * inner + h * dim + e] = f32_to_bf16(os[e] * rstd * wr[i] * (g / (1.0f + expf(-g))));
    }
  }
}

// sums: float32 [n_partials][n_tokens][ld], partial_stride elements between partial sums.  w2: bfloat16 [heads * dim][rank];
// w0, bonus, weight: float32 [heads * dim].  out: bfloat16 [n_tokens][heads * dim].  Token t belongs to sequence t.
extern "C" int cwm_wkv_token(const float* sums, long ld, int n_partials, long partial_stride, const void* w2, int rank,
                             const float* w0, const float* bonus, const float* weight, float eps, void* out, float* state,
                             long state_ld, const int* slots, int n_slots, int n_tokens, int heads, int dim, hipStream_t stream) {
  CWM_REQUIRE(n_tokens >= 0 && n_tokens <= 65535 && heads >= 1 && n_partials >= 1, "wkv_token: bad sizes");
  CWM_REQUIRE(dim >= 1 && dim <= GLA_MAX_DIM, "wkv_token: heads of %d rows are outside 1..%d", dim, GLA_MAX_DIM);
  CWM_REQUIRE(rank >= 1 && rank <= 4096, "wkv_token: a rank of %d is outside 1..4096", rank);
  CWM_REQUIRE(ld >= 4L * heads * dim + rank && eps > 0.f, "wkv_token: rows of %ld values are too short", ld);
  CWM_REQUIRE(sums && w2 && w0 && bonus && weight && out && state && slots, "wkv_token: arguments missing");
  CWM_REQUIRE(state_ld >= cwm_gla_state_elems(heads, dim, dim), "wkv_token: a state row of %ld elements is too short", state_ld);
  if (n_tokens == 0) return 0;
  hipLaunchKernelGGL(wkv_token_kernel, dim3(heads, n_tokens), dim3(GLA_THREADS), sizeof(float) * rank, stream, sums, ld, n_partials,
                     partial_stride, (const bf16_t*)w2, rank, w0, bonus, weight, eps, (bf16_t*)out, state, state_ld, slots, n_slots,
                     heads, dim, gla_split(dim, dim));
  return cwm_launch_status("wkv_token");
}
