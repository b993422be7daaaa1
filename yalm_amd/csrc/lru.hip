// A gated linear recurrence on every channel of its own (a real-gated linear recurrent unit).  With u the block's input (float32,
// behind its short convolution), cut into blocks of n channels, per token
//     r = sigmoid(R_b u_b + r0),   i = sigmoid(I_b u_b + i0)           (R_b, I_b: n x n, one pair a block)
//     a = exp(s r),   S <- a S + sqrt(1 - a^2) i u,   out = S gelu(z + z0)
// s < 0 a number a channel, z the other branch's product.  sqrt(1 - a^2) is formed as sqrt(-expm1(2 s r)), so that a decay
// close to one keeps its digits.  Everything is float32; with bfloat16 matrices the gates' products run on the matrix cores
// with u as the sum of two bfloat16 numbers, so that u is not rounded to 16 bits on the way.
//
// Steps of prompts, a tile of 64 tokens of one sequence at a time, all tiles at once:
//   lru_gates*_kernel  the gates, and the recurrence inside the tile from S = 0: P_t the product of the decays from the tile's
//                      start up to t, Q_t the state that the tile's own tokens make; the tile's last P and Q once more, in `ends`;
//   lru_carry_kernel   the states in front of the tiles, a thread a channel (over `ends`), and the state behind the text;
//   lru_finish_kernel  out = (P S_in + Q) gelu(z + z0).
// Steps of single tokens: lru_step_kernel does all of it, sixteen lanes a channel; many of them go through the gates' kernel (tiles
// of 64 rows, P = a and Q the token's own share) and lru_finish_kernel.
#include "common.h"
#include "yalm_hip.h"

namespace {
constexpr int LG_T = PAGE, LG_N = 64, LG_K = 32, LG_THREADS = 256, LG_Q = LG_T / 4;      // tokens, channels, k of a stage; tokens of a quarter
constexpr int LG_ZROW = LG_N + 1;

struct LruArgs {
  const float* u;                                // [T, W]
  const float* bias;                             // [2, W]: r0, i0
  const float* slope;                            // [W]: s
  float *P, *Q, *ends;                           // [T, W] each; [tiles, 2, W]
  const int *cu_seqlens, *seq_tile0;             // seq_tile0 null: the rows are single tokens, tiles are 64 rows
  int T, B, W, n;
};

__device__ __forceinline__ float sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float gelu(float z) { return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z))); }
// a and sqrt(1 - a^2) i u of one token and channel
__device__ __forceinline__ void lru_terms(float zr, float zi, float slope, float u, float& a, float& b) {
  const float la = slope * sigmoid(zr);
  a = expf(la);
  b = sqrtf(-expm1f(2.0f * la)) * sigmoid(zi) * u;
}

struct LruTile { int first, rows; };
__device__ __forceinline__ LruTile lru_tile(const LruArgs& x, int tile) {
  if (x.seq_tile0 == nullptr) return {tile * LG_T, min(LG_T, x.T - tile * LG_T)};
  int lo = 0, hi = x.B - 1;                        // the last sequence whose first tile is not behind this one
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (x.seq_tile0[mid] <= tile) lo = mid; else hi = mid - 1;
  }
  const int first = x.cu_seqlens[lo] + (tile - x.seq_tile0[lo]) * LG_T;
  return {first, min(LG_T, x.cu_seqlens[lo + 1] - first)};
}

// From the gates' products of a tile (s_z [2][64 tokens][LG_ZROW], without bias) to P and Q.  A thread a channel and a
// quarter of the tokens; s_ends [4][64][2].  Called by all threads behind a barrier.
__device__ __forceinline__ void lru_tile_scan(const LruArgs& x, const LruTile tile, const float* s_z, float* s_ends, int c0, int c_end) {
  const int ch = threadIdx.x % LG_N, quarter = threadIdx.x / LG_N, c = c0 + ch;
  const bool ok = c < c_end, scan = x.seq_tile0 != nullptr;
  const int cc = min(c, c_end - 1);
  const float br = x.bias[cc], bi = x.bias[x.W + cc], slope = x.slope[cc];
  float p[LG_Q], q[LG_Q], uu[LG_Q];
#pragma unroll
  for (int i = 0; i < LG_Q; ++i) uu[i] = x.u[(size_t)(tile.first + min(quarter * LG_Q + i, tile.rows - 1)) * x.W + cc];
  float A = 1.f, S = 0.f;
#pragma unroll
  for (int i = 0; i < LG_Q; ++i) {
    const int t = quarter * LG_Q + i;
    float a, b;
    lru_terms(s_z[t * LG_ZROW + ch] + br, s_z[(LG_T + t) * LG_ZROW + ch] + bi, slope, uu[i], a, b);
    if (scan) {
      if (t >= tile.rows) a = 1.f, b = 0.f;        // behind the text: nothing changes any more
      A *= a;
      S = fmaf(a, S, b);
      p[i] = A, q[i] = S;
    } else {
      p[i] = a, q[i] = b;
    }
  }
  if (scan) {                                      // what the quarters in front have made
    s_ends[(quarter * LG_N + ch) * 2] = A;
    s_ends[(quarter * LG_N + ch) * 2 + 1] = S;
    __syncthreads();
    float pa = 1.f, ps = 0.f;
    for (int k = 0; k < quarter; ++k) {
      const float ka = s_ends[(k * LG_N + ch) * 2], ks = s_ends[(k * LG_N + ch) * 2 + 1];
      ps = fmaf(ka, ps, ks);
      pa *= ka;
    }
#pragma unroll
    for (int i = 0; i < LG_Q; ++i) {
      q[i] = fmaf(p[i], ps, q[i]);
      p[i] *= pa;
    }
    if (quarter == 3 && ok) {
      float* e = x.ends + (size_t)blockIdx.x * 2 * x.W + c;
      e[0] = p[LG_Q - 1];
      e[x.W] = q[LG_Q - 1];
    }
  }
  if (!ok) return;
#pragma unroll
  for (int i = 0; i < LG_Q; ++i) {
    const int t = quarter * LG_Q + i;
    if (t < tile.rows) {
      const size_t at = (size_t)(tile.first + t) * x.W + c;
      x.P[at] = p[i];
      x.Q[at] = q[i];
    }
  }
}

// Any sizes and both storage types of the matrices: float32 multiply-adds, a thread 16 tokens and one channel of both gates.
template <typename TW>
__global__ __launch_bounds__(LG_THREADS) void lru_gates_kernel(LruArgs x, const TW* __restrict__ w) {
  __shared__ float s_u[LG_T][LG_K + 1], s_w[2][LG_N][LG_K + 1];
  __shared__ float s_z[2 * LG_T * LG_ZROW], s_ends[4 * LG_N * 2];
  const LruTile tile = lru_tile(x, blockIdx.x);
  if (tile.rows <= 0) return;
  const int n = x.n, per_block = ((n + LG_N - 1) / LG_N);
  const int blk = blockIdx.y / per_block, n0 = blockIdx.y % per_block * LG_N, tid = threadIdx.x, ch = tid % LG_N, quarter = tid / LG_N;
  float acc[2][LG_Q];
#pragma unroll
  for (int i = 0; i < LG_Q; ++i) acc[0][i] = acc[1][i] = 0.f;
  for (int k0 = 0; k0 < n; k0 += LG_K) {
    for (int i = tid; i < LG_T * LG_K; i += LG_THREADS) {
      const int t = i / LG_K, k = k0 + i % LG_K;
      s_u[t][i % LG_K] = t < tile.rows && k < n ? x.u[(size_t)(tile.first + t) * x.W + blk * n + k] : 0.f;
    }
    for (int i = tid; i < 2 * LG_N * LG_K; i += LG_THREADS) {
      const int m = i / (LG_N * LG_K), o = i / LG_K % LG_N, k = k0 + i % LG_K;
      s_w[m][o][i % LG_K] = n0 + o < n && k < n ? to_f32(w[((size_t)m * x.W + blk * n + n0 + o) * n + k]) : 0.f;
    }
    __syncthreads();
#pragma unroll 4
    for (int k = 0; k < LG_K; ++k) {
      const float wr = s_w[0][ch][k], wi = s_w[1][ch][k];
#pragma unroll
      for (int i = 0; i < LG_Q; ++i) {
        const float v = s_u[quarter * LG_Q + i][k];
        acc[0][i] = fmaf(wr, v, acc[0][i]);
        acc[1][i] = fmaf(wi, v, acc[1][i]);
      }
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < LG_Q; ++i)
#pragma unroll
    for (int m = 0; m < 2; ++m) s_z[(m * LG_T + quarter * LG_Q + i) * LG_ZROW + ch] = acc[m][i];
  __syncthreads();
  lru_tile_scan(x, tile, s_z, s_ends, blk * n + n0, (blk + 1) * n);
}

// bfloat16 matrices on the matrix cores (n a multiple of 8): v_mfma_f32_32x32x16_bf16 (operand rows = lane % 32, eight k a
// lane at k offset 8 (lane / 32); result column = lane % 32, rows 8 (r / 4) + 4 (lane / 32) + r % 4).  A wave 32 tokens and 32
// channels of both gates; u = hi + lo.  The next stage's operands wait in registers.
typedef __attribute__((ext_vector_type(8))) __bf16 lg_bf16x8;
typedef __attribute__((ext_vector_type(16))) float lg_f32x16;
constexpr int LG_ROW = LG_K + 8;
__global__ __launch_bounds__(LG_THREADS) void lru_gates_mfma_kernel(LruArgs x, const bf16* __restrict__ w) {
  constexpr size_t STAGE = (size_t)(2 * LG_T + 2 * LG_N) * LG_ROW * sizeof(bf16), Z = (size_t)2 * LG_T * LG_ZROW * sizeof(float);
  __shared__ __attribute__((aligned(16))) unsigned char raw[STAGE > Z ? STAGE : Z];
  __shared__ float s_ends[4 * LG_N * 2];
  bf16* s_hi = reinterpret_cast<bf16*>(raw);      // [64][LG_ROW]
  bf16* s_lo = s_hi + LG_T * LG_ROW;
  bf16* s_w = s_lo + LG_T * LG_ROW;               // [2][64][LG_ROW]
  const LruTile tile = lru_tile(x, blockIdx.x);
  if (tile.rows <= 0) return;
  const int n = x.n, per_block = ((n + LG_N - 1) / LG_N);
  const int blk = blockIdx.y / per_block, n0 = blockIdx.y % per_block * LG_N, tid = threadIdx.x;
  const int wave = tid / WAVE, lane = tid % WAVE, wm = wave / 2, wn = wave % 2, li = lane % 32, lh = lane / 32;
  const int lrow = tid / 4, lk = tid % 4 * 8;      // what this thread stages: 8 values of row lrow of u and of both matrices
  const bool u_ok = lrow < tile.rows, w_ok = n0 + lrow < n;
  const float* up = x.u + (size_t)(tile.first + (u_ok ? lrow : 0)) * x.W + blk * n + lk;
  const bf16* wp = w + ((size_t)blk * n + n0 + (w_ok ? lrow : 0)) * n + lk;
  float4 ua, ub;
  lg_bf16x8 wr, wi;
  const lg_bf16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
  auto fetch = [&](int k0) {
    const bool k_ok = k0 + lk < n;
    ua = ub = make_float4(0.f, 0.f, 0.f, 0.f);
    wr = wi = zero;
    if (u_ok && k_ok) {
      ua = *reinterpret_cast<const float4*>(up + k0);
      ub = *reinterpret_cast<const float4*>(up + k0 + 4);
    }
    if (w_ok && k_ok) {
      wr = *reinterpret_cast<const lg_bf16x8*>(wp + k0);
      wi = *reinterpret_cast<const lg_bf16x8*>(wp + (size_t)x.W * n + k0);
    }
  };
  lg_f32x16 acc[2];
#pragma unroll
  for (int r = 0; r < 16; ++r) acc[0][r] = acc[1][r] = 0.f;
  fetch(0);
  for (int k0 = 0; k0 < n; k0 += LG_K) {
    {
      const float v[8] = {ua.x, ua.y, ua.z, ua.w, ub.x, ub.y, ub.z, ub.w};
      lg_bf16x8 hi, lo;
#pragma unroll
      for (int k = 0; k < 8; ++k) {
        hi[k] = static_cast<bf16>(v[k]);
        lo[k] = static_cast<bf16>(v[k] - static_cast<float>(hi[k]));
      }
      *reinterpret_cast<lg_bf16x8*>(s_hi + lrow * LG_ROW + lk) = hi;
      *reinterpret_cast<lg_bf16x8*>(s_lo + lrow * LG_ROW + lk) = lo;
      *reinterpret_cast<lg_bf16x8*>(s_w + lrow * LG_ROW + lk) = wr;
      *reinterpret_cast<lg_bf16x8*>(s_w + (LG_N + lrow) * LG_ROW + lk) = wi;
    }
    __syncthreads();
    if (k0 + LG_K < n) fetch(k0 + LG_K);
#pragma unroll
    for (int ks = 0; ks < LG_K; ks += 16) {
      const lg_bf16x8 hi = *reinterpret_cast<const lg_bf16x8*>(s_hi + (wm * 32 + li) * LG_ROW + ks + lh * 8);
      const lg_bf16x8 lo = *reinterpret_cast<const lg_bf16x8*>(s_lo + (wm * 32 + li) * LG_ROW + ks + lh * 8);
#pragma unroll
      for (int m = 0; m < 2; ++m) {
        const lg_bf16x8 f = *reinterpret_cast<const lg_bf16x8*>(s_w + (m * LG_N + wn * 32 + li) * LG_ROW + ks + lh * 8);
        acc[m] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(lo, f, acc[m], 0, 0, 0);
        acc[m] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(hi, f, acc[m], 0, 0, 0);
      }
    }
    __syncthreads();
  }
  float* s_z = reinterpret_cast<float*>(raw);      // the last stage is read
#pragma unroll
  for (int m = 0; m < 2; ++m)
#pragma unroll
    for (int r = 0; r < 16; ++r)
      s_z[(m * LG_T + wm * 32 + 8 * (r / 4) + 4 * lh + r % 4) * LG_ZROW + wn * 32 + li] = acc[m][r];
  __syncthreads();
  lru_tile_scan(x, tile, s_z, s_ends, blk * n + n0, (blk + 1) * n);
}

// ends [tile][0] <- the state in front of the tile; state [slot] <- the state behind the text.  A thread a (sequence, channel).
__global__ __launch_bounds__(WAVE) void lru_carry_kernel(float* __restrict__ ends, float* __restrict__ state,
                                                         const int* __restrict__ cu_seqlens, const int* __restrict__ seq_slot,
                                                         const int* __restrict__ seq_tile0, int W) {
  const int b = blockIdx.y, c = blockIdx.x * WAVE + threadIdx.x;
  if (c >= W) return;
  const int slot = seq_slot[b], n_tiles = (cu_seqlens[b + 1] - cu_seqlens[b] + LG_T - 1) / LG_T;
  float S = slot >= 0 ? state[(size_t)slot * W + c] : 0.f;
  float* e = ends + (size_t)seq_tile0[b] * 2 * W + c;
  constexpr int AHEAD = 8;
  for (int k0 = 0; k0 < n_tiles; k0 += AHEAD) {
    float a[AHEAD], q[AHEAD];
#pragma unroll
    for (int k = 0; k < AHEAD; ++k) {
      const size_t at = (size_t)min(k0 + k, n_tiles - 1) * 2 * W;
      a[k] = e[at];
      q[k] = e[at + W];
    }
#pragma unroll
    for (int k = 0; k < AHEAD; ++k) {
      if (k0 + k < n_tiles) {
        e[(size_t)(k0 + k) * 2 * W] = S;
        S = fmaf(a[k], S, q[k]);
      }
    }
  }
  if (slot >= 0) state[(size_t)slot * W + c] = S;
}

// out = (P S_in + Q) gelu(z + z0): S_in from `ends` (prompts), or with seq_tile0 null the sequence's state, which the new one
// replaces (row t is sequence t's one token; a padding row gives zeros).  VEC neighbours a thread.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void lru_finish_kernel(const float* __restrict__ P, const float* __restrict__ Q,
                                                         const float* __restrict__ ends, float* __restrict__ state,
                                                         const float* __restrict__ z, long z_row, const float* __restrict__ z_bias,
                                                         T* __restrict__ out, const int* __restrict__ tok_seq,
                                                         const int* __restrict__ cu_seqlens, const int* __restrict__ seq_slot,
                                                         const int* __restrict__ seq_tile0, int W) {
  struct __attribute__((aligned(VEC * sizeof(float)))) F { float v[VEC]; };
  struct __attribute__((aligned(VEC * sizeof(T)))) O { T v[VEC]; };
  const int t = blockIdx.x, c = (blockIdx.y * 256 + threadIdx.x) * VEC;
  if (c >= W) return;
  const size_t at = (size_t)t * W + c;
  const F p = *reinterpret_cast<const F*>(P + at), q = *reinterpret_cast<const F*>(Q + at);
  const F y = *reinterpret_cast<const F*>(z + (size_t)t * z_row + c), yb = *reinterpret_cast<const F*>(z_bias + c);
  F s = {};
  float* own = nullptr;
  bool padding = false;
  if (seq_tile0 != nullptr) {
    const int b = tok_seq[t];
    s = *reinterpret_cast<const F*>(ends + (size_t)(seq_tile0[b] + (t - cu_seqlens[b]) / LG_T) * 2 * W + c);
  } else {
    const int slot = seq_slot[t];
    padding = slot < 0;
    if (!padding) {
      own = state + (size_t)slot * W + c;
      s = *reinterpret_cast<const F*>(own);
    }
  }
  O o;
#pragma unroll
  for (int k = 0; k < VEC; ++k) {
    s.v[k] = fmaf(p.v[k], s.v[k], q.v[k]);
    o.v[k] = from_f32<T>(padding ? 0.f : s.v[k] * gelu(y.v[k] + yb.v[k]));
  }
  if (own != nullptr) *reinterpret_cast<F*>(own) = s;
  *reinterpret_cast<O*>(out + at) = o;
}

// A step of single tokens (row t is sequence t's): sixteen lanes a channel, LS_ROWS rows at a time.
constexpr int LS_LANES = 16, LS_ROWS = 8, LS_CH = 256 / LS_LANES;
template <typename TW, typename T, bool VEC>
__global__ __launch_bounds__(256) void lru_step_kernel(const float* __restrict__ u, const TW* __restrict__ w, const float* __restrict__ bias,
                                                       const float* __restrict__ slope, const float* __restrict__ z, long z_row,
                                                       const float* __restrict__ z_bias, float* __restrict__ state,
                                                       const int* __restrict__ seq_slot, T* __restrict__ out, int n_rows, int W, int n) {
  const int lane = threadIdx.x % LS_LANES, c = blockIdx.x * LS_CH + threadIdx.x / LS_LANES, r0 = blockIdx.y * LS_ROWS;
  if (c >= W) return;                              // whole groups of lanes: the exchanges below stay inside a group
  const int rows = min(LS_ROWS, n_rows - r0), blk = c / n;
  const TW* wr = w + (size_t)c * n;
  const TW* wi = wr + (size_t)W * n;
  const float* ub = u + (size_t)r0 * W + blk * n;
  // what the lane's own row will need is asked for first
  const int row = r0 + min(lane, rows - 1), slot = seq_slot[row];
  const float y = z[(size_t)row * z_row + c] + z_bias[c], own = u[(size_t)row * W + c];
  const float S0 = slot >= 0 ? state[(size_t)slot * W + c] : 0.f;
  float acc[LS_ROWS][2];
#pragma unroll
  for (int r = 0; r < LS_ROWS; ++r) acc[r][0] = acc[r][1] = 0.f;
  constexpr int K = VEC ? 4 : 1;
  for (int k = lane * K; k < n; k += LS_LANES * K) {
    float a[K], b[K];
    if constexpr (VEC) {
      struct __attribute__((aligned(4 * sizeof(TW)))) W4 { TW v[4]; };
      const W4 a4 = *reinterpret_cast<const W4*>(wr + k), b4 = *reinterpret_cast<const W4*>(wi + k);
#pragma unroll
      for (int e = 0; e < 4; ++e) a[e] = to_f32(a4.v[e]), b[e] = to_f32(b4.v[e]);
    } else {
      a[0] = to_f32(wr[k]), b[0] = to_f32(wi[k]);
    }
#pragma unroll
    for (int r = 0; r < LS_ROWS; ++r) {
      const float* p = ub + (size_t)min(r, rows - 1) * W + k;
      float v[K];
      if constexpr (VEC) {
        const float4 v4 = *reinterpret_cast<const float4*>(p);
        v[0] = v4.x, v[1] = v4.y, v[2] = v4.z, v[3] = v4.w;
      } else {
        v[0] = p[0];
      }
#pragma unroll
      for (int e = 0; e < K; ++e) {
        acc[r][0] = fmaf(a[e], v[e], acc[r][0]);
        acc[r][1] = fmaf(b[e], v[e], acc[r][1]);
      }
    }
  }
  float zr = 0.f, zi = 0.f;
#pragma unroll
  for (int r = 0; r < LS_ROWS; ++r) {
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
      for (int o = LS_LANES / 2; o > 0; o >>= 1) acc[r][m] += __shfl_xor(acc[r][m], o, WAVE);
    if (lane == r) zr = acc[r][0], zi = acc[r][1];
  }
  if (lane >= rows) return;
  float a, b;
  lru_terms(zr + bias[c], zi + bias[W + c], slope[c], own, a, b);
  const float S = fmaf(a, S0, b);
  if (slot >= 0) state[(size_t)slot * W + c] = S;
  out[(size_t)row * W + c] = from_f32<T>(slot >= 0 ? S * gelu(y) : 0.f);
}

bool lru_sizes_ok(int W, int n) { return n > 0 && W > 0 && W % n == 0 && (long)(W / n) * ceil_div(n, LG_N) <= 65535 && ceil_div(W, 256) <= 65535; }

template <typename T>
int lru_finish_launch(const float* P, const float* Q, const float* ends, float* state, const float* z, long z_row, const float* z_bias,
                      void* out, const int* tok_seq, const int* cu_seqlens, const int* seq_slot, const int* seq_tile0, int T_, int W,
                      hipStream_t stream) {
  const bool vec = W % 4 == 0 && z_row % 4 == 0 && ((((uintptr_t)P) | ((uintptr_t)Q) | ((uintptr_t)ends) | ((uintptr_t)state) | ((uintptr_t)z) |
                                                     ((uintptr_t)z_bias) | ((uintptr_t)out)) & 15) == 0;
  if (vec)
    lru_finish_kernel<T, 4><<<dim3(T_, ceil_div(W, 1024)), 256, 0, stream>>>(P, Q, ends, state, z, z_row, z_bias, (T*)out, tok_seq,
                                                                            cu_seqlens, seq_slot, seq_tile0, W);
  else
    lru_finish_kernel<T, 1><<<dim3(T_, ceil_div(W, 256)), 256, 0, stream>>>(P, Q, ends, state, z, z_row, z_bias, (T*)out, tok_seq,
                                                                           cu_seqlens, seq_slot, seq_tile0, W);
  return launch_status();
}
}  // namespace

extern "C" int yalm_lru(const float* u, const void* w, int w_dtype, const float* bias, const float* slope, const float* z, long z_row,
                        const float* z_bias, float* state, float* P, float* Q, float* ends, const int* tok_seq,
                        const int* cu_seqlens, const int* seq_slot, const int* seq_tile0, int n_tiles, void* out, int out_dtype, int T,
                        int B, int W, int n, int force_simple, hipStream_t stream) {
  if (T <= 0 || B <= 0) return YALM_OK;
  const bool prompts = seq_tile0 != nullptr;
  if (!lru_sizes_ok(W, n) || z_row < W || B > 65535 || P == nullptr || Q == nullptr || (!prompts && T != B) ||
      (prompts && (ends == nullptr || n_tiles <= 0 || tok_seq == nullptr)))
    return YALM_ERR_ARG;
  if ((w_dtype != YALM_F32 && w_dtype != YALM_BF16) || (out_dtype != YALM_F32 && out_dtype != YALM_BF16)) return YALM_ERR_DTYPE;
  const LruArgs x = {u, bias, slope, P, Q, ends, cu_seqlens, seq_tile0, T, B, W, n};
  const dim3 grid(prompts ? n_tiles : ceil_div(T, LG_T), W / n * ceil_div(n, LG_N));
  if (w_dtype == YALM_F32)
    lru_gates_kernel<float><<<grid, LG_THREADS, 0, stream>>>(x, (const float*)w);
  else if (!force_simple && n % 8 == 0 && ((((uintptr_t)u) | ((uintptr_t)w)) & 15) == 0)
    lru_gates_mfma_kernel<<<grid, LG_THREADS, 0, stream>>>(x, (const bf16*)w);
  else
    lru_gates_kernel<bf16><<<grid, LG_THREADS, 0, stream>>>(x, (const bf16*)w);
  if (prompts)
    lru_carry_kernel<<<dim3(ceil_div(W, WAVE), B), WAVE, 0, stream>>>(ends, state, cu_seqlens, seq_slot, seq_tile0, W);
  int rc = launch_status();
  if (rc != YALM_OK) return rc;
  if (out_dtype == YALM_F32)
    return lru_finish_launch<float>(P, Q, ends, state, z, z_row, z_bias, out, tok_seq, cu_seqlens, seq_slot, seq_tile0, T, W, stream);
  return lru_finish_launch<bf16>(P, Q, ends, state, z, z_row, z_bias, out, tok_seq, cu_seqlens, seq_slot, seq_tile0, T, W, stream);
}

extern "C" int yalm_lru_step(const float* u, const void* w, int w_dtype, const float* bias, const float* slope, const float* z,
                             long z_row, const float* z_bias, float* state, const int* seq_slot, void* out, int out_dtype, int B, int W,
                             int n, hipStream_t stream) {
  if (B <= 0) return YALM_OK;
  if (!lru_sizes_ok(W, n) || z_row < W || ceil_div(B, LS_ROWS) > 65535) return YALM_ERR_ARG;
  if ((w_dtype != YALM_F32 && w_dtype != YALM_BF16) || (out_dtype != YALM_F32 && out_dtype != YALM_BF16)) return YALM_ERR_DTYPE;
  const dim3 grid(ceil_div(W, LS_CH), ceil_div(B, LS_ROWS));
  const bool vec = n % 4 == 0 && ((((uintptr_t)u) | ((uintptr_t)w)) & 15) == 0;
#define STEP(TW_, TO_, V_) \
  lru_step_kernel<TW_, TO_, V_><<<grid, 256, 0, stream>>>(u, (const TW_*)w, bias, slope, z, z_row, z_bias, state, seq_slot, (TO_*)out, B, W, n)
#define STEP_V(TW_, TO_) do { if (vec) STEP(TW_, TO_, true); else STEP(TW_, TO_, false); } while (0)
  if (w_dtype == YALM_F32) {
    if (out_dtype == YALM_F32) STEP_V(float, float);
    else STEP_V(float, bf16);
  } else {
    if (out_dtype == YALM_F32) STEP_V(bf16, float);
    else STEP_V(bf16, bf16);
  }
#undef STEP_V
#undef STEP
  return launch_status();
}
