// Linear attention under a decay of one fixed number a head (lightning attention): per head, with the state S [d, dv] in
// float32,
//     q = silu(z_q),  k = silu(z_k),  v = silu(z_v)
//     S <- g S + k v^T,   o = S^T q
// from the projections z_q | z_k | z_v (float32, columns of a wider row).  Everything behind the projections is float32.
// Single tokens and sizes that the tiles do not take: diag_scan.h's walk.
//
// Prompts go a tile of 64 tokens at a time on the matrix cores, in float32: with n the tile's tokens,
//     o_t = g^(t + 1) S_0^T q_t + sum over s <= t of g^(t - s) (q_t . k_s) v_s,
//     S_n = g^n S_0 + sum over s of g^(n - 1 - s) k_s v_s^T.
// No power below the zeroth is ever formed; the powers g^0 .. g^64 of every head are a table (made in float64), so that a decay
// of one, or one close to it, loses nothing.  lightning_tiles_kernel (every tile and head at once) makes the second sum of o and the scaled
// queries and keys; tile_scan.h's walk over the tiles the products with S_0 and the state.
#include "tile_scan.h"
#include "yalm_hip.h"

namespace {
constexpr int LT_POWERS = GT + 1;                // of a head: g^0 .. g^64
constexpr int LT_THREADS = 256, LT_NWAVES = LT_THREADS / WAVE;

// z sigmoid(z); the reciprocal instruction is good to one unit in the last place
__device__ __forceinline__ float fast_silu(float z) { return z * __builtin_amdgcn_rcpf(1.0f + __expf(-z)); }

struct LightningOp {
  static constexpr bool KEYS = true, LOW = false;
  struct Row { float f; };
  const float* proj;                             // z_q | z_k | z_v at its first columns
  const float* powers;                           // [heads][LT_POWERS]
  long row;                                      // elements of a row
  int Hd, Hv, d, dv;
  __device__ Row begin(int h, int, bool) const { return {powers[h * LT_POWERS + 1]}; }
  __device__ void fetch(int t, int h, int r, float* z) const {
    z[0] = proj[(size_t)t * row + h * d + r];
    z[1] = proj[(size_t)t * row + Hd + h * d + r];
  }
  __device__ void form(const Row& m, const float* z, const float*, float& q, float& f, float& k) const {
    q = fast_silu(z[0]);
    k = fast_silu(z[1]);
    f = m.f;
  }
  __device__ float value(int t, int h, int j) const { return proj[(size_t)t * row + 2 * Hd + h * dv + j]; }
  __device__ static float act(float v) { return fast_silu(v); }
  __device__ int low_size() const { return 0; }
  __device__ float low(int, int) const { return 0.f; }
};

// qd [tile][head][64][DP], kd [tile][head][DP][64] and gd [tile][head][DP] as tile_scan.h wants them; raw = the second sum
// of o.  VEC: heads, rows and addresses allow loads of four elements.
template <int DP, bool VEC>
__global__ __launch_bounds__(LT_THREADS) void lightning_tiles_kernel(LightningOp op, float* __restrict__ raw, float* __restrict__ qd,
                                                                     float* __restrict__ kd, float* __restrict__ gd,
                                                                     const int* __restrict__ cu_seqlens,
                                                                     const int* __restrict__ seq_tile0, int B, int n_heads) {
  constexpr int ROW = DP + 4;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* s_q = lds;                               // [64][ROW]
  float* s_k = s_q + GT * ROW;                    // [64][ROW]
  __shared__ __attribute__((aligned(16))) float s_a[GT * GA_ROW];      // scores [64][GA_ROW]
  __shared__ float s_pow[LT_POWERS];
  const int gt = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int b = seq_of_tile(seq_tile0, B, gt);
  const int p0 = (gt - seq_tile0[b]) * GT, first = cu_seqlens[b] + p0, n = min(GT, cu_seqlens[b + 1] - first);
  if (n <= 0) return;
  const int wave = tid / WAVE, lane = tid % WAVE, li = lane % 16, lq = lane / 16;
  const int d = op.d, dv = op.dv;
  for (int i = tid; i < LT_POWERS; i += LT_THREADS) s_pow[i] = op.powers[h * LT_POWERS + i];
  // the first columns' values, in the order of the last product's operand: asked for first, needed last
  const int n_cols = (dv + 15) / 16;
  float vb[GT / 4];
  auto load_values = [&](int col) {
    const int j = col * 16 + li;
#pragma unroll
    for (int i = 0; i < GT / 4; ++i) {
      const int s = 16 * (i / 4) + 4 * lq + i % 4;
      vb[i] = op.value(first + min(s, n - 1), h, min(j, dv - 1));      // behind the text the score is zero
    }
  };
  constexpr int PER = GT * DP / 4 / LT_THREADS;    // runs of four elements a thread and operand
  float4 q4[PER], k4[PER];
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int at = tid + i * LT_THREADS, t = at / (DP / 4), e = at % (DP / 4) * 4;
    const float* src = op.proj + (size_t)(first + t) * op.row + h * d + e;
    q4[i] = k4[i] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (t < n) {
      if constexpr (VEC) {
        if (e < d) {
          q4[i] = *reinterpret_cast<const float4*>(src);
          k4[i] = *reinterpret_cast<const float4*>(src + op.Hd);
        }
      } else {
        float q[4] = {0.f, 0.f, 0.f, 0.f}, k[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int u = 0; u < 4; ++u)
          if (e + u < d) q[u] = src[u], k[u] = src[op.Hd + u];
        q4[i] = make_float4(q[0], q[1], q[2], q[3]), k4[i] = make_float4(k[0], k[1], k[2], k[3]);
      }
    }
  }
  if (wave < n_cols) load_values(wave);
  lds_barrier();                                  // the powers
  const size_t at_h = (size_t)gt * n_heads + h;
#pragma unroll
  for (int i = 0; i < PER; ++i) {                 // silu(0) = 0: what lies behind the text and behind d stays zero
    const int at = tid + i * LT_THREADS, t = at / (DP / 4), e = at % (DP / 4) * 4;
    const float4 q = make_float4(fast_silu(q4[i].x), fast_silu(q4[i].y), fast_silu(q4[i].z), fast_silu(q4[i].w));
    const float4 k = make_float4(fast_silu(k4[i].x), fast_silu(k4[i].y), fast_silu(k4[i].z), fast_silu(k4[i].w));
    *reinterpret_cast<float4*>(s_q + t * ROW + e) = q;
    *reinterpret_cast<float4*>(s_k + t * ROW + e) = k;
    const float g = s_pow[t + 1];
    *reinterpret_cast<float4*>(qd + (at_h * GT + t) * DP + e) = make_float4(q.x * g, q.y * g, q.z * g, q.w * g);
  }
  for (int e = tid; e < DP; e += LT_THREADS) gd[at_h * DP + e] = s_pow[n];
  lds_barrier();
#pragma unroll 2
  for (int at = tid; at < DP * GT / 4; at += LT_THREADS) {
    const int e = at / (GT / 4), t = at % (GT / 4) * 4;
    float k[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) k[u] = t + u < n ? s_k[(t + u) * ROW + e] * s_pow[n - 1 - t - u] : 0.f;
    *reinterpret_cast<float4*>(kd + (at_h * DP + e) * GT + t) = make_float4(k[0], k[1], k[2], k[3]);
  }
  // scores: wave w the rows of block w (a tile has as many blocks as the workgroup waves)
  static_assert(GNB == LT_NWAVES, "");
  for (int j = 0; j <= wave; ++j) {
    gf32x4 acc[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll 2
    for (int m = 0; m < DP / 16; ++m) {
      const int e = 16 * m + 4 * lq;
      const float4 a = *reinterpret_cast<const float4*>(s_q + (wave * GB + li) * ROW + e);
      const float4 x = *reinterpret_cast<const float4*>(s_k + (j * GB + li) * ROW + e);
#pragma unroll
      for (int r = 0; r < 4; ++r) acc[r & 1] = mfma4(el(a, r), el(x, r), acc[r & 1]);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = wave * GB + 4 * lq + r, s = j * GB + li;
      s_a[t * GA_ROW + s] = s <= t ? (acc[0][r] + acc[1][r]) * s_pow[t - s] : 0.f;
    }
  }
  lds_barrier();
  for (int col = wave; col < n_cols; col += LT_NWAVES) {
    if (col != wave) load_values(col);
    const int j = col * 16 + li;
#pragma unroll
    for (int i = 0; i < GT / 4; ++i) vb[i] = fast_silu(vb[i]);
#pragma unroll
    for (int i = 0; i < GNB; ++i) {
      gf32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int m = 0; m <= i; ++m) {
        const float4 a = *reinterpret_cast<const float4*>(s_a + (i * GB + li) * GA_ROW + 16 * m + 4 * lq);
#pragma unroll
        for (int r = 0; r < 4; ++r) acc = mfma4(el(a, r), vb[4 * m + r], acc);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = i * GB + 4 * lq + r;
        if (t < n && j < dv) raw[(size_t)(first + t) * op.Hv + h * dv + j] = acc[r];
      }
    }
  }
}

int lightning_padded_dim(int d) { return d <= 32 ? 32 : d <= 64 ? 64 : d <= 128 ? 128 : 0; }

template <int DP>
int lightning_tiles_launch(const LightningOp& op, bool vec, float* state, float* raw, float* qd, float* kd, float* gd,
                           const int* cu_seqlens, const int* seq_slot, const int* seq_tile0, int n_tiles, int B, int n_heads,
                           hipStream_t stream) {
  constexpr size_t lds = (size_t)2 * GT * (DP + 4) * sizeof(float);
  static LdsAllowance allowance[2];
  const void* kernel = vec ? reinterpret_cast<const void*>(lightning_tiles_kernel<DP, true>)
                           : reinterpret_cast<const void*>(lightning_tiles_kernel<DP, false>);
  int rc = allow_dynamic_lds(allowance[vec], kernel, (int)lds);
  if (rc != YALM_OK) return rc;
  const dim3 grid(n_tiles, n_heads);
  if (vec) lightning_tiles_kernel<DP, true><<<grid, LT_THREADS, lds, stream>>>(op, raw, qd, kd, gd, cu_seqlens, seq_tile0, B, n_heads);
  else lightning_tiles_kernel<DP, false><<<grid, LT_THREADS, lds, stream>>>(op, raw, qd, kd, gd, cu_seqlens, seq_tile0, B, n_heads);
  rc = launch_status();
  if (rc != YALM_OK) return rc;
  return scan_carry_launch<DP>(op, state, raw, qd, kd, gd, cu_seqlens, seq_slot, seq_tile0, B, n_heads, stream);
}
}  // namespace

extern "C" int yalm_lightning(const float* proj, long row, const float* powers, float* state, float* raw, const int* cu_seqlens,
                              const int* seq_slot, int T, int B, int n_heads, int d, int dv, hipStream_t stream) {
  if (T <= 0 || B <= 0) return YALM_OK;
  if (n_heads <= 0 || d <= 0 || d > 256 || dv <= 0 || row < (long)n_heads * (2 * d + dv)) return YALM_ERR_ARG;
  const LightningOp op = {proj, powers, row, n_heads * d, n_heads * dv, d, dv};
#define SCAN(NR_, LANES_, NC_, TOK_) \
  return diag_scan_launch<LightningOp, NR_, LANES_, NC_, TOK_>(op, state, raw, cu_seqlens, seq_slot, B, n_heads, d, dv, 0, stream)
  // steps of single tokens: more columns a workgroup, which then forms a head's operands less often
  if (d <= 32) SCAN(4, 8, 2, 8);
  if (d <= 64) SCAN(4, 16, 2, 8);
  if (d <= 128 && T == B) SCAN(8, 16, 4, 8);
  if (d <= 128) SCAN(8, 16, 1, 16);
  SCAN(8, 32, 2, 8);
#undef SCAN
}

extern "C" int yalm_lightning_tiles_fit(int d) { return d > 0 ? lightning_padded_dim(d) : 0; }

extern "C" int yalm_lightning_tiles(const float* proj, long row, const float* powers, float* state, float* raw, float* qd, float* kd,
                                    float* gd, const int* cu_seqlens, const int* seq_slot, const int* seq_tile0, int n_tiles, int T,
                                    int B, int n_heads, int d, int dv, hipStream_t stream) {
  if (T <= 0 || B <= 0 || n_tiles <= 0) return YALM_OK;
  const int dp = yalm_lightning_tiles_fit(d);
  if (n_heads <= 0 || n_heads > 65535 || B > 65535 || dv <= 0 || ceil_div(dv, 16) > 65535 || dp == 0 ||
      row < (long)n_heads * (2 * d + dv) || ((((uintptr_t)qd) | ((uintptr_t)kd) | ((uintptr_t)gd)) & 15))
    return YALM_ERR_ARG;
  const LightningOp op = {proj, powers, row, n_heads * d, n_heads * dv, d, dv};
  const bool vec = d % 4 == 0 && row % 4 == 0 && (((uintptr_t)proj) & 15) == 0;
#define TILES(DP_) return lightning_tiles_launch<DP_>(op, vec, state, raw, qd, kd, gd, cu_seqlens, seq_slot, seq_tile0, n_tiles, B, n_heads, stream)
  if (dp == 32) TILES(32);
  if (dp == 64) TILES(64);
  TILES(128);
#undef TILES
}
