// Gated linear attention: per head, with the state S [d, dv] in float32,
//     f = sigmoid(z)^(1 / tau),  z = W_2 (W_1 h) + b     (a decay per head and key channel, by a low-rank product)
//     S <- diag(f) S + k v^T,   o = S^T (q_scale q)
// and each head's o is divided by its root mean square over dv, multiplied by a weight shared by the heads and by
// silu(g).  Everything behind the projections q | k | v | g | W_1 h (float32) is float32, W_2's product included: a
// thread that forms a row of f keeps that row of W_2 (its first 16 elements) in registers and reads a token's W_1 h
// from LDS.  The power of the sigmoid is exp(-softplus(-z) / tau), so that neither end of z loses digits.  The walk
// over the tokens is diag_scan.h's.
//
// Prompts go a tile of 64 tokens at a time on the matrix cores, in float32 (v_mfma_f32_16x16x4_f32).  With L_t the sum of
// ln f over the tile's tokens up to and including t (a number a channel),
//     o_t = (q_t e^L_t) S_0 + sum over s <= t of (sum over channels of q_t k_s e^(L_t - L_s)) v_s,
//     S_64 = diag(e^L_63) S_0 + sum over s of (k_s e^(L_63 - L_s)) v_s^T.
// gla_tiles_kernel (every tile and head at once): the decays and their sums, the three scaled operands above, and the
// second sum of o.  No e^(-L) is ever formed, whatever the decays: the tile is cut into four blocks of 16 tokens;
// between blocks the exponent is split at the blocks' borders into parts that are each <= 0, and inside a block every
// (t, s, channel) has its own e^(L_t - L_s).  scan_carry_kernel (a workgroup 16 columns of a head, the tiles in order): the
// products with S_0 and the state (tile_scan.h).
#include "tile_scan.h"
#include "yalm_hip.h"

namespace {
constexpr int GLA_ROW_LOW = 16;                  // elements of W_2's row in registers; longer rows go on in memory

struct GlaOp {
  static constexpr bool KEYS = true, LOW = true;
  struct Row {
    float w2[GLA_ROW_LOW];
    const float* rest;
    float bias;
  };
  const float* proj;
  const float* w2;                               // [heads * d, padded rank], zeros behind the rank
  const float* bias;                             // [heads * d]
  int Hd, Hv, N, d, dv, rank;
  float q_scale, inv_tau;
  __device__ int padded() const { return (rank + 3) / 4 * 4; }
  __device__ Row begin(int h, int r, bool ok) const {
    Row m;
    m.rest = w2 + (size_t)(ok ? h * d + r : 0) * padded();
#pragma unroll
    for (int i = 0; i < GLA_ROW_LOW; ++i) m.w2[i] = i < padded() ? m.rest[i] : 0.f;
    m.bias = ok ? bias[h * d + r] : 0.f;
    return m;
  }
  __device__ void fetch(int t, int h, int r, float* z) const {
    z[0] = proj[(size_t)t * N + h * d + r];
    z[1] = proj[(size_t)t * N + Hd + h * d + r];
  }
  __device__ void form(const Row& m, const float* x, const float* low, float& q, float& f, float& k) const {
    const int rp = padded();
    float z = m.bias;
#pragma unroll
    for (int i = 0; i < GLA_ROW_LOW; i += 4) {
      if (i < rp) {
        const float4 a = *reinterpret_cast<const float4*>(low + i);
        z = fmaf(m.w2[i], a.x, fmaf(m.w2[i + 1], a.y, fmaf(m.w2[i + 2], a.z, fmaf(m.w2[i + 3], a.w, z))));
      }
    }
    for (int i = GLA_ROW_LOW; i < rp; i += 4) {
      const float4 a = *reinterpret_cast<const float4*>(low + i), w = *reinterpret_cast<const float4*>(m.rest + i);
      z = fmaf(w.x, a.x, fmaf(w.y, a.y, fmaf(w.z, a.z, fmaf(w.w, a.w, z))));
    }
    // -ln sigmoid(z) = max(-z, 0) + ln(1 + e^-|z|): an error of it is an error of f in proportion, so that the rounding of
    // 1 + e^-|z| is no more than that of f itself
    const float softplus = fmaxf(-z, 0.f) + __logf(1.0f + __expf(-fabsf(z)));
    f = __expf(-softplus * inv_tau);
    q = x[0] * q_scale;
    k = x[1];
  }
  __device__ float value(int t, int h, int j) const { return proj[(size_t)t * N + 2 * Hd + h * dv + j]; }
  __device__ static float act(float v) { return v; }
  __device__ int low_size() const { return rank; }
  __device__ float low(int t, int i) const { return proj[(size_t)t * N + 2 * Hd + 2 * Hv + i]; }
};
}  // namespace

namespace {
constexpr int GLA_TILES_LDS = 160 * 1024;

// qd [tile][head][64][DP] = q e^L, kd [tile][head][DP][64] = k e^(L_63 - L), gd [tile][head][DP] = e^L_63; raw = the second
// sum of o.  A thread owns one channel of one block of 16 tokens.
template <int DP>
__global__ __launch_bounds__(GNB * DP) void gla_tiles_kernel(GlaOp op, float* __restrict__ raw, float* __restrict__ qd,
                                                             float* __restrict__ kd, float* __restrict__ gd,
                                                             const int* __restrict__ cu_seqlens, const int* __restrict__ seq_tile0,
                                                             int B, int n_heads) {
  constexpr int ROW = DP + 4, NWAVES = GNB * DP / WAVE;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* s_q = lds;                               // [64][ROW]  q
  float* s_k = s_q + GT * ROW;                    // [64][ROW]  k
  float* s_c = s_k + GT * ROW;                    // [64][ROW]  the sums of log2 f from the token's block's start
  float* s_base = s_c + GT * ROW;                 // [5][DP]    the same at the blocks' borders, from the tile's start
  float* s_a = s_base + (GNB + 1) * DP;           // [64][GA_ROW] scores; before them the tokens' short vectors [64][rp]
  const int gt = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int b = seq_of_tile(seq_tile0, B, gt);
  const int p0 = (gt - seq_tile0[b]) * GT, first = cu_seqlens[b] + p0, n = min(GT, cu_seqlens[b + 1] - first);
  if (n <= 0) return;
  const int ch = tid % DP, sb = tid / DP, wave = tid / WAVE, lane = tid % WAVE, li = lane % 16, lq = lane / 16;
  const int d = op.d, dv = op.dv, N = op.N, rp = op.padded();
  const bool ch_ok = ch < d;
  // the block's values, in the order of the last product's operand: asked for first, needed last
  const int n_cols = (dv + 15) / 16;
  float vb[GT / 4];
  auto load_values = [&](int col) {
    const int j = col * 16 + li;
#pragma unroll
    for (int i = 0; i < GT / 4; ++i) {
      const int s = 16 * (i / 4) + 4 * lq + i % 4;
      vb[i] = j < dv && s < n ? op.value(first + s, h, j) : 0.f;
    }
  };
  for (int i = tid; i < GT * rp; i += GNB * DP) {
    const int t = i / rp, e = i % rp;
    s_a[i] = t < n && e < op.rank ? op.low(first + t, e) : 0.f;
  }
  float q[GB], k[GB], c[GB];
#pragma unroll
  for (int u = 0; u < GB; ++u) {
    const int t = sb * GB + u;
    const bool ok = ch_ok && t < n;
    const float* row = op.proj + (size_t)(first + t) * N + h * d + ch;
    q[u] = ok ? row[0] * op.q_scale : 0.f;
    k[u] = ok ? row[op.Hd] : 0.f;
  }
  if (wave < n_cols) load_values(wave);
  lds_barrier();
  {
    const float* w = op.w2 + (size_t)(ch_ok ? h * d + ch : 0) * rp;
    const float bias = ch_ok ? op.bias[h * d + ch] : 0.f;
#pragma unroll
    for (int u = 0; u < GB; ++u) c[u] = bias;
    for (int i = 0; i < rp; i += 4) {
      const float4 w4 = *reinterpret_cast<const float4*>(w + i);
#pragma unroll
      for (int u = 0; u < GB; ++u) {
        const float4 a = *reinterpret_cast<const float4*>(s_a + (sb * GB + u) * rp + i);
        c[u] = fmaf(w4.x, a.x, fmaf(w4.y, a.y, fmaf(w4.z, a.z, fmaf(w4.w, a.w, c[u]))));
      }
    }
    float sum = 0.f;
#pragma unroll
    for (int u = 0; u < GB; ++u) {
      const float softplus = fmaxf(-c[u], 0.f) + __logf(1.0f + __expf(-fabsf(c[u])));
      sum += ch_ok && sb * GB + u < n ? -softplus * op.inv_tau * 1.4426950408889634f : 0.f;
      c[u] = sum;
    }
    s_base[(sb + 1) * DP + ch] = sum;             // the block's own sum, added up below
#pragma unroll
    for (int u = 0; u < GB; ++u) {
      const int at = (sb * GB + u) * ROW + ch;
      s_q[at] = q[u], s_k[at] = k[u], s_c[at] = c[u];
    }
  }
  lds_barrier();
  float base[GNB + 1];                            // log2 of the decay from the tile's start to the blocks' borders
  base[0] = 0.f;
#pragma unroll
  for (int i = 1; i <= GNB; ++i) base[i] = base[i - 1] + s_base[i * DP + ch];
  float mine = 0.f, after = 0.f;                  // up to this thread's block; from its end to the tile's end
#pragma unroll
  for (int i = 0; i < GNB; ++i) {
    if (i < sb) mine = base[i + 1];
    if (i > sb) after += s_base[(i + 1) * DP + ch];
  }
  lds_barrier();                                // the blocks' sums are read: the borders' take their place
  if (sb == 0) {
#pragma unroll
    for (int i = 0; i <= GNB; ++i) s_base[i * DP + ch] = base[i];
  }
  {
    const size_t at = (size_t)gt * n_heads + h;
    float* qo = qd + (at * GT + sb * GB) * DP + ch;
    float* ko = kd + (at * DP + ch) * GT + sb * GB;
#pragma unroll
    for (int u = 0; u < GB; ++u) qo[(size_t)u * DP] = q[u] * exp2f(mine + c[u]);
    const float end = c[GB - 1];
#pragma unroll
    for (int u = 0; u < GB; u += 4) {
      float4 o;
      o.x = k[u] * exp2f(end - c[u] + after);
      o.y = k[u + 1] * exp2f(end - c[u + 1] + after);
      o.z = k[u + 2] * exp2f(end - c[u + 2] + after);
      o.w = k[u + 3] * exp2f(end - c[u + 3] + after);
      *reinterpret_cast<float4*>(ko + u) = o;
    }
    if (sb == 0) gd[at * DP + ch] = exp2f(base[GNB]);
  }
  lds_barrier();
  // scores inside a block: a thread a pair t > s
  for (int p = ch; p < GB * (GB - 1) / 2; p += DP) {
    int t = (int)((1.0f + sqrtf(1.0f + 8.0f * (float)p)) * 0.5f);
    if (t * (t - 1) / 2 > p) --t;
    if (t * (t + 1) / 2 <= p) ++t;
    const int rt = sb * GB + t, rs = sb * GB + p - t * (t - 1) / 2;
    float acc0 = 0.f, acc1 = 0.f;
#pragma unroll 2
    for (int i = 0; i < DP; i += 4) {
      const float4 a = *reinterpret_cast<const float4*>(s_q + rt * ROW + i), x = *reinterpret_cast<const float4*>(s_k + rs * ROW + i);
      const float4 ct = *reinterpret_cast<const float4*>(s_c + rt * ROW + i), cs = *reinterpret_cast<const float4*>(s_c + rs * ROW + i);
      acc0 = fmaf(a.x * x.x, __builtin_amdgcn_exp2f(ct.x - cs.x), acc0);
      acc1 = fmaf(a.y * x.y, __builtin_amdgcn_exp2f(ct.y - cs.y), acc1);
      acc0 = fmaf(a.z * x.z, __builtin_amdgcn_exp2f(ct.z - cs.z), acc0);
      acc1 = fmaf(a.w * x.w, __builtin_amdgcn_exp2f(ct.w - cs.w), acc1);
    }
    s_a[rt * GA_ROW + rs] = acc0 + acc1;
    s_a[rs * GA_ROW + rt] = 0.f;                  // s does not see t
  }
  {                                               // a token on itself, where the exponent is 0: DP / 16 lanes a token, 16 channels a lane
    constexpr int LT = DP / GB;
    const int rt = sb * GB + ch / LT;
    float acc = 0.f;
#pragma unroll
    for (int i = 0; i < 16; i += 4) {
      const int e = (ch % LT) * 16 + i;
      const float4 a = *reinterpret_cast<const float4*>(s_q + rt * ROW + e), x = *reinterpret_cast<const float4*>(s_k + rt * ROW + e);
      acc += (a.x * x.x + a.y * x.y) + (a.z * x.z + a.w * x.w);
    }
#pragma unroll
    for (int o = LT / 2; o > 0; o >>= 1) acc += __shfl_xor(acc, o, WAVE);
    if (ch % LT == 0) s_a[rt * GA_ROW + rt] = acc;
  }
  // scores between blocks i > j: (q e^(L_t - border i)) (e^(border i - border j + 1)) (k e^(border j + 1 - L_s))
  for (int p = wave; p < GNB * (GNB - 1) / 2; p += NWAVES) {
    const int i = p < 1 ? 1 : p < 3 ? 2 : 3, j = p - i * (i - 1) / 2;
    const int rt = i * GB + li, rs = j * GB + li;
    gf32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
    for (int m = 0; m < DP / 16; ++m) {
      const int e = 16 * m + 4 * lq;
      const float4 a = *reinterpret_cast<const float4*>(s_q + rt * ROW + e), x = *reinterpret_cast<const float4*>(s_k + rs * ROW + e);
      const float4 ct = *reinterpret_cast<const float4*>(s_c + rt * ROW + e), cs = *reinterpret_cast<const float4*>(s_c + rs * ROW + e);
      const float4 bi = *reinterpret_cast<const float4*>(s_base + i * DP + e), bj = *reinterpret_cast<const float4*>(s_base + (j + 1) * DP + e);
      const float4 ej = *reinterpret_cast<const float4*>(s_c + (j * GB + GB - 1) * ROW + e);
#pragma unroll
      for (int r = 0; r < 4; ++r)
        acc = mfma4(el(a, r) * __builtin_amdgcn_exp2f(el(ct, r) + (el(bi, r) - el(bj, r))),
                    el(x, r) * __builtin_amdgcn_exp2f(el(ej, r) - el(cs, r)), acc);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) s_a[(i * GB + 4 * lq + r) * GA_ROW + j * GB + li] = acc[r];
  }
  lds_barrier();
  for (int col = wave; col < n_cols; col += NWAVES) {
    if (col != wave) load_values(col);
    const int j = col * 16 + li;
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

size_t gla_tiles_lds(int dp, int rank) {
  const int rp = (rank + 3) / 4 * 4;
  return ((size_t)3 * GT * (dp + 4) + (GNB + 1) * dp + (size_t)GT * (rp > GA_ROW ? rp : GA_ROW)) * sizeof(float);
}

int gla_padded_dim(int d) { return d <= 32 ? 32 : d <= 64 ? 64 : d <= 128 ? 128 : 0; }

template <int DP>
int gla_tiles_launch(const GlaOp& op, float* state, float* raw, float* qd, float* kd, float* gd, const int* cu_seqlens,
                     const int* seq_slot, const int* seq_tile0, int n_tiles, int B, int n_heads, hipStream_t stream) {
  static LdsAllowance allowance;
  const size_t lds = gla_tiles_lds(DP, op.rank);
  int rc = allow_dynamic_lds(allowance, reinterpret_cast<const void*>(gla_tiles_kernel<DP>), GLA_TILES_LDS);
  if (rc != YALM_OK) return rc;
  gla_tiles_kernel<DP><<<dim3(n_tiles, n_heads), GNB * DP, lds, stream>>>(op, raw, qd, kd, gd, cu_seqlens, seq_tile0, B, n_heads);
  rc = launch_status();
  if (rc != YALM_OK) return rc;
  return scan_carry_launch<DP>(op, state, raw, qd, kd, gd, cu_seqlens, seq_slot, seq_tile0, B, n_heads, stream);
}
}  // namespace

extern "C" int yalm_gla(const float* proj, const float* w2, const float* bias, const float* w_norm, float* state, float* raw,
                        const int* cu_seqlens, const int* seq_slot, void* out, int T, int B, int n_heads, int d, int dv, int rank,
                        float q_scale, float inv_tau, float eps, int out_dtype, hipStream_t stream) {
  if (T <= 0 || B <= 0) return YALM_OK;
  if (n_heads <= 0 || d <= 0 || d > 256 || dv <= 0 || rank <= 0 || rank > 256 || (((uintptr_t)w2) & 15)) return YALM_ERR_ARG;
  if (out_dtype != YALM_F32 && out_dtype != YALM_BF16) return YALM_ERR_DTYPE;
  const int Hd = n_heads * d, Hv = n_heads * dv, N = 2 * Hd + 2 * Hv + rank;
  const GlaOp op = {proj, w2, bias, Hd, Hv, N, d, dv, rank, q_scale, inv_tau};
  const size_t low = (size_t)((rank + 3) / 4 * 4);
  int rc;
#define SCAN(NR_, LANES_, NC_, TOK_) \
  rc = diag_scan_launch<GlaOp, NR_, LANES_, NC_, TOK_>(op, state, raw, cu_seqlens, seq_slot, B, n_heads, d, dv, low, stream)
  // steps of single tokens: more columns a workgroup, which then forms a head's operands less often
  if (d <= 32) SCAN(4, 8, 2, 8);
  else if (d <= 64) SCAN(4, 16, 2, 8);
  else if (d <= 128 && T == B) SCAN(8, 16, 4, 8);
  else if (d <= 128) SCAN(8, 16, 1, 16);
  else SCAN(8, 32, 2, 8);
#undef SCAN
  if (rc != YALM_OK) return rc;
  return heads_norm_launch(raw, w_norm, proj + 2 * Hd + Hv, N, out, T, n_heads, dv, eps, out_dtype, stream);
}

extern "C" int yalm_gla_tiles_fit(int d, int rank) {
  const int dp = gla_padded_dim(d);
  return d > 0 && dp > 0 && rank > 0 && gla_tiles_lds(dp, rank) <= GLA_TILES_LDS ? dp : 0;
}

extern "C" int yalm_gla_tiles(const float* proj, const float* w2, const float* bias, const float* w_norm, float* state, float* raw,
                              float* qd, float* kd, float* gd, const int* cu_seqlens, const int* seq_slot, const int* seq_tile0,
                              int n_tiles, void* out, int T, int B, int n_heads, int d, int dv, int rank, float q_scale,
                              float inv_tau, float eps, int out_dtype, hipStream_t stream) {
  if (T <= 0 || B <= 0 || n_tiles <= 0) return YALM_OK;
  const int dp = yalm_gla_tiles_fit(d, rank);
  if (n_heads <= 0 || n_heads > 65535 || B > 65535 || dv <= 0 || ceil_div(dv, 16) > 65535 || dp == 0 ||
      ((((uintptr_t)w2) | ((uintptr_t)qd) | ((uintptr_t)kd) | ((uintptr_t)gd)) & 15))
    return YALM_ERR_ARG;
  if (out_dtype != YALM_F32 && out_dtype != YALM_BF16) return YALM_ERR_DTYPE;
  const int Hd = n_heads * d, Hv = n_heads * dv, N = 2 * Hd + 2 * Hv + rank;
  const GlaOp op = {proj, w2, bias, Hd, Hv, N, d, dv, rank, q_scale, inv_tau};
  const int rc = dp == 32   ? gla_tiles_launch<32>(op, state, raw, qd, kd, gd, cu_seqlens, seq_slot, seq_tile0, n_tiles, B, n_heads, stream)
                 : dp == 64 ? gla_tiles_launch<64>(op, state, raw, qd, kd, gd, cu_seqlens, seq_slot, seq_tile0, n_tiles, B, n_heads, stream)
                            : gla_tiles_launch<128>(op, state, raw, qd, kd, gd, cu_seqlens, seq_slot, seq_tile0, n_tiles, B, n_heads, stream);
  if (rc != YALM_OK) return rc;
  return heads_norm_launch(raw, w_norm, proj + 2 * Hd + Hv, N, out, T, n_heads, dv, eps, out_dtype, stream);
}
