// Gated linear attention: per head, with the state S [d, dv] in float32,
//     f = sigmoid(z)^(1 / tau),  z = W_2 (W_1 h) + b     (a decay per head and key channel, by a low-rank product)
//     S <- diag(f) S + k v^T,   o = S^T (q_scale q)
// and each head's o is divided by its root mean square over dv, multiplied by a weight shared by the heads and by
// silu(g).  Everything behind the projections q | k | v | g | W_1 h (float32) is float32, W_2's product included: a
// thread that forms a row of f keeps that row of W_2 (its first 16 elements) in registers and reads a token's W_1 h
// from LDS.  The power of the sigmoid is exp(-softplus(-z) / tau), so that neither end of z loses digits.  The walk
// over the tokens is diag_scan.h's.
#include "diag_scan.h"
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
    const float softplus = fmaxf(-z, 0.f) + log1pf(expf(-fabsf(z)));      // -ln sigmoid(z)
    f = expf(-softplus * inv_tau);
    q = x[0] * q_scale;
    k = x[1];
  }
  __device__ float value(int t, int h, int j) const { return proj[(size_t)t * N + 2 * Hd + h * dv + j]; }
  __device__ int low_size() const { return rank; }
  __device__ float low(int t, int i) const { return proj[(size_t)t * N + 2 * Hd + 2 * Hv + i]; }
};
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
  if (d <= 32) SCAN(4, 8, 2, 8);
  else if (d <= 64) SCAN(4, 16, 2, 8);
  else if (d <= 128) SCAN(4, 32, 2, 8);
  else SCAN(8, 32, 2, 8);
#undef SCAN
  if (rc != YALM_OK) return rc;
  return heads_norm_launch(raw, w_norm, proj + 2 * Hd + Hv, N, out, T, n_heads, dv, eps, out_dtype, stream);
}
