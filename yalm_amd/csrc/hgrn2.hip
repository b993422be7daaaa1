// The gated linear recurrence whose forget gate also decides what is written (HGRN2).  Per head, with the state S
// [d, dv] in float32:
//     q = silu(z_q),  f = l + (1 - l) sigmoid(z_f + b)          (l the gate's lower bound, per head and channel)
//     S <- diag(f) S + (1 - f) v^T,   o = S^T q
// and each head's o is divided by its root mean square over dv and multiplied by a weight shared by the heads.
// Everything behind the projections z_q | z_f | v (float32) is float32; the walk over the tokens is diag_scan.h's.
#include "diag_scan.h"
#include "yalm_hip.h"

namespace {
struct Hgrn2Op {
  static constexpr bool KEYS = false, LOW = false;
  struct Row { float bias, lower; };
  const float* proj;
  const float* f_bias;
  const float* lower;
  int Hd, N, d, dv;                               // heads * d, the projections' row
  __device__ Row begin(int h, int r, bool ok) const {
    return {ok ? f_bias[h * d + r] : 0.f, ok ? lower[h * d + r] : 0.f};
  }
  __device__ void fetch(int t, int h, int r, float* z) const {
    z[0] = proj[(size_t)t * N + h * d + r];
    z[1] = proj[(size_t)t * N + Hd + h * d + r];
  }
  __device__ void form(const Row& m, const float* z, const float*, float& q, float& f, float&) const {
    q = z[0] / (1.0f + expf(-z[0]));
    f = m.lower + (1.0f - m.lower) / (1.0f + expf(-(z[1] + m.bias)));
  }
  __device__ float value(int t, int h, int j) const { return proj[(size_t)t * N + 2 * Hd + h * dv + j]; }
  __device__ static float act(float v) { return v; }
  __device__ int low_size() const { return 0; }
  __device__ float low(int, int) const { return 0.f; }
};
}  // namespace

extern "C" int yalm_hgrn2(const float* proj, const float* f_bias, const float* lower, const float* w_norm, float* state,
                          float* raw, const int* cu_seqlens, const int* seq_slot, void* out, int T, int B, int n_heads,
                          int d, int dv, float eps, int out_dtype, hipStream_t stream) {
  if (T <= 0 || B <= 0) return YALM_OK;
  if (n_heads <= 0 || d <= 0 || d > 256 || dv <= 0) return YALM_ERR_ARG;
  if (out_dtype != YALM_F32 && out_dtype != YALM_BF16) return YALM_ERR_DTYPE;
  const Hgrn2Op op = {proj, f_bias, lower, n_heads * d, 2 * n_heads * d + n_heads * dv, d, dv};
  int rc;
#define SCAN(NR_, LANES_, NC_, TOK_) \
  rc = diag_scan_launch<Hgrn2Op, NR_, LANES_, NC_, TOK_>(op, state, raw, cu_seqlens, seq_slot, B, n_heads, d, dv, 0, stream)
  if (d <= 32) SCAN(4, 8, 1, 16);
  else if (d <= 64) SCAN(8, 8, 1, 16);
  else if (d <= 128) SCAN(16, 8, 1, 16);
  else SCAN(32, 8, 1, 16);
#undef SCAN
  if (rc != YALM_OK) return rc;
  return heads_norm_launch(raw, w_norm, nullptr, 0, out, T, n_heads, dv, eps, out_dtype, stream);
}
