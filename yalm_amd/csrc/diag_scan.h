// A linear recurrence with a diagonal decay, token by token, in float32.  Per head, with the state S [d, dv]:
//     S <- diag(f_t) S + k_t v_t^T,   o_t = S^T q_t
// where q, f and k (d numbers each a token and head) are formed from the projections by an `Op`, and k is either a
// number of its own (Op::KEYS) or 1 - f (what the decay forgets of a row is what the row takes in).
//
// diag_scan_kernel: every column of S runs the recurrence on its own.  A workgroup owns COLS columns of one (sequence,
// head) and walks the sequence's tokens of the step in order; a column is spread over LANES lanes, each with NR
// consecutive rows of NC columns in registers, so that what a lane reads of q, f and k serves NC columns (the state is
// kept column by column, [slot][head][column][row]).  The operands of TOK tokens at a time are formed once by the whole
// workgroup (from projections that were asked for a group ahead and waited in registers) and wait in LDS, where the
// lanes read them four at a time; a lane (a quad of lanes, where a column has more than eight) leaves its share of a
// column's read-out in LDS and goes on to the next token, and the shares of a group's tokens are summed afterwards by
// all threads at once, so that no token waits for LDS to exchange between lanes.
//
// heads_norm_kernel: out[t, h, :] = o[t, h, :] / sqrt(mean(o[t, h, :]^2) + eps) * w, optionally times silu of a gate;
// a wave a (token, head).
//
// An Op is a small struct handed over by value:
//   KEYS                        whether k is a number of its own
//   LOW                         whether form() reads a short vector a token (`low`, low_size() floats padded to a multiple of 4)
//   Row begin(h, r, ok)         what a thread that forms row r of head h keeps in registers
//   fetch(t, h, r, z)           two floats of token t's projections (plain loads)
//   form(row, z, low, q, f, k)  the operands from them
//   value(t, h, j), act(z)      a plain load of what v_t[j] is made of, and v_t[j] from it;  low(t, i) the short vector's elements
#pragma once
#include "common.h"

namespace {
constexpr int DS_THREADS = 256;

// the value of another lane of the same quad (a DPP quad_perm control)
template <int CTRL>
__device__ __forceinline__ float quad_swap(float v) {
  return __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), CTRL, 0xF, 0xF, true));
}

template <class Op, int NR, int LANES, int NC, int TOK>
__global__ __launch_bounds__(DS_THREADS) void diag_scan_kernel(Op op, float* __restrict__ state, float* __restrict__ raw,
                                                               const int* __restrict__ cu_seqlens,
                                                               const int* __restrict__ seq_slot, int n_heads, int d, int dv) {
  constexpr int DP = NR * LANES;                  // rows as the lanes count them (zeros behind d); divides DS_THREADS
  constexpr int GROUPS = DS_THREADS / LANES, COLS = GROUPS * NC;
  constexpr int EL = TOK * DP / DS_THREADS;       // elements a thread forms for a group of tokens
  constexpr int VL = (TOK * COLS + DS_THREADS - 1) / DS_THREADS;     // values it fetches (threads behind TOK * COLS: none)
  constexpr int SHARES = LANES > 8 ? LANES / 4 : LANES;         // shares of a column's read-out that go through LDS
  static_assert(NR % 4 == 0 && (LANES == 8 || LANES == 16 || LANES == 32) && DS_THREADS % DP == 0 && EL >= 1, "");
  __shared__ __attribute__((aligned(16))) float s_q[TOK][DP];
  __shared__ __attribute__((aligned(16))) float s_f[TOK][DP];
  __shared__ __attribute__((aligned(16))) float s_k[Op::KEYS ? TOK : 1][Op::KEYS ? DP : 4];
  __shared__ __attribute__((aligned(16))) float s_v[TOK][COLS];
  __shared__ __attribute__((aligned(16))) float s_part[TOK][COLS][SHARES];
  extern __shared__ __attribute__((aligned(16))) float s_low[];              // Op::LOW: [2][TOK][padded size]
  const int b = blockIdx.x, h = blockIdx.y, c0 = blockIdx.z * COLS, tid = threadIdx.x;
  const int group = tid / LANES, rl = tid % LANES, j0 = c0 + group * NC, r0 = rl * NR;
  const int slot = seq_slot[b];
  const int t0 = cu_seqlens[b], t1 = cu_seqlens[b + 1];
  const int HV = n_heads * dv;
  if (slot < 0) {                                 // a padding row: no state is touched, its result is zeros
    for (int t = t0; t < t1; ++t)
      if (tid < COLS && c0 + tid < dv) raw[(size_t)t * HV + h * dv + c0 + tid] = 0.f;
    return;
  }
  float* sp = state + ((size_t)slot * n_heads + h) * dv * d;
  const bool vec = d % 4 == 0 && (((uintptr_t)state) & 15) == 0;
  float s[NC][NR];
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const float* col = sp + (size_t)min(j0 + c, dv - 1) * d;
#pragma unroll
    for (int i = 0; i < NR; i += 4) {
      if (vec && r0 + i + 3 < d && j0 + c < dv) {
        const float4 v4 = *reinterpret_cast<const float4*>(col + r0 + i);
        s[c][i] = v4.x, s[c][i + 1] = v4.y, s[c][i + 2] = v4.z, s[c][i + 3] = v4.w;
      } else {
#pragma unroll
        for (int k = 0; k < 4; ++k) s[c][i + k] = (r0 + i + k < d && j0 + c < dv) ? col[r0 + i + k] : 0.f;
      }
    }
  }
  // the thread forms row gr of the tokens gt, gt + DS_THREADS / DP, ... of a group, and fetches the values of column vc
  // of the tokens vt, vt + DS_THREADS / COLS, ...: always the same row and column
  const int gr = tid % DP, gt = tid / DP, vc = tid % COLS, vt = tid / COLS;
  const bool row_ok = gr < d, col_ok = c0 + vc < dv;
  const typename Op::Row mine = op.begin(h, gr, row_ok);
  const int rp = Op::LOW ? (op.low_size() + 3) / 4 * 4 : 0;
  float z[EL][2], zv[VL], zl = 0.f;
  auto fetch = [&](int tc) {                      // a group's operands into registers: asked for a group ahead
#pragma unroll
    for (int k = 0; k < EL; ++k) {
      op.fetch(min(tc + gt + k * (DS_THREADS / DP), t1 - 1), h, min(gr, d - 1), z[k]);      // no branch: what lies behind is not used
    }
#pragma unroll
    for (int k = 0; k < VL; ++k) {
      zv[k] = op.value(min(tc + vt + k * (DS_THREADS / COLS), t1 - 1), h, min(c0 + vc, dv - 1));
    }
  };
  auto low_at = [&](int tc, int i) {              // element i of the group's short vectors, tokens one behind the other
    const int t = tc + i / rp, e = i % rp;
    return t < t1 && e < op.low_size() ? op.low(t, e) : 0.f;
  };
  if (t1 > t0) fetch(t0);
  if constexpr (Op::LOW) {                        // the short vectors are a group further ahead: LDS holds the group's, a register the next one's
    for (int i = tid; i < TOK * rp; i += DS_THREADS) s_low[i] = low_at(t0, i);
    if (tid < TOK * rp) zl = low_at(t0 + TOK, tid);
  }
  int turn = 0;
  for (int tc = t0; tc < t1; tc += TOK, turn ^= 1) {
    const int n = min(TOK, t1 - tc);
    lds_barrier();                              // the group before is read
    auto form = [&](int k) {
      const int tt = gt + k * (DS_THREADS / DP);
      float q, f, kk = 0.f;
      op.form(mine, z[k], s_low + (turn * TOK + tt) * rp, q, f, kk);
      s_q[tt][gr] = row_ok ? q : 0.f;
      s_f[tt][gr] = row_ok ? f : 0.f;
      if constexpr (Op::KEYS) s_k[tt][gr] = row_ok ? kk : 0.f;
    };
    if (n == TOK) {                               // a whole group: no branch between a thread's elements
#pragma unroll
      for (int k = 0; k < EL; ++k) form(k);
    } else {
#pragma unroll
      for (int k = 0; k < EL; ++k)
        if (gt + k * (DS_THREADS / DP) < n) form(k);
    }
#pragma unroll
    for (int k = 0; k < VL; ++k)
      if (vt + k * (DS_THREADS / COLS) < TOK) s_v[vt + k * (DS_THREADS / COLS)][vc] = Op::act(zv[k]);
    if (tc + TOK < t1) {
      fetch(tc + TOK);
      if constexpr (Op::LOW) {
        float* next = s_low + (turn ^ 1) * TOK * rp;
        for (int i = tid; i < TOK * rp; i += DS_THREADS) next[i] = i == tid ? zl : low_at(tc + TOK, i);
        if (tid < TOK * rp && tc + 2 * TOK < t1) zl = low_at(tc + 2 * TOK, tid);
      }
    }
    lds_barrier();
    auto token = [&](int tt) {
      float v[NC], acc[NC][2];
#pragma unroll
      for (int c = 0; c < NC; ++c) {
        v[c] = s_v[tt][group * NC + c];
        acc[c][0] = acc[c][1] = 0.f;
      }
#pragma unroll
      for (int i = 0; i < NR; i += 4) {
        const float4 f4 = *reinterpret_cast<const float4*>(&s_f[tt][r0 + i]);
        const float4 q4 = *reinterpret_cast<const float4*>(&s_q[tt][r0 + i]);
        const float f[4] = {f4.x, f4.y, f4.z, f4.w}, q[4] = {q4.x, q4.y, q4.z, q4.w};
        float k[4] = {0.f, 0.f, 0.f, 0.f};
        if constexpr (Op::KEYS) {
          const float4 k4 = *reinterpret_cast<const float4*>(&s_k[tt][r0 + i]);
          k[0] = k4.x, k[1] = k4.y, k[2] = k4.z, k[3] = k4.w;
        }
#pragma unroll
        for (int c = 0; c < NC; ++c)
#pragma unroll
          for (int u = 0; u < 4; ++u) {
            float& x = s[c][i + u];
            if constexpr (Op::KEYS) x = fmaf(f[u], x, k[u] * v[c]);
            else x = fmaf(f[u], x - v[c], v[c]);              // f S + (1 - f) v
            acc[c][u & 1] = fmaf(x, q[u], acc[c][u & 1]);
          }
      }
#pragma unroll
      for (int c = 0; c < NC; ++c) {
        float sum = acc[c][0] + acc[c][1];
        if constexpr (LANES > 8) {                // the four lanes of a quad first
          sum += quad_swap<0xB1>(sum);            // lane ^ 1
          sum += quad_swap<0x4E>(sum);            // lane ^ 2
          if ((rl & 3) == 0) s_part[tt][group * NC + c][rl >> 2] = sum;
        } else {
          s_part[tt][group * NC + c][rl] = sum;
        }
      }
    };
    if (n == TOK) {                               // a whole group: its tokens unrolled, so that a token's reads of LDS stand under the token before
#pragma unroll
      for (int tt = 0; tt < TOK; ++tt) token(tt);
    } else {
      for (int tt = 0; tt < n; ++tt) token(tt);
    }
    lds_barrier();
    // a column's read-out is the sum over its lanes: VL (token, column) pairs a thread
#pragma unroll
    for (int k = 0; k < VL; ++k) {
      const int tt = vt + k * (DS_THREADS / COLS);
      if (tt < n && col_ok) {
        float sum[SHARES / 4];                    // in pairs, pairs of pairs, ...
#pragma unroll
        for (int i = 0; i < SHARES / 4; ++i) {
          const float4 a = *reinterpret_cast<const float4*>(&s_part[tt][vc][4 * i]);
          sum[i] = (a.x + a.y) + (a.z + a.w);
        }
#pragma unroll
        for (int w = SHARES / 8; w > 0; w /= 2)
#pragma unroll
          for (int i = 0; i < w; ++i) sum[i] = sum[2 * i] + sum[2 * i + 1];
        raw[(size_t)(tc + tt) * HV + h * dv + c0 + vc] = sum[0];
      }
    }
  }
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    if (j0 + c >= dv) continue;
    float* col = sp + (size_t)(j0 + c) * d;
#pragma unroll
    for (int i = 0; i < NR; i += 4) {
      if (vec && r0 + i + 3 < d) {
        *reinterpret_cast<float4*>(col + r0 + i) = make_float4(s[c][i], s[c][i + 1], s[c][i + 2], s[c][i + 3]);
      } else {
#pragma unroll
        for (int k = 0; k < 4; ++k)
          if (r0 + i + k < d) col[r0 + i + k] = s[c][i + k];
      }
    }
  }
}

// gate (optional): float32, row t's at gate + t * gate_row, head h's at h * dv
template <typename T>
__global__ __launch_bounds__(4 * WAVE) void heads_norm_kernel(const float* __restrict__ raw, const float* __restrict__ w,
                                                             const float* __restrict__ gate, long gate_row, T* __restrict__ out,
                                                             long n_rows, int n_heads, int dv, float eps) {
  const long row = (long)blockIdx.x * 4 + threadIdx.x / WAVE;
  const int lane = threadIdx.x % WAVE;
  if (row >= n_rows) return;
  const float* src = raw + row * dv;
  const float* g = gate == nullptr ? nullptr : gate + (row / n_heads) * gate_row + (row % n_heads) * dv;
  float ss = 0.f;
  for (int i = lane; i < dv; i += WAVE) ss = fmaf(src[i], src[i], ss);
  ss = wave_sum(ss);
  const float f = 1.0f / sqrtf(ss / (float)dv + eps);
  for (int i = lane; i < dv; i += WAVE) {
    float v = src[i] * f * w[i];
    if (g != nullptr) v *= g[i] / (1.0f + expf(-g[i]));
    out[row * dv + i] = from_f32<T>(v);
  }
}

// The gated form for dv a multiple of 4 up to 256: LPR lanes a (token, head), four elements a lane, everything asked for
// before the first sum.
template <typename T, int LPR>
__global__ __launch_bounds__(4 * WAVE) void heads_norm_gate_kernel(const float* __restrict__ raw, const float* __restrict__ w,
                                                                  const float* __restrict__ gate, long gate_row, T* __restrict__ out,
                                                                  long n_rows, int n_heads, int dv, float eps) {
  const long row = (long)blockIdx.x * (4 * WAVE / LPR) + threadIdx.x / LPR;
  const int i = threadIdx.x % LPR * 4;
  const bool ok = row < n_rows && i < dv;
  float4 v = make_float4(0.f, 0.f, 0.f, 0.f), g = v, ww = v;
  if (ok) {
    v = *reinterpret_cast<const float4*>(raw + row * dv + i);
    g = *reinterpret_cast<const float4*>(gate + (row / n_heads) * gate_row + (row % n_heads) * dv + i);
    ww = *reinterpret_cast<const float4*>(w + i);
  }
  float ss = (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w);
#pragma unroll
  for (int o = LPR / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, WAVE);
  const float f = 1.0f / sqrtf(ss / (float)dv + eps);
  auto gated = [&](float x, float y, float z) { return x * f * y * (z / (1.0f + expf(-z))); };
  if (ok) {
    T* o = out + row * dv + i;
    o[0] = from_f32<T>(gated(v.x, ww.x, g.x));
    o[1] = from_f32<T>(gated(v.y, ww.y, g.y));
    o[2] = from_f32<T>(gated(v.z, ww.z, g.z));
    o[3] = from_f32<T>(gated(v.w, ww.w, g.w));
  }
}

template <typename T>
int heads_norm_gate_launch(const float* raw, const float* w, const float* gate, long gate_row, void* out, long n_rows, int n_heads,
                           int dv, float eps, hipStream_t stream) {
#define HN(LPR_)                                                                                                         \
  heads_norm_gate_kernel<T, LPR_><<<ceil_div(n_rows, 4 * WAVE / LPR_), 4 * WAVE, 0, stream>>>(raw, w, gate, gate_row, (T*)out, \
                                                                                             n_rows, n_heads, dv, eps)
  if (dv <= 32) HN(8);
  else if (dv <= 64) HN(16);
  else if (dv <= 128) HN(32);
  else HN(64);
#undef HN
  return launch_status();
}

template <class Op, int NR, int LANES, int NC, int TOK>
int diag_scan_launch(const Op& op, float* state, float* raw, const int* cu_seqlens, const int* seq_slot, int B, int n_heads,
                     int d, int dv, size_t low_elements, hipStream_t stream) {
  constexpr int COLS = DS_THREADS / LANES * NC;
  if (n_heads > 65535 || ceil_div(dv, COLS) > 65535) return YALM_ERR_ARG;
  dim3 grid(B, n_heads, ceil_div(dv, COLS));
  diag_scan_kernel<Op, NR, LANES, NC, TOK><<<grid, DS_THREADS, low_elements * 2 * TOK * sizeof(float), stream>>>(
      op, state, raw, cu_seqlens, seq_slot, n_heads, d, dv);
  return launch_status();
}

static inline int heads_norm_launch(const float* raw, const float* w, const float* gate, long gate_row, void* out, int T, int n_heads,
                                    int dv, float eps, int out_dtype, hipStream_t stream) {
  const long n_rows = (long)T * n_heads;
  if (gate != nullptr && dv % 4 == 0 && dv <= 256 && gate_row % 4 == 0 &&
      ((((uintptr_t)raw) | ((uintptr_t)w) | ((uintptr_t)gate)) & 15) == 0)
    return out_dtype == YALM_F32 ? heads_norm_gate_launch<float>(raw, w, gate, gate_row, out, n_rows, n_heads, dv, eps, stream)
                                 : heads_norm_gate_launch<bf16>(raw, w, gate, gate_row, out, n_rows, n_heads, dv, eps, stream);
  const int blocks = ceil_div(n_rows, 4);
  if (out_dtype == YALM_F32)
    heads_norm_kernel<float><<<blocks, 4 * WAVE, 0, stream>>>(raw, w, gate, gate_row, (float*)out, n_rows, n_heads, dv, eps);
  else
    heads_norm_kernel<bf16><<<blocks, 4 * WAVE, 0, stream>>>(raw, w, gate, gate_row, (bf16*)out, n_rows, n_heads, dv, eps);
  return launch_status();
}
}  // namespace
