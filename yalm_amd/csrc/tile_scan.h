// Linear recurrences of diag_scan.h a tile of 64 tokens at a time on the matrix cores, in float32 (v_mfma_f32_16x16x4_f32):
// what their kernels share.  A design's own kernel works every tile and head at once and leaves, per tile and head,
//     qd [64][DP]   the queries times the decays from the tile's start up to and including their token,
//     kd [DP][64]   the keys times the decays behind their token up to the tile's end (zeros behind the text),
//     gd [DP]       the decays of the whole tile,
// and in raw the part of o that the tile's own tokens make.  scan_carry_kernel then walks a sequence's tiles in order (a
// workgroup 16 columns of a head): the products with the carried state and the state itself.  A wave owns 32 rows of S in
// the layout of a matrix instruction's result, which is also its operand in the next tile's product when k is counted in
// that order; the waves' shares of o meet in LDS.
//
// An Op is a small struct handed over by value with d, dv, Hv (the elements of a row of raw), value(t, h, j) (a plain load of
// what v_t[j] is made of) and act (v_t[j] from it).
#pragma once
#include <type_traits>

#include "diag_scan.h"

namespace {
constexpr int GT = PAGE, GB = 16, GNB = GT / GB;       // tokens of a tile and of a block, blocks
constexpr int GA_ROW = GT + 4;                   // LDS row of the tile's score matrix
typedef __attribute__((ext_vector_type(4))) float gf32x4;
__device__ __forceinline__ gf32x4 mfma4(float a, float b, gf32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }
__device__ __forceinline__ float el(const float4& v, int i) { return i == 0 ? v.x : i == 1 ? v.y : i == 2 ? v.z : v.w; }

// the sequence of tile gt (the last b with seq_tile0[b] <= gt)
__device__ __forceinline__ int seq_of_tile(const int* __restrict__ seq_tile0, int B, int gt) {
  int lo = 0, hi = B - 1;
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (seq_tile0[mid] <= gt) lo = mid; else hi = mid - 1;
  }
  return lo;
}

// The state over the tiles of a sequence, and its share of o added to raw.  NW waves, wave w the rows 32 w .. 32 w + 31.
// WHOLE: dv is a multiple of 16, so that every tile but a sequence's last one is stored without a branch (behind a branch
// the compiler would wait for the operands that are still on their way).
template <class Op, int NW, bool WHOLE>
__global__ __launch_bounds__(NW * WAVE) void scan_carry_kernel(Op op, float* __restrict__ state, float* __restrict__ raw,
                                                               const float* __restrict__ qd, const float* __restrict__ kd,
                                                              const float* __restrict__ gd, const int* __restrict__ cu_seqlens,
                                                              const int* __restrict__ seq_slot, const int* __restrict__ seq_tile0,
                                                              int n_heads) {
  constexpr int DP = 32 * NW, TB = GNB / NW > 0 ? GNB / NW : 1;      // row blocks of o a wave adds up
  static_assert(GNB % NW == 0, "");
  __shared__ gf32x4 s_o[2][NW][GNB][WAVE];
  // heads run fastest: with a number of heads that is a multiple of the chip's eight parts, the workgroups of one head (which
  // read the same scaled queries and keys) share a second-level cache
  const int b = blockIdx.z, h = blockIdx.x, tid = threadIdx.x, lane = tid % WAVE, li = lane % 16, lq = lane / 16;
  const int wave = __builtin_amdgcn_readfirstlane(tid / WAVE);
  const int j = blockIdx.y * 16 + li, d = op.d, dv = op.dv;
  const int slot = seq_slot[b], start = cu_seqlens[b], len = cu_seqlens[b + 1] - start, tile0 = seq_tile0[b];
  const int n_tiles = (len + GT - 1) / GT;
  const bool col_ok = j < dv;
  float* sp = state + (((size_t)max(slot, 0) * n_heads + h) * dv + min(j, dv - 1)) * d;
  gf32x4 S[2];
#pragma unroll
  for (int R = 0; R < 2; ++R)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int e = 32 * wave + 16 * R + 4 * lq + r;
      S[R][r] = slot >= 0 && col_ok && e < d ? sp[e] : 0.f;
    }
  struct Operands {
    float4 q[GNB][2], k[2][GNB], g[2];
    float v[GT / 4], o[TB][4];
  };
  auto load = [&](int tile, Operands& x) {
    const size_t at = (size_t)(tile0 + tile) * n_heads + h;
    const float* qp = qd + at * GT * DP + 32 * wave + 4 * lq;
    const float* kp = kd + (at * DP + 32 * wave) * GT + 4 * lq;
    const int first = start + tile * GT, n = min(GT, len - tile * GT);
#pragma unroll
    for (int R = 0; R < 2; ++R) {
      x.g[R] = *reinterpret_cast<const float4*>(gd + at * DP + 32 * wave + 16 * R + 4 * lq);
#pragma unroll
      for (int i = 0; i < GNB; ++i) {
        x.q[i][R] = *reinterpret_cast<const float4*>(qp + (size_t)(i * GB + li) * DP + 16 * R);
        x.k[R][i] = *reinterpret_cast<const float4*>(kp + (size_t)(16 * R + li) * GT + i * GB);
      }
    }
#pragma unroll
    for (int i = 0; i < GT / 4; ++i) {
      const int s = 16 * (i / 4) + 4 * lq + i % 4;
      x.v[i] = op.value(first + min(s, n - 1), h, min(j, dv - 1));       // behind the text k is zero
    }
#pragma unroll
    for (int i = 0; i < TB; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = (wave * TB + i) * GB + 4 * lq + r;
        x.o[i][r] = raw[(size_t)(first + min(t, n - 1)) * op.Hv + h * dv + min(j, dv - 1)];
      }
  };
  auto work = [&](int tile, const Operands& x, auto whole) {
    const int first = start + tile * GT, n = min(GT, len - tile * GT), buf = tile & 1;
    gf32x4 acc[GNB];
#pragma unroll
    for (int i = 0; i < GNB; ++i) acc[i] = (gf32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int R = 0; R < 2; ++R)
#pragma unroll
      for (int r = 0; r < 4; ++r)
#pragma unroll
        for (int i = 0; i < GNB; ++i) acc[i] = mfma4(el(x.q[i][R], r), S[R][r], acc[i]);
#pragma unroll
    for (int R = 0; R < 2; ++R)
#pragma unroll
      for (int r = 0; r < 4; ++r) S[R][r] *= el(x.g[R], r);
#pragma unroll
    for (int i = 0; i < GT / 4; ++i)
#pragma unroll
      for (int R = 0; R < 2; ++R) S[R] = mfma4(el(x.k[R][i / 4], i % 4), Op::act(x.v[i]), S[R]);
#pragma unroll
    for (int i = 0; i < GNB; ++i) s_o[buf][wave][i][lane] = acc[i];
    lds_barrier();                                // the next tile's operands stay in flight
#pragma unroll
    for (int i = 0; i < TB; ++i) {
      gf32x4 sum = s_o[buf][0][wave * TB + i][lane];
#pragma unroll
      for (int w = 1; w < NW; ++w) sum += s_o[buf][w][wave * TB + i][lane];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = (wave * TB + i) * GB + 4 * lq + r;
        if (decltype(whole)::value || (t < n && col_ok)) raw[(size_t)(first + t) * op.Hv + h * dv + j] = x.o[i][r] + sum[r];
      }
    }
  };
  Operands even, odd;                             // the next tile's operands are asked for before this tile's products
  if (n_tiles <= 0) return;
  const std::integral_constant<bool, WHOLE> inner;
  int tile = 0;
  load(0, even);
  for (; tile + 2 < n_tiles; tile += 2) {
    load(tile + 1, odd);
    __builtin_amdgcn_sched_barrier(0);
    work(tile, even, inner);
    load(tile + 2, even);
    __builtin_amdgcn_sched_barrier(0);
    work(tile + 1, odd, inner);
  }
  if (tile + 1 < n_tiles) {
    load(tile + 1, odd);
    work(tile, even, inner);
    work(tile + 1, odd, std::false_type{});
  } else {
    work(tile, even, std::false_type{});
  }
  if (slot < 0 || !col_ok) return;
#pragma unroll
  for (int R = 0; R < 2; ++R)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int e = 32 * wave + 16 * R + 4 * lq + r;
      if (e < d) sp[e] = S[R][r];
    }
}

template <int DP, class Op>
int scan_carry_launch(const Op& op, float* state, float* raw, const float* qd, const float* kd, const float* gd, const int* cu_seqlens,
                      const int* seq_slot, const int* seq_tile0, int B, int n_heads, hipStream_t stream) {
  const dim3 grid(n_heads, ceil_div(op.dv, 16), B);
  if (op.dv % 16 == 0)
    scan_carry_kernel<Op, DP / 32, true><<<grid, DP / 32 * WAVE, 0, stream>>>(op, state, raw, qd, kd, gd, cu_seqlens, seq_slot,
                                                                         seq_tile0, n_heads);
  else
    scan_carry_kernel<Op, DP / 32, false><<<grid, DP / 32 * WAVE, 0, stream>>>(op, state, raw, qd, kd, gd, cu_seqlens, seq_slot,
                                                                          seq_tile0, n_heads);
  return launch_status();
}
}  // namespace
