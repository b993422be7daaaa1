// Kernels of layers that norm a sublayer's OUTPUT before it joins the residual stream
// (x <- x + rms(y) * w) or the SUM of both (x <- LN(alpha x + y)), of the PolyNorm activation, of an elementwise squash in
// a norm's place (tanh(alpha x) * w + b), and of a row's RMS norm under a sigmoid gate.  Everything is float32 arithmetic, on a
// row per workgroup where a row has sums; inputs from GEMMs are float32, outputs go to the compute dtype.
#include "common.h"
#include "yalm_hip.h"

namespace {

constexpr int ROW_THREADS = 256;
constexpr int ROW_WAVES = ROW_THREADS / WAVE;

template <typename T>
__global__ __launch_bounds__(ROW_THREADS) void cast_kernel(const float* __restrict__ x, T* __restrict__ out, long n) {
  long i = (long)blockIdx.x * ROW_THREADS + threadIdx.x;
  const long step = (long)gridDim.x * ROW_THREADS;
  for (; i < n; i += step) out[i] = from_f32<T>(x[i]);
}

// x[r] += y[r] * rsqrt(mean(y[r]^2) + eps) * w; if h is given: h[r] = T(x[r]), or with next_w the norm that reads
// the stream next, h[r] = T(x[r] * rsqrt(mean(x[r]^2) + next_eps) * next_w)
template <typename W, typename T, int NT, int PER>
__global__ __launch_bounds__(NT) void norm_add_kernel(const float* __restrict__ y, const W* __restrict__ w, float eps,
                                                      float* __restrict__ x, T* __restrict__ h, const float* __restrict__ next_w,
                                                      float next_eps, int D) {
  // PER > 0: the row fits PER values a thread; y is read once and the new x stays in registers for the second norm
  __shared__ float red[NT / WAVE];
  const size_t row = (size_t)blockIdx.x * D;
  float keep[PER > 0 ? PER : 1];
  float ss = 0.f;
  if (PER > 0) {
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      const int i = threadIdx.x + j * NT;
      keep[j] = i < D ? y[row + i] : 0.f;
      ss += keep[j] * keep[j];
    }
  } else {
    for (int i = threadIdx.x; i < D; i += NT) {
      const float v = y[row + i];
      ss += v * v;
    }
  }
  ss = block_sum<NT / WAVE>(ss, red);
  const float scale = 1.0f / sqrtf(ss / (float)D + eps);
  float ss2 = 0.f;
  if (PER > 0) {
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      const int i = threadIdx.x + j * NT;
      if (i < D) {
        const float v = x[row + i] + keep[j] * scale * to_f32(w[i]);
        x[row + i] = v;
        keep[j] = v;
        ss2 += v * v;
        if (h != nullptr && next_w == nullptr) h[row + i] = from_f32<T>(v);
      }
    }
  } else {
    for (int i = threadIdx.x; i < D; i += NT) {
      const float v = x[row + i] + y[row + i] * scale * to_f32(w[i]);
      x[row + i] = v;
      ss2 += v * v;
      if (h != nullptr && next_w == nullptr) h[row + i] = from_f32<T>(v);
    }
  }
  if (h == nullptr || next_w == nullptr) return;
  ss2 = block_sum<NT / WAVE>(ss2, red);
  const float scale2 = 1.0f / sqrtf(ss2 / (float)D + next_eps);
  if (PER > 0) {
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      const int i = threadIdx.x + j * NT;
      if (i < D) h[row + i] = from_f32<T>(keep[j] * scale2 * next_w[i]);
    }
  } else {
    for (int i = threadIdx.x; i < D; i += NT) h[row + i] = from_f32<T>(x[row + i] * scale2 * next_w[i]);   // its own stores
  }
}

// The layer norm of a weighted sum: n[r] = LN(alpha * x[row(r)] + y[r]) (y may be null), LN(v) = (v - mean) / sqrt(mean of
// the squared deviations + eps) * w + b.  STORE_X: x[r] = n[r] (the stream after a layer that norms the sum).  h, if given:
// h[r] = T(n[r]), or with next_w the layer norm that reads the stream next, h[r] = T(LN(n[r]; next_w, next_b, next_eps)).
// PER > 0: the row fits PER values a thread and stays in registers from the sum to the last result; PER = 0: any
// width (STORE_X then keeps the row in x, else it is formed again for every pass).
template <typename T, int NT, int PER, bool STORE_X>
__global__ __launch_bounds__(NT) void layer_norm_kernel(float* __restrict__ x, const float* __restrict__ y, float alpha,
                                                        const int* __restrict__ row_index, const float* __restrict__ w,
                                                        const float* __restrict__ b, float eps, T* __restrict__ h,
                                                        const float* __restrict__ next_w, const float* __restrict__ next_b,
                                                        float next_eps, int D) {
  __shared__ float red[NT / WAVE];
  const size_t row = (size_t)blockIdx.x * D;
  float* xr = x + (size_t)(row_index != nullptr ? row_index[blockIdx.x] : (int)blockIdx.x) * D;
  const float inv_d = 1.0f / (float)D;
  float keep[PER > 0 ? PER : 1];
  auto each = [&](auto f) {                        // f(element, place in keep)
    if constexpr (PER > 0) {
#pragma unroll
      for (int j = 0; j < PER; ++j) {
        const int i = threadIdx.x + j * NT;
        if (i < D) f(i, j);
      }
    } else {
      for (int i = threadIdx.x; i < D; i += NT) f(i, 0);
    }
  };
  auto input = [&](int i) { return fmaf(alpha, xr[i], y != nullptr ? y[row + i] : 0.f); };
  // v(i, j): the row's element at the present stage
  auto at = [&](int i, int j) {
    if constexpr (PER > 0) return keep[j];
    else return STORE_X ? xr[i] : input(i);
  };
  float sum = 0.f;
  each([&](int i, int j) {
    const float v = input(i);
    if constexpr (PER > 0) keep[j] = v;
    else if (STORE_X) xr[i] = v;                   // a thread reads back its own stores only
    sum += v;
  });
  const float mean = block_sum<NT / WAVE>(sum, red) * inv_d;
  float ss = 0.f;
  each([&](int i, int j) {
    const float dv = at(i, j) - mean;
    ss = fmaf(dv, dv, ss);
  });
  const float r = 1.0f / sqrtf(block_sum<NT / WAVE>(ss, red) * inv_d + eps);
  const bool second = h != nullptr && next_w != nullptr;
  float sum2 = 0.f;
  each([&](int i, int j) {
    const float n = fmaf((at(i, j) - mean) * r, w[i], b[i]);
    if constexpr (PER > 0) keep[j] = n;
    if (STORE_X) xr[i] = n;
    if (h != nullptr && !second) h[row + i] = from_f32<T>(n);
    sum2 += n;
  });
  if (!second) return;
  auto normed = [&](int i, int j) {
    if constexpr (PER > 0) return keep[j];
    else return STORE_X ? xr[i] : fmaf((input(i) - mean) * r, w[i], b[i]);
  };
  const float mean2 = block_sum<NT / WAVE>(sum2, red) * inv_d;
  float ss2 = 0.f;
  each([&](int i, int j) {
    const float dv = normed(i, j) - mean2;
    ss2 = fmaf(dv, dv, ss2);
  });
  const float r2 = 1.0f / sqrtf(block_sum<NT / WAVE>(ss2, red) * inv_d + next_eps);
  each([&](int i, int j) { h[row + i] = from_f32<T>(fmaf((normed(i, j) - mean2) * r2, next_w[i], next_b[i])); });
}

// An elementwise squash in a norm's place, n(v) = tanh(alpha v) * w + b.  y null: h[r] = T(n(x[row(r)])).  Else x[r] += mult *
// n(y[r] + y_bias), and h (may be null) receives the new x, or with next_w the squash that reads the stream next, of the new
// x.  A thread has VEC neighbours of a row.
template <typename T, int VEC>
__global__ __launch_bounds__(ROW_THREADS) void squash_kernel(float* __restrict__ x, const float* __restrict__ y,
                                                             const float* __restrict__ y_bias, float mult,
                                                             const int* __restrict__ row_index, float alpha,
                                                             const float* __restrict__ w, const float* __restrict__ b,
                                                             T* __restrict__ h, float next_alpha, const float* __restrict__ next_w,
                                                             const float* __restrict__ next_b, int D) {
  struct __attribute__((aligned(VEC * sizeof(float)))) F { float v[VEC]; };
  struct __attribute__((aligned(VEC * sizeof(T)))) O { T v[VEC]; };
  const int i = (blockIdx.y * ROW_THREADS + threadIdx.x) * VEC;
  if (i >= D) return;
  auto load = [&](const float* p) { return *reinterpret_cast<const F*>(p); };
  const size_t at = (size_t)blockIdx.x * D + i;
  float* xp = x + (row_index != nullptr ? (size_t)row_index[blockIdx.x] * D + i : at);
  const F ww = load(w + i), bb = load(b + i);
  F xv = load(xp);
  O o;
  if (y == nullptr) {
#pragma unroll
    for (int k = 0; k < VEC; ++k) o.v[k] = from_f32<T>(fmaf(tanhf(alpha * xv.v[k]), ww.v[k], bb.v[k]));
    *reinterpret_cast<O*>(h + at) = o;
    return;
  }
  F yv = load(y + at);
  if (y_bias != nullptr) {
    const F yb = load(y_bias + i);
#pragma unroll
    for (int k = 0; k < VEC; ++k) yv.v[k] += yb.v[k];
  }
#pragma unroll
  for (int k = 0; k < VEC; ++k) xv.v[k] = fmaf(mult, fmaf(tanhf(alpha * yv.v[k]), ww.v[k], bb.v[k]), xv.v[k]);
  *reinterpret_cast<F*>(xp) = xv;
  if (h == nullptr) return;
  if (next_w != nullptr) {
    const F nw = load(next_w + i), nb = load(next_b + i);
#pragma unroll
    for (int k = 0; k < VEC; ++k) o.v[k] = from_f32<T>(fmaf(tanhf(next_alpha * xv.v[k]), nw.v[k], nb.v[k]));
  } else {
#pragma unroll
    for (int k = 0; k < VEC; ++k) o.v[k] = from_f32<T>(xv.v[k]);
  }
  *reinterpret_cast<O*>(h + at) = o;
}

// out[r, i] = x[r, i] / sqrt(mean(x[r]^2) + eps) * w[i] * sigmoid(gate[r, i]), i < n: a workgroup a row; the rows of gate and
// out are gate_row and out_row apart.  PER > 0: the row fits PER values a thread; PER = 0: any length.
template <typename T, int NT, int PER>
__global__ __launch_bounds__(NT) void rms_gate_kernel(const float* __restrict__ x, const float* __restrict__ w, float eps,
                                                      const float* __restrict__ gate, long gate_row, T* __restrict__ out,
                                                      long out_row, int n) {
  __shared__ float red[NT / WAVE];
  const float* xr = x + (size_t)blockIdx.x * n;
  const float* gr = gate + (size_t)blockIdx.x * gate_row;
  T* o = out + (size_t)blockIdx.x * out_row;
  float ss = 0.f;
  auto gated = [&](float v, float s, float wi, float z) { return from_f32<T>(v * s * wi / (1.0f + expf(-z))); };
  if constexpr (PER > 0) {
    float v[PER], z[PER], g[PER];
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      const int i = threadIdx.x + j * NT;
      v[j] = i < n ? xr[i] : 0.f;
      z[j] = i < n ? gr[i] : 0.f;
      g[j] = i < n ? w[i] : 0.f;
    }
#pragma unroll
    for (int j = 0; j < PER; ++j) ss = fmaf(v[j], v[j], ss);
    const float s = 1.0f / sqrtf(block_sum<NT / WAVE>(ss, red) / (float)n + eps);
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      const int i = threadIdx.x + j * NT;
      if (i < n) o[i] = gated(v[j], s, g[j], z[j]);
    }
  } else {
    for (int i = threadIdx.x; i < n; i += NT) ss = fmaf(xr[i], xr[i], ss);
    const float s = 1.0f / sqrtf(block_sum<NT / WAVE>(ss, red) / (float)n + eps);
    for (int i = threadIdx.x; i < n; i += NT) o[i] = gated(xr[i], s, w[i], gr[i]);
  }
}

// out = a N(z) + b N(z^2) + c N(z^3) + e, N(v) = v / sqrt(mean(v^2) + eps) over the row.  PER > 0: the row fits PER
// values a thread and is read once (kept in registers between the sums and the result); PER = 0: any width, read twice.
template <typename T, int NT, int PER>
__global__ __launch_bounds__(NT) void polynorm_kernel(const float* __restrict__ z, const float* __restrict__ coef, float eps,
                                                      T* __restrict__ out, int F) {
  constexpr int ROW_THREADS = NT, ROW_WAVES = NT / WAVE;
  __shared__ float red[ROW_WAVES];
  const size_t row = (size_t)blockIdx.x * F;
  float s2 = 0.f, s4 = 0.f, s6 = 0.f;
  float keep[PER > 0 ? PER : 1];
  if (PER > 0) {
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      const int i = threadIdx.x + j * ROW_THREADS;
      const float v = i < F ? z[row + i] : 0.f;
      keep[j] = v;
      const float v2 = v * v;
      s2 += v2;
      s4 += v2 * v2;
      s6 += v2 * v2 * v2;
    }
  } else {
    for (int i = threadIdx.x; i < F; i += ROW_THREADS) {
      const float v = z[row + i];
      const float v2 = v * v;
      s2 += v2;
      s4 += v2 * v2;
      s6 += v2 * v2 * v2;
    }
  }
  s2 = block_sum<ROW_WAVES>(s2, red);
  s4 = block_sum<ROW_WAVES>(s4, red);
  s6 = block_sum<ROW_WAVES>(s6, red);
  const float r1 = coef[0] / sqrtf(s2 / (float)F + eps);
  const float r2 = coef[1] / sqrtf(s4 / (float)F + eps);
  const float r3 = coef[2] / sqrtf(s6 / (float)F + eps);
  const float e = coef[3];
  if (PER > 0) {
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      const int i = threadIdx.x + j * ROW_THREADS;
      const float v = keep[j];
      if (i < F) out[row + i] = from_f32<T>(v * r1 + v * v * r2 + v * v * v * r3 + e);
    }
  } else {
    for (int i = threadIdx.x; i < F; i += ROW_THREADS) {
      const float v = z[row + i];
      out[row + i] = from_f32<T>(v * r1 + v * v * r2 + v * v * v * r3 + e);
    }
  }
}

template <typename T>
int polynorm_launch(const float* z, const float* coef, float eps, void* out, int R, int F, hipStream_t stream) {
  if (F < 2048) polynorm_kernel<T, 256, 8><<<R, 256, 0, stream>>>(z, coef, eps, (T*)out, F);
  else if (F <= 8192) polynorm_kernel<T, 1024, 8><<<R, 1024, 0, stream>>>(z, coef, eps, (T*)out, F);
  else if (F <= 32768) polynorm_kernel<T, 1024, 32><<<R, 1024, 0, stream>>>(z, coef, eps, (T*)out, F);
  else polynorm_kernel<T, 1024, 0><<<R, 1024, 0, stream>>>(z, coef, eps, (T*)out, F);
  return launch_status();
}

}  // namespace

extern "C" int yalm_cast(const float* x, void* out, long n, int out_dtype, hipStream_t stream) {
  if (n <= 0) return YALM_OK;
  const int blocks = (int)((n + ROW_THREADS - 1) / ROW_THREADS < 4096 ? (n + ROW_THREADS - 1) / ROW_THREADS : 4096);
  if (out_dtype == YALM_BF16)
    cast_kernel<bf16><<<blocks, ROW_THREADS, 0, stream>>>(x, (bf16*)out, n);
  else if (out_dtype == YALM_F32)
    cast_kernel<float><<<blocks, ROW_THREADS, 0, stream>>>(x, (float*)out, n);
  else
    return YALM_ERR_DTYPE;
  return launch_status();
}

template <typename W, typename T>
static int norm_add_launch(const float* y, const void* w, float eps, float* x, void* h, const float* next_w, float next_eps,
                           int R, int D, hipStream_t stream) {
  if (D < 2048)
    norm_add_kernel<W, T, 256, 8><<<R, 256, 0, stream>>>(y, (const W*)w, eps, x, (T*)h, next_w, next_eps, D);
  else if (D <= 8192)
    norm_add_kernel<W, T, 1024, 8><<<R, 1024, 0, stream>>>(y, (const W*)w, eps, x, (T*)h, next_w, next_eps, D);
  else
    norm_add_kernel<W, T, 1024, 0><<<R, 1024, 0, stream>>>(y, (const W*)w, eps, x, (T*)h, next_w, next_eps, D);
  return launch_status();
}

extern "C" int yalm_norm_add(const float* y, const void* w, int w_dtype, float eps, float* x, void* h_out, int h_dtype,
                             const float* next_w, float next_eps, int R, int D, hipStream_t stream) {
  if (R <= 0) return YALM_OK;
  if (D <= 0) return YALM_ERR_ARG;
  if (w_dtype != YALM_F32 && w_dtype != YALM_BF16) return YALM_ERR_DTYPE;
  if (h_out != nullptr && h_dtype != YALM_F32 && h_dtype != YALM_BF16) return YALM_ERR_DTYPE;
  const bool hb = h_out != nullptr && h_dtype == YALM_BF16;
  if (w_dtype == YALM_F32)
    return hb ? norm_add_launch<float, bf16>(y, w, eps, x, h_out, next_w, next_eps, R, D, stream)
              : norm_add_launch<float, float>(y, w, eps, x, h_out, next_w, next_eps, R, D, stream);
  return hb ? norm_add_launch<bf16, bf16>(y, w, eps, x, h_out, next_w, next_eps, R, D, stream)
            : norm_add_launch<bf16, float>(y, w, eps, x, h_out, next_w, next_eps, R, D, stream);
}

template <typename T, bool STORE_X>
static int layer_norm_launch(float* x, const float* y, float alpha, const int* row_index, const float* w, const float* b,
                             float eps, void* h, const float* next_w, const float* next_b, float next_eps, int R, int D,
                             hipStream_t stream) {
#define LN(NT_, PER_)                                                                                                    \
  layer_norm_kernel<T, NT_, PER_, STORE_X><<<R, NT_, 0, stream>>>(x, y, alpha, row_index, w, b, eps, (T*)h, next_w, next_b, \
                                                                  next_eps, D)
  if (D <= 1024) LN(256, 4);
  else if (D <= 4096) LN(1024, 4);
  else if (D <= 16384) LN(1024, 16);
  else LN(1024, 0);
#undef LN
  return launch_status();
}

extern "C" int yalm_layer_norm(float* x, const float* y, float alpha, const int* row_index, const float* w, const float* b,
                               float eps, int store_x, void* h, int h_dtype, const float* next_w, const float* next_b,
                               float next_eps, int R, int D, hipStream_t stream) {
  if (R <= 0) return YALM_OK;
  if (D <= 0 || w == nullptr || b == nullptr || (store_x && row_index != nullptr) || (!store_x && h == nullptr) ||
      (next_w != nullptr && (next_b == nullptr || h == nullptr)))
    return YALM_ERR_ARG;
  if (h != nullptr && h_dtype != YALM_F32 && h_dtype != YALM_BF16) return YALM_ERR_DTYPE;
#define LN(T_, S_) layer_norm_launch<T_, S_>(x, y, alpha, row_index, w, b, eps, h, next_w, next_b, next_eps, R, D, stream)
  const bool hb = h != nullptr && h_dtype == YALM_BF16;
  if (store_x) return hb ? LN(bf16, true) : LN(float, true);
  return hb ? LN(bf16, false) : LN(float, false);
#undef LN
}

extern "C" int yalm_polynorm(const float* z, const float* coef, float eps, void* out, int out_dtype, int R, int F,
                             hipStream_t stream) {
  if (R <= 0) return YALM_OK;
  if (F <= 0) return YALM_ERR_ARG;
  if (out_dtype == YALM_BF16) return polynorm_launch<bf16>(z, coef, eps, out, R, F, stream);
  if (out_dtype == YALM_F32) return polynorm_launch<float>(z, coef, eps, out, R, F, stream);
  return YALM_ERR_DTYPE;
}

template <typename T>
static int squash_launch(float* x, const float* y, const float* y_bias, float mult, const int* row_index, float alpha,
                         const float* w, const float* b, void* h, float next_alpha, const float* next_w, const float* next_b,
                         int R, int D, hipStream_t stream) {
  const bool vec = D % 4 == 0 && ((((uintptr_t)x) | ((uintptr_t)y) | ((uintptr_t)y_bias) | ((uintptr_t)w) | ((uintptr_t)b) |
                                   ((uintptr_t)h) | ((uintptr_t)next_w) | ((uintptr_t)next_b)) & 15) == 0;
  const dim3 grid(R, ceil_div(D, ROW_THREADS * (vec ? 4 : 1)));
#define SQ(V_) \
  squash_kernel<T, V_><<<grid, ROW_THREADS, 0, stream>>>(x, y, y_bias, mult, row_index, alpha, w, b, (T*)h, next_alpha, next_w, next_b, D)
  if (vec) SQ(4);
  else SQ(1);
#undef SQ
  return launch_status();
}

extern "C" int yalm_squash(float* x, const float* y, const float* y_bias, float mult, const int* row_index, float alpha,
                           const float* w, const float* b, void* h, int h_dtype, float next_alpha, const float* next_w,
                           const float* next_b, int R, int D, hipStream_t stream) {
  if (R <= 0) return YALM_OK;
  if (D <= 0 || ceil_div(D, ROW_THREADS) > 65535 || w == nullptr || b == nullptr || (y == nullptr && h == nullptr) ||
      (y == nullptr && (y_bias != nullptr || next_w != nullptr)) || (y != nullptr && row_index != nullptr) ||
      (next_w != nullptr && (next_b == nullptr || h == nullptr)))
    return YALM_ERR_ARG;
  if (h != nullptr && h_dtype != YALM_F32 && h_dtype != YALM_BF16) return YALM_ERR_DTYPE;
  if (h != nullptr && h_dtype == YALM_BF16)
    return squash_launch<bf16>(x, y, y_bias, mult, row_index, alpha, w, b, h, next_alpha, next_w, next_b, R, D, stream);
  return squash_launch<float>(x, y, y_bias, mult, row_index, alpha, w, b, h, next_alpha, next_w, next_b, R, D, stream);
}

template <typename T>
static int rms_gate_launch(const float* x, const float* w, float eps, const float* gate, long gate_row, void* out, long out_row,
                           int R, int n, hipStream_t stream) {
#define RG(NT_, PER_) rms_gate_kernel<T, NT_, PER_><<<R, NT_, 0, stream>>>(x, w, eps, gate, gate_row, (T*)out, out_row, n)
  if (n <= 1024) RG(256, 4);
  else if (n <= 2048) RG(512, 4);
  else if (n <= 8192) RG(1024, 8);
  else RG(1024, 0);
#undef RG
  return launch_status();
}

extern "C" int yalm_rms_gate(const float* x, const float* w, float eps, const float* gate, long gate_row, void* out,
                             long out_row, int out_dtype, int R, int n, hipStream_t stream) {
  if (R <= 0) return YALM_OK;
  if (n <= 0 || gate_row < n || out_row < n || w == nullptr || gate == nullptr) return YALM_ERR_ARG;
  if (out_dtype == YALM_F32) return rms_gate_launch<float>(x, w, eps, gate, gate_row, out, out_row, R, n, stream);
  if (out_dtype == YALM_BF16) return rms_gate_launch<bf16>(x, w, eps, gate, gate_row, out, out_row, R, n, stream);
  return YALM_ERR_DTYPE;
}
