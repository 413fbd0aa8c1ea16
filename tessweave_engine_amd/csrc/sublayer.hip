// Kernels of a layer arrangement that norms AFTER each sum:
//
//   x <- w * unit(alpha * x + scale * y),  unit(v) = v / sqrt(mean(v^2) + eps)
//
// x is the float32 residual stream, y a sublayer's float32 result (or split-K partial sums that are added up
// here, in index order), scale an optional per-channel factor, w the norm's weight. The normed row is written
// back to x and, rounded once, to `out` in the compute type, which is what the next sublayer's products read.
// Also here: the square of relu, in place, for a feed-forward without a gate.
#include "tw_common.h"

struct ResidualNormArgs {
  float* x;                 // [n][hidden]
  const float* y; long ldy; // [n][ldy] or null
  const float* add; int splits; size_t add_stride;   // [splits][n][hidden] or null
  const float* scale;       // [hidden] or null
  const float* w;           // [hidden]
  void* out;                // [n][hidden], compute type, or null
  int hidden;
  float alpha, eps;
};

// PER groups of four consecutive elements a thread, the row in registers between the two passes.
template <typename T, int PER>
__global__ __launch_bounds__(1024) void residual_norm_vec4_kernel(ResidualNormArgs a) {
  __shared__ float lds[16];
  const int row = blockIdx.x;
  const int chunks = a.hidden / 4;
  float* x = a.x + (size_t)row * a.hidden;
  f32x4 v[PER];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    v[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (c < chunks) {
      f32x4 yv = {0.f, 0.f, 0.f, 0.f};
      if (a.add) {
        for (int s = 0; s < a.splits; ++s)
          yv += *reinterpret_cast<const f32x4*>(a.add + s * a.add_stride + (size_t)row * a.hidden + 4 * c);
      } else if (a.y) {
        yv = *reinterpret_cast<const f32x4*>(a.y + (size_t)row * a.ldy + 4 * c);
      }
      if (a.scale) yv *= *reinterpret_cast<const f32x4*>(a.scale + 4 * c);
      const f32x4 xv = *reinterpret_cast<const f32x4*>(x + 4 * c);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        v[i][e] = __fmaf_rn(a.alpha, xv[e], yv[e]);
        ss = __fmaf_rn(v[i][e], v[i][e], ss);
      }
    }
  }
  const float total = tw_block_sum(ss, lds);
  const float rinv = 1.f / sqrtf(total / (float)a.hidden + a.eps);
  T* out = a.out ? (T*)a.out + (size_t)row * a.hidden : nullptr;
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    if (c < chunks) {
      const f32x4 wv = *reinterpret_cast<const f32x4*>(a.w + 4 * c);
      f32x4 r;
#pragma unroll
      for (int e = 0; e < 4; ++e) r[e] = v[i][e] * rinv * wv[e];
      *reinterpret_cast<f32x4*>(x + 4 * c) = r;
      if (out) {
#pragma unroll
        for (int e = 0; e < 4; ++e) out[4 * c + e] = tw_from_float<T>(r[e]);
      }
    }
  }
}

// Any row length: the sums are parked in x between the two passes (a thread reads back only what it wrote).
template <typename T>
__global__ void residual_norm_kernel(ResidualNormArgs a) {
  __shared__ float lds[16];
  const int row = blockIdx.x;
  float* x = a.x + (size_t)row * a.hidden;
  float ss = 0.f;
  for (int c = threadIdx.x; c < a.hidden; c += blockDim.x) {
    float yv = 0.f;
    if (a.add) {
      for (int s = 0; s < a.splits; ++s) yv += a.add[s * a.add_stride + (size_t)row * a.hidden + c];
    } else if (a.y) {
      yv = a.y[(size_t)row * a.ldy + c];
    }
    if (a.scale) yv *= a.scale[c];
    const float v = __fmaf_rn(a.alpha, x[c], yv);
    x[c] = v;
    ss = __fmaf_rn(v, v, ss);
  }
  const float total = tw_block_sum(ss, lds);
  const float rinv = 1.f / sqrtf(total / (float)a.hidden + a.eps);
  T* out = a.out ? (T*)a.out + (size_t)row * a.hidden : nullptr;
  for (int c = threadIdx.x; c < a.hidden; c += blockDim.x) {
    const float r = x[c] * rinv * a.w[c];
    x[c] = r;
    if (out) out[c] = tw_from_float<T>(r);
  }
}

template <typename T>
static void residual_norm_launch(const ResidualNormArgs& a, int n, hipStream_t stream) {
  const bool aligned = a.hidden % 4 == 0 && (uintptr_t)a.x % 16 == 0 && (uintptr_t)a.w % 16 == 0 &&
                       (!a.y || ((uintptr_t)a.y % 16 == 0 && a.ldy % 4 == 0)) &&
                       (!a.add || ((uintptr_t)a.add % 16 == 0 && a.add_stride % 4 == 0)) &&
                       (!a.scale || (uintptr_t)a.scale % 16 == 0);
  const int chunks = a.hidden / 4;
  if (aligned && chunks <= 4096) {
    const int per = chunks <= 1024 ? 1 : (chunks <= 2048 ? 2 : 4);
    int threads = (chunks + per - 1) / per;
    threads = (threads + 63) / 64 * 64;
    if (per == 1) residual_norm_vec4_kernel<T, 1><<<n, threads, 0, stream>>>(a);
    else if (per == 2) residual_norm_vec4_kernel<T, 2><<<n, threads, 0, stream>>>(a);
    else residual_norm_vec4_kernel<T, 4><<<n, threads, 0, stream>>>(a);
  } else {
    residual_norm_kernel<T><<<n, 256, 0, stream>>>(a);
  }
}

extern "C" int tw_residual_norm(int out_dtype, float* x, const float* y, long ldy, const float* add, int splits,
                                long add_stride, const float* scale, const float* w, void* out, int n, int hidden,
                                float alpha, float eps, hipStream_t stream) {
  TW_REQUIRE(x && w && n >= 0 && hidden > 0 && eps > 0.f);
  TW_REQUIRE(add == nullptr || (splits > 0 && add_stride >= (long)n * hidden));
  TW_REQUIRE(y == nullptr || ldy >= hidden);
  if (n == 0) return 0;
  ResidualNormArgs a{x, add ? nullptr : y, ldy, add, splits, (size_t)add_stride, scale, w, out, hidden, alpha, eps};
  if (out_dtype == TW_DTYPE_BF16) residual_norm_launch<bf16_t>(a, n, stream);
  else if (out_dtype == TW_DTYPE_F32) residual_norm_launch<float>(a, n, stream);
  else return TW_ERR_BAD_ARGUMENT;
  return TW_LAUNCH_RESULT();
}

// ---- x <- max(x, 0)^2 in place ---------------------------------------------------------------------------
template <typename T>
__global__ void relu_squared_kernel(T* __restrict__ x, long ld, int cols, long total) {
  const long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= total) return;
  const long row = i / cols;
  const int col = (int)(i % cols);
  T* p = x + row * ld + col;
  const float v = fmaxf(tw_to_float(*p), 0.f);
  *p = tw_from_float<T>(v * v);
}

// The same from split-K partial sums of the product before (float32 [splits][n][cols], added in index order): one
// rounding, and no kernel of its own for the sums.
template <typename T>
__global__ void relu_squared_sums_kernel(const float* __restrict__ partial, int splits, T* __restrict__ x, long ld, int cols,
                                         long total) {
  const long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= total) return;
  float v = 0.f;
  for (int s = 0; s < splits; ++s) v += partial[(size_t)s * total + i];
  v = fmaxf(v, 0.f);
  x[(i / cols) * ld + i % cols] = tw_from_float<T>(v * v);
}

extern "C" int tw_relu_squared(int dtype, void* x, long ld, int n, int cols, const float* partial, int splits,
                               hipStream_t stream) {
  TW_REQUIRE(x && n >= 0 && cols > 0 && ld >= cols && (partial == nullptr || splits > 0));
  if (n == 0) return 0;
  const long total = (long)n * cols;
  const int blocks = tw_div_up(total, 256);
  if (partial) {
    if (dtype == TW_DTYPE_BF16) relu_squared_sums_kernel<bf16_t><<<blocks, 256, 0, stream>>>(partial, splits, (bf16_t*)x, ld, cols, total);
    else if (dtype == TW_DTYPE_F32) relu_squared_sums_kernel<float><<<blocks, 256, 0, stream>>>(partial, splits, (float*)x, ld, cols, total);
    else return TW_ERR_BAD_ARGUMENT;
    return TW_LAUNCH_RESULT();
  }
  if (dtype == TW_DTYPE_BF16) relu_squared_kernel<bf16_t><<<blocks, 256, 0, stream>>>((bf16_t*)x, ld, cols, total);
  else if (dtype == TW_DTYPE_F32) relu_squared_kernel<float><<<blocks, 256, 0, stream>>>((float*)x, ld, cols, total);
  else return TW_ERR_BAD_ARGUMENT;
  return TW_LAUNCH_RESULT();
}

// ---- a norm on the sublayer's RESULT: x <- x + mult * w * unit(y) -------------------------------------------------
// y is a sublayer's float32 result (or split-K partial sums that are added up here, in index order); its statistic is
// float32; the sum goes back into the float32 stream x and, rounded once, to `out` in the compute type, which is what
// the next sublayer's products read (such an arrangement's sublayers read the stream itself). A block a row, four
// elements a thread and pass where rows and addresses allow; the row of y stays in registers between the two passes
// up to 4,096 elements, longer rows are read again.
struct AddNormedArgs {
  float* x;
  const float* y; long ldy;
  const float* add; int splits; size_t add_stride;
  const float* w;
  void* out;
  int hidden;
  float mult, eps;
};

template <typename T, bool VEC>
__global__ __launch_bounds__(256) void add_normed_kernel(AddNormedArgs a) {
  __shared__ float lds[16];
  constexpr int W = VEC ? 4 : 1;
  constexpr int KEEP = 4;
  const int row = blockIdx.x;
  const int units = a.hidden / W;
  float* x = a.x + (size_t)row * a.hidden;
  auto load = [&](int u, float* v) {
#pragma unroll
    for (int e = 0; e < W; ++e) v[e] = 0.f;
    if (a.add) {
      for (int s = 0; s < a.splits; ++s) {
        const float* p = a.add + s * a.add_stride + (size_t)row * a.hidden + (size_t)u * W;
        if (VEC) {
          const f32x4 t = *reinterpret_cast<const f32x4*>(p);
#pragma unroll
          for (int e = 0; e < W; ++e) v[e] += t[e];
        } else {
          v[0] += p[0];
        }
      }
    } else {
      const float* p = a.y + (size_t)row * a.ldy + (size_t)u * W;
      if (VEC) {
        const f32x4 t = *reinterpret_cast<const f32x4*>(p);
#pragma unroll
        for (int e = 0; e < W; ++e) v[e] = t[e];
      } else {
        v[0] = p[0];
      }
    }
  };
  float kept[KEEP][W];
  float ss = 0.f;
  int i = 0;
  for (int u = threadIdx.x; u < units; u += blockDim.x, ++i) {
    float v[W];
    load(u, v);
#pragma unroll
    for (int e = 0; e < W; ++e) ss = __fmaf_rn(v[e], v[e], ss);
    if (i < KEEP) {
#pragma unroll
      for (int e = 0; e < W; ++e) kept[i][e] = v[e];
    }
  }
  const float total = tw_block_sum(ss, lds);
  const float f = a.mult / sqrtf(total / (float)a.hidden + a.eps);
  T* out = a.out ? (T*)a.out + (size_t)row * a.hidden : nullptr;
  i = 0;
  for (int u = threadIdx.x; u < units; u += blockDim.x, ++i) {
    float v[W];
    if (i < KEEP) {
#pragma unroll
      for (int e = 0; e < W; ++e) v[e] = kept[i][e];
    } else {
      load(u, v);
    }
#pragma unroll
    for (int e = 0; e < W; ++e) {
      const int c = u * W + e;
      const float r = __fmaf_rn(v[e] * f, a.w[c], x[c]);
      x[c] = r;
      if (out) out[c] = tw_from_float<T>(r);
    }
  }
}

extern "C" int tw_add_normed(int out_dtype, float* x, const float* y, long ldy, const float* add, int splits, long add_stride,
                             const float* w, void* out, int n, int hidden, float mult, float eps, hipStream_t stream) {
  TW_REQUIRE(x && w && (y || add) && n >= 0 && hidden > 0 && eps > 0.f);
  TW_REQUIRE(add == nullptr || (splits > 0 && add_stride >= (long)n * hidden));
  TW_REQUIRE(add != nullptr || ldy >= hidden);
  if (n == 0) return 0;
  AddNormedArgs a{x, add ? nullptr : y, ldy, add, splits, (size_t)add_stride, w, out, hidden, mult, eps};
  const bool vec = hidden % 4 == 0 && (add ? ((uintptr_t)add % 16 == 0 && add_stride % 4 == 0)
                                           : ((uintptr_t)y % 16 == 0 && ldy % 4 == 0));
  if (out_dtype == TW_DTYPE_BF16) {
    if (vec) add_normed_kernel<bf16_t, true><<<n, 256, 0, stream>>>(a);
    else add_normed_kernel<bf16_t, false><<<n, 256, 0, stream>>>(a);
  } else if (out_dtype == TW_DTYPE_F32) {
    if (vec) add_normed_kernel<float, true><<<n, 256, 0, stream>>>(a);
    else add_normed_kernel<float, false><<<n, 256, 0, stream>>>(a);
  } else {
    return TW_ERR_BAD_ARGUMENT;
  }
  return TW_LAUNCH_RESULT();
}

// ---- activations of a plain product, in place: kind 1 max(x, 0)^2 (above), 2 the exact gelu, x Phi(x) -------------
__device__ __forceinline__ float sl_act(float v, int kind) {
  if (kind == 2) return 0.5f * v * (1.f + erff(v * 0.70710678118654752f));
  v = fmaxf(v, 0.f);
  return v * v;
}

template <typename T>
__global__ void activation_kernel(T* __restrict__ x, long ld, int cols, long total, const float* __restrict__ partial, int splits,
                                  int kind) {
  const long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= total) return;
  T* p = x + (i / cols) * ld + i % cols;
  float v = 0.f;
  if (partial) {
    for (int s = 0; s < splits; ++s) v += partial[(size_t)s * total + i];
  } else {
    v = tw_to_float(*p);
  }
  *p = tw_from_float<T>(sl_act(v, kind));
}

extern "C" int tw_activation(int dtype, void* x, long ld, int n, int cols, const float* partial, int splits, int kind,
                             hipStream_t stream) {
  TW_REQUIRE(x && n >= 0 && cols > 0 && ld >= cols && (partial == nullptr || splits > 0) && (kind == 1 || kind == 2));
  if (n == 0) return 0;
  const long total = (long)n * cols;
  const int blocks = tw_div_up(total, 256);
  if (dtype == TW_DTYPE_BF16) activation_kernel<bf16_t><<<blocks, 256, 0, stream>>>((bf16_t*)x, ld, cols, total, partial, splits, kind);
  else if (dtype == TW_DTYPE_F32) activation_kernel<float><<<blocks, 256, 0, stream>>>((float*)x, ld, cols, total, partial, splits, kind);
  else return TW_ERR_BAD_ARGUMENT;
  return TW_LAUNCH_RESULT();
}

// ---- out <- out * sigmoid(gate), element by element (an output gate in front of the output product) ---------------
template <typename T, typename G>
__global__ void sigmoid_gate_kernel(T* __restrict__ out, long ld_out, const G* __restrict__ gate, long ld_g, int cols, long total) {
  const long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= total) return;
  const long row = i / cols;
  const int col = (int)(i % cols);
  T* p = out + row * ld_out + col;
  const float z = tw_to_float(gate[row * ld_g + col]);
  *p = tw_from_float<T>(tw_to_float(*p) / (1.f + expf(-z)));
}

extern "C" int tw_sigmoid_gate(int dtype, void* out, long ld_out, const void* gate, long ld_g, int gate_f32, int n, int cols,
                               hipStream_t stream) {
  TW_REQUIRE(out && gate && n >= 0 && cols > 0 && ld_out >= cols && ld_g >= cols);
  if (n == 0) return 0;
  const long total = (long)n * cols;
  const int blocks = tw_div_up(total, 256);
  if (dtype == TW_DTYPE_BF16 && gate_f32)
    sigmoid_gate_kernel<bf16_t, float><<<blocks, 256, 0, stream>>>((bf16_t*)out, ld_out, (const float*)gate, ld_g, cols, total);
  else if (dtype == TW_DTYPE_BF16)
    sigmoid_gate_kernel<bf16_t, bf16_t><<<blocks, 256, 0, stream>>>((bf16_t*)out, ld_out, (const bf16_t*)gate, ld_g, cols, total);
  else if (dtype == TW_DTYPE_F32)
    sigmoid_gate_kernel<float, float><<<blocks, 256, 0, stream>>>((float*)out, ld_out, (const float*)gate, ld_g, cols, total);
  else return TW_ERR_BAD_ARGUMENT;
  return TW_LAUNCH_RESULT();
}

// ---- x <- cap * tanh(x / cap) over float32 values (a soft cap of the logits) ---------------------------------------
__global__ void softcap_values_kernel(float* __restrict__ x, long total, float cap) {
  const long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (i < total) x[i] = cap * tanhf(x[i] / cap);
}

extern "C" int tw_softcap_values(float* x, long total, float cap, hipStream_t stream) {
  TW_REQUIRE(x && total >= 0 && cap > 0.f);
  if (total == 0) return 0;
  softcap_values_kernel<<<tw_div_up(total, 256), 256, 0, stream>>>(x, total, cap);
  return TW_LAUNCH_RESULT();
}

// ---- several results side by side, each normed, summed into the stream: x <- x + sum_b mult_b * w_b * unit(y_b) ----
// Every y_b [n][hidden] is float32, or the split-K partial sums of a product that are added up here, in index order. A
// block a row.
#define TW_NORMED_SUM_MOST 4
struct NormedSumArgs {
  float* x;
  const float* y[TW_NORMED_SUM_MOST];
  const float* w[TW_NORMED_SUM_MOST];
  float mult[TW_NORMED_SUM_MOST];
  int splits[TW_NORMED_SUM_MOST];       // partial sums of y_b (1: y_b itself), n * hidden floats apart
  size_t stride;
  int count, hidden;
  float eps;
};

// PER groups of four consecutive elements a thread, COUNT results: all rows are on their way before the first is used, and
// their sums of squares meet in one reduction.
template <int COUNT, int PER>
__global__ __launch_bounds__(1024) void add_normed_sum_vec4_kernel(NormedSumArgs a) {
  __shared__ float lds[COUNT][16];
  const size_t row0 = (size_t)blockIdx.x * a.hidden;
  const int chunks = a.hidden / 4;
  f32x4 v[COUNT][PER];
  float ss[COUNT];
#pragma unroll
  for (int b = 0; b < COUNT; ++b) {
    ss[b] = 0.f;
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int c = threadIdx.x + i * blockDim.x;
      v[b][i] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (c < chunks) {
        const float* y = a.y[b] + row0 + 4 * c;
#pragma unroll 8
        for (int s = 0; s < a.splits[b]; ++s) v[b][i] += *reinterpret_cast<const f32x4*>(y + s * a.stride);
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) ss[b] = __fmaf_rn(v[b][i][e], v[b][i][e], ss[b]);
    }
  }
  const int wave = threadIdx.x / TW_WAVE, waves = blockDim.x / TW_WAVE;
#pragma unroll
  for (int b = 0; b < COUNT; ++b) {
    const float t = tw_wave_sum(ss[b]);
    if (threadIdx.x % TW_WAVE == 0) lds[b][wave] = t;
  }
  __syncthreads();
  float f[COUNT];
#pragma unroll
  for (int b = 0; b < COUNT; ++b) {
    float t = 0.f;
    for (int w = 0; w < waves; ++w) t += lds[b][w];
    f[b] = a.mult[b] / sqrtf(t / (float)a.hidden + a.eps);
  }
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    if (c < chunks) {
      f32x4* x = reinterpret_cast<f32x4*>(a.x + row0 + 4 * c);
      f32x4 sum = *x;
#pragma unroll
      for (int b = 0; b < COUNT; ++b)
#pragma unroll
        for (int e = 0; e < 4; ++e) sum[e] = __fmaf_rn(v[b][i][e] * f[b], a.w[b][4 * c + e], sum[e]);
      *x = sum;
    }
  }
}

// Any row length: every result is read twice.
__global__ __launch_bounds__(256) void add_normed_sum_kernel(NormedSumArgs a) {
  __shared__ float lds[16];
  const size_t row0 = (size_t)blockIdx.x * a.hidden;
  for (int b = 0; b < a.count; ++b) {
    const float* y = a.y[b] + row0;
    auto value = [&](int c) {
      float v = 0.f;
      for (int s = 0; s < a.splits[b]; ++s) v += y[s * a.stride + c];
      return v;
    };
    float ss = 0.f;
    for (int c = threadIdx.x; c < a.hidden; c += 256) {
      const float v = value(c);
      ss = __fmaf_rn(v, v, ss);
    }
    const float f = a.mult[b] / sqrtf(tw_block_sum(ss, lds) / (float)a.hidden + a.eps);
    for (int c = threadIdx.x; c < a.hidden; c += 256) a.x[row0 + c] = __fmaf_rn(value(c) * f, a.w[b][c], a.x[row0 + c]);
  }
}

template <int COUNT>
static void add_normed_sum_launch(const NormedSumArgs& a, int n, hipStream_t stream) {
  const int chunks = a.hidden / 4;
  const int per = chunks <= 1024 ? 1 : 2;
  const int threads = (tw_div_up(chunks, per) + 63) / 64 * 64;
  if (per == 1) add_normed_sum_vec4_kernel<COUNT, 1><<<n, threads, 0, stream>>>(a);
  else add_normed_sum_vec4_kernel<COUNT, 2><<<n, threads, 0, stream>>>(a);
}

extern "C" int tw_add_normed_sum(float* x, int count, const float* const* ys, const int* splits, const float* const* ws,
                                 const float* mults, int n, int hidden, float eps, hipStream_t stream) {
  TW_REQUIRE(x && ys && splits && ws && mults && n >= 0 && hidden > 0 && eps > 0.f && count > 0 && count <= TW_NORMED_SUM_MOST);
  NormedSumArgs a{};
  a.x = x;
  a.stride = (size_t)n * hidden;
  a.count = count;
  a.hidden = hidden;
  a.eps = eps;
  bool vec = hidden % 4 == 0 && (uintptr_t)x % 16 == 0;
  for (int b = 0; b < count; ++b) {
    TW_REQUIRE(ys[b] && ws[b] && splits[b] > 0);
    a.y[b] = ys[b];
    a.w[b] = ws[b];
    a.mult[b] = mults[b];
    a.splits[b] = splits[b];
    vec = vec && (uintptr_t)ys[b] % 16 == 0;
  }
  if (n == 0) return 0;
  if (vec && hidden <= 8192) {
    if (count == 1) add_normed_sum_launch<1>(a, n, stream);
    else if (count == 2) add_normed_sum_launch<2>(a, n, stream);
    else if (count == 3) add_normed_sum_launch<3>(a, n, stream);
    else add_normed_sum_launch<4>(a, n, stream);
  } else {
    add_normed_sum_kernel<<<n, 256, 0, stream>>>(a);
  }
  return TW_LAUNCH_RESULT();
}

// ---- x += y over float32 values --------------------------------------------------------------------------------------
__global__ void add_values_kernel(float* __restrict__ x, const float* __restrict__ y, long total) {
  const long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (i < total) x[i] += y[i];
}

extern "C" int tw_add_values(float* x, const float* y, long total, hipStream_t stream) {
  TW_REQUIRE(x && y && total >= 0);
  if (total == 0) return 0;
  add_values_kernel<<<tw_div_up(total, 256), 256, 0, stream>>>(x, y, total);
  return TW_LAUNCH_RESULT();
}

// ---- layer norms: a sublayer's result normed into the stream, and the stream normed for the next sublayer ------------
//   x <- x + [norm1](y),  out <- norm2(x),    norm(v) = (v - mean) / sqrt(mean((v - mean)^2) + eps) * w + b
// Every step is optional: no y (norm2 alone), no norm1 (y is added as it is), no out. y is float32 rows, or split-K partial
// sums that are added up here in index order, and / or the rows of a token's routed experts, weighted (pair i's row is
// pos[i]; a choice without a row adds nothing). Statistics and sums are float32; out is rounded once to the compute type.
// rows (or null): the rows of x and y that out's rows are formed from; x then stays as it is. A block a row.
struct LayerNormArgs {
  float* x;
  const float* y; long ldy;
  const float* add; int splits; size_t add_stride;
  const float* pair_rows; const int* pos; const float* pair_weights; int top;      // [.][hidden], [n][top], [n][top]
  const float* w1; const float* b1;
  const float* w2; const float* b2;
  void* out;
  const int* rows;
  int hidden;
  float eps;
};

// PER groups of four consecutive elements a thread, the row in registers.
template <typename T, int PER>
__global__ __launch_bounds__(1024) void layer_norm_vec4_kernel(LayerNormArgs a) {
  __shared__ float lds[16];
  const int row = a.rows ? a.rows[blockIdx.x] : blockIdx.x;
  const int chunks = a.hidden / 4;
  float* x = a.x + (size_t)row * a.hidden;
  const bool has_y = a.y || a.add || a.top > 0;
  f32x4 xv[PER], yv[PER];
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    xv[i] = yv[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (c < chunks) {
      xv[i] = *reinterpret_cast<const f32x4*>(x + 4 * c);
      if (a.add) {
        const float* p = a.add + (size_t)row * a.hidden + 4 * c;
#pragma unroll 8
        for (int s = 0; s < a.splits; ++s) yv[i] += *reinterpret_cast<const f32x4*>(p + s * a.add_stride);
      } else if (a.y) {
        yv[i] = *reinterpret_cast<const f32x4*>(a.y + (size_t)row * a.ldy + 4 * c);
      }
#pragma unroll 4
      for (int r = 0; r < a.top; ++r) {
        const int at = a.pos[(size_t)row * a.top + r];
        if (at >= 0) yv[i] += a.pair_weights[(size_t)row * a.top + r] * *reinterpret_cast<const f32x4*>(a.pair_rows + (size_t)at * a.hidden + 4 * c);
      }
    }
  }
  // (mean, one over the deviation) of a row in registers
  auto statistics = [&](const f32x4 (&v)[PER], float& mean, float& rinv) {
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < PER; ++i) s += (v[i][0] + v[i][1]) + (v[i][2] + v[i][3]);
    mean = tw_block_sum(s, lds) / (float)a.hidden;
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < PER; ++i)
      if (threadIdx.x + i * blockDim.x < chunks) {
#pragma unroll
        for (int e = 0; e < 4; ++e) ss = __fmaf_rn(v[i][e] - mean, v[i][e] - mean, ss);
      }
    rinv = 1.f / sqrtf(tw_block_sum(ss, lds) / (float)a.hidden + a.eps);
  };
  if (has_y) {
    float mean = 0.f, rinv = 1.f;
    if (a.w1) statistics(yv, mean, rinv);
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int c = threadIdx.x + i * blockDim.x;
      if (c < chunks) {
        if (a.w1) {
          const f32x4 w = *reinterpret_cast<const f32x4*>(a.w1 + 4 * c), b = *reinterpret_cast<const f32x4*>(a.b1 + 4 * c);
#pragma unroll
          for (int e = 0; e < 4; ++e) yv[i][e] = __fmaf_rn((yv[i][e] - mean) * rinv, w[e], b[e]);
        }
        xv[i] += yv[i];
        if (!a.rows) *reinterpret_cast<f32x4*>(x + 4 * c) = xv[i];
      }
    }
  }
  if (!a.out) return;
  float mean, rinv;
  statistics(xv, mean, rinv);
  T* out = (T*)a.out + (size_t)blockIdx.x * a.hidden;
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    if (c < chunks) {
      const f32x4 w = *reinterpret_cast<const f32x4*>(a.w2 + 4 * c), b = *reinterpret_cast<const f32x4*>(a.b2 + 4 * c);
#pragma unroll
      for (int e = 0; e < 4; ++e) out[4 * c + e] = tw_from_float<T>(__fmaf_rn((xv[i][e] - mean) * rinv, w[e], b[e]));
    }
  }
}

// Any row length and alignment: what a pass needs is formed anew.
template <typename T>
__global__ __launch_bounds__(256) void layer_norm_kernel(LayerNormArgs a) {
  __shared__ float lds[16];
  const int row = a.rows ? a.rows[blockIdx.x] : blockIdx.x;
  float* x = a.x + (size_t)row * a.hidden;
  const bool has_y = a.y || a.add || a.top > 0;
  auto result = [&](int c) {
    float v = 0.f;
    if (a.add) {
      for (int s = 0; s < a.splits; ++s) v += a.add[s * a.add_stride + (size_t)row * a.hidden + c];
    } else if (a.y) {
      v = a.y[(size_t)row * a.ldy + c];
    }
    for (int r = 0; r < a.top; ++r) {
      const int at = a.pos[(size_t)row * a.top + r];
      if (at >= 0) v += a.pair_weights[(size_t)row * a.top + r] * a.pair_rows[(size_t)at * a.hidden + c];
    }
    return v;
  };
  auto statistics = [&](auto value, float& mean, float& rinv) {
    float s = 0.f, ss = 0.f;
    for (int c = threadIdx.x; c < a.hidden; c += 256) s += value(c);
    mean = tw_block_sum(s, lds) / (float)a.hidden;
    for (int c = threadIdx.x; c < a.hidden; c += 256) {
      const float d = value(c) - mean;
      ss = __fmaf_rn(d, d, ss);
    }
    rinv = 1.f / sqrtf(tw_block_sum(ss, lds) / (float)a.hidden + a.eps);
  };
  float mean1 = 0.f, rinv1 = 1.f, mean2 = 0.f, rinv2 = 1.f;
  if (has_y && a.w1) statistics(result, mean1, rinv1);
  auto sum = [&](int c) {
    if (!has_y) return x[c];
    const float y = result(c);
    return x[c] + (a.w1 ? __fmaf_rn((y - mean1) * rinv1, a.w1[c], a.b1[c]) : y);
  };
  if (a.out) statistics(sum, mean2, rinv2);
  T* out = (T*)a.out + (size_t)blockIdx.x * a.hidden;
  for (int c = threadIdx.x; c < a.hidden; c += 256) {
    const float v = sum(c);
    if (has_y && !a.rows) x[c] = v;
    if (a.out) out[c] = tw_from_float<T>(__fmaf_rn((v - mean2) * rinv2, a.w2[c], a.b2[c]));
  }
}

template <typename T>
static void layer_norm_launch(const LayerNormArgs& a, int n, hipStream_t stream) {
  auto ok = [](const void* p) { return (uintptr_t)p % 16 == 0; };            // (null is)
  const bool vec = a.hidden % 4 == 0 && ok(a.x) && ok(a.y) && a.ldy % 4 == 0 && ok(a.add) && a.add_stride % 4 == 0 &&
                   ok(a.pair_rows) && ok(a.w1) && ok(a.b1) && ok(a.w2) && ok(a.b2);
  const int chunks = a.hidden / 4;
  if (vec && chunks <= 4096) {
    const int per = chunks <= 1024 ? 1 : chunks <= 2048 ? 2 : 4;
    const int threads = (tw_div_up(chunks, per) + 63) / 64 * 64;
    if (per == 1) layer_norm_vec4_kernel<T, 1><<<n, threads, 0, stream>>>(a);
    else if (per == 2) layer_norm_vec4_kernel<T, 2><<<n, threads, 0, stream>>>(a);
    else layer_norm_vec4_kernel<T, 4><<<n, threads, 0, stream>>>(a);
  } else {
    layer_norm_kernel<T><<<n, 256, 0, stream>>>(a);
  }
}

extern "C" int tw_layer_norm(int out_dtype, float* x, const float* y, long ldy, const float* add, int splits, long add_stride,
                             const float* pair_rows, const int* pos, const float* pair_weights, int top, const float* w1,
                             const float* b1, const float* w2, const float* b2, void* out, const int* rows, int n_out, int hidden,
                             float eps, hipStream_t stream) {
  TW_REQUIRE(x && n_out >= 0 && hidden > 0 && eps > 0.f && (out || !rows) && top >= 0);
  TW_REQUIRE((!out || (w2 && b2)) && (!w1 || b1));
  TW_REQUIRE(!add || (splits > 0 && !y));
  TW_REQUIRE(!y || ldy >= hidden);
  TW_REQUIRE(top == 0 || (pair_rows && pos && pair_weights));
  if (n_out == 0) return 0;
  LayerNormArgs a{x, y, ldy, add, splits, (size_t)add_stride, pair_rows, pos, pair_weights, top, w1, b1, w2, b2, out, rows, hidden, eps};
  if (out_dtype == TW_DTYPE_BF16) layer_norm_launch<bf16_t>(a, n_out, stream);
  else if (out_dtype == TW_DTYPE_F32) layer_norm_launch<float>(a, n_out, stream);
  else return TW_ERR_BAD_ARGUMENT;
  return TW_LAUNCH_RESULT();
}
