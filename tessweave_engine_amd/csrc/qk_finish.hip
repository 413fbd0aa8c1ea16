// What stands between the projections and the attention of a mixer whose queries and keys are normed as WHOLE rows and
// whose values are its keys: per token
//
//   q <- rotate(w_q * unit(q)),  k <- rotate(w_k * unit(k)),  v = k as it came (before norm and rotation)
//
// unit(.) over all heads of the row at once (H D elements of q, G D of k), rotation of the first `rot` elements of
// every head (pairing 0: element j with j + rot / 2; 1: element 2 j with 2 j + 1), by the angles of the token's
// position. q and k come as float32 rows (the results of short convolutions); statistics, weights and rotation are
// float32, and each result is rounded once to the compute type. The queries go to q_out with heads of Dp elements
// (tails of zeros), keys and values into the token's page slot:
//   keys [pages][G][P][Dp], values [pages][G][Dp][P] (transposed inside a page).
#include "tw_common.h"

struct QkFinishArgs {
  const float* src; long ld;
  int q_col, k_col;
  const float* wq; const float* wk;
  const float* cos_t; const float* sin_t;      // [n][rot / 2]
  void* q_out; long ld_q;
  void* keys; void* values; const int* slots;
  int H, G, D, Dp, rot, pairing, P;
  float eps;
};

__device__ __forceinline__ float qf_turned(const float* row, const float* w, float rinv, int base, int d, int rot, int pairing,
                                           const float* cs, const float* sn) {
  // element d of a head that starts at row[base]: normed, then turned if d < rot
  auto normed = [&](int e) { return row[base + e] * rinv * w[base + e]; };
  if (d >= rot) return normed(d);
  const int half = rot / 2;
  int pair, other;
  bool first;
  if (pairing == 1) {
    pair = d >> 1;
    first = (d & 1) == 0;
    other = first ? d + 1 : d - 1;
  } else {
    first = d < half;
    pair = first ? d : d - half;
    other = first ? d + half : d - half;
  }
  const float mine = normed(d), theirs = normed(other);
  const float c = cs[pair], s = sn[pair];
  // (u, v) -> (u c - v s, v c + u s)
  return first ? __fmaf_rn(mine, c, -__fmul_rn(theirs, s)) : __fmaf_rn(mine, c, __fmul_rn(theirs, s));
}

template <typename T>
__global__ __launch_bounds__(256) void qk_finish_kernel(QkFinishArgs a) {
  __shared__ float lds[16];
  const int n = blockIdx.x;
  const float* row = a.src + (size_t)n * a.ld;
  const int nq = a.H * a.D, nk = a.G * a.D;
  float sq = 0.f, sk = 0.f;
  for (int i = threadIdx.x; i < nq; i += blockDim.x) sq = __fmaf_rn(row[a.q_col + i], row[a.q_col + i], sq);
  for (int i = threadIdx.x; i < nk; i += blockDim.x) sk = __fmaf_rn(row[a.k_col + i], row[a.k_col + i], sk);
  const float tq = tw_block_sum(sq, lds);
  const float tk = tw_block_sum(sk, lds);
  const float rq = 1.f / sqrtf(tq / (float)nq + a.eps), rk = 1.f / sqrtf(tk / (float)nk + a.eps);
  const float* cs = a.cos_t + (size_t)n * (a.rot / 2);
  const float* sn = a.sin_t + (size_t)n * (a.rot / 2);
  T* q = (T*)a.q_out + (size_t)n * a.ld_q;
  for (int i = threadIdx.x; i < a.H * a.Dp; i += blockDim.x) {
    const int head = i / a.Dp, d = i % a.Dp;
    float v = 0.f;
    if (d < a.D) v = qf_turned(row + a.q_col, a.wq, rq, head * a.D, d, a.rot, a.pairing, cs, sn);
    q[i] = tw_from_float<T>(v);
  }
  const int slot = a.slots[n];
  if (slot < 0) return;
  const int page = slot / a.P, at = slot % a.P;
  for (int i = threadIdx.x; i < a.G * a.Dp; i += blockDim.x) {
    const int kvh = i / a.Dp, d = i % a.Dp;
    float k = 0.f, v = 0.f;
    if (d < a.D) {
      k = qf_turned(row + a.k_col, a.wk, rk, kvh * a.D, d, a.rot, a.pairing, cs, sn);
      v = row[a.k_col + kvh * a.D + d];
    }
    ((T*)a.keys)[(((size_t)page * a.G + kvh) * a.P + at) * a.Dp + d] = tw_from_float<T>(k);
    ((T*)a.values)[(((size_t)page * a.G + kvh) * a.Dp + d) * a.P + at] = tw_from_float<T>(v);
  }
}

extern "C" int tw_qk_finish(int dtype, const float* src, long ld, int q_col, int k_col, const float* wq, const float* wk,
                            const float* cos_t, const float* sin_t, void* q_out, long ld_q, void* keys, void* values,
                            const int* slots, int n, int H, int G, int D, int Dp, int rot, int pairing, int page_size,
                            float eps, hipStream_t stream) {
  TW_REQUIRE(src && wq && wk && q_out && keys && values && slots && n >= 0 && H > 0 && G > 0 && D > 0 && Dp >= D);
  TW_REQUIRE(rot >= 0 && rot % 2 == 0 && rot <= D && (rot == 0 || (cos_t && sin_t)) && (pairing == 0 || pairing == 1));
  TW_REQUIRE(q_col >= 0 && k_col >= 0 && ld >= q_col + (long)H * D && ld >= k_col + (long)G * D && ld_q >= (long)H * Dp);
  TW_REQUIRE(page_size > 0 && eps > 0.f);
  if (n == 0) return 0;
  QkFinishArgs a{src, ld, q_col, k_col, wq, wk, cos_t, sin_t, q_out, ld_q, keys, values, slots, H, G, D, Dp, rot, pairing,
                 page_size, eps};
  if (dtype == TW_DTYPE_BF16) qk_finish_kernel<bf16_t><<<n, 256, 0, stream>>>(a);
  else if (dtype == TW_DTYPE_F32) qk_finish_kernel<float><<<n, 256, 0, stream>>>(a);
  else return TW_ERR_BAD_ARGUMENT;
  return TW_LAUNCH_RESULT();
}

// ---- queries and keys normed per head, without a rotation ----------------------------------------------------------
// What stands between the projections and the attention of a mixer whose heads are normed one by one and whose positions
// enter as a temperature of the queries:
//
//   q <- temperature(p) * unit(q_h),  k <- unit(k_g),  v as it comes;   temperature(p) = 1 + coef * ln(floor((p + 1) / every) + 1)
//
// unit(.) over a head's D elements. q, k and v are columns of float32 rows; each result is rounded once to the compute
// type: queries to q_out with heads of Dp elements (tails of zeros), keys and values (of E elements) into the token's page
// slot, keys [pages][G][P][Dp], values [pages][G][Dp][P]. One wave a (token, head): H query heads, then G key/value heads.
struct HeadFinishArgs {
  const float* src; long ld;
  int q_col, k_col, v_col;
  const int* positions;
  void* q_out; long ld_q;
  void* keys; void* values; const int* slots;
  int n, H, G, D, E, Dp, P;
  int every;                    // 0: no temperature
  float coef, eps;
};

template <typename T>
__global__ __launch_bounds__(256) void head_finish_kernel(HeadFinishArgs a) {
  const long unit = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (unit >= (long)a.n * (a.H + a.G)) return;
  const int lane = threadIdx.x & 63;
  const int n = (int)(unit / (a.H + a.G)), head = (int)(unit % (a.H + a.G));
  const bool query = head < a.H;
  const int g = head - a.H;
  const float* row = a.src + (size_t)n * a.ld;
  const float* x = row + (query ? a.q_col + head * a.D : a.k_col + g * a.D);
  float v[4], ss = 0.f;                           // D <= 256
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int d = lane + 64 * i;
    v[i] = d < a.D ? x[d] : 0.f;
    ss = __fmaf_rn(v[i], v[i], ss);
  }
  float f = 1.f / sqrtf(tw_wave_sum(ss) / (float)a.D + a.eps);
  if (query) {
    if (a.every > 0) f *= __fmaf_rn(a.coef, logf((float)((a.positions[n] + 1) / a.every + 1)), 1.f);
    T* q = (T*)a.q_out + (size_t)n * a.ld_q + (size_t)head * a.Dp;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = lane + 64 * i;
      if (d < a.Dp) q[d] = tw_from_float<T>(v[i] * f);
    }
    return;
  }
  const int slot = a.slots[n];
  if (slot < 0) return;
  const int page = slot / a.P, at = slot % a.P;
  T* k = (T*)a.keys + (((size_t)page * a.G + g) * a.P + at) * a.Dp;
  T* vals = (T*)a.values + ((size_t)page * a.G + g) * a.Dp * a.P + at;
  const float* value = row + a.v_col + g * a.E;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int d = lane + 64 * i;
    if (d < a.Dp) {
      k[d] = tw_from_float<T>(v[i] * f);
      vals[(size_t)d * a.P] = tw_from_float<T>(d < a.E ? value[d] : 0.f);
    }
  }
}

extern "C" int tw_head_finish(int dtype, const float* src, long ld, int q_col, int k_col, int v_col, const int* positions,
                              void* q_out, long ld_q, void* keys, void* values, const int* slots, int n, int H, int G, int D,
                              int E, int Dp, int page_size, int every, float coef, float eps, hipStream_t stream) {
  TW_REQUIRE(src && positions && q_out && keys && values && slots && n >= 0 && H > 0 && G > 0 && D > 0 && E > 0);
  TW_REQUIRE(Dp >= D && Dp >= E && Dp <= 256 && q_col >= 0 && k_col >= 0 && v_col >= 0 && ld >= q_col + (long)H * D &&
             ld >= k_col + (long)G * D && ld >= v_col + (long)G * E && ld_q >= (long)H * Dp);
  TW_REQUIRE(page_size > 0 && eps > 0.f && every >= 0);
  if (n == 0) return 0;
  HeadFinishArgs a{src, ld, q_col, k_col, v_col, positions, q_out, ld_q, keys, values, slots, n, H, G, D, E, Dp, page_size,
                   every, coef, eps};
  const int blocks = tw_div_up((long)n * (H + G), 4);
  if (dtype == TW_DTYPE_BF16) head_finish_kernel<bf16_t><<<blocks, 256, 0, stream>>>(a);
  else if (dtype == TW_DTYPE_F32) head_finish_kernel<float><<<blocks, 256, 0, stream>>>(a);
  else return TW_ERR_BAD_ARGUMENT;
  return TW_LAUNCH_RESULT();
}

// ---- rotated queries and keys, normed or not, values of their own, gates -----------------------------------------
// What stands between one packed projection and the attention over pages. Per token:
//
//   q <- rotate(norm(q)),  k <- rotate(norm(k)),  v <- v_scale * v,  gate <- sigmoid(g)         (bias added first, if any)
//
// norm: 0 none; 1 per head, weights of D elements that all heads share; 2 over the whole row at once, weights over the row
// (x / sqrt(mean(x^2) + eps) * w). Rotation of the first `rot` elements of every head (pairing as above). A head may have
// M = 2 MAPS, each with D elements of its own that are rotated like a head: a key then holds both maps side by side, and
// every (head, map) is a query of its own whose other half is zeros, so that plain attention over M H query heads and G key
// heads of M D elements gives every map's scores against the same values.
//   src   float32 rows, or the split-K sums of the projection [splits][n][ld], added up here in index order
//   q_out [n][H M][Dp], keys [pages][G][P][Dp], values [pages][G][Dp][P] in the compute type (tails of zeros)
//   gate  float32 [n][H]
// k_col < 0: no keys and values (a layer that reads another's pages); g_col < 0: no gate. One workgroup a token: q and k
// meet in LDS.
struct RowsFinishArgs {
  const float* src; long ld; int splits; size_t split_stride;
  const float* bias;
  int q_col, k_col, v_col, g_col;
  const float* wq; const float* wk; int norm;
  const float* cos_t; const float* sin_t;
  int rot, pairing;
  void* q_out; long ld_q;
  void* keys; void* values; const int* slots;
  float* gate;
  int H, G, M, D, E, Dp, P;
  float eps, v_scale;
  bool vec;                     // columns, row length and addresses allow 16-byte accesses
};

__device__ __forceinline__ float rf_rotated(const float* x, int d, int rot, int pairing, const float* cs, const float* sn) {
  if (d >= rot) return x[d];
  int pair, other;
  bool first;
  if (pairing == 1) {
    pair = d >> 1;
    first = (d & 1) == 0;
    other = d ^ 1;
  } else {
    const int half = rot / 2;
    first = d < half;
    pair = first ? d : d - half;
    other = first ? d + half : d - half;
  }
  const float c = cs[pair], s = sn[pair];
  return first ? __fmaf_rn(x[d], c, -__fmul_rn(x[other], s)) : __fmaf_rn(x[d], c, __fmul_rn(x[other], s));
}

template <typename T>
__device__ __forceinline__ void rf_store4(T* p, const float (&v)[4]) {
  struct alignas(4 * sizeof(T)) Four { T e[4]; };
  Four f;
#pragma unroll
  for (int j = 0; j < 4; ++j) f.e[j] = tw_from_float<T>(v[j]);
  *reinterpret_cast<Four*>(p) = f;
}

template <typename T>
__global__ __launch_bounds__(256) void rows_finish_kernel(RowsFinishArgs a) {
  extern __shared__ __attribute__((aligned(16))) float rf_lds[];
  __shared__ float red[16];
  const int n = blockIdx.x, tid = threadIdx.x;
  const float* row = a.src + (size_t)n * a.ld;
  const int nq = a.H * a.M * a.D, nk = a.k_col >= 0 ? a.G * a.M * a.D : 0;
  float* q_s = rf_lds;
  float* k_s = rf_lds + (nq + 3) / 4 * 4;
  auto column = [&](int c) {
    float v = row[c];
    for (int s = 1; s < a.splits; ++s) v += row[s * a.split_stride + c];
    return a.bias ? v + a.bias[c] : v;
  };
  auto four = [&](int c) {
    f32x4 v = *reinterpret_cast<const f32x4*>(row + c);
#pragma unroll 8
    for (int s = 1; s < a.splits; ++s) v += *reinterpret_cast<const f32x4*>(row + s * a.split_stride + c);
    if (a.bias) v += *reinterpret_cast<const f32x4*>(a.bias + c);
    return v;
  };
  // the row's queries and keys into LDS, their squares summed on the way
  auto stage = [&](float* dst, int col, int count) {
    float ss = 0.f;
    if (a.vec) {
      for (int i = 4 * tid; i < count; i += 1024) {
        f32x4 v;
        if (i + 4 <= count) v = four(col + i);
        else {
#pragma unroll
          for (int j = 0; j < 4; ++j) v[j] = i + j < count ? column(col + i + j) : 0.f;
        }
#pragma unroll
        for (int j = 0; j < 4; ++j) ss = __fmaf_rn(v[j], v[j], ss);
        *reinterpret_cast<f32x4*>(dst + i) = v;
      }
    } else {
      for (int i = tid; i < count; i += 256) {
        const float v = column(col + i);
        ss = __fmaf_rn(v, v, ss);
        dst[i] = v;
      }
    }
    return ss;
  };
  float sq = stage(q_s, a.q_col, nq), sk = nk ? stage(k_s, a.k_col, nk) : 0.f;
  const int slot = nk ? a.slots[n] : -1;
  const int page = slot >= 0 ? slot / a.P : 0, at = slot >= 0 ? slot % a.P : 0;
  if (slot >= 0) {                                    // values: straight from the row into the page
    for (int i = tid; i < a.G * a.Dp; i += 256) {
      const int g = i / a.Dp, e = i - g * a.Dp;
      const float v = e < a.E ? column(a.v_col + g * a.E + e) * a.v_scale : 0.f;
      ((T*)a.values)[(((size_t)page * a.G + g) * a.Dp + e) * a.P + at] = tw_from_float<T>(v);
    }
  }
  if (a.g_col >= 0)
    for (int i = tid; i < a.H; i += 256) a.gate[(size_t)n * a.H + i] = 1.f / (1.f + expf(-column(a.g_col + i)));
  if (a.norm == 2) {
    sq = tw_block_sum(sq, red);
    const float rq = 1.f / sqrtf(sq / (float)nq + a.eps);
    for (int i = tid; i < nq; i += 256) q_s[i] = q_s[i] * rq * a.wq[i];
    if (nk) {
      sk = tw_block_sum(sk, red);
      const float rk = 1.f / sqrtf(sk / (float)nk + a.eps);
      for (int i = tid; i < nk; i += 256) k_s[i] = k_s[i] * rk * a.wk[i];
    }
  } else if (a.norm == 1) {
    __syncthreads();
    const int lane = tid & 63, heads_q = a.H * a.M, heads = heads_q + (nk ? a.G * a.M : 0);
    for (int head = tid >> 6; head < heads; head += 4) {
      float* x = head < heads_q ? q_s + head * a.D : k_s + (head - heads_q) * a.D;
      const float* w = head < heads_q ? a.wq : a.wk;
      float v[4], ss = 0.f;                           // D <= 256
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = lane + 64 * i;
        v[i] = d < a.D ? x[d] : 0.f;
        ss = __fmaf_rn(v[i], v[i], ss);
      }
      const float f = 1.f / sqrtf(tw_wave_sum(ss) / (float)a.D + a.eps);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = lane + 64 * i;
        if (d < a.D) x[d] = v[i] * f * w[d];
      }
    }
  }
  __syncthreads();
  const float* cs = a.cos_t + (size_t)n * (a.rot / 2);
  const float* sn = a.sin_t + (size_t)n * (a.rot / 2);
  const int pieces = a.Dp / 4;
  T* q = (T*)a.q_out + (size_t)n * a.ld_q;
  for (int i = tid; i < a.H * a.M * pieces; i += 256) {
    const int vh = i / pieces, d0 = (i - vh * pieces) * 4;
    const int from = a.M == 2 ? (vh & 1) * a.D : 0;   // where the map's elements lie among the key's
    float v[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int d = d0 + j - from;
      v[j] = d >= 0 && d < a.D ? rf_rotated(q_s + vh * a.D, d, a.rot, a.pairing, cs, sn) : 0.f;
    }
    rf_store4<T>(q + (size_t)vh * a.Dp + d0, v);
  }
  if (slot < 0) return;
  for (int i = tid; i < a.G * pieces; i += 256) {
    const int g = i / pieces, d0 = (i - g * pieces) * 4;
    float v[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int d = d0 + j, m = d >= a.D ? 1 : 0;
      v[j] = d < a.M * a.D ? rf_rotated(k_s + (g * a.M + m) * a.D, d - m * a.D, a.rot, a.pairing, cs, sn) : 0.f;
    }
    rf_store4<T>((T*)a.keys + (((size_t)page * a.G + g) * a.P + at) * a.Dp + d0, v);
  }
}

extern "C" int tw_rows_finish(int dtype, const float* src, long ld, int splits, long split_stride, const float* bias, int q_col,
                              int k_col, int v_col, int g_col, int norm, const float* wq, const float* wk, const float* cos_t,
                              const float* sin_t, int rot, int pairing, void* q_out, long ld_q, void* keys, void* values,
                              const int* slots, float* gate, int n, int H, int G, int M, int D, int E, int Dp, int page_size,
                              float eps, float v_scale, hipStream_t stream) {
  TW_REQUIRE(src && q_out && n >= 0 && H > 0 && G > 0 && (M == 1 || M == 2) && D > 0 && D <= 256 && splits >= 1);
  TW_REQUIRE(Dp % 16 == 0 && Dp >= M * D && Dp <= 256 && q_col >= 0 && ld >= q_col + (long)H * M * D && ld_q >= (long)H * M * Dp);
  TW_REQUIRE(splits == 1 || split_stride >= (long)n * ld);
  TW_REQUIRE(k_col < 0 || (keys && values && slots && page_size > 0 && E > 0 && E <= Dp && v_col >= 0 &&
                           ld >= k_col + (long)G * M * D && ld >= v_col + (long)G * E));
  TW_REQUIRE(g_col < 0 || (gate && ld >= (long)g_col + H));
  TW_REQUIRE(norm >= 0 && norm <= 2 && (norm == 0 || (wq && (wk || k_col < 0) && eps > 0.f)));
  TW_REQUIRE(rot >= 0 && rot % 2 == 0 && rot <= D && (rot == 0 || (cos_t && sin_t)) && (pairing == 0 || pairing == 1));
  TW_REQUIRE((uintptr_t)q_out % 16 == 0 && ld_q % 4 == 0 && (k_col < 0 || (uintptr_t)keys % 16 == 0));
  const int nq = H * M * D, nk = k_col < 0 ? 0 : G * M * D;
  const size_t lds = ((size_t)(nq + 3) / 4 * 4 + (size_t)(nk + 3) / 4 * 4) * sizeof(float);
  TW_REQUIRE(lds <= 128 * 1024);
  if (n == 0) return 0;
  const bool vec = ld % 4 == 0 && split_stride % 4 == 0 && q_col % 4 == 0 && (k_col < 0 || k_col % 4 == 0) &&
                   (uintptr_t)src % 16 == 0 && (!bias || (uintptr_t)bias % 16 == 0);
  RowsFinishArgs a{src, ld, splits, (size_t)split_stride, bias, q_col, k_col, v_col, g_col, wq, wk, norm, cos_t, sin_t, rot, pairing,
                   q_out, ld_q, keys, values, slots, gate, H, G, M, D, E, Dp, page_size > 0 ? page_size : 1, eps, v_scale, vec};
  static bool allowed = false;
  if (!allowed) {
    hipError_t e = hipFuncSetAttribute((const void*)rows_finish_kernel<bf16_t>, hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024);
    if (e == hipSuccess)
      e = hipFuncSetAttribute((const void*)rows_finish_kernel<float>, hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024);
    if (e != hipSuccess) return (int)e;
    allowed = true;
  }
  if (dtype == TW_DTYPE_BF16) rows_finish_kernel<bf16_t><<<n, 256, lds, stream>>>(a);
  else if (dtype == TW_DTYPE_F32) rows_finish_kernel<float><<<n, 256, lds, stream>>>(a);
  else return TW_ERR_BAD_ARGUMENT;
  return TW_LAUNCH_RESULT();
}

// ---- two maps of a head combined -----------------------------------------------------------------------------------
// Differential attention: a1 and a2 (E elements each of Dp, float32) are what a head's two maps give over the same values;
//   o = a1 - lambda a2,   out = o / sqrt(mean(o^2) + eps) * factor * gate            (gate: one number a (token, head), or null)
// rounded once to the compute type, heads Ep elements apart (tails of zeros). A wave a (token, head).
template <typename T>
__global__ __launch_bounds__(256) void map_difference_kernel(const float* __restrict__ src, long ld, const float* __restrict__ gate,
                                                             T* __restrict__ out, long ld_out, int n, int H, int E, int Dp,
                                                             int Ep, float lambda, float factor, float eps) {
  const long unit = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (unit >= (long)n * H) return;
  const int lane = threadIdx.x & 63, row = (int)(unit / H), head = (int)(unit % H);
  const float* a1 = src + (size_t)row * ld + (size_t)head * 2 * Dp;
  const float* a2 = a1 + Dp;
  float v[4], ss = 0.f;                               // E <= 256
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int e = lane + 64 * i;
    v[i] = e < E ? __fmaf_rn(-lambda, a2[e], a1[e]) : 0.f;
    ss = __fmaf_rn(v[i], v[i], ss);
  }
  float f = factor / sqrtf(tw_wave_sum(ss) / (float)E + eps);
  if (gate) f *= gate[(size_t)row * H + head];
  T* dst = out + (size_t)row * ld_out + (size_t)head * Ep;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int e = lane + 64 * i;
    if (e < Ep) dst[e] = tw_from_float<T>(v[i] * f);
  }
}

extern "C" int tw_map_difference(int dtype, const float* src, long ld, const float* gate, void* out, long ld_out, int n, int H,
                                 int E, int Dp, int Ep, float lambda, float factor, float eps, hipStream_t stream) {
  TW_REQUIRE(src && out && n >= 0 && H > 0 && E > 0 && E <= 256 && Dp >= E && Ep >= E && Ep <= 256 && eps > 0.f);
  TW_REQUIRE(ld >= 2L * H * Dp && ld_out >= (long)H * Ep);
  if (n == 0) return 0;
  const int blocks = tw_div_up((long)n * H, 4);
  if (dtype == TW_DTYPE_BF16)
    map_difference_kernel<bf16_t><<<blocks, 256, 0, stream>>>(src, ld, gate, (bf16_t*)out, ld_out, n, H, E, Dp, Ep, lambda, factor, eps);
  else if (dtype == TW_DTYPE_F32)
    map_difference_kernel<float><<<blocks, 256, 0, stream>>>(src, ld, gate, (float*)out, ld_out, n, H, E, Dp, Ep, lambda, factor, eps);
  else return TW_ERR_BAD_ARGUMENT;
  return TW_LAUNCH_RESULT();
}
