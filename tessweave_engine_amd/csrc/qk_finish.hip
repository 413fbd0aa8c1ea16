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
// The angles are positions times freq + rest (rest, or null: what float32 rounded off the frequencies), formed here with the
// product's rounding error beside it.
//   q_out [n][H M][Dp], keys [pages][G][P][Dp], values [pages][G][Dp][P] in the compute type (tails of zeros)
//   gate  float32 [n][H]
// k_col < 0: no keys and values (a layer that reads another's pages); g_col < 0: no gate. A token's q and k
// meet in LDS.
struct RowsFinishArgs {
  const float* src; long ld; int splits; size_t split_stride;
  const float* bias;
  int q_col, k_col, v_col, g_col;
  const float* wq; const float* wk; int norm;
  const int* positions; const float* freq; const float* rest;
  int rot, pairing;
  void* q_out; long ld_q;
  void* keys; void* values; const int* slots;
  float* gate;
  int H, G, M, D, E, Dp, P;
  float eps, v_scale;
  bool vec;                     // columns, row length and addresses allow 16-byte accesses
  int n;                        // tokens
};

#define RF_TILE 16              /* tokens whose values one workgroup writes in steps of many rows */
#define RF_FEW 64               /* up to this many rows a token's workgroup is wide and writes its own values */

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

// Elements d .. d + 3 of a head; whole (sizes allow it): in 16-byte pieces, d a multiple of 4.
__device__ __forceinline__ f32x4 rf_rotated4(const float* x, int d, int D, int rot, int pairing, const float* cs, const float* sn, bool whole) {
  f32x4 v;
  if (!whole) {
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = d + j >= 0 && d + j < D ? rf_rotated(x, d + j, rot, pairing, cs, sn) : 0.f;
    return v;
  }
  if (d < 0 || d >= D) return f32x4{0.f, 0.f, 0.f, 0.f};
  v = *reinterpret_cast<const f32x4*>(x + d);
  if (d >= rot) return v;
  if (pairing == 1) {
    const float c0 = cs[d / 2], c1 = cs[d / 2 + 1], s0 = sn[d / 2], s1 = sn[d / 2 + 1];
    return f32x4{__fmaf_rn(v[0], c0, -__fmul_rn(v[1], s0)), __fmaf_rn(v[1], c0, __fmul_rn(v[0], s0)),
                 __fmaf_rn(v[2], c1, -__fmul_rn(v[3], s1)), __fmaf_rn(v[3], c1, __fmul_rn(v[2], s1))};
  }
  const int half = rot / 2;
  const bool first = d < half;
  const int pair = first ? d : d - half;
  const f32x4 other = *reinterpret_cast<const f32x4*>(x + (first ? d + half : d - half));
  const f32x4 c = *reinterpret_cast<const f32x4*>(cs + pair), s = *reinterpret_cast<const f32x4*>(sn + pair);
#pragma unroll
  for (int j = 0; j < 4; ++j) v[j] = first ? __fmaf_rn(v[j], c[j], -__fmul_rn(other[j], s[j])) : __fmaf_rn(v[j], c[j], __fmul_rn(other[j], s[j]));
  return v;
}

// Sum over the 16 lanes of a row of the wave; every lane gets it.
template <int CTRL>
__device__ __forceinline__ float rf_turned_row(float v) {
  return __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), CTRL, 0xf, 0xf, true));
}
__device__ __forceinline__ float rf_row_sum(float v) {
  v += rf_turned_row<0x128>(v);
  v += rf_turned_row<0x124>(v);
  v += rf_turned_row<0x122>(v);
  v += rf_turned_row<0x121>(v);
  return v;
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
__device__ __forceinline__ void rf_store4(T* p, f32x4 v) {
  const float e[4] = {v[0], v[1], v[2], v[3]};
  rf_store4<T>(p, e);
}

// One column of a token's row: its split-K sums added up in index order, then the bias.
__device__ __forceinline__ float rf_column(const RowsFinishArgs& a, const float* row, int c) {
  float v = row[c];
  for (int s = 1; s < a.splits; ++s) v += row[s * a.split_stride + c];
  return a.bias ? v + a.bias[c] : v;
}

// The values of 16 tokens: a thread takes one element of one head and writes it for all of them, eight tokens a store where
// they are neighbours in a page (values lie transposed there).
template <typename T>
__device__ void rf_values(const RowsFinishArgs& a, int tile, int column_block) {
  const int i = column_block * blockDim.x + threadIdx.x;
  if (i >= a.G * a.Dp) return;
  const int g = i / a.Dp, e = i - g * a.Dp, t0 = tile * RF_TILE;
  const bool real = e < a.E;
  float v[RF_TILE];
#pragma unroll
  for (int j = 0; j < RF_TILE; ++j) v[j] = real && t0 + j < a.n ? rf_column(a, a.src + (size_t)(t0 + j) * a.ld, a.v_col + g * a.E + e) : 0.f;
#pragma unroll
  for (int half = 0; half < RF_TILE; half += 8) {
    const int t = t0 + half;
    if (t >= a.n) return;
    const int first = a.slots[t];
    bool together = first >= 0 && first % 8 == 0 && a.P % 8 == 0 && t + 8 <= a.n;
    if (together) {
#pragma unroll
      for (int j = 1; j < 8; ++j) together = together && a.slots[t + j] == first + j;
    }
    auto place = [&](int slot) { return (T*)a.values + (((size_t)(slot / a.P) * a.G + g) * a.Dp + e) * a.P + slot % a.P; };
    if (together) {
      T* to = place(first);
#pragma unroll
      for (int q = 0; q < 8; q += 4) {
        float four[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) four[j] = v[half + q + j] * a.v_scale;
        rf_store4<T>(to + q, four);
      }
    } else {
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const int slot = t + j < a.n ? a.slots[t + j] : -1;
        if (slot >= 0) *place(slot) = tw_from_float<T>(v[half + j] * a.v_scale);
      }
    }
  }
}

// Workgroups 0 .. n - 1: a token each. Steps of many rows: the workgroups behind them write the values, 16 tokens each
// (value_blocks a tile); else a token's workgroup writes its own. Every 16-byte piece of q, k and v is one thread's, so
// that all of a row is on its way at once.
template <typename T, int THREADS>
__global__ __launch_bounds__(THREADS) void rows_finish_kernel(RowsFinishArgs a, int value_blocks) {
  extern __shared__ __attribute__((aligned(16))) float rf_lds[];
  __shared__ float red[16];
  __shared__ __attribute__((aligned(16))) float cs[128], sn[128];                  // rot <= 256
  const int n = blockIdx.x, tid = threadIdx.x;
  if (n >= a.n) {
    rf_values<T>(a, (n - a.n) / value_blocks, (n - a.n) % value_blocks);
    return;
  }
  const float* row = a.src + (size_t)n * a.ld;
  const bool keys = a.k_col >= 0;
  const int nq = a.H * a.M * a.D, nk = keys ? a.G * a.M * a.D : 0, nv = keys && !value_blocks ? a.G * a.E : 0;
  const int pq = (nq + 3) / 4, pk = (nk + 3) / 4, pv = (nv + 3) / 4;
  float* q_s = rf_lds;
  float* k_s = q_s + 4 * pq;
  float* v_s = k_s + 4 * pk;
  const int slot = keys ? a.slots[n] : -1;
  float sq = 0.f, sk = 0.f;
  for (int i = tid; i < pq + pk + pv; i += THREADS) {
    const int in_q = i < pq, in_k = !in_q && i < pq + pk;
    const int at = 4 * (in_q ? i : in_k ? i - pq : i - pq - pk);
    const int count = in_q ? nq : in_k ? nk : nv;
    const int col = (in_q ? a.q_col : in_k ? a.k_col : a.v_col) + at;
    f32x4 v;
    if (a.vec && at + 4 <= count) {
      v = *reinterpret_cast<const f32x4*>(row + col);
#pragma unroll 8
      for (int s = 1; s < a.splits; ++s) v += *reinterpret_cast<const f32x4*>(row + s * a.split_stride + col);
      if (a.bias) v += *reinterpret_cast<const f32x4*>(a.bias + col);
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = at + j < count ? rf_column(a, row, col + j) : 0.f;
    }
    if (a.norm == 2) {
      float ss = 0.f;
#pragma unroll
      for (int j = 0; j < 4; ++j) ss = __fmaf_rn(v[j], v[j], ss);
      if (in_q) sq += ss;
      else if (in_k) sk += ss;
    }
    *reinterpret_cast<f32x4*>(rf_lds + 4 * i) = v;
  }
  for (int i = THREADS - 1 - tid; i < a.rot / 2; i += THREADS) {    // (the last threads: they have the fewest pieces)
    const float p = (float)a.positions[n], f = a.freq[i];
    const float angle = __fmul_rn(p, f);
    const float off = a.rest ? __fmaf_rn(p, a.rest[i], __fmaf_rn(p, f, -angle)) : 0.f;    // (a few hundredths at most)
    float s, c;
    sincosf(angle, &s, &c);
    const float off2 = off * off, so = off * __fmaf_rn(-off2, 1.f / 6.f, 1.f), co = -0.5f * off2;
    sn[i] = __fmaf_rn(so, c, __fmaf_rn(co, s, s));
    cs[i] = __fmaf_rn(-so, s, __fmaf_rn(co, c, c));
  }
  if (a.g_col >= 0)
    for (int i = THREADS - 1 - tid; i < a.H; i += THREADS)
      a.gate[(size_t)n * a.H + i] = 1.f / (1.f + expf(-rf_column(a, row, a.g_col + i)));
  auto scale_row = [&](float* x, int count, float f, const float* w) {
    for (int i = 4 * tid; i < count; i += 4 * THREADS) {
      f32x4 v = *reinterpret_cast<const f32x4*>(x + i) * f;
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] *= i + j < count ? w[i + j] : 0.f;
      *reinterpret_cast<f32x4*>(x + i) = v;
    }
  };
  if (a.norm == 2) {
    sq = tw_block_sum(sq, red);
    const float rq = 1.f / sqrtf(sq / (float)nq + a.eps);
    scale_row(q_s, nq, rq, a.wq);
    if (nk) {
      sk = tw_block_sum(sk, red);
      const float rk = 1.f / sqrtf(sk / (float)nk + a.eps);
      scale_row(k_s, nk, rk, a.wk);
    }
  } else if (a.norm == 1) {
    __syncthreads();
    // 16 lanes a head
    const int lane = tid & 15, heads_q = a.H * a.M, heads = heads_q + (nk ? a.G * a.M : 0);
    for (int head = tid >> 4; head < heads; head += THREADS / 16) {
      float* x = head < heads_q ? q_s + head * a.D : k_s + (head - heads_q) * a.D;
      const float* w = head < heads_q ? a.wq : a.wk;
      float ss = 0.f;
      for (int d = lane; d < a.D; d += 16) ss = __fmaf_rn(x[d], x[d], ss);
      const float f = 1.f / sqrtf(rf_row_sum(ss) / (float)a.D + a.eps);
      for (int d = lane; d < a.D; d += 16) x[d] = x[d] * f * w[d];
    }
  }
  __syncthreads();
  const int pieces = a.Dp / 4;
  const int page = slot >= 0 ? slot / a.P : 0, at = slot >= 0 ? slot % a.P : 0;
  T* q = (T*)a.q_out + (size_t)n * a.ld_q;
  const int heads_q = a.H * a.M, heads_k = slot >= 0 ? a.G : 0;
  const bool whole = a.D % 4 == 0 && a.rot % 8 == 0;                 // four elements turn alike, with four others or among themselves
  for (int i = tid; i < (heads_q + heads_k) * pieces; i += THREADS) {
    const int head = i / pieces, d0 = (i - head * pieces) * 4;
    if (head < heads_q) {
      const int from = a.M == 2 ? (head & 1) * a.D : 0;              // where the map's elements lie among the key's
      rf_store4<T>(q + (size_t)head * a.Dp + d0, rf_rotated4(q_s + head * a.D, d0 - from, a.D, a.rot, a.pairing, cs, sn, whole));
    } else {
      const int g = head - heads_q;
      f32x4 v;
      if (whole || a.M == 1) {
        const int m = a.M == 2 && d0 >= a.D ? 1 : 0;
        v = rf_rotated4(k_s + (g * a.M + m) * a.D, d0 - m * a.D, a.D, a.rot, a.pairing, cs, sn, whole);
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int d = d0 + j, m = d >= a.D ? 1 : 0;
          v[j] = d < 2 * a.D ? rf_rotated(k_s + (g * 2 + m) * a.D, d - m * a.D, a.rot, a.pairing, cs, sn) : 0.f;
        }
      }
      rf_store4<T>((T*)a.keys + (((size_t)page * a.G + g) * a.P + at) * a.Dp + d0, v);
    }
  }
  if (value_blocks || slot < 0) return;
  for (int i = tid; i < a.G * a.Dp; i += THREADS) {
    const int g = i / a.Dp, e = i - g * a.Dp;
    ((T*)a.values)[(((size_t)page * a.G + g) * a.Dp + e) * a.P + at] = tw_from_float<T>(e < a.E ? v_s[g * a.E + e] * a.v_scale : 0.f);
  }
}

template <typename T, int THREADS>
static int rows_finish_launch(const RowsFinishArgs& a, size_t lds, int value_blocks, hipStream_t stream) {
  static bool allowed = false;
  if (!allowed) {
    const hipError_t e = hipFuncSetAttribute((const void*)rows_finish_kernel<T, THREADS>, hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024);
    if (e != hipSuccess) return (int)e;
    allowed = true;
  }
  rows_finish_kernel<T, THREADS><<<a.n + value_blocks * tw_div_up(a.n, RF_TILE), THREADS, lds, stream>>>(a, value_blocks);
  return TW_LAUNCH_RESULT();
}

extern "C" int tw_rows_finish(int dtype, const float* src, long ld, int splits, long split_stride, const float* bias, int q_col,
                              int k_col, int v_col, int g_col, int norm, const float* wq, const float* wk,
                              const int* positions, const float* freq, const float* rest, int rot, int pairing, void* q_out, long ld_q, void* keys, void* values,
                              const int* slots, float* gate, int n, int H, int G, int M, int D, int E, int Dp, int page_size,
                              float eps, float v_scale, hipStream_t stream) {
  TW_REQUIRE(src && q_out && n >= 0 && H > 0 && G > 0 && (M == 1 || M == 2) && D > 0 && D <= 256 && splits >= 1);
  TW_REQUIRE(Dp % 16 == 0 && Dp >= M * D && Dp <= 256 && q_col >= 0 && ld >= q_col + (long)H * M * D && ld_q >= (long)H * M * Dp);
  TW_REQUIRE(splits == 1 || split_stride >= (long)n * ld);
  TW_REQUIRE(k_col < 0 || (keys && values && slots && page_size > 0 && E > 0 && E <= Dp && v_col >= 0 &&
                           ld >= k_col + (long)G * M * D && ld >= v_col + (long)G * E));
  TW_REQUIRE(g_col < 0 || (gate && ld >= (long)g_col + H));
  TW_REQUIRE(norm >= 0 && norm <= 2 && (norm == 0 || (wq && (wk || k_col < 0) && eps > 0.f)));
  TW_REQUIRE(rot >= 0 && rot % 2 == 0 && rot <= D && (rot == 0 || (positions && freq)) && (pairing == 0 || pairing == 1));
  TW_REQUIRE((uintptr_t)q_out % 16 == 0 && ld_q % 4 == 0 && (k_col < 0 || (uintptr_t)keys % 16 == 0));
  const int nq = H * M * D, nk = k_col < 0 ? 0 : G * M * D, nv = k_col < 0 ? 0 : G * E;
  const size_t lds = ((size_t)(nq + 3) / 4 + (size_t)(nk + 3) / 4 + (n <= RF_FEW ? (size_t)(nv + 3) / 4 : 0)) * 16;
  TW_REQUIRE(lds <= 128 * 1024);
  if (n == 0) return 0;
  const bool vec = ld % 4 == 0 && split_stride % 4 == 0 && q_col % 4 == 0 && (k_col < 0 || (k_col % 4 == 0 && v_col % 4 == 0)) &&
                   (uintptr_t)src % 16 == 0 && (!bias || (uintptr_t)bias % 16 == 0);
  const RowsFinishArgs a{src, ld, splits, (size_t)split_stride, bias, q_col, k_col, v_col, g_col, wq, wk, norm, positions, freq, rest, rot, pairing,
                         q_out, ld_q, keys, values, slots, gate, H, G, M, D, E, Dp, page_size > 0 ? page_size : 1, eps, v_scale, vec, n};
  const int value_blocks = k_col >= 0 && n > RF_FEW ? tw_div_up((long)G * Dp, 256) : 0;
  if (dtype == TW_DTYPE_BF16)
    return n <= RF_FEW ? rows_finish_launch<bf16_t, 1024>(a, lds, 0, stream) : rows_finish_launch<bf16_t, 256>(a, lds, value_blocks, stream);
  if (dtype == TW_DTYPE_F32)
    return n <= RF_FEW ? rows_finish_launch<float, 1024>(a, lds, 0, stream) : rows_finish_launch<float, 256>(a, lds, value_blocks, stream);
  return TW_ERR_BAD_ARGUMENT;
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
