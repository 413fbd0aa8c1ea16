// A feed-forward of routed experts: every token runs the `top` experts with the largest router scores.
//
//   z = W_router h (float32)      s = sigmoid(z)      chosen: the `top` largest (the lowest index wins a tie)
//   out = sum over the chosen experts e of  expert_e(s_e * h)         (the score multiplies the expert's INPUT)
//   expert(y): down( glu(gate y, up y) ), glu as TW_GLU_SWISH_LIMITED with the experts' limit
//
// A second kind of expert and of weighting (`kind` 1 of tw_moe_experts, `mode` 1 of tw_moe_route):
//   z = W_router h + b        chosen: the `top` largest      p = softmax over the chosen logits alone
//   out = sum over the chosen experts e of  p_e * expert_e(h)         (the weight multiplies the expert's OUTPUT)
//   expert(y): down( gelu(up y) ), the exact gelu y Phi(y); no gate matrix
//
// A third (`kind` 2, `mode` 2): gated experts whose weights multiply their outputs, a softmax over ALL logits, and experts
// without matrices:
//   s = softmax(W_router h) over X + identity logits    chosen: the `top` largest of s + correction
//   p = s of the chosen over their sum (+ 1e-20)        expert(y): down( silu(gate y) * up y ); the last `identity`
//   out = sum over the chosen experts e of  p_e * expert_e(h)          experts return h itself
//
// A fourth (`kind` 3, `mode` 0 with groups): plain experts whose weights are scaled scores that multiply their outputs,
//   s = sigmoid(W_router h); the experts stand in `groups` equal groups of neighbours, a group's score is the sum of its two
//   largest s, only experts of the best `keep` groups can be chosen;     p = scale * s of the chosen
//   out = sum over the chosen experts e of  p_e * expert_e(h)         expert(y): down( max(up y, 0)^2 )
//
// A step runs in six launches (four where there are few pairs: see PLAN below) whose shapes depend only on the number
// of rows: route; plan (every expert's rows are laid out one expert after the other, each expert's share padded to whole
// tiles of 16 rows; which expert a tile belongs to is a table on the device, tiles nobody uses say -1); gather (the
// scaled, rounded input rows in that order); two grouped products on the matrix unit, one workgroup a (tile, range of
// columns), whose weights are the tile's expert's; combine (each token adds its experts' rows in the order it chose
// them; a choice of an identity expert adds the input row itself). No launch waits for the
// host, so the whole runs inside a captured graph.
//
// The experts' matrices lie stacked, K padded to a multiple of 32 by zeros and rows to a multiple of 16, in the order the
// matrix unit's fragments are read: [X][rows / 16][K / (4 EPF)][piece 0..3][row 0..15][EPF] (EPF: the elements of 16
// bytes), so that a wave's load of one fragment is 1 KB of consecutive memory (eight cache lines; row-major, its 16 rows
// are 16 lines, and the loads queue for the cache's tag lookups):
//   gate, up [X][Fd][Cd], down [X][C16][Fd]   (Fd, Cd: the inner size and the width rounded up to 32, C16: the width
//   rounded up to 16). The gathered rows and the activations between the two products lie the same way.
#include "gemm_shared.h"

#define TW_MOE_MAX_EXPERTS 1024
#define TW_MOE_TILE 16
#define TW_MOE_WIDE 4                 /* tiles a workgroup takes at once in steps of many rows */
#define TW_MOE_SPLITK_TILES 64        /* up to this many tiles a step, the waves of a workgroup split K */

// ---- route ---------------------------------------------------------------------------------------------------
// Four consecutive elements of a row as floats.
__device__ __forceinline__ f32x4 moe_four(const float* p) { return *reinterpret_cast<const f32x4*>(p); }
__device__ __forceinline__ f32x4 moe_four(const bf16_t* p) {
  const bf16x4 v = *reinterpret_cast<const bf16x4*>(p);
  return f32x4{(float)v[0], (float)v[1], (float)v[2], (float)v[3]};
}

// A workgroup takes R rows: a wave forms two experts' logits for all of them at a time, four elements a lane and load,
// several loads in flight before the first is used (a logit is a chain of loads from memory, and their latency is all it
// costs: few rows get many waves each, many rows share a read of the router). Then a wave a row chooses.
template <typename T, int R, int WAVES>
__global__ __launch_bounds__(64 * WAVES) void moe_route_kernel(const T* __restrict__ h, long ld_h, const float* __restrict__ router,
                                                               const float* __restrict__ bias, int mode, int n, int C, int X,
                                                               int top, int* __restrict__ ids, float* __restrict__ weights,
                                                               int groups, int keep, float scale) {
  __shared__ float z_s[R][TW_MOE_MAX_EXPERTS];
  __shared__ float score_s[R][TW_MOE_MAX_EXPERTS];   // mode 2: the softmax over all logits (z: what decides the choice); groups: theirs
  const int row0 = blockIdx.x * R, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const T* x[R];
#pragma unroll
  for (int r = 0; r < R; ++r) x[r] = h + (size_t)min(row0 + r, n - 1) * ld_h;
  const bool vec = C % 4 == 0 && ld_h % 4 == 0 && ((uintptr_t)h % 16 == 0) && ((uintptr_t)router % 16 == 0);
  for (int e = 2 * wave; e < X; e += 2 * WAVES) {
    const float* w0 = router + (size_t)e * C;
    const float* w1 = router + (size_t)min(e + 1, X - 1) * C;
    float s0[R], s1[R];
#pragma unroll
    for (int r = 0; r < R; ++r) s0[r] = s1[r] = 0.f;
    if (vec) {
#pragma unroll 4
      for (int c = 4 * lane; c < C; c += 256) {
        const f32x4 a = *reinterpret_cast<const f32x4*>(w0 + c);
        const f32x4 b = *reinterpret_cast<const f32x4*>(w1 + c);
#pragma unroll
        for (int r = 0; r < R; ++r) {
          const f32x4 xv = moe_four(x[r] + c);
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            s0[r] = __fmaf_rn(a[j], xv[j], s0[r]);
            s1[r] = __fmaf_rn(b[j], xv[j], s1[r]);
          }
        }
      }
    } else {
      for (int c = lane; c < C; c += 64) {
#pragma unroll
        for (int r = 0; r < R; ++r) {
          const float xv = tw_to_float(x[r][c]);
          s0[r] = __fmaf_rn(w0[c], xv, s0[r]);
          s1[r] = __fmaf_rn(w1[c], xv, s1[r]);
        }
      }
    }
    const bool biased = bias && mode != 2;
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const float t0 = tw_wave_sum(s0[r]), t1 = tw_wave_sum(s1[r]);
      if (lane == 0) {
        z_s[r][e] = t0 + (biased ? bias[e] : 0.f);
        if (e + 1 < X) z_s[r][e + 1] = t1 + (biased ? bias[e + 1] : 0.f);
      }
    }
  }
  __syncthreads();
  if (wave >= R || row0 + wave >= n) return;
  const int row = row0 + wave;
  float* z = z_s[wave];
  float* score = score_s[wave];
  if (mode == 2) {
    float most = -INFINITY, sum = 0.f;
    for (int e = lane; e < X; e += 64) most = fmaxf(most, z[e]);
    most = tw_wave_max(most);
    for (int e = lane; e < X; e += 64) {
      score[e] = expf(z[e] - most);
      sum += score[e];
    }
    sum = tw_wave_sum(sum);
    for (int e = lane; e < X; e += 64) {             // (a lane reads and writes its own experts only)
      score[e] /= sum;
      z[e] = score[e] + (bias ? bias[e] : 0.f);
    }
    __builtin_amdgcn_wave_barrier();
    __threadfence_block();
  }
  if (keep < groups) {
    // the two largest logits of every group (lanes share a group where there are few), then the groups' ranks
    const int size = X / groups;
    int share = 1;
    while (2 * share * groups <= 64) share *= 2;
    for (int g0 = 0; g0 < groups; g0 += 64 / share) {
      const int grp = g0 + lane / share;
      float b1 = -INFINITY, b2 = -INFINITY;
      if (grp < groups)
        for (int e = lane % share; e < size; e += share) {
          const float v = z[grp * size + e];
          b2 = fmaxf(b2, fminf(b1, v));
          b1 = fmaxf(b1, v);
        }
      for (int o = share / 2; o > 0; o >>= 1) {
        const float o1 = __shfl_xor(b1, o, TW_WAVE), o2 = __shfl_xor(b2, o, TW_WAVE);
        b2 = fmaxf(fminf(b1, o1), fmaxf(b2, o2));
        b1 = fmaxf(b1, o1);
      }
      if (grp < groups && lane % share == 0)
        score[grp] = 1.f / (1.f + expf(-b1)) + (size > 1 ? 1.f / (1.f + expf(-b2)) : 0.f);
    }
    __builtin_amdgcn_wave_barrier();
    __threadfence_block();
    unsigned kept = 0;                               // of groups lane, lane + 64, ..
    for (int i = 0, grp = lane; grp < groups; grp += 64, ++i) {
      const float mine = score[grp];
      int rank = 0;
      for (int j = 0; j < groups; ++j) rank += score[j] > mine || (score[j] == mine && j < grp) ? 1 : 0;
      kept |= rank < keep ? 1u << i : 0u;
    }
    __builtin_amdgcn_wave_barrier();
    __threadfence_block();
    for (int i = 0, grp = lane; grp < groups; grp += 64, ++i) score[grp] = (kept >> i) & 1u ? 1.f : 0.f;
    __builtin_amdgcn_wave_barrier();
    __threadfence_block();
    for (int e = lane; e < X; e += 64)
      if (score[e / size] == 0.f) z[e] = -INFINITY;
    __builtin_amdgcn_wave_barrier();
    __threadfence_block();
  }
  for (int r = 0; r < top; ++r) {
    float best = -INFINITY;
    int at = 0x7fffffff;
    for (int e = lane; e < X; e += 64) {
      const float v = z[e];
      if (v > best || (v == best && e < at)) { best = v; at = e; }
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ov = __shfl_xor(best, o, TW_WAVE);
      const int oa = __shfl_xor(at, o, TW_WAVE);
      if (ov > best || (ov == best && oa < at)) { best = ov; at = oa; }
    }
    at = min(at, X - 1);                             // (no logit compares as the largest if all are NaN)
    if (lane == 0) {
      ids[(size_t)row * top + r] = at;
      weights[(size_t)row * top + r] = mode == 2 ? score[at] : mode == 1 ? best : scale / (1.f + expf(-best));
      z[at] = -INFINITY;
    }
    __builtin_amdgcn_wave_barrier();
    __threadfence_block();
  }
  if (mode == 1 && lane == 0) {
    // the softmax over the chosen logits alone (the first chosen is the largest), in the order they were chosen
    float* w = weights + (size_t)row * top;
    const float first = w[0];
    float sum = 0.f;
    for (int r = 0; r < top; ++r) {
      w[r] = expf(w[r] - first);
      sum += w[r];
    }
    for (int r = 0; r < top; ++r) w[r] = w[r] / sum;
  }
  if (mode == 2 && lane == 0) {
    float* w = weights + (size_t)row * top;
    float sum = 1e-20f;
    for (int r = 0; r < top; ++r) sum += w[r];
    for (int r = 0; r < top; ++r) w[r] = w[r] / sum;
  }
}

extern "C" int tw_moe_route(int dtype, const void* h, long ld_h, const float* router, const float* bias, int mode, int n, int C,
                            int X, int top, int* ids, float* weights, int groups, int keep, float scale, hipStream_t stream) {
  TW_REQUIRE(h && router && ids && weights && n >= 0 && C > 0 && ld_h >= C && mode >= 0 && mode <= 2);
  TW_REQUIRE(X > 0 && X <= TW_MOE_MAX_EXPERTS && top > 0 && top <= X);
  TW_REQUIRE(groups >= 1 && X % groups == 0 && keep >= 1 && keep <= groups && top <= keep * (X / groups));
  TW_REQUIRE(mode == 0 || (keep == groups && scale == 1.f));
  if (n == 0) return 0;
#define TW_MOE_ROUTE(T)                                                                                                 \
  do {                                                                                                                  \
    if (n <= 64) moe_route_kernel<T, 1, 16><<<n, 1024, 0, stream>>>((const T*)h, ld_h, router, bias, mode, n, C, X, top, ids, weights, groups, keep, scale); \
    else if (n <= 512) moe_route_kernel<T, 1, 4><<<n, 256, 0, stream>>>((const T*)h, ld_h, router, bias, mode, n, C, X, top, ids, weights, groups, keep, scale); \
    else moe_route_kernel<T, 4, 8><<<tw_div_up(n, 4), 512, 0, stream>>>((const T*)h, ld_h, router, bias, mode, n, C, X, top, ids, weights, groups, keep, scale); \
  } while (0)
  if (dtype == TW_DTYPE_BF16) TW_MOE_ROUTE(bf16_t);
  else if (dtype == TW_DTYPE_F32) TW_MOE_ROUTE(float);
  else return TW_ERR_BAD_ARGUMENT;
#undef TW_MOE_ROUTE
  return TW_LAUNCH_RESULT();
}

// ---- plan ----------------------------------------------------------------------------------------------------
// items = n * top pairs (token, choice). pos[item]: the pair's row in the experts' order; src_item[row]: the pair of a
// row, -1 for padding (a pair whose expert is number X or above, one without matrices, gets no row: pos -1); tile_expert[tile]: the expert of rows 16 tile .., -1 for a tile behind the last one in use.
// Which of an expert's rows a pair gets depends on the order the atomics arrive in; no result depends on it, since
// every row is computed for itself and a token adds its rows in the order of its choices.
__global__ __launch_bounds__(1024) void moe_plan_kernel(const int* __restrict__ ids, int items, int X, int* __restrict__ pos,
                                                        int* __restrict__ src_item, int* __restrict__ tile_expert,
                                                        int capacity, int tiles, int unit) {
  __shared__ int count[TW_MOE_MAX_EXPERTS];
  __shared__ int offset[TW_MOE_MAX_EXPERTS + 1];
  for (int e = threadIdx.x; e < X; e += blockDim.x) count[e] = 0;
  for (int r = threadIdx.x; r < capacity; r += blockDim.x) src_item[r] = -1;
  for (int t = threadIdx.x; t < tiles; t += blockDim.x) tile_expert[t] = -1;
  __syncthreads();
  for (int i = threadIdx.x; i < items; i += blockDim.x) pos[i] = ids[i] < X ? atomicAdd(&count[ids[i]], 1) : -1;
  __syncthreads();
  if (threadIdx.x == 0) {
    int at = 0;
    for (int e = 0; e < X; ++e) {
      offset[e] = at;
      at += (count[e] + unit - 1) / unit * unit;
    }
    offset[X] = at;
  }
  __syncthreads();
  for (int e = threadIdx.x; e < X; e += blockDim.x)
    for (int t = offset[e] / TW_MOE_TILE; t < offset[e + 1] / TW_MOE_TILE; ++t) tile_expert[t] = e;
  for (int i = threadIdx.x; i < items; i += blockDim.x) {
    if (ids[i] >= X) continue;
    const int row = offset[ids[i]] + pos[i];
    pos[i] = row;
    src_item[row] = i;
  }
}

// The rows an expert's share is padded to: one tile, or, once the experts have a tile's rows each on average, the
// TW_MOE_WIDE tiles that one workgroup of the grouped products then takes against one read of the expert's matrices.
static int moe_unit(long items, int X) { return items >= (long)TW_MOE_TILE * X ? TW_MOE_TILE * TW_MOE_WIDE : TW_MOE_TILE; }

extern "C" long tw_moe_capacity(long items, int X) {
  // rows the experts' order can take: every expert's share rounded up to whole units (never fewer for more items)
  const long unit = moe_unit(items, X);
  return (items + (long)X * (unit - 1) + unit - 1) / unit * unit;
}

extern "C" int tw_moe_plan(const int* ids, int items, int X, int* pos, int* src_item, int* tile_expert, int capacity,
                           hipStream_t stream) {
  TW_REQUIRE(ids && pos && src_item && tile_expert && items >= 0 && X > 0 && X <= TW_MOE_MAX_EXPERTS);
  TW_REQUIRE(capacity >= tw_moe_capacity(items, X) && capacity % TW_MOE_TILE == 0);
  if (items == 0) return 0;
  moe_plan_kernel<<<1, 1024, 0, stream>>>(ids, items, X, pos, src_item, tile_expert, capacity, capacity / TW_MOE_TILE,
                                          moe_unit(items, X));
  return TW_LAUNCH_RESULT();
}

// ---- gather: xs[row] = round(weight * h[token]) in the experts' order, zeros in padding rows and behind C ----------
// A workgroup takes a tile's 16 rows and every gridDim.y-th group of 16 pieces of them: a thread a (row, piece), so that what
// a wave writes is consecutive (xs lies in fragment order).
template <typename T>
__global__ __launch_bounds__(256) void moe_gather_kernel(const T* __restrict__ h, long ld_h, const float* __restrict__ weights,
                                                         const int* __restrict__ src_item, const int* __restrict__ tile_expert,
                                                         T* __restrict__ xs, int C, int Cd, int top) {
  const int tile = blockIdx.x;
  if (tile_expert[tile] < 0) return;
  constexpr int EPF = Elem<T>::kPerFrag;
  const int r = threadIdx.x % TW_MOE_TILE;
  const int item = src_item[tile * TW_MOE_TILE + r];
  const float w = weights && item >= 0 ? weights[item] : 1.f;             // (no weights: they multiply the experts' outputs instead)
  const T* src = h + (item >= 0 ? (size_t)(item / top) * ld_h : 0);
  const bool vec = ld_h % EPF == 0 && (uintptr_t)h % 16 == 0;
  T* dst = xs + (size_t)tile * Cd * TW_MOE_TILE;
#pragma unroll 4
  for (int p = threadIdx.x / TW_MOE_TILE + 16 * blockIdx.y; p < Cd / EPF; p += 16 * gridDim.y) {
    typename Elem<T>::Frag v = Elem<T>::zero();
    const int c = p * EPF;
    if (item >= 0) {
      if (vec && c + EPF <= C) {
        v = tw_load_frag(src + c);
        if (weights) {
#pragma unroll
          for (int e = 0; e < EPF; ++e) v[e] = tw_from_float<T>(w * tw_to_float(v[e]));
        }
      } else {
#pragma unroll
        for (int e = 0; e < EPF; ++e)
          if (c + e < C) v[e] = tw_from_float<T>(w * tw_to_float(src[c + e]));
      }
    }
    *reinterpret_cast<typename Elem<T>::Frag*>(dst + ((size_t)p * TW_MOE_TILE + r) * EPF) = v;
  }
}

// ---- the grouped products ---------------------------------------------------------------------------------------
// One workgroup: a tile of 16 rows against 4 waves x NT x 16 columns of its expert's matrix W[ex] ([N][K], K a multiple
// of 32). GLU: W and W2 are gate and up, the result glu(gate, up) goes out in the compute type; otherwise the float32
// product. Operands go from memory straight into fragments (lane = 16 * piece + row reads 16 bytes).
// SPLITK (steps of few rows, where the tiles in use are too few to fill the chip and every one streams its expert's whole
// matrix): the four waves share one range of NT x 16 columns and take every fourth step over K each; their sums meet in
// LDS and are added in the order of the waves.
// MT > 1 (steps of many rows, whose experts' shares are padded to MT tiles): a workgroup takes MT tiles of one expert
// against every fragment of the expert's matrices it reads.
template <int N> struct MoeCount { static constexpr int value = N; };
// ACT 0: the float32 product; 1: gate and up with the limited swish; 2: one matrix with the exact gelu; 3: gate and up with
// SiLU; 4: one matrix with the square of relu (1 to 4 write the next product's rows in the compute type).
// PLAN (the first product of steps of at most 64 (token, choice) pairs whose weights multiply outputs): there is no plan
// and no gather launch. Every wave finds the tiles itself, lane i holding pair i: a pair whose expert has 16 m pairs before
// it opens a tile, the tiles are numbered in the order of the pairs that open them, and the rows are read where they lie in
// h. The tile's first workgroup writes what the second product and the combination read: tile_expert, pos.
struct MoePairs {
  const int* ids;       // [items]
  int items, top, X;
  long ld_h;
  int* tile_expert;
  int* pos;
};
template <typename T, int ACT, int NT, bool SPLITK = false, int MT = 1, bool PLAN = false>
__global__ __launch_bounds__(256) void moe_grouped_kernel(const T* __restrict__ A, long lda, const T* __restrict__ W,
                                                          const T* __restrict__ W2, const int* __restrict__ tile_expert,
                                                          void* __restrict__ out, long ldo, int N, int K, float limit,
                                                          MoePairs pairs = {}) {
  constexpr int EPF = Elem<T>::kPerFrag;
  constexpr bool GLU = ACT == 1 || ACT == 3;
  const int tile = blockIdx.x * MT;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int r = lane & 15, g = lane >> 4;
  int ex, row_of_lane = 0;                           // PLAN: the row of h that lane's row r of the tile is
  if constexpr (PLAN) {
    const int mine = lane < pairs.items ? pairs.ids[lane] : -1;
    const bool real = mine >= 0 && mine < pairs.X;
    int before = 0;                                  // pairs of the same expert before this one
    for (int i = 0; i < pairs.items; ++i) {
      const int other = __builtin_amdgcn_readlane(mine, i);
      before += (i < lane && other == mine) ? 1 : 0;
    }
    const unsigned long long opens = __ballot(real && before % TW_MOE_TILE == 0);
    int opener = -1;                                 // the pair that opens this tile
    {
      unsigned long long left = opens;
      for (int i = 0; i < tile && left; ++i) left &= left - 1;
      if (left) opener = __ffsll((unsigned long long)left) - 1;
    }
    const bool leads = blockIdx.y == 0 && wave == 0;
    if (leads && tile == 0 && lane < pairs.items && !real) pairs.pos[lane] = -1;
    if (opener < 0) {
      if (leads && lane == 0) pairs.tile_expert[tile] = -1;
      return;
    }
    ex = __builtin_amdgcn_readlane(mine, opener);
    const int from = __builtin_amdgcn_readlane(before, opener);
    const bool here = real && mine == ex && before >= from && before < from + TW_MOE_TILE;
    unsigned long long members = __ballot(here);
    if (leads) {
      if (lane == 0) pairs.tile_expert[tile] = ex;
      if (here) pairs.pos[lane] = tile * TW_MOE_TILE + before - from;
    }
    // row j of the tile is its j-th member; rows behind the last repeat the first (nobody reads what they give)
    int pair = opener;
    for (int i = 0; i < TW_MOE_TILE && members; ++i) {
      const int m = __ffsll((unsigned long long)members) - 1;
      members &= members - 1;
      if (i == r) pair = m;
    }
    row_of_lane = pair / pairs.top;
  } else {
    ex = tile_expert[tile];
    if (ex < 0) return;
  }
  const int col0 = (SPLITK ? blockIdx.y : blockIdx.y * 4 + wave) * 16 * NT;
  if (col0 >= N) return;
  constexpr int KSTEP = 4 * EPF;
  constexpr int BLK = 64 * EPF;                      // elements of one step's fragment of a tile: lane l's at l * EPF
  constexpr int k_stride = (SPLITK ? 4 : 1) * BLK;    // (k counts the elements of a tile's fragments, step after step)
  const int k_first = SPLITK ? wave * BLK : 0;
  const size_t tile_elems = (size_t)K * TW_MOE_TILE;  // all steps of one tile of 16 rows
  const int n_blocks = (N + 15) / 16;
  const T* a_ptr = PLAN ? A + (size_t)row_of_lane * pairs.ld_h + g * EPF : A + (size_t)tile * tile_elems + lane * EPF;
  const T* w_ptr[NT];
  const T* w2_ptr[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const size_t at = ((size_t)ex * n_blocks + min(col0 / 16 + t, n_blocks - 1)) * tile_elems + lane * EPF;
    w_ptr[t] = W + at;
    w2_ptr[t] = GLU ? W2 + at : nullptr;
  }
  f32x4 acc[MT][NT], acc2[MT][NT];
#pragma unroll
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int t = 0; t < NT; ++t) acc[m][t] = acc2[m][t] = f32x4{0.f, 0.f, 0.f, 0.f};
  // U steps' operands are on their way before the first is used: what bounds this loop is the latency of memory
  auto steps = [&](int k, auto count) {
    constexpr int U = decltype(count)::value;
    typename Elem<T>::Frag a[U][MT], b[U][NT], b2[U][NT];
#pragma unroll
    for (int u = 0; u < U; ++u) {
#pragma unroll
      for (int m = 0; m < MT; ++m) a[u][m] = tw_load_frag(PLAN ? a_ptr + (k + u * k_stride) / TW_MOE_TILE
                                                                          : a_ptr + (size_t)m * tile_elems + k + u * k_stride);
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        // (few rows: an expert's matrices are read once a step)
        b[u][t] = SPLITK ? tw_load_frag_stream(w_ptr[t] + k + u * k_stride) : tw_load_frag(w_ptr[t] + k + u * k_stride);
        if (GLU) b2[u][t] = SPLITK ? tw_load_frag_stream(w2_ptr[t] + k + u * k_stride) : tw_load_frag(w2_ptr[t] + k + u * k_stride);
      }
    }
    __builtin_amdgcn_sched_barrier(0);               // (the scheduler would put each load in front of its use to save registers)
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int t = 0; t < NT; ++t)
#pragma unroll
        for (int m = 0; m < MT; ++m) {
          tw_mma16(acc[m][t], a[u][m], b[u][t]);
          if (GLU) tw_mma16(acc2[m][t], a[u][m], b2[u][t]);
        }
  };
  constexpr int U = MT > 1 ? 2 : GLU ? 4 : (NT > 2 ? 4 : 8);
  int k = k_first;
  const int k_end = (int)tile_elems;
  for (; k + (U - 1) * k_stride < k_end; k += U * k_stride) steps(k, MoeCount<U>());
  for (; k < k_end; k += k_stride) steps(k, MoeCount<1>());
  static_assert(!SPLITK || MT == 1);
  if constexpr (SPLITK) {
    __shared__ f32x4 part[GLU ? 2 : 1][3][NT][64];
    if (wave > 0) {
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        part[0][wave - 1][t][lane] = acc[0][t];
        if (GLU) part[GLU ? 1 : 0][wave - 1][t][lane] = acc2[0][t];
      }
    }
    __syncthreads();
    if (wave > 0) return;
#pragma unroll
    for (int w = 0; w < 3; ++w)
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        acc[0][t] += part[0][w][t][lane];
        if (GLU) acc2[0][t] += part[GLU ? 1 : 0][w][t][lane];
      }
  }
#pragma unroll
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const int col = col0 + t * 16 + r;
      if (col >= N) continue;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        if (ACT != 0) {
          // the activations are the next product's rows: in fragment order too (ldo: the elements of a row)
          const size_t at = (size_t)(tile + m) * ldo * TW_MOE_TILE + ((size_t)(col / EPF) * TW_MOE_TILE + 4 * g + j) * EPF + col % EPF;
          const float z = acc[m][t][j];
          ((T*)out)[at] = tw_from_float<T>(ACT == 1 ? tw_swish_limited(z, acc2[m][t][j], limit)
                                               : ACT == 3 ? tw_silu(z) * acc2[m][t][j]
                                               : ACT == 4 ? fmaxf(z, 0.f) * fmaxf(z, 0.f)
                                               : 0.5f * z * (1.f + erff(z * 0.70710678118654752f)));
        } else {
          ((float*)out)[(size_t)((tile + m) * TW_MOE_TILE + 4 * g + j) * ldo + col] = acc[m][t][j];
        }
      }
    }
}

// ---- combine: x[token] += its experts' rows, in the order of its choices ------------------------------------------
// A workgroup takes 1,024 columns of a row, four a thread where rows and addresses allow 16-byte accesses.
// weights (or null): a factor on each of the token's rows; accumulate 0: x is written, not added to. more (or null):
// float32 [splits][n][C] partial sums of something else that belongs to the same result (a shared expert's last product
// with its K ranges not yet added up): added here, in index order, before the experts' rows.
// A choice without a row (pos -1) is an expert that returns h itself.
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void moe_combine_kernel(float* __restrict__ x, long ld_x, const float* __restrict__ ys,
                                                          long ld_y, const int* __restrict__ pos, int C, int top,
                                                          const float* __restrict__ weights, int accumulate,
                                                          const float* __restrict__ more, int splits, size_t more_stride,
                                                          const T* __restrict__ h, long ld_h) {
  const int row = blockIdx.x;
  const int c = blockIdx.y * 1024 + threadIdx.x * 4;
  if (c >= C) return;
  const T* own = h + (size_t)row * ld_h + c;
  if constexpr (VEC) {
    f32x4 sum = {0.f, 0.f, 0.f, 0.f};
    if (more)
      for (int s = 0; s < splits; ++s) sum += *reinterpret_cast<const f32x4*>(more + s * more_stride + (size_t)row * C + c);
    for (int r = 0; r < top; ++r) {
      const int at = pos[(size_t)row * top + r];
      f32x4 y;
      if (at >= 0) y = *reinterpret_cast<const f32x4*>(ys + (size_t)at * ld_y + c);
      else y = f32x4{tw_to_float(own[0]), tw_to_float(own[1]), tw_to_float(own[2]), tw_to_float(own[3])};
      if (weights) sum += weights[(size_t)row * top + r] * y;
      else sum += y;
    }
    f32x4* dst = reinterpret_cast<f32x4*>(x + (size_t)row * ld_x + c);
    if (accumulate) *dst += sum;
    else *dst = sum;
  } else {
    for (int j = 0; j < 4 && c + j < C; ++j) {
      float sum = 0.f;
      if (more)
        for (int s = 0; s < splits; ++s) sum += more[s * more_stride + (size_t)row * C + c + j];
      for (int r = 0; r < top; ++r) {
        const int at = pos[(size_t)row * top + r];
        sum += (weights ? weights[(size_t)row * top + r] : 1.f) * (at >= 0 ? ys[(size_t)at * ld_y + c + j] : tw_to_float(own[j]));
      }
      if (accumulate) x[(size_t)row * ld_x + c + j] += sum;
      else x[(size_t)row * ld_x + c + j] = sum;
    }
  }
}

// The two grouped products of a step: kind 0 gated with the limited swish, 1 up alone with gelu, 2 gated with SiLU, 3 up alone
// with the square of relu.
template <typename T, int ACT>
static void moe_products(const T* xs, const T* gate, const T* up, const T* down, const int* tile_expert, T* act, float* ys, int C,
                         int Cd, int Fd, float limit, int tiles, bool wide, hipStream_t stream) {
  constexpr bool PLAIN = ACT == 2 || ACT == 4;
  const T* first = PLAIN ? up : gate;
  const T* second = PLAIN ? nullptr : up;
  if (tiles <= TW_MOE_SPLITK_TILES) {
    // few rows: most tiles hold one or two rows and each streams its expert's matrices once; the waves then split K
    moe_grouped_kernel<T, ACT, 2, true><<<dim3(tiles, tw_div_up(Fd, 16 * 2)), 256, 0, stream>>>(
        xs, Cd, first, second, tile_expert, act, Fd, Fd, Cd, limit);
    moe_grouped_kernel<T, 0, 2, true><<<dim3(tiles, tw_div_up(C, 16 * 2)), 256, 0, stream>>>(
        act, Fd, down, nullptr, tile_expert, ys, C, C, Fd, 0.f);
  } else if (wide) {
    moe_grouped_kernel<T, ACT, 2, false, TW_MOE_WIDE><<<dim3(tiles / TW_MOE_WIDE, tw_div_up(Fd, 4 * 16 * 2)), 256, 0, stream>>>(
        xs, Cd, first, second, tile_expert, act, Fd, Fd, Cd, limit);
    moe_grouped_kernel<T, 0, 2, false, TW_MOE_WIDE><<<dim3(tiles / TW_MOE_WIDE, tw_div_up(C, 4 * 16 * 2)), 256, 0, stream>>>(
        act, Fd, down, nullptr, tile_expert, ys, C, C, Fd, 0.f);
  } else {
    moe_grouped_kernel<T, ACT, 2><<<dim3(tiles, tw_div_up(Fd, 4 * 16 * 2)), 256, 0, stream>>>(
        xs, Cd, first, second, tile_expert, act, Fd, Fd, Cd, limit);
    moe_grouped_kernel<T, 0, 4><<<dim3(tiles, tw_div_up(C, 4 * 16 * 4)), 256, 0, stream>>>(
        act, Fd, down, nullptr, tile_expert, ys, C, C, Fd, 0.f);
  }
}

struct MoeStep {
  const void *h, *gate, *up, *down;
  long ld_h, ld_x;
  const float* weights;
  const int *ids, *src_item, *tile_expert, *pos;
  void *xs, *act;
  float *ys, *x;
  const float* more;
  int n, top, X, C, Cd, Fd, capacity, kind, accumulate, more_splits;
  float limit;
  bool wide, few;
};

template <typename T, int ACT>
static void moe_products_few(const MoeStep& s, hipStream_t stream) {
  constexpr bool PLAIN = ACT == 2 || ACT == 4;
  // (every tile is opened by a pair of its own, and the tiles in use never exceed what a plan could need)
  const int tiles = s.n * s.top < s.capacity / TW_MOE_TILE ? s.n * s.top : s.capacity / TW_MOE_TILE;
  const MoePairs pairs{s.ids, s.n * s.top, s.top, s.X, s.ld_h, const_cast<int*>(s.tile_expert), const_cast<int*>(s.pos)};
  moe_grouped_kernel<T, ACT, 2, true, 1, true><<<dim3(tiles, tw_div_up(s.Fd, 16 * 2)), 256, 0, stream>>>(
      (const T*)s.h, s.Cd, (const T*)(PLAIN ? s.up : s.gate), (const T*)(PLAIN ? nullptr : s.up), nullptr, s.act, s.Fd, s.Fd,
      s.Cd, s.limit, pairs);
  moe_grouped_kernel<T, 0, 2, true><<<dim3(tiles, tw_div_up(s.C, 16 * 2)), 256, 0, stream>>>(
      (const T*)s.act, s.Fd, (const T*)s.down, nullptr, s.tile_expert, s.ys, s.C, s.C, s.Fd, 0.f);
}

// Can the first product find its tiles and rows itself? (few pairs, rows of h that are whole fragments)
static bool moe_few(int dtype, const void* h, long ld_h, int n, int top, int C, int Cd, int kind) {
  const int epf = dtype == TW_DTYPE_BF16 ? 8 : 4;
  return kind != 0 && n * top <= 64 && C == Cd && C % (4 * epf) == 0 && ld_h % epf == 0 && (uintptr_t)h % 16 == 0;
}

template <typename T>
static void moe_run(const MoeStep& s, hipStream_t stream) {
  if (s.few) {
    if (s.kind == 1) moe_products_few<T, 2>(s, stream);
    else if (s.kind == 2) moe_products_few<T, 3>(s, stream);
    else moe_products_few<T, 4>(s, stream);
  } else {
    const int pieces = tw_div_up(s.Cd, 16 * Elem<T>::kPerFrag);
    moe_gather_kernel<T><<<dim3(s.capacity / TW_MOE_TILE, pieces < 4 ? pieces : 4), 256, 0, stream>>>((const T*)s.h, s.ld_h, s.kind == 0 ? s.weights : nullptr, s.src_item,
                                                         s.tile_expert, (T*)s.xs, s.C, s.Cd, s.top);
    const int tiles = s.capacity / TW_MOE_TILE;
#define TW_MOE_PRODUCTS(ACT)                                                                                            \
    moe_products<T, ACT>((const T*)s.xs, (const T*)s.gate, (const T*)s.up, (const T*)s.down, s.tile_expert, (T*)s.act,    \
                         s.ys, s.C, s.Cd, s.Fd, s.limit, tiles, s.wide, stream)
    if (s.kind == 0) TW_MOE_PRODUCTS(1);
    else if (s.kind == 1) TW_MOE_PRODUCTS(2);
    else if (s.kind == 2) TW_MOE_PRODUCTS(3);
    else TW_MOE_PRODUCTS(4);
#undef TW_MOE_PRODUCTS
  }
  if (!s.x) return;                                  // (whoever reads ys and pos adds them up)
  const dim3 grid(s.n, tw_div_up(s.C, 1024));
  const size_t more_stride = (size_t)s.n * s.C;
  const float* weights = s.kind == 0 ? nullptr : s.weights;
  if (s.C % 4 == 0 && s.ld_x % 4 == 0 && (uintptr_t)s.x % 16 == 0 && (uintptr_t)s.ys % 16 == 0 && (uintptr_t)s.more % 16 == 0)
    moe_combine_kernel<T, true><<<grid, 256, 0, stream>>>(s.x, s.ld_x, s.ys, s.C, s.pos, s.C, s.top, weights, s.accumulate, s.more,
                                                          s.more_splits, more_stride, (const T*)s.h, s.ld_h);
  else
    moe_combine_kernel<T, false><<<grid, 256, 0, stream>>>(s.x, s.ld_x, s.ys, s.C, s.pos, s.C, s.top, weights, s.accumulate, s.more,
                                                           s.more_splits, more_stride, (const T*)s.h, s.ld_h);
}

// h [n][C] (compute type) -> x [n][C] float32 += the routed experts' results. ids, weights [n * top] come from
// tw_moe_route (ids of X and above, where the weights multiply outputs: experts that return h). Scratch: pos [n * top],
// src_item [capacity], tile_expert [capacity / 16] (int32), xs [capacity][Cd], act [capacity][Fd] (compute type),
// ys [capacity][C] (float32), capacity = tw_moe_capacity(n * top, X). x null: the experts' rows stay in ys, unweighted, pair i's
// in row pos[i] (kinds whose weights multiply outputs).
extern "C" int tw_moe_experts(int dtype, const void* h, long ld_h, const int* ids, const float* weights, int n, int top, int X,
                              const void* gate, const void* up, const void* down, int C, int Cd, int Fd, float limit,
                              int* pos, int* src_item, int* tile_expert, void* xs, void* act, float* ys, int capacity,
                              float* x, long ld_x, int kind, int accumulate, const float* more, int more_splits,
                              hipStream_t stream) {
  TW_REQUIRE(h && ids && weights && up && down && pos && src_item && tile_expert && xs && act && ys && (x || (kind != 0 && !more)));
  TW_REQUIRE(((kind == 0 || kind == 2) && gate) || kind == 1 || kind == 3);
  TW_REQUIRE(more == nullptr || more_splits > 0);
  if (kind == 1 || kind == 3) gate = up;            // (never read: the alignment test below wants a pointer)
  TW_REQUIRE(n >= 0 && top > 0 && C > 0 && Cd >= C && Cd % 32 == 0 && Fd > 0 && Fd % 32 == 0 && ld_h >= C && (!x || ld_x >= C));
  TW_REQUIRE((uintptr_t)xs % 16 == 0 && (uintptr_t)act % 16 == 0 && (uintptr_t)gate % 16 == 0 && (uintptr_t)up % 16 == 0 &&
             (uintptr_t)down % 16 == 0);
  TW_REQUIRE(dtype == TW_DTYPE_BF16 || dtype == TW_DTYPE_F32);
  if (n == 0) return 0;
  const bool few = moe_few(dtype, h, ld_h, n, top, C, Cd, kind);
  if (!few) {
    const int code = tw_moe_plan(ids, n * top, X, pos, src_item, tile_expert, capacity, stream);
    if (code) return code;
  }
  const bool wide = moe_unit((long)n * top, X) == TW_MOE_TILE * TW_MOE_WIDE;
  TW_REQUIRE(!wide || capacity % (TW_MOE_TILE * TW_MOE_WIDE) == 0);
  const MoeStep s{h, gate, up, down, ld_h, ld_x, weights, ids, src_item, tile_expert, pos, xs, act, ys, x, more,
                  n, top, X, C, Cd, Fd, capacity, kind, accumulate, more_splits, limit, wide, few};
  if (dtype == TW_DTYPE_BF16) moe_run<bf16_t>(s, stream);
  else moe_run<float>(s, stream);
  return TW_LAUNCH_RESULT();
}
