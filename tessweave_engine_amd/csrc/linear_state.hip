// Linear recurrences with a matrix state per head that decays from token to token:
//
//   S_t = d_t S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t         (S: [D][E] per head and request, float32)
//
// in two forms, chosen by what the decay depends on (`act`: q, k and v pass SiLU when they are read):
//   head     d_t is one number: delta = softplus(raw + dt_bias_h), d_t = exp(-exp(A_log_h) delta), k_t = delta * b_t and
//            o_t += skip_h v_t: the state-space recurrence of Mamba-2 (Dao and Gu, "Transformers are SSMs"). `share` heads
//            in a row read the same q and b (the recurrence's C and B).
//            Or d_t is a constant of the head (`decay`), k_t as it comes: lightning attention (Qin et al., "Lightning
//            Attention-2: A Free Lunch for Handling Unlimited Sequence Lengths in Large Language Models").
//   channel  d_t is a diagonal matrix over the key elements, given by its logarithms (float32 rows): gated linear
//            attention (Yang et al., "Gated Linear Attention Transformers with Hardware-Efficient Training").
//
// q, k and v are columns of float32 rows; decays, states and all products are float32. State layout: [H][Ep][Dp] (a
// value column's keys are contiguous; Dp, Ep: D and E rounded up to 16, the tails are zeros).
//
// ls_walk: sequences of a few tokens, token by token: the step is bound by reading and writing S once.
// ls_chunk: longer portions, 16 tokens at once on the matrix unit. With L_i the running sum of the logarithms of d inside
// the chunk (a vector over the key elements in the channel form):
//   o_i = (exp(L_i) q_i) . S0 + sum_{j <= i} (exp(L_i - L_j) q_i . k_j) v_j
//   S   = exp(L_last) S0 + sum_j (exp(L_last - L_j) k_j) v_j^T
// In the channel form the exponentials between tokens are factors of q and k: both are taken against the chunk's middle
// (q exp(L_i - L_mid), k exp(L_mid - L_j), S0 exp(L_mid)), so that an exponent spans half a chunk. A chunk in which some
// half decays by more than e^-60 forms its pairs one by one instead (every exponent at most 0).
//
// Portions with few (head, column) workgroups are cut into segments: a first launch leaves the state each segment alone
// would build from zero, a scan turns those into the states the segments start from (and writes the request's new
// state), and the main launch walks all segments at once.
#include "tw_common.h"

#define LS_L 16
#define LS_RANGE (-60.f)
enum { LS_HEAD, LS_CHANNEL, LS_FIXED };     // what a kernel's decay is: a step's number a head, a number a key element, a head's constant

struct LsArgs {
  const float* src; long ld;            // q of head h at q_col + h / share * D, k at k_col + h / share * D, v at v_col + h * E
  int q_col, k_col, v_col, share;
  const float* logs; long ld_logs;      // channel: logarithm of head h's decay at h * D, or (logs null, walked steps only)
  const float* low; long ld_low; int rank;          // what tw_decay_logs forms it from: rows [n][rank],
  const float* up; const float* up_bias; float tau; // up [rank][H D], its bias
  const float* raw; long ld_raw;        // head: the step size before its bias at raw_col + h
  int raw_col;
  const float* dt_bias; const float* A_log; const float* skip;   // [H]
  float* state;
  const int* q_start; const int* state_slots;
  int seq0;
  float* out; long ld_out;              // [rows][H E]
  int H, D, E, Dp, Ep;
  float q_scale;
  const float* decay;                   // head: [H] constants in (0, 1] (then raw, dt_bias, A_log are not read), or null
  bool act;                             // q, k and v pass SiLU
  bool vec;                             // q and k of every head and row are whole 16-byte pieces
};

struct LsSegments {
  float* states;       // [sequence - seq0][H][segments][Ep][Dp]
  float* logs;         // [sequence - seq0][H][segments][2][Dp]: the logarithm of a segment's whole decay, in two parts
  int len, count;      // tokens a segment (a multiple of LS_L), the most segments of a sequence
};

__device__ __forceinline__ float ls_softplus(float x) { return x > 20.f ? x : log1pf(expf(x)); }
__device__ __forceinline__ float ls_log_decay(float x, float tau) {        // log sigmoid(x) / tau
  return (x >= 0.f ? -log1pf(expf(-x)) : x - log1pf(expf(x))) / tau;
}

template <int CTRL>
__device__ __forceinline__ float ls_turned(float v) {
  return __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), CTRL, 0xf, 0xf, true));
}
template <int N>
__device__ __forceinline__ float ls_below(float v) {          // the value N lanes below in the row of 16, 0 where there is none
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x110 + N, 0xf, 0xf, false));
}
// sum over LPC neighbouring lanes (4, 16, 32 or 64); every lane gets it
template <int LPC>
__device__ __forceinline__ float ls_sum(float v) {
  if constexpr (LPC == 4) {
    v += ls_turned<0xB1>(v);          // inside a quad: lanes 1 0 3 2, then 2 3 0 1
    v += ls_turned<0x4E>(v);
  } else {
    v += ls_turned<0x128>(v);         // the row rotated by 8 lanes, then by 4, 2, 1
    v += ls_turned<0x124>(v);
    v += ls_turned<0x122>(v);
    v += ls_turned<0x121>(v);
    if constexpr (LPC >= 32) {
      auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
      v = __uint_as_float(a[0]) + __uint_as_float(a[1]);
    }
    if constexpr (LPC == 64) {
      auto b = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
      v = __uint_as_float(b[0]) + __uint_as_float(b[1]);
    }
  }
  return v;
}

__device__ __forceinline__ float ls_silu(float z) { return z / (1.f + expf(-z)); }

__device__ __forceinline__ void ls_lds_barrier() {            // (loads from memory stay on their way across it)
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
}

// elements d0 .. d0 + 3 of a vector of D, zeros behind its end. vec: D is a multiple of 4 and the address of 16 bytes.
__device__ __forceinline__ f32x4 ls_four(const float* p, int d0, int D, bool vec) {
  f32x4 v = {0.f, 0.f, 0.f, 0.f};
  if (vec) {
    if (d0 < D) v = *reinterpret_cast<const f32x4*>(p + d0);
  } else {
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (d0 + j < D) v[j] = p[d0 + j];
  }
  return v;
}

// ---- token by token -------------------------------------------------------------------------------------------------
// grid (column blocks, H, n_seqs). LPC lanes hold a value column, four key elements each; a thread holds its elements of
// CPT columns. Decays given by their low-rank product: the workgroup's threads share out (key element, part of the rank).
template <int LPC, int CPT, int FORM>
__global__ __launch_bounds__(256) void ls_walk_kernel(LsArgs a) {
  constexpr bool CHANNEL = FORM == LS_CHANNEL, fixed = FORM == LS_FIXED;
  constexpr int CW = 256 / LPC;                               // columns a pass
  const int seq = a.seq0 + blockIdx.z, head = blockIdx.y;
  const int r0 = a.q_start[seq], r1 = a.q_start[seq + 1];
  if (r1 <= r0) return;
  const int d0 = 4 * (threadIdx.x % LPC);
  const int e0 = blockIdx.x * CW * CPT + threadIdx.x / LPC;
  const bool held = d0 < a.Dp;
  float* S_mem = a.state + ((size_t)a.state_slots[seq] * a.H + head) * (size_t)a.Ep * a.Dp;
  f32x4 S[CPT];
#pragma unroll
  for (int c = 0; c < CPT; ++c) {
    const int e = e0 + c * CW;
    S[c] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (held && e < a.Ep) S[c] = __builtin_nontemporal_load(reinterpret_cast<const f32x4*>(S_mem + (size_t)e * a.Dp + d0));
  }
  const int group = head / a.share;
  float rate = 0.f, bias = 0.f, skip = 0.f;                  // (a constant decay: its value, or its logarithm, in `rate`)
  if constexpr (fixed) {
    rate = a.decay[head];
  } else if (!CHANNEL) {
    rate = -expf(a.A_log[head]);
    bias = a.dt_bias[head];
    skip = a.skip ? a.skip[head] : 0.f;
  }
  constexpr int KM = 4 * LPC, PARTS = 256 / KM;               // key elements, threads that share one's product
  __shared__ float part_s[CHANNEL ? PARTS : 1][KM];
  __shared__ __attribute__((aligned(16))) float decay_s[KM];
  for (int t = r0; t < r1; ++t) {
    const float* row = a.src + (size_t)t * a.ld;
    const float* q = row + a.q_col + (size_t)group * a.D;
    const float* k = row + a.k_col + (size_t)group * a.D;
    f32x4 qv = ls_four(q, d0, a.D, a.vec), kv = ls_four(k, d0, a.D, a.vec), dv;
    if (fixed && a.act) {
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        qv[j] = ls_silu(qv[j]);
        kv[j] = ls_silu(kv[j]);
      }
    }
    if constexpr (CHANNEL) {
      if (a.logs) {
        dv = ls_four(a.logs + (size_t)t * a.ld_logs + (size_t)head * a.D, d0, a.D, false);
#pragma unroll
        for (int j = 0; j < 4; ++j) dv[j] = expf(dv[j]);      // (behind the last element: 1)
      } else {
        const float* low = a.low + (size_t)t * a.ld_low;
        const int d = threadIdx.x % KM, part = threadIdx.x / KM;
        const size_t stride = (size_t)a.H * a.D;
        const float* up = a.up + (size_t)head * a.D + min(d, a.D - 1);
        float z = 0.f;
#pragma unroll 8
        for (int r = part; r < a.rank; r += PARTS) z = __fmaf_rn(up[r * stride], low[r], z);
        part_s[part][d] = z;
        ls_lds_barrier();
        if (threadIdx.x < KM) {
          float sum = part_s[0][d];
#pragma unroll
          for (int i = 1; i < PARTS; ++i) sum += part_s[i][d];
          decay_s[d] = d < a.D ? expf(ls_log_decay(sum + a.up_bias[(size_t)head * a.D + d], a.tau)) : 1.f;
        }
        ls_lds_barrier();
        dv = *reinterpret_cast<const f32x4*>(&decay_s[d0]);
      }
    } else if (fixed) {
      dv = f32x4{rate, rate, rate, rate};
    } else {
      const float step = ls_softplus(a.raw[(size_t)t * a.ld_raw + a.raw_col + head] + bias);
      const float decay = expf(rate * step);
      kv *= step;
      dv = f32x4{decay, decay, decay, decay};
    }
    qv *= a.q_scale;
    const float* v = row + a.v_col + (size_t)head * a.E;
#pragma unroll
    for (int c = 0; c < CPT; ++c) {
      const int e = e0 + c * CW;
      float x = e < a.E ? v[e] : 0.f;
      if (fixed && a.act) x = ls_silu(x);
      float o = 0.f;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        S[c][j] = __fmaf_rn(dv[j], S[c][j], kv[j] * x);
        o = __fmaf_rn(S[c][j], qv[j], o);
      }
      o = ls_sum<LPC>(o);
      if (d0 == 0 && e < a.E) a.out[(size_t)t * a.ld_out + (size_t)head * a.E + e] = CHANNEL ? o : __fmaf_rn(skip, x, o);
    }
  }
#pragma unroll
  for (int c = 0; c < CPT; ++c) {
    const int e = e0 + c * CW;
    if (held && e < a.Ep) __builtin_nontemporal_store(S[c], reinterpret_cast<f32x4*>(S_mem + (size_t)e * a.Dp + d0));
  }
}

// ---- 16 tokens at once ----------------------------------------------------------------------------------------------
// grid (slices of 64 value columns * H, segments, n_seqs). A wave owns 16 value columns; lane (r, g) = (lane % 16,
// lane / 16) holds S[16 dt + 4 g + 0..3][its column r] for every tile dt of the key elements: the layout that is both the
// B operand of Q S and the accumulator of K^T V. BUILD: only the segment's own state, from zero.
template <int DT, int FORM, bool BUILD>
__global__ __launch_bounds__(256) void ls_chunk_kernel(LsArgs a, LsSegments sg) {
  constexpr bool CHANNEL = FORM == LS_CHANNEL, fixed = FORM == LS_FIXED;
  constexpr int DM = 16 * DT, QS = DM + 4;
  constexpr int NU = (2 * DM + 255) / 256;                    // (key element, half of the chunk) pairs a thread stages
  __shared__ __attribute__((aligned(16))) float q_s[BUILD ? 1 : LS_L][QS];
  __shared__ __attribute__((aligned(16))) float k_s[LS_L][QS];
  __shared__ __attribute__((aligned(16))) float l_s[CHANNEL && !BUILD ? LS_L : 1][QS];   // running sums, for chunks of pairs one by one
  __shared__ __attribute__((aligned(16))) float f_s[CHANNEL ? 3 : 1][DM];    // factors of S: before the read-out, behind it, behind the sum
  __shared__ float v_s[LS_L][68];
  __shared__ f32x4 part_s[BUILD ? 1 : 256];
  __shared__ float cum_s[LS_L], step_s[LS_L], tail_s[LS_L];   // head form: L_i, delta_i, delta_i exp(L_last - L_i)
  __shared__ int wide_s[4];
  const int slices = (a.Ep + 63) / 64;
  const int slice = blockIdx.x % slices, head = blockIdx.x / slices;
  const int seq = a.seq0 + blockIdx.z;
  const int q_first = a.q_start[seq], q_last = a.q_start[seq + 1];
  const int first = q_first + blockIdx.y * sg.len;
  if (first >= q_last) return;
  const int last = min(first + sg.len, q_last);
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int r = lane & 15, g = lane >> 4;
  const int tiles = a.Dp / 16, group = head / a.share;
  const int e_col = slice * 64 + wave * 16 + r;
  const bool on = slice * 64 + wave * 16 < a.Ep;
  const size_t one = (size_t)a.Ep * a.Dp;
  float* seg_state = sg.states + (((size_t)blockIdx.z * a.H + head) * sg.count + blockIdx.y) * one;
  float* own_state = a.state + ((size_t)a.state_slots[seq] * a.H + head) * one;
  f32x4 S[DT];
#pragma unroll
  for (int t = 0; t < DT; ++t) {
    S[t] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (!BUILD && on && t < tiles)
      S[t] = *reinterpret_cast<const f32x4*>((sg.count > 1 ? seg_state : own_state) + (size_t)e_col * a.Dp + 16 * t + 4 * g);
  }
  float rate = 0.f, bias = 0.f, skip = 0.f;                  // (a constant decay: its value, or its logarithm, in `rate`)
  if constexpr (fixed) {
    rate = logf(a.decay[head]);
  } else if (!CHANNEL) {
    rate = -expf(a.A_log[head]);
    bias = a.dt_bias[head];
    skip = a.skip ? a.skip[head] : 0.f;
  }

  // a chunk's rows on their way: a thread takes a key element of eight tokens (its half of the chunk) and four values
  float rq[NU][8], rk[NU][8], rl[NU][8], rv[4], rraw = 0.f;
  float whole[NU];                                            // channel form: logarithm of the segment's decay so far
  float whole_head = 0.f;
#pragma unroll
  for (int u = 0; u < NU; ++u) whole[u] = 0.f;
  auto request = [&](int c0) __attribute__((always_inline)) {
#pragma unroll
    for (int u = 0; u < NU; ++u) {
      const int item = threadIdx.x + 256 * u;
      const int half = item / DM, d = item - half * DM;
      const bool in_d = half < 2 && d < a.D;
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const int t = c0 + 8 * half + i;
        const bool ok = in_d && t < last;
        const float* row = a.src + (size_t)(ok ? t : first) * a.ld;
        if (!BUILD) rq[u][i] = ok ? row[a.q_col + group * a.D + d] : 0.f;
        rk[u][i] = ok ? row[a.k_col + group * a.D + d] : 0.f;
        if (CHANNEL) rl[u][i] = ok ? a.logs[(size_t)t * a.ld_logs + (size_t)head * a.D + d] : 0.f;
      }
    }
    const int t = c0 + (threadIdx.x >> 4);
    const bool ok = t < last;
    const float* row = a.src + (size_t)(ok ? t : first) * a.ld + a.v_col + (size_t)head * a.E;
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const int e = slice * 64 + (threadIdx.x & 15) + 16 * x;
      rv[x] = ok && e < a.E ? row[e] : 0.f;
    }
    if (!CHANNEL && !fixed && threadIdx.x < LS_L) {
      const int tt = c0 + threadIdx.x;
      rraw = tt < last ? a.raw[(size_t)tt * a.ld_raw + a.raw_col + head] : 0.f;
    }
  };
  request(first);
  for (int c0 = first; c0 < last; c0 += LS_L) {
    float total[NU];                                          // this thread's half, for its key element
    if (CHANNEL) {
      bool wide = false;
#pragma unroll
      for (int u = 0; u < NU; ++u) {
        total[u] = 0.f;
#pragma unroll
        for (int i = 0; i < 8; ++i) total[u] += rl[u][i];
        wide |= total[u] < LS_RANGE;
        whole[u] += total[u];
      }
      const bool any = __any(wide);
      if (lane == 0) wide_s[wave] = any ? 1 : 0;
    }
    ls_lds_barrier();                                         // the chunk before has been worked on by every wave
    const bool pairs = CHANNEL && (wide_s[0] | wide_s[1] | wide_s[2] | wide_s[3]) != 0;

    // ---- the chunk's rows into LDS --------------------------------------------------------------------------------
    if (fixed && a.act) {
#pragma unroll
      for (int u = 0; u < NU; ++u)
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          if (!BUILD) rq[u][i] = ls_silu(rq[u][i]);
          rk[u][i] = ls_silu(rk[u][i]);
        }
#pragma unroll
      for (int x = 0; x < 4; ++x) rv[x] = ls_silu(rv[x]);
    }
    if (CHANNEL) {
#pragma unroll
      for (int u = 0; u < NU; ++u) {
        const int item = threadIdx.x + 256 * u;
        const int half = item / DM, d = item - half * DM;
        if (half >= 2 || d >= a.Dp) continue;
        // `mid` taken as the end of the first half: sums of logarithms from there (half 1) or up to there (half 0)
        float upto = 0.f;                                     // L_i - L_(start of this half)
        float other = 0.f;
        if (pairs && d < a.D) {                               // the other half's whole sum
#pragma unroll
          for (int i = 0; i < 8; ++i) {
            const int t = c0 + 8 * (1 - half) + i;
            if (t < last) other += a.logs[(size_t)t * a.ld_logs + (size_t)head * a.D + d];
          }
        }
        if (!pairs) {
          if (half == 0) {
            f_s[0][d] = expf(total[u]);                       // exp(L_mid)
            f_s[1][d] = 1.f;
          } else {
            f_s[2][d] = expf(total[u]);                       // exp(L_last - L_mid)
          }
        } else if (half == 0) {
          f_s[0][d] = 1.f;
          f_s[1][d] = expf(total[u] + other);
          f_s[2][d] = 1.f;
        }
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          upto += rl[u][i];
          const int row = 8 * half + i;
          if (!pairs) {
            const float from_mid = half == 0 ? upto - total[u] : upto;       // L_i - L_mid
            if (!BUILD) q_s[row][d] = rq[u][i] * a.q_scale * expf(from_mid);
            k_s[row][d] = rk[u][i] * expf(-from_mid);
          } else {
            const float L = half == 0 ? upto : upto + other;
            if (!BUILD) {
              q_s[row][d] = rq[u][i] * a.q_scale * expf(L);
              l_s[row][d] = L;
            }
            k_s[row][d] = rk[u][i] * expf(half == 0 ? (total[u] - upto) + other : total[u] - upto);   // exp(L_last - L_j)
          }
        }
      }
    } else {
#pragma unroll
      for (int u = 0; u < NU; ++u) {
        const int item = threadIdx.x + 256 * u;
        const int half = item / DM, d = item - half * DM;
        if (half >= 2 || d >= a.Dp) continue;
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          if (!BUILD) q_s[8 * half + i][d] = rq[u][i] * a.q_scale;
          k_s[8 * half + i][d] = rk[u][i];
        }
      }
      if (threadIdx.x < LS_L) {                               // (one row of 16 lanes)
        const bool in = c0 + (int)threadIdx.x < last;
        const float step = !in ? 0.f : fixed ? 1.f : ls_softplus(rraw + bias);
        const float lg = rate * step;
        float L = lg;
        L += ls_below<1>(L);
        L += ls_below<2>(L);
        L += ls_below<4>(L);
        L += ls_below<8>(L);
        const float L_last = __shfl(L, LS_L - 1, TW_WAVE);
        cum_s[threadIdx.x] = L;
        step_s[threadIdx.x] = step;
        tail_s[threadIdx.x] = step * expf(L_last - L);
      }
    }
#pragma unroll
    for (int x = 0; x < 4; ++x) v_s[threadIdx.x >> 4][(threadIdx.x & 15) + 16 * x] = rv[x];
    ls_lds_barrier();
    if (c0 + LS_L < last) request(c0 + LS_L);

    f32x4 w = {0.f, 0.f, 0.f, 0.f};                           // W[token r][token 4 g + e]
    if (!BUILD) {
      if (!pairs) {
        f32x4 p = {0.f, 0.f, 0.f, 0.f};                       // over this wave's share of the key elements
        for (int t = wave; t < tiles; t += 4) {
          const f32x4 kf = *reinterpret_cast<const f32x4*>(&k_s[r][16 * t + 4 * g]);
          const f32x4 qf = *reinterpret_cast<const f32x4*>(&q_s[r][16 * t + 4 * g]);
          tw_mma16(p, kf, qf);                                // p[e]: k_(4 g + e) . q_r
        }
        part_s[wave * 64 + lane] = p;
      } else {
        const int i = threadIdx.x >> 4, j = threadIdx.x & 15;
        float sum = 0.f;
        if (j <= i && c0 + i < last) {
          const float* q = a.src + (size_t)(c0 + i) * a.ld + a.q_col + group * a.D;
          const float* k = a.src + (size_t)(c0 + j) * a.ld + a.k_col + group * a.D;
          for (int d = 0; d < a.D; ++d) sum = __fmaf_rn(q[d] * a.q_scale * k[d], expf(l_s[i][d] - l_s[j][d]), sum);
        }
        reinterpret_cast<float*>(part_s)[i * LS_L + j] = sum;
      }
      ls_lds_barrier();
      if (pairs) {
        w = *reinterpret_cast<const f32x4*>(reinterpret_cast<const float*>(part_s) + r * LS_L + 4 * g);
      } else {
        w = (part_s[lane] + part_s[64 + lane]) + (part_s[128 + lane] + part_s[192 + lane]);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int j = 4 * g + e;
          if (CHANNEL) w[e] = j <= r ? w[e] : 0.f;
          else w[e] = j <= r ? w[e] * step_s[j] * expf(cum_s[r] - cum_s[j]) : 0.f;
        }
      }
    }
    if (on) {
      f32x4 vf;                                               // values of tokens 4 g .. 4 g + 3, column r of the wave's
#pragma unroll
      for (int e = 0; e < 4; ++e) vf[e] = v_s[4 * g + e][wave * 16 + r];
      if (CHANNEL) {
#pragma unroll
        for (int t = 0; t < DT; ++t)
          if (t < tiles) S[t] *= *reinterpret_cast<const f32x4*>(&f_s[0][16 * t + 4 * g]);
      }
      if (!BUILD) {
        f32x4 o = {0.f, 0.f, 0.f, 0.f}, o2 = {0.f, 0.f, 0.f, 0.f};        // (two chains of products instead of one)
#pragma unroll
        for (int t = 0; t < DT; t += 2) {
          if (t < tiles) tw_mma16_k4(o, *reinterpret_cast<const f32x4*>(&q_s[r][16 * t + 4 * g]), S[t]);
          if (t + 1 < tiles) tw_mma16_k4(o2, *reinterpret_cast<const f32x4*>(&q_s[r][16 * (t + 1) + 4 * g]), S[t + 1]);
        }
        o += o2;
        if (!CHANNEL) {
#pragma unroll
          for (int e = 0; e < 4; ++e) o[e] = __fmaf_rn(skip, vf[e], o[e] * expf(cum_s[4 * g + e]));
        }
        tw_mma16_k4(o, w, vf);                                // o[e]: token 4 g + e
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int t = c0 + 4 * g + e;
          if (t < last && e_col < a.E) a.out[(size_t)t * a.ld_out + (size_t)head * a.E + e_col] = o[e];
        }
      }
      // the state behind the chunk
      float all = 1.f;
      if (!CHANNEL) {
        all = expf(cum_s[LS_L - 1]);
#pragma unroll
        for (int e = 0; e < 4; ++e) vf[e] *= tail_s[4 * g + e];
      }
#pragma unroll
      for (int t = 0; t < DT; ++t) {
        if (t < tiles) {
          f32x4 kf;
#pragma unroll
          for (int e = 0; e < 4; ++e) kf[e] = k_s[4 * g + e][16 * t + r];
          if (CHANNEL) S[t] *= *reinterpret_cast<const f32x4*>(&f_s[1][16 * t + 4 * g]);
          else S[t] *= all;
          tw_mma16_k4(S[t], kf, vf);
          if (CHANNEL) S[t] *= *reinterpret_cast<const f32x4*>(&f_s[2][16 * t + 4 * g]);
        }
      }
    }
    if (!CHANNEL && BUILD) whole_head += cum_s[LS_L - 1];
  }
  if (on && (BUILD || sg.count == 1)) {
    float* dst = BUILD ? seg_state : own_state;
#pragma unroll
    for (int t = 0; t < DT; ++t)
      if (t < tiles) *reinterpret_cast<f32x4*>(dst + (size_t)e_col * a.Dp + 16 * t + 4 * g) = S[t];
  }
  if (BUILD && slice == 0) {
    float* logs = sg.logs + (((size_t)blockIdx.z * a.H + head) * sg.count + blockIdx.y) * 2 * a.Dp;
    if (CHANNEL) {
#pragma unroll
      for (int u = 0; u < NU; ++u) {
        const int item = threadIdx.x + 256 * u;
        const int half = item / DM, d = item - half * DM;
        if (half < 2 && d < a.Dp) logs[half * a.Dp + d] = whole[u];
      }
    } else if (threadIdx.x == 0) {
      logs[0] = whole_head;
    }
  }
}

// Segments' own states -> the states they start from, in place; the request's state goes from old to new.
// grid (groups of four state elements / 256, H, n_seqs)
template <int FORM>
__global__ __launch_bounds__(256) void ls_scan_kernel(LsArgs a, LsSegments sg) {
  constexpr bool CHANNEL = FORM == LS_CHANNEL;
  const int head = blockIdx.y, seq = a.seq0 + blockIdx.z;
  const int rows = a.q_start[seq + 1] - a.q_start[seq];
  const size_t one = (size_t)a.Ep * a.Dp;
  const size_t at = ((size_t)blockIdx.x * 256 + threadIdx.x) * 4;
  if (rows <= 0 || at >= one) return;
  const int d = (int)(at % a.Dp);
  const int segments = (rows + sg.len - 1) / sg.len;
  const size_t base = ((size_t)blockIdx.z * a.H + head) * sg.count;
  f32x4* own = reinterpret_cast<f32x4*>(a.state + ((size_t)a.state_slots[seq] * a.H + head) * one + at);
  f32x4 S = *own;
#pragma unroll 4
  for (int p = 0; p < segments; ++p) {
    f32x4* mem = reinterpret_cast<f32x4*>(sg.states + (base + p) * one + at);
    const float* logs = sg.logs + (base + p) * 2 * a.Dp;
    const f32x4 built = *mem;
    f32x4 decay;
    if (CHANNEL) {
#pragma unroll
      for (int j = 0; j < 4; ++j) decay[j] = expf(logs[d + j] + logs[a.Dp + d + j]);
    } else {
      const float f = expf(logs[0]);
      decay = f32x4{f, f, f, f};
    }
    *mem = S;
#pragma unroll
    for (int j = 0; j < 4; ++j) S[j] = __fmaf_rn(decay[j], S[j], built[j]);
  }
  *own = S;
}

// Segments of a launch whose longest portion has max_q_len tokens: enough that the chip's CUs all have a few workgroups,
// each at least four chunks long.
static void ls_segments(int n_seqs, int max_q_len, int H, int Ep, int* len, int* count) {
  const int chunks = tw_div_up(max_q_len, LS_L);
  const long groups = (long)n_seqs * H * ((Ep + 63) / 64);
  long want = tw_div_up(1024, groups);
  if (want > chunks / 4) want = chunks / 4;
  if (want < 1) want = 1;
  const int per = tw_div_up(chunks, want);
  *len = per * LS_L;
  *count = tw_div_up(chunks, per);
}

extern "C" long tw_linear_state_workspace_floats(int n_seqs, int max_q_len, int H, int Dp, int Ep) {
  if (n_seqs <= 0 || max_q_len <= 0) return 0;
  int len, count;
  ls_segments(n_seqs, max_q_len, H, Ep, &len, &count);
  return count > 1 ? (long)n_seqs * H * count * ((long)Ep * Dp + 2L * Dp) : 0;
}

template <int FORM>
static int ls_walk_launch(const LsArgs& a, int n_seqs, hipStream_t stream) {
  // few (sequence, head) pairs: two columns a thread spread a head over more workgroups; else eight
#define LS_WALK(LPC)                                                                                                   \
  do {                                                                                                                 \
    constexpr int CW = 256 / LPC;                                                                                      \
    if ((long)n_seqs * a.H >= 512 && a.Ep >= 8 * CW)                                                                   \
      ls_walk_kernel<LPC, 8, FORM><<<dim3(tw_div_up(a.Ep, 8 * CW), a.H, n_seqs), 256, 0, stream>>>(a);              \
    else if (a.Ep >= 2 * CW)                                                                                           \
      ls_walk_kernel<LPC, 2, FORM><<<dim3(tw_div_up(a.Ep, 2 * CW), a.H, n_seqs), 256, 0, stream>>>(a);              \
    else                                                                                                               \
      ls_walk_kernel<LPC, 1, FORM><<<dim3(tw_div_up(a.Ep, CW), a.H, n_seqs), 256, 0, stream>>>(a);                  \
  } while (0)
  if (a.Dp <= 16) LS_WALK(4);
  else if (a.Dp <= 64) LS_WALK(16);
  else if (a.Dp <= 128) LS_WALK(32);
  else LS_WALK(64);
#undef LS_WALK
  return TW_LAUNCH_RESULT();
}

template <int DT, int FORM>
static int ls_chunk_launch(const LsArgs& a, const LsSegments& sg, int n_seqs, hipStream_t stream) {
  const dim3 grid((unsigned)((a.Ep + 63) / 64 * a.H), (unsigned)sg.count, (unsigned)n_seqs);
  if (sg.count > 1) {
    ls_chunk_kernel<DT, FORM, true><<<grid, 256, 0, stream>>>(a, sg);
    ls_scan_kernel<FORM><<<dim3(tw_div_up((long)a.Ep * a.Dp, 1024), a.H, n_seqs), 256, 0, stream>>>(a, sg);
  }
  ls_chunk_kernel<DT, FORM, false><<<grid, 256, 0, stream>>>(a, sg);
  return TW_LAUNCH_RESULT();
}

template <int FORM>
static int ls_launch(const LsArgs& a, const LsSegments& sg, int n_seqs, int walk, hipStream_t stream) {
  if (walk) return ls_walk_launch<FORM>(a, n_seqs, stream);
  if (a.Dp <= 64) return ls_chunk_launch<4, FORM>(a, sg, n_seqs, stream);
  if (a.Dp <= 128) return ls_chunk_launch<8, FORM>(a, sg, n_seqs, stream);
  return ls_chunk_launch<16, FORM>(a, sg, n_seqs, stream);
}

// Sequences seq0 .. seq0 + n_seqs - 1. logs given, or, walked, what they are formed from (low, up, up_bias, tau): the
// channel form; else the head form (raw, dt_bias, A_log; skip or null; or decay [H] alone, then act != 0 puts q, k and v through SiLU). walk != 0: token by token; else chunks, for portions
// of up to max_q_len tokens.
extern "C" int tw_linear_state(const float* src, long ld, int q_col, int k_col, int v_col, int share, const float* logs,
                               long ld_logs, const float* low, long ld_low, int rank, const float* up,
                               const float* up_bias, float tau, const float* raw, long ld_raw, int raw_col, const float* dt_bias,
                               const float* A_log, const float* skip, float* state, const int* q_start,
                               const int* state_slots, int seq0, int n_seqs, int max_q_len, float* out, long ld_out, int H,
                               int D, int E, float q_scale, const float* decay, int act, int walk, float* workspace,
                               long workspace_floats, hipStream_t stream) {
  TW_REQUIRE(src && state && q_start && state_slots && out && (logs || low || decay || (raw && dt_bias && A_log)));
  TW_REQUIRE((!decay || (!logs && !low)) && (!act || decay));
  TW_REQUIRE(!low || (walk && up && up_bias && rank > 0 && ld_low >= rank && tau > 0.f));
  TW_REQUIRE(seq0 >= 0 && n_seqs >= 0 && max_q_len >= 1 && H > 0 && D > 0 && D <= 256 && E > 0 && share > 0 && H % share == 0);
  TW_REQUIRE(q_col >= 0 && k_col >= 0 && v_col >= 0 && ld >= (long)max(q_col, k_col) + (long)(H / share) * D &&
             ld >= (long)v_col + (long)H * E && ld_out >= (long)H * E);
  TW_REQUIRE(logs ? ld_logs >= (long)H * D : (low || decay) ? true : (raw_col >= 0 && ld_raw >= (long)raw_col + H));
  TW_REQUIRE((uintptr_t)state % 16 == 0 && n_seqs <= 65535 && H <= 65535);
  if (n_seqs == 0) return 0;
  const int Dp = (D + 15) / 16 * 16, Ep = (E + 15) / 16 * 16;
  LsArgs a{src, ld, q_col, k_col, v_col, share, logs, ld_logs, low, ld_low, rank, up, up_bias, tau, raw, ld_raw, raw_col,
           dt_bias, A_log, skip, state, q_start,
           state_slots, seq0, out, ld_out, H, D, E, Dp, Ep, q_scale, decay, act != 0,
           D % 4 == 0 && ld % 4 == 0 && q_col % 4 == 0 && k_col % 4 == 0 && (uintptr_t)src % 16 == 0};
  LsSegments sg{nullptr, nullptr, 0, 1};
  if (!walk) {
    ls_segments(n_seqs, max_q_len, H, Ep, &sg.len, &sg.count);
    if (sg.count > 1) {
      TW_REQUIRE(workspace && (uintptr_t)workspace % 16 == 0 &&
                 workspace_floats >= tw_linear_state_workspace_floats(n_seqs, max_q_len, H, Dp, Ep));
      sg.states = workspace;
      sg.logs = workspace + (size_t)n_seqs * H * sg.count * Ep * Dp;
    }
    TW_REQUIRE(sg.count <= 65535);
  }
  if (logs || low) return ls_launch<LS_CHANNEL>(a, sg, n_seqs, walk, stream);
  return decay ? ls_launch<LS_FIXED>(a, sg, n_seqs, walk, stream) : ls_launch<LS_HEAD>(a, sg, n_seqs, walk, stream);
}

// ---- the logarithms of a channel's decay --------------------------------------------------------------------------
// out[n][c] = log sigmoid(z) / tau, z = sum_r low[n][r] * up[r][c] + bias[c]: a low-rank product (its first half comes from
// a packed projection), the sigmoid and its root. up is held [rank][channels]. 8 tokens a block, a channel a thread.
#define LS_GATE_TOKENS 8
#define LS_GATE_RANK 64
__global__ __launch_bounds__(256) void ls_decay_kernel(const float* __restrict__ low, long ld, const float* __restrict__ up,
                                                       const float* __restrict__ bias, float tau, float* __restrict__ out,
                                                       long ld_out, int n, int rank, int channels) {
  __shared__ float low_s[LS_GATE_TOKENS][LS_GATE_RANK];
  const int n0 = blockIdx.y * LS_GATE_TOKENS, c = blockIdx.x * 256 + threadIdx.x;
  const int rows = min(LS_GATE_TOKENS, n - n0);
  float z[LS_GATE_TOKENS];
#pragma unroll
  for (int t = 0; t < LS_GATE_TOKENS; ++t) z[t] = 0.f;
  for (int r0 = 0; r0 < rank; r0 += LS_GATE_RANK) {
    const int rs = min(LS_GATE_RANK, rank - r0);
    __syncthreads();
    for (int i = threadIdx.x; i < rows * rs; i += 256) low_s[i / rs][i % rs] = low[(size_t)(n0 + i / rs) * ld + r0 + i % rs];
    __syncthreads();
    if (c < channels) {
#pragma unroll 8
      for (int rr = 0; rr < rs; ++rr) {
        const float w = up[(size_t)(r0 + rr) * channels + c];
#pragma unroll
        for (int t = 0; t < LS_GATE_TOKENS; ++t) z[t] = __fmaf_rn(w, low_s[t][rr], z[t]);   // (rows behind the last hold anything)
      }
    }
  }
  if (c >= channels) return;
  const float b = bias[c];
#pragma unroll
  for (int t = 0; t < LS_GATE_TOKENS; ++t) {
    if (t >= rows) break;
    out[(size_t)(n0 + t) * ld_out + c] = ls_log_decay(z[t] + b, tau);
  }
}

extern "C" int tw_decay_logs(const float* low, long ld, const float* up, const float* bias, float tau, float* out, long ld_out,
                             int n, int rank, int channels, hipStream_t stream) {
  TW_REQUIRE(low && up && bias && out && n >= 0 && rank > 0 && channels > 0 && ld >= rank && ld_out >= channels && tau > 0.f);
  if (n == 0) return 0;
  ls_decay_kernel<<<dim3(tw_div_up(channels, 256), tw_div_up(n, LS_GATE_TOKENS)), 256, 0, stream>>>(low, ld, up, bias, tau, out,
                                                                                                    ld_out, n, rank, channels);
  return TW_LAUNCH_RESULT();
}

// ---- a gate, then a norm in equal parts -----------------------------------------------------------------------------
// out[n] = [.. u_p / sqrt(mean(u_p^2) + eps) ..] * weight over `parts` equal parts u_p of u = y * silu(gate), rounded to the
// compute type. THREADS 256: a block a (token, part); 64: a wave. AFTER: u = y, and the normed row is multiplied by
// sigmoid(gate) and by `scale` before it is rounded.
template <typename T, int THREADS, bool AFTER>
__global__ __launch_bounds__(256) void gate_group_norm_kernel(const float* __restrict__ y, long ld_y, const float* __restrict__ gate,
                                                              long ld_g, const float* __restrict__ weight, T* __restrict__ out,
                                                              long ld_out, int n, int parts, int size, float eps, float scale) {
  __shared__ float lds[16];
  const long unit = (long)blockIdx.x * (256 / THREADS) + threadIdx.x / THREADS;
  if (unit >= (long)n * parts) return;                        // (a whole block or a whole wave)
  const int lane = threadIdx.x % THREADS;
  const int row = (int)(unit / parts), c0 = (int)(unit % parts) * size;
  const float* src = y + (size_t)row * ld_y + c0;
  const float* g = gate + (size_t)row * ld_g + c0;
  constexpr int KEEP = 8;
  float kept[KEEP];
  float ss = 0.f;
  auto value = [&](int c) {
    if (AFTER) return src[c];
    const float z = g[c];
    return src[c] * (z / (1.f + expf(-z)));
  };
  auto finished = [&](float v, float rinv, int c) {
    const float r = v * rinv * weight[c0 + c];
    return AFTER ? r * (scale / (1.f + expf(-g[c]))) : r;
  };
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int c = lane + i * THREADS;
    kept[i] = c < size ? value(c) : 0.f;
    ss = __fmaf_rn(kept[i], kept[i], ss);
  }
  for (int c = lane + KEEP * THREADS; c < size; c += THREADS) {
    const float v = value(c);
    ss = __fmaf_rn(v, v, ss);
  }
  const float sum = THREADS == 64 ? tw_wave_sum(ss) : tw_block_sum(ss, lds);
  const float rinv = 1.f / sqrtf(sum / (float)size + eps);
  T* dst = out + (size_t)row * ld_out + c0;
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int c = lane + i * THREADS;
    if (c < size) dst[c] = tw_from_float<T>(finished(kept[i], rinv, c));
  }
  for (int c = lane + KEEP * THREADS; c < size; c += THREADS) dst[c] = tw_from_float<T>(finished(value(c), rinv, c));
}

template <typename T, bool AFTER>
static void gate_group_norm_launch(const float* y, long ld_y, const float* gate, long ld_g, const float* weight, void* out,
                                   long ld_out, int n, int parts, int size, float eps, float scale, hipStream_t stream) {
  const long units = (long)n * parts;
  if (size > 512)
    gate_group_norm_kernel<T, 256, AFTER><<<(unsigned)units, 256, 0, stream>>>(y, ld_y, gate, ld_g, weight, (T*)out, ld_out, n, parts, size, eps, scale);
  else
    gate_group_norm_kernel<T, 64, AFTER><<<tw_div_up(units, 4), 256, 0, stream>>>(y, ld_y, gate, ld_g, weight, (T*)out, ld_out, n, parts, size, eps, scale);
}

// after != 0: the gate (sigmoid) and `scale` behind the norm; else the gate (SiLU) in front of it.
extern "C" int tw_gate_group_norm(int dtype, const float* y, long ld_y, const float* gate, long ld_g, const float* weight,
                                  void* out, long ld_out, int n, int parts, int size, float eps, int after, float scale,
                                  hipStream_t stream) {
  TW_REQUIRE(y && gate && weight && out && n >= 0 && parts > 0 && size > 0 && eps > 0.f);
  TW_REQUIRE(ld_y >= (long)parts * size && ld_g >= (long)parts * size && ld_out >= (long)parts * size);
  if (n == 0) return 0;
#define TW_GATE_NORM(T)                                                                                                      \
  do {                                                                                                                       \
    if (after) gate_group_norm_launch<T, true>(y, ld_y, gate, ld_g, weight, out, ld_out, n, parts, size, eps, scale, stream);  \
    else gate_group_norm_launch<T, false>(y, ld_y, gate, ld_g, weight, out, ld_out, n, parts, size, eps, 1.f, stream);         \
  } while (0)
  if (dtype == TW_DTYPE_BF16) TW_GATE_NORM(bf16_t);
  else if (dtype == TW_DTYPE_F32) TW_GATE_NORM(float);
  else return TW_ERR_BAD_ARGUMENT;
#undef TW_GATE_NORM
  return TW_LAUNCH_RESULT();
}
