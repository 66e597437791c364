// Gated delta rule with short-convolved, unit-normalised queries and keys, for gfx950.
//
// Per value head (state S: d x dv, fp32), token by token:
//   S <- g S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q
// with g = exp(-exp(A_log) softplus(a + dt_bias)), beta = sigmoid(b), k and q divided by
// sqrt(sum(x^2) + 1e-6), q also multiplied by d^(-1/2); value head h reads query/key head
// h / (heads / kv_heads).
//
//   gated_delta_scan    a portion of any length: the recurrence itself, in fp32 vector arithmetic.
//   gated_delta_step    one token per sequence with everything around it: the short convolutions on
//                       their ring of past inputs, silu, unit norms, gates, the state update, the
//                       output norm and the output gate.
//   gated_rms_norm      o / rms(o) * w * silu(gate) * scale, behind the scan.
//
// The scan takes 16 tokens at a time, all of it in fp32 (fp32 MFMA, which has twice the rate of the
// vector unit).  With the decays multiplied up inside the block, G_t = g_1 .. g_t:
//   u_t = beta_t (v_t - G_t S0^T k_t) - sum_{s<t} A_ts u_s,   A_ts = beta_t (k_t . k_s) G_t / G_s
//   o_t = G_t S0^T q_t + sum_{s<=t} P_ts u_s,                 P_ts = (q_t . k_s) G_t / G_s
//   S16 = G_16 S0 + sum_s k_s (G_16 / G_s) u_s^T
// so with T = (I + A)^-1, U = T R.  At 16 tokens the products inside a block are a seventh of those
// with the state for 128 channels.  The quotients of decays are exponentials of differences of log
// decays: none of them overflows, and a decay of zero is zero.
//   gated_delta_prepare  T, P, the decays and the norm factors of every block, all blocks at once, one
//                        wavefront each; T by forward substitution (a power series in A would lose
//                        digits to cancellation)
//   gated_delta_scan     walks the blocks with the state in MFMA accumulators.  The accumulator layout
//                        (column = lane % 16, rows 4 (lane / 16) + i) is the second operand of
//                        instruction i as it stands when the contraction runs over rows {i, 4 + i,
//                        8 + i, 12 + i}, so neither the state nor U is ever moved between lanes.
#include "stream_common.hpp"

namespace based {

constexpr float kUnitEps = 1e-6f;
constexpr int kBlk = 16;            // tokens per block
// what gated_delta_prepare leaves per (sequence, head, block): T and P row-major, then 16 each of G_t,
// nk_t G_16 / G_t, beta_t, nq_t G_t and nk_t G_t, with nq_t and nk_t what turns q_t and k_t into unit vectors
constexpr int kPrepT = 0, kPrepP = 256, kPrepG = 512, kPrepTail = 528, kPrepBeta = 544, kPrepGq = 560, kPrepGk = 576;
constexpr int kPrepFloats = BASED_DELTA_PREP_FLOATS;

struct DeltaArgs {
  const void* q;
  const void* k;
  const void* v;
  const void* a;
  const void* bt;
  const void* a_log;
  const void* dt_bias;
  float* state;  // (B, H, d, dvp)
  float* o;      // (B, L, H, dv)
  float* prep;   // (B, H, blocks, kPrepFloats)
  int B, L, H, G, d, dv, dvp, blocks;
  long x_sb, x_sl;  // strides of q, k, v
  long g_sb, g_sl;  // strides of a, bt
  int fresh, vec;
};

template <typename T> __device__ __forceinline__ float log_decay_of(float a, const void* a_log, const void* dt_bias, int h) {
  const float dt = softplus_f(a + to_f32(static_cast<const T*>(dt_bias)[h]));
  return -expf(to_f32(static_cast<const T*>(a_log)[h])) * dt;
}

__device__ __forceinline__ f32x4 mfma_f32(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// 4 consecutive channels of a row of d as they lie in memory.  Fetched without a condition (channels
// past the end come from the row's start) and cleared where they are used: a load in a branch or
// in front of a select is waited for on the spot.  LAY: 0 element by element, 1 whole aligned groups, 2 whole
// groups of rows that fill the tile (nothing to clear).
template <typename T, int LAY> struct Four {
  typedef __attribute__((ext_vector_type(4))) T t4;
  t4 r;
  __device__ __forceinline__ void load(const T* row, int e, int d) {
    if constexpr (LAY == 2) {
      r = *reinterpret_cast<const t4*>(row + e);
    } else if constexpr (LAY == 1) {
      r = *reinterpret_cast<const t4*>(row + (e < d ? e : 0));
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i) r[i] = row[e + i < d ? e + i : 0];
    }
  }
  __device__ __forceinline__ f32x4 get(int e, int d) const {
    f32x4 x;
#pragma unroll
    for (int i = 0; i < 4; ++i) x[i] = LAY == 2 || e + i < d ? to_f32(r[i]) : 0.f;
    return x;
  }
};

template <typename T, bool VEC>
__global__ __launch_bounds__(256) void gated_delta_prepare_kernel(const DeltaArgs a) {
  __shared__ __attribute__((aligned(16))) float s_a[4][kBlk][kBlk + 4];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l16 = lane & 15, quad = lane >> 4;
  const long n_items = (long)a.B * a.H * a.blocks;
  const long item0 = (long)blockIdx.x * 4 + wave;
  const bool live = item0 < n_items;
  const long item = live ? item0 : n_items - 1;
  const int blk = (int)(item % a.blocks);
  const int h = (int)(item / a.blocks % a.H), b = (int)(item / a.blocks / a.H), hk = h / (a.H / a.G);
  const int t0 = blk * kBlk, tok = t0 + l16;
  const bool in = tok < a.L;
  const long row = in ? tok : a.L - 1;
  const T* q = static_cast<const T*>(a.q) + b * a.x_sb + row * a.x_sl + (long)hk * a.d;
  const T* k = static_cast<const T*>(a.k) + b * a.x_sb + row * a.x_sl + (long)hk * a.d;
  const long gate = b * a.g_sb + row * a.g_sl + h;
  // token l16's gates, in every lane of that number
  const float beta = in ? sigmoid_f(to_f32(static_cast<const T*>(a.bt)[gate])) : 0.f;
  float lg = in ? log_decay_of<T>(to_f32(static_cast<const T*>(a.a)[gate]), a.a_log, a.dt_bias, h) : 0.f;
  lg = fmaxf(lg, -200.f);  // exp(-200) is zero in fp32
  f32x4 kk = {0.f, 0.f, 0.f, 0.f}, qk = kk;
  float sq = 0.f, sk = 0.f;
  for (int e0 = 0; e0 < a.d; e0 += 64) {
    Four<T, VEC ? 1 : 0> xr[4], yr[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      xr[j].load(q, e0 + j * 16 + quad * 4, a.d);
      yr[j].load(k, e0 + j * 16 + quad * 4, a.d);
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const f32x4 x = xr[j].get(e0 + j * 16 + quad * 4, a.d), y = yr[j].get(e0 + j * 16 + quad * 4, a.d);
      if (e0 + j * 16 < a.d) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          sq = __builtin_fmaf(x[i], x[i], sq);
          sk = __builtin_fmaf(y[i], y[i], sk);
          kk = mfma_f32(y[i], y[i], kk);
          qk = mfma_f32(x[i], y[i], qk);
        }
      }
    }
  }
  sq += __shfl_xor(sq, 16, 64), sk += __shfl_xor(sk, 16, 64);
  sq += __shfl_xor(sq, 32, 64), sk += __shfl_xor(sk, 32, 64);
  const float fq = in ? 1.0f / (sqrtf((float)a.d) * sqrtf(sq + kUnitEps)) : 0.f, fk = in ? 1.0f / sqrtf(sk + kUnitEps) : 0.f;
  // log G of token l16, in 64 bits: behind a token that forgets nearly everything the differences of
  // these sums still have to carry the ordinary decays
  double lc = lg;
#pragma unroll
  for (int m = 1; m < 16; m <<= 1) {
    const double up = __shfl_up(lc, m, 16);
    if (l16 >= m) lc += up;
  }
  const double lc_end = __shfl(lc, 15, 64);
  float* out = a.prep + item * kPrepFloats;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int t = quad * 4 + i;  // row; l16 is the column s
    const double lc_t = __shfl(lc, t, 64);
    const float beta_t = __shfl(beta, t, 64), fq_t = __shfl(fq, t, 64), fk_t = __shfl(fk, t, 64);
    const float ratio = l16 <= t ? expf(fminf((float)(lc_t - lc), 0.f)) : 0.f;
    s_a[wave][t][l16] = l16 < t ? beta_t * kk[i] * fk_t * fk * ratio : 0.f;
    if (live) out[kPrepP + t * kBlk + l16] = qk[i] * fq_t * fk * ratio;
  }
  if (live && quad == 0) {
    const float G = expf((float)lc);
    out[kPrepG + l16] = G;
    out[kPrepTail + l16] = fk * expf(fminf((float)(lc_end - lc), 0.f));
    out[kPrepBeta + l16] = beta;
    out[kPrepGq + l16] = fq * G;
    out[kPrepGk + l16] = fk * G;
  }
  __syncthreads();
  // column l16 of T: x_t = [t = l16] - sum_{s<t} A_ts x_s
  float x[kBlk];
#pragma unroll
  for (int t = 0; t < kBlk; ++t) {
    float acc = t == l16 ? 1.f : 0.f;
#pragma unroll
    for (int s4 = 0; s4 < t; s4 += 4) {
      const f32x4 r = *reinterpret_cast<const f32x4*>(&s_a[wave][t][s4]);
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (s4 + j < t) acc = __builtin_fmaf(-r[j], x[s4 + j], acc);
    }
    x[t] = acc;
  }
  if (live && quad == 0) {
#pragma unroll
    for (int t = 0; t < kBlk; ++t) out[kPrepT + t * kBlk + l16] = x[t];
  }
}

// RB: 16-row blocks of the state; RS: wavefronts that share a 16-column tile, RB / RS row blocks each
// (their partial products with the state are added up through LDS).  Four wavefronts per workgroup.
// Queries and keys go from memory into the operands as they are: the factors that make unit vectors of
// them are factors of rows of the products, and have been multiplied into the decays.
template <typename T, int RB, int RS, int LAY>
__global__ __launch_bounds__(256) void gated_delta_scan_kernel(const DeltaArgs a) {
  static_assert(RB % RS == 0 && 4 % RS == 0, "row blocks divide among the wavefronts of a tile");
  constexpr int CT = 4 / RS, RBW = RB / RS;
  __shared__ __attribute__((aligned(16))) f32x4 s_part[2][RS > 1 ? CT * RS * 2 * 64 : 1];
  const int tid = threadIdx.x, lane = tid & 63, l16 = lane & 15, quad = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int ct = wave / RS, rs = wave % RS, row0 = rs * RBW * 16;
  // (the quotients are formed in vector registers: brought back so that every base address is a scalar)
  const int b = __builtin_amdgcn_readfirstlane(blockIdx.x / a.H), h = blockIdx.x - b * a.H;
  const int hk = __builtin_amdgcn_readfirstlane(h / (a.H / a.G));
  const int col = (blockIdx.y * CT + ct) * 16 + l16;
  const bool col_in = col < a.dv;
  const int vcol = col_in ? col : 0;
  const T* q = static_cast<const T*>(a.q) + b * a.x_sb + (long)hk * a.d;
  const T* k = static_cast<const T*>(a.k) + b * a.x_sb + (long)hk * a.d;
  const T* v = static_cast<const T*>(a.v) + b * a.x_sb + (long)h * a.dv;
  const float* prep = a.prep + ((long)b * a.H + h) * a.blocks * kPrepFloats;
  float* st = a.state + ((long)b * a.H + h) * a.d * a.dvp + vcol;
  float* o = a.o + ((long)b * a.L * a.H + h) * a.dv + vcol;
  const int last_blk = (a.L - 1) / kBlk, x_sl = (int)a.x_sl, o_sl = a.H * a.dv;

  f32x4 S[RBW];
#pragma unroll
  for (int r = 0; r < RBW; ++r)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int row = row0 + r * 16 + quad * 4 + i;
      const bool in = !a.fresh && col_in && row < a.d;
      S[r][i] = in ? st[(long)row * a.dvp] : 0.f;
    }

  // What a block needs from memory, asked for two blocks ahead into two sets of registers that take turns.
  struct Stage {
    Four<T, LAY> k[RBW], q[RBW];
    T kt[RBW][4], v[4];
    f32x4 t, p, gk, gq, tail, beta;
    float last;
  };
  auto fetch = [&](Stage& s, int blk) {
    const float* pr = prep + (long)blk * kPrepFloats;
    // rows past the last token are fetched from it, and a block that lies behind it from the block before
    const int at = (blk < last_blk ? blk : last_blk) * kBlk, left = a.L - 1 - at;
    const T* kb = k + (long)at * a.x_sl;
    const T* qb = q + (long)at * a.x_sl;
    const T* vb = v + (long)at * a.x_sl;
    const unsigned mine = (unsigned)((l16 < left ? l16 : left) * x_sl);
#pragma unroll
    for (int r = 0; r < RBW; ++r) {
      s.k[r].load(kb + mine, row0 + r * 16 + quad * 4, a.d);
      s.q[r].load(qb + mine, row0 + r * 16 + quad * 4, a.d);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = quad * 4 + i;
      const unsigned off = (unsigned)((t < left ? t : left) * x_sl);
#pragma unroll
      for (int r = 0; r < RBW; ++r) {
        const int row = row0 + r * 16 + l16;
        s.kt[r][i] = kb[off + (unsigned)(LAY == 2 || row < a.d ? row : 0)];
      }
      s.v[i] = vb[off + (unsigned)vcol];
    }
    s.t = *reinterpret_cast<const f32x4*>(pr + kPrepT + l16 * kBlk + quad * 4);
    s.p = *reinterpret_cast<const f32x4*>(pr + kPrepP + l16 * kBlk + quad * 4);
    s.gk = *reinterpret_cast<const f32x4*>(pr + kPrepGk + quad * 4);
    s.gq = *reinterpret_cast<const f32x4*>(pr + kPrepGq + quad * 4);
    s.tail = *reinterpret_cast<const f32x4*>(pr + kPrepTail + quad * 4);
    s.beta = *reinterpret_cast<const f32x4*>(pr + kPrepBeta + quad * 4);
    s.last = pr[kPrepG + kBlk - 1];
  };

  const f32x4 none = {0.f, 0.f, 0.f, 0.f};
  auto block = [&](Stage& s, int blk, int buf) {
    f32x4 kf[RBW], qf[RBW], kt[RBW];
#pragma unroll
    for (int r = 0; r < RBW; ++r) {
      kf[r] = s.k[r].get(row0 + r * 16 + quad * 4, a.d);
      qf[r] = s.q[r].get(row0 + r * 16 + quad * 4, a.d);
#pragma unroll
      for (int i = 0; i < 4; ++i) kt[r][i] = LAY == 2 || row0 + r * 16 + l16 < a.d ? to_f32(s.kt[r][i]) : 0.f;
    }
    // copies of their own: values that are used later in the block would otherwise stay in the registers the
    // next load wants, and the load's result be moved (and waited for) at the end of the loop
    f32x4 tm = s.t, pm = s.p, gk = s.gk, gq = s.gq, tail = s.tail, beta = s.beta;
    float last = s.last;
    asm volatile("" : "+v"(tm), "+v"(pm), "+v"(gk), "+v"(gq), "+v"(tail), "+v"(beta), "+v"(last));
    float vv[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) vv[i] = to_f32(s.v[i]);
    fetch(s, blk + 2 < a.blocks ? blk + 2 : a.blocks - 1);
    // two sums each for keys and queries: a product that waits for the one before it leaves the pipe idle
    f32x4 kq[2][2] = {{none, none}, {none, none}};
#pragma unroll
    for (int r = 0; r < RBW; ++r)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        kq[0][i & 1] = mfma_f32(kf[r][i], S[r][i], kq[0][i & 1]);
        kq[1][i & 1] = mfma_f32(qf[r][i], S[r][i], kq[1][i & 1]);
      }
    f32x4 ks = kq[0][0] + kq[0][1], qs = kq[1][0] + kq[1][1];
    if constexpr (RS > 1) {
      f32x4* part = &s_part[buf][ct * RS * 2 * 64];
      part[(rs * 2 + 0) * 64 + lane] = ks;
      part[(rs * 2 + 1) * 64 + lane] = qs;
      // the waves exchange data through LDS only: what is on its way from memory is not waited for
      __builtin_amdgcn_fence(__ATOMIC_RELEASE, "workgroup", "local");
      __builtin_amdgcn_s_barrier();
      __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "workgroup", "local");
      ks = part[lane];
      qs = part[64 + lane];
#pragma unroll
      for (int r = 1; r < RS; ++r) {
        ks += part[(r * 2 + 0) * 64 + lane];
        qs += part[(r * 2 + 1) * 64 + lane];
      }
    }
    float r4[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) r4[i] = beta[i] * (vv[i] - gk[i] * ks[i]);
    f32x4 u = mfma_f32(tm[0], r4[0], none), u1 = mfma_f32(tm[1], r4[1], none);
    u = mfma_f32(tm[2], r4[2], u), u1 = mfma_f32(tm[3], r4[3], u1);
#pragma unroll
    for (int r = 0; r < RBW; ++r) S[r] *= last;
    u += u1;
    float ut[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) ut[i] = u[i] * tail[i];
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int r = 0; r < RBW; ++r) S[r] = mfma_f32(kt[r][i], ut[i], S[r]);
    f32x4 oo = gq * qs;
    f32x4 o1 = mfma_f32(pm[1], u[1], none);
    oo = mfma_f32(pm[0], u[0], oo);
    o1 = mfma_f32(pm[3], u[3], o1);
    oo = mfma_f32(pm[2], u[2], oo);
    oo += o1;
    if (rs == 0 && col_in) {
      float* ob = o + (long)blk * kBlk * o_sl;
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (blk * kBlk + quad * 4 + i < a.L) ob[(quad * 4 + i) * o_sl] = oo[i];
    }
  };

  Stage s0, s1;
  // (kept apart: the wait for a set counts the loads behind it, and takes the least favourable order of
  // those in front of the loop and in it)
  fetch(s0, 0);
  __builtin_amdgcn_sched_barrier(0);
  fetch(s1, 1);
  __builtin_amdgcn_sched_barrier(0);
  // The number of blocks is even (an empty one changes nothing): a way out between the two would make
  // copies of the registers that are being loaded, and wait for them.
  for (int blk = 0; blk < a.blocks; blk += 2) {
    block(s0, blk, 0);
    block(s1, blk + 1, 1);
  }
#pragma unroll
  for (int r = 0; r < RBW; ++r)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int row = row0 + r * 16 + quad * 4 + i;
      if (col_in && row < a.d) st[(long)row * a.dvp] = S[r][i];
    }
}

// ---- o / rms(o) * w * silu(gate) * scale: LPR (8 or 16) lanes per (token, head) ----
struct GatedNormArgs {
  const float* o;  // (B, L, H, dv)
  const void* w;
  const void* gate;
  void* y;
  long rows;  // B L H
  int L, H, dv;
  long g_sb, g_sl, y_sb, y_sl;
  float eps, scale;
};

template <typename T, bool VEC, int LPR>
__global__ __launch_bounds__(256) void gated_rms_norm_kernel(const GatedNormArgs a) {
  constexpr int N = VEC ? Pack<T>::kN : 1;
  const long row0 = (long)blockIdx.x * (256 / LPR) + threadIdx.x / LPR;
  const bool live = row0 < a.rows;
  const long row = live ? row0 : a.rows - 1;
  const int lane = threadIdx.x % LPR;
  const int h = (int)(row % a.H);
  const long bl = row / a.H;
  const long b = bl / a.L, l = bl % a.L;
  const float* o = a.o + row * a.dv;
  const T* gate = static_cast<const T*>(a.gate) + b * a.g_sb + l * a.g_sl + (long)h * a.dv;
  T* y = static_cast<T*>(a.y) + b * a.y_sb + l * a.y_sl + (long)h * a.dv;
  const T* w = static_cast<const T*>(a.w);
  float ss = 0.f;
  for (int p = lane; p * N < a.dv; p += LPR) {
    float x[N];
    if constexpr (VEC) {
      load_vec<float, N>(o + p * N, x);
    } else {
      x[0] = o[p];
    }
#pragma unroll
    for (int j = 0; j < N; ++j) ss = __builtin_fmaf(x[j], x[j], ss);
  }
  const float r = 1.0f / sqrtf((LPR == 16 ? sum16(ss) : sum8(ss)) / (float)a.dv + a.eps);
  for (int p = lane; p * N < a.dv; p += LPR) {
    float x[N], g[N], wv[N], out[N];
    if constexpr (VEC) {
      load_vec<float, N>(o + p * N, x);
      load_vec<T, N>(gate + p * N, g);
      load_vec<T, N>(w + p * N, wv);
    } else {
      x[0] = o[p], g[0] = to_f32(gate[p]), wv[0] = to_f32(w[p]);
    }
#pragma unroll
    for (int j = 0; j < N; ++j) out[j] = x[j] * r * wv[j] * silu_exact(g[j]) * a.scale;
    if (live) {
      if constexpr (VEC)
        store_vec<T, N>(y + p * N, out);
      else
        y[p] = from_f32<T>(out[0]);
    }
  }
}

template <typename T> void launch_gated_norm(const GatedNormArgs& a, bool vec, hipStream_t s) {
  const bool narrow = a.dv <= 8 * (vec ? Pack<T>::kN : 1);
  const int per = narrow ? 32 : 16;
  const dim3 grid((unsigned)((a.rows + per - 1) / per)), block(256);
  if (vec) {
    if (narrow)
      hipLaunchKernelGGL((gated_rms_norm_kernel<T, true, 8>), grid, block, 0, s, a);
    else
      hipLaunchKernelGGL((gated_rms_norm_kernel<T, true, 16>), grid, block, 0, s, a);
  } else {
    if (narrow)
      hipLaunchKernelGGL((gated_rms_norm_kernel<T, false, 8>), grid, block, 0, s, a);
    else
      hipLaunchKernelGGL((gated_rms_norm_kernel<T, false, 16>), grid, block, 0, s, a);
  }
}

// ---- one token per sequence, one workgroup per (sequence, value head) ----
struct DeltaStepArgs {
  const void* x;       // (B, C): the projections that go through the short convolution
  const void* conv_w;  // (taps, C)
  void* ring;          // (B, taps, C)
  const void* a;
  const void* bt;
  const void* gate;
  const void* a_log;
  const void* dt_bias;
  const void* norm_w;
  float* state;
  void* y;
  const int32_t* pos;
  int pos_host;
  int B, H, G, d, dv, dvp, C, taps, k_off, v_off;
  long x_sb, g_sb, gate_sb, y_sb, ring_sb;
  float eps, scale;
};

// NT threads, RPT rows of the state per thread.
template <typename T, int NT, int RPT>
__global__ __launch_bounds__(NT) void gated_delta_step_kernel(const DeltaStepArgs a) {
  extern __shared__ float smem[];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int b = blockIdx.x / a.H, h = blockIdx.x % a.H, share = a.H / a.G, hk = h / share;
  const int pos = row_pos(a.pos, a.pos_host, b);
  if (pos < 0) return;
  const int cq_n = a.dvp / 4, rg_n = NT / cq_n;
  float* sq = smem;                 // [d]
  float* sk = sq + a.d;             // [d]
  float* sv = sk + a.d;             // [dvp]
  float* su = sv + a.dvp;           // [dvp]
  float* so = su + a.dvp;           // [dvp]
  float* sc = so + a.dvp;           // [8]: sum q^2, sum k^2, sum q k, decay, beta
  float* pk = sc + 8;               // [rg_n][dvp] partial S^T k
  float* pq = pk + rg_n * a.dvp;    // [rg_n][dvp]
  // the state is asked for first
  const int cq = tid % cq_n, rgi = tid / cq_n;
  const bool act = rgi < rg_n;
  float* st = a.state + ((long)b * a.H + h) * a.d * a.dvp;
  f32x4 S[RPT];
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int row = rgi + i * rg_n;
    const bool in = act && row < a.d;
    const f32x4 x = *reinterpret_cast<const f32x4*>(st + (long)(in ? row : 0) * a.dvp + cq * 4);
    const float keep = in && pos > 0 ? 1.f : 0.f;
    // (a select, not a product: a fresh state may hold anything)
#pragma unroll
    for (int j = 0; j < 4; ++j) S[i][j] = keep != 0.f ? x[j] : 0.f;
  }
  // short convolutions and silu
  const T* x = static_cast<const T*>(a.x) + b * a.x_sb;
  const T* cw = static_cast<const T*>(a.conv_w);
  T* ring = static_cast<T*>(a.ring) + b * a.ring_sb;
  for (int i = tid; i < 2 * a.d + a.dv; i += NT) {
    const int ch = i < a.d ? hk * a.d + i : (i < 2 * a.d ? a.k_off + hk * a.d + i - a.d : a.v_off + h * a.dv + i - 2 * a.d);
    const T now = x[ch];
    float acc = ring_dot<T>(ring + ch, cw + ch, a.C, a.taps, pos);
    acc = __builtin_fmaf(to_f32(cw[(long)(a.taps - 1) * a.C + ch]), to_f32(now), acc);
    const float val = round_to<T>(silu_exact(acc));
    (i < a.d ? sq[i] : i < 2 * a.d ? sk[i - a.d] : sv[i - 2 * a.d]) = val;
    // a slot that no reader of this step looks at; shared query/key heads have one writer
    if (i >= 2 * a.d || h % share == 0) ring[(long)(pos % a.taps) * a.C + ch] = now;
  }
  if (tid == 0) {
    sc[3] = expf(log_decay_of<T>(to_f32(static_cast<const T*>(a.a)[b * a.g_sb + h]), a.a_log, a.dt_bias, h));
    sc[4] = sigmoid_f(to_f32(static_cast<const T*>(a.bt)[b * a.g_sb + h]));
  }
  __syncthreads();
  if (wave == 0) {
    float qq = 0.f, kk = 0.f, qk = 0.f;
    for (int i = lane; i < a.d; i += 64) {
      qq = __builtin_fmaf(sq[i], sq[i], qq);
      kk = __builtin_fmaf(sk[i], sk[i], kk);
      qk = __builtin_fmaf(sq[i], sk[i], qk);
    }
    qq = wave_sum(qq), kk = wave_sum(kk), qk = wave_sum(qk);
    if (lane == 0) sc[0] = qq, sc[1] = kk, sc[2] = qk;
  }
  if (act) {
    f32x4 ak = {0.f, 0.f, 0.f, 0.f}, aq = ak;
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
      const int row = rgi + i * rg_n;
      const float kv = row < a.d ? sk[row] : 0.f, qv = row < a.d ? sq[row] : 0.f;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        ak[j] = __builtin_fmaf(S[i][j], kv, ak[j]);
        aq[j] = __builtin_fmaf(S[i][j], qv, aq[j]);
      }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      pk[rgi * a.dvp + cq * 4 + j] = ak[j];
      pq[rgi * a.dvp + cq * 4 + j] = aq[j];
    }
  }
  __syncthreads();
  const float fq = 1.0f / (sqrtf((float)a.d) * sqrtf(sc[0] + kUnitEps)), fk = 1.0f / sqrtf(sc[1] + kUnitEps);
  const float g = sc[3], beta = sc[4], kq = sc[2] * fq * fk;
  for (int c = tid; c < a.dvp; c += NT) {
    float tk = 0.f, tq = 0.f;
    for (int r = 0; r < rg_n; ++r) {
      tk += pk[r * a.dvp + c];
      tq += pq[r * a.dvp + c];
    }
    const float u = c < a.dv ? beta * (sv[c] - g * fk * tk) : 0.f;
    su[c] = u;
    so[c] = c < a.dv ? __builtin_fmaf(kq, u, g * fq * tq) : 0.f;
  }
  __syncthreads();
  if (act) {
    float uj[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) uj[j] = su[cq * 4 + j];
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
      const int row = rgi + i * rg_n;
      if (row < a.d) {
        const float kv = sk[row] * fk;
        f32x4 n;
#pragma unroll
        for (int j = 0; j < 4; ++j) n[j] = __builtin_fmaf(kv, uj[j], g * S[i][j]);
        *reinterpret_cast<f32x4*>(st + (long)row * a.dvp + cq * 4) = n;
      }
    }
  }
  float ss = 0.f;
  for (int c = lane; c < a.dv; c += 64) ss = __builtin_fmaf(so[c], so[c], ss);
  const float r = 1.0f / sqrtf(wave_sum(ss) / (float)a.dv + a.eps);
  T* y = static_cast<T*>(a.y) + b * a.y_sb + (long)h * a.dv;
  const T* gate = static_cast<const T*>(a.gate) + b * a.gate_sb + (long)h * a.dv;
  for (int c = tid; c < a.dv; c += NT)
    y[c] = from_f32<T>(so[c] * r * to_f32(static_cast<const T*>(a.norm_w)[c]) * silu_exact(to_f32(gate[c])) * a.scale);
}

template <typename T, int RB, int RS, int LAY> void launch_delta_scan_split(const DeltaArgs& a, hipStream_t s) {
  const int cols = 16 * (4 / RS);
  const dim3 grid((unsigned)(a.B * a.H), (unsigned)((a.dv + cols - 1) / cols));
  hipLaunchKernelGGL((gated_delta_scan_kernel<T, RB, RS, LAY>), grid, dim3(256), 0, s, a);
}

// Tiles are shared by as many wavefronts as it takes to give every SIMD one; tall ones always, for their
// registers.
template <typename T, int RB, int LAY> void launch_delta_scan_lay(const DeltaArgs& a, hipStream_t s) {
  const long tiles = (long)a.B * a.H * ((a.dv + 15) / 16);
  constexpr bool kFour = RB % 4 == 0, kOnlyFour = kFour && (LAY == 0 || (RB > 12 && sizeof(T) == 4));
  if constexpr (kFour) {
    if (tiles < 512 || kOnlyFour) {
      launch_delta_scan_split<T, RB, 4, LAY>(a, s);
      return;
    }
  }
  if constexpr (!kOnlyFour) {
    if constexpr (RB % 2 == 0) {
      if (tiles < 1024 || RB > 8) {
        launch_delta_scan_split<T, RB, 2, LAY>(a, s);
        return;
      }
    }
    if constexpr (RB <= 8) launch_delta_scan_split<T, RB, 1, LAY>(a, s);
  }
}

template <typename T, int RB> void launch_delta_scan(const DeltaArgs& a, hipStream_t s) {
  if (!a.vec)
    launch_delta_scan_lay<T, RB, 0>(a, s);
  else if (a.d < RB * 16)
    launch_delta_scan_lay<T, RB, 1>(a, s);
  else
    launch_delta_scan_lay<T, RB, 2>(a, s);
}

template <typename T> void launch_delta(const DeltaArgs& a, hipStream_t s) {
  const long items = (long)a.B * a.H * a.blocks;
  const dim3 grid((unsigned)((items + 3) / 4));
  if (a.vec)
    hipLaunchKernelGGL((gated_delta_prepare_kernel<T, true>), grid, dim3(256), 0, s, a);
  else
    hipLaunchKernelGGL((gated_delta_prepare_kernel<T, false>), grid, dim3(256), 0, s, a);
  const int rb = (a.d + 15) / 16;
  if (rb <= 1)
    launch_delta_scan<T, 1>(a, s);
  else if (rb <= 2)
    launch_delta_scan<T, 2>(a, s);
  else if (rb <= 3)
    launch_delta_scan<T, 3>(a, s);
  else if (rb <= 4)
    launch_delta_scan<T, 4>(a, s);
  else if (rb <= 6)
    launch_delta_scan<T, 6>(a, s);
  else if (rb <= 8)
    launch_delta_scan<T, 8>(a, s);
  else if (rb <= 12)
    launch_delta_scan<T, 12>(a, s);
  else
    launch_delta_scan<T, 16>(a, s);
}

template <typename T, int NT, int RPT> void launch_delta_step_rows(const DeltaStepArgs& a, hipStream_t s) {
  const int rg_n = NT / (a.dvp / 4);
  const size_t bytes = (size_t)(2 * a.d + 3 * a.dvp + 8 + 2 * rg_n * a.dvp) * sizeof(float);
  hipLaunchKernelGGL((gated_delta_step_kernel<T, NT, RPT>), dim3((unsigned)(a.B * a.H)), dim3(NT), bytes, s, a);
}

constexpr int kDeltaStepMaxThreads = 512, kDeltaStepMaxRows = 32;

// About eight 16-byte pieces of the state per thread: enough in flight, and a small state does not pay
// for the barriers of many wavefronts.
template <typename T> void launch_delta_step(const DeltaStepArgs& a, hipStream_t s) {
  const int cq_n = a.dvp / 4;
  auto rows = [&](int nt) { return (a.d + nt / cq_n - 1) / (nt / cq_n); };
  if (cq_n <= 128 && rows(128) <= 8)
    launch_delta_step_rows<T, 128, 8>(a, s);
  else if (rows(256) <= 8)
    launch_delta_step_rows<T, 256, 8>(a, s);
  else if (rows(512) <= 8)
    launch_delta_step_rows<T, 512, 8>(a, s);
  else if (rows(512) <= 16)
    launch_delta_step_rows<T, 512, 16>(a, s);
  else
    launch_delta_step_rows<T, 512, 32>(a, s);
}

}  // namespace based

extern "C" BASED_API int based_gated_delta_scan(const void* q, const void* k, const void* v, const void* a_gate, const void* b_gate,
                                                const void* a_log, const void* dt_bias, float* state, float* work, float* o,
                                                int64_t B, int64_t L, int64_t H, int64_t G, int64_t D, int64_t DV, int64_t state_row, int64_t x_sb,
                                                int64_t x_sl, int64_t g_sb, int64_t g_sl, int fresh, int io_dtype, void* stream) {
  using namespace based;
  BASED_REQUIRE(q && k && v && a_gate && b_gate && a_log && dt_bias && state && work && o, BASED_ERR_ARG, "gated_delta_scan: null pointer argument");
  BASED_REQUIRE(B >= 0 && L >= 0 && H > 0 && G > 0 && D > 0 && DV > 0, BASED_ERR_ARG, "gated_delta_scan: bad sizes");
  BASED_REQUIRE(H % G == 0, BASED_ERR_SHAPE, "gated_delta_scan: %ld heads do not divide into %ld query/key heads", (long)H, (long)G);
  BASED_REQUIRE(D <= 256, BASED_ERR_SHAPE, "gated_delta_scan: query/key size %ld (at most 256)", (long)D);
  BASED_REQUIRE(state_row >= DV, BASED_ERR_ARG, "gated_delta_scan: state rows of %ld for a value size of %ld", (long)state_row, (long)DV);
  BASED_REQUIRE(io_dtype == BASED_BF16 || io_dtype == BASED_F32, BASED_ERR_DTYPE, "gated_delta_scan: bad dtype");
  BASED_REQUIRE(B * H < (1ll << 31) && L < (1ll << 31) && DV < (1ll << 20), BASED_ERR_SHAPE, "gated_delta_scan: grid too large");
  if (B == 0 || L == 0) return BASED_OK;
  const int64_t blocks = 2 * ((L + 2 * kBlk - 1) / (2 * kBlk));
  BASED_REQUIRE(B * H * blocks < (1ll << 32), BASED_ERR_SHAPE, "gated_delta_scan: grid too large");
  BASED_REQUIRE(x_sl < (1ll << 26) && H * DV < (1ll << 26), BASED_ERR_SHAPE, "gated_delta_scan: rows too long");
  BASED_REQUIRE(aligned_to(work, 16), BASED_ERR_ALIGN, "gated_delta_scan: the work space must be 16-byte aligned");
  // groups of four channels as one load
  const int vec = D % 4 == 0 && x_sb % 4 == 0 && x_sl % 4 == 0 && aligned_to(q, 16) && aligned_to(k, 16);
  const DeltaArgs a{q,      k,      v,      a_gate, b_gate,  a_log,          dt_bias,     state, o,    work, (int)B, (int)L,
                    (int)H, (int)G, (int)D, (int)DV, (int)state_row, (int)blocks, x_sb,  x_sl, g_sb, g_sl,   fresh, vec};
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (io_dtype == BASED_BF16)
    launch_delta<__bf16>(a, s);
  else
    launch_delta<float>(a, s);
  return check_launch("gated_delta_scan");
}

extern "C" BASED_API int based_gated_rms_norm(const float* o, const void* weight, const void* gate, void* y, int64_t B, int64_t L,
                                              int64_t H, int64_t DV, int64_t g_sb, int64_t g_sl, int64_t y_sb, int64_t y_sl,
                                              float eps, float scale, int io_dtype, void* stream) {
  using namespace based;
  BASED_REQUIRE(o && weight && gate && y, BASED_ERR_ARG, "gated_rms_norm: null pointer argument");
  BASED_REQUIRE(B >= 0 && L >= 0 && H > 0 && DV > 0, BASED_ERR_ARG, "gated_rms_norm: bad sizes");
  BASED_REQUIRE(io_dtype == BASED_BF16 || io_dtype == BASED_F32, BASED_ERR_DTYPE, "gated_rms_norm: bad dtype");
  const int64_t rows = B * L * H;
  BASED_REQUIRE(rows < (1ll << 33), BASED_ERR_SHAPE, "gated_rms_norm: grid too large");
  if (rows == 0) return BASED_OK;
  const GatedNormArgs a{o, weight, gate, y, (long)rows, (int)L, (int)H, (int)DV, g_sb, g_sl, y_sb, y_sl, eps, scale};
  const int n = io_dtype == BASED_BF16 ? 8 : 4;
  const bool vec = DV % n == 0 && g_sb % n == 0 && g_sl % n == 0 && y_sb % n == 0 && y_sl % n == 0 && aligned_to(o, 16) &&
                   aligned_to(weight, 16) && aligned_to(gate, 16) && aligned_to(y, 16);
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (io_dtype == BASED_BF16)
    launch_gated_norm<__bf16>(a, vec, s);
  else
    launch_gated_norm<float>(a, vec, s);
  return check_launch("gated_rms_norm");
}

extern "C" BASED_API int based_gated_delta_step(const void* x, const void* conv_w, void* ring, const void* a_gate, const void* b_gate,
                                                const void* out_gate, const void* a_log, const void* dt_bias, const void* norm_w,
                                                float* state, void* y, const int32_t* pos, int64_t pos_host, int64_t B, int64_t H,
                                                int64_t G, int64_t D, int64_t DV, int64_t state_row, int64_t C, int taps,
                                                int64_t k_off, int64_t v_off, int64_t x_sb, int64_t g_sb, int64_t gate_sb,
                                                int64_t y_sb, int64_t ring_sb, float eps, float scale, int io_dtype, void* stream) {
  using namespace based;
  BASED_REQUIRE(x && conv_w && ring && a_gate && b_gate && out_gate && a_log && dt_bias && norm_w && state && y, BASED_ERR_ARG,
                "gated_delta_step: null pointer argument");
  BASED_REQUIRE(B >= 0 && H > 0 && G > 0 && D > 0 && DV > 0 && pos_host >= 0, BASED_ERR_ARG, "gated_delta_step: bad sizes");
  BASED_REQUIRE(H % G == 0, BASED_ERR_SHAPE, "gated_delta_step: %ld heads do not divide into %ld query/key heads", (long)H, (long)G);
  BASED_REQUIRE(taps >= 1 && taps <= 8, BASED_ERR_SHAPE, "gated_delta_step: %d taps (1 to 8)", taps);
  BASED_REQUIRE(state_row >= DV && state_row % 4 == 0 && aligned_to(state, 16), BASED_ERR_ALIGN,
                "gated_delta_step: state rows must be whole 16-byte pieces");
  BASED_REQUIRE(D <= 256 && state_row <= 512 && D * state_row <= 65536, BASED_ERR_SHAPE,
                "gated_delta_step: a state of %ld x %ld per head is too large", (long)D, (long)state_row);
  BASED_REQUIRE(G * D <= k_off && k_off + G * D <= v_off && v_off + H * DV <= C, BASED_ERR_ARG, "gated_delta_step: bad channel layout");
  BASED_REQUIRE(io_dtype == BASED_BF16 || io_dtype == BASED_F32, BASED_ERR_DTYPE, "gated_delta_step: bad dtype");
  BASED_REQUIRE(B * H < (1ll << 31), BASED_ERR_SHAPE, "gated_delta_step: grid too large");
  if (B == 0) return BASED_OK;
  const DeltaStepArgs a{x,      conv_w, ring,   a_gate,  b_gate,         out_gate, a_log, dt_bias, norm_w,     state, y,
                        pos,    (int)pos_host, (int)B, (int)H,  (int)G, (int)D,   (int)DV, (int)state_row, (int)C, taps, (int)k_off,
                        (int)v_off, x_sb, g_sb, gate_sb, y_sb, ring_sb, eps, scale};
  hipStream_t s = static_cast<hipStream_t>(stream);
  const int rg_n = kDeltaStepMaxThreads / ((int)state_row / 4);
  BASED_REQUIRE((D + rg_n - 1) / rg_n <= kDeltaStepMaxRows, BASED_ERR_SHAPE, "gated_delta_step: a state of %ld x %ld per head is too large",
                (long)D, (long)state_row);
  if (io_dtype == BASED_BF16)
    launch_delta_step<__bf16>(a, s);
  else
    launch_delta_step<float>(a, s);
  return check_launch("gated_delta_step");
}
