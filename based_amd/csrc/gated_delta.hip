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
// The scan walks tokens rather than blocks of tokens: 32-bit products are required, fp32 MFMA has
// the rate of the vector unit, and the blocked form needs about twice the products of the
// recurrence.  How a prompt is cut then cannot change more than the rounding of the carried state.
// Three products per state element and token:
//   * S^T k and S^T q are taken in one pass over the state BEFORE the update,
//     o = g S0^T q + (k . q) u, so that one reduction per token is on the dependent path;
//   * the decay is not multiplied into the state: the state is kept divided by the running product
//     of decays G, S = G Z, Z += k (u / G)^T, and Z is brought back to G = 1 when G gets small.
// A wavefront holds 8 CPL columns: lane = 8 column groups x 8 row groups, RPL rows x CPL columns in
// registers; the sums over rows are three DPP additions within 8 lanes.  Queries, keys and values
// of 16 tokens at a time are normalised and laid out in LDS in fp32 (two buffers), the raw ones of
// the tile after that being on their way in registers.
#include "stream_common.hpp"

namespace based {

constexpr float kUnitEps = 1e-6f;
constexpr int kDeltaTile = 16;               // tokens staged together
constexpr float kRescaleBelow = 1e-9f;       // running decay at which the stored state is brought back to scale 1

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
  int B, L, H, G, d, dv, dvp;
  long x_sb, x_sl;  // strides of q, k, v
  long g_sb, g_sl;  // strides of a, bt
  int fresh;
};

template <typename T> __device__ __forceinline__ float decay_of(float a, const void* a_log, const void* dt_bias, int h) {
  const float dt = softplus_f(a + to_f32(static_cast<const T*>(dt_bias)[h]));
  return expf(-expf(to_f32(static_cast<const T*>(a_log)[h])) * dt);
}

// E consecutive elements as they lie in memory; VEC: aligned to their size (16 bytes at most)
template <typename T, int E> struct Raw {
  static constexpr int kPer = E * (int)sizeof(T) > 16 ? 16 / (int)sizeof(T) : E;
  typedef __attribute__((ext_vector_type(kPer))) T piece_t;
  piece_t p[E / kPer];
  __device__ __forceinline__ float get(int i) const { return to_f32(p[i / kPer][i % kPer]); }
  template <bool VEC> __device__ __forceinline__ void load(const T* src, int valid) {
#pragma unroll
    for (int i = 0; i < E / kPer; ++i) {
      if constexpr (VEC) {
        // whole pieces are inside the row or outside of it
        const piece_t x = *reinterpret_cast<const piece_t*>(src + (i * kPer < valid ? i * kPer : 0));
#pragma unroll
        for (int j = 0; j < kPer; ++j) p[i][j] = i * kPer < valid ? x[j] : (T)0.0f;
      } else {
#pragma unroll
        for (int j = 0; j < kPer; ++j) {
          const T x = src[i * kPer + j < valid ? i * kPer + j : 0];
          p[i][j] = i * kPer + j < valid ? x : (T)0.0f;
        }
      }
    }
  }
};

template <typename T, int RPL, int CPL, int NW, bool VEC>
__global__ __launch_bounds__(64 * NW) void gated_delta_scan_kernel(const DeltaArgs a) {
  constexpr int D = RPL * 8;            // rows held (d <= D)
  constexpr int COLS = NW * 8 * CPL;    // columns of the workgroup
  constexpr int E = RPL / 2;            // channels of q and of k a staging thread brings: 16 threads per token
  constexpr int PASSES = 4 / NW;        // tokens per pass: 4 NW
  constexpr int EV = 2 * CPL;           // value channels a staging thread brings
  __shared__ __attribute__((aligned(16))) float s_k[2][kDeltaTile][D];
  __shared__ __attribute__((aligned(16))) float s_q[2][kDeltaTile][D];
  __shared__ __attribute__((aligned(16))) float s_v[2][kDeltaTile][COLS];
  __shared__ __attribute__((aligned(16))) float s_g[2][kDeltaTile][4];  // decay, beta, k . q
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, rg = lane & 7, cg = lane >> 3;
  const int b = blockIdx.x / a.H, h = blockIdx.x % a.H, hk = h / (a.H / a.G);
  const int col_wg = blockIdx.y * COLS, my_col = wave * 8 * CPL + cg * CPL;  // within the workgroup
  const T* q = static_cast<const T*>(a.q) + b * a.x_sb + (long)hk * a.d;
  const T* k = static_cast<const T*>(a.k) + b * a.x_sb + (long)hk * a.d;
  const T* v = static_cast<const T*>(a.v) + b * a.x_sb + (long)h * a.dv;
  const T* ga = static_cast<const T*>(a.a) + b * a.g_sb + h;
  const T* gb = static_cast<const T*>(a.bt) + b * a.g_sb + h;

  float S[RPL][CPL];
  float* st = a.state + ((long)b * a.H + h) * a.d * a.dvp + col_wg + my_col;
#pragma unroll
  for (int i = 0; i < RPL; ++i) {
    const int row = (i >> 2) * 32 + rg * 4 + (i & 3);
#pragma unroll
    for (int c = 0; c < CPL; ++c) {
      const bool in = !a.fresh && row < a.d && col_wg + my_col + c < a.dv;
      S[i][c] = in ? st[(long)row * a.dvp + c] : 0.f;
    }
  }

  // staging roles
  const int part = tid & 15, tok0 = tid >> 4;               // q, k: channels part * E ..
  const int vtok = tid / (4 * NW), vch = (tid % (4 * NW)) * EV;
  Raw<T, E> rq[PASSES], rk[PASSES];
  Raw<T, EV> rv;
  T ra[PASSES], rb[PASSES];
  auto fetch = [&](int l0) {
#pragma unroll
    for (int p = 0; p < PASSES; ++p) {
      const int l = l0 + p * 4 * NW + tok0;
      const long row = l < a.L ? l : a.L - 1;
      const int left = a.d - part * E;
      rq[p].template load<VEC>(q + row * a.x_sl + (left > 0 ? part * E : 0), left);
      rk[p].template load<VEC>(k + row * a.x_sl + (left > 0 ? part * E : 0), left);
      ra[p] = ga[row * a.g_sl];
      rb[p] = gb[row * a.g_sl];
    }
    const int l = l0 + vtok;
    const long row = l < a.L ? l : a.L - 1;
    const int left = a.dv - col_wg - vch;
    rv.template load<VEC>(v + row * a.x_sl + (left > 0 ? col_wg + vch : 0), left);
  };
  const float q_scale = 1.0f / sqrtf((float)a.d);
  auto stage = [&](int buf) {
#pragma unroll
    for (int p = 0; p < PASSES; ++p) {
      const int t = p * 4 * NW + tok0;
      float qq = 0.f, kk = 0.f, qk = 0.f;
#pragma unroll
      for (int i = 0; i < E; ++i) {
        const float x = rq[p].get(i), y = rk[p].get(i);
        qq = __builtin_fmaf(x, x, qq);
        kk = __builtin_fmaf(y, y, kk);
        qk = __builtin_fmaf(x, y, qk);
      }
      qq = sum16(qq), kk = sum16(kk), qk = sum16(qk);
      const float fq = q_scale / sqrtf(qq + kUnitEps), fk = 1.0f / sqrtf(kk + kUnitEps);
#pragma unroll
      for (int i = 0; i < E; ++i) {
        s_q[buf][t][part * E + i] = rq[p].get(i) * fq;
        s_k[buf][t][part * E + i] = rk[p].get(i) * fk;
      }
      if (part == 0) {
        s_g[buf][t][0] = decay_of<T>(to_f32(ra[p]), a.a_log, a.dt_bias, h);
        s_g[buf][t][1] = sigmoid_f(to_f32(rb[p]));
        s_g[buf][t][2] = qk * fq * fk;
      }
    }
#pragma unroll
    for (int i = 0; i < EV; ++i) s_v[buf][vtok][vch + i] = rv.get(i);
  };

  fetch(0);
  stage(0);
  float G = 1.0f;
  int buf = 0;
  const bool writer = rg == 0;
  float* op = a.o + ((long)b * a.L * a.H + h) * a.dv + col_wg + my_col;
  const int cols_left = a.dv - col_wg - my_col;
  for (int l0 = 0; l0 < a.L; l0 += kDeltaTile, buf ^= 1) {
    __syncthreads();  // this tile is laid out; everyone is done with the other buffer
    const bool more = l0 + kDeltaTile < a.L;
    if (more) fetch(l0 + kDeltaTile);
    const int n = a.L - l0 < kDeltaTile ? a.L - l0 : kDeltaTile;
    f32x4 kn[RPL / 4], qn[RPL / 4], gn;
    float vn[CPL];
    auto load_token = [&](int t) {
#pragma unroll
      for (int i = 0; i < RPL / 4; ++i) {
        kn[i] = *reinterpret_cast<const f32x4*>(&s_k[buf][t][i * 32 + rg * 4]);
        qn[i] = *reinterpret_cast<const f32x4*>(&s_q[buf][t][i * 32 + rg * 4]);
      }
      gn = *reinterpret_cast<const f32x4*>(&s_g[buf][t][0]);
#pragma unroll
      for (int c = 0; c < CPL; ++c) vn[c] = s_v[buf][t][my_col + c];
    };
    load_token(0);
    for (int t = 0; t < n; ++t) {
      f32x4 kc[RPL / 4], qc[RPL / 4];
      float vc[CPL];
#pragma unroll
      for (int i = 0; i < RPL / 4; ++i) kc[i] = kn[i], qc[i] = qn[i];
#pragma unroll
      for (int c = 0; c < CPL; ++c) vc[c] = vn[c];
      const float g = gn[0], beta = gn[1], kq = gn[2];
      load_token(t + 1 < n ? t + 1 : t);
      float sk[CPL], sq[CPL];
#pragma unroll
      for (int c = 0; c < CPL; ++c) {
        float k0 = 0.f, k1 = 0.f, q0 = 0.f, q1 = 0.f;
#pragma unroll
        for (int i = 0; i < RPL; i += 2) {
          k0 = __builtin_fmaf(S[i][c], kc[i >> 2][i & 3], k0);
          q0 = __builtin_fmaf(S[i][c], qc[i >> 2][i & 3], q0);
          k1 = __builtin_fmaf(S[i + 1][c], kc[i >> 2][(i & 3) + 1], k1);
          q1 = __builtin_fmaf(S[i + 1][c], qc[i >> 2][(i & 3) + 1], q1);
        }
        sk[c] = sum8(k0 + k1);
        sq[c] = sum8(q0 + q1);
      }
      G *= g;  // the same in every lane
      float o[CPL], u[CPL];
#pragma unroll
      for (int c = 0; c < CPL; ++c) {
        u[c] = beta * (vc[c] - G * sk[c]);
        o[c] = __builtin_fmaf(kq, u[c], G * sq[c]);
      }
      if (G < kRescaleBelow) {
#pragma unroll
        for (int i = 0; i < RPL; ++i)
#pragma unroll
          for (int c = 0; c < CPL; ++c) S[i][c] *= G;
        G = 1.0f;
      }
      const float inv = __builtin_amdgcn_rcpf(G);
#pragma unroll
      for (int c = 0; c < CPL; ++c) {
        const float uz = u[c] * inv;
#pragma unroll
        for (int i = 0; i < RPL; ++i) S[i][c] = __builtin_fmaf(kc[i >> 2][i & 3], uz, S[i][c]);
      }
      if (writer) {
        float* dst = op + (long)(l0 + t) * a.H * a.dv;
        if (CPL == 4 && (a.dv & 3) == 0) {
          if (cols_left > 0) *reinterpret_cast<f32x4*>(dst) = f32x4{o[0], o[1 % CPL], o[2 % CPL], o[3 % CPL]};
        } else {
#pragma unroll
          for (int c = 0; c < CPL; ++c)
            if (c < cols_left) dst[c] = o[c];
        }
      }
    }
    if (more) stage(buf ^ 1);
  }
#pragma unroll
  for (int i = 0; i < RPL; ++i) {
    const int row = (i >> 2) * 32 + rg * 4 + (i & 3);
#pragma unroll
    for (int c = 0; c < CPL; ++c)
      if (row < a.d && c < cols_left) st[(long)row * a.dvp + c] = S[i][c] * G;
  }
}

// ---- o / rms(o) * w * silu(gate) * scale: 16 lanes per (token, head) ----
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

template <typename T, bool VEC>
__global__ __launch_bounds__(256) void gated_rms_norm_kernel(const GatedNormArgs a) {
  constexpr int N = VEC ? Pack<T>::kN : 1;
  const long row0 = (long)blockIdx.x * 16 + (threadIdx.x >> 4);
  const bool live = row0 < a.rows;
  const long row = live ? row0 : a.rows - 1;
  const int lane = threadIdx.x & 15;
  const int h = (int)(row % a.H);
  const long bl = row / a.H;
  const long b = bl / a.L, l = bl % a.L;
  const float* o = a.o + row * a.dv;
  const T* gate = static_cast<const T*>(a.gate) + b * a.g_sb + l * a.g_sl + (long)h * a.dv;
  T* y = static_cast<T*>(a.y) + b * a.y_sb + l * a.y_sl + (long)h * a.dv;
  const T* w = static_cast<const T*>(a.w);
  float ss = 0.f;
  for (int p = lane; p * N < a.dv; p += 16) {
    float x[N];
    if constexpr (VEC) {
      load_vec<float, N>(o + p * N, x);
    } else {
      x[0] = o[p];
    }
#pragma unroll
    for (int j = 0; j < N; ++j) ss = __builtin_fmaf(x[j], x[j], ss);
  }
  const float r = 1.0f / sqrtf(sum16(ss) / (float)a.dv + a.eps);
  for (int p = lane; p * N < a.dv; p += 16) {
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

constexpr int kDeltaStepThreads = 512;

template <typename T, int RPT>
__global__ __launch_bounds__(kDeltaStepThreads) void gated_delta_step_kernel(const DeltaStepArgs a) {
  extern __shared__ float smem[];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int b = blockIdx.x / a.H, h = blockIdx.x % a.H, share = a.H / a.G, hk = h / share;
  const int pos = row_pos(a.pos, a.pos_host, b);
  if (pos < 0) return;
  const int cq_n = a.dvp / 4, rg_n = kDeltaStepThreads / cq_n;
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
  for (int i = tid; i < 2 * a.d + a.dv; i += kDeltaStepThreads) {
    const int ch = i < a.d ? hk * a.d + i : (i < 2 * a.d ? a.k_off + hk * a.d + i - a.d : a.v_off + h * a.dv + i - 2 * a.d);
    const T now = x[ch];
    float acc = 0.f;
    for (int j = 0; j < a.taps - 1; ++j) {
      const int p = pos - (a.taps - 1) + j;
      if (p >= 0) acc = __builtin_fmaf(to_f32(cw[(long)j * a.C + ch]), to_f32(ring[(long)(p % a.taps) * a.C + ch]), acc);
    }
    acc = __builtin_fmaf(to_f32(cw[(long)(a.taps - 1) * a.C + ch]), to_f32(now), acc);
    const float val = round_to<T>(silu_exact(acc));
    (i < a.d ? sq[i] : i < 2 * a.d ? sk[i - a.d] : sv[i - 2 * a.d]) = val;
    // a slot that no reader of this step looks at; shared query/key heads have one writer
    if (i >= 2 * a.d || h % share == 0) ring[(long)(pos % a.taps) * a.C + ch] = now;
  }
  if (tid == 0) {
    sc[3] = decay_of<T>(to_f32(static_cast<const T*>(a.a)[b * a.g_sb + h]), a.a_log, a.dt_bias, h);
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
  for (int c = tid; c < a.dvp; c += kDeltaStepThreads) {
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
  for (int c = tid; c < a.dv; c += kDeltaStepThreads)
    y[c] = from_f32<T>(so[c] * r * to_f32(static_cast<const T*>(a.norm_w)[c]) * silu_exact(to_f32(gate[c])) * a.scale);
}

template <typename T, int RPL, int CPL, int NW> void launch_delta_scan_vec(const DeltaArgs& a, bool vec, hipStream_t s) {
  const dim3 grid((unsigned)(a.B * a.H), (unsigned)((a.dv + NW * 8 * CPL - 1) / (NW * 8 * CPL))), block(64 * NW);
  if (vec)
    hipLaunchKernelGGL((gated_delta_scan_kernel<T, RPL, CPL, NW, true>), grid, block, 0, s, a);
  else
    hipLaunchKernelGGL((gated_delta_scan_kernel<T, RPL, CPL, NW, false>), grid, block, 0, s, a);
}

// More columns per lane spend fewer instructions per state element, fewer columns make more
// wavefronts: enough of them for two per SIMD are wanted first.
template <typename T, int RPL> void launch_delta_scan(const DeltaArgs& a, bool vec, hipStream_t s) {
  const long cols = (long)a.B * a.H * a.dv;
  if (cols >= 32l * 2048 && a.dv > 64)
    launch_delta_scan_vec<T, RPL, 4, 4>(a, vec, s);
  else if (cols >= 16l * 2048 && a.dv > 32)
    launch_delta_scan_vec<T, RPL, 2, 4>(a, vec, s);
  else
    launch_delta_scan_vec<T, RPL, 1, 4>(a, vec, s);
}

template <typename T, int RPT> void launch_delta_step(const DeltaStepArgs& a, hipStream_t s) {
  const int rg_n = kDeltaStepThreads / (a.dvp / 4);
  const size_t bytes = (size_t)(2 * a.d + 3 * a.dvp + 8 + 2 * rg_n * a.dvp) * sizeof(float);
  hipLaunchKernelGGL((gated_delta_step_kernel<T, RPT>), dim3((unsigned)(a.B * a.H)), dim3(kDeltaStepThreads), bytes, s, a);
}

}  // namespace based

extern "C" BASED_API int based_gated_delta_scan(const void* q, const void* k, const void* v, const void* a_gate, const void* b_gate,
                                                const void* a_log, const void* dt_bias, float* state, float* o, int64_t B, int64_t L,
                                                int64_t H, int64_t G, int64_t D, int64_t DV, int64_t state_row, int64_t x_sb,
                                                int64_t x_sl, int64_t g_sb, int64_t g_sl, int fresh, int io_dtype, void* stream) {
  using namespace based;
  BASED_REQUIRE(q && k && v && a_gate && b_gate && a_log && dt_bias && state && o, BASED_ERR_ARG, "gated_delta_scan: null pointer argument");
  BASED_REQUIRE(B >= 0 && L >= 0 && H > 0 && G > 0 && D > 0 && DV > 0, BASED_ERR_ARG, "gated_delta_scan: bad sizes");
  BASED_REQUIRE(H % G == 0, BASED_ERR_SHAPE, "gated_delta_scan: %ld heads do not divide into %ld query/key heads", (long)H, (long)G);
  BASED_REQUIRE(D <= 256, BASED_ERR_SHAPE, "gated_delta_scan: query/key size %ld (at most 256)", (long)D);
  BASED_REQUIRE(state_row >= DV, BASED_ERR_ARG, "gated_delta_scan: state rows of %ld for a value size of %ld", (long)state_row, (long)DV);
  BASED_REQUIRE(io_dtype == BASED_BF16 || io_dtype == BASED_F32, BASED_ERR_DTYPE, "gated_delta_scan: bad dtype");
  BASED_REQUIRE(B * H < (1ll << 31) && L < (1ll << 31) && DV < (1ll << 20), BASED_ERR_SHAPE, "gated_delta_scan: grid too large");
  if (B == 0 || L == 0) return BASED_OK;
  const DeltaArgs a{q,      k,      v,      a_gate,  b_gate, a_log,          dt_bias, state, o,    (int)B, (int)L,
                    (int)H, (int)G, (int)D, (int)DV, (int)state_row, x_sb, x_sl,  g_sb,  g_sl, fresh};
  hipStream_t s = static_cast<hipStream_t>(stream);
  // staging pieces: half a lane's rows (16 bytes at most) of q and k, 2 .. 8 elements of v
  const bool vec = D % 16 == 0 && DV % 8 == 0 && x_sb % 8 == 0 && x_sl % 8 == 0 && aligned_to(q, 16) && aligned_to(k, 16) && aligned_to(v, 16);
#define BASED_DELTA_ROWS(T)                              \
  if (D <= 32)                                           \
    launch_delta_scan<T, 4>(a, vec, s);                  \
  else if (D <= 64)                                      \
    launch_delta_scan<T, 8>(a, vec, s);                  \
  else if (D <= 128)                                     \
    launch_delta_scan<T, 16>(a, vec, s);                 \
  else                                                   \
    launch_delta_scan<T, 32>(a, vec, s);
  if (io_dtype == BASED_BF16) {
    BASED_DELTA_ROWS(__bf16)
  } else {
    BASED_DELTA_ROWS(float)
  }
#undef BASED_DELTA_ROWS
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
  BASED_REQUIRE((rows + 15) / 16 < (1ll << 31), BASED_ERR_SHAPE, "gated_rms_norm: grid too large");
  if (rows == 0) return BASED_OK;
  const GatedNormArgs a{o, weight, gate, y, (long)rows, (int)L, (int)H, (int)DV, g_sb, g_sl, y_sb, y_sl, eps, scale};
  const int n = io_dtype == BASED_BF16 ? 8 : 4;
  const bool vec = DV % n == 0 && g_sb % n == 0 && g_sl % n == 0 && y_sb % n == 0 && y_sl % n == 0 && aligned_to(o, 16) &&
                   aligned_to(weight, 16) && aligned_to(gate, 16) && aligned_to(y, 16);
  const dim3 grid((unsigned)((rows + 15) / 16)), block(256);
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (io_dtype == BASED_BF16) {
    if (vec)
      hipLaunchKernelGGL((gated_rms_norm_kernel<__bf16, true>), grid, block, 0, s, a);
    else
      hipLaunchKernelGGL((gated_rms_norm_kernel<__bf16, false>), grid, block, 0, s, a);
  } else {
    if (vec)
      hipLaunchKernelGGL((gated_rms_norm_kernel<float, true>), grid, block, 0, s, a);
    else
      hipLaunchKernelGGL((gated_rms_norm_kernel<float, false>), grid, block, 0, s, a);
  }
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
  const int rg_n = kDeltaStepThreads / ((int)state_row / 4), rows = ((int)D + rg_n - 1) / rg_n;
#define BASED_DELTA_STEP(T)                 \
  if (rows <= 4)                            \
    launch_delta_step<T, 4>(a, s);          \
  else if (rows <= 8)                       \
    launch_delta_step<T, 8>(a, s);          \
  else if (rows <= 16)                      \
    launch_delta_step<T, 16>(a, s);         \
  else                                      \
    launch_delta_step<T, 32>(a, s);
  BASED_REQUIRE(rows <= 32, BASED_ERR_SHAPE, "gated_delta_step: a state of %ld x %ld per head is too large", (long)D, (long)state_row);
  if (io_dtype == BASED_BF16) {
    BASED_DELTA_STEP(__bf16)
  } else {
    BASED_DELTA_STEP(float)
  }
#undef BASED_DELTA_STEP
  return check_launch("gated_delta_step");
}
