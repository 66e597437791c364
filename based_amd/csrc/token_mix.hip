// Token mixing in front of a time-mixing layer, the low-rank decay of its channels, and two element-wise
// operations of a per-layer token input, for gfx950:
//
//   token_mix:      y_s,t = x_t + (x_{t-1} - x_t) * mu_s for several mixes s of the same input; the input
//                   before a portion comes from a ring (B, 2, D), slot p % 2 holds position p.
//   channel_decay:  log2 of exp(-exp(w2 tanh(h) + w0)) per channel, in fp32.
//   gelu_mul:       gelu_tanh(g) * table[index], the gate of a per-token embedding.
//   softcap:        cap * tanh(x / cap) in place.
//   token_side_step: a per-layer token input for single tokens, r = residual + mult * x and
//                   proj(gelu_tanh(gate r) * table[index]) in one launch, a few workgroups per token.
#include "stream_common.hpp"

namespace based {

struct TokenMixArgs {
  const void* x;
  const void* mu;  // (S, D)
  void* y;         // (S, B, L, D)
  void* ring;      // (B, 2, D) or null
  const int32_t* pos;
  int pos_host;
  int B, L, D, S;
  long x_sb, x_sl, ring_sb;
};

constexpr int kMixTile = 4;  // tokens per thread

template <typename T, int N> __device__ __forceinline__ void load_some(const T* p, float (&out)[N]) {
  if constexpr (N == 1)
    out[0] = to_f32(*p);
  else
    load_vec<T, N>(p, out);
}
template <typename T, int N> __device__ __forceinline__ void store_some(T* p, const float (&in)[N]) {
  if constexpr (N == 1)
    *p = from_f32<T>(in[0]);
  else
    store_vec<T, N>(p, in);
}

// A thread owns N consecutive channels and walks kMixTile tokens.
template <typename T, int N>
__global__ __launch_bounds__(256) void token_mix_kernel(const TokenMixArgs a) {
  const int c0 = (blockIdx.x * 256 + threadIdx.x) * N;
  if (c0 >= a.D) return;
  const int b = blockIdx.z, l0 = blockIdx.y * kMixTile;
  const int start = row_pos(a.pos, a.pos_host, b);
  if (start < 0) return;
  const T* x = static_cast<const T*>(a.x) + b * a.x_sb + c0;
  T* ring = a.ring != nullptr ? static_cast<T*>(a.ring) + b * a.ring_sb + c0 : nullptr;
  const int ntok = a.L - l0 < kMixTile ? a.L - l0 : kMixTile;
  float in[kMixTile][N], before[N];
#pragma unroll
  for (int t = 0; t < kMixTile; ++t) load_some<T, N>(x + (long)(l0 + (t < ntok ? t : ntok - 1)) * a.x_sl, in[t]);
#pragma unroll
  for (int c = 0; c < N; ++c) before[c] = 0.f;
  if (l0 > 0)
    load_some<T, N>(x + (long)(l0 - 1) * a.x_sl, before);
  else if (ring != nullptr && start > 0)
    load_some<T, N>(ring + (long)((start - 1) & 1) * a.D, before);
  for (int s = 0; s < a.S; ++s) {
    float mu[N];
    load_some<T, N>(static_cast<const T*>(a.mu) + (long)s * a.D + c0, mu);
    T* y = static_cast<T*>(a.y) + (((long)s * a.B + b) * a.L + l0) * a.D + c0;
#pragma unroll
    for (int t = 0; t < kMixTile; ++t)
      if (t < ntok) {
        float out[N];
#pragma unroll
        for (int c = 0; c < N; ++c) out[c] = __builtin_fmaf((t > 0 ? in[t > 0 ? t - 1 : 0][c] : before[c]) - in[t][c], mu[c], in[t][c]);
        store_some<T, N>(y + (long)t * a.D, out);
      }
  }
  // the portion's last input goes into the ring; the thread that has read the old one writes it
  if (ring != nullptr && blockIdx.y == 0) {
    float last[N];
    load_some<T, N>(x + (long)(a.L - 1) * a.x_sl, last);
    store_some<T, N>(ring + (long)((start + a.L - 1) & 1) * a.D, last);
  }
}

// ---- log2 decay of every channel: -exp(w2 tanh(h) + w0) log2(e) ----
struct ChannelDecayArgs {
  const void* h;   // (rows, R)
  const void* w2;  // (C, R)
  const void* w0;  // (C)
  float* y;        // (rows, C)
  long rows, h_sr;
  int C, R;
};

constexpr float kLog2e = 1.4426950408889634f;

constexpr int kDecayRows = 16;

// Any element type and size: 16 rows of tanh(h) in LDS, a thread per channel.
template <typename T>
__global__ __launch_bounds__(256) void channel_decay_kernel(const ChannelDecayArgs a) {
  extern __shared__ float th[];  // [kDecayRows][R]
  const long r0 = (long)blockIdx.x * kDecayRows;
  const int n = a.rows - r0 < kDecayRows ? (int)(a.rows - r0) : kDecayRows;
  for (int i = threadIdx.x; i < n * a.R; i += 256)
    th[i] = tanh_f(to_f32(static_cast<const T*>(a.h)[(r0 + i / a.R) * a.h_sr + i % a.R]));
  __syncthreads();
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= a.C) return;
  const T* w = static_cast<const T*>(a.w2) + (long)c * a.R;
  const float w0 = to_f32(static_cast<const T*>(a.w0)[c]);
  float acc[kDecayRows];
#pragma unroll
  for (int r = 0; r < kDecayRows; ++r) acc[r] = w0;
  for (int j = 0; j < a.R; ++j) {
    const float wj = to_f32(w[j]);
#pragma unroll
    for (int r = 0; r < kDecayRows; ++r) acc[r] = __builtin_fmaf(wj, th[(r < n ? r : 0) * a.R + j], acc[r]);
  }
#pragma unroll
  for (int r = 0; r < kDecayRows; ++r)
    if (r < n) a.y[(r0 + r) * a.C + c] = -expf(acc[r]) * kLog2e;
}

__device__ __forceinline__ f32x4 mfma16(bf16x8 a, bf16x8 b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }

// bf16, R a multiple of 8 up to 256, C of 4: a wavefront keeps tanh(h) of 16 rows, as two bf16 numbers each, and walks the
// channels of its part 16 at a time.
template <int KC>
__global__ __launch_bounds__(256) void channel_decay_mfma_kernel(const ChannelDecayArgs a) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l16 = lane & 15, quad = lane >> 4;
  const long row = (long)blockIdx.x * 64 + wave * 16 + l16;
  const long rr = row < a.rows ? row : a.rows - 1;
  const __bf16* h = static_cast<const __bf16*>(a.h) + rr * a.h_sr;
  bf16x8 raw[KC], hi[KC], lo[KC];
#pragma unroll
  for (int k = 0; k < KC; ++k) {
    const int e = k * 32 + quad * 8;
    raw[k] = *reinterpret_cast<const bf16x8*>(h + (e < a.R ? e : 0));
  }
  const int per = ((a.C + (int)gridDim.y - 1) / (int)gridDim.y + 15) / 16 * 16;
  const int c_lo = blockIdx.y * per, c_hi = c_lo + per < a.C ? c_lo + per : a.C;
  bf16x8 w[KC];
  bf16x4 w0;
  auto fetch = [&](int c0) {
    const int c = c0 + l16 < a.C ? c0 + l16 : a.C - 1, cq = c0 + quad * 4 < a.C ? c0 + quad * 4 : 0;
#pragma unroll
    for (int k = 0; k < KC; ++k) {
      const int e = k * 32 + quad * 8;
      w[k] = *reinterpret_cast<const bf16x8*>(static_cast<const __bf16*>(a.w2) + (c * a.R + (e < a.R ? e : 0)));
    }
    w0 = *reinterpret_cast<const bf16x4*>(static_cast<const __bf16*>(a.w0) + cq);
  };
  if (c_lo < c_hi) fetch(c_lo);
#pragma unroll
  for (int k = 0; k < KC; ++k)
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const float t = k * 32 + quad * 8 < a.R ? tanh_f(to_f32(raw[k][j])) : 0.f;
      hi[k][j] = (__bf16)t;
      lo[k][j] = (__bf16)(t - (float)hi[k][j]);
    }
  for (int c0 = c_lo; c0 < c_hi; c0 += 16) {
    f32x4 acc;
#pragma unroll
    for (int i = 0; i < 4; ++i) acc[i] = to_f32(w0[i]);
#pragma unroll
    for (int k = 0; k < KC; ++k) {
      acc = mfma16(w[k], hi[k], acc);
      acc = mfma16(w[k], lo[k], acc);
    }
    if (c0 + 16 < c_hi) fetch(c0 + 16);
    // lane: row l16, channels 4 quad + i
    f32x4 out;
#pragma unroll
    for (int i = 0; i < 4; ++i) out[i] = -exp_f(acc[i]) * kLog2e;
    if (row < a.rows && c0 + quad * 4 < c_hi) *reinterpret_cast<f32x4*>(a.y + row * a.C + c0 + quad * 4) = out;
  }
}

// ---- gelu_tanh(g) * table[index] ----
struct GeluMulArgs {
  const void* g;
  const void* table;
  const int64_t* index;
  void* y;
  long rows, t_sr, t_n;
  int n;
  long g_sr;
};

template <typename T>
__global__ __launch_bounds__(256) void gelu_mul_kernel(const GeluMulArgs a) {
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= a.rows * a.n) return;
  const long row = i / a.n;
  const int c = (int)(i % a.n);
  const long src = a.index[row];
  const bool bad = src < 0 || src >= a.t_n;
  const float e = to_f32(static_cast<const T*>(a.table)[(bad ? 0 : src) * a.t_sr + c]);
  const float g = to_f32(static_cast<const T*>(a.g)[row * a.g_sr + c]);
  static_cast<T*>(a.y)[i] = from_f32<T>(bad ? __builtin_nanf("") : gelu_tanh_f(g) * e);
}

template <typename T>
__global__ __launch_bounds__(256) void softcap_kernel(T* x, long n, float cap) {
  constexpr int N = Pack<T>::kN;
  const long i0 = ((long)blockIdx.x * 256 + threadIdx.x) * N;
  if (i0 + N <= n) {
    float v[N];
    load_vec<T, N>(x + i0, v);
#pragma unroll
    for (int j = 0; j < N; ++j) v[j] = cap * tanh_f(v[j] / cap);
    store_vec<T, N>(x + i0, v);
  } else {
    for (long i = i0; i < n; ++i) x[i] = from_f32<T>(cap * tanh_f(to_f32(x[i]) / cap));
  }
}

// ---- a token input for single tokens ----
struct SideStepArgs {
  const __bf16* x;       // (M, D)
  const float* res_in;   // (M, D)
  float* res_out;        // (M, D)
  const __bf16* gate_w;  // (n, D)
  const __bf16* proj_w;  // (D, n)
  const __bf16* table;
  const int64_t* index;
  __bf16* y;             // (M, D)
  long x_sr, t_sr, t_n;
  int D, n, d_rows;
  float mult;
};

constexpr int kSideThreads = 1024, kSideWaves = kSideThreads / 64;
constexpr int kSideMaxDim = 4096, kSideMaxInner = 512;

// C: 512-channel pieces of a row a lane holds of each gate row (D <= 512 C).  Several workgroups per token: each forms the whole
// gate and d_rows rows of the product behind it; the first one writes the residual.
template <int C>
__global__ __launch_bounds__(kSideThreads) void token_side_step_kernel(const SideStepArgs a) {
  __shared__ __attribute__((aligned(16))) __bf16 row[512 * C];
  __shared__ __attribute__((aligned(16))) __bf16 inner[kSideMaxInner];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const long m = blockIdx.x;
  const int d0 = blockIdx.y * a.d_rows, d1 = d0 + a.d_rows < a.D ? d0 + a.d_rows : a.D;
  // the first gate rows and the first pieces of proj are asked for before anything else
  constexpr int GU = C >= 8 ? 1 : C >= 4 ? 2 : 4;  // gate rows in flight together
  bf16x8 g8[GU][C];
  auto fetch = [&](int j0) {
#pragma unroll
    for (int u = 0; u < GU; ++u)
#pragma unroll
      for (int c = 0; c < C; ++c) {
        const int e = (c * 64 + lane) * 8, j = j0 + u;
        g8[u][c] = *reinterpret_cast<const bf16x8*>(a.gate_w + (long)(j < a.n ? j : 0) * a.D + (e < a.D ? e : 0));
      }
  };
  fetch(wave * GU);
  // rows of proj are `lpr` lanes wide where that is a power of two up to 16, else one lane walks a row
  const int pieces = a.n / 8, lpr = pieces <= 16 && (pieces & (pieces - 1)) == 0 ? pieces : 1;
  const int first = d0 + tid / lpr, step = kSideThreads / lpr, piece = (tid % lpr) * 8;
  constexpr int PU = 2;  // rows of proj in flight together
  bf16x8 p8[PU];
#pragma unroll
  for (int u = 0; u < PU; ++u) {
    const int d = first + u * step;
    p8[u] = *reinterpret_cast<const bf16x8*>(a.proj_w + (long)(d < d1 ? d : d0) * a.n + piece);
  }
  const long src = a.index[m];
  const bool bad = src < 0 || src >= a.t_n;
  for (int e = tid * 4; e < 512 * C; e += kSideThreads * 4) {
    f32x4 r = {0.f, 0.f, 0.f, 0.f};
    if (e < a.D) {
      const bf16x4 x = *reinterpret_cast<const bf16x4*>(a.x + m * a.x_sr + e);
      if (a.res_in != nullptr) {
        r = *reinterpret_cast<const f32x4*>(a.res_in + m * a.D + e);
#pragma unroll
        for (int j = 0; j < 4; ++j) r[j] = __builtin_fmaf(a.mult, to_f32(x[j]), r[j]);
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j) r[j] = to_f32(x[j]);
      }
      if (blockIdx.y == 0) *reinterpret_cast<f32x4*>(a.res_out + m * a.D + e) = r;
    }
    bf16x4 o;
#pragma unroll
    for (int j = 0; j < 4; ++j) o[j] = (__bf16)r[j];
    *reinterpret_cast<bf16x4*>(row + e) = o;  // (zeros behind the row)
  }
  lds_barrier();
  for (int j0 = wave * GU; j0 < a.n; j0 += kSideWaves * GU) {
    if (j0 != wave * GU) fetch(j0);
    float acc[GU], e[GU];
#pragma unroll
    for (int u = 0; u < GU; ++u) {
      acc[u] = 0.f;
      e[u] = to_f32(a.table[(bad ? 0 : src) * a.t_sr + (j0 + u < a.n ? j0 + u : 0)]);
    }
#pragma unroll
    for (int c = 0; c < C; ++c) {
      float x[8];
      load_vec<__bf16, 8>(row + (c * 64 + lane) * 8, x);
#pragma unroll
      for (int u = 0; u < GU; ++u)
#pragma unroll
        for (int i = 0; i < 8; ++i) acc[u] = __builtin_fmaf(to_f32(g8[u][c][i]), x[i], acc[u]);
    }
#pragma unroll
    for (int u = 0; u < GU; ++u) {
      float v = sum16(acc[u]);
      v += __shfl_xor(v, 16, 64);
      v += __shfl_xor(v, 32, 64);
      if (lane == 0 && j0 + u < a.n) inner[j0 + u] = (__bf16)(bad ? __builtin_nanf("") : gelu_tanh_f(round_to<__bf16>(v)) * e[u]);
    }
  }
  lds_barrier();
  for (int t0 = d0; t0 < d1; t0 += PU * step) {  // (the same rounds for every lane: lanes of a row add up together)
    float acc[PU];
#pragma unroll
    for (int u = 0; u < PU; ++u) {
      const int d = t0 + tid / lpr + u * step;
      const __bf16* w = a.proj_w + (long)(d < d1 ? d : d0) * a.n;
      if (t0 != d0) p8[u] = *reinterpret_cast<const bf16x8*>(w + piece);
      acc[u] = 0.f;
      float x[8];
      load_vec<__bf16, 8>(inner + piece, x);
#pragma unroll
      for (int i = 0; i < 8; ++i) acc[u] = __builtin_fmaf(to_f32(p8[u][i]), x[i], acc[u]);
      if (lpr == 1) {
#pragma unroll 4
        for (int c = 8; c < a.n; c += 8) {
          float wv[8];
          load_vec<__bf16, 8>(w + c, wv);
          load_vec<__bf16, 8>(inner + c, x);
#pragma unroll
          for (int i = 0; i < 8; ++i) acc[u] = __builtin_fmaf(wv[i], x[i], acc[u]);
        }
      }
    }
#pragma unroll
    for (int u = 0; u < PU; ++u) {
      if (lpr >= 2) acc[u] = dpp_move_add<0xB1>(acc[u]);   // quad_perm [1,0,3,2]
      if (lpr >= 4) acc[u] = dpp_move_add<0x4E>(acc[u]);   // quad_perm [2,3,0,1]
      if (lpr >= 8) acc[u] = dpp_move_add<0x141>(acc[u]);  // row_half_mirror
      if (lpr >= 16) acc[u] = dpp_move_add<0x140>(acc[u]); // row_mirror
      const int d = t0 + tid / lpr + u * step;
      if (tid % lpr == 0 && d < d1) a.y[m * a.D + d] = (__bf16)acc[u];
    }
  }
}

}  // namespace based

extern "C" BASED_API int based_token_mix(const void* x, const void* mu, void* y, void* ring, const int32_t* pos, int64_t pos_host,
                                         int64_t B, int64_t L, int64_t D, int64_t S, int64_t x_sb, int64_t x_sl, int64_t ring_sb,
                                         int io_dtype, void* stream) {
  using namespace based;
  BASED_REQUIRE(x && mu && y, BASED_ERR_ARG, "token_mix: null pointer argument");
  BASED_REQUIRE(B >= 0 && L >= 0 && D > 0 && S > 0 && pos_host >= 0 && pos_host + L < (1ll << 31), BASED_ERR_ARG, "token_mix: bad sizes");
  BASED_REQUIRE(io_dtype == BASED_BF16 || io_dtype == BASED_F32, BASED_ERR_DTYPE, "token_mix: bad dtype");
  BASED_REQUIRE(B < 65536 && (L + kMixTile - 1) / kMixTile < 65536 && D < (1ll << 28), BASED_ERR_SHAPE, "token_mix: grid too large");
  if (B == 0 || L == 0) return BASED_OK;
  const int n = io_dtype == BASED_BF16 ? 8 : 4;
  const bool vec = D % n == 0 && x_sb % n == 0 && x_sl % n == 0 && ring_sb % n == 0 && aligned_to(x, 16) && aligned_to(mu, 16) &&
                   aligned_to(y, 16) && aligned_to(ring, 16);
  const TokenMixArgs a{x, mu, y, ring, pos, (int)pos_host, (int)B, (int)L, (int)D, (int)S, x_sb, x_sl, ring_sb};
  const int per = vec ? n : 1;
  const dim3 grid((unsigned)((D / per + 255) / 256), (unsigned)((L + kMixTile - 1) / kMixTile), (unsigned)B), block(256);
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (io_dtype == BASED_BF16) {
    if (vec)
      hipLaunchKernelGGL((token_mix_kernel<__bf16, 8>), grid, block, 0, s, a);
    else
      hipLaunchKernelGGL((token_mix_kernel<__bf16, 1>), grid, block, 0, s, a);
  } else {
    if (vec)
      hipLaunchKernelGGL((token_mix_kernel<float, 4>), grid, block, 0, s, a);
    else
      hipLaunchKernelGGL((token_mix_kernel<float, 1>), grid, block, 0, s, a);
  }
  return check_launch("token_mix");
}

extern "C" BASED_API int based_channel_decay(const void* h, const void* w2, const void* w0, float* y, int64_t rows, int64_t h_sr,
                                             int64_t C, int64_t R, int io_dtype, void* stream) {
  using namespace based;
  BASED_REQUIRE(h && w2 && w0 && y, BASED_ERR_ARG, "channel_decay: null pointer argument");
  BASED_REQUIRE(rows >= 0 && C > 0 && R > 0 && rows < (1ll << 31) && C < (1ll << 22), BASED_ERR_ARG, "channel_decay: bad sizes");
  BASED_REQUIRE(R <= 1024, BASED_ERR_SHAPE, "channel_decay: rank %ld (at most 1024)", (long)R);
  BASED_REQUIRE(io_dtype == BASED_BF16 || io_dtype == BASED_F32, BASED_ERR_DTYPE, "channel_decay: bad dtype");
  if (rows == 0) return BASED_OK;
  const ChannelDecayArgs a{h, w2, w0, y, (long)rows, (long)h_sr, (int)C, (int)R};
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (io_dtype == BASED_BF16 && R % 8 == 0 && R <= 256 && C % 4 == 0 && C * R < (1ll << 31) && h_sr % 8 == 0 &&
      aligned_to(h, 16) && aligned_to(w2, 16) && aligned_to(w0, 8) && aligned_to(y, 16)) {
    // parts of the channels: enough workgroups for short portions, few times tanh for long ones
    const int64_t blocks = (rows + 63) / 64, parts = blocks >= 512 ? 2 : (1024 + blocks - 1) / blocks;
    const dim3 grid((unsigned)blocks, (unsigned)(parts < (C + 63) / 64 ? parts : (C + 63) / 64));
    const int kc = (int)((R + 31) / 32);
    if (kc <= 1)
      hipLaunchKernelGGL((channel_decay_mfma_kernel<1>), grid, dim3(256), 0, s, a);
    else if (kc <= 2)
      hipLaunchKernelGGL((channel_decay_mfma_kernel<2>), grid, dim3(256), 0, s, a);
    else if (kc <= 4)
      hipLaunchKernelGGL((channel_decay_mfma_kernel<4>), grid, dim3(256), 0, s, a);
    else
      hipLaunchKernelGGL((channel_decay_mfma_kernel<8>), grid, dim3(256), 0, s, a);
    return check_launch("channel_decay");
  }
  const dim3 grid((unsigned)((rows + kDecayRows - 1) / kDecayRows), (unsigned)((C + 255) / 256));
  const size_t bytes = (size_t)kDecayRows * R * sizeof(float);
  if (io_dtype == BASED_BF16)
    hipLaunchKernelGGL(channel_decay_kernel<__bf16>, grid, dim3(256), bytes, s, a);
  else
    hipLaunchKernelGGL(channel_decay_kernel<float>, grid, dim3(256), bytes, s, a);
  return check_launch("channel_decay");
}

extern "C" BASED_API int based_gelu_mul(const void* g, const void* table, const int64_t* index, void* y, int64_t rows, int64_t n,
                                        int64_t g_sr, int64_t table_sr, int64_t table_n, int io_dtype, void* stream) {
  using namespace based;
  BASED_REQUIRE(g && table && index && y, BASED_ERR_ARG, "gelu_mul: null pointer argument");
  BASED_REQUIRE(rows >= 0 && n > 0 && table_n > 0 && rows * n < (1ll << 38), BASED_ERR_ARG, "gelu_mul: bad sizes");
  BASED_REQUIRE(io_dtype == BASED_BF16 || io_dtype == BASED_F32, BASED_ERR_DTYPE, "gelu_mul: bad dtype");
  if (rows == 0) return BASED_OK;
  const GeluMulArgs a{g, table, index, y, (long)rows, (long)table_sr, (long)table_n, (int)n, (long)g_sr};
  const dim3 grid((unsigned)((rows * n + 255) / 256));
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (io_dtype == BASED_BF16)
    hipLaunchKernelGGL(gelu_mul_kernel<__bf16>, grid, dim3(256), 0, s, a);
  else
    hipLaunchKernelGGL(gelu_mul_kernel<float>, grid, dim3(256), 0, s, a);
  return check_launch("gelu_mul");
}

extern "C" BASED_API int based_softcap(void* x, int64_t n, float cap, int io_dtype, void* stream) {
  using namespace based;
  BASED_REQUIRE(x || n == 0, BASED_ERR_ARG, "softcap: null pointer argument");
  BASED_REQUIRE(n >= 0 && n < (1ll << 38) && cap > 0.f, BASED_ERR_ARG, "softcap: bad sizes");
  BASED_REQUIRE(io_dtype == BASED_BF16 || io_dtype == BASED_F32, BASED_ERR_DTYPE, "softcap: bad dtype");
  BASED_REQUIRE(aligned_to(x, 16), BASED_ERR_ALIGN, "softcap: x must be 16-byte aligned");
  if (n == 0) return BASED_OK;
  hipStream_t s = static_cast<hipStream_t>(stream);
  const int per = io_dtype == BASED_BF16 ? 8 : 4;
  const dim3 grid((unsigned)((n + 256 * per - 1) / (256 * per)));
  if (io_dtype == BASED_BF16)
    hipLaunchKernelGGL(softcap_kernel<__bf16>, grid, dim3(256), 0, s, static_cast<__bf16*>(x), (long)n, cap);
  else
    hipLaunchKernelGGL(softcap_kernel<float>, grid, dim3(256), 0, s, static_cast<float*>(x), (long)n, cap);
  return check_launch("softcap");
}

extern "C" BASED_API int based_token_side_step(const void* x, const float* residual_in, float* residual_out, const void* gate_w,
                                               const void* proj_w, const void* table, const int64_t* index, void* y, int64_t M, int64_t D,
                                               int64_t n, int64_t x_sr, int64_t table_sr, int64_t table_n, float mult, void* stream) {
  using namespace based;
  BASED_REQUIRE(x && residual_out && gate_w && proj_w && table && index && y, BASED_ERR_ARG, "token_side_step: null pointer argument");
  BASED_REQUIRE(M >= 0 && D > 0 && n > 0 && table_n > 0 && M < (1ll << 31), BASED_ERR_ARG, "token_side_step: bad sizes");
  BASED_REQUIRE(D % 8 == 0 && D <= kSideMaxDim && n % 8 == 0 && n <= kSideMaxInner, BASED_ERR_SHAPE,
                "token_side_step: sizes %ld and %ld (multiples of 8, at most %d and %d)", (long)D, (long)n, kSideMaxDim, kSideMaxInner);
  BASED_REQUIRE(x_sr % 4 == 0 && aligned_to(x, 8) && aligned_to(residual_in, 16) && aligned_to(residual_out, 16) && aligned_to(gate_w, 16) &&
                    aligned_to(proj_w, 16),
                BASED_ERR_ALIGN, "token_side_step: rows must be whole 16-byte pieces");
  BASED_REQUIRE(residual_in != residual_out, BASED_ERR_ARG, "token_side_step: residual_out must not be residual_in");
  if (M == 0) return BASED_OK;
  // rows of the second product per workgroup: 256 or more, and no more workgroups than compute units
  const int most = M < 256 ? (int)(256 / M) : 1, wanted = (int)((D + 255) / 256), parts = wanted < most ? wanted : most;
  const int d_rows = (int)((D + parts - 1) / parts);
  const SideStepArgs a{static_cast<const __bf16*>(x), residual_in, residual_out, static_cast<const __bf16*>(gate_w),
                       static_cast<const __bf16*>(proj_w), static_cast<const __bf16*>(table), index, static_cast<__bf16*>(y), (long)x_sr,
                       (long)table_sr, (long)table_n, (int)D, (int)n, d_rows, mult};
  hipStream_t s = static_cast<hipStream_t>(stream);
  const dim3 grid((unsigned)M, (unsigned)((D + d_rows - 1) / d_rows)), block(kSideThreads);
  const int chunks = (int)((D + 511) / 512);
  if (chunks <= 1)
    hipLaunchKernelGGL((token_side_step_kernel<1>), grid, block, 0, s, a);
  else if (chunks <= 2)
    hipLaunchKernelGGL((token_side_step_kernel<2>), grid, block, 0, s, a);
  else if (chunks <= 4)
    hipLaunchKernelGGL((token_side_step_kernel<4>), grid, block, 0, s, a);
  else
    hipLaunchKernelGGL((token_side_step_kernel<8>), grid, block, 0, s, a);
  return check_launch("token_side_step");
}
