// The two element-wise operations in front of a mixer with a streamed input, for gfx950:
//
//   add_norm:     r = residual + mult * x  (fp32; r = x without a residual),
//                 y = norm(r) * w, norm the layer norm without a bias
//                 (r - mean) / sqrt(var + eps) or the RMS norm r / sqrt(mean(r^2) + eps).
//                 The norm sees the fp32 sum, not a rounded copy of it.  Optionally x is divided by its own
//                 RMS and weighted before it is added, and r also receives a vector and a row of a table
//                 (the embedding of the row's token, once more); without a norm y is the rounded sum.
//   stream_conv:  y_t = [x_t +] act(bias + sum_j w[j] x_{t - taps + 1 + j}), a causal convolution
//                 per channel over a sequence that arrives in portions of any length.  The inputs
//                 of earlier portions come from a ring (B, taps, D): slot p % taps holds the input
//                 at position p, so that the step of a single token writes a slot that no other
//                 reader of the same step looks at.
//
// Both are streams of 16-byte accesses; the convolution keeps the last taps - 1 inputs of its
// channels in registers and walks a tile of tokens, so every input is read once (plus a halo of
// taps - 1 rows per tile).
#include "stream_common.hpp"

namespace based {

enum { kNormRms = BASED_NORM_RMS, kNormLayer = BASED_NORM_LAYER, kNormNone = BASED_NORM_NONE };

struct AddNormArgs {
  const void* x;
  const float* res_in;
  const void* w;
  void* y;
  float* res_out;
  long rows;
  int D;
  long x_sr, ri_sr, y_sr, ro_sr;
  float eps, mult;
  int kind;
  StreamAddends add;
};

// One wavefront per row, the row in registers: NV pieces of 8 elements per lane (D <= 512 NV, D % 8 == 0).
// ADD: with what `StreamAddends` brings, or without a norm.
template <typename T, int NV, bool ADD>
__global__ __launch_bounds__(256) void add_norm_kernel(const AddNormArgs a) {
  const long row = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (row >= a.rows) return;
  const int lane = threadIdx.x & 63;
  const T* x = static_cast<const T*>(a.x) + row * a.x_sr;
  const T* w = static_cast<const T*>(a.w);
  float v[NV][8], wt[NV][8];
  bool live[NV];
#pragma unroll
  for (int c = 0; c < NV; ++c) {
    const int e = (c * 64 + lane) * 8;
    live[c] = e < a.D;
    load_vec<T, 8>(x + (live[c] ? e : 0), v[c]);
    if (!ADD || w != nullptr) load_vec<T, 8>(w + (live[c] ? e : 0), wt[c]);
  }
  float extra[ADD ? NV : 1][8];
  if constexpr (ADD) {
    const StreamAddends& m = a.add;
    long src = row;
    bool poison = false;
    if (m.rows != nullptr && m.rows_index != nullptr) {
      src = m.rows_index[row];
      poison = src < 0 || src >= m.rows_n;
      src = poison ? 0 : src;
    }
    float pw[NV][8];
    if (m.post_w != nullptr) {
#pragma unroll
      for (int c = 0; c < NV; ++c) load_vec<T, 8>(static_cast<const T*>(m.post_w) + (live[c] ? (c * 64 + lane) * 8 : 0), pw[c]);
    }
#pragma unroll
    for (int c = 0; c < NV; ++c) {
      const int e = live[c] ? (c * 64 + lane) * 8 : 0;
      float a8[8], b8[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) a8[i] = b8[i] = 0.f;
      if (m.vec != nullptr) load_vec<T, 8>(static_cast<const T*>(m.vec) + e, a8);
      if (m.rows != nullptr) load_vec<T, 8>(static_cast<const T*>(m.rows) + src * m.rows_sr + e, b8);
#pragma unroll
      for (int i = 0; i < 8; ++i) extra[c][i] = poison ? __builtin_nanf("") : a8[i] + b8[i];
    }
    if (m.post_w != nullptr) {
      float ss = 0.f;
#pragma unroll
      for (int c = 0; c < NV; ++c)
#pragma unroll
        for (int i = 0; i < 8; ++i) ss = live[c] ? __builtin_fmaf(v[c][i], v[c][i], ss) : ss;
      const float r = 1.0f / sqrtf(wave_sum(ss) / (float)a.D + m.post_eps);
#pragma unroll
      for (int c = 0; c < NV; ++c)
#pragma unroll
        for (int i = 0; i < 8; ++i) v[c][i] = v[c][i] * r * pw[c][i];
    }
  }
  if (a.res_in != nullptr) {
    const float* r = a.res_in + row * a.ri_sr;
#pragma unroll
    for (int c = 0; c < NV; ++c) {
      float rv[8];
      load_vec<float, 8>(r + (live[c] ? (c * 64 + lane) * 8 : 0), rv);
#pragma unroll
      for (int i = 0; i < 8; ++i) v[c][i] = __builtin_fmaf(a.mult, v[c][i], rv[i]);
    }
  }
  if constexpr (ADD) {
#pragma unroll
    for (int c = 0; c < NV; ++c)
#pragma unroll
      for (int i = 0; i < 8; ++i) v[c][i] += extra[c][i];
  }
  float s = 0.f;
#pragma unroll
  for (int c = 0; c < NV; ++c) {
    if (live[c]) {
      if (a.res_out != nullptr) store_vec<float, 8>(a.res_out + row * a.ro_sr + (c * 64 + lane) * 8, v[c]);
#pragma unroll
      for (int i = 0; i < 8; ++i) s += v[c][i];
    }
  }
  if constexpr (ADD) {
    if (a.kind == kNormNone) {
#pragma unroll
      for (int c = 0; c < NV; ++c)
        if (live[c]) store_vec<T, 8>(static_cast<T*>(a.y) + row * a.y_sr + (c * 64 + lane) * 8, v[c]);
      return;
    }
  }
  const float mean = a.kind == kNormLayer ? wave_sum(s) / (float)a.D : 0.f;
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < NV; ++c)
    if (live[c]) {
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        v[c][i] -= mean;
        ss = __builtin_fmaf(v[c][i], v[c][i], ss);
      }
    }
  const float rstd = 1.0f / sqrtf(wave_sum(ss) / (float)a.D + a.eps);
#pragma unroll
  for (int c = 0; c < NV; ++c)
    if (live[c]) {
      float o[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) o[i] = v[c][i] * rstd * wt[c][i];
      store_vec<T, 8>(static_cast<T*>(a.y) + row * a.y_sr + (c * 64 + lane) * 8, o);
    }
}

// Rows of any length and alignment: one workgroup per row, element by element, the row read again
// for every pass (it is in the cache).
template <typename T>
__global__ __launch_bounds__(256) void add_norm_any_kernel(const AddNormArgs a) {
  __shared__ float part[4];
  const long row = blockIdx.x;
  const T* x = static_cast<const T*>(a.x) + row * a.x_sr;
  const T* w = static_cast<const T*>(a.w);
  const float* r = a.res_in != nullptr ? a.res_in + row * a.ri_sr : nullptr;
  auto block_sum = [&](float v) {
    v = wave_sum(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) part[threadIdx.x >> 6] = v;
    __syncthreads();
    return part[0] + part[1] + part[2] + part[3];
  };
  const StreamAddends& m = a.add;
  const T* pw = static_cast<const T*>(m.post_w);
  const T* vec = static_cast<const T*>(m.vec);
  const T* add_row = nullptr;
  bool poison = false;
  if (m.rows != nullptr) {
    long src = m.rows_index != nullptr ? m.rows_index[row] : row;
    poison = m.rows_index != nullptr && (src < 0 || src >= m.rows_n);
    add_row = static_cast<const T*>(m.rows) + (poison ? 0 : src) * m.rows_sr;
  }
  float post = 1.f;
  if (pw != nullptr) {
    float ss = 0.f;
    for (int e = threadIdx.x; e < a.D; e += 256) ss = __builtin_fmaf(to_f32(x[e]), to_f32(x[e]), ss);
    post = 1.0f / sqrtf(block_sum(ss) / (float)a.D + m.post_eps);
  }
  auto sum_at = [&](int e) {
    float v = to_f32(x[e]);
    if (pw != nullptr) v = v * post * to_f32(pw[e]);
    if (r != nullptr) v = __builtin_fmaf(a.mult, v, r[e]);
    const float more = (vec != nullptr ? to_f32(vec[e]) : 0.f) + (add_row != nullptr ? to_f32(add_row[e]) : 0.f);
    return poison ? __builtin_nanf("") : v + more;
  };
  if (a.kind == kNormNone) {
    for (int e = threadIdx.x; e < a.D; e += 256) {
      const float v = sum_at(e);
      if (a.res_out != nullptr) a.res_out[row * a.ro_sr + e] = v;
      static_cast<T*>(a.y)[row * a.y_sr + e] = from_f32<T>(v);
    }
    return;
  }
  float mean = 0.f;
  if (a.kind == kNormLayer) {
    float s = 0.f;
    for (int e = threadIdx.x; e < a.D; e += 256) s += sum_at(e);
    mean = block_sum(s) / (float)a.D;
  }
  float ss = 0.f;
  for (int e = threadIdx.x; e < a.D; e += 256) {
    const float d = sum_at(e) - mean;
    ss = __builtin_fmaf(d, d, ss);
  }
  const float rstd = 1.0f / sqrtf(block_sum(ss) / (float)a.D + a.eps);
  for (int e = threadIdx.x; e < a.D; e += 256) {
    const float v = sum_at(e);
    if (a.res_out != nullptr) a.res_out[row * a.ro_sr + e] = v;
    static_cast<T*>(a.y)[row * a.y_sr + e] = from_f32<T>((v - mean) * rstd * to_f32(w[e]));
  }
}

template <typename T, bool ADD> void launch_add_norm_rows(const AddNormArgs& a, bool vec, hipStream_t s) {
  if (!vec || a.D > 4096) {
    hipLaunchKernelGGL(add_norm_any_kernel<T>, dim3((unsigned)a.rows), dim3(256), 0, s, a);
    return;
  }
  const dim3 grid((unsigned)((a.rows + 3) / 4)), block(256);
  const int nv = (a.D + 511) / 512;
  if (nv <= 1)
    hipLaunchKernelGGL((add_norm_kernel<T, 1, ADD>), grid, block, 0, s, a);
  else if (nv <= 2)
    hipLaunchKernelGGL((add_norm_kernel<T, 2, ADD>), grid, block, 0, s, a);
  else if (nv <= 4)
    hipLaunchKernelGGL((add_norm_kernel<T, 4, ADD>), grid, block, 0, s, a);
  else
    hipLaunchKernelGGL((add_norm_kernel<T, 8, ADD>), grid, block, 0, s, a);
}

template <typename T> void launch_add_norm(const AddNormArgs& a, bool vec, hipStream_t s) {
  if (a.kind == kNormNone || a.add.post_w != nullptr || a.add.vec != nullptr || a.add.rows != nullptr)
    launch_add_norm_rows<T, true>(a, vec, s);
  else
    launch_add_norm_rows<T, false>(a, vec, s);
}

struct StreamConvArgs {
  const void* x;
  const void* w;     // (taps, D)
  const void* bias;  // (D) or null
  void* y;
  void* ring;  // (B, taps, D) or null
  const int32_t* pos;
  int pos_host;
  int L, D;
  long x_sb, x_sl, y_sb, y_sl, ring_sb;
  int silu, add_input;
};

constexpr int kStreamTile = 8;  // tokens per thread; at least taps - 1, so that only the first tile looks into the ring

template <typename T, int N> __device__ __forceinline__ void load_n(const T* p, float (&out)[N]) {
  if constexpr (N == 1)
    out[0] = to_f32(*p);
  else
    load_vec<T, N>(p, out);
}

// A thread owns N consecutive channels (16 bytes, or a single one) and walks kStreamTile tokens.
template <typename T, int K, int N>
__global__ __launch_bounds__(256) void stream_conv_kernel(const StreamConvArgs a) {
  static_assert(K - 1 <= kStreamTile, "the ring serves the first tile only");
  const int c0 = (blockIdx.x * 256 + threadIdx.x) * N;
  if (c0 >= a.D) return;
  const int b = blockIdx.z, l0 = blockIdx.y * kStreamTile;
  const int start = row_pos(a.pos, a.pos_host, b);
  const T* x = static_cast<const T*>(a.x) + b * a.x_sb + c0;
  T* y = static_cast<T*>(a.y) + b * a.y_sb + c0;
  const T* wp = static_cast<const T*>(a.w) + c0;
  T* ring = a.ring != nullptr ? static_cast<T*>(a.ring) + b * a.ring_sb + c0 : nullptr;
  float w[K][N], bias[N];
#pragma unroll
  for (int j = 0; j < K; ++j) load_n<T, N>(wp + (long)j * a.D, w[j]);
#pragma unroll
  for (int c = 0; c < N; ++c) bias[c] = 0.f;
  if (a.bias != nullptr) load_n<T, N>(static_cast<const T*>(a.bias) + c0, bias);

  const int ntok = a.L - l0 < kStreamTile ? a.L - l0 : kStreamTile;
  float in[kStreamTile][N];
#pragma unroll
  for (int t = 0; t < kStreamTile; ++t) load_n<T, N>(x + (long)(l0 + (t < ntok ? t : ntok - 1)) * a.x_sl, in[t]);
  float win[K][N];  // win[j]: the input taps - 1 - j before the current token
#pragma unroll
  for (int j = 0; j < K - 1; ++j) {
    const int l = l0 - (K - 1) + j;
#pragma unroll
    for (int c = 0; c < N; ++c) win[j][c] = 0.f;
    if (l >= 0)
      load_n<T, N>(x + (long)l * a.x_sl, win[j]);
    else if (ring != nullptr && start + l >= 0)
      load_n<T, N>(ring + (long)((start + l) % K) * a.D, win[j]);
  }
#pragma unroll
  for (int t = 0; t < kStreamTile; ++t) {
    if (t < ntok) {
      float out[N];
#pragma unroll
      for (int c = 0; c < N; ++c) {
        win[K - 1][c] = in[t][c];
        float acc = bias[c];
#pragma unroll
        for (int j = 0; j < K; ++j) acc = __builtin_fmaf(w[j][c], win[j][c], acc);
        if (a.silu) acc = silu_exact(acc);
        out[c] = a.add_input ? acc + in[t][c] : acc;
#pragma unroll
        for (int j = 0; j < K - 1; ++j) win[j][c] = win[j + 1][c];
      }
      if constexpr (N == 1)
        y[(long)(l0 + t) * a.y_sl] = from_f32<T>(out[0]);
      else
        store_vec<T, N>(y + (long)(l0 + t) * a.y_sl, out);
    }
  }
  // the last inputs of the portion go into the ring; the thread that has read the old ones writes them
  if (ring != nullptr && blockIdx.y == 0) {
#pragma unroll
    for (int j = 0; j < (K > 1 ? K - 1 : 1); ++j) {
      const int l = a.L - 1 - j;
      if (l >= 0) {
        float last[N];
        load_n<T, N>(x + (long)l * a.x_sl, last);
        T* slot = ring + (long)((start + l) % K) * a.D;
        if constexpr (N == 1)
          *slot = from_f32<T>(last[0]);
        else
          store_vec<T, N>(slot, last);
      }
    }
  }
}

template <typename T, int K> void launch_stream_conv_taps(const StreamConvArgs& a, int B, bool vec, hipStream_t s) {
  const int n = vec ? Pack<T>::kN : 1;
  const dim3 grid((unsigned)((a.D / n + 255) / 256), (unsigned)((a.L + kStreamTile - 1) / kStreamTile), (unsigned)B), block(256);
  if (vec)
    hipLaunchKernelGGL((stream_conv_kernel<T, K, Pack<T>::kN>), grid, block, 0, s, a);
  else
    hipLaunchKernelGGL((stream_conv_kernel<T, K, 1>), grid, block, 0, s, a);
}

template <typename T> void launch_stream_conv(const StreamConvArgs& a, int B, int taps, bool vec, hipStream_t s) {
  switch (taps) {
    case 1: launch_stream_conv_taps<T, 1>(a, B, vec, s); break;
    case 2: launch_stream_conv_taps<T, 2>(a, B, vec, s); break;
    case 3: launch_stream_conv_taps<T, 3>(a, B, vec, s); break;
    case 4: launch_stream_conv_taps<T, 4>(a, B, vec, s); break;
    case 5: launch_stream_conv_taps<T, 5>(a, B, vec, s); break;
    case 6: launch_stream_conv_taps<T, 6>(a, B, vec, s); break;
    case 7: launch_stream_conv_taps<T, 7>(a, B, vec, s); break;
    default: launch_stream_conv_taps<T, 8>(a, B, vec, s); break;
  }
}

}  // namespace based

extern "C" BASED_API int based_add_norm_addends(const void* x, const float* residual_in, const void* weight, void* y,
                                                float* residual_out, int64_t rows, int64_t D, int64_t x_sr, int64_t ri_sr,
                                                int64_t y_sr, int64_t ro_sr, float eps, int kind, float mult, const void* post_weight,
                                                float post_eps, const void* add_vec, const void* add_rows, const int64_t* add_index,
                                                int64_t add_sr, int64_t add_n, int io_dtype, void* stream) {
  using namespace based;
  BASED_REQUIRE(x && y && (weight || kind == kNormNone), BASED_ERR_ARG, "add_norm: null pointer argument");
  BASED_REQUIRE(rows >= 0 && D > 0 && rows < (1ll << 31) && D < (1ll << 30), BASED_ERR_ARG, "add_norm: bad sizes");
  BASED_REQUIRE(kind == kNormRms || kind == kNormLayer || kind == kNormNone, BASED_ERR_ARG, "add_norm: unknown norm %d", kind);
  BASED_REQUIRE(io_dtype == BASED_BF16 || io_dtype == BASED_F32, BASED_ERR_DTYPE, "add_norm: bad dtype");
  BASED_REQUIRE(residual_in == nullptr || residual_out != residual_in, BASED_ERR_ARG,
                "add_norm: residual_out must not be residual_in");
  BASED_REQUIRE(add_rows == nullptr || add_n > 0, BASED_ERR_ARG, "add_norm: the added rows need their number");
  BASED_REQUIRE(add_rows == nullptr || add_index != nullptr || add_n >= rows, BASED_ERR_ARG, "add_norm: too few rows to add");
  if (rows == 0) return BASED_OK;
  const bool vec = D % 8 == 0 && x_sr % 8 == 0 && y_sr % 8 == 0 && ri_sr % 4 == 0 && ro_sr % 4 == 0 && add_sr % 8 == 0 &&
                   aligned_to(x, 16) && aligned_to(weight, 16) && aligned_to(y, 16) && aligned_to(residual_in, 16) &&
                   aligned_to(residual_out, 16) && aligned_to(post_weight, 16) && aligned_to(add_vec, 16) && aligned_to(add_rows, 16);
  const AddNormArgs a{x,     residual_in, weight, y,   residual_out, (long)rows, (int)D, x_sr, ri_sr, y_sr, ro_sr, eps, mult, kind,
                      {post_weight, add_vec, add_rows, add_index, add_sr, add_n, post_eps}};
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (io_dtype == BASED_BF16)
    launch_add_norm<__bf16>(a, vec, s);
  else
    launch_add_norm<float>(a, vec, s);
  return check_launch("add_norm");
}

extern "C" BASED_API int based_add_norm(const void* x, const float* residual_in, const void* weight, void* y,
                                        float* residual_out, int64_t rows, int64_t D, int64_t x_sr, int64_t ri_sr,
                                        int64_t y_sr, int64_t ro_sr, float eps, int kind, float mult, int io_dtype,
                                        void* stream) {
  using namespace based;
  BASED_REQUIRE(kind == kNormRms || kind == kNormLayer, BASED_ERR_ARG, "add_norm: unknown norm %d", kind);
  return based_add_norm_addends(x, residual_in, weight, y, residual_out, rows, D, x_sr, ri_sr, y_sr, ro_sr, eps, kind, mult, nullptr,
                                0.f, nullptr, nullptr, nullptr, 0, 0, io_dtype, stream);
}

extern "C" BASED_API int based_stream_conv(const void* x, const void* weight, const void* bias, void* y, void* ring,
                                           const int32_t* pos, int64_t pos_host, int64_t B, int64_t L, int64_t D, int taps,
                                           int64_t x_sb, int64_t x_sl, int64_t y_sb, int64_t y_sl, int64_t ring_sb,
                                           int activation, int add_input, int io_dtype, void* stream) {
  using namespace based;
  BASED_REQUIRE(x && weight && y, BASED_ERR_ARG, "stream_conv: null pointer argument");
  BASED_REQUIRE(x != y, BASED_ERR_ARG, "stream_conv: the output must not be the input");
  BASED_REQUIRE(B >= 0 && L >= 0 && D > 0 && pos_host >= 0 && pos_host + L < (1ll << 31), BASED_ERR_ARG, "stream_conv: bad sizes");
  BASED_REQUIRE(taps >= 1 && taps <= 8, BASED_ERR_SHAPE, "stream_conv: %d taps (1 to 8)", taps);
  BASED_REQUIRE(activation == BASED_ACT_NONE || activation == BASED_ACT_SILU, BASED_ERR_ARG, "stream_conv: unknown activation");
  BASED_REQUIRE(io_dtype == BASED_BF16 || io_dtype == BASED_F32, BASED_ERR_DTYPE, "stream_conv: bad dtype");
  BASED_REQUIRE(B < 65536 && (L + kStreamTile - 1) / kStreamTile < 65536 && D < (1ll << 28), BASED_ERR_SHAPE,
                "stream_conv: grid too large");
  if (B == 0 || L == 0) return BASED_OK;
  const int n = io_dtype == BASED_BF16 ? 8 : 4;
  const bool vec = D % n == 0 && x_sb % n == 0 && x_sl % n == 0 && y_sb % n == 0 && y_sl % n == 0 && ring_sb % n == 0 &&
                   aligned_to(x, 16) && aligned_to(y, 16) && aligned_to(weight, 16) && aligned_to(bias, 16) && aligned_to(ring, 16);
  const StreamConvArgs a{x,    weight, bias, y,    ring, pos,     (int)pos_host, (int)L, (int)D,
                         x_sb, x_sl,   y_sb, y_sl, ring_sb, activation == BASED_ACT_SILU, add_input};
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (io_dtype == BASED_BF16)
    launch_stream_conv<__bf16>(a, (int)B, taps, vec, s);
  else
    launch_stream_conv<float>(a, (int)B, taps, vec, s);
  return check_launch("stream_conv");
}
