// Real-gated linear recurrent unit for gfx950 (Griffin: Mixing Gated Linear Recurrences with Local
// Attention for Efficient Language Models).  Per channel, in fp32:
//   r = sigmoid(ra u + rb),  i = sigmoid(ri u + ib)      ra, ri block-diagonal: n x n per block
//   log a = -c r softplus(lam),   S_t = a S_{t-1} + sqrt(1 - a^2) i u,   out = S * gelu_tanh(y)
//
//   rglru_gates  both gate products of 64 tokens x 64 channels on MFMA (bf16, or fp32 MFMA for fp32
//                tensors), with the decay a and the input x = sqrt(1 - a^2) i u formed behind them, in
//                fp32; and, for its 64 tokens, what the recurrence does to any state that enters
//                them: S -> P S + X.
//   rglru_scan   64 tokens per thread and channel: the state that enters them from the (P, X) of the
//                segments before, then the recurrence and the output gate.
//   rglru_step   one token per sequence: the short convolution on its ring of past inputs, the gates,
//                the state update and the output gate.
#include "stream_common.hpp"

namespace based {

constexpr int kSeg = 64;  // tokens per segment

struct RglruArgs {
  const void* u;  // (B, L, W), strides
  const void* y;
  const void* ra;  // (blocks, n, n) [out, in]
  const void* rb;
  const void* ri;
  const void* ib;
  const void* lam;
  float* ga;   // (B, L, W) decay
  float* gx;   // (B, L, W) input
  float* agg;  // (B, segments + 1, 2, W): P and X; entry 0 is the state that enters the call
  float* state;  // (B, W)
  void* out;
  int B, L, W, n, segs;
  long u_sb, u_sl, y_sb, y_sl, o_sb, o_sl;
  float c;
  int fresh;
};

template <typename T> struct GateMma;
template <> struct GateMma<__bf16> {
  static constexpr int kK = 32;  // contraction per instruction
  typedef bf16x8 frag_t;
  static constexpr int kPer = 8;
  static __device__ __forceinline__ f32x4 run(frag_t a, frag_t b, f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
  }
};
template <> struct GateMma<float> {
  static constexpr int kK = 4;
  typedef float frag_t;
  static constexpr int kPer = 1;
  static __device__ __forceinline__ f32x4 run(frag_t a, frag_t b, f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
  }
};

__device__ __forceinline__ void lru_gates(float zr, float zi, float sp, float u, float c, float& a, float& x) {
  const float r = sigmoid_f(zr), i = sigmoid_f(zi);
  const float log_a = -c * r * sp;
  a = expf(log_a);
  x = sqrtf(-expm1f(2.0f * log_a)) * i * u;
}

// grid: x = segment of the sequence, y = 64-channel tile within its block (ceil(n / 64) per block), z = sequence
template <typename T>
__global__ __launch_bounds__(256) void rglru_gates_kernel(const RglruArgs a) {
  typedef GateMma<T> M;
  constexpr int KT = 32;                               // contraction staged at a time
  constexpr int PAD = 16 / (int)sizeof(T);
  constexpr int KS = KT + PAD;
  constexpr int SPAD = 4;
  __shared__ __attribute__((aligned(16))) T s_u[64 * KS], s_r[64 * KS], s_i[64 * KS];
  __shared__ float s_a[64][64 + SPAD], s_x[64][64 + SPAD];  // [token][channel]
  __shared__ float s_const[3][64];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, quad = lane >> 4;
  const int tiles = (a.n + 63) / 64;
  const int blk = blockIdx.y / tiles, c0 = (blockIdx.y % tiles) * 64;  // first output channel within the block
  const int b = blockIdx.z, seg = blockIdx.x, l0 = seg * kSeg;
  const T* u = static_cast<const T*>(a.u) + b * a.u_sb + (long)blk * a.n;
  const T* ra = static_cast<const T*>(a.ra) + (long)blk * a.n * a.n;
  const T* ri = static_cast<const T*>(a.ri) + (long)blk * a.n * a.n;
  if (tid < 64) {
    const int ch = c0 + tid < a.n ? c0 + tid : a.n - 1, w = blk * a.n + ch;
    s_const[0][tid] = to_f32(static_cast<const T*>(a.rb)[w]);
    s_const[1][tid] = to_f32(static_cast<const T*>(a.ib)[w]);
    s_const[2][tid] = softplus_f(to_f32(static_cast<const T*>(a.lam)[w]));
  }
  f32x4 zr[4], zi[4];  // wavefront: 16 tokens (columns) x 64 channels (rows)
#pragma unroll
  for (int i = 0; i < 4; ++i) zr[i] = zi[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  constexpr int V = Pack<T>::kN;
  const bool vec = a.n % V == 0 && a.u_sb % V == 0 && a.u_sl % V == 0 && ((uintptr_t)a.u & 15) == 0 && ((uintptr_t)a.ra & 15) == 0 &&
                   ((uintptr_t)a.ri & 15) == 0;
  for (int k0 = 0; k0 < a.n; k0 += KT) {
    __syncthreads();
    for (int p = tid; p < 64 * (KT / V); p += 256) {
      const int row = p / (KT / V), e = (p % (KT / V)) * V;
      const int tok = l0 + row < a.L ? l0 + row : a.L - 1;
      const int ch = c0 + row < a.n ? c0 + row : a.n - 1;
      typedef typename Pack<T>::type vec_t;
      if (vec) {
        const bool in = k0 + e < a.n;
        const int k = in ? k0 + e : 0;
        vec_t xu = *reinterpret_cast<const vec_t*>(u + tok * a.u_sl + k);
        vec_t xr = *reinterpret_cast<const vec_t*>(ra + (long)ch * a.n + k);
        vec_t xi = *reinterpret_cast<const vec_t*>(ri + (long)ch * a.n + k);
        if (!in) {
#pragma unroll
          for (int j = 0; j < V; ++j) xu[j] = xr[j] = xi[j] = (T)0.0f;
        }
        *reinterpret_cast<vec_t*>(&s_u[row * KS + e]) = xu;
        *reinterpret_cast<vec_t*>(&s_r[row * KS + e]) = xr;
        *reinterpret_cast<vec_t*>(&s_i[row * KS + e]) = xi;
      } else {
#pragma unroll
        for (int j = 0; j < V; ++j) {
          const bool in = k0 + e + j < a.n;
          const int k = in ? k0 + e + j : 0;
          const T xu = u[tok * a.u_sl + k], xr = ra[(long)ch * a.n + k], xi = ri[(long)ch * a.n + k];
          s_u[row * KS + e + j] = in ? xu : (T)0.0f;
          s_r[row * KS + e + j] = in ? xr : (T)0.0f;
          s_i[row * KS + e + j] = in ? xi : (T)0.0f;
        }
      }
    }
    __syncthreads();
#pragma unroll
    for (int kk = 0; kk < KT; kk += M::kK) {
      const int e = kk + quad * M::kPer;
      const typename M::frag_t fu = *reinterpret_cast<const typename M::frag_t*>(&s_u[(wave * 16 + l16) * KS + e]);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        zr[i] = M::run(*reinterpret_cast<const typename M::frag_t*>(&s_r[(i * 16 + l16) * KS + e]), fu, zr[i]);
        zi[i] = M::run(*reinterpret_cast<const typename M::frag_t*>(&s_i[(i * 16 + l16) * KS + e]), fu, zi[i]);
      }
    }
  }
  // lane: token wave*16 + l16, channels i*16 + quad*4 ..
  const int tl = wave * 16 + l16, tok = l0 + tl;
  const bool tok_in = tok < a.L;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int ch = i * 16 + quad * 4;
    f32x4 ov, xv;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int cc = c0 + ch + j < a.n ? c0 + ch + j : a.n - 1;
      const float uv = to_f32(u[(tok_in ? tok : a.L - 1) * a.u_sl + cc]);
      float av, x;
      lru_gates(zr[i][j] + s_const[0][ch + j], zi[i][j] + s_const[1][ch + j], s_const[2][ch + j], uv, a.c, av, x);
      ov[j] = av, xv[j] = x;
    }
    *reinterpret_cast<f32x4*>(&s_a[tl][ch]) = ov;
    *reinterpret_cast<f32x4*>(&s_x[tl][ch]) = xv;
  }
  __syncthreads();
  // the tile in rows of 64 channels, and the segment's effect on a state that enters it
  const int ntok = a.L - l0 < kSeg ? a.L - l0 : kSeg;
  const int nch = a.n - c0 < 64 ? a.n - c0 : 64;
  const long base = ((long)b * a.L + l0) * a.W + (long)blk * a.n + c0;
  for (int p = tid; p < ntok * 64; p += 256) {
    const int t = p >> 6, ch = p & 63;
    if (ch < nch) {
      a.ga[base + (long)t * a.W + ch] = s_a[t][ch];
      a.gx[base + (long)t * a.W + ch] = s_x[t][ch];
    }
  }
  if (tid < nch) {
    float P = 1.f, X = 0.f;
    for (int t = 0; t < ntok; ++t) {
      const float av = s_a[t][tid];
      P *= av;
      X = __builtin_fmaf(av, X, s_x[t][tid]);
    }
    const int w = blk * a.n + c0 + tid;
    float* g = a.agg + ((long)b * (a.segs + 1) + seg + 1) * 2 * a.W + w;
    g[0] = P;
    g[a.W] = X;
    if (seg == 0) {
      float* g0 = a.agg + (long)b * (a.segs + 1) * 2 * a.W + w;
      g0[0] = 0.f;
      g0[a.W] = a.fresh ? 0.f : a.state[(long)b * a.W + w];
    }
  }
}

// grid: x = 256-channel tile, y = segment, z = sequence
template <typename T>
__global__ __launch_bounds__(256) void rglru_scan_kernel(const RglruArgs a) {
  const int w = blockIdx.x * 256 + threadIdx.x;
  if (w >= a.W) return;
  const int seg = blockIdx.y, b = blockIdx.z, l0 = seg * kSeg;
  const float* g = a.agg + (long)b * (a.segs + 1) * 2 * a.W + w;
  float S = 0.f;
#pragma unroll 8
  for (int i = 0; i <= seg; ++i) S = __builtin_fmaf(g[(long)i * 2 * a.W], S, g[(long)i * 2 * a.W + a.W]);
  const int ntok = a.L - l0 < kSeg ? a.L - l0 : kSeg;
  const float* pa = a.ga + ((long)b * a.L + l0) * a.W + w;
  const float* px = a.gx + ((long)b * a.L + l0) * a.W + w;
  const T* py = static_cast<const T*>(a.y) + b * a.y_sb + l0 * a.y_sl + w;
  T* po = static_cast<T*>(a.out) + b * a.o_sb + l0 * a.o_sl + w;
  constexpr int U = 8;
  int t = 0;
  for (; t + U <= ntok; t += U) {
    float av[U], xv[U], yv[U];
#pragma unroll
    for (int i = 0; i < U; ++i) {
      av[i] = pa[(long)(t + i) * a.W];
      xv[i] = px[(long)(t + i) * a.W];
      yv[i] = to_f32(py[(t + i) * a.y_sl]);
    }
#pragma unroll
    for (int i = 0; i < U; ++i) {
      S = __builtin_fmaf(av[i], S, xv[i]);
      po[(t + i) * a.o_sl] = from_f32<T>(S * gelu_tanh_f(yv[i]));
    }
  }
  for (; t < ntok; ++t) {
    S = __builtin_fmaf(pa[(long)t * a.W], S, px[(long)t * a.W]);
    po[t * a.o_sl] = from_f32<T>(S * gelu_tanh_f(to_f32(py[t * a.y_sl])));
  }
  if (seg == a.segs - 1) a.state[(long)b * a.W + w] = S;
}

// ---- one token per sequence ----
struct RglruStepArgs {
  const void* x;  // (B, W): input of the short convolution
  const void* y;
  const void* conv_w;  // (taps, W)
  const void* conv_b;
  void* ring;  // (B, taps, W)
  const void* ra;
  const void* rb;
  const void* ri;
  const void* ib;
  const void* lam;
  float* state;
  void* out;
  const int32_t* pos;
  int pos_host;
  int B, W, n, taps;
  long x_sb, y_sb, o_sb, ring_sb;
  float c;
};

constexpr int kLruRows = 8;  // sequences held at a time

// A workgroup takes 32 output channels of one block (a wavefront 8 of them, 8 lanes per channel) and
// up to kLruRows sequences; the convolved inputs of the whole block go through LDS.
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void rglru_step_kernel(const RglruStepArgs a) {
  constexpr int N = VEC ? Pack<T>::kN : 1;
  extern __shared__ __attribute__((aligned(16))) float s_u[];  // [kLruRows][n rounded up to 4]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int tiles = (a.n + 31) / 32;
  const int blk = blockIdx.x / tiles, tile = blockIdx.x % tiles, m0 = blockIdx.y * kLruRows;
  const int rows = a.B - m0 < kLruRows ? a.B - m0 : kLruRows;
  const int ns = (a.n + 3) & ~3;  // rows of whole 16-byte pieces
  for (int i = tid; i < kLruRows * a.n; i += 256) {
    const int m = i / a.n, k = i % a.n, ch = blk * a.n + k;
    float val = 0.f;
    if (m < rows) {
      const int b = m0 + m, pos = row_pos(a.pos, a.pos_host, b);
      const T now = static_cast<const T*>(a.x)[b * a.x_sb + ch];
      const T* cw = static_cast<const T*>(a.conv_w) + ch;
      T* ring = static_cast<T*>(a.ring) + b * a.ring_sb + ch;
      float acc = a.conv_b != nullptr ? to_f32(static_cast<const T*>(a.conv_b)[ch]) : 0.f;
      for (int j = 0; j < a.taps - 1; ++j) {
        const int p = pos - (a.taps - 1) + j;
        if (p >= 0) acc = __builtin_fmaf(to_f32(cw[(long)j * a.W]), to_f32(ring[(long)(p % a.taps) * a.W]), acc);
      }
      acc = __builtin_fmaf(to_f32(cw[(long)(a.taps - 1) * a.W]), to_f32(now), acc);
      val = round_to<T>(acc);
      // a slot that no reader of this step looks at; one tile of the block writes it
      if (tile == 0 && pos >= 0) ring[(long)(pos % a.taps) * a.W] = now;
    }
    s_u[m * ns + k] = val;
  }
  __syncthreads();
  const int ch = tile * 32 + wave * 8 + (lane >> 3), part = lane & 7;
  const bool ok = ch < a.n;
  const int cc = ok ? ch : a.n - 1;
  const T* wr = static_cast<const T*>(a.ra) + ((long)blk * a.n + cc) * a.n;
  const T* wi = static_cast<const T*>(a.ri) + ((long)blk * a.n + cc) * a.n;
  float zr[kLruRows], zi[kLruRows];
#pragma unroll
  for (int m = 0; m < kLruRows; ++m) zr[m] = zi[m] = 0.f;
#pragma unroll 2
  for (int k = part * N; k < a.n; k += 8 * N) {
    float r[N], q[N];
    if constexpr (VEC) {
      load_vec<T, N>(wr + k, r);
      load_vec<T, N>(wi + k, q);
    } else {
      r[0] = to_f32(wr[k]), q[0] = to_f32(wi[k]);
    }
#pragma unroll
    for (int m = 0; m < kLruRows; ++m) {
      float uv[N];
      if constexpr (VEC)
        load_vec<float, N>(&s_u[m * ns + k], uv);
      else
        uv[0] = s_u[m * ns + k];
#pragma unroll
      for (int j = 0; j < N; ++j) {
        zr[m] = __builtin_fmaf(r[j], uv[j], zr[m]);
        zi[m] = __builtin_fmaf(q[j], uv[j], zi[m]);
      }
    }
  }
  float my_r = 0.f, my_i = 0.f;
#pragma unroll
  for (int m = 0; m < kLruRows; ++m) {
    const float sr = sum8(zr[m]), si = sum8(zi[m]);
    my_r = part == m ? sr : my_r;
    my_i = part == m ? si : my_i;
  }
  // lane `part` finishes sequence m0 + part
  if (ok && part < rows) {
    const int b = m0 + part, w = blk * a.n + ch;
    const int pos = row_pos(a.pos, a.pos_host, b);
    float av, x;
    lru_gates(my_r + to_f32(static_cast<const T*>(a.rb)[w]), my_i + to_f32(static_cast<const T*>(a.ib)[w]),
              softplus_f(to_f32(static_cast<const T*>(a.lam)[w])), s_u[part * ns + ch], a.c, av, x);
    float* sp = a.state + (long)b * a.W + w;
    const float old = *sp;
    const float S = pos > 0 ? __builtin_fmaf(av, old, x) : x;
    *sp = S;
    static_cast<T*>(a.out)[b * a.o_sb + w] = from_f32<T>(S * gelu_tanh_f(to_f32(static_cast<const T*>(a.y)[b * a.y_sb + w])));
  }
}

}  // namespace based

extern "C" BASED_API int based_rglru_prefill(const void* u, const void* y, const void* ra, const void* rb, const void* ri, const void* ib,
                                             const void* lam, float* work_a, float* work_x, float* work_agg, float* state, void* out,
                                             int64_t B, int64_t L, int64_t W, int64_t blocks, int64_t u_sb, int64_t u_sl, int64_t y_sb,
                                             int64_t y_sl, int64_t o_sb, int64_t o_sl, float c, int fresh, int io_dtype, void* stream) {
  using namespace based;
  BASED_REQUIRE(u && y && ra && rb && ri && ib && lam && work_a && work_x && work_agg && state && out, BASED_ERR_ARG,
                "rglru_prefill: null pointer argument");
  BASED_REQUIRE(B >= 0 && L >= 0 && W > 0 && blocks > 0, BASED_ERR_ARG, "rglru_prefill: bad sizes");
  BASED_REQUIRE(W % blocks == 0, BASED_ERR_SHAPE, "rglru_prefill: %ld channels do not divide into %ld blocks", (long)W, (long)blocks);
  BASED_REQUIRE(io_dtype == BASED_BF16 || io_dtype == BASED_F32, BASED_ERR_DTYPE, "rglru_prefill: bad dtype");
  const int64_t n = W / blocks, segs = (L + kSeg - 1) / kSeg, tiles = blocks * ((n + 63) / 64);
  BASED_REQUIRE(B < 65536 && segs < 65536 && tiles < 65536 && L < (1ll << 31), BASED_ERR_SHAPE, "rglru_prefill: grid too large");
  if (B == 0 || L == 0) return BASED_OK;
  const RglruArgs a{u,      y,      ra,     rb,     ri,        ib,   lam,  work_a, work_x, work_agg, state, out, (int)B,
                    (int)L, (int)W, (int)n, (int)segs, u_sb, u_sl, y_sb,   y_sl,   o_sb,     o_sl,  c,   fresh};
  hipStream_t s = static_cast<hipStream_t>(stream);
  const dim3 g1((unsigned)segs, (unsigned)tiles, (unsigned)B), g2((unsigned)((W + 255) / 256), (unsigned)segs, (unsigned)B), block(256);
  if (io_dtype == BASED_BF16) {
    hipLaunchKernelGGL(rglru_gates_kernel<__bf16>, g1, block, 0, s, a);
    hipLaunchKernelGGL(rglru_scan_kernel<__bf16>, g2, block, 0, s, a);
  } else {
    hipLaunchKernelGGL(rglru_gates_kernel<float>, g1, block, 0, s, a);
    hipLaunchKernelGGL(rglru_scan_kernel<float>, g2, block, 0, s, a);
  }
  return check_launch("rglru_prefill");
}

extern "C" BASED_API int based_rglru_step(const void* x, const void* y, const void* conv_w, const void* conv_b, void* ring, const void* ra,
                                          const void* rb, const void* ri, const void* ib, const void* lam, float* state, void* out,
                                          const int32_t* pos, int64_t pos_host, int64_t B, int64_t W, int64_t blocks, int taps,
                                          int64_t x_sb, int64_t y_sb, int64_t o_sb, int64_t ring_sb, float c, int io_dtype,
                                          void* stream) {
  using namespace based;
  BASED_REQUIRE(x && y && conv_w && ring && ra && rb && ri && ib && lam && state && out, BASED_ERR_ARG, "rglru_step: null pointer argument");
  BASED_REQUIRE(B >= 0 && W > 0 && blocks > 0 && pos_host >= 0, BASED_ERR_ARG, "rglru_step: bad sizes");
  BASED_REQUIRE(W % blocks == 0, BASED_ERR_SHAPE, "rglru_step: %ld channels do not divide into %ld blocks", (long)W, (long)blocks);
  BASED_REQUIRE(taps >= 1 && taps <= 8, BASED_ERR_SHAPE, "rglru_step: %d taps (1 to 8)", taps);
  BASED_REQUIRE(io_dtype == BASED_BF16 || io_dtype == BASED_F32, BASED_ERR_DTYPE, "rglru_step: bad dtype");
  const int64_t n = W / blocks, tiles = blocks * ((n + 31) / 32), mt = (B + kLruRows - 1) / kLruRows;
  BASED_REQUIRE(n <= 2048, BASED_ERR_SHAPE, "rglru_step: blocks of %ld channels (at most 2048)", (long)n);
  BASED_REQUIRE(tiles < (1ll << 31) && mt < 65536, BASED_ERR_SHAPE, "rglru_step: grid too large");
  if (B == 0) return BASED_OK;
  const RglruStepArgs a{x,  y,  conv_w, conv_b, ring, ra, rb, ri, ib, lam, state, out, pos, (int)pos_host, (int)B, (int)W, (int)n, taps, x_sb,
                        y_sb, o_sb, ring_sb, c};
  const int v = io_dtype == BASED_BF16 ? 8 : 4;
  const bool vec = n % v == 0 && aligned_to(ra, 16) && aligned_to(ri, 16);
  const dim3 grid((unsigned)tiles, (unsigned)mt), block(256);
  const size_t bytes = (size_t)kLruRows * ((n + 3) & ~3) * sizeof(float);
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (io_dtype == BASED_BF16) {
    if (vec)
      hipLaunchKernelGGL((rglru_step_kernel<__bf16, true>), grid, block, bytes, s, a);
    else
      hipLaunchKernelGGL((rglru_step_kernel<__bf16, false>), grid, block, bytes, s, a);
  } else {
    if (vec)
      hipLaunchKernelGGL((rglru_step_kernel<float, true>), grid, block, bytes, s, a);
    else
      hipLaunchKernelGGL((rglru_step_kernel<float, false>), grid, block, bytes, s, a);
  }
  return check_launch("rglru_step");
}
