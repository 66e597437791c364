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
  a = exp_f(log_a);
  x = __builtin_amdgcn_sqrtf(one_minus_square(a, log_a)) * i * u;
}

// grid: x = segment of the sequence, y = 64-channel tile within its block (ceil(n / 64) per block), z = sequence
template <typename T>
__global__ __launch_bounds__(256) void rglru_gates_kernel(const RglruArgs a) {
  typedef GateMma<T> M;
  constexpr int KT = 128 / (int)sizeof(T);             // contraction staged at a time
  constexpr int PAD = 16 / (int)sizeof(T);
  constexpr int KS = KT + PAD;
  constexpr int SPAD = 4;
  // the operands, and after them the decays and inputs of the tile
  constexpr int kOperands = 3 * 64 * KS * (int)sizeof(T), kTile = 2 * 64 * (64 + SPAD) * 4;
  __shared__ __attribute__((aligned(16))) char s_mem[kOperands > kTile ? kOperands : kTile];
  T* s_u = reinterpret_cast<T*>(s_mem);
  T* s_r = s_u + 64 * KS;
  T* s_i = s_r + 64 * KS;
  float(*s_a)[64 + SPAD] = reinterpret_cast<float(*)[64 + SPAD]>(s_mem);  // [token][channel]
  float(*s_x)[64 + SPAD] = s_a + 64;
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
    typedef typename Pack<T>::type vec_t;
    constexpr int PIECES = 64 * (KT / V) / 256;
    if (vec) {
      vec_t xu[PIECES], xr[PIECES], xi[PIECES];
#pragma unroll
      for (int i = 0; i < PIECES; ++i) {
        const int p = i * 256 + tid, row = p / (KT / V), e = (p % (KT / V)) * V;
        const int tok = l0 + row < a.L ? l0 + row : a.L - 1, ch = c0 + row < a.n ? c0 + row : a.n - 1;
        const int k = k0 + e < a.n ? k0 + e : 0;
        xu[i] = *reinterpret_cast<const vec_t*>(u + tok * a.u_sl + k);
        xr[i] = *reinterpret_cast<const vec_t*>(ra + (long)ch * a.n + k);
        xi[i] = *reinterpret_cast<const vec_t*>(ri + (long)ch * a.n + k);
      }
#pragma unroll
      for (int i = 0; i < PIECES; ++i) {
        const int p = i * 256 + tid, row = p / (KT / V), e = (p % (KT / V)) * V;
        const bool in = k0 + e < a.n;
#pragma unroll
        for (int j = 0; j < V; ++j) {
          xu[i][j] = in ? xu[i][j] : (T)0.0f;
          xr[i][j] = in ? xr[i][j] : (T)0.0f;
          xi[i][j] = in ? xi[i][j] : (T)0.0f;
        }
        *reinterpret_cast<vec_t*>(&s_u[row * KS + e]) = xu[i];
        *reinterpret_cast<vec_t*>(&s_r[row * KS + e]) = xr[i];
        *reinterpret_cast<vec_t*>(&s_i[row * KS + e]) = xi[i];
      }
    } else {
      for (int p = tid; p < 64 * KT; p += 256) {
        const int row = p / KT, e = p % KT;
        const int tok = l0 + row < a.L ? l0 + row : a.L - 1, ch = c0 + row < a.n ? c0 + row : a.n - 1;
        const bool in = k0 + e < a.n;
        const int k = in ? k0 + e : 0;
        const T xu = u[tok * a.u_sl + k], xr = ra[(long)ch * a.n + k], xi = ri[(long)ch * a.n + k];
        s_u[row * KS + e] = in ? xu : (T)0.0f;
        s_r[row * KS + e] = in ? xr : (T)0.0f;
        s_i[row * KS + e] = in ? xi : (T)0.0f;
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
  __syncthreads();  // the operands are done with
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

// C consecutive channels as floats / from floats
template <typename T, int C> __device__ __forceinline__ void load_ch(const T* p, float (&out)[C]) {
  typedef __attribute__((ext_vector_type(C))) T vec_t;
  const vec_t x = *reinterpret_cast<const vec_t*>(p);
#pragma unroll
  for (int c = 0; c < C; ++c) out[c] = to_f32(x[c]);
}

// grid: x = tile of 256 C channels, y = segment, z = sequence; C channels per thread
template <typename T, int C>
__global__ __launch_bounds__(256) void rglru_scan_kernel(const RglruArgs a) {
  const int w = (blockIdx.x * 256 + threadIdx.x) * C;
  if (w >= a.W) return;
  const int seg = blockIdx.y, b = blockIdx.z, l0 = seg * kSeg;
  const float* g = a.agg + (long)b * (a.segs + 1) * 2 * a.W + w;
  float S[C];
#pragma unroll
  for (int c = 0; c < C; ++c) S[c] = 0.f;
  constexpr int U = 8;
  for (int i0 = 0; i0 <= seg; i0 += U) {
    float P[U][C], X[U][C];
#pragma unroll
    for (int i = 0; i < U; ++i) {
      const long at = (long)(i0 + i <= seg ? i0 + i : seg) * 2 * a.W;
      load_ch<float, C>(g + at, P[i]);
      load_ch<float, C>(g + at + a.W, X[i]);
    }
#pragma unroll
    for (int i = 0; i < U; ++i)
#pragma unroll
      for (int c = 0; c < C; ++c) S[c] = i0 + i <= seg ? __builtin_fmaf(P[i][c], S[c], X[i][c]) : S[c];
  }
  const int ntok = a.L - l0 < kSeg ? a.L - l0 : kSeg;
  const float* pa = a.ga + ((long)b * a.L + l0) * a.W + w;
  const float* px = a.gx + ((long)b * a.L + l0) * a.W + w;
  const T* py = static_cast<const T*>(a.y) + b * a.y_sb + l0 * a.y_sl + w;
  T* po = static_cast<T*>(a.out) + b * a.o_sb + l0 * a.o_sl + w;
  for (int t0 = 0; t0 < ntok; t0 += U) {
    float av[U][C], xv[U][C], yv[U][C];
#pragma unroll
    for (int i = 0; i < U; ++i) {
      const int t = t0 + i < ntok ? t0 + i : ntok - 1;
      load_ch<float, C>(pa + (long)t * a.W, av[i]);
      load_ch<float, C>(px + (long)t * a.W, xv[i]);
      load_ch<T, C>(py + t * a.y_sl, yv[i]);
    }
#pragma unroll
    for (int i = 0; i < U; ++i) {
      if (t0 + i < ntok) {
        typedef __attribute__((ext_vector_type(C))) T vec_t;
        vec_t o;
#pragma unroll
        for (int c = 0; c < C; ++c) {
          S[c] = __builtin_fmaf(av[i][c], S[c], xv[i][c]);
          o[c] = from_f32<T>(S[c] * gelu_tanh_f(yv[i][c]));
        }
        *reinterpret_cast<vec_t*>(po + (t0 + i) * a.o_sl) = o;
      }
    }
  }
  if (seg == a.segs - 1) {
#pragma unroll
    for (int c = 0; c < C; ++c) a.state[(long)b * a.W + w + c] = S[c];
  }
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

// a piece of a gate row: 16 bytes, or one element
template <typename T, bool VEC> struct LruPiece {
  typedef typename Pack<T>::type type;
  static __device__ __forceinline__ float get(type x, int i) { return to_f32(x[i]); }
};
template <typename T> struct LruPiece<T, false> {
  typedef T type;
  static __device__ __forceinline__ float get(type x, int) { return to_f32(x); }
};

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
  const int ch = tile * 32 + wave * 8 + (lane >> 3), part = lane & 7;
  const bool ok = ch < a.n;
  const int cc = ok ? ch : a.n - 1;
  // What does not depend on a position is asked for first: the first pieces of the gate rows, and what the
  // lane needs that finishes sequence m0 + part.
  const T* wr = static_cast<const T*>(a.ra) + ((long)blk * a.n + cc) * a.n;
  const T* wi = static_cast<const T*>(a.ri) + ((long)blk * a.n + cc) * a.n;
  typedef typename LruPiece<T, VEC>::type piece_t;
  piece_t pr[2], pi[2];
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int k = (part + 8 * i) * N;
    pr[i] = *reinterpret_cast<const piece_t*>(wr + (k < a.n ? k : 0));
    pi[i] = *reinterpret_cast<const piece_t*>(wi + (k < a.n ? k : 0));
  }
  const int bp = m0 + (part < rows ? part : 0), wc = blk * a.n + cc;
  const T rb = static_cast<const T*>(a.rb)[wc], ib = static_cast<const T*>(a.ib)[wc], lam = static_cast<const T*>(a.lam)[wc];
  const T yv = static_cast<const T*>(a.y)[bp * a.y_sb + wc];
  const float old = a.state[(long)bp * a.W + wc];
  const int pos_p = row_pos(a.pos, a.pos_host, bp);

  // the convolved inputs of the block: `share` threads per channel, each with every share-th sequence, four of
  // them in flight together
  const int share = a.n >= 256 ? 1 : 256 / a.n;
  for (int k = tid % (256 / share); k < a.n; k += 256 / share) {
    if (tid / (256 / share) >= share) break;
    const int chn = blk * a.n + k;
    const T* cw = static_cast<const T*>(a.conv_w) + chn;
    const float bias = a.conv_b != nullptr ? to_f32(static_cast<const T*>(a.conv_b)[chn]) : 0.f;
    for (int mb = tid / (256 / share); mb < rows; mb += 4 * share) {
      int pos[4];
      T now[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int m = mb + j * share < rows ? mb + j * share : rows - 1;
        pos[j] = row_pos(a.pos, a.pos_host, m0 + m);
        now[j] = static_cast<const T*>(a.x)[(m0 + m) * a.x_sb + chn];
      }
      float acc[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[j] = bias;
      for (int t0 = 0; t0 < a.taps - 1; t0 += 3) {
        T xv[4][3], cv[3];
#pragma unroll
        for (int t = 0; t < 3; ++t) {
          cv[t] = cw[(long)(t0 + t < a.taps - 1 ? t0 + t : 0) * a.W];
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            const int m = mb + j * share < rows ? mb + j * share : rows - 1;
            const int p = pos[j] - (a.taps - 1) + t0 + t;
            const bool in = t0 + t < a.taps - 1 && p >= 0;
            xv[j][t] = static_cast<const T*>(a.ring)[(m0 + m) * a.ring_sb + (long)(in ? p % a.taps : 0) * a.W + chn];
          }
        }
#pragma unroll
        for (int t = 0; t < 3; ++t)
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            const int p = pos[j] - (a.taps - 1) + t0 + t;
            const bool in = t0 + t < a.taps - 1 && p >= 0;
            acc[j] = in ? __builtin_fmaf(to_f32(cv[t]), to_f32(xv[j][t]), acc[j]) : acc[j];
          }
      }
      const float c_last = to_f32(cw[(long)(a.taps - 1) * a.W]);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int m = mb + j * share;
        if (m < rows) {
          s_u[m * ns + k] = round_to<T>(__builtin_fmaf(c_last, to_f32(now[j]), acc[j]));
          // a slot that no reader of this step looks at; one tile of the block writes it
          if (tile == 0 && pos[j] >= 0) static_cast<T*>(a.ring)[(m0 + m) * a.ring_sb + (long)(pos[j] % a.taps) * a.W + chn] = now[j];
        }
      }
    }
  }
  for (int i = tid; i < (kLruRows - rows) * ns; i += 256) s_u[rows * ns + i] = 0.f;
  __syncthreads();
  float zr[kLruRows], zi[kLruRows];
#pragma unroll
  for (int m = 0; m < kLruRows; ++m) zr[m] = zi[m] = 0.f;
  for (int k = part * N, it = 0; k < a.n; k += 8 * N, ++it) {
    const piece_t rp = it == 0 ? pr[0] : it == 1 ? pr[1] : *reinterpret_cast<const piece_t*>(wr + k);
    const piece_t ip = it == 0 ? pi[0] : it == 1 ? pi[1] : *reinterpret_cast<const piece_t*>(wi + k);
    float r[N], q[N];
#pragma unroll
    for (int j = 0; j < N; ++j) {
      r[j] = LruPiece<T, VEC>::get(rp, j);
      q[j] = LruPiece<T, VEC>::get(ip, j);
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
    float av, x;
    lru_gates(my_r + to_f32(rb), my_i + to_f32(ib), softplus_f(to_f32(lam)), s_u[part * ns + ch], a.c, av, x);
    const float S = pos_p > 0 ? __builtin_fmaf(av, old, x) : x;
    a.state[(long)bp * a.W + wc] = S;
    static_cast<T*>(a.out)[bp * a.o_sb + wc] = from_f32<T>(S * gelu_tanh_f(to_f32(yv)));
  }
}

template <typename T> void launch_rglru_prefill(const RglruArgs& a, int tiles, bool pairs, hipStream_t s) {
  const int per = pairs ? 512 : 256;
  const dim3 g1((unsigned)a.segs, (unsigned)tiles, (unsigned)a.B);
  const dim3 g2((unsigned)((a.W + per - 1) / per), (unsigned)a.segs, (unsigned)a.B), block(256);
  hipLaunchKernelGGL(rglru_gates_kernel<T>, g1, block, 0, s, a);
  if (pairs)
    hipLaunchKernelGGL((rglru_scan_kernel<T, 2>), g2, block, 0, s, a);
  else
    hipLaunchKernelGGL((rglru_scan_kernel<T, 1>), g2, block, 0, s, a);
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
  const bool pairs = W % 2 == 0 && y_sb % 2 == 0 && y_sl % 2 == 0 && o_sb % 2 == 0 && o_sl % 2 == 0 && aligned_to(y, 8) &&
                     aligned_to(out, 8) && aligned_to(work_a, 8) && aligned_to(work_x, 8) && aligned_to(work_agg, 8);
  if (io_dtype == BASED_BF16)
    launch_rglru_prefill<__bf16>(a, (int)tiles, pairs, s);
  else
    launch_rglru_prefill<float>(a, (int)tiles, pairs, s);
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
