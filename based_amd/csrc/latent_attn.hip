// Attention over a cache of latents, for gfx950.  A token's cache row is its normalised latent (R channels)
// and one rotated key part (rot channels) that all heads share; head h's key is [rotated part | uk_h c] and its
// value uv_h c.  Prompts expand the rows they see to keys and values (a matrix product) and attend those.
// A single token stays in the latent space: with q~ = uk^T q a score is q~ . c + q_rot . k_rot, the weighted
// sum of the latents is formed once per head, and uv_h is applied to that sum.
//
//   latent_write   norm and rotation of a portion's rows, into the cache
//   latent_query   one token per sequence: q~ and the rotated q of every head, and the token's cache row
//   latent_step    scores, softmax and weighted latents, the keys of a sequence dealt to several workgroups
//   latent_values  their partial results put together, times uv
// The first and the last have a form on MFMA for 16 sequences at a time.
#include "stream_common.hpp"

namespace based {

struct LatentArgs {
  const void* x;      // (B, L, R + rot): latent, rotated part
  const void* norm_w; // (R)
  void* cache;        // (B, S, R + rot)
  const float* cos_t; // (n_pos, rot / 2)
  const float* sin_t;
  const int32_t* pos;
  int pos_host, n_pos;
  int B, L, S, R, rot, half_split;
  long x_sb, x_sl, c_sb, c_st;
  float eps;
  // single tokens
  const void* q;      // (B, H * (rot + d)), a head's rotated channels first
  const void* w;      // (H * (rot + d + dv), R + rot): of each head rot rows, then uk (d rows), then uv (dv rows)
  float* qa;          // (B, H, R + rot)
  float* part;        // (B, splits, H, R)
  float* part_ml;     // (B, splits, H, 2): running maximum, running sum
  void* o;            // (B, H * dv)
  int H, d, dv, splits, window;
  long q_sb, w_sr, o_sb;
  float scale, out_scale;
};

// channel c of a rotated part, with its partner
template <typename T>
__device__ __forceinline__ float turned(const T* x, int c, int pos, const LatentArgs& a) {
  const int half = a.rot / 2;
  int pair, partner;
  float sgn;
  if (a.half_split) {
    pair = c < half ? c : c - half;
    partner = c < half ? c + half : c - half;
    sgn = c < half ? -1.f : 1.f;
  } else {
    pair = c >> 1;
    partner = c ^ 1;
    sgn = (c & 1) ? 1.f : -1.f;
  }
  const long t = (long)pos * half + pair;
  return to_f32(x[c]) * a.cos_t[t] + sgn * to_f32(x[partner]) * a.sin_t[t];
}

// One wavefront writes one row.
template <typename T>
__device__ __forceinline__ void write_row(const LatentArgs& a, const T* x, T* out, int pos, int lane) {
  float ss = 0.f;
  for (int c = lane; c < a.R; c += 64) ss = __builtin_fmaf(to_f32(x[c]), to_f32(x[c]), ss);
  const float r = 1.0f / sqrtf(wave_sum(ss) / (float)a.R + a.eps);
  for (int c = lane; c < a.R; c += 64) out[c] = from_f32<T>(to_f32(x[c]) * r * to_f32(static_cast<const T*>(a.norm_w)[c]));
  for (int c = lane; c < a.rot; c += 64) out[a.R + c] = from_f32<T>(turned(x + a.R, c, pos, a));
}

template <typename T>
__global__ __launch_bounds__(256) void latent_write_kernel(const LatentArgs a) {
  const long item = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= (long)a.B * a.L) return;
  const int b = (int)(item / a.L), l = (int)(item % a.L), pos = a.pos_host + l;
  write_row<T>(a, static_cast<const T*>(a.x) + b * a.x_sb + l * a.x_sl, static_cast<T*>(a.cache) + b * a.c_sb + pos * a.c_st, pos,
               threadIdx.x & 63);
}

// Rows of whole 16-byte pieces, LPR (16, 32 or 64) lanes each; bf16.
template <int LPR>
__global__ __launch_bounds__(256) void latent_write_vec_kernel(const LatentArgs a) {
  constexpr int KEEP = 2;
  const long item0 = (long)blockIdx.x * (256 / LPR) + threadIdx.x / LPR;
  const bool live = item0 < (long)a.B * a.L;
  const long item = live ? item0 : 0;
  const int lane = threadIdx.x % LPR;
  const int b = (int)(item / a.L), l = (int)(item % a.L), pos = a.pos_host + l;
  const __bf16* x = static_cast<const __bf16*>(a.x) + b * a.x_sb + l * a.x_sl;
  __bf16* out = static_cast<__bf16*>(a.cache) + b * a.c_sb + pos * a.c_st;
  float v[KEEP][8], w[KEEP][8];
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int e = (i * LPR + lane) * 8;
    load_vec<__bf16, 8>(x + (e < a.R ? e : 0), v[i]);
    load_vec<__bf16, 8>(static_cast<const __bf16*>(a.norm_w) + (e < a.R ? e : 0), w[i]);
  }
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < KEEP; ++i)
#pragma unroll
    for (int j = 0; j < 8; ++j) ss = (i * LPR + lane) * 8 < a.R ? __builtin_fmaf(v[i][j], v[i][j], ss) : ss;
  ss = sum16(ss);
  if (LPR >= 32) ss += __shfl_xor(ss, 16, 64);
  if (LPR >= 64) ss += __shfl_xor(ss, 32, 64);
  const float r = 1.0f / sqrtf(ss / (float)a.R + a.eps);
  if (!live) return;
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int e = (i * LPR + lane) * 8;
#pragma unroll
    for (int j = 0; j < 8; ++j) v[i][j] *= r * w[i][j];
    if (e < a.R) store_vec<__bf16, 8>(out + e, v[i]);
  }
  for (int c = lane; c < a.rot; c += LPR) out[a.R + c] = (__bf16)turned(x + a.R, c, pos, a);
}

// ---- one token per sequence ----
constexpr int kQueryCols = 128;  // latent channels per workgroup of latent_query
constexpr int kQueryRows = 4;    // sequences at a time

// The cache row and the rotated queries of sequence b, by one workgroup.
template <typename T> __device__ __forceinline__ void query_row(const LatentArgs& a, int b) {
  const int tid = threadIdx.x, W = a.R + a.rot;
  if (b >= a.B) return;
  const int pos = row_pos(a.pos, a.pos_host, b);
  if (pos < 0 || pos >= a.S || (a.rot > 0 && pos >= a.n_pos)) return;
  if (tid < 64) {
    write_row<T>(a, static_cast<const T*>(a.x) + b * a.x_sb, static_cast<T*>(a.cache) + b * a.c_sb + pos * a.c_st, pos, tid);
  } else {
    for (int i = tid - 64; i < a.H * a.rot; i += 192) {
      const int h = i / a.rot, c = i % a.rot;
      const T* q = static_cast<const T*>(a.q) + b * a.q_sb + (long)h * (a.rot + a.d);
      a.qa[((long)b * a.H + h) * W + a.R + c] = round_to<T>(turned(q, c, pos, a));
    }
  }
}

// N: elements per load (8 or 1); kQueryRows sequences per workgroup.  In x, workgroups 0 .. H * ceil(R / kQueryCols) - 1 form q~, the
// rest (one per sequence) write the cache row and rotate the queries.
template <typename T, int N>
__global__ __launch_bounds__(256) void latent_query_kernel(const LatentArgs a) {
  constexpr int LANES = kQueryCols / N, GROUPS = 256 / LANES > 0 ? 256 / LANES : 1;
  __shared__ float qs[kQueryRows][256];
  __shared__ float part[GROUPS][kQueryRows][kQueryCols];
  const int tid = threadIdx.x, W = a.R + a.rot, col_blocks = (a.R + kQueryCols - 1) / kQueryCols;
  if ((int)blockIdx.x >= a.H * col_blocks) {
    query_row<T>(a, blockIdx.y * kQueryRows + blockIdx.x - a.H * col_blocks);
    return;
  }
  const int h = blockIdx.x / col_blocks, r0 = (blockIdx.x % col_blocks) * kQueryCols;
  const int b0 = blockIdx.y * kQueryRows;
  const int piece = tid % LANES, grp = tid / LANES, col = r0 + piece * N;
  const T* w = static_cast<const T*>(a.w) + ((long)h * (a.rot + a.d + a.dv) + a.rot) * a.w_sr;
  {
    const int rows = a.B - b0 < kQueryRows ? a.B - b0 : kQueryRows;
    float acc[kQueryRows][N];
#pragma unroll
    for (int m = 0; m < kQueryRows; ++m)
#pragma unroll
      for (int j = 0; j < N; ++j) acc[m][j] = 0.f;
    for (int d0 = 0; d0 < a.d; d0 += 256) {
      const int nd = a.d - d0 < 256 ? a.d - d0 : 256;
      __syncthreads();
      for (int i = tid; i < rows * nd; i += 256)
        qs[i / nd][i % nd] = to_f32(static_cast<const T*>(a.q)[(long)(b0 + i / nd) * a.q_sb + (long)h * (a.rot + a.d) + a.rot + d0 + i % nd]);
      __syncthreads();
#pragma unroll 4
      for (int d = grp; d < nd; d += GROUPS) {
        float wv[N];
        const T* p = w + (long)(d0 + d) * a.w_sr + (col < a.R ? col : 0);
        if constexpr (N == 1)
          wv[0] = to_f32(*p);
        else
          load_vec<T, N>(p, wv);
#pragma unroll
        for (int m = 0; m < kQueryRows; ++m)
#pragma unroll
          for (int j = 0; j < N; ++j) acc[m][j] = __builtin_fmaf(wv[j], qs[m < rows ? m : 0][d], acc[m][j]);
      }
    }
    __syncthreads();
#pragma unroll
    for (int m = 0; m < kQueryRows; ++m)
#pragma unroll
      for (int j = 0; j < N; ++j) part[grp][m][piece * N + j] = acc[m][j];
    __syncthreads();
    for (int i = tid; i < rows * kQueryCols; i += 256) {
      const int m = i / kQueryCols, c = i % kQueryCols;
      float s = 0.f;
#pragma unroll
      for (int g = 0; g < GROUPS; ++g) s += part[g][m][c];
      if (r0 + c < a.R) a.qa[((long)(b0 + m) * a.H + h) * W + r0 + c] = s;
    }
  }
}

__device__ __forceinline__ f32x4 latent_mfma(bf16x8 a, bf16x8 b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }

// The same for 16 sequences per workgroup, bf16 rows of whole 16-byte pieces: uk is turned round in LDS, 64 of a head's channels at a time.
constexpr int kTileRows = 16;
constexpr int kTileMinRows = 8;  // sequences from which these forms are used

__global__ __launch_bounds__(256) void latent_query_mfma_kernel(const LatentArgs a) {
  constexpr int KD = 64, KS = KD + 8;
  __shared__ __attribute__((aligned(16))) __bf16 ut[kQueryCols * KS];  // [latent channel][channel of the head]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, quad = lane >> 4, W = a.R + a.rot;
  const int col_blocks = (a.R + kQueryCols - 1) / kQueryCols;
  if ((int)blockIdx.x >= a.H * col_blocks) {
    query_row<__bf16>(a, blockIdx.y * kTileRows + blockIdx.x - a.H * col_blocks);
    return;
  }
  const int h = blockIdx.x / col_blocks, r0 = (blockIdx.x % col_blocks) * kQueryCols, b0 = blockIdx.y * kTileRows;
  const __bf16* w = static_cast<const __bf16*>(a.w) + ((long)h * (a.rot + a.d + a.dv) + a.rot) * a.w_sr;
  const __bf16* q = static_cast<const __bf16*>(a.q) + (long)(b0 + l16 < a.B ? b0 + l16 : b0) * a.q_sb + (long)h * (a.rot + a.d) + a.rot;
  const int k4 = tid & 15, e = (tid >> 4) * 8;  // this thread's (4 channels of the head x 8 of the latent)
  const int col = r0 + e < a.R ? r0 + e : 0;
  f32x4 acc[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
  for (int d0 = 0; d0 < a.d; d0 += KD) {
    bf16x8 wf[4], qf[2];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = d0 + k4 * 4 + r;
      wf[r] = *reinterpret_cast<const bf16x8*>(w + (long)(d < a.d ? d : 0) * a.w_sr + col);
    }
#pragma unroll
    for (int s = 0; s < 2; ++s) {  // (channels past the end are zero here, anything in ut)
      const int d = d0 + s * 32 + quad * 8;
      qf[s] = *reinterpret_cast<const bf16x8*>(q + (d < a.d ? d : 0));
      if (d >= a.d) qf[s] = bf16x8{};
    }
    if (d0 > 0) lds_barrier();
#pragma unroll
    for (int j = 0; j < 8; ++j) *reinterpret_cast<bf16x4*>(&ut[(e + j) * KS + k4 * 4]) = bf16x4{wf[0][j], wf[1][j], wf[2][j], wf[3][j]};
    lds_barrier();
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int s = 0; s < 2; ++s)
        acc[i] = latent_mfma(qf[s], *reinterpret_cast<const bf16x8*>(&ut[((wave * 2 + i) * 16 + l16) * KS + s * 32 + quad * 8]), acc[i]);
  }
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int r = r0 + (wave * 2 + i) * 16 + l16;
#pragma unroll
    for (int m = 0; m < 4; ++m) {
      const int b = b0 + quad * 4 + m;
      if (b < a.B && r < a.R) a.qa[((long)b * a.H + h) * W + r] = acc[i][m];
    }
  }
}

// The keys of one split: first key and their number.
__device__ __forceinline__ void split_range(const LatentArgs& a, int pos, int split, int& k0, int& n) {
  const int lo = pos - a.window + 1 > 0 ? pos - a.window + 1 : 0, all = pos - lo + 1;
  const int per = ((all + a.splits - 1) / a.splits + 15) / 16 * 16;
  k0 = lo + split * per;
  n = all - split * per;
  n = n < 0 ? 0 : n > per ? per : n;
}

// Any element type and size: one workgroup per (sequence, head, split).
constexpr int kLatentMax = 1024;  // latent and rotated channels

template <typename T>
__global__ __launch_bounds__(256) void latent_step_any_kernel(const LatentArgs a) {
  __shared__ float qs[kLatentMax];
  __shared__ float ps[256];
  __shared__ float red[8];
  const int tid = threadIdx.x, W = a.R + a.rot;
  const int h = blockIdx.x % a.H, split = (blockIdx.x / a.H) % a.splits, b = blockIdx.x / (a.H * a.splits);
  const int pos = row_pos(a.pos, a.pos_host, b);
  if (pos < 0 || pos >= a.S) return;
  int first, n;
  split_range(a, pos, split, first, n);
  const T* cache = static_cast<const T*>(a.cache) + b * a.c_sb;
  for (int c = tid; c < W; c += 256) qs[c] = a.qa[((long)b * a.H + h) * W + c];
  float acc[kLatentMax / 256], m_run = -INFINITY, l_run = 0.f;
#pragma unroll
  for (int i = 0; i < kLatentMax / 256; ++i) acc[i] = 0.f;
  __syncthreads();
  for (int k0 = 0; k0 < n; k0 += 256) {
    const int nk = n - k0 < 256 ? n - k0 : 256;
    float s = -INFINITY;
    if (tid < nk) {
      const T* row = cache + (long)(first + k0 + tid) * a.c_st;
      float dot = 0.f;
      for (int c = 0; c < W; ++c) dot = __builtin_fmaf(qs[c], to_f32(row[c]), dot);
      s = dot * a.scale;
    }
    float mx = s;
#pragma unroll
    for (int m = 32; m >= 1; m >>= 1) mx = fmaxf(mx, __shfl_xor(mx, m, 64));
    if ((tid & 63) == 0) red[tid >> 6] = mx;
    __syncthreads();
    const float m_new = fmaxf(fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])), m_run);
    const float alpha = expf(m_run - m_new), p = expf(s - m_new);
    m_run = m_new;
    ps[tid] = p;
    const float sum = wave_sum(p);
    if ((tid & 63) == 0) red[4 + (tid >> 6)] = sum;
    __syncthreads();
    l_run = l_run * alpha + red[4] + red[5] + red[6] + red[7];
#pragma unroll
    for (int i = 0; i < kLatentMax / 256; ++i) {
      const int c = i * 256 + tid;
      if (c < a.R) {
        float v = acc[i] * alpha;
        for (int j = 0; j < nk; ++j) v = __builtin_fmaf(ps[j], to_f32(cache[(long)(first + k0 + j) * a.c_st + c]), v);
        acc[i] = v;
      }
    }
    __syncthreads();
  }
  const long at = ((long)b * a.splits + split) * a.H + h;
#pragma unroll
  for (int i = 0; i < kLatentMax / 256; ++i) {
    const int c = i * 256 + tid;
    if (c < a.R) a.part[at * a.R + c] = acc[i];
  }
  if (tid == 0) {
    a.part_ml[2 * at] = m_run;
    a.part_ml[2 * at + 1] = l_run;
  }
}

// bf16, MFMA: 16 heads per workgroup, 64 keys at a time; a wavefront forms the scores of 16 of them and a
// quarter of the weighted latents.  KC: 32-channel pieces of a row (rounded up); RT: 16-channel tiles of the latent per
// wavefront (rounded up).  R and rot multiples of 8.
template <int KC, int RT>
__global__ __launch_bounds__(256, 1) void latent_step_mfma_kernel(const LatentArgs a) {
  constexpr int KS = 64 + 8;  // keys per LDS row
  constexpr int RMAX = RT * 64;
  __shared__ __attribute__((aligned(16))) __bf16 vt[RMAX * KS];  // [latent channel][key]
  __shared__ __attribute__((aligned(16))) __bf16 ps[16 * KS];    // [head][key]
  __shared__ float wmax[4][16], wsum[4][16];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, quad = lane >> 4, W = a.R + a.rot;
  const int b = blockIdx.x, split = blockIdx.y, h0 = blockIdx.z * 16;
  const int pos = row_pos(a.pos, a.pos_host, b);
  if (pos < 0 || pos >= a.S) return;
  int first, n;
  split_range(a, pos, split, first, n);
  const __bf16* cache = static_cast<const __bf16*>(a.cache) + b * a.c_sb + (long)first * a.c_st;
  const long at = ((long)b * a.splits + split) * a.H + h0 + l16;  // of this lane's head
  const bool head_in = h0 + l16 < a.H;
  if (n == 0) {
    if (head_in && tid < 16) a.part_ml[2 * at] = -INFINITY, a.part_ml[2 * at + 1] = 0.f;
    return;
  }
  typedef __attribute__((ext_vector_type(4))) uint32_t u32x4;
  constexpr int VU = 16 * (RMAX / 8) / 256 > 0 ? 16 * (RMAX / 8) / 256 : 1;  // (4 keys x 8 channels) pieces per thread
  bf16x8 kf[KC];
  u32x4 vf[VU][4];
  auto fetch = [&](int k0) {
    const int key = k0 + wave * 16 + l16;
    const __bf16* row = cache + (long)(key < n ? key : n - 1) * a.c_st;
#pragma unroll
    for (int c = 0; c < KC; ++c) {
      const int e = c * 32 + quad * 8;
      kf[c] = *reinterpret_cast<const bf16x8*>(row + (e < W ? e : 0));
    }
#pragma unroll
    for (int i = 0; i < VU; ++i) {
      const int p = i * 256 + tid, k4 = p & 15, e = (p >> 4) * 8;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int vk = k0 + k4 * 4 + r;
        vf[i][r] = *reinterpret_cast<const u32x4*>(cache + (long)(vk < n ? vk : n - 1) * a.c_st + (e < a.R ? e : 0));
      }
    }
  };
  fetch(0);
  // queries of this lane's head, the score scale in them
  bf16x8 qf[KC];
  const float* q = a.qa + ((long)b * a.H + (head_in ? h0 + l16 : 0)) * W;
#pragma unroll
  for (int c = 0; c < KC; ++c) {
    const int e = c * 32 + quad * 8;
    float x[8];
    load_vec<float, 8>(q + (e < W ? e : 0), x);
#pragma unroll
    for (int j = 0; j < 8; ++j) qf[c][j] = (__bf16)(e < W ? x[j] : 0.f);
  }
  const float scale2 = a.scale * 1.4426950408889634f;
  f32x4 acc[RT];
#pragma unroll
  for (int i = 0; i < RT; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m_run = -INFINITY, l_run = 0.f;
  for (int k0 = 0; k0 < n; k0 += 64) {
    lds_barrier();
#pragma unroll
    for (int i = 0; i < VU; ++i) {
      const int p = i * 256 + tid, k4 = p & 15, e = (p >> 4) * 8;
      if (e < RMAX) {
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          bf16x4 col;
#pragma unroll
          for (int r = 0; r < 4; ++r) col[r] = __builtin_bit_cast(bf16x8, vf[i][r])[j];
          *reinterpret_cast<bf16x4*>(&vt[(e + j) * KS + k4 * 4]) = col;
        }
      }
    }
    // scores: column = head l16, rows = keys 4 quad + i of this wavefront's 16
    f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int c = 0; c < KC; ++c) s = latent_mfma(kf[c], qf[c], s);
    if (k0 + 64 < n) fetch(k0 + 64);
    float mx = -INFINITY;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      s[i] = k0 + wave * 16 + quad * 4 + i < n ? s[i] * scale2 : -INFINITY;
      mx = fmaxf(mx, s[i]);
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    if (quad == 0) wmax[wave][l16] = mx;
    lds_barrier();
    const float m_new = fmaxf(m_run, fmaxf(fmaxf(wmax[0][l16], wmax[1][l16]), fmaxf(wmax[2][l16], wmax[3][l16])));
    const float alpha = __builtin_amdgcn_exp2f(m_run - m_new);
    m_run = m_new;
    bf16x4 p4;
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float p = __builtin_amdgcn_exp2f(s[i] - m_new);
      sum += p;
      p4[i] = (__bf16)p;
    }
    *reinterpret_cast<bf16x4*>(&ps[l16 * KS + wave * 16 + quad * 4]) = p4;
    sum += __shfl_xor(sum, 16, 64);
    sum += __shfl_xor(sum, 32, 64);
    if (quad == 0) wsum[wave][l16] = sum;
    lds_barrier();
    l_run = l_run * alpha + wsum[0][l16] + wsum[1][l16] + wsum[2][l16] + wsum[3][l16];
    const bf16x8 pf0 = *reinterpret_cast<const bf16x8*>(&ps[l16 * KS + quad * 8]);
    const bf16x8 pf1 = *reinterpret_cast<const bf16x8*>(&ps[l16 * KS + 32 + quad * 8]);
#pragma unroll
    for (int i = 0; i < RT; ++i) {
      const __bf16* v = &vt[((wave * RT + i) * 16 + l16) * KS + quad * 8];
      acc[i] *= alpha;
      acc[i] = latent_mfma(*reinterpret_cast<const bf16x8*>(v), pf0, acc[i]);
      acc[i] = latent_mfma(*reinterpret_cast<const bf16x8*>(v + 32), pf1, acc[i]);
    }
  }
  if (!head_in) return;
#pragma unroll
  for (int i = 0; i < RT; ++i) {
    const int r = (wave * RT + i) * 16 + quad * 4;
    if (r < a.R) *reinterpret_cast<f32x4*>(a.part + at * a.R + r) = acc[i];
  }
  if (wave == 0 && quad == 0) {
    a.part_ml[2 * at] = m_run * 0.6931471805599453f;  // natural units, as the other form leaves it
    a.part_ml[2 * at + 1] = l_run;
  }
}

constexpr int kValueRows = 4;   // sequences at a time
constexpr int kValueCols = 16;  // value channels per workgroup
constexpr int kMaxSplits = 64;

template <typename T, int N>
__global__ __launch_bounds__(256) void latent_values_kernel(const LatentArgs a) {
  __shared__ __attribute__((aligned(16))) float lat[kValueRows][kLatentMax];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int h = blockIdx.x, b0 = blockIdx.y * kValueRows, j0 = blockIdx.z * kValueCols;
  const int rows = a.B - b0 < kValueRows ? a.B - b0 : kValueRows;
  // this wavefront's rows of uv are asked for first
  constexpr int JU = kValueCols / 4;
  const T* w = static_cast<const T*>(a.w) + ((long)h * (a.rot + a.d + a.dv) + a.rot + a.d) * a.w_sr;
  const int j1 = j0 + kValueCols < a.dv ? j0 + kValueCols : a.dv, j = j0 + wave * JU;
  float wv[JU][N];
  auto load_rows = [&](int c) {
#pragma unroll
    for (int u = 0; u < JU; ++u) {
      const T* p = w + (long)(j + u < j1 ? j + u : j0) * a.w_sr + (c < a.R ? c : 0);
      if constexpr (N == 1)
        wv[u][0] = to_f32(*p);
      else
        load_vec<T, N>(p, wv[u]);
    }
  };
  load_rows(lane * N);
  // what each split counts for: exp(m_s - max) / sum
  __shared__ float share[kValueRows][kMaxSplits];
  for (int m = wave; m < rows; m += 4) {
    const int pos = row_pos(a.pos, a.pos_host, b0 + m);
    const bool ok = pos >= 0 && pos < a.S;
    const float* ml = a.part_ml + 2 * ((long)(b0 + m) * a.splits * a.H + h);
    float ms[kMaxSplits / 64], ls[kMaxSplits / 64], mx = -INFINITY, l = 0.f;
#pragma unroll
    for (int i = 0; i < kMaxSplits / 64; ++i) {
      const int s = i * 64 + lane;
      const bool in = ok && s < a.splits;
      ms[i] = in ? ml[2 * (long)s * a.H] : -INFINITY;
      ls[i] = in ? ml[2 * (long)s * a.H + 1] : 0.f;
      mx = fmaxf(mx, ms[i]);
    }
#pragma unroll
    for (int x = 32; x >= 1; x >>= 1) mx = fmaxf(mx, __shfl_xor(mx, x, 64));
#pragma unroll
    for (int i = 0; i < kMaxSplits / 64; ++i) {
      ms[i] = ms[i] == -INFINITY ? 0.f : expf(ms[i] - mx);
      l = __builtin_fmaf(ms[i], ls[i], l);
    }
    l = wave_sum(l);
#pragma unroll
    for (int i = 0; i < kMaxSplits / 64; ++i) share[m][i * 64 + lane] = l > 0.f ? ms[i] / l : 0.f;
  }
  lds_barrier();
  // (a split without keys has left nothing in its part: it is not read)
  const float* p0 = a.part + ((long)b0 * a.splits * a.H + h) * a.R;
  const long p_row = (long)a.splits * a.H * a.R, p_split = (long)a.H * a.R;
  constexpr int SU = 8;  // splits whose parts are in flight together
  if (a.R % 4 == 0 && (reinterpret_cast<uintptr_t>(a.part) & 15) == 0) {
    const int pieces = a.R / 4;
    for (int i = tid; i < rows * pieces; i += 256) {
      const int m = i / pieces, c = i % pieces * 4;
      f32x4 v = {0.f, 0.f, 0.f, 0.f};
      for (int s0 = 0; s0 < a.splits; s0 += SU) {
        f32x4 x[SU];
        float f[SU];
#pragma unroll
        for (int s = 0; s < SU; ++s) {
          f[s] = s0 + s < a.splits ? share[m][s0 + s] : 0.f;
          x[s] = *reinterpret_cast<const f32x4*>(p0 + m * p_row + (f[s] != 0.f ? (s0 + s) * p_split : 0) + c);
        }
#pragma unroll
        for (int s = 0; s < SU; ++s)
#pragma unroll
          for (int j = 0; j < 4; ++j) v[j] = f[s] != 0.f ? __builtin_fmaf(f[s], x[s][j], v[j]) : v[j];
      }
      *reinterpret_cast<f32x4*>(&lat[m][c]) = v;
    }
  } else {
    for (int i = tid; i < rows * a.R; i += 256) {
      const int m = i / a.R, c = i % a.R;
      float v = 0.f;
      for (int s = 0; s < a.splits; ++s) {
        const float f = share[m][s];
        if (f != 0.f) v = __builtin_fmaf(f, p0[m * p_row + s * p_split + c], v);
      }
      lat[m][c] = v;
    }
  }
  lds_barrier();
  {
    float acc[JU][kValueRows];
#pragma unroll
    for (int u = 0; u < JU; ++u)
#pragma unroll
      for (int m = 0; m < kValueRows; ++m) acc[u][m] = 0.f;
    for (int c = lane * N; c < a.R; c += 64 * N) {
      if (c >= 64 * N) load_rows(c);
#pragma unroll
      for (int m = 0; m < kValueRows; ++m)
#pragma unroll
        for (int i = 0; i < N; ++i) {
          const float x = lat[m < rows ? m : 0][c + i];
#pragma unroll
          for (int u = 0; u < JU; ++u) acc[u][m] = __builtin_fmaf(wv[u][i], x, acc[u][m]);
        }
    }
#pragma unroll
    for (int u = 0; u < JU; ++u)
#pragma unroll
      for (int m = 0; m < kValueRows; ++m) {
        float s = sum16(acc[u][m]);
        s += __shfl_xor(s, 16, 64);
        s += __shfl_xor(s, 32, 64);
        if (m < rows && lane == 0 && j + u < j1) static_cast<T*>(a.o)[(long)(b0 + m) * a.o_sb + (long)h * a.dv + j + u] = from_f32<T>(s * a.out_scale);
      }
  }
}

// The same for 16 sequences per workgroup, bf16: KC 32-channel pieces of the latent (rounded up), 64 value channels per workgroup.
// R a multiple of 8, part 16-byte aligned.
template <int KC>
__global__ __launch_bounds__(256) void latent_values_mfma_kernel(const LatentArgs a) {
  constexpr int RS = KC * 32 + 8;
  __shared__ __attribute__((aligned(16))) __bf16 lat[kTileRows * RS];
  __shared__ float share[kTileRows][kMaxSplits];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, quad = lane >> 4;
  const int h = blockIdx.x, b0 = blockIdx.y * kTileRows, j = blockIdx.z * 64 + wave * 16 + l16;
  const int rows = a.B - b0 < kTileRows ? a.B - b0 : kTileRows;
  // this lane's row of uv is asked for first
  const __bf16* w = static_cast<const __bf16*>(a.w) + ((long)h * (a.rot + a.d + a.dv) + a.rot + a.d + (j < a.dv ? j : 0)) * a.w_sr;
  bf16x8 wf[KC];
#pragma unroll
  for (int c = 0; c < KC; ++c) {
    const int e = c * 32 + quad * 8;
    wf[c] = *reinterpret_cast<const bf16x8*>(w + (e < a.R ? e : 0));
  }
  {  // what each split counts for: exp(m_s - max) / sum; 16 lanes per row
    const int m = tid >> 4, b = b0 + (m < rows ? m : 0);
    const int pos = row_pos(a.pos, a.pos_host, b);
    const bool ok = m < rows && pos >= 0 && pos < a.S;
    const float* ml = a.part_ml + 2 * ((long)b * a.splits * a.H + h);
    constexpr int N = kMaxSplits / 16;
    float ms[N], ls[N], mx = -INFINITY, l = 0.f;
#pragma unroll
    for (int i = 0; i < N; ++i) {
      const int s = i * 16 + (tid & 15);
      const bool in = ok && s < a.splits;
      ms[i] = in ? ml[2 * (long)s * a.H] : -INFINITY;
      ls[i] = in ? ml[2 * (long)s * a.H + 1] : 0.f;
      mx = fmaxf(mx, ms[i]);
    }
#pragma unroll
    for (int x = 8; x >= 1; x >>= 1) mx = fmaxf(mx, __shfl_xor(mx, x, 64));
#pragma unroll
    for (int i = 0; i < N; ++i) {
      ms[i] = ms[i] == -INFINITY ? 0.f : expf(ms[i] - mx);
      l = __builtin_fmaf(ms[i], ls[i], l);
    }
    l = sum16(l);
#pragma unroll
    for (int i = 0; i < N; ++i) share[m][i * 16 + (tid & 15)] = l > 0.f ? ms[i] / l : 0.f;
  }
  lds_barrier();
  // (a split without keys has left nothing in its part: it is not read)
  const float* p0 = a.part + ((long)b0 * a.splits * a.H + h) * a.R;
  const long p_row = (long)a.splits * a.H * a.R, p_split = (long)a.H * a.R;
  constexpr int PIECES = KC * 8, IU = 4, SU = 2;  // 4-channel pieces of a row; pieces and splits in flight together
  for (int i0 = tid; i0 < kTileRows * PIECES; i0 += 256 * IU) {
    f32x4 v[IU];
#pragma unroll
    for (int u = 0; u < IU; ++u) v[u] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int s0 = 0; s0 < a.splits; s0 += SU) {
      f32x4 x[IU][SU];
      float f[IU][SU];
#pragma unroll
      for (int u = 0; u < IU; ++u)
#pragma unroll
        for (int s = 0; s < SU; ++s) {
          const int m = (i0 + u * 256) / PIECES, c = (i0 + u * 256) % PIECES * 4;
          const bool in = m < rows && c < a.R;
          f[u][s] = in && s0 + s < a.splits ? share[m][s0 + s] : 0.f;
          x[u][s] = *reinterpret_cast<const f32x4*>(p0 + (f[u][s] != 0.f ? m * p_row + (s0 + s) * p_split + c : 0));
        }
#pragma unroll
      for (int u = 0; u < IU; ++u)
#pragma unroll
        for (int s = 0; s < SU; ++s)
#pragma unroll
          for (int k = 0; k < 4; ++k) v[u][k] = f[u][s] != 0.f ? __builtin_fmaf(f[u][s], x[u][s][k], v[u][k]) : v[u][k];
    }
#pragma unroll
    for (int u = 0; u < IU; ++u) {
      const int m = (i0 + u * 256) / PIECES, c = (i0 + u * 256) % PIECES * 4;
      *reinterpret_cast<bf16x4*>(&lat[m * RS + c]) = bf16x4{(__bf16)v[u][0], (__bf16)v[u][1], (__bf16)v[u][2], (__bf16)v[u][3]};
    }
  }
  lds_barrier();
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int c = 0; c < KC; ++c) acc = latent_mfma(*reinterpret_cast<const bf16x8*>(&lat[l16 * RS + c * 32 + quad * 8]), wf[c], acc);
#pragma unroll
  for (int m = 0; m < 4; ++m)
    if (quad * 4 + m < rows && j < a.dv)
      static_cast<__bf16*>(a.o)[(long)(b0 + quad * 4 + m) * a.o_sb + (long)h * a.dv + j] = (__bf16)(acc[m] * a.out_scale);
}

static int latent_check(const char* who, const LatentArgs& a, int64_t last, int io_dtype) {
  BASED_REQUIRE(a.x && a.norm_w && a.cache, BASED_ERR_ARG, "%s: null pointer argument", who);
  BASED_REQUIRE(a.B >= 0 && a.L >= 0 && a.S > 0 && a.R > 0 && a.rot >= 0 && a.rot % 2 == 0, BASED_ERR_ARG, "%s: bad sizes", who);
  BASED_REQUIRE(a.R + a.rot <= kLatentMax, BASED_ERR_SHAPE, "%s: cache rows of %d channels (at most %d)", who, a.R + a.rot, kLatentMax);
  BASED_REQUIRE(a.rot == 0 || (a.cos_t && a.sin_t), BASED_ERR_ARG, "%s: rotary tables missing", who);
  BASED_REQUIRE(last < a.S, BASED_ERR_SHAPE, "%s: position %ld does not fit a cache of %d rows", who, (long)last, a.S);
  BASED_REQUIRE(a.rot == 0 || last < a.n_pos, BASED_ERR_SHAPE, "%s: rotary tables end before position %ld", who, (long)last);
  BASED_REQUIRE(io_dtype == BASED_BF16 || io_dtype == BASED_F32, BASED_ERR_DTYPE, "%s: bad dtype", who);
  return BASED_OK;
}

template <int KC, int RT> void launch_latent_mfma(const LatentArgs& a, hipStream_t s) {
  hipLaunchKernelGGL((latent_step_mfma_kernel<KC, RT>), dim3((unsigned)a.B, (unsigned)a.splits, (unsigned)((a.H + 15) / 16)), dim3(256), 0,
                     s, a);
}

template <typename T> void launch_latent_query(const LatentArgs& a, bool vec, hipStream_t s) {
  const dim3 grid((unsigned)(a.H * ((a.R + kQueryCols - 1) / kQueryCols) + kQueryRows), (unsigned)((a.B + kQueryRows - 1) / kQueryRows));
  if (vec)
    hipLaunchKernelGGL((latent_query_kernel<T, Pack<T>::kN>), grid, dim3(256), 0, s, a);
  else
    hipLaunchKernelGGL((latent_query_kernel<T, 1>), grid, dim3(256), 0, s, a);
}

template <typename T> void launch_latent_values(const LatentArgs& a, bool vec, hipStream_t s) {
  const dim3 grid((unsigned)a.H, (unsigned)((a.B + kValueRows - 1) / kValueRows), (unsigned)((a.dv + kValueCols - 1) / kValueCols));
  if (vec)
    hipLaunchKernelGGL((latent_values_kernel<T, Pack<T>::kN>), grid, dim3(256), 0, s, a);
  else
    hipLaunchKernelGGL((latent_values_kernel<T, 1>), grid, dim3(256), 0, s, a);
}

static bool launch_latent_step_mfma(const LatentArgs& a, hipStream_t s) {
  const int kc = (a.R + a.rot + 31) / 32, rt = (a.R + 63) / 64;
  if (kc <= 3 && rt <= 1)
    launch_latent_mfma<3, 1>(a, s);
  else if (kc <= 5 && rt <= 2)
    launch_latent_mfma<5, 2>(a, s);
  else if (kc <= 10 && rt <= 4)
    launch_latent_mfma<10, 4>(a, s);
  else if (kc <= 18 && rt <= 8)
    launch_latent_mfma<18, 8>(a, s);
  else
    return false;
  return true;
}

}  // namespace based

extern "C" BASED_API int based_latent_write(const void* x, const void* norm_w, void* cache, int64_t start, int64_t B, int64_t L, int64_t S,
                                            int64_t R, int64_t rot, int64_t x_sb, int64_t x_sl, int64_t c_sb, int64_t c_st, float eps,
                                            const float* rope_cos, const float* rope_sin, int64_t rope_len, int half_split, int io_dtype,
                                            void* stream) {
  using namespace based;
  BASED_REQUIRE(start >= 0 && start + L < (1ll << 31), BASED_ERR_SHAPE, "latent_write: sequence too long");
  LatentArgs a{};
  a.x = x, a.norm_w = norm_w, a.cache = cache, a.cos_t = rope_cos, a.sin_t = rope_sin, a.pos_host = (int)start, a.n_pos = (int)rope_len;
  a.B = (int)B, a.L = (int)L, a.S = (int)S, a.R = (int)R, a.rot = (int)rot, a.half_split = half_split;
  a.x_sb = x_sb, a.x_sl = x_sl, a.c_sb = c_sb, a.c_st = c_st, a.eps = eps;
  const int rc = latent_check("latent_write", a, start + L - 1, io_dtype);
  if (rc != BASED_OK) return rc;
  if (B == 0 || L == 0) return BASED_OK;
  hipStream_t s = static_cast<hipStream_t>(stream);
  const int64_t rows = B * L;
  BASED_REQUIRE(rows < (1ll << 31), BASED_ERR_SHAPE, "latent_write: grid too large");
  const bool vec = io_dtype == BASED_BF16 && R % 8 == 0 && x_sb % 8 == 0 && x_sl % 8 == 0 && c_sb % 8 == 0 && c_st % 8 == 0 &&
                   aligned_to(x, 16) && aligned_to(cache, 16) && aligned_to(norm_w, 16);
  if (vec && R <= 256)
    hipLaunchKernelGGL(latent_write_vec_kernel<16>, dim3((unsigned)((rows + 15) / 16)), dim3(256), 0, s, a);
  else if (vec && R <= 512)
    hipLaunchKernelGGL(latent_write_vec_kernel<32>, dim3((unsigned)((rows + 7) / 8)), dim3(256), 0, s, a);
  else if (vec)
    hipLaunchKernelGGL(latent_write_vec_kernel<64>, dim3((unsigned)((rows + 3) / 4)), dim3(256), 0, s, a);
  else if (io_dtype == BASED_BF16)
    hipLaunchKernelGGL(latent_write_kernel<__bf16>, dim3((unsigned)((rows + 3) / 4)), dim3(256), 0, s, a);
  else
    hipLaunchKernelGGL(latent_write_kernel<float>, dim3((unsigned)((rows + 3) / 4)), dim3(256), 0, s, a);
  return check_launch("latent_write");
}

extern "C" BASED_API int based_latent_step(const void* q, const void* x, const void* norm_w, const void* weight, void* cache, float* work_q,
                                           float* work_part, float* work_ml, void* o, const int32_t* pos, int64_t pos_host, int64_t B,
                                           int64_t H, int64_t D, int64_t DV, int64_t S, int64_t R, int64_t rot, int64_t splits,
                                           int64_t q_sb, int64_t x_sb, int64_t w_sr, int64_t c_sb, int64_t c_st, int64_t o_sb,
                                           int64_t window, float scale, float eps, float out_scale, const float* rope_cos,
                                           const float* rope_sin, int64_t rope_len, int half_split, int io_dtype, void* stream) {
  using namespace based;
  BASED_REQUIRE(q && weight && work_q && work_part && work_ml && o, BASED_ERR_ARG, "latent_step: null pointer argument");
  BASED_REQUIRE(H > 0 && D > 0 && DV > 0 && window > 0 && window < (1ll << 31) && splits > 0 && splits < 65536 && pos_host >= 0 &&
                    pos_host < (1ll << 31),
                BASED_ERR_ARG, "latent_step: bad sizes");
  BASED_REQUIRE(splits <= kMaxSplits, BASED_ERR_SHAPE, "latent_step: %ld splits (at most %d)", (long)splits, kMaxSplits);
  BASED_REQUIRE(B < 65536 * kValueRows && B * H * splits < (1ll << 31) && H < 65536, BASED_ERR_SHAPE, "latent_step: grid too large");
  LatentArgs a{};
  a.x = x, a.norm_w = norm_w, a.cache = cache, a.cos_t = rope_cos, a.sin_t = rope_sin, a.pos = pos, a.pos_host = (int)pos_host;
  a.n_pos = (int)rope_len, a.B = (int)B, a.L = 1, a.S = (int)S, a.R = (int)R, a.rot = (int)rot, a.half_split = half_split;
  a.x_sb = x_sb, a.c_sb = c_sb, a.c_st = c_st, a.eps = eps, a.q = q, a.w = weight, a.qa = work_q, a.part = work_part, a.part_ml = work_ml;
  a.o = o, a.H = (int)H, a.d = (int)D, a.dv = (int)DV, a.splits = (int)splits, a.window = (int)window;
  a.q_sb = q_sb, a.w_sr = w_sr, a.o_sb = o_sb, a.scale = scale, a.out_scale = out_scale;
  const int rc = latent_check("latent_step", a, pos != nullptr ? 0 : pos_host, io_dtype);
  if (rc != BASED_OK) return rc;
  if (B == 0) return BASED_OK;
  hipStream_t s = static_cast<hipStream_t>(stream);
  const int n = io_dtype == BASED_BF16 ? 8 : 4;
  const bool vec = R % n == 0 && w_sr % n == 0 && aligned_to(weight, 16);
  const bool tiles = io_dtype == BASED_BF16 && vec && B >= kTileMinRows;
  if (tiles && D % 8 == 0 && rot % 8 == 0 && q_sb % 8 == 0 && aligned_to(q, 16))
    hipLaunchKernelGGL(latent_query_mfma_kernel, dim3((unsigned)(H * ((R + kQueryCols - 1) / kQueryCols) + kTileRows),
                       (unsigned)((B + kTileRows - 1) / kTileRows)), dim3(256), 0, s, a);
  else if (io_dtype == BASED_BF16)
    launch_latent_query<__bf16>(a, vec, s);
  else
    launch_latent_query<float>(a, vec, s);
  const bool mfma = io_dtype == BASED_BF16 && R % 8 == 0 && rot % 8 == 0 && c_sb % 8 == 0 && c_st % 8 == 0 && aligned_to(cache, 16) &&
                    aligned_to(work_q, 16) && aligned_to(work_part, 16);
  if (!mfma || !launch_latent_step_mfma(a, s)) {
    const dim3 grid((unsigned)(B * H * splits));
    if (io_dtype == BASED_BF16)
      hipLaunchKernelGGL(latent_step_any_kernel<__bf16>, grid, dim3(256), 0, s, a);
    else
      hipLaunchKernelGGL(latent_step_any_kernel<float>, grid, dim3(256), 0, s, a);
  }
  const dim3 tile_grid((unsigned)H, (unsigned)((B + kTileRows - 1) / kTileRows), (unsigned)((DV + 63) / 64));
  if (tiles && aligned_to(work_part, 16) && R <= 256)
    hipLaunchKernelGGL(latent_values_mfma_kernel<8>, tile_grid, dim3(256), 0, s, a);
  else if (tiles && aligned_to(work_part, 16) && R <= 512)
    hipLaunchKernelGGL(latent_values_mfma_kernel<16>, tile_grid, dim3(256), 0, s, a);
  else if (io_dtype == BASED_BF16)
    launch_latent_values<__bf16>(a, vec, s);
  else
    launch_latent_values<float>(a, vec, s);
  return check_launch("latent_step");
}
