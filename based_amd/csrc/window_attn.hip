// Causal softmax attention over a sliding window of any size with grouped heads, for gfx950:
// position i attends j with 0 <= i - j < window; query head h reads key/value head h / (H / G);
// key and value sizes may differ.  In the same launches: rotary positions on the leading
// rotary_dim channels of q and k (interleaved pairs (2i, 2i + 1), or half-split pairs
// (i, i + rotary_dim / 2)) and the value norm v / sqrt(mean(v^2) + eps).
//
// The cache holds one row per token and key/value head: dim key channels (rotated), then vdim
// value channels (normalised), (B, S, G, dim + vdim).
//
//   window_kv_write      a portion's keys and values into the cache
//   window_prefill_mfma  bf16: 128 (token, head) rows per workgroup, 32 per wavefront.  The heads of
//                        a group are rows of the same tile, so that a key tile is fetched once for
//                        all of them and a tile of tokens is short against the window.  Scores are
//                        formed transposed (keys x queries), which leaves the weights in the lanes
//                        that the product with the values wants them in.
//   window_prefill_any   any element type and size: one wavefront per query
//   window_step          one token per sequence: rotation, value norm, cache write and attention,
//                        one workgroup per (sequence, key/value head)
#include "stream_common.hpp"

namespace based {

struct WindowArgs {
  const void* q;
  const void* k;
  const void* v;
  void* kv;
  void* o;
  const float* cos_t;  // (n_pos, rot / 2) or null
  const float* sin_t;
  const int32_t* pos;
  int pos_host, n_pos;
  int B, L, H, G, d, dv, S;
  long q_sb, q_sl, k_sb, k_sl, v_sb, v_sl, o_sb, o_sl;  // heads are contiguous blocks of d / dv
  long kv_sb, kv_st;
  int rot, half_split, window, norm_v;
  float scale, eps, out_scale;
};

// partner and sign of channel c in the rotation: x'_c = x_c cos + sgn * x_partner sin
__device__ __forceinline__ void rope_pair(int c, int rot, int half_split, int& pair, int& partner, float& sgn) {
  if (half_split) {
    const int h = rot / 2;
    pair = c < h ? c : c - h;
    partner = c < h ? c + h : c - h;
    sgn = c < h ? -1.f : 1.f;
  } else {
    pair = c >> 1;
    partner = c ^ 1;
    sgn = (c & 1) ? 1.f : -1.f;
  }
}

template <typename T>
__device__ __forceinline__ float rotated(const T* row, int c, int pos, const WindowArgs& a) {
  const float x = to_f32(row[c]);
  if (c >= a.rot) return x;
  int pair, partner;
  float sgn;
  rope_pair(c, a.rot, a.half_split, pair, partner, sgn);
  const long t = (long)pos * (a.rot / 2) + pair;
  return x * a.cos_t[t] + sgn * to_f32(row[partner]) * a.sin_t[t];
}

// What turns 8 channels from c on (c and the rotary size multiples of 8): angles, and for half-split pairs
// the partners.  Loaded without a condition (what is not rotated reads the table's start and its own
// channels) and applied later, so that every load of a row is on its way before the first is waited for.
template <bool HALF> struct Turn8 {
  float cs[HALF ? 8 : 4], sn[HALF ? 8 : 4], partner[8];
  __device__ __forceinline__ void load(const __bf16* row, int c, int pos, const WindowArgs& a) {
    const bool in = c < a.rot;
    const int half = a.rot / 2;
    if constexpr (HALF) {
      const int pair = in ? (c < half ? c : c - half) : 0;
      const long t = in ? (long)pos * half + pair : 0;
      load_vec<float, 8>((a.rot > 0 ? a.cos_t : reinterpret_cast<const float*>(a.kv)) + t, cs);
      load_vec<float, 8>((a.rot > 0 ? a.sin_t : reinterpret_cast<const float*>(a.kv)) + t, sn);
      load_vec<__bf16, 8>(row + (in ? (c < half ? c + half : c - half) : 0), partner);
    } else {
      const long t = in ? (long)pos * half + c / 2 : 0;
      load_vec<float, 4>((a.rot > 0 ? a.cos_t : reinterpret_cast<const float*>(a.kv)) + t, cs);
      load_vec<float, 4>((a.rot > 0 ? a.sin_t : reinterpret_cast<const float*>(a.kv)) + t, sn);
    }
  }
  __device__ __forceinline__ void apply(float (&x)[8], int c, const WindowArgs& a) const {
    if (c >= a.rot) return;
    if constexpr (HALF) {
      const float sgn = c < a.rot / 2 ? -1.f : 1.f;
#pragma unroll
      for (int j = 0; j < 8; ++j) x[j] = x[j] * cs[j] + sgn * partner[j] * sn[j];
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float u = x[2 * j], v = x[2 * j + 1];
        x[2 * j] = u * cs[j] - v * sn[j];
        x[2 * j + 1] = v * cs[j] + u * sn[j];
      }
    }
  }
};

// One wavefront per (token, key/value head).
template <typename T>
__global__ __launch_bounds__(256) void window_kv_write_kernel(const WindowArgs a) {
  const long item = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= (long)a.B * a.L * a.G) return;
  const int lane = threadIdx.x & 63;
  const int g = (int)(item % a.G);
  const long bl = item / a.G;
  const int l = (int)(bl % a.L), b = (int)(bl / a.L);
  const int pos = a.pos_host + l;
  const T* k = static_cast<const T*>(a.k) + b * a.k_sb + l * a.k_sl + (long)g * a.d;
  const T* v = static_cast<const T*>(a.v) + b * a.v_sb + l * a.v_sl + (long)g * a.dv;
  T* out = static_cast<T*>(a.kv) + b * a.kv_sb + pos * a.kv_st + (long)g * (a.d + a.dv);
  float ss = 0.f;
  for (int c = lane; c < a.dv; c += 64) ss = __builtin_fmaf(to_f32(v[c]), to_f32(v[c]), ss);
  const float r = a.norm_v ? 1.0f / sqrtf(wave_sum(ss) / (float)a.dv + a.eps) : 1.0f;
  for (int c = lane; c < a.d; c += 64) out[c] = from_f32<T>(rotated(k, c, pos, a));
  for (int c = lane; c < a.dv; c += 64) out[a.d + c] = from_f32<T>(to_f32(v[c]) * r);
}

// The same with 16-byte pieces: LPI (8, 16 or 32) lanes per (token, key/value head), one piece of the key and
// one of the value each.  d, dv and every stride multiples of 8, pointers 16-byte aligned.
template <int LPI, bool HALF>
__global__ __launch_bounds__(256) void window_kv_write_vec_kernel(const WindowArgs a) {
  const long item0 = (long)blockIdx.x * (256 / LPI) + threadIdx.x / LPI;
  const long n_items = (long)a.B * a.L * a.G;
  const bool live = item0 < n_items;
  const long item = live ? item0 : n_items - 1;
  const int c = (threadIdx.x % LPI) * 8;
  const int g = (int)(item % a.G);
  const long bl = item / a.G;
  const int l = (int)(bl % a.L), b = (int)(bl / a.L);
  const int pos = a.pos_host + l;
  const __bf16* k = static_cast<const __bf16*>(a.k) + b * a.k_sb + l * a.k_sl + (long)g * a.d;
  const __bf16* v = static_cast<const __bf16*>(a.v) + b * a.v_sb + l * a.v_sl + (long)g * a.dv;
  __bf16* out = static_cast<__bf16*>(a.kv) + b * a.kv_sb + pos * a.kv_st + (long)g * (a.d + a.dv);
  const int ck = c < a.d ? c : 0, cv = c < a.dv ? c : 0;
  float x[8], y[8];
  Turn8<HALF> turn;
  load_vec<__bf16, 8>(k + ck, x);
  load_vec<__bf16, 8>(v + cv, y);
  turn.load(k, ck, pos, a);
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < 8; ++j) ss = __builtin_fmaf(y[j], y[j], ss);
  ss = c < a.dv ? ss : 0.f;
  ss = LPI == 8 ? sum8(ss) : sum16(ss);
  if (LPI == 32) ss += __shfl_xor(ss, 16, 64);
  const float r = a.norm_v ? 1.0f / sqrtf(ss / (float)a.dv + a.eps) : 1.0f;
  turn.apply(x, ck, a);
#pragma unroll
  for (int j = 0; j < 8; ++j) y[j] *= r;
  if (live && c < a.d) store_vec<__bf16, 8>(out + c, x);
  if (live && c < a.dv) store_vec<__bf16, 8>(out + a.d + c, y);
}

// ---- prefill, bf16, MFMA ----
// KC: 32-channel pieces of the key size; VC: 32-channel pieces of the value size (both rounded up;
// channels past the real sizes are zeros).
constexpr int kTileKeys = 64;
constexpr int kTileRows = 128;  // (token, head) rows per workgroup

__device__ __forceinline__ f32x4 mfma_bf16(bf16x8 a, bf16x8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}

template <int KC, int VC, bool HALF>
__global__ __launch_bounds__(256, KC <= 3 && VC <= 2 ? 3 : 1) void window_prefill_mfma_kernel(const WindowArgs a) {
  constexpr int D = KC * 32, DV = VC * 32;
  constexpr int KS = D + 8, VS = kTileKeys + 8;  // LDS row strides: 16-lane reads of 16 bytes meet every bank once
  __shared__ __attribute__((aligned(16))) __bf16 lds_k[kTileKeys * KS];
  __shared__ __attribute__((aligned(16))) __bf16 lds_v[DV * VS];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, quad = lane >> 4;
  const int bg = blockIdx.y, b = bg / a.G, g = bg % a.G;
  const int qpk = a.H / a.G;
  const int n_rows = a.L * qpk;
  const int r0 = blockIdx.x * kTileRows;
  const int r_end = r0 + kTileRows < n_rows ? r0 + kTileRows : n_rows;
  const int row_w = r0 + wave * 32;  // first row of this wavefront
  const __bf16* kv = static_cast<const __bf16*>(a.kv) + b * a.kv_sb + (long)g * (a.d + a.dv);

  // queries: lane holds channels quad*8 + 32 c .. of row l16 (+16): the MFMA's second operand.  Turned and
  // rounded after the first tile of keys has been asked for.
  bf16x8 qf[2][KC];
  int qpos[2], qtok[2], qhead[2];
  const __bf16* qrow[2];
#pragma unroll
  for (int t = 0; t < 2; ++t) {
    const int row = row_w + t * 16 + l16;
    const int rr = row < n_rows ? row : n_rows - 1;
    qtok[t] = rr / qpk;
    qhead[t] = g * qpk + rr % qpk;
    qpos[t] = a.pos_host + qtok[t];
    qrow[t] = static_cast<const __bf16*>(a.q) + b * a.q_sb + qtok[t] * a.q_sl + (long)qhead[t] * a.d;
#pragma unroll
    for (int c = 0; c < KC; ++c) {
      const int e = c * 32 + quad * 8;
      qf[t][c] = *reinterpret_cast<const bf16x8*>(qrow[t] + (e < a.d ? e : 0));
    }
  }
  const int wave_lo_tok = a.pos_host + (row_w < n_rows ? row_w : n_rows - 1) / qpk;
  const int wave_hi_row = row_w + 31 < n_rows ? row_w + 31 : n_rows - 1;
  const int wave_hi_tok = a.pos_host + wave_hi_row / qpk;

  f32x4 acc[2][2 * VC];
#pragma unroll
  for (int t = 0; t < 2; ++t)
#pragma unroll
    for (int i = 0; i < 2 * VC; ++i) acc[t][i] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m_run[2] = {-INFINITY, -INFINITY}, l_run[2] = {0.f, 0.f};
  const float scale2 = fabsf(a.scale) * 1.4426950408889634f;  // scores in powers of two; the sign is the queries'

  const int first_pos = a.pos_host + r0 / qpk, last_pos = a.pos_host + (r_end - 1) / qpk;
  const int lo = first_pos - a.window + 1 > 0 ? first_pos - a.window + 1 : 0;

  // staging: keys as 16-byte pieces of rows; values as 4 keys x 8 channels, turned on the way
  constexpr int KP = kTileKeys * (D / 8) / 256;  // pieces per thread
  constexpr int VP = 16 * (DV / 8) / 256 > 0 ? 16 * (DV / 8) / 256 : 1;
  typedef __attribute__((ext_vector_type(4))) uint32_t u32x4;
  u32x4 kbuf[KP];
  u32x4 vbuf[VP][4];
  const u32x4 zero4 = {0u, 0u, 0u, 0u};
  // rows past the last key and channels past the sizes are fetched from valid places and cleared in `stage`
  const int st32 = (int)a.kv_st;
  auto fetch = [&](int k0) {
    const __bf16* tile = kv + (long)k0 * a.kv_st;
    const int last = last_pos - k0;
#pragma unroll
    for (int i = 0; i < KP; ++i) {
      const int p = i * 256 + tid, key = p / (D / 8), e = (p % (D / 8)) * 8;
      kbuf[i] = *reinterpret_cast<const u32x4*>(tile + ((key <= last ? key : last) * st32 + (e < a.d ? e : 0)));
    }
#pragma unroll
    for (int i = 0; i < VP; ++i) {
      const int p = i * 256 + tid, k4 = p & 15, e = (p >> 4) * 8;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = k4 * 4 + r;
        vbuf[i][r] = *reinterpret_cast<const u32x4*>(tile + ((key <= last ? key : last) * st32 + a.d + (e < a.dv ? e : 0)));
      }
    }
  };
  auto stage = [&]() {
#pragma unroll
    for (int i = 0; i < KP; ++i) {
      const int p = i * 256 + tid, key = p / (D / 8), e = (p % (D / 8)) * 8;
      *reinterpret_cast<u32x4*>(&lds_k[key * KS + e]) = e < a.d ? kbuf[i] : zero4;
    }
#pragma unroll
    for (int i = 0; i < VP; ++i) {
      const int p = i * 256 + tid, k4 = p & 15, e = (p >> 4) * 8;
      if (e < DV) {
#pragma unroll
        for (int r = 0; r < 4; ++r) vbuf[i][r] = e < a.dv ? vbuf[i][r] : zero4;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          bf16x4 col;
#pragma unroll
          for (int r = 0; r < 4; ++r) col[r] = __builtin_bit_cast(bf16x8, vbuf[i][r])[j];
          *reinterpret_cast<bf16x4*>(&lds_v[(e + j) * VS + k4 * 4]) = col;
        }
      }
    }
  };

  fetch(lo);
  if (a.rot > 0) {
    constexpr int CB = KC == 3 ? 1 : KC < 4 ? KC : 4;
#pragma unroll
    for (int c0 = 0; c0 < KC; c0 += CB) {
      Turn8<HALF> turn[2][CB];
#pragma unroll
      for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int c = 0; c < CB; ++c) turn[t][c].load(qrow[t], (c0 + c) * 32 + quad * 8, qpos[t], a);
#pragma unroll
      for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int c = 0; c < CB; ++c) {
          float x[8];
#pragma unroll
          for (int j = 0; j < 8; ++j) x[j] = to_f32(qf[t][c0 + c][j]);
          turn[t][c].apply(x, (c0 + c) * 32 + quad * 8, a);
#pragma unroll
          for (int j = 0; j < 8; ++j) qf[t][c0 + c][j] = (__bf16)x[j];
        }
    }
  }
  if (a.scale < 0.f) {
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int c = 0; c < KC; ++c)
#pragma unroll
        for (int j = 0; j < 8; ++j) qf[t][c][j] = -qf[t][c][j];
  }
  if (D > a.d) {
#pragma unroll
    for (int c = 0; c < KC; ++c)
      if (c * 32 + quad * 8 >= a.d) {
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
          for (int j = 0; j < 8; ++j) qf[t][c][j] = (__bf16)0.f;
      }
  }
  for (int k0 = lo; k0 <= last_pos; k0 += kTileKeys) {
    __syncthreads();  // every wavefront is done with the tile before
    stage();
    __syncthreads();
    if (k0 + kTileKeys <= last_pos) fetch(k0 + kTileKeys);
#pragma unroll
    for (int h = 0; h < 2; ++h) {
      // 32 keys at a time: does any row of this wavefront see one of them, does every row see all?
      const int kh = k0 + h * 32;
      if (kh > wave_hi_tok || kh + 31 <= wave_lo_tok - a.window) continue;
      const bool all = kh + 31 <= wave_lo_tok && kh > wave_hi_tok - a.window;
      f32x4 s[2][2];
#pragma unroll
      for (int kt = 0; kt < 2; ++kt) {
#pragma unroll
        for (int t = 0; t < 2; ++t) s[t][kt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int c = 0; c < KC; ++c) {
          const bf16x8 kf = *reinterpret_cast<const bf16x8*>(&lds_k[(h * 32 + kt * 16 + l16) * KS + c * 32 + quad * 8]);
#pragma unroll
          for (int t = 0; t < 2; ++t) s[t][kt] = mfma_bf16(kf, qf[t][c], s[t][kt]);
        }
      }
      bf16x8 pf[2];
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        float mx = -INFINITY;
        const int d0 = qpos[t] - kh - quad * 4;
#pragma unroll
        for (int kt = 0; kt < 2; ++kt)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            float sc = s[t][kt][i];
            if (!all) sc = (unsigned)(d0 - kt * 16 - i) < (unsigned)a.window ? sc : -INFINITY;
            s[t][kt][i] = sc;
            mx = fmaxf(mx, sc);
          }
        mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
        mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
        if (__any(mx > m_run[t])) {
          const float m_new = fmaxf(m_run[t], mx);
          // no key seen yet: every weight is 2^-inf = 0
          const float alpha = __builtin_amdgcn_exp2f((m_run[t] - (m_new == -INFINITY ? 0.f : m_new)) * scale2);
          m_run[t] = m_new;
          l_run[t] *= alpha;
#pragma unroll
          for (int i = 0; i < 2 * VC; ++i) acc[t][i] *= alpha;
        }
        const float m2 = m_run[t] == -INFINITY ? 0.f : m_run[t] * scale2;
        float sum = 0.f;
#pragma unroll
        for (int kt = 0; kt < 2; ++kt)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const float p = __builtin_amdgcn_exp2f(__builtin_fmaf(s[t][kt][i], scale2, -m2));
            sum += p;
            pf[t][kt * 4 + i] = (__bf16)p;
          }
        l_run[t] += sum;  // this lane's keys; the four lane groups are added at the end
      }
#pragma unroll
      for (int i = 0; i < 2 * VC; ++i) {
        const __bf16* vp = &lds_v[(i * 16 + l16) * VS + h * 32 + quad * 4];
        const bf16x4 v0 = *reinterpret_cast<const bf16x4*>(vp), v1 = *reinterpret_cast<const bf16x4*>(vp + 16);
        const bf16x8 vf = __builtin_shufflevector(v0, v1, 0, 1, 2, 3, 4, 5, 6, 7);
#pragma unroll
        for (int t = 0; t < 2; ++t) acc[t][i] = mfma_bf16(vf, pf[t], acc[t][i]);
      }
    }
  }
#pragma unroll
  for (int t = 0; t < 2; ++t) {
    float l = l_run[t];
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    const float inv = a.out_scale / l;
    if (row_w + t * 16 + l16 < n_rows) {
      __bf16* op = static_cast<__bf16*>(a.o) + b * a.o_sb + qtok[t] * a.o_sl + (long)qhead[t] * a.dv;
#pragma unroll
      for (int i = 0; i < 2 * VC; ++i) {
        const int e = i * 16 + quad * 4;
        if (e < a.dv) {
          bf16x4 o;
#pragma unroll
          for (int j = 0; j < 4; ++j) o[j] = (__bf16)(acc[t][i][j] * inv);
          *reinterpret_cast<bf16x4*>(op + e) = o;
        }
      }
    }
  }
}

// ---- prefill, any element type and any sizes: one wavefront per (token, query head) ----
constexpr int kAnyMaxDim = 512;  // largest key / value size

template <typename T>
__global__ __launch_bounds__(64) void window_prefill_any_kernel(const WindowArgs a) {
  __shared__ float qs[kAnyMaxDim];
  __shared__ float ps[64];
  const int lane = threadIdx.x, l = blockIdx.x, h = blockIdx.y, b = blockIdx.z;
  const int g = h / (a.H / a.G), pos = a.pos_host + l;
  const T* q = static_cast<const T*>(a.q) + b * a.q_sb + l * a.q_sl + (long)h * a.d;
  const T* kv = static_cast<const T*>(a.kv) + b * a.kv_sb + (long)g * (a.d + a.dv);
  for (int c = lane; c < a.d; c += 64) qs[c] = round_to<T>(rotated(q, c, pos, a));
  float acc[kAnyMaxDim / 64];
#pragma unroll
  for (int i = 0; i < kAnyMaxDim / 64; ++i) acc[i] = 0.f;
  float m_run = -INFINITY, l_run = 0.f;
  const int lo = pos - a.window + 1 > 0 ? pos - a.window + 1 : 0;
  __syncthreads();
  for (int k0 = lo; k0 <= pos; k0 += 64) {
    const int key = k0 + lane;
    float s = -INFINITY;
    if (key <= pos) {
      const T* kr = kv + (long)key * a.kv_st;
      float dot = 0.f;
      for (int c = 0; c < a.d; ++c) dot = __builtin_fmaf(qs[c], to_f32(kr[c]), dot);
      s = dot * a.scale;
    }
    float mx = s;
#pragma unroll
    for (int m = 32; m >= 1; m >>= 1) mx = fmaxf(mx, __shfl_xor(mx, m, 64));
    const float m_new = fmaxf(m_run, mx);
    const float alpha = expf(m_run - m_new), p = expf(s - m_new);
    m_run = m_new;
    l_run = l_run * alpha + wave_sum(p);
    __syncthreads();
    ps[lane] = p;
    __syncthreads();
    const int n = pos - k0 + 1 < 64 ? pos - k0 + 1 : 64;
#pragma unroll
    for (int i = 0; i < kAnyMaxDim / 64; ++i) {
      const int c = i * 64 + lane;
      if (c < a.dv) {
        float v = acc[i] * alpha;
        for (int j = 0; j < n; ++j) v = __builtin_fmaf(ps[j], to_f32(kv[(long)(k0 + j) * a.kv_st + a.d + c]), v);
        acc[i] = v;
      }
    }
  }
  T* o = static_cast<T*>(a.o) + b * a.o_sb + l * a.o_sl + (long)h * a.dv;
  const float inv = a.out_scale / l_run;
#pragma unroll
  for (int i = 0; i < kAnyMaxDim / 64; ++i) {
    const int c = i * 64 + lane;
    if (c < a.dv) o[c] = from_f32<T>(acc[i] * inv);
  }
}

// ---- one token per sequence ----
constexpr int kStepThreads = 256;
constexpr int kStepKeys = 256;  // keys per round of the running softmax

template <typename T, int N> struct RawPiece {
  typedef typename Pack<T>::type type;
  static __device__ __forceinline__ float get(type x, int i) { return to_f32(x[i]); }
};
template <typename T> struct RawPiece<T, 1> {
  typedef T type;
  static __device__ __forceinline__ float get(type x, int) { return to_f32(x); }
};

// QT: query heads of the group served together (the group is walked QT heads at a time).
// VEC: 16-byte pieces of the rows (sizes and strides multiples of the piece); otherwise element by element.
template <typename T, int QT, bool VEC>
__global__ __launch_bounds__(kStepThreads) void window_step_kernel(const WindowArgs a, int part_floats) {
  constexpr int N = VEC ? Pack<T>::kN : 1;
  extern __shared__ float smem[];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int b = blockIdx.x / a.G, g = blockIdx.x % a.G;
  const int qpk = a.H / a.G;
  const int pos = row_pos(a.pos, a.pos_host, b);
  if (pos < 0 || pos >= a.S || (a.rot > 0 && pos >= a.n_pos)) return;  // a position the cache does not hold
  float* qs = smem;                        // [QT][d]
  float* sc = qs + QT * a.d;               // [QT][kStepKeys]
  float* stat = sc + QT * kStepKeys;       // [3][QT]: running maximum, running sum, rescale of the current keys
  float* part = stat + 3 * QT;             // [QT][parts][vp2 * N], partial outputs
  float* knew = part + part_floats;        // [d] and [dv]: the row of the new token, as the cache holds it
  float* vnew = knew + a.d;
  const T* k = static_cast<const T*>(a.k) + b * a.k_sb + (long)g * a.d;
  const T* v = static_cast<const T*>(a.v) + b * a.v_sb + (long)g * a.dv;
  T* kv = static_cast<T*>(a.kv) + b * a.kv_sb + (long)g * (a.d + a.dv);
  const int lo = pos - a.window + 1 > 0 ? pos - a.window + 1 : 0;
  // lanes per key: the smallest power of two that covers the row in N-element pieces, 64 at most
  const int pieces = (a.d + N - 1) / N;
  int lpk = 1;
  while (lpk < pieces && lpk < 64) lpk <<= 1;
  const int keys_at_once = kStepThreads / lpk, my_key = tid / lpk, my_piece = tid % lpk;
  // lanes per value row, likewise; then the partial sums that are left for LDS
  int vp2 = 1;
  while (vp2 * N < a.dv) vp2 <<= 1;  // <= kStepThreads
  const int v_groups = kStepThreads / vp2, my_vp = tid % vp2, my_vg = tid / vp2;
  const int parts = vp2 < 64 ? kStepThreads / 64 : v_groups, my_part = vp2 < 64 ? wave : my_vg;
  const bool v_in = my_vp * N < a.dv;
  constexpr int KU = 4;  // rows whose loads are in flight together
  typedef typename RawPiece<T, N>::type raw_t;
  auto load_row = [&](int j, int n, int first, int piece, int k0) -> raw_t {
    return *reinterpret_cast<const raw_t*>(kv + (long)(k0 + (j < n ? j : n - 1)) * a.kv_st + first + piece * N);
  };
  // the first rows of the cache are asked for before anything else; the new token's row is not in it yet
  // and is taken from LDS
  const int n_first = pos - lo + 1 < kStepKeys ? pos - lo + 1 : kStepKeys;
  const int kp = my_piece < pieces ? my_piece : 0, vp = v_in ? my_vp : 0;
  raw_t xk[KU], xv[KU];
#pragma unroll
  for (int u = 0; u < KU; ++u) xk[u] = load_row(u * keys_at_once + my_key, n_first, 0, kp, lo);
#pragma unroll
  for (int u = 0; u < KU; ++u) xv[u] = load_row(u * v_groups + my_vg, n_first, a.d, vp, lo);
  {
    T* out = kv + (long)pos * a.kv_st;
    if (wave == 0) {
      float ss = 0.f;
      for (int c = lane; c < a.dv; c += 64) ss = __builtin_fmaf(to_f32(v[c]), to_f32(v[c]), ss);
      const float r = a.norm_v ? 1.0f / sqrtf(wave_sum(ss) / (float)a.dv + a.eps) : 1.0f;
      for (int c = lane; c < a.dv; c += 64) {
        const T x = from_f32<T>(to_f32(v[c]) * r);
        out[a.d + c] = x;
        vnew[c] = to_f32(x);
      }
    } else {
      for (int c = tid - 64; c < a.d; c += kStepThreads - 64) {
        const T x = from_f32<T>(rotated(k, c, pos, a));
        out[c] = x;
        knew[c] = to_f32(x);
      }
    }
  }

  for (int h0 = 0; h0 < qpk; h0 += QT) {
    if (h0 > 0) __syncthreads();  // the round before is done with LDS
    for (int i = tid; i < QT * a.d; i += kStepThreads) {
      const int hh = i / a.d, c = i % a.d;
      const int h = g * qpk + (h0 + hh < qpk ? h0 + hh : h0);
      const T* q = static_cast<const T*>(a.q) + b * a.q_sb + (long)h * a.d;
      qs[i] = round_to<T>(rotated(q, c, pos, a));
    }
    if (tid < QT) {
      stat[tid] = -INFINITY;
      stat[QT + tid] = 0.f;
    }
    __syncthreads();
    float qr[QT][N];  // this lane's piece of every query
#pragma unroll
    for (int hh = 0; hh < QT; ++hh)
#pragma unroll
      for (int i = 0; i < N; ++i) qr[hh][i] = my_piece < pieces ? qs[hh * a.d + (my_piece < pieces ? my_piece : 0) * N + i] : 0.f;
    float acc[QT][N];
#pragma unroll
    for (int hh = 0; hh < QT; ++hh)
#pragma unroll
      for (int i = 0; i < N; ++i) acc[hh][i] = 0.f;
    for (int k0 = lo; k0 <= pos; k0 += kStepKeys) {
      const int n = pos - k0 + 1 < kStepKeys ? pos - k0 + 1 : kStepKeys;
      if (k0 > lo) __syncthreads();
      // the pieces of row j as floats; the last row of all is the new token's
      auto floats = [&](raw_t x, const float* fresh, int piece, int j, float (&f)[N]) {
        const bool is_new = k0 + j == pos;
#pragma unroll
        for (int i = 0; i < N; ++i) {
          const float nv = fresh[piece * N + i], ov = RawPiece<T, N>::get(x, i);
          f[i] = is_new ? nv : ov;
        }
      };
      const bool first = h0 == 0 && k0 == lo;
      for (int j0 = 0; j0 < n; j0 += KU * keys_at_once) {
        if (!first || j0 > 0) {
#pragma unroll
          for (int u = 0; u < KU; ++u) xk[u] = load_row(j0 + u * keys_at_once + my_key, n, 0, kp, k0);
        }
#pragma unroll
        for (int u = 0; u < KU; ++u) {
          const int j = j0 + u * keys_at_once + my_key;
          float f[N];
          floats(xk[u], knew, kp, j, f);
          float dot[QT];
#pragma unroll
          for (int hh = 0; hh < QT; ++hh) {
            dot[hh] = 0.f;
#pragma unroll
            for (int i = 0; i < N; ++i) dot[hh] = __builtin_fmaf(f[i], qr[hh][i], dot[hh]);
          }
          for (int p = my_piece + lpk; p < pieces; p += lpk) {  // rows of more than 64 pieces
            float y[N];
            floats(load_row(j, n, 0, p, k0), knew, p, j, y);
#pragma unroll
            for (int hh = 0; hh < QT; ++hh)
#pragma unroll
              for (int i = 0; i < N; ++i) dot[hh] = __builtin_fmaf(y[i], qs[hh * a.d + p * N + i], dot[hh]);
          }
#pragma unroll
          for (int hh = 0; hh < QT; ++hh) {
            if (lpk == 8) {
              dot[hh] = sum8(dot[hh]);
            } else if (lpk == 16) {
              dot[hh] = sum16(dot[hh]);
            } else {
              for (int m = 1; m < lpk; m <<= 1) dot[hh] += __shfl_xor(dot[hh], m, 64);
            }
            if (my_piece == 0 && j < n) sc[hh * kStepKeys + j] = dot[hh] * a.scale;
          }
        }
      }
      if (!first) {
        // the first value rows are on their way during the softmax
#pragma unroll
        for (int u = 0; u < KU; ++u) xv[u] = load_row(my_vg + u * v_groups, n, a.d, vp, k0);
      }
      __syncthreads();
      for (int hh = wave; hh < QT; hh += kStepThreads / 64) {
        float s[kStepKeys / 64], mx = -INFINITY;
#pragma unroll
        for (int i = 0; i < kStepKeys / 64; ++i) {
          const int j = i * 64 + lane;
          s[i] = j < n ? sc[hh * kStepKeys + j] : -INFINITY;
          mx = fmaxf(mx, s[i]);
        }
#pragma unroll
        for (int m = 32; m >= 1; m >>= 1) mx = fmaxf(mx, __shfl_xor(mx, m, 64));
        const float m_old = stat[hh], m_new = fmaxf(m_old, mx);
        float sum = 0.f;
#pragma unroll
        for (int i = 0; i < kStepKeys / 64; ++i) {
          const float p = expf(s[i] - m_new);
          sc[hh * kStepKeys + i * 64 + lane] = p;
          sum += p;
        }
        sum = wave_sum(sum);
        const float alpha = expf(m_old - m_new);
        if (lane == 0) {
          stat[hh] = m_new;
          stat[QT + hh] = stat[QT + hh] * alpha + sum;
          stat[2 * QT + hh] = alpha;
        }
      }
      __syncthreads();
      if (k0 > lo) {
#pragma unroll
        for (int hh = 0; hh < QT; ++hh)
#pragma unroll
          for (int i = 0; i < N; ++i) acc[hh][i] *= stat[2 * QT + hh];
      }
      for (int j0 = my_vg; j0 < n; j0 += KU * v_groups) {
        if (j0 != my_vg) {
#pragma unroll
          for (int u = 0; u < KU; ++u) xv[u] = load_row(j0 + u * v_groups, n, a.d, vp, k0);
        }
#pragma unroll
        for (int u = 0; u < KU; ++u) {
          const int j = j0 + u * v_groups;
          float f[N];
          floats(xv[u], vnew, vp, j, f);
#pragma unroll
          for (int hh = 0; hh < QT; ++hh) {
            const float p = j < n ? sc[hh * kStepKeys + j] : 0.f;
#pragma unroll
            for (int i = 0; i < N; ++i) acc[hh][i] = j < n ? __builtin_fmaf(p, f[i], acc[hh][i]) : acc[hh][i];
          }
        }
      }
    }
#pragma unroll
    for (int hh = 0; hh < QT; ++hh) {
      for (int m = vp2; m < 64; m <<= 1) {
#pragma unroll
        for (int i = 0; i < N; ++i) acc[hh][i] += __shfl_xor(acc[hh][i], m, 64);
      }
      if (vp2 >= 64 || lane < vp2) {
#pragma unroll
        for (int i = 0; i < N; ++i) part[((hh * parts + my_part) * vp2 + my_vp) * N + i] = acc[hh][i];
      }
    }
    __syncthreads();
    for (int i = tid; i < QT * a.dv; i += kStepThreads) {
      const int hh = i / a.dv, c = i % a.dv;
      if (h0 + hh < qpk) {
        float s = 0.f;
        for (int p = 0; p < parts; ++p) s += part[(hh * parts + p) * vp2 * N + c];
        T* o = static_cast<T*>(a.o) + b * a.o_sb + (long)(g * qpk + h0 + hh) * a.dv;
        o[c] = from_f32<T>(s * (a.out_scale / stat[QT + hh]));
      }
    }
  }
}

// The same for bf16 rows of whole 16-byte pieces: queries, the new key and the new value are turned and
// normalised in the registers of the lanes that use them, the new token starts the running softmax, and the
// cached keys before it follow, so that everything the launch reads is asked for at its start and a window
// of w needs w - 1 rows.  Products of queries and keys are dot-product instructions on bf16 pairs.
// LPK, VP2: lanes per key row and per value row (powers of two), 0: whatever the sizes ask for.
template <int QT, bool HALF, int LPK, int VP2>
__global__ __launch_bounds__(kStepThreads) void window_step_vec_kernel(const WindowArgs a) {
  constexpr int N = 8, KU = 4;
  extern __shared__ float smem[];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int b = blockIdx.x / a.G, g = blockIdx.x % a.G;
  const int qpk = a.H / a.G;
  const int pos = row_pos(a.pos, a.pos_host, b);
  if (pos < 0 || pos >= a.S || (a.rot > 0 && pos >= a.n_pos)) return;  // a position the cache does not hold
  float* sc = smem;                   // [QT][kStepKeys]
  float* stat = sc + QT * kStepKeys;  // [3][QT]: running maximum, running sum, rescale of the current keys
  float* part = stat + 3 * QT;        // [QT][parts][vp2 * 8], partial outputs
  const __bf16* k = static_cast<const __bf16*>(a.k) + b * a.k_sb + (long)g * a.d;
  const __bf16* v = static_cast<const __bf16*>(a.v) + b * a.v_sb + (long)g * a.dv;
  __bf16* kv = static_cast<__bf16*>(a.kv) + b * a.kv_sb + (long)g * (a.d + a.dv);
  const int lo = pos - a.window + 1 > 0 ? pos - a.window + 1 : 0;
  const int old = pos - lo;  // cached keys this token sees
  int lpk = LPK, vp2 = VP2;
  if constexpr (LPK == 0) {
    lpk = 1;
    while (lpk * N < a.d) lpk <<= 1;
  }
  if constexpr (VP2 == 0) {
    vp2 = 1;
    while (vp2 * N < a.dv) vp2 <<= 1;
  }
  const int keys_at_once = kStepThreads / lpk, my_key = tid / lpk, my_piece = tid % lpk;
  const int v_groups = kStepThreads / vp2, my_vp = tid % vp2, my_vg = tid / vp2;
  const int parts = kStepThreads / 64;
  const bool k_in = my_piece * N < a.d, v_in = my_vp * N < a.dv;
  const int ke = k_in ? my_piece * N : 0, ve = v_in ? my_vp * N : 0;
  const int st32 = (int)a.kv_st;
  auto row = [&](int k0, int j, int n) { return kv + (long)k0 * a.kv_st + (n > 0 ? (j < n ? j : n - 1) : 0) * st32; };

  const int n_first = old < kStepKeys ? old : kStepKeys;
  bf16x8 xk[KU], xv[KU], qraw[QT];
#pragma unroll
  for (int u = 0; u < KU; ++u) xk[u] = *reinterpret_cast<const bf16x8*>(row(lo, u * keys_at_once + my_key, n_first) + ke);
#pragma unroll
  for (int u = 0; u < KU; ++u) xv[u] = *reinterpret_cast<const bf16x8*>(row(lo, u * v_groups + my_vg, n_first) + a.d + ve);
  auto q_row = [&](int hh) { return static_cast<const __bf16*>(a.q) + b * a.q_sb + (long)(g * qpk + (hh < qpk ? hh : qpk - 1)) * a.d; };
#pragma unroll
  for (int hh = 0; hh < QT; ++hh) qraw[hh] = *reinterpret_cast<const bf16x8*>(q_row(hh) + ke);
  const bf16x8 knew_raw = *reinterpret_cast<const bf16x8*>(k + ke), vnew_raw = *reinterpret_cast<const bf16x8*>(v + ve);
  Turn8<HALF> turn;
  turn.load(k, ke, pos, a);

  // the new value: normalised by the lanes that share the row
  float vn[N];
  {
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < N; ++i) {
      vn[i] = v_in ? to_f32(vnew_raw[i]) : 0.f;
      ss = __builtin_fmaf(vn[i], vn[i], ss);
    }
    if constexpr (VP2 == 8) {
      ss = sum8(ss);
    } else if constexpr (VP2 == 16) {
      ss = sum16(ss);
    } else {
      for (int m = 1; m < vp2; m <<= 1) ss += __shfl_xor(ss, m, 64);
    }
    const float r = a.norm_v ? 1.0f / sqrtf(ss / (float)a.dv + a.eps) : 1.0f;
    bf16x8 o;
#pragma unroll
    for (int i = 0; i < N; ++i) {
      o[i] = (__bf16)(vn[i] * r);
      vn[i] = to_f32(o[i]);
    }
    if (my_vg == 0 && v_in) *reinterpret_cast<bf16x8*>(kv + (long)pos * a.kv_st + a.d + ve) = o;
  }
  typedef __attribute__((ext_vector_type(4))) uint32_t u32x4;
  auto turned = [&](bf16x8 raw, const Turn8<HALF>& t) -> u32x4 {
    float x[N];
#pragma unroll
    for (int i = 0; i < N; ++i) x[i] = to_f32(raw[i]);
    t.apply(x, ke, a);
    bf16x8 y;
#pragma unroll
    for (int i = 0; i < N; ++i) y[i] = (__bf16)(k_in ? x[i] : 0.f);
    return __builtin_bit_cast(u32x4, y);
  };
  const u32x4 knew = turned(knew_raw, turn);
  if (my_key == 0 && k_in) *reinterpret_cast<u32x4*>(kv + (long)pos * a.kv_st + ke) = knew;
  auto dot8 = [](u32x4 x, u32x4 y) {
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const uint32_t xi = x[i], yi = y[i];  // (a bit cast of a vector's element as such takes element 0)
      s = __builtin_amdgcn_fdot2_f32_bf16(__builtin_bit_cast(bf16x2, xi), __builtin_bit_cast(bf16x2, yi), s, false);
    }
    return s;
  };
  auto over_pieces = [&](float x) {
    if constexpr (LPK == 8) {
      x = sum8(x);
    } else if constexpr (LPK == 16) {
      x = sum16(x);
    } else {
      for (int m = 1; m < lpk; m <<= 1) x += __shfl_xor(x, m, 64);
    }
    return x;
  };

  for (int h0 = 0; h0 < qpk; h0 += QT) {
    if (h0 > 0) __syncthreads();  // the round before is done with LDS
    u32x4 q[QT];
    Turn8<HALF> tq = turn;
    if (h0 > 0) {
#pragma unroll
      for (int hh = 0; hh < QT; ++hh) qraw[hh] = *reinterpret_cast<const bf16x8*>(q_row(h0 + hh) + ke);
    }
#pragma unroll
    for (int hh = 0; hh < QT; ++hh) {
      if constexpr (HALF)
        load_vec<__bf16, 8>(q_row(h0 + hh) + (ke < a.rot ? (ke < a.rot / 2 ? ke + a.rot / 2 : ke - a.rot / 2) : 0), tq.partner);
      q[hh] = turned(qraw[hh], tq);
    }
    // the new token: maximum = its score, weight 1
    float s_new[QT], acc[QT][N];
#pragma unroll
    for (int hh = 0; hh < QT; ++hh) {
      s_new[hh] = over_pieces(dot8(knew, q[hh])) * a.scale;
#pragma unroll
      for (int i = 0; i < N; ++i) acc[hh][i] = my_vg == 0 ? vn[i] : 0.f;
      if (tid == 0) {
        stat[hh] = s_new[hh];
        stat[QT + hh] = 1.f;
      }
    }
    for (int k0 = lo; k0 < pos; k0 += kStepKeys) {
      const int n = pos - k0 < kStepKeys ? pos - k0 : kStepKeys;
      const bool first = h0 == 0 && k0 == lo;
      if (k0 > lo) __syncthreads();
      for (int j0 = 0; j0 < n; j0 += KU * keys_at_once) {
        if (!first || j0 > 0) {
#pragma unroll
          for (int u = 0; u < KU; ++u) xk[u] = *reinterpret_cast<const bf16x8*>(row(k0, j0 + u * keys_at_once + my_key, n) + ke);
        }
#pragma unroll
        for (int u = 0; u < KU; ++u) {
          const int j = j0 + u * keys_at_once + my_key;
#pragma unroll
          for (int hh = 0; hh < QT; ++hh) {
            const float s = over_pieces(dot8(__builtin_bit_cast(u32x4, xk[u]), q[hh]));
            if (my_piece == 0 && j < n) sc[hh * kStepKeys + j] = s * a.scale;
          }
        }
      }
      if (!first) {
        // the first value rows are on their way during the softmax
#pragma unroll
        for (int u = 0; u < KU; ++u) xv[u] = *reinterpret_cast<const bf16x8*>(row(k0, u * v_groups + my_vg, n) + a.d + ve);
      }
      __syncthreads();
      for (int hh = wave; hh < QT; hh += kStepThreads / 64) {
        float s[kStepKeys / 64], mx = -INFINITY;
#pragma unroll
        for (int i = 0; i < kStepKeys / 64; ++i) {
          const int j = i * 64 + lane;
          const float x = sc[hh * kStepKeys + j];
          s[i] = j < n ? x : -INFINITY;
          mx = fmaxf(mx, s[i]);
        }
#pragma unroll
        for (int m = 32; m >= 1; m >>= 1) mx = fmaxf(mx, __shfl_xor(mx, m, 64));
        const float m_old = stat[hh], m_new = fmaxf(m_old, mx);
        float sum = 0.f;
#pragma unroll
        for (int i = 0; i < kStepKeys / 64; ++i) {
          const float p = exp_f(s[i] - m_new);
          sc[hh * kStepKeys + i * 64 + lane] = p;
          sum += p;
        }
        sum = wave_sum(sum);
        const float alpha = exp_f(m_old - m_new);
        if (lane == 0) {
          stat[hh] = m_new;
          stat[QT + hh] = stat[QT + hh] * alpha + sum;
          stat[2 * QT + hh] = alpha;
        }
      }
      __syncthreads();
#pragma unroll
      for (int hh = 0; hh < QT; ++hh) {
        const float alpha = stat[2 * QT + hh];
#pragma unroll
        for (int i = 0; i < N; ++i) acc[hh][i] *= alpha;
      }
      for (int j0 = my_vg; j0 < n; j0 += KU * v_groups) {
        if (j0 != my_vg) {
#pragma unroll
          for (int u = 0; u < KU; ++u) xv[u] = *reinterpret_cast<const bf16x8*>(row(k0, j0 + u * v_groups, n) + a.d + ve);
        }
#pragma unroll
        for (int u = 0; u < KU; ++u) {
          const int j = j0 + u * v_groups;
#pragma unroll
          for (int hh = 0; hh < QT; ++hh) {
            const float p = j < n ? sc[hh * kStepKeys + (j < n ? j : 0)] : 0.f;
#pragma unroll
            for (int i = 0; i < N; ++i) acc[hh][i] = __builtin_fmaf(p, to_f32(xv[u][i]), acc[hh][i]);
          }
        }
      }
    }
#pragma unroll
    for (int hh = 0; hh < QT; ++hh) {
      if constexpr (VP2 != 0) {
#pragma unroll
        for (int m = VP2; m < 64; m <<= 1)
#pragma unroll
          for (int i = 0; i < N; ++i) acc[hh][i] += __shfl_xor(acc[hh][i], m, 64);
      } else {
        for (int m = vp2; m < 64; m <<= 1) {
#pragma unroll
          for (int i = 0; i < N; ++i) acc[hh][i] += __shfl_xor(acc[hh][i], m, 64);
        }
      }
      if (lane < vp2) {
#pragma unroll
        for (int i = 0; i < N; ++i) part[((hh * parts + wave) * vp2 + my_vp) * N + i] = acc[hh][i];
      }
    }
    __syncthreads();
#pragma unroll
    for (int hh = 0; hh < QT; ++hh) {
      if (h0 + hh < qpk) {
        const float inv = a.out_scale / stat[QT + hh];
        for (int c = tid; c < a.dv; c += kStepThreads) {
          float s = 0.f;
#pragma unroll
          for (int p = 0; p < kStepThreads / 64; ++p) s += part[(hh * parts + p) * vp2 * N + c];
          static_cast<__bf16*>(a.o)[b * a.o_sb + (long)(g * qpk + h0 + hh) * a.dv + c] = (__bf16)(s * inv);
        }
      }
    }
  }
}

template <bool HALF, int LPK, int VP2> void launch_window_step_lanes(const WindowArgs& a, int vp2, hipStream_t s) {
  const int qpk = a.H / a.G;
  const dim3 grid((unsigned)(a.B * a.G)), block(kStepThreads);
  auto bytes = [&](int qt) { return (size_t)qt * (kStepKeys + 3 + kStepThreads / 64 * vp2 * 8) * sizeof(float); };
  if (qpk == 1)
    hipLaunchKernelGGL((window_step_vec_kernel<1, HALF, LPK, VP2>), grid, block, bytes(1), s, a);
  else if (qpk == 2)
    hipLaunchKernelGGL((window_step_vec_kernel<2, HALF, LPK, VP2>), grid, block, bytes(2), s, a);
  else if (qpk <= 4 || bytes(8) > 64 * 1024)
    hipLaunchKernelGGL((window_step_vec_kernel<4, HALF, LPK, VP2>), grid, block, bytes(4), s, a);
  else
    hipLaunchKernelGGL((window_step_vec_kernel<8, HALF, LPK, VP2>), grid, block, bytes(8), s, a);
}

template <bool HALF> void launch_window_step_vec(const WindowArgs& a, hipStream_t s) {
  int lpk = 1, vp2 = 1;
  while (lpk * 8 < a.d) lpk <<= 1;
  while (vp2 * 8 < a.dv) vp2 <<= 1;
  if (lpk == 8 && vp2 == 8)
    launch_window_step_lanes<HALF, 8, 8>(a, vp2, s);
  else if (lpk == 8 && vp2 == 16)
    launch_window_step_lanes<HALF, 8, 16>(a, vp2, s);
  else if (lpk == 16 && vp2 == 16)
    launch_window_step_lanes<HALF, 16, 16>(a, vp2, s);
  else
    launch_window_step_lanes<HALF, 0, 0>(a, vp2, s);
}

template <typename T, bool VEC> void launch_window_step(const WindowArgs& a, hipStream_t s) {
  const int qpk = a.H / a.G;
  const dim3 grid((unsigned)(a.B * a.G)), block(kStepThreads);
  constexpr int N = VEC ? Pack<T>::kN : 1;
  int vp2 = 1;
  while (vp2 * N < a.dv) vp2 <<= 1;
  const int parts = vp2 < 64 ? kStepThreads / 64 : kStepThreads / vp2;
  auto part_floats = [&](int qt) { return qt * parts * vp2 * N; };
  auto bytes = [&](int qt) { return (size_t)(qt * (a.d + kStepKeys + 3) + part_floats(qt) + a.d + a.dv) * sizeof(float); };
  if (qpk == 1)
    hipLaunchKernelGGL((window_step_kernel<T, 1, VEC>), grid, block, bytes(1), s, a, part_floats(1));
  else if (qpk == 2)
    hipLaunchKernelGGL((window_step_kernel<T, 2, VEC>), grid, block, bytes(2), s, a, part_floats(2));
  else if (qpk <= 4 || bytes(8) > 64 * 1024)
    hipLaunchKernelGGL((window_step_kernel<T, 4, VEC>), grid, block, bytes(4), s, a, part_floats(4));
  else
    hipLaunchKernelGGL((window_step_kernel<T, 8, VEC>), grid, block, bytes(8), s, a, part_floats(8));
}

template <int LPI> void launch_kv_write(const WindowArgs& a, hipStream_t s) {
  const long items = (long)a.B * a.L * a.G;
  const dim3 grid((unsigned)((items + 256 / LPI - 1) / (256 / LPI)));
  if (a.half_split)
    hipLaunchKernelGGL((window_kv_write_vec_kernel<LPI, true>), grid, dim3(256), 0, s, a);
  else
    hipLaunchKernelGGL((window_kv_write_vec_kernel<LPI, false>), grid, dim3(256), 0, s, a);
}

template <int KC, int VC> void launch_window_mfma_pairs(const WindowArgs& a, dim3 grid, hipStream_t s) {
  if (a.half_split)
    hipLaunchKernelGGL((window_prefill_mfma_kernel<KC, VC, true>), grid, dim3(256), 0, s, a);
  else
    hipLaunchKernelGGL((window_prefill_mfma_kernel<KC, VC, false>), grid, dim3(256), 0, s, a);
}

template <int KC> void launch_window_mfma(const WindowArgs& a, dim3 grid, hipStream_t s) {
  const int vc = (a.dv + 31) / 32;
  if (vc <= 1)
    launch_window_mfma_pairs<KC, 1>(a, grid, s);
  else if (vc <= 2)
    launch_window_mfma_pairs<KC, 2>(a, grid, s);
  else if (vc <= 4)
    launch_window_mfma_pairs<KC, 4>(a, grid, s);
  else
    launch_window_mfma_pairs<KC, 8>(a, grid, s);
}

static int window_check(const char* who, const WindowArgs& a, int64_t n_rope, int io_dtype, int64_t last) {
  BASED_REQUIRE(a.q && a.k && a.v && a.kv && a.o, BASED_ERR_ARG, "%s: null pointer argument", who);
  BASED_REQUIRE(a.B >= 0 && a.L >= 0 && a.H > 0 && a.G > 0 && a.d > 0 && a.dv > 0 && a.S > 0, BASED_ERR_ARG, "%s: bad sizes", who);
  BASED_REQUIRE(a.H % a.G == 0, BASED_ERR_SHAPE, "%s: %d query heads do not divide into %d key/value heads", who, a.H, a.G);
  BASED_REQUIRE(a.d <= kAnyMaxDim && a.dv <= kAnyMaxDim, BASED_ERR_SHAPE, "%s: head sizes %d / %d (at most %d)", who, a.d, a.dv,
                kAnyMaxDim);
  BASED_REQUIRE(a.window > 0, BASED_ERR_ARG, "%s: window %d", who, a.window);
  BASED_REQUIRE(a.rot >= 0 && a.rot <= a.d && a.rot % 2 == 0, BASED_ERR_SHAPE, "%s: rotary size %d of %d channels", who, a.rot, a.d);
  BASED_REQUIRE(a.rot == 0 || (a.cos_t && a.sin_t), BASED_ERR_ARG, "%s: rotary tables missing", who);
  BASED_REQUIRE(io_dtype == BASED_BF16 || io_dtype == BASED_F32, BASED_ERR_DTYPE, "%s: bad dtype", who);
  BASED_REQUIRE(last < a.S, BASED_ERR_SHAPE, "%s: position %ld does not fit a cache of %d rows", who, (long)last, a.S);
  BASED_REQUIRE(a.rot == 0 || last < n_rope, BASED_ERR_SHAPE, "%s: rotary tables end before position %ld", who, (long)last);
  return BASED_OK;
}

static bool window_vec(const WindowArgs& a, int n) {
  return a.d % n == 0 && a.dv % n == 0 && a.q_sb % n == 0 && a.q_sl % n == 0 && a.k_sb % n == 0 && a.k_sl % n == 0 &&
         a.v_sb % n == 0 && a.v_sl % n == 0 && a.o_sb % n == 0 && a.o_sl % n == 0 && a.kv_sb % n == 0 && a.kv_st % n == 0 &&
         aligned_to(a.q, 16) && aligned_to(a.k, 16) && aligned_to(a.v, 16) && aligned_to(a.kv, 16) && aligned_to(a.o, 16);
}

// The attention of a portion whose keys and values are in place.
static void launch_window_attend(const WindowArgs& a, bool vec, int io_dtype, hipStream_t s) {
  if (vec) {
    const dim3 grid((unsigned)(((long)a.L * (a.H / a.G) + kTileRows - 1) / kTileRows), (unsigned)(a.B * a.G));
    const int kc = (int)((a.d + 31) / 32);
    if (kc <= 1)
      launch_window_mfma<1>(a, grid, s);
    else if (kc <= 2)
      launch_window_mfma<2>(a, grid, s);
    else if (kc <= 3)
      launch_window_mfma<3>(a, grid, s);
    else if (kc <= 4)
      launch_window_mfma<4>(a, grid, s);
    else
      launch_window_mfma<8>(a, grid, s);
  } else {
    const dim3 grid((unsigned)a.L, (unsigned)a.H, (unsigned)a.B);
    if (io_dtype == BASED_BF16)
      hipLaunchKernelGGL(window_prefill_any_kernel<__bf16>, grid, dim3(64), 0, s, a);
    else
      hipLaunchKernelGGL(window_prefill_any_kernel<float>, grid, dim3(64), 0, s, a);
  }
}

}  // namespace based

extern "C" BASED_API int based_window_attn_prefill(
    const void* q, const void* k, const void* v, void* kv_cache, void* o, int64_t start, int64_t B, int64_t L, int64_t H, int64_t G,
    int64_t D, int64_t DV, int64_t S, int64_t q_sb, int64_t q_sl, int64_t k_sb, int64_t k_sl, int64_t v_sb, int64_t v_sl,
    int64_t o_sb, int64_t o_sl, int64_t kv_sb, int64_t kv_st, int64_t window, float scale, int norm_v, float eps, float out_scale,
    const float* rope_cos, const float* rope_sin, int64_t rope_len, int64_t rotary_dim, int half_split, int io_dtype, void* stream) {
  using namespace based;
  BASED_REQUIRE(start >= 0 && start + L < (1ll << 31) && window < (1ll << 31) && L * H < (1ll << 31), BASED_ERR_SHAPE,
                "window_attn_prefill: sequence too long");
  const WindowArgs a{q,       k,       v,      kv_cache, o,        rope_cos, rope_sin, nullptr, (int)start, (int)rope_len,
                     (int)B,  (int)L,  (int)H, (int)G,   (int)D,   (int)DV,  (int)S,   q_sb,    q_sl,       k_sb,
                     k_sl,    v_sb,    v_sl,   o_sb,     o_sl,     kv_sb,    kv_st,    (int)rotary_dim, half_split, (int)window,
                     norm_v,  scale,   eps,    out_scale};
  const int rc = window_check("window_attn_prefill", a, rope_len, io_dtype, start + L - 1);
  if (rc != BASED_OK) return rc;
  BASED_REQUIRE(B * G < 65536 && B < 65536 && H < 65536, BASED_ERR_SHAPE, "window_attn_prefill: grid too large");
  if (B == 0 || L == 0) return BASED_OK;
  hipStream_t s = static_cast<hipStream_t>(stream);
  // pieces of 8 channels are turned whole: the rotary size is a multiple of 8 (16 in half-split pairs)
  const bool vec = io_dtype == BASED_BF16 && D <= 256 && DV <= 256 && rotary_dim % (half_split ? 16 : 8) == 0 && window_vec(a, 8);
  const int64_t items = B * L * G;
  BASED_REQUIRE(items < (1ll << 32), BASED_ERR_SHAPE, "window_attn_prefill: grid too large");
  if (vec) {
    const int64_t widest = D > DV ? D : DV;
    widest <= 64 ? launch_kv_write<8>(a, s) : widest <= 128 ? launch_kv_write<16>(a, s) : launch_kv_write<32>(a, s);
  } else if (io_dtype == BASED_BF16)
    hipLaunchKernelGGL(window_kv_write_kernel<__bf16>, dim3((unsigned)((items + 3) / 4)), dim3(256), 0, s, a);
  else
    hipLaunchKernelGGL(window_kv_write_kernel<float>, dim3((unsigned)((items + 3) / 4)), dim3(256), 0, s, a);
  launch_window_attend(a, vec, io_dtype, s);
  return check_launch("window_attn_prefill");
}

extern "C" BASED_API int based_window_attn_attend(const void* q, const void* kv, void* o, int64_t start, int64_t B, int64_t L, int64_t H,
                                                  int64_t G, int64_t D, int64_t DV, int64_t S, int64_t q_sb, int64_t q_sl, int64_t o_sb,
                                                  int64_t o_sl, int64_t kv_sb, int64_t kv_st, int64_t window, float scale,
                                                  float out_scale, const float* rope_cos, const float* rope_sin, int64_t rope_len,
                                                  int64_t rotary_dim, int half_split, int io_dtype, void* stream) {
  using namespace based;
  BASED_REQUIRE(start >= 0 && start + L < (1ll << 31) && window < (1ll << 31) && L * H < (1ll << 31), BASED_ERR_SHAPE,
                "window_attn_attend: sequence too long");
  // k and v are not read: the rows are there already
  const WindowArgs a{q,      q,      q,      const_cast<void*>(kv), o,       rope_cos, rope_sin, nullptr, (int)start, (int)rope_len,
                     (int)B, (int)L, (int)H, (int)G,                (int)D,  (int)DV,  (int)S,   q_sb,    q_sl,       0,
                     0,      0,      0,      o_sb,                  o_sl,    kv_sb,    kv_st,    (int)rotary_dim, half_split, (int)window,
                     0,      scale,  0.f,    out_scale};
  const int rc = window_check("window_attn_attend", a, rope_len, io_dtype, start + L - 1);
  if (rc != BASED_OK) return rc;
  BASED_REQUIRE(B * G < 65536 && B < 65536 && H < 65536, BASED_ERR_SHAPE, "window_attn_attend: grid too large");
  if (B == 0 || L == 0) return BASED_OK;
  const bool vec = io_dtype == BASED_BF16 && D <= 256 && DV <= 256 && rotary_dim % (half_split ? 16 : 8) == 0 && window_vec(a, 8);
  launch_window_attend(a, vec, io_dtype, static_cast<hipStream_t>(stream));
  return check_launch("window_attn_attend");
}

extern "C" BASED_API int based_window_attn_step(
    const void* q, const void* k, const void* v, void* kv_cache, void* o, const int32_t* pos, int64_t pos_host, int64_t B, int64_t H,
    int64_t G, int64_t D, int64_t DV, int64_t S, int64_t q_sb, int64_t k_sb, int64_t v_sb, int64_t o_sb, int64_t kv_sb,
    int64_t kv_st, int64_t window, float scale, int norm_v, float eps, float out_scale, const float* rope_cos,
    const float* rope_sin, int64_t rope_len, int64_t rotary_dim, int half_split, int io_dtype, void* stream) {
  using namespace based;
  BASED_REQUIRE(pos_host >= 0 && pos_host < (1ll << 31) && window < (1ll << 31), BASED_ERR_SHAPE, "window_attn_step: bad position");
  const WindowArgs a{q,      k,      v,      kv_cache, o,       rope_cos, rope_sin, pos,  (int)pos_host, (int)rope_len,
                     (int)B, 1,      (int)H, (int)G,   (int)D,  (int)DV,  (int)S,   q_sb, 0,             k_sb,
                     0,      v_sb,   0,      o_sb,     0,       kv_sb,    kv_st,    (int)rotary_dim, half_split, (int)window,
                     norm_v, scale,  eps,    out_scale};
  const int rc = window_check("window_attn_step", a, rope_len, io_dtype, pos != nullptr ? 0 : pos_host);
  if (rc != BASED_OK) return rc;
  BASED_REQUIRE(B * G < (1ll << 31), BASED_ERR_SHAPE, "window_attn_step: grid too large");
  const int n = io_dtype == BASED_BF16 ? 8 : 4;
  const bool vec = window_vec(a, n);
  BASED_REQUIRE(vec || DV <= kStepThreads, BASED_ERR_SHAPE, "window_attn_step: value size %ld with unaligned rows (at most %d)",
                (long)DV, kStepThreads);
  if (B == 0) return BASED_OK;
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (io_dtype == BASED_BF16 && vec && rotary_dim % (half_split ? 16 : 8) == 0)
    half_split ? launch_window_step_vec<true>(a, s) : launch_window_step_vec<false>(a, s);
  else if (io_dtype == BASED_BF16)
    vec ? launch_window_step<__bf16, true>(a, s) : launch_window_step<__bf16, false>(a, s);
  else
    vec ? launch_window_step<float, true>(a, s) : launch_window_step<float, false>(a, s);
  return check_launch("window_attn_step");
}
