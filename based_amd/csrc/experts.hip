// Mixture of experts with sigmoid routing for gfx950.  Of E small gated feed-forwards a token takes the `top`
// with the largest scores s = sigmoid(W_router h); each reads s * h, and their outputs are added:
//   y = sum_e down_e(silu(gate_e(s h)) * up_e(s h))
// (s multiplies the sums of gate and up in fp32, which is the same thing.)
//
//   expert_route    scores in fp32, the choice, and for grouped products each choice's place among its
//                   expert's rows; a single workgroup (up to 32 tokens) also does what the next two do
//   expert_plan     rows of every expert rounded up to tiles, which expert a tile belongs to, and the choices in
//                   that order
//   expert_scatter  the last part, where there are too many choices for one workgroup
//   expert_gemm     MFMA product of a tile of rows with its expert's matrices, gathered and scattered by that
//                   order: gate and up with the activation behind them, then down
//   expert_sum      the choices of a token added up (with one choice the product writes the token's row)
//   expert_route_row  the same for few tokens, with the norm in front of the layer
//   expert_rows     few tokens, fp32, or rows that are no whole 16-byte pieces: dot products, one choice at a time
#include "stream_common.hpp"

namespace based {

constexpr int kMaxExperts = 256;

struct RouteArgs {
  const void* h;  // (N, D)
  const void* w;  // (E, D)
  int32_t* ids;   // (N, top)
  float* scores;  // (N, top)
  int32_t* rank;  // (N, top) or null
  int32_t* counts;  // (E), with rank; zero on entry unless one workgroup does everything
  // one workgroup for all tokens: the plan too
  int32_t* tile_first;
  int32_t* tile_expert;
  int32_t* order;
  int tile_rows;
  long n, h_sr;
  int D, E, top;
};

__device__ __forceinline__ f32x4 expert_mfma(bf16x8 a, bf16x8 b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }

// Tiles of every expert from its count, by threads 0 .. 255; scan: 256 ints of LDS.  Called by a whole workgroup.
__device__ __forceinline__ void plan_tiles(const int* counts, int* scan, int* first_of, int32_t* tile_first, int32_t* tile_expert, int E, int tile_rows) {
  const int e = threadIdx.x;
  const int tiles = e < E ? (counts[e] + tile_rows - 1) / tile_rows : 0;
  if (e < 256) scan[e] = tiles;
  __syncthreads();
  for (int m = 1; m < 256; m <<= 1) {
    const int add = e < 256 && e >= m ? scan[e - m] : 0;
    __syncthreads();
    if (e < 256) scan[e] += add;
    __syncthreads();
  }
  if (e < E) {
    const int first = scan[e] - tiles;
    first_of[e] = first;
    tile_first[e] = first;
    for (int t = 0; t < tiles; ++t) tile_expert[first + t] = e;
  }
  if (e == 255) tile_first[E] = scan[255];
  __syncthreads();
}

// ET: tiles of 16 experts (bf16 MFMA); 0: element by element.  NW wavefronts.  SPLIT: they share 16 TT tokens, a part of the row each;
// otherwise 16 tokens each.
template <typename T, int ET, int NW, bool SPLIT, int TT>
__global__ __launch_bounds__(64 * NW) void expert_route_kernel(const RouteArgs a) {
  constexpr int NT = 64 * NW, TOK = ET == 0 ? 16 : SPLIT ? 16 * TT : 16 * NW;
  extern __shared__ float logits[];  // [NW (SPLIT) or 1][TOK][E]
  __shared__ int hist[kMaxExperts], base[kMaxExperts], scan[256];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, quad = lane >> 4;
  const long n0 = (long)blockIdx.x * TOK;
  const int n = a.n - n0 < TOK ? (int)(a.n - n0) : TOK;
  for (int e = tid; e < a.E; e += NT) hist[e] = 0;
  if constexpr (ET > 0) {
    f32x4 acc[ET][TT];
#pragma unroll
    for (int t = 0; t < ET; ++t)
#pragma unroll
      for (int x = 0; x < TT; ++x) acc[t][x] = f32x4{0.f, 0.f, 0.f, 0.f};
    const __bf16* h[TT];
#pragma unroll
    for (int x = 0; x < TT; ++x) {
      const int tok = (SPLIT ? 0 : wave * 16) + x * 16 + l16;
      h[x] = static_cast<const __bf16*>(a.h) + (n0 + (tok < n ? tok : 0)) * a.h_sr;
    }
    const __bf16* w[ET];
#pragma unroll
    for (int t = 0; t < ET; ++t) {
      const int e = t * 16 + l16;
      w[t] = static_cast<const __bf16*>(a.w) + (long)(e < a.E ? e : 0) * a.D;
    }
    const int pieces = (a.D + 31) / 32, per = SPLIT ? (pieces + NW - 1) / NW : pieces;
    const int p0 = SPLIT ? wave * per : 0, p1 = p0 + per < pieces ? p0 + per : pieces;
    constexpr int PU = ET <= 4 ? 4 : 2;  // pieces whose loads are in flight together
    for (int p = p0; p < p1; p += PU) {
      bf16x8 x8[PU][TT], w8[PU][ET];
#pragma unroll
      for (int u = 0; u < PU; ++u) {
        const int c = (p + u) * 32 + quad * 8;
        const bool in = p + u < p1 && c < a.D;
#pragma unroll
        for (int x = 0; x < TT; ++x) x8[u][x] = *reinterpret_cast<const bf16x8*>(h[x] + (in ? c : 0));
#pragma unroll
        for (int t = 0; t < ET; ++t) w8[u][t] = *reinterpret_cast<const bf16x8*>(w[t] + (in ? c : 0));
      }
#pragma unroll
      for (int u = 0; u < PU; ++u) {
        const bool in = p + u < p1 && (p + u) * 32 + quad * 8 < a.D;
#pragma unroll
        for (int x = 0; x < TT; ++x) {
#pragma unroll
          for (int j = 0; j < 8; ++j) x8[u][x][j] = in ? x8[u][x][j] : (__bf16)0.f;
#pragma unroll
          for (int t = 0; t < ET; ++t) acc[t][x] = expert_mfma(w8[u][t], x8[u][x], acc[t][x]);
        }
      }
    }
    // column = token l16, rows = experts 4 quad + i
#pragma unroll
    for (int t = 0; t < ET; ++t)
#pragma unroll
      for (int x = 0; x < TT; ++x)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int e = t * 16 + quad * 4 + i;
          if (e < a.E) logits[((SPLIT ? wave * TOK : wave * 16) + x * 16 + l16) * a.E + e] = acc[t][x][i];
        }
    __syncthreads();
    for (int i = tid; i < TOK * a.E; i += NT) {
      float z = logits[i];
      if constexpr (SPLIT) {
#pragma unroll
        for (int v = 1; v < NW; ++v) z += logits[v * TOK * a.E + i];
      }
      logits[i] = 1.0f / (1.0f + expf(-z));
    }
  } else {
    for (int i = tid; i < TOK * a.E; i += NT) {
      const int t = i / a.E, e = i % a.E;
      const T* h = static_cast<const T*>(a.h) + (n0 + (t < n ? t : 0)) * a.h_sr;
      const T* w = static_cast<const T*>(a.w) + (long)e * a.D;
      float z = 0.f;
      for (int c = 0; c < a.D; ++c) z = __builtin_fmaf(to_f32(w[c]), to_f32(h[c]), z);
      logits[i] = 1.0f / (1.0f + expf(-z));
    }
  }
  __syncthreads();
  // 16 lanes per token
  const int sub = tid & 15;
  for (int t = tid >> 4; t < TOK; t += NT / 16) {
    float* s = logits + t * a.E;
    for (int j = 0; j < a.top; ++j) {
      float best = -2.f;
      int at = 0;
      for (int e = sub; e < a.E; e += 16)
        if (s[e] > best) best = s[e], at = e;
#pragma unroll
      for (int m = 8; m >= 1; m >>= 1) {
        const float ov = __shfl_xor(best, m, 16);
        const int oa = __shfl_xor(at, m, 16);
        if (ov > best || (ov == best && oa < at)) best = ov, at = oa;
      }
      if (at % 16 == sub) s[at] = -1.f;  // taken
      if (sub == 0 && t < n) {
        const long slot = (n0 + t) * a.top + j;
        a.ids[slot] = at;
        a.scores[slot] = best;
        if (a.rank != nullptr) a.rank[slot] = atomicAdd(&hist[at], 1);
      }
    }
  }
  if (a.rank == nullptr) return;
  __syncthreads();
  if (a.order != nullptr) {
    plan_tiles(hist, scan, base, a.tile_first, a.tile_expert, a.E, a.tile_rows);
    for (int e = tid; e < a.E; e += NT) a.counts[e] = hist[e];
  } else {
    for (int e = tid; e < a.E; e += NT) base[e] = hist[e] > 0 ? atomicAdd(&a.counts[e], hist[e]) : 0;
    __syncthreads();
  }
  for (int t = tid >> 4; t < n; t += NT / 16) {
    if (sub != 0) continue;
    for (int j = 0; j < a.top; ++j) {
      const long slot = (n0 + t) * a.top + j;  // (this thread has written it)
      if (a.order != nullptr)
        a.order[(long)base[a.ids[slot]] * a.tile_rows + a.rank[slot]] = (int32_t)slot;
      else
        a.rank[slot] += base[a.ids[slot]];
    }
  }
}

// Few tokens: one workgroup each, router rows as whole lines.  With norm_w (bf16) the token's row is formed first: r = res_in + mult * x
// (fp32, into res_out), h = norm(r) * norm_w (into h_out).
struct RouteRowArgs {
  RouteArgs r;
  const float* res_in;
  float* res_out;
  const __bf16* norm_w;
  __bf16* h_out;
  float mult, eps;
  int kind;
};

constexpr int kRouteRowMax = 4096;  // channels

__global__ __launch_bounds__(512) void expert_route_row_kernel(const RouteRowArgs a) {
  __shared__ __attribute__((aligned(16))) __bf16 row[kRouteRowMax];
  __shared__ float s[kMaxExperts], part[16];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, D = a.r.D, E = a.r.E;
  const long n = blockIdx.x;
  const __bf16* x = static_cast<const __bf16*>(a.r.h) + n * a.r.h_sr;
  const int e8 = tid * 8;
  const bool in = e8 < D;
  float v[8];
  load_vec<__bf16, 8>(x + (in ? e8 : 0), v);
  if (a.norm_w != nullptr) {
    float w8[8], r8[8];
    load_vec<__bf16, 8>(a.norm_w + (in ? e8 : 0), w8);
#pragma unroll
    for (int i = 0; i < 8; ++i) r8[i] = 0.f;
    if (a.res_in != nullptr) load_vec<float, 8>(a.res_in + n * D + (in ? e8 : 0), r8);
    const float mult = a.res_in != nullptr ? a.mult : 1.0f;
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      v[i] = in ? __builtin_fmaf(mult, v[i], r8[i]) : 0.f;
      sum += v[i];
    }
    auto all = [&](float q, int at) {
      q = sum16(q);
      q += __shfl_xor(q, 16, 64);
      q += __shfl_xor(q, 32, 64);
      if (lane == 0) part[at + wave] = q;
      __syncthreads();
      float t = 0.f;
#pragma unroll
      for (int i = 0; i < 8; ++i) t += part[at + i];
      return t;
    };
    if (a.res_out != nullptr && in) store_vec<float, 8>(a.res_out + n * D + e8, v);
    const float mean = a.kind == BASED_NORM_LAYER ? all(sum, 0) / (float)D : 0.f;
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      v[i] = in ? v[i] - mean : 0.f;
      ss = __builtin_fmaf(v[i], v[i], ss);
    }
    const float rstd = 1.0f / sqrtf(all(ss, 8) / (float)D + a.eps);
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] *= rstd * w8[i];
    if (in) store_vec<__bf16, 8>(a.h_out + n * D + e8, v);
  }
  if (in) store_vec<__bf16, 8>(row + e8, v);
  __syncthreads();
  constexpr int EU = 4;  // experts whose rows are in flight together
  for (int e0 = wave * EU; e0 < E; e0 += 8 * EU) {
    float acc[EU];
#pragma unroll
    for (int u = 0; u < EU; ++u) acc[u] = 0.f;
#pragma unroll 2
    for (int c = lane * 8; c < D; c += 512) {
      float h8[8];
      load_vec<__bf16, 8>(row + c, h8);
#pragma unroll
      for (int u = 0; u < EU; ++u) {
        float w8[8];
        load_vec<__bf16, 8>(static_cast<const __bf16*>(a.r.w) + (long)(e0 + u < E ? e0 + u : 0) * D + c, w8);
#pragma unroll
        for (int i = 0; i < 8; ++i) acc[u] = __builtin_fmaf(w8[i], h8[i], acc[u]);
      }
    }
#pragma unroll
    for (int u = 0; u < EU; ++u) {
      float z = sum16(acc[u]);
      z += __shfl_xor(z, 16, 64);
      z += __shfl_xor(z, 32, 64);
      if (lane == 0 && e0 + u < E) s[e0 + u] = 1.0f / (1.0f + expf(-z));
    }
  }
  __syncthreads();
  if (wave != 0) return;
  float mine[kMaxExperts / 64];
#pragma unroll
  for (int i = 0; i < kMaxExperts / 64; ++i) mine[i] = i * 64 + lane < E ? s[i * 64 + lane] : -2.f;
  for (int j = 0; j < a.r.top; ++j) {
    float best = -3.f;
    int at = 0;
#pragma unroll
    for (int i = 0; i < kMaxExperts / 64; ++i)
      if (mine[i] > best) best = mine[i], at = i * 64 + lane;
#pragma unroll
    for (int m = 32; m >= 1; m >>= 1) {
      const float ov = __shfl_xor(best, m, 64);
      const int oa = __shfl_xor(at, m, 64);
      if (ov > best || (ov == best && oa < at)) best = ov, at = oa;
    }
#pragma unroll
    for (int i = 0; i < kMaxExperts / 64; ++i) mine[i] = i * 64 + lane == at ? -2.f : mine[i];
    if (lane == 0) {
      a.r.ids[n * a.r.top + j] = at;
      a.r.scores[n * a.r.top + j] = best;
    }
  }
}

constexpr long kPlanSlots = 8192;  // choices that the planning workgroup puts in order by itself

constexpr int kPlanThreads = 1024;

__global__ __launch_bounds__(kPlanThreads) void expert_plan_kernel(const int32_t* counts, const int32_t* __restrict__ ids,
                                                                   const int32_t* __restrict__ rank, int32_t* tile_first,
                                                                   int32_t* tile_expert, int32_t* __restrict__ order, long slots, int E,
                                                                   int tile_rows) {
  __shared__ int scan[256], first_of[kMaxExperts];
  plan_tiles(counts, scan, first_of, tile_first, tile_expert, E, tile_rows);
  if (slots <= kPlanSlots) {
    // (the loads of the unrolled places are independent of each other)
#pragma unroll 4
    for (int i = threadIdx.x; i < (int)slots; i += kPlanThreads) order[(long)first_of[ids[i]] * tile_rows + rank[i]] = i;
  }
}

__global__ __launch_bounds__(256) void expert_scatter_kernel(const int32_t* ids, const int32_t* rank, const int32_t* tile_first, int32_t* order,
                                                             long slots, int tile_rows) {
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i < slots) order[(long)tile_first[ids[i]] * tile_rows + rank[i]] = (int32_t)i;
}

// ---- grouped products ----
struct ExpertGemmArgs {
  const __bf16* x;       // PAIRED: (N, K) rows gathered by order / top; otherwise (tiles * rows, K) in order
  const __bf16* w;       // PAIRED: (E, 2 F, K), up rows then gate rows; otherwise (E, F, K)
  __bf16* y;             // PAIRED: (tiles * rows, F); otherwise (slots, F) scattered by order
  const int32_t* order;
  const int32_t* counts;
  const int32_t* tile_first;
  const int32_t* tile_expert;
  const float* scores;   // (slots), PAIRED
  long x_sr;
  int E, F, K, top, col_tiles, tiles;
};

constexpr int kGemmK = 64;
constexpr int kBand = 8;

// Workgroups are dealt to the eight dies in turn: those of one die take neighbouring tiles, which share rows and matrices.
__device__ __forceinline__ int tile_of_block(int i, int n) {
  const int die = i & 7, k = i >> 3, per = n / 8, more = n % 8;
  return die * per + (die < more ? die : more) + k;
}

// BM rows and BN rows of the weights (PAIRED: half of them up, half gate) per workgroup; AHEAD rounds of 64 channels on their
// way from memory.
template <int BM, int BN, int AHEAD, int BUF, bool PAIRED>
__global__ __launch_bounds__(256, 2) void expert_gemm_kernel(const ExpertGemmArgs a) {
  // rows of 128 bytes lie side by side, the eight 16-byte pieces of a row turned by half its number: neither the rows that
  // eight lanes write nor the sixteen that a tile reads meet a bank twice
  constexpr int KS = kGemmK;
  auto place = [](int r, int p) { return r * KS + ((p ^ (r >> 1)) & 7) * 8; };
  constexpr int WM = BM >= 128 ? 2 : 1, WN = 4 / WM, MT = BM / 16 / WM, NT = BN / 32 / WN, HALF = BN / 2;
  constexpr int AP = BM / 32, BP = BN / 32;  // 16-byte pieces per thread
  __shared__ __attribute__((aligned(16))) __bf16 xs[BUF][BM * KS], ws[BUF][BN * KS];
  __shared__ int slot_of[BM];
  // bands of kBand row tiles, walked down the rows first: what is in flight on a die shares its rows and its matrices
  const int id = tile_of_block(blockIdx.x, gridDim.x), band = id / (kBand * a.col_tiles), in_band = id % (kBand * a.col_tiles);
  const int deep = a.tiles - band * kBand < kBand ? a.tiles - band * kBand : kBand;
  const int tile = band * kBand + in_band % deep, f0 = in_band / deep * (PAIRED ? HALF : BN);
  if (tile >= a.tile_first[a.E]) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, quad = lane >> 4, wm = wave % WM, wn = wave / WM;
  const int e = a.tile_expert[tile], r0 = (tile - a.tile_first[e]) * BM;
  const int rows = a.counts[e] - r0 < BM ? a.counts[e] - r0 : BM;
  for (int i = tid; i < BM; i += 256) slot_of[i] = a.order[(long)tile * BM + (i < rows ? i : 0)];
  lds_barrier();
  typedef __attribute__((ext_vector_type(4))) uint32_t u32x4;
  const int piece = (tid & 7) * 8;  // of the 64 channels of a round
  const __bf16* xrow[AP];
#pragma unroll
  for (int i = 0; i < AP; ++i) {
    const int r = i * 32 + (tid >> 3);
    xrow[i] = a.x + (PAIRED ? (long)(slot_of[r] / a.top) * a.x_sr : ((long)tile * BM + (r < rows ? r : 0)) * a.x_sr);
  }
  const __bf16* wbase = a.w + (long)e * (PAIRED ? 2 * a.F : a.F) * a.K;
  int wrow[BP];
#pragma unroll
  for (int i = 0; i < BP; ++i) {
    const int r = i * 32 + (tid >> 3);
    const int f = PAIRED ? f0 + (r % HALF) : f0 + r;
    wrow[i] = ((PAIRED && r >= HALF ? a.F : 0) + (f < a.F ? f : a.F - 1)) * a.K;
  }
  u32x4 xb[AHEAD][AP], wb[AHEAD][BP];
  const u32x4 zero = {0u, 0u, 0u, 0u};
  auto fetch = [&](int k0, u32x4 (&x)[AP], u32x4 (&w)[BP]) {
    const int c = k0 + piece < a.K ? k0 + piece : 0;
#pragma unroll
    for (int i = 0; i < AP; ++i) x[i] = *reinterpret_cast<const u32x4*>(xrow[i] + c);
#pragma unroll
    for (int i = 0; i < BP; ++i) w[i] = *reinterpret_cast<const u32x4*>(wbase + (wrow[i] + c));
  };
  f32x4 acc[2][NT][MT];
#pragma unroll
  for (int p = 0; p < 2; ++p)
#pragma unroll
    for (int i = 0; i < NT; ++i)
#pragma unroll
      for (int j = 0; j < MT; ++j) acc[p][i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  auto stage = [&](int k0, int buf, const u32x4 (&x)[AP], const u32x4 (&w)[BP]) {
    const bool in = k0 + piece < a.K;
#pragma unroll
    for (int i = 0; i < AP; ++i) *reinterpret_cast<u32x4*>(&xs[buf][place(i * 32 + (tid >> 3), tid & 7)]) = in ? x[i] : zero;
#pragma unroll
    for (int i = 0; i < BP; ++i) *reinterpret_cast<u32x4*>(&ws[buf][place(i * 32 + (tid >> 3), tid & 7)]) = w[i];
  };
  auto multiply = [&](int buf) {
#pragma unroll
    for (int kk = 0; kk < kGemmK; kk += 32) {
      bf16x8 xf[MT];
#pragma unroll
      for (int j = 0; j < MT; ++j) xf[j] = *reinterpret_cast<const bf16x8*>(&xs[buf][place((wm * MT + j) * 16 + l16, kk / 8 + quad)]);
#pragma unroll
      for (int p = 0; p < 2; ++p)
#pragma unroll
        for (int i = 0; i < NT; ++i) {
          const bf16x8 wf = *reinterpret_cast<const bf16x8*>(&ws[buf][place(p * HALF + (wn * NT + i) * 16 + l16, kk / 8 + quad)]);
#pragma unroll
          for (int j = 0; j < MT; ++j) acc[p][i][j] = expert_mfma(wf, xf[j], acc[p][i][j]);
        }
    }
  };
#pragma unroll
  for (int s = 0; s < AHEAD; ++s) fetch(s * kGemmK, xb[s], wb[s]);
  // (rounds past the end multiply by zeros: every stage of the loops is the same)
  if constexpr (BUF == 1) {
    for (int k00 = 0; k00 < a.K; k00 += AHEAD * kGemmK) {
#pragma unroll
      for (int s = 0; s < AHEAD; ++s) {
        const int k0 = k00 + s * kGemmK;
        lds_barrier();
        stage(k0, 0, xb[s], wb[s]);
        lds_barrier();
        fetch(k0 + AHEAD * kGemmK, xb[s], wb[s]);
        multiply(0);
      }
    }
  } else {
    // one barrier per round: the next round goes into the other half of LDS while this one is multiplied
    constexpr int U = AHEAD % 2 == 0 ? AHEAD : 2 * AHEAD;
    stage(0, 0, xb[0], wb[0]);
    fetch(AHEAD * kGemmK, xb[0], wb[0]);
    lds_barrier();
    for (int k00 = 0; k00 < a.K; k00 += U * kGemmK) {
#pragma unroll
      for (int s = 0; s < U; ++s) {
        const int k1 = k00 + (s + 1) * kGemmK;
        multiply(s & 1);
        stage(k1, (s + 1) & 1, xb[(s + 1) % AHEAD], wb[(s + 1) % AHEAD]);
        fetch(k1 + AHEAD * kGemmK, xb[(s + 1) % AHEAD], wb[(s + 1) % AHEAD]);
        lds_barrier();
      }
    }
  }
  // column = row l16 of the tile's rows, rows = features 4 quad + i
#pragma unroll
  for (int j = 0; j < MT; ++j) {
    const int r = (wm * MT + j) * 16 + l16;
    if (r >= rows) continue;
    const int slot = slot_of[r];
    if constexpr (PAIRED) {
      const float s = a.scores[slot];
      __bf16* y = a.y + ((long)tile * BM + r) * a.F;
#pragma unroll
      for (int i = 0; i < NT; ++i) {
        const int f = f0 + (wn * NT + i) * 16 + quad * 4;
        if (f < a.F) {
          bf16x4 o;
#pragma unroll
          for (int m = 0; m < 4; ++m) o[m] = (__bf16)(silu_exact(acc[1][i][j][m] * s) * (acc[0][i][j][m] * s));
          *reinterpret_cast<bf16x4*>(y + f) = o;
        }
      }
    } else {
      __bf16* y = a.y + (long)slot * a.F;
#pragma unroll
      for (int p = 0; p < 2; ++p)
#pragma unroll
        for (int i = 0; i < NT; ++i) {
          const int f = f0 + p * HALF + (wn * NT + i) * 16 + quad * 4;
          if (f < a.F) {
            bf16x4 o;
#pragma unroll
            for (int m = 0; m < 4; ++m) o[m] = (__bf16)acc[p][i][j][m];
            *reinterpret_cast<bf16x4*>(y + f) = o;
          }
        }
    }
  }
}

template <int BM, int BN, int AHEAD, int BUF, bool PAIRED> void launch_expert_gemm(ExpertGemmArgs a, hipStream_t s) {
  const int cols = PAIRED ? BN / 2 : BN;
  a.col_tiles = (a.F + cols - 1) / cols;
  hipLaunchKernelGGL((expert_gemm_kernel<BM, BN, AHEAD, BUF, PAIRED>), dim3((unsigned)(a.col_tiles * a.tiles)), dim3(256), 0, s, a);
}

template <bool PAIRED> void launch_expert_product(const ExpertGemmArgs& a, int rows, hipStream_t s) {
  if (rows == BASED_EXPERT_TILE_ROWS_SMALL)
    launch_expert_gemm<BASED_EXPERT_TILE_ROWS_SMALL, 128, 4, 1, PAIRED>(a, s);
  else if (a.F >= 256 && (long)a.tiles * a.F >= (PAIRED ? 512 * 128 : 512 * 256))
    launch_expert_gemm<BASED_EXPERT_TILE_ROWS, 256, 1, 1, PAIRED>(a, s);
  else
    launch_expert_gemm<BASED_EXPERT_TILE_ROWS, 128, 2, 1, PAIRED>(a, s);
}

// y[n] = sum of the rows of its choices
__global__ __launch_bounds__(256) void expert_sum_kernel(const __bf16* x, __bf16* y, long n, int D, int top) {
  const int pieces = D / 8;
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= n * pieces) return;
  const long row = i / pieces;
  const int c = (int)(i % pieces) * 8;
  float s[8];
#pragma unroll
  for (int j = 0; j < 8; ++j) s[j] = 0.f;
  for (int t = 0; t < top; ++t) {
    float v[8];
    load_vec<__bf16, 8>(x + (row * top + t) * D + c, v);
#pragma unroll
    for (int j = 0; j < 8; ++j) s[j] += v[j];
  }
  store_vec<__bf16, 8>(y + row * D + c, s);
}

// ---- one choice at a time ----
struct ExpertRowsArgs {
  const void* x;   // first product: (N, K); second: (N * top, K)
  const void* w;   // (E, 2 F, K) / (E, F, K)
  void* y;         // (N * top, F) / (N, F)
  const int32_t* ids;
  const float* scores;
  long n, x_sr;
  int F, K, top;
};

constexpr int kRowsFeatures = 16;  // features per workgroup

template <int LPR> __device__ __forceinline__ float lanes_sum(float v) {
  if constexpr (LPR == 8) return sum8(v);
  v = sum16(v);
  if constexpr (LPR >= 32) v += __shfl_xor(v, 16, 64);
  if constexpr (LPR >= 64) v += __shfl_xor(v, 32, 64);
  return v;
}

// LPR lanes share a dot product; a workgroup takes kRowsFeatures features of one choice (gate and up) or token (down).
template <typename T, int N, int LPR, bool PAIRED>
__global__ __launch_bounds__(256) void expert_rows_kernel(const ExpertRowsArgs a) {
  const int lane = threadIdx.x % LPR, grp = threadIdx.x / LPR;
  constexpr int GROUPS = 256 / LPR;
  const long item = blockIdx.x;  // choice or token
  const int f1 = (int)(blockIdx.y + 1) * kRowsFeatures < a.F ? (int)(blockIdx.y + 1) * kRowsFeatures : a.F;
  constexpr int FU = GROUPS >= kRowsFeatures ? 1 : kRowsFeatures / GROUPS;  // features per group of lanes, in flight together
  int f[FU];
#pragma unroll
  for (int u = 0; u < FU; ++u) f[u] = blockIdx.y * kRowsFeatures + u * GROUPS + grp;
  auto load = [&](const T* p, float (&v)[N]) {
    if constexpr (N == 1)
      v[0] = to_f32(*p);
    else
      load_vec<T, N>(p, v);
  };
  if constexpr (PAIRED) {
    const T* x = static_cast<const T*>(a.x) + item / a.top * a.x_sr;
    const T* w = static_cast<const T*>(a.w) + (long)a.ids[item] * 2 * a.F * a.K;
    float up[FU], gate[FU];
#pragma unroll
    for (int u = 0; u < FU; ++u) up[u] = gate[u] = 0.f;
#pragma unroll 2
    for (int c = lane * N; c < a.K; c += LPR * N) {
      float xv[N];
      load(x + c, xv);
#pragma unroll
      for (int u = 0; u < FU; ++u) {
        const long row = f[u] < f1 ? f[u] : 0;
        float uv[N], gv[N];
        load(w + row * a.K + c, uv);
        load(w + (a.F + row) * a.K + c, gv);
#pragma unroll
        for (int j = 0; j < N; ++j) {
          up[u] = __builtin_fmaf(uv[j], xv[j], up[u]);
          gate[u] = __builtin_fmaf(gv[j], xv[j], gate[u]);
        }
      }
    }
    const float s = a.scores[item];
#pragma unroll
    for (int u = 0; u < FU; ++u) {
      const float uu = lanes_sum<LPR>(up[u]), gg = lanes_sum<LPR>(gate[u]);
      if (lane == 0 && f[u] < f1) static_cast<T*>(a.y)[item * a.F + f[u]] = from_f32<T>(silu_exact(gg * s) * (uu * s));
    }
  } else {
    float acc[FU];
#pragma unroll
    for (int u = 0; u < FU; ++u) acc[u] = 0.f;
    for (int t = 0; t < a.top; ++t) {
      const T* x = static_cast<const T*>(a.x) + (item * a.top + t) * a.x_sr;
      const T* w = static_cast<const T*>(a.w) + (long)a.ids[item * a.top + t] * a.F * a.K;
#pragma unroll 2
      for (int c = lane * N; c < a.K; c += LPR * N) {
        float xv[N];
        load(x + c, xv);
#pragma unroll
        for (int u = 0; u < FU; ++u) {
          float wv[N];
          load(w + (long)(f[u] < f1 ? f[u] : 0) * a.K + c, wv);
#pragma unroll
          for (int j = 0; j < N; ++j) acc[u] = __builtin_fmaf(wv[j], xv[j], acc[u]);
        }
      }
    }
#pragma unroll
    for (int u = 0; u < FU; ++u) {
      const float s = lanes_sum<LPR>(acc[u]);
      if (lane == 0 && f[u] < f1) static_cast<T*>(a.y)[item * a.F + f[u]] = from_f32<T>(s);
    }
  }
}

template <typename T, int N, bool PAIRED> void launch_expert_rows(const ExpertRowsArgs& a, long items, hipStream_t s) {
  const dim3 grid((unsigned)items, (unsigned)((a.F + kRowsFeatures - 1) / kRowsFeatures));
  const int pieces = (a.K + N - 1) / N;
  if (pieces <= 8)
    hipLaunchKernelGGL((expert_rows_kernel<T, N, 8, PAIRED>), grid, dim3(256), 0, s, a);
  else if (pieces <= 16)
    hipLaunchKernelGGL((expert_rows_kernel<T, N, 16, PAIRED>), grid, dim3(256), 0, s, a);
  else if (pieces <= 32)
    hipLaunchKernelGGL((expert_rows_kernel<T, N, 32, PAIRED>), grid, dim3(256), 0, s, a);
  else
    hipLaunchKernelGGL((expert_rows_kernel<T, N, 64, PAIRED>), grid, dim3(256), 0, s, a);
}

template <typename T, bool PAIRED> void launch_expert_rows_vec(const ExpertRowsArgs& a, bool vec, long items, hipStream_t s) {
  if (vec)
    launch_expert_rows<T, Pack<T>::kN, PAIRED>(a, items, s);
  else
    launch_expert_rows<T, 1, PAIRED>(a, items, s);
}

constexpr int kRouteOneWg = 32;  // tokens that one workgroup routes, of up to 32 experts (16 of more): it makes the plan too

template <int ET> void launch_route_tiles(const RouteArgs& a, hipStream_t s) {
  const size_t one = (size_t)16 * a.E * sizeof(float);
  constexpr int NW = ET <= 4 ? 8 : 4;
  if constexpr (ET <= 2) {
    if (a.n > 16 && a.n <= kRouteOneWg) {
      hipLaunchKernelGGL((expert_route_kernel<__bf16, ET, NW, true, 2>), dim3(1), dim3(64 * NW), 2 * NW * one, s, a);
      return;
    }
  }
  if (a.n >= 4096)
    hipLaunchKernelGGL((expert_route_kernel<__bf16, ET, 4, false, 1>), dim3((unsigned)((a.n + 63) / 64)), dim3(256), 4 * one, s, a);
  else
    hipLaunchKernelGGL((expert_route_kernel<__bf16, ET, NW, true, 1>), dim3((unsigned)((a.n + 15) / 16)), dim3(64 * NW), NW * one, s, a);
}

static bool route_is_single(const RouteArgs& a, bool vec) { return a.n <= (vec && a.E <= 32 ? kRouteOneWg : 16); }

template <typename T> void launch_route(RouteArgs a, bool vec, hipStream_t s) {
  const dim3 grid((unsigned)((a.n + 15) / 16));
  if (!route_is_single(a, vec)) a.order = nullptr;
  if constexpr (sizeof(T) == 2) {
    const int et = (a.E + 15) / 16;
    if (vec && et <= 1)
      return launch_route_tiles<1>(a, s);
    if (vec && et <= 2)
      return launch_route_tiles<2>(a, s);
    if (vec && et <= 4)
      return launch_route_tiles<4>(a, s);
    if (vec && et <= 8)
      return launch_route_tiles<8>(a, s);
  }
  hipLaunchKernelGGL((expert_route_kernel<T, 0, 4, false, 1>), grid, dim3(256), (size_t)16 * a.E * sizeof(float), s, a);
}

static bool route_vec(const RouteArgs& a) {
  return a.D % 8 == 0 && a.h_sr % 8 == 0 && a.E <= 128 && aligned_to(a.h, 16) && aligned_to(a.w, 16);
}

static int route_check(const char* who, const RouteArgs& a) {
  BASED_REQUIRE(a.n >= 0 && a.D > 0 && a.E > 0 && a.top > 0 && a.top <= a.E, BASED_ERR_ARG, "%s: bad sizes", who);
  BASED_REQUIRE(a.E <= kMaxExperts, BASED_ERR_SHAPE, "%s: %d experts (at most %d)", who, a.E, kMaxExperts);
  BASED_REQUIRE(a.n * a.top < (1ll << 31), BASED_ERR_SHAPE, "%s: too many choices", who);
  return BASED_OK;
}

}  // namespace based

/* Tiles of BASED_EXPERT_TILE_ROWS or BASED_EXPERT_TILE_ROWS_SMALL rows. */
static int expert_tile_rows(int64_t slots, int64_t E) { return slots >= 256 * E ? BASED_EXPERT_TILE_ROWS : BASED_EXPERT_TILE_ROWS_SMALL; }

extern "C" BASED_API int64_t based_expert_tiles(int64_t n, int64_t E, int64_t top) {
  if (n <= 0 || E <= 0 || top <= 0) return 0;
  const int64_t rows = expert_tile_rows(n * top, E);
  return n * top / rows + (E < n * top ? E : n * top);
}

extern "C" BASED_API int64_t based_expert_tile_rows(int64_t n, int64_t E, int64_t top) { return expert_tile_rows(n * top, E); }

extern "C" BASED_API int based_expert_grouped(const void* h, const void* router, const void* w1, const void* w2, int32_t* ids, float* scores,
                                              int32_t* rank, int32_t* counts, int32_t* tile_first, int32_t* tile_expert, int32_t* order,
                                              void* work_act, void* work_out, void* y, int64_t n, int64_t D, int64_t F, int64_t E, int64_t top,
                                              int64_t h_sr, void* stream) {
  using namespace based;
  BASED_REQUIRE(h && router && w1 && w2 && ids && scores && rank && counts && tile_first && tile_expert && order && work_act && y,
                BASED_ERR_ARG, "expert_grouped: null pointer argument");
  BASED_REQUIRE(F > 0 && D < (1ll << 28), BASED_ERR_ARG, "expert_grouped: bad sizes");
  BASED_REQUIRE(top == 1 || work_out != nullptr, BASED_ERR_ARG, "expert_grouped: several choices per token need work_out");
  BASED_REQUIRE(D % 8 == 0 && F % 8 == 0 && h_sr % 8 == 0 && 2 * F * D < (1ll << 31), BASED_ERR_SHAPE,
                "expert_grouped: sizes %ld and %ld must be multiples of 8", (long)D, (long)F);
  BASED_REQUIRE(aligned_to(h, 16) && aligned_to(w1, 16) && aligned_to(w2, 16) && aligned_to(work_act, 16) && aligned_to(work_out, 16) &&
                    aligned_to(y, 16),
                BASED_ERR_ALIGN, "expert_grouped: tensors must be 16-byte aligned");
  RouteArgs r{h, router, ids, scores, rank, counts, tile_first, tile_expert, order, 0, (long)n, (long)h_sr, (int)D, (int)E, (int)top};
  const int rc = route_check("expert_grouped", r);
  if (rc != BASED_OK) return rc;
  if (n == 0) return BASED_OK;
  const int64_t slots = n * top;
  const int rows = expert_tile_rows(slots, E);
  const int64_t tiles = based_expert_tiles(n, E, top);
  BASED_REQUIRE(tiles * ((F > D ? F : D) / 64 + 1) < (1ll << 31), BASED_ERR_SHAPE, "expert_grouped: too many rows");
  hipStream_t s = static_cast<hipStream_t>(stream);
  r.tile_rows = rows;
  const bool vec = route_vec(r);
  launch_route<__bf16>(r, vec, s);
  if (!route_is_single(r, vec)) {
    hipLaunchKernelGGL(expert_plan_kernel, dim3(1), dim3(kPlanThreads), 0, s, counts, ids, rank, tile_first, tile_expert, order, (long)slots, (int)E,
                       rows);
    if (slots > kPlanSlots)
      hipLaunchKernelGGL(expert_scatter_kernel, dim3((unsigned)((slots + 255) / 256)), dim3(256), 0, s, ids, rank, tile_first, order,
                         (long)slots, rows);
  }
  const ExpertGemmArgs a{static_cast<const __bf16*>(h), static_cast<const __bf16*>(w1), static_cast<__bf16*>(work_act), order, counts, tile_first,
                         tile_expert, scores, (long)h_sr, (int)E, (int)F, (int)D, (int)top, 0, (int)tiles};
  __bf16* out = static_cast<__bf16*>(top == 1 ? y : work_out);
  const ExpertGemmArgs a2{static_cast<const __bf16*>(work_act), static_cast<const __bf16*>(w2), out, order, counts, tile_first,
                          tile_expert, scores, (long)F, (int)E, (int)D, (int)F, (int)top, 0, (int)tiles};
  launch_expert_product<true>(a, rows, s);
  launch_expert_product<false>(a2, rows, s);
  if (top > 1)
    hipLaunchKernelGGL(expert_sum_kernel, dim3((unsigned)((n * (D / 8) + 255) / 256)), dim3(256), 0, s, out, static_cast<__bf16*>(y), (long)n,
                       (int)D, (int)top);
  return check_launch("expert_grouped");
}

extern "C" BASED_API int based_expert_rows(const void* x, const float* residual_in, float* residual_out, const void* norm_weight, void* work_h,
                                           float mult, int norm_kind, float eps, const void* router, const void* w1, const void* w2,
                                           int32_t* ids, float* scores, void* work_act, void* y, int64_t n, int64_t D, int64_t F, int64_t E,
                                           int64_t top, int64_t x_sr, int io_dtype, void* stream) {
  using namespace based;
  BASED_REQUIRE(x && router && w1 && w2 && ids && scores && work_act && y, BASED_ERR_ARG, "expert_rows: null pointer argument");
  BASED_REQUIRE(F > 0 && D < (1 << 20) && F < (1 << 20), BASED_ERR_SHAPE, "expert_rows: grid too large");
  BASED_REQUIRE(io_dtype == BASED_BF16 || io_dtype == BASED_F32, BASED_ERR_DTYPE, "expert_rows: bad dtype");
  RouteArgs r{x, router, ids, scores, nullptr, nullptr, nullptr, nullptr, nullptr, 0, (long)n, (long)x_sr, (int)D, (int)E, (int)top};
  const int rc = route_check("expert_rows", r);
  if (rc != BASED_OK) return rc;
  const bool by_row = io_dtype == BASED_BF16 && D % 8 == 0 && D <= kRouteRowMax && x_sr % 8 == 0 && aligned_to(x, 16) && aligned_to(router, 16);
  if (norm_weight != nullptr) {
    BASED_REQUIRE(by_row, BASED_ERR_SHAPE, "expert_rows: the norm takes bf16 rows of a multiple of 8 up to %d channels", kRouteRowMax);
    BASED_REQUIRE(work_h && (norm_kind == BASED_NORM_RMS || norm_kind == BASED_NORM_LAYER) && residual_out != residual_in, BASED_ERR_ARG,
                  "expert_rows: bad norm arguments");
    BASED_REQUIRE(aligned_to(norm_weight, 16) && aligned_to(residual_in, 16) && aligned_to(residual_out, 16) && aligned_to(work_h, 16),
                  BASED_ERR_ALIGN, "expert_rows: tensors must be 16-byte aligned");
  }
  if (n == 0) return BASED_OK;
  hipStream_t s = static_cast<hipStream_t>(stream);
  const void* h = norm_weight != nullptr ? work_h : x;
  const int64_t h_sr = norm_weight != nullptr ? D : x_sr;
  if (norm_weight != nullptr || (by_row && n <= 16)) {
    const RouteRowArgs a{r, residual_in, residual_out, static_cast<const __bf16*>(norm_weight), static_cast<__bf16*>(work_h), mult, eps, norm_kind};
    hipLaunchKernelGGL(expert_route_row_kernel, dim3((unsigned)n), dim3(512), 0, s, a);
  } else if (io_dtype == BASED_BF16) {
    launch_route<__bf16>(r, route_vec(r), s);
  } else {
    launch_route<float>(r, false, s);
  }
  const int p = io_dtype == BASED_BF16 ? 8 : 4;
  const bool vec1 = D % p == 0 && h_sr % p == 0 && aligned_to(h, 16) && aligned_to(w1, 16);
  const bool vec2 = F % p == 0 && aligned_to(work_act, 16) && aligned_to(w2, 16);
  const ExpertRowsArgs a1{h, w1, work_act, ids, scores, (long)n, (long)h_sr, (int)F, (int)D, (int)top};
  const ExpertRowsArgs a2{work_act, w2, y, ids, scores, (long)n, (long)F, (int)D, (int)F, (int)top};
  if (io_dtype == BASED_BF16) {
    launch_expert_rows_vec<__bf16, true>(a1, vec1, n * top, s);
    launch_expert_rows_vec<__bf16, false>(a2, vec2, n, s);
  } else {
    launch_expert_rows_vec<float, true>(a1, vec1, n * top, s);
    launch_expert_rows_vec<float, false>(a2, vec2, n, s);
  }
  return check_launch("expert_rows");
}
