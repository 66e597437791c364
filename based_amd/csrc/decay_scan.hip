// Linear attention with decaying states for gfx950.  Per head (state S: d x dv, fp32), token by token, either
//
//   channel decays (a decay per key channel and token, a bonus for the current token):
//     o_t = (S + diag(u) k_t v_t^T)^T q_t,   then  S <- diag(w_t) S + k_t v_t^T
//   head decays (one constant per head):
//     S <- w_h S + k_t v_t^T,   then  o_t = S^T q_t
//
// with silu on q, k and v first where asked for.  Decays come as base-2 logarithms.  The state lies by
// value channel, (B, H, dv, dp): rows of dp >= d key channels.
//
//   decay_scan_mfma   bf16: walks 64 tokens at a time with the state in MFMA accumulators, 16 value channels
//                     per wavefront.  Long sequences are cut into segments: a first pass leaves what every
//                     segment adds to the state, `decay_join` turns that into the state at every segment's
//                     start, and the second pass starts there.
//   decay_scan_any    any element type and size: a thread holds some key channels of one value channel.
//   decay_step        one token per sequence; for channel decays with the low-rank decay in front and the
//                     head norm and gate behind.
//   group_norm_gate   o / rms(o) * w * act(g) over groups of a row.
//
// Inside 64 tokens, with P_ts the weight of v_s in o_t, o = P v + (q scaled by the decay since the start) S0.
// All scaling is by decays over tokens that lie in between, never by an inverse, so nothing overflows:
//   * s and t in the same 16 tokens: k_s, multiplied by one more decay at each step, is passed from token to
//     token (a lane is a token) and meets every q on its way;
//   * s in an earlier 16 tokens: k_s decayed to the end of its 16, q_t to the start of its own, and to q
//     also what lies between.
// fp32 numbers enter a bf16 product as pairs (a number rounded to bf16, and the rest rounded to bf16), so
// an operand keeps 16 bits and the sums 24.
#include "stream_common.hpp"

namespace based {

constexpr int kScanTokens = 64;

struct DecayScanArgs {
  const void* q;
  const void* k;
  const void* v;
  const float* lw;       // (B, L, H * d) contiguous: log2 of the channel decays, or null
  const float* head_lw;  // (2, H): log2 of the head decays, then the decays, or null
  const void* u;         // (H, d)
  float* state;          // (B, H, dv, dp)
  float* seg;            // (B, H, segs, dv, dp) work, null with one segment
  float* seg_lw;         // (B, H, segs, dp) work: channel decays over a segment
  void* o;               // (B, L, H * dv)
  int B, L, H, d, dv, dp;
  long q_sb, q_sl, k_sb, k_sl, v_sb, v_sl, o_sb, o_sl;
  int segs, seg_chunks;  // segments, and 64-token pieces in each
  int silu, fresh;
};

template <int CTRL> __device__ __forceinline__ float row_moved(float x) {  // lanes without a source receive 0
  return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, x), CTRL, 0xf, 0xf, true));
}
// Products along the 16 lanes of a row, of several independent numbers at once.  A DPP multiplication leaves a lane
// without a source as it is, which is the multiplication by one that is wanted; the compiler has no builtin that
// says so.  A register must not be read through DPP in the two issue slots after it was written: four numbers in turn
// keep that distance by themselves, the first ones are kept from what stands before by the s_nop.
//   prefix[i]: product over lanes 0 .. l of w[i];  suffix[i]: over lanes l .. 15
//   before[i] *= prefix of the lane before (nothing for lane 0);  after[i] *= suffix of the lane behind (nothing for lane 15)
#define BASED_ROW_STEP(ctrl) \
  "v_mul_f32_dpp %0, %0, %0 " ctrl " row_mask:0xf bank_mask:0xf\n\t" \
  "v_mul_f32_dpp %1, %1, %1 " ctrl " row_mask:0xf bank_mask:0xf\n\t" \
  "v_mul_f32_dpp %2, %2, %2 " ctrl " row_mask:0xf bank_mask:0xf\n\t" \
  "v_mul_f32_dpp %3, %3, %3 " ctrl " row_mask:0xf bank_mask:0xf\n\t"
#define BASED_ROW_LAST(ctrl) \
  "v_mul_f32_dpp %4, %0, %4 " ctrl " row_mask:0xf bank_mask:0xf\n\t" \
  "v_mul_f32_dpp %5, %1, %5 " ctrl " row_mask:0xf bank_mask:0xf\n\t" \
  "v_mul_f32_dpp %6, %2, %6 " ctrl " row_mask:0xf bank_mask:0xf\n\t" \
  "v_mul_f32_dpp %7, %3, %7 " ctrl " row_mask:0xf bank_mask:0xf"
__device__ __forceinline__ void row_prefix4(float* prefix, float* before) {
  asm volatile("s_nop 1\n\t" BASED_ROW_STEP("row_shr:1") BASED_ROW_STEP("row_shr:2") BASED_ROW_STEP("row_shr:4")
               BASED_ROW_STEP("row_shr:8") BASED_ROW_LAST("row_shr:1")
               : "+v"(prefix[0]), "+v"(prefix[1]), "+v"(prefix[2]), "+v"(prefix[3]), "+v"(before[0]), "+v"(before[1]), "+v"(before[2]),
                 "+v"(before[3]));
}
__device__ __forceinline__ void row_suffix4(float* suffix, float* after) {
  asm volatile("s_nop 1\n\t" BASED_ROW_STEP("row_shl:1") BASED_ROW_STEP("row_shl:2") BASED_ROW_STEP("row_shl:4")
               BASED_ROW_STEP("row_shl:8") BASED_ROW_LAST("row_shl:1")
               : "+v"(suffix[0]), "+v"(suffix[1]), "+v"(suffix[2]), "+v"(suffix[3]), "+v"(after[0]), "+v"(after[1]), "+v"(after[2]),
                 "+v"(after[3]));
}
#undef BASED_ROW_STEP
#undef BASED_ROW_LAST
// sum over the four lanes l16, l16 + 16, + 32, + 48, in all of them
__device__ __forceinline__ float quad_rows_sum(float x) {
  x += __shfl_xor(x, 16, 64);
  return x + __shfl_xor(x, 32, 64);
}

__device__ __forceinline__ f32x4 mfma_16(bf16x8 a, bf16x8 b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }
// two numbers as packed pairs of bf16: rounded, and what the rounding left
__device__ __forceinline__ void split2(float a, float b, uint32_t& hi, uint32_t& lo) {
  hi = pack_bf16(a, b);
  lo = pack_bf16(a - __builtin_bit_cast(float, hi << 16), b - __builtin_bit_cast(float, hi & 0xffff0000u));
}
typedef __attribute__((ext_vector_type(4))) uint32_t u32x4;
// eight numbers in the order of an MFMA operand
__device__ __forceinline__ void split8(const float* x, bf16x8& hi, bf16x8& lo) {
  u32x4 h, l;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    uint32_t a, b;
    split2(x[2 * i], x[2 * i + 1], a, b);
    h[i] = a, l[i] = b;
  }
  hi = __builtin_bit_cast(bf16x8, h);
  lo = __builtin_bit_cast(bf16x8, l);
}
// the halves of a packed pair as they are
__device__ __forceinline__ void store_pair(__bf16* p, __bf16* q, uint32_t x) {
  *reinterpret_cast<uint16_t*>(p) = (uint16_t)x;
  *reinterpret_cast<uint16_t*>(q) = (uint16_t)(x >> 16);
}

// HALVES wavefronts (1 or 2) share the key channels of 16 tokens, DT 32-channel pieces each (d <= 32 DT HALVES, d % 4 == 0), so
// that what a lane holds of a token stays in registers; their parts of P are added through LDS.  Channels of a piece are held by the lanes in the
// order of the accumulators: element e < 4 of a lane in 16-lane row `quad` is channel 4 quad + e, e >= 4
// channel 16 + 4 quad + e - 4; every contraction over channels uses that order on both sides.
template <int DT, int HALVES, bool CHANNEL> struct ScanLds {
  static constexpr int CH = 32 * DT * HALVES, RS = CH + 8, TS = kScanTokens + 8;
  __bf16 q_hi[kScanTokens * RS];                 // q scaled to the start of the 64 tokens; head decays: q itself
  __bf16 q_lo[CHANNEL ? kScanTokens * RS : 8];
  union {
    struct {
      __bf16 hi[kScanTokens * RS];               // k decayed to the end of its 16 tokens; head decays: k itself
      __bf16 lo[CHANNEL ? kScanTokens * RS : 8];
    } k;
    struct {
      __bf16 hi[kScanTokens * TS], lo[kScanTokens * TS];  // P, [t][s]
      f32x4 part[HALVES > 1 ? 4 * 4 * 64 : 1];            // the second half's part of P, as its lanes hold it
    } p;
  };
  __bf16 kt_hi[CH * TS], kt_lo[CH * TS];         // k decayed to the end of the 64 tokens, [channel][token]
  __bf16 vt[64 * HALVES * TS];                            // v, [channel][token]
  float total[4][CH], all[CH];                   // decay over each 16 tokens, and over the 64
};

template <int DT, int HALVES, bool CHANNEL, bool STATE_ONLY>
__global__ __launch_bounds__(256 * HALVES, 2) void decay_scan_mfma_kernel(const DecayScanArgs a) {
  typedef ScanLds<DT, HALVES, CHANNEL> Lds;
  constexpr int RS = Lds::RS, TS = Lds::TS, E = DT * 8, DA = DT * HALVES;
  extern __shared__ __attribute__((aligned(16))) char scan_lds[];
  Lds& lds = *reinterpret_cast<Lds*>(scan_lds);
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), l16 = lane & 15, quad = lane >> 4;
  const int blk = wave & 3, half = wave >> 2, ch0 = half * 32 * DT;  // this wavefront's 16 tokens of 64, and its key channels
  const int b = blockIdx.x / a.H, h = blockIdx.x % a.H, sg = blockIdx.z;
  const int col_base = blockIdx.y * 64 * HALVES, dv0 = col_base + wave * 16;
  const bool has_cols = dv0 < a.dv, col_in = dv0 + l16 < a.dv;
  const __bf16* qp = static_cast<const __bf16*>(a.q) + b * a.q_sb + (long)h * a.d;
  const __bf16* kp = static_cast<const __bf16*>(a.k) + b * a.k_sb + (long)h * a.d;
  const __bf16* vp = static_cast<const __bf16*>(a.v) + b * a.v_sb + (long)h * a.dv;
  const float* lwp = CHANNEL ? a.lw + ((long)b * a.L) * a.H * a.d + (long)h * a.d : nullptr;
  const float head_l2 = CHANNEL ? 0.f : a.head_lw[h];
  const long bh = (long)b * a.H + h;
  float* st = a.state + (bh * a.dv + (col_in ? dv0 + l16 : 0)) * a.dp;

  // channel of element e of piece c
  auto chan = [&](int c, int f) { return ch0 + c * 32 + f * 16 + quad * 4; };
  auto chan_of = [&](int i) { return ch0 + (i >> 3) * 32 + ((i >> 2) & 1) * 16 + quad * 4 + (i & 3); };

  // state: tile ct holds key channels 16 ct + 4 quad + i of value channel dv0 + l16
  f32x4 S[2 * DA];
  {
    const float* from = a.segs > 1 ? a.seg + ((bh * a.segs + sg) * a.dv + (col_in ? dv0 + l16 : 0)) * a.dp : st;
    const bool zero = STATE_ONLY || (a.segs == 1 && a.fresh);
#pragma unroll
    for (int ct = 0; ct < 2 * DA; ++ct) {
      const int ch = ct * 16 + quad * 4;
      S[ct] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (!zero && col_in && ch < a.d) S[ct] = *reinterpret_cast<const f32x4*>(from + ch);
    }
  }
  float seg_total = 1.f;  // (state pass, channel decays) decay of the segment so far, of the channel that is this thread's number

  struct Stage {
    bf16x4 q[STATE_ONLY ? 1 : 2 * DT], k[2 * DT], v[4];
    f32x4 lw[CHANNEL ? 2 * DT : 1];
  };
  const int first = sg * a.seg_chunks, chunks = (a.L + kScanTokens - 1) / kScanTokens;
  const int last = first + a.seg_chunks < chunks ? first + a.seg_chunks : chunks;
  // the rows of this wavefront's 16 tokens, unconditionally (places past the end are cleared at use): the place of the
  // 64 tokens is the same for all lanes, and what lies behind it fits 32 bits
  auto fetch = [&](Stage& s, int chunk) {
    const int left = a.L - chunk * kScanTokens, mine = blk * 16 + l16, t = mine < left ? mine : left - 1;
    const long t0 = (long)chunk * kScanTokens;
    const __bf16* q0 = qp + t0 * a.q_sl;
    const __bf16* k0 = kp + t0 * a.k_sl;
    const __bf16* v0 = vp + t0 * a.v_sl;
    const float* w0 = CHANNEL ? lwp + t0 * a.H * a.d : nullptr;
    const int tq = t * (int)a.q_sl, tk = t * (int)a.k_sl, tv = t * (int)a.v_sl, tw = t * a.H * a.d;
#pragma unroll
    for (int g = 0; g < 2 * DT; ++g) {
      const int ch = chan(g >> 1, g & 1) < a.d ? chan(g >> 1, g & 1) : 0;
      if constexpr (!STATE_ONLY) s.q[g] = *reinterpret_cast<const bf16x4*>(q0 + (tq + ch));
      s.k[g] = *reinterpret_cast<const bf16x4*>(k0 + (tk + ch));
      if constexpr (CHANNEL) s.lw[g] = *reinterpret_cast<const f32x4*>(w0 + (tw + ch));
    }
#pragma unroll
    for (int f = 0; f < 4; ++f) {
      const int col = col_base + half * 64 + quad * 16 + f * 4;
      s.v[f] = *reinterpret_cast<const bf16x4*>(v0 + (tv + (col < a.dv ? col : 0)));
    }
  };

  // the next 64 tokens are asked for as soon as these are in registers, or where those are scarce behind P
  constexpr bool LATE = CHANNEL && !STATE_ONLY && HALVES > 1;
  Stage cur;
  if (first < last) fetch(cur, first);
  for (int chunk = first; chunk < last; ++chunk) {
    const int left = a.L - chunk * kScanTokens, n = left < kScanTokens ? left : kScanTokens;
    const int t = blk * 16 + l16;  // this lane's token
    const bool live = t < n;
    float q[STATE_ONLY ? 1 : E], k[E], w[CHANNEL ? E : 1];
#pragma unroll
    for (int i = 0; i < E; ++i) {
      if constexpr (!STATE_ONLY) q[i] = to_f32(cur.q[i >> 2][i & 3]);
      k[i] = to_f32(cur.k[i >> 2][i & 3]);
    }
    if (a.silu) {  // (one branch for all of them)
#pragma unroll
      for (int i = 0; i < E; ++i) {
        if constexpr (!STATE_ONLY) q[i] = round_to<__bf16>(silu_exact(q[i]));
        k[i] = round_to<__bf16>(silu_exact(k[i]));
      }
    }
#pragma unroll
    for (int g = 0; g < 2 * DT; ++g) {
      const bool in = live && chan(g >> 1, g & 1) < a.d;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        if constexpr (!STATE_ONLY) q[g * 4 + j] = in ? q[g * 4 + j] : 0.f;
        k[g * 4 + j] = in ? k[g * 4 + j] : 0.f;
        if constexpr (CHANNEL) w[g * 4 + j] = in ? __builtin_amdgcn_exp2f(cur.lw[g][j]) : 1.f;
      }
    }

    if constexpr (HALVES > 1) __builtin_amdgcn_sched_barrier(0);
    f32x4 diag = {0.f, 0.f, 0.f, 0.f};  // the weights inside the 16 tokens: column t, rows s = 4 quad + i
    if constexpr (CHANNEL && !STATE_ONLY) {
      const int rel = l16 - quad * 4;  // row i is j tokens back where rel = j + i
      float sum = 0.f;
#pragma unroll
      for (int g = 0; g < 2 * DT; ++g) {
        const int ch = chan(g >> 1, g & 1) < a.d ? chan(g >> 1, g & 1) : 0;
        const bf16x4 u = *reinterpret_cast<const bf16x4*>(static_cast<const __bf16*>(a.u) + (long)h * a.d + ch);
#pragma unroll
        for (int j = 0; j < 4; ++j) sum = __builtin_fmaf(q[g * 4 + j] * to_f32(u[j]), k[g * 4 + j], sum);
      }
      sum = quad_rows_sum(sum);
#pragma unroll
      for (int i = 0; i < 4; ++i) diag[i] = rel == i ? sum : diag[i];
      float x[E], before[E];
#pragma unroll
      for (int i = 0; i < E; ++i) {
        x[i] = row_moved<0x111>(k[i]);
        before[i] = row_moved<0x111>(w[i]);  // of the token before
      }
      constexpr int kUnroll = 3;  // (few steps in flight: registers are scarce)
#pragma unroll kUnroll
      for (int j = 1; j < 16; ++j) {
        sum = 0.f;
#pragma unroll
        for (int i = 0; i < E; ++i) {
          sum = __builtin_fmaf(q[i], x[i], sum);
          x[i] = row_moved<0x111>(x[i]) * before[i];
        }
        sum = quad_rows_sum(sum);
#pragma unroll
        for (int i = 0; i < 4; ++i) diag[i] = rel == j + i ? sum : diag[i];
      }
    }

    __builtin_amdgcn_sched_barrier(0);
    uint32_t vv[8];
    {
      float v[16];
#pragma unroll
      for (int j = 0; j < 16; ++j) v[j] = to_f32(cur.v[j >> 2][j & 3]);
      if (a.silu) {
#pragma unroll
        for (int j = 0; j < 16; ++j) v[j] = silu_exact(v[j]);
      }
#pragma unroll
      for (int f = 0; f < 4; ++f) {
        const bool in = live && col_base + half * 64 + quad * 16 + f * 4 < a.dv;
#pragma unroll
        for (int j = 0; j < 2; ++j) vv[f * 2 + j] = in ? pack_bf16(v[f * 4 + 2 * j], v[f * 4 + 2 * j + 1]) : 0u;
      }
    }
    if (!LATE && chunk + 1 < last) fetch(cur, chunk + 1);
    lds_barrier();  // every wavefront is done with the 64 tokens before
#pragma unroll
    for (int j = 0; j < 8; ++j)
      store_pair(&lds.vt[(half * 64 + quad * 16 + 2 * j) * TS + t], &lds.vt[(half * 64 + quad * 16 + 2 * j + 1) * TS + t], vv[j]);
    if constexpr (CHANNEL) {
      if constexpr (HALVES > 1) __builtin_amdgcn_sched_barrier(0);
      // q decayed from the start of these 16 tokens, k to their end
      if constexpr (!STATE_ONLY) {
        float prefix[E];
#pragma unroll
        for (int i = 0; i < E; ++i) prefix[i] = w[i];
#pragma unroll
        for (int i = 0; i < E; i += 4) row_prefix4(prefix + i, q + i);
      }
#pragma unroll
      for (int i = 0; i < E; i += 4) row_suffix4(w + i, k + i);
      // (the product over all 16 is lane 0's suffix)
      if (l16 == 0) {
#pragma unroll
        for (int i = 0; i < E; i += 4) *reinterpret_cast<f32x4*>(&lds.total[blk][chan_of(i)]) = f32x4{w[i], w[i + 1], w[i + 2], w[i + 3]};
      }
      if constexpr (!STATE_ONLY) {
#pragma unroll
        for (int c = 0; c < DT; ++c) {
          bf16x8 hi, lo;
          split8(k + c * 8, hi, lo);
          *reinterpret_cast<bf16x8*>(&lds.k.hi[t * RS + ch0 + c * 32 + quad * 8]) = hi;
          *reinterpret_cast<bf16x8*>(&lds.k.lo[t * RS + ch0 + c * 32 + quad * 8]) = lo;
        }
      }
    } else {
      const float f = __builtin_amdgcn_exp2f(head_l2 * (float)(n - 1 - t > 0 ? n - 1 - t : 0));
#pragma unroll
      for (int i = 0; i < E; i += 2) {
        uint32_t hi, lo;
        split2(k[i] * f, k[i + 1] * f, hi, lo);
        store_pair(&lds.kt_hi[chan_of(i) * TS + t], &lds.kt_hi[(chan_of(i) + 1) * TS + t], hi);
        store_pair(&lds.kt_lo[chan_of(i) * TS + t], &lds.kt_lo[(chan_of(i) + 1) * TS + t], lo);
      }
      if constexpr (!STATE_ONLY) {
#pragma unroll
        for (int c = 0; c < DT; ++c) {
          u32x4 q4, k4;
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            q4[e] = pack_bf16(q[c * 8 + 2 * e], q[c * 8 + 2 * e + 1]);
            k4[e] = pack_bf16(k[c * 8 + 2 * e], k[c * 8 + 2 * e + 1]);
          }
          *reinterpret_cast<u32x4*>(&lds.k.hi[t * RS + ch0 + c * 32 + quad * 8]) = k4;
          *reinterpret_cast<u32x4*>(&lds.q_hi[t * RS + ch0 + c * 32 + quad * 8]) = q4;
        }
      }
    }
    lds_barrier();

    if constexpr (CHANNEL) {
      const int ch = threadIdx.x;
      if (ch < Lds::CH) {
        const float all = (lds.total[0][ch] * lds.total[1][ch]) * (lds.total[2][ch] * lds.total[3][ch]);
        lds.all[ch] = all;
        if constexpr (STATE_ONLY) seg_total *= all;
      }
    }
    f32x4 P[STATE_ONLY ? 1 : 4];  // P^T tiles: column t of this wavefront's 16 tokens, rows s of 16 tokens j
    if constexpr (CHANNEL) {
#pragma unroll
      for (int i = 0; i < E; i += 4) {
        f32x4 x = {k[i], k[i + 1], k[i + 2], k[i + 3]};
#pragma unroll
        for (int m = 1; m < 4; ++m)  // the 16-token groups behind this one
          if (m > blk) x *= *reinterpret_cast<const f32x4*>(&lds.total[m][chan_of(i)]);
#pragma unroll
        for (int e = 0; e < 4; e += 2) {
          const int ch = chan_of(i) + e;
          uint32_t hi, lo;
          split2(x[e], x[e + 1], hi, lo);
          store_pair(&lds.kt_hi[ch * TS + t], &lds.kt_hi[(ch + 1) * TS + t], hi);
          store_pair(&lds.kt_lo[ch * TS + t], &lds.kt_lo[(ch + 1) * TS + t], lo);
        }
      }
      if constexpr (!STATE_ONLY) {
#pragma unroll
        for (int j = 0; j < 4; ++j) P[j] = f32x4{0.f, 0.f, 0.f, 0.f};
        // q scaled to the start of its own 16 tokens, then by the groups in between, nearest first
#pragma unroll
        for (int step = 1; step <= 4; ++step) {
          __builtin_amdgcn_sched_barrier(0);
          const int j = blk - step;  // the last round scales to the start of the 64 tokens
          if (j < -1) break;
          bf16x8 hi[DT], lo[DT];
#pragma unroll
          for (int c = 0; c < DT; ++c) split8(q + c * 8, hi[c], lo[c]);
          if (j >= 0) {
            f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int c = 0; c < DT; ++c) {
              const bf16x8 kh = *reinterpret_cast<const bf16x8*>(&lds.k.hi[(j * 16 + l16) * RS + ch0 + c * 32 + quad * 8]);
              const bf16x8 kl = *reinterpret_cast<const bf16x8*>(&lds.k.lo[(j * 16 + l16) * RS + ch0 + c * 32 + quad * 8]);
              acc = mfma_16(kh, hi[c], acc);
              acc = mfma_16(kl, hi[c], acc);
              acc = mfma_16(kh, lo[c], acc);
            }
#pragma unroll
            for (int m = 0; m < 3; ++m) P[m] = m == j ? acc : P[m];
#pragma unroll
            for (int i = 0; i < E; i += 4) {
              const f32x4 f = *reinterpret_cast<const f32x4*>(&lds.total[j][chan_of(i)]);
#pragma unroll
              for (int e = 0; e < 4; ++e) q[i + e] *= f[e];
            }
          } else {
#pragma unroll
            for (int c = 0; c < DT; ++c) {
              *reinterpret_cast<bf16x8*>(&lds.q_hi[t * RS + ch0 + c * 32 + quad * 8]) = hi[c];
              *reinterpret_cast<bf16x8*>(&lds.q_lo[t * RS + ch0 + c * 32 + quad * 8]) = lo[c];
            }
          }
        }
#pragma unroll
        for (int m = 0; m < 4; ++m) P[m] = m == blk ? diag : P[m];
      }
    } else if constexpr (!STATE_ONLY) {
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        P[j] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (j > blk) continue;
#pragma unroll
        for (int c = 0; c < DT; ++c) {
          const bf16x8 k8 = *reinterpret_cast<const bf16x8*>(&lds.k.hi[(j * 16 + l16) * RS + ch0 + c * 32 + quad * 8]);
          const bf16x8 q8 = *reinterpret_cast<const bf16x8*>(&lds.q_hi[t * RS + ch0 + c * 32 + quad * 8]);
          P[j] = mfma_16(k8, q8, P[j]);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int dist = t - (j * 16 + quad * 4 + i);
          P[j][i] = dist >= 0 ? P[j][i] * __builtin_amdgcn_exp2f(head_l2 * (float)dist) : 0.f;
        }
      }
    }
    lds_barrier();  // k is not read any more: P goes into its place
    if constexpr (!STATE_ONLY) {
      if constexpr (HALVES > 1) {
        if (half == 1) {
#pragma unroll
          for (int j = 0; j < 4; ++j) lds.p.part[(blk * 4 + j) * 64 + lane] = P[j];
        }
        lds_barrier();
        if (half == 0) {
#pragma unroll
          for (int j = 0; j < 4; ++j) P[j] += lds.p.part[(blk * 4 + j) * 64 + lane];
        }
      }
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        typedef __attribute__((ext_vector_type(2))) uint32_t u32x2;
        u32x2 hi, lo;
#pragma unroll
        for (int i = 0; i < 2; ++i) {
          uint32_t x, y;
          split2(P[j][2 * i], P[j][2 * i + 1], x, y);
          hi[i] = x, lo[i] = y;
        }
        if (half == 0 && j <= (blk | 1)) {
          *reinterpret_cast<u32x2*>(&lds.p.hi[t * TS + j * 16 + quad * 4]) = hi;
          *reinterpret_cast<u32x2*>(&lds.p.lo[t * TS + j * 16 + quad * 4]) = lo;
        }
      }
      lds_barrier();
    }
    if (LATE && chunk + 1 < last) fetch(cur, chunk + 1);
    if (has_cols) {
      bf16x8 v8[2];
#pragma unroll
      for (int g = 0; g < 2; ++g) v8[g] = *reinterpret_cast<const bf16x8*>(&lds.vt[(wave * 16 + l16) * TS + g * 32 + quad * 8]);
      if constexpr (!STATE_ONLY) {
        bf16x8 sh[DA], sl[DA];
#pragma unroll
        for (int c = 0; c < DA; ++c) {
          const float x[8] = {S[2 * c][0], S[2 * c][1], S[2 * c][2], S[2 * c][3], S[2 * c + 1][0], S[2 * c + 1][1], S[2 * c + 1][2], S[2 * c + 1][3]};
          split8(x, sh[c], sl[c]);
        }
#pragma unroll
        for (int tb = 0; tb < 4; ++tb) {
          if (tb > 0 && DA > 1) __builtin_amdgcn_sched_barrier(0);  // (one group's operands in registers at a time)
          const int tok = tb * 16 + l16;
          f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int c = 0; c < DA; ++c) {
            const bf16x8 qh = *reinterpret_cast<const bf16x8*>(&lds.q_hi[tok * RS + c * 32 + quad * 8]);
            acc = mfma_16(sh[c], qh, acc);
            acc = mfma_16(sl[c], qh, acc);
            if constexpr (CHANNEL) {
              const bf16x8 ql = *reinterpret_cast<const bf16x8*>(&lds.q_lo[tok * RS + c * 32 + quad * 8]);
              acc = mfma_16(sh[c], ql, acc);
            }
          }
          if constexpr (!CHANNEL) acc *= __builtin_amdgcn_exp2f(head_l2 * (float)(tok + 1));
#pragma unroll
          for (int g = 0; g < 2; ++g) {
            if (g * 2 > tb) continue;
            const bf16x8 ph = *reinterpret_cast<const bf16x8*>(&lds.p.hi[tok * TS + g * 32 + quad * 8]);
            const bf16x8 pl = *reinterpret_cast<const bf16x8*>(&lds.p.lo[tok * TS + g * 32 + quad * 8]);
            acc = mfma_16(v8[g], ph, acc);
            acc = mfma_16(v8[g], pl, acc);
          }
          if (tok < n && dv0 + quad * 4 < a.dv) {
            bf16x4 out;
#pragma unroll
            for (int i = 0; i < 4; ++i) out[i] = (__bf16)acc[i];
            *reinterpret_cast<bf16x4*>(static_cast<__bf16*>(a.o) + b * a.o_sb + (long)(chunk * kScanTokens + tok) * a.o_sl +
                                       (long)h * a.dv + dv0 + quad * 4) = out;
          }
        }
      }
      // the state behind the 64 tokens
#pragma unroll
      for (int ct = 0; ct < 2 * DA; ++ct) {
        if (HALVES > 1 && ct % 2 == 0) __builtin_amdgcn_sched_barrier(0);
        if constexpr (CHANNEL) {
          S[ct] *= *reinterpret_cast<const f32x4*>(&lds.all[ct * 16 + quad * 4]);
        } else {
          S[ct] *= __builtin_amdgcn_exp2f(head_l2 * (float)n);
        }
#pragma unroll
        for (int g = 0; g < 2; ++g) {
          const bf16x8 kh = *reinterpret_cast<const bf16x8*>(&lds.kt_hi[(ct * 16 + l16) * TS + g * 32 + quad * 8]);
          const bf16x8 kl = *reinterpret_cast<const bf16x8*>(&lds.kt_lo[(ct * 16 + l16) * TS + g * 32 + quad * 8]);
          S[ct] = mfma_16(kh, v8[g], S[ct]);
          S[ct] = mfma_16(kl, v8[g], S[ct]);
        }
      }
    }
  }
  if constexpr (CHANNEL && STATE_ONLY) {
    if (blockIdx.y == 0 && threadIdx.x < a.d) a.seg_lw[(bh * a.segs + sg) * a.dp + threadIdx.x] = seg_total;
  }
  if (!has_cols) return;
  float* to = st;
  if constexpr (STATE_ONLY) to = a.seg + ((bh * a.segs + sg) * a.dv + (col_in ? dv0 + l16 : 0)) * a.dp;
  if (STATE_ONLY || sg == a.segs - 1) {
#pragma unroll
    for (int ct = 0; ct < 2 * DA; ++ct) {
      const int ch = ct * 16 + quad * 4;
      if (col_in && ch < a.d) *reinterpret_cast<f32x4*>(to + ch) = S[ct];
    }
  }
}

// What each segment adds -> the state at its start, four key channels of a value channel per thread.
__global__ __launch_bounds__(256) void decay_join_kernel(const DecayScanArgs a) {
  const int pieces = a.dp / 4;
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= (long)a.B * a.H * a.dv * pieces) return;
  const int ch = (int)(i % pieces) * 4;
  const long row = i / pieces, bh = row / a.dv, col = row % a.dv;
  if (ch >= a.d) return;
  float* st = a.state + (bh * a.dv + col) * a.dp + ch;
  f32x4 S = {0.f, 0.f, 0.f, 0.f};
  if (!a.fresh) S = *reinterpret_cast<const f32x4*>(st);
  const float head_l2 = a.lw != nullptr ? 0.f : a.head_lw[bh % a.H];
  for (int s = 0; s < a.segs; ++s) {
    float* p = a.seg + ((bh * a.segs + s) * a.dv + col) * a.dp + ch;
    f32x4 add = {0.f, 0.f, 0.f, 0.f};
    if (s + 1 < a.segs) add = *reinterpret_cast<const f32x4*>(p);
    *reinterpret_cast<f32x4*>(p) = S;
    if (s + 1 == a.segs) return;
    f32x4 l;
    if (a.lw != nullptr) {
      l = *reinterpret_cast<const f32x4*>(a.seg_lw + (bh * a.segs + s) * a.dp + ch);
    } else {
      const int lo = s * a.seg_chunks * kScanTokens, hi = (s + 1) * a.seg_chunks * kScanTokens;
      const float f = __builtin_amdgcn_exp2f(head_l2 * (float)((hi < a.L ? hi : a.L) - lo));
      l = f32x4{f, f, f, f};
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) S[j] = __builtin_fmaf(S[j], l[j], add[j]);
  }
}

// ---- any element type and size ----
// 16 lanes per value channel, channels l16 + 16 i of the key; 16 value channels per workgroup.
template <typename T, int CPT, bool CHANNEL>
__global__ __launch_bounds__(256) void decay_scan_any_kernel(const DecayScanArgs a) {
  constexpr int kTile = 8;  // tokens staged at once
  constexpr int CH = 16 * CPT;
  __shared__ float sq[kTile][CH], sk[kTile][CH], sw[CHANNEL ? kTile : 1][CH], sv[kTile][16];
  const int tid = threadIdx.x, l16 = tid & 15, col = tid >> 4;
  const int b = blockIdx.x / a.H, h = blockIdx.x % a.H, dv0 = blockIdx.y * 16;
  const bool col_in = dv0 + col < a.dv;
  const T* qp = static_cast<const T*>(a.q) + b * a.q_sb + (long)h * a.d;
  const T* kp = static_cast<const T*>(a.k) + b * a.k_sb + (long)h * a.d;
  const T* vp = static_cast<const T*>(a.v) + b * a.v_sb + (long)h * a.dv;
  float* st = a.state + (((long)b * a.H + h) * a.dv + (col_in ? dv0 + col : 0)) * a.dp;
  float S[CPT], u[CPT];
  const float head_w = CHANNEL ? 0.f : a.head_lw[a.H + h];
#pragma unroll
  for (int i = 0; i < CPT; ++i) {
    const int c = l16 + 16 * i;
    S[i] = !a.fresh && col_in && c < a.d ? st[c] : 0.f;
    u[i] = CHANNEL && c < a.d ? to_f32(static_cast<const T*>(a.u)[(long)h * a.d + c]) : 0.f;
  }
  auto active = [&](T x) { return a.silu ? round_to<T>(silu_exact(to_f32(x))) : to_f32(x); };
  for (int t0 = 0; t0 < a.L; t0 += kTile) {
    const int n = a.L - t0 < kTile ? a.L - t0 : kTile;
    __syncthreads();
    for (int i = tid; i < kTile * CH; i += 256) {
      const int t = i / CH, c = i % CH;
      const bool in = t < n && c < a.d;
      sq[t][c] = in ? active(qp[(t0 + t) * a.q_sl + c]) : 0.f;
      sk[t][c] = in ? active(kp[(t0 + t) * a.k_sl + c]) : 0.f;
      if constexpr (CHANNEL) sw[t][c] = in ? exp2f(a.lw[(((long)b * a.L + t0 + t) * a.H + h) * a.d + c]) : 1.f;
    }
    for (int i = tid; i < kTile * 16; i += 256) {
      const int t = i / 16, c = i % 16;
      sv[t][c] = t < n && dv0 + c < a.dv ? active(vp[(t0 + t) * a.v_sl + dv0 + c]) : 0.f;
    }
    __syncthreads();
    for (int t = 0; t < n; ++t) {
      const float v = sv[t][col];
      float o = 0.f;
#pragma unroll
      for (int i = 0; i < CPT; ++i) {
        const int c = l16 + 16 * i;
        const float kv = sk[t][c] * v;
        if constexpr (CHANNEL) {
          o = __builtin_fmaf(__builtin_fmaf(u[i], kv, S[i]), sq[t][c], o);
          S[i] = __builtin_fmaf(sw[t][c], S[i], kv);
        } else {
          S[i] = __builtin_fmaf(head_w, S[i], kv);
          o = __builtin_fmaf(S[i], sq[t][c], o);
        }
      }
      o = sum16(o);
      if (l16 == 0 && col_in) static_cast<T*>(a.o)[b * a.o_sb + (t0 + t) * a.o_sl + (long)h * a.dv + dv0 + col] = from_f32<T>(o);
    }
  }
#pragma unroll
  for (int i = 0; i < CPT; ++i) {
    const int c = l16 + 16 * i;
    if (col_in && c < a.d) st[c] = S[i];
  }
}

// ---- one token per sequence: one workgroup per (sequence, head) ----
struct DecayStepArgs {
  const void* q;
  const void* k;
  const void* v;
  const float* head_lw;
  const void* u;
  const void* hid;   // (B, R): the low-rank part of the channel decays before tanh
  const void* w2;    // (H * d, R)
  const void* w0;    // (H * d)
  const void* gate;  // (B, H * dv)
  const void* norm_w;
  float* state;
  void* o;
  const int32_t* pos;
  int pos_host;
  int B, H, d, dv, dp, R;
  long q_sb, k_sb, v_sb, h_sb, g_sb, o_sb;
  int silu;
  float eps;
};

// NT threads; LPR lanes per value channel, four key channels each; RPT value channels per thread.
template <typename T, int NT, int LPR, int RPT, bool CHANNEL>
__global__ __launch_bounds__(NT) void decay_step_kernel(const DecayStepArgs a) {
  extern __shared__ float smem[];
  constexpr int kRows = NT / LPR;  // value channels at a time
  const int tid = threadIdx.x, lane = tid & 63;
  const int b = blockIdx.x / a.H, h = blockIdx.x % a.H;
  const int pos = row_pos(a.pos, a.pos_host, b);
  if (pos < 0) return;
  float* sq = smem;             // [4 LPR], zeros behind d
  float* sk = sq + 4 * LPR;     // [4 LPR]
  float* sw = sk + 4 * LPR;     // [4 LPR]
  float* su = sw + 4 * LPR;     // [4 LPR]
  float* sv = su + 4 * LPR;     // [RPT * kRows]
  float* so = sv + RPT * kRows; // [RPT * kRows]
  float* th = so + RPT * kRows; // [R]
  // the state is asked for first
  const int piece = tid % LPR, r0 = tid / LPR, c0 = piece * 4;
  const bool in_c = c0 < a.d;
  float* st = a.state + ((long)b * a.H + h) * a.dv * a.dp;
  f32x4 S[RPT];
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int row = r0 + i * kRows;
    const bool in = in_c && row < a.dv;
    const f32x4 x = *reinterpret_cast<const f32x4*>(st + (in ? (long)row * a.dp + c0 : 0));
#pragma unroll
    for (int j = 0; j < 4; ++j) S[i][j] = in && pos > 0 && c0 + j < a.d ? x[j] : 0.f;
  }
  auto active = [&](T x) { return a.silu ? round_to<T>(silu_exact(to_f32(x))) : to_f32(x); };
  for (int c = tid; c < 4 * LPR; c += NT) {
    const bool in = c < a.d;
    const long at = (long)h * a.d + (in ? c : 0);
    const T xq = static_cast<const T*>(a.q)[b * a.q_sb + at], xk = static_cast<const T*>(a.k)[b * a.k_sb + at];
    sq[c] = in ? active(xq) : 0.f;
    sk[c] = in ? active(xk) : 0.f;
    if constexpr (CHANNEL) su[c] = in ? to_f32(static_cast<const T*>(a.u)[at]) : 0.f;
  }
  for (int c = tid; c < RPT * kRows; c += NT)
    sv[c] = c < a.dv ? active(static_cast<const T*>(a.v)[b * a.v_sb + (long)h * a.dv + c]) : 0.f;
  if constexpr (CHANNEL) {
    for (int j = tid; j < a.R; j += NT) th[j] = tanh_f(to_f32(static_cast<const T*>(a.hid)[b * a.h_sb + j]));
    __syncthreads();
    // four lanes per key channel
    for (int c = tid >> 2; c < 4 * LPR; c += NT / 4) {
      const bool in = c < a.d;
      const long at = (long)h * a.d + (in ? c : 0);
      const T* w = static_cast<const T*>(a.w2) + at * a.R;
      float z = 0.f;
      for (int j = tid & 3; j < a.R; j += 4) z = __builtin_fmaf(to_f32(w[j]), th[j], z);
      z += __shfl_xor(z, 1, 64);
      z += __shfl_xor(z, 2, 64);
      z += to_f32(static_cast<const T*>(a.w0)[at]);
      if ((tid & 3) == 0) sw[c] = in ? expf(-expf(z)) : 0.f;
    }
  }
  __syncthreads();
  float q[4], k[4], w[4], u[4];
  const float head_w = CHANNEL ? 0.f : a.head_lw[a.H + h];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    q[j] = sq[c0 + j], k[j] = sk[c0 + j];
    w[j] = CHANNEL ? sw[c0 + j] : head_w;
    u[j] = CHANNEL ? su[c0 + j] : 0.f;
  }
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int row = r0 + i * kRows;
    const float v = sv[row];
    float o = 0.f;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const float kv = k[j] * v;
      if constexpr (CHANNEL) {
        o = __builtin_fmaf(__builtin_fmaf(u[j], kv, S[i][j]), q[j], o);
        S[i][j] = __builtin_fmaf(w[j], S[i][j], kv);
      } else {
        S[i][j] = __builtin_fmaf(w[j], S[i][j], kv);
        o = __builtin_fmaf(S[i][j], q[j], o);
      }
    }
    if (in_c && row < a.dv) *reinterpret_cast<f32x4*>(st + (long)row * a.dp + c0) = S[i];
    if constexpr (LPR == 8) {
      o = sum8(o);
    } else if constexpr (LPR >= 16) {
      o = sum16(o);
      if constexpr (LPR >= 32) o += __shfl_xor(o, 16, 64);
      if constexpr (LPR >= 64) o += __shfl_xor(o, 32, 64);
    }
    if (piece == 0) so[row] = o;
  }
  __syncthreads();
  T* out = static_cast<T*>(a.o) + b * a.o_sb + (long)h * a.dv;
  if constexpr (CHANNEL) {
    float ss = 0.f;
    for (int c = lane; c < a.dv; c += 64) ss = __builtin_fmaf(so[c], so[c], ss);
    const float r = 1.0f / sqrtf(wave_sum(ss) / (float)a.dv + a.eps);
    const T* gate = static_cast<const T*>(a.gate) + b * a.g_sb + (long)h * a.dv;
    const T* nw = static_cast<const T*>(a.norm_w) + (long)h * a.dv;
    for (int c = tid; c < a.dv; c += NT) out[c] = from_f32<T>(so[c] * r * to_f32(nw[c]) * silu_exact(to_f32(gate[c])));
  } else {
    for (int c = tid; c < a.dv; c += NT) out[c] = from_f32<T>(so[c]);
  }
}

// ---- o / rms(o) * w * act(g) over groups of n elements of a row ----
struct GroupNormArgs {
  const void* o;
  const void* w;     // (G, n)
  const void* gate;
  void* y;
  long rows;         // B L G
  int L, G, n;
  long o_sb, o_sl, g_sb, g_sl, y_sb, y_sl;
  float eps, scale;
  int sigmoid;
};

template <typename T, bool VEC, int LPR>
__global__ __launch_bounds__(256) void group_norm_gate_kernel(const GroupNormArgs a) {
  constexpr int N = VEC ? Pack<T>::kN : 1;
  constexpr int KEEP = LPR == 64 ? 4 : 2;  // pieces of the row a lane keeps between the two passes
  const long row0 = (long)blockIdx.x * (256 / LPR) + threadIdx.x / LPR;
  const bool live = row0 < a.rows;
  const long row = live ? row0 : a.rows - 1;
  const int lane = threadIdx.x % LPR;
  const int g = (int)(row % a.G);
  const long bl = row / a.G, b = bl / a.L, l = bl % a.L;
  const T* o = static_cast<const T*>(a.o) + b * a.o_sb + l * a.o_sl + (long)g * a.n;
  const T* gate = static_cast<const T*>(a.gate) + b * a.g_sb + l * a.g_sl + (long)g * a.n;
  T* y = static_cast<T*>(a.y) + b * a.y_sb + l * a.y_sl + (long)g * a.n;
  const T* w = static_cast<const T*>(a.w) + (long)g * a.n;
  auto load = [&](const T* p, float (&x)[N]) {
    if constexpr (VEC)
      load_vec<T, N>(p, x);
    else
      x[0] = to_f32(*p);
  };
  float keep[KEEP][N], gk[KEEP][N], wk[KEEP][N];
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int e = (lane + i * LPR) * N;
    load(o + (e < a.n ? e : 0), keep[i]);
    load(gate + (e < a.n ? e : 0), gk[i]);
    load(w + (e < a.n ? e : 0), wk[i]);
  }
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < KEEP; ++i)
#pragma unroll
    for (int j = 0; j < N; ++j) ss = (lane + i * LPR) * N < a.n ? __builtin_fmaf(keep[i][j], keep[i][j], ss) : ss;
  for (int e = (lane + KEEP * LPR) * N; e < a.n; e += LPR * N) {
    float x[N];
    load(o + e, x);
#pragma unroll
    for (int j = 0; j < N; ++j) ss = __builtin_fmaf(x[j], x[j], ss);
  }
  ss = LPR == 8 ? sum8(ss) : LPR == 16 ? sum16(ss) : wave_sum(ss);
  const float r = a.scale / sqrtf(ss / (float)a.n + a.eps);
  auto finish = [&](int e, const float (&x)[N], const float (&gv)[N], const float (&wv)[N]) {
    float out[N];
#pragma unroll
    for (int j = 0; j < N; ++j) out[j] = x[j] * r * wv[j] * (a.sigmoid ? sigmoid_f(gv[j]) : silu_exact(gv[j]));
    if (live) {
      if constexpr (VEC)
        store_vec<T, N>(y + e, out);
      else
        y[e] = from_f32<T>(out[0]);
    }
  };
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int e = (lane + i * LPR) * N;
    if (e < a.n) finish(e, keep[i], gk[i], wk[i]);
  }
  for (int e = (lane + KEEP * LPR) * N; e < a.n; e += LPR * N) {
    float x[N], gv[N], wv[N];
    load(o + e, x);
    load(gate + e, gv);
    load(w + e, wv);
    finish(e, x, gv, wv);
  }
}

template <typename T, bool VEC> void launch_group_norm(const GroupNormArgs& a, hipStream_t s) {
  const int N = VEC ? Pack<T>::kN : 1;
  const int lpr = a.n <= 8 * N ? 8 : a.n <= 32 * N ? 16 : 64;
  const int per = 256 / lpr;
  const dim3 grid((unsigned)((a.rows + per - 1) / per)), block(256);
  if (lpr == 8)
    hipLaunchKernelGGL((group_norm_gate_kernel<T, VEC, 8>), grid, block, 0, s, a);
  else if (lpr == 16)
    hipLaunchKernelGGL((group_norm_gate_kernel<T, VEC, 16>), grid, block, 0, s, a);
  else
    hipLaunchKernelGGL((group_norm_gate_kernel<T, VEC, 64>), grid, block, 0, s, a);
}

template <int DT, int HALVES, bool CHANNEL> int launch_decay_mfma(const DecayScanArgs& a, hipStream_t s) {
  const size_t bytes = sizeof(ScanLds<DT, HALVES, CHANNEL>);
  if (bytes > 64 * 1024) {
    static const hipError_t once = [&] {
      hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(decay_scan_mfma_kernel<DT, HALVES, CHANNEL, false>),
                                         hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes);
      if (e != hipSuccess) return e;
      return hipFuncSetAttribute(reinterpret_cast<const void*>(decay_scan_mfma_kernel<DT, HALVES, CHANNEL, true>),
                                 hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes);
    }();
    BASED_REQUIRE(once == hipSuccess, BASED_ERR_LAUNCH, "decay_scan: %zu bytes of LDS refused: %s", bytes, hipGetErrorString(once));
  }
  const int cols = 64 * HALVES;
  dim3 grid((unsigned)(a.B * a.H), (unsigned)((a.dv + cols - 1) / cols), (unsigned)a.segs);
  if (a.segs > 1) {
    dim3 all_but_last = grid;
    all_but_last.z -= 1;
    hipLaunchKernelGGL((decay_scan_mfma_kernel<DT, HALVES, CHANNEL, true>), all_but_last, dim3(256 * HALVES), bytes, s, a);
    const long items = (long)a.B * a.H * a.dv * (a.dp / 4);
    hipLaunchKernelGGL(decay_join_kernel, dim3((unsigned)((items + 255) / 256)), dim3(256), 0, s, a);
  }
  hipLaunchKernelGGL((decay_scan_mfma_kernel<DT, HALVES, CHANNEL, false>), grid, dim3(256 * HALVES), bytes, s, a);
  return BASED_OK;
}

template <bool CHANNEL> int launch_decay_scan_mfma(const DecayScanArgs& a, hipStream_t s) {
  if (a.d <= 32) return launch_decay_mfma<1, 1, CHANNEL>(a, s);
  if (a.d <= 64) return launch_decay_mfma<2, 1, CHANNEL>(a, s);
  return launch_decay_mfma<2, 2, CHANNEL>(a, s);
}

template <typename T, bool CHANNEL> void launch_decay_scan_any(const DecayScanArgs& a, hipStream_t s) {
  const dim3 grid((unsigned)(a.B * a.H), (unsigned)((a.dv + 15) / 16));
  const int cpt = (a.d + 15) / 16;
  if (cpt <= 4)
    hipLaunchKernelGGL((decay_scan_any_kernel<T, 4, CHANNEL>), grid, dim3(256), 0, s, a);
  else if (cpt <= 8)
    hipLaunchKernelGGL((decay_scan_any_kernel<T, 8, CHANNEL>), grid, dim3(256), 0, s, a);
  else
    hipLaunchKernelGGL((decay_scan_any_kernel<T, 16, CHANNEL>), grid, dim3(256), 0, s, a);
}

template <typename T, int NT, int LPR, int RPT, bool CHANNEL> void launch_decay_step_block(const DecayStepArgs& a, hipStream_t s) {
  const size_t bytes = (size_t)(16 * LPR + 2 * RPT * (NT / LPR) + (CHANNEL ? a.R : 0)) * sizeof(float);
  hipLaunchKernelGGL((decay_step_kernel<T, NT, LPR, RPT, CHANNEL>), dim3((unsigned)(a.B * a.H)), dim3(NT), bytes, s, a);
}

// Few rows of the state per thread, so that all of it is in flight at once.
template <typename T, int LPR, bool CHANNEL> void launch_decay_step_rows(const DecayStepArgs& a, hipStream_t s) {
  auto rows = [&](int nt) { return (a.dv + nt / LPR - 1) / (nt / LPR); };
  if (rows(256) <= 2)
    launch_decay_step_block<T, 256, LPR, 2, CHANNEL>(a, s);
  else if (rows(256) <= 4)
    launch_decay_step_block<T, 256, LPR, 4, CHANNEL>(a, s);
  else if (rows(256) <= 8)
    launch_decay_step_block<T, 256, LPR, 8, CHANNEL>(a, s);
  else if (rows(512) <= 8)
    launch_decay_step_block<T, 512, LPR, 8, CHANNEL>(a, s);
  else
    launch_decay_step_block<T, 1024, LPR, 16, CHANNEL>(a, s);
}

template <typename T, bool CHANNEL> void launch_decay_step(const DecayStepArgs& a, hipStream_t s) {
  const int pieces = (a.d + 3) / 4;
  if (pieces <= 8)
    launch_decay_step_rows<T, 8, CHANNEL>(a, s);
  else if (pieces <= 16)
    launch_decay_step_rows<T, 16, CHANNEL>(a, s);
  else if (pieces <= 32)
    launch_decay_step_rows<T, 32, CHANNEL>(a, s);
  else
    launch_decay_step_rows<T, 64, CHANNEL>(a, s);
}

// Segments of a scan: enough workgroups to give every SIMD two wavefronts, none shorter than four pieces of 64 tokens.
static int decay_segments(int64_t B, int64_t L, int64_t H, int64_t D, int64_t DV) {
  const int64_t cols = D <= 64 ? 64 : 128, chunks = (L + kScanTokens - 1) / kScanTokens, wgs = B * H * ((DV + cols - 1) / cols);
  int64_t segs = ((D <= 64 ? 512 : 256) + wgs - 1) / wgs;
  if (segs > chunks / 4) segs = chunks / 4;
  if (segs > 64) segs = 64;
  return segs < 2 ? 1 : (int)segs;
}

}  // namespace based

extern "C" BASED_API int64_t based_decay_scan_work(int64_t B, int64_t L, int64_t H, int64_t D, int64_t DV, int64_t state_row) {
  if (B <= 0 || L <= 0 || H <= 0 || D <= 0 || DV <= 0) return 0;
  const int64_t segs = based::decay_segments(B, L, H, D, DV);
  return segs <= 1 ? 0 : B * H * segs * (DV + 1) * state_row;
}

extern "C" BASED_API int based_decay_scan(const void* q, const void* k, const void* v, const float* channel_log2, const float* head_decay,
                                          const void* bonus, float* state, float* work, void* o, int64_t B, int64_t L, int64_t H,
                                          int64_t D, int64_t DV, int64_t state_row, int64_t q_sb, int64_t q_sl, int64_t k_sb,
                                          int64_t k_sl, int64_t v_sb, int64_t v_sl, int64_t o_sb, int64_t o_sl, int activation, int fresh,
                                          int io_dtype, void* stream) {
  using namespace based;
  BASED_REQUIRE(q && k && v && state && o, BASED_ERR_ARG, "decay_scan: null pointer argument");
  BASED_REQUIRE((channel_log2 != nullptr) != (head_decay != nullptr), BASED_ERR_ARG, "decay_scan: decays per channel or per head");
  BASED_REQUIRE((channel_log2 != nullptr) == (bonus != nullptr), BASED_ERR_ARG, "decay_scan: the bonus belongs to channel decays");
  BASED_REQUIRE(B >= 0 && L >= 0 && H > 0 && D > 0 && DV > 0, BASED_ERR_ARG, "decay_scan: bad sizes");
  BASED_REQUIRE(D <= 256, BASED_ERR_SHAPE, "decay_scan: key size %ld (at most 256)", (long)D);
  BASED_REQUIRE(state_row >= D && state_row % 4 == 0 && aligned_to(state, 16) && aligned_to(work, 16), BASED_ERR_ALIGN,
                "decay_scan: state rows must be whole 16-byte pieces");
  BASED_REQUIRE(activation == BASED_ACT_NONE || activation == BASED_ACT_SILU, BASED_ERR_ARG, "decay_scan: unknown activation");
  BASED_REQUIRE(io_dtype == BASED_BF16 || io_dtype == BASED_F32, BASED_ERR_DTYPE, "decay_scan: bad dtype");
  BASED_REQUIRE(B * H < (1ll << 31) && L < (1ll << 31) && DV < (1ll << 20), BASED_ERR_SHAPE, "decay_scan: grid too large");
  BASED_REQUIRE(q_sl < (1ll << 24) && k_sl < (1ll << 24) && v_sl < (1ll << 24) && H * D < (1ll << 24), BASED_ERR_SHAPE, "decay_scan: rows too long");
  if (B == 0 || L == 0) return BASED_OK;
  DecayScanArgs a{q,    k,    v,    channel_log2, head_decay, bonus, state, nullptr, nullptr, o,    (int)B, (int)L, (int)H, (int)D, (int)DV,
                  (int)state_row, q_sb, q_sl, k_sb, k_sl, v_sb, v_sl, o_sb, o_sl, 1, (int)((L + kScanTokens - 1) / kScanTokens),
                  activation == BASED_ACT_SILU, fresh};
  hipStream_t s = static_cast<hipStream_t>(stream);
  const bool vec = io_dtype == BASED_BF16 && D <= 128 && D % 4 == 0 && DV % 4 == 0 && q_sb % 4 == 0 && q_sl % 4 == 0 && k_sb % 4 == 0 &&
                   k_sl % 4 == 0 && v_sb % 4 == 0 && v_sl % 4 == 0 && o_sb % 4 == 0 && o_sl % 4 == 0 && aligned_to(q, 8) &&
                   aligned_to(k, 8) && aligned_to(v, 8) && aligned_to(o, 8) && aligned_to(bonus, 8) && aligned_to(channel_log2, 16);
  if (vec) {
    const int segs = decay_segments(B, L, H, D, DV);
    if (segs > 1) {
      BASED_REQUIRE(work != nullptr, BASED_ERR_ARG, "decay_scan: no work space");
      a.seg_chunks = (a.seg_chunks + segs - 1) / segs;
      a.segs = (int)(((L + kScanTokens - 1) / kScanTokens + a.seg_chunks - 1) / a.seg_chunks);
      a.seg = work;
      a.seg_lw = work + B * H * a.segs * DV * state_row;
    }
    const int rc = channel_log2 != nullptr ? launch_decay_scan_mfma<true>(a, s) : launch_decay_scan_mfma<false>(a, s);
    if (rc != BASED_OK) return rc;
  } else if (io_dtype == BASED_BF16) {
    channel_log2 != nullptr ? launch_decay_scan_any<__bf16, true>(a, s) : launch_decay_scan_any<__bf16, false>(a, s);
  } else {
    channel_log2 != nullptr ? launch_decay_scan_any<float, true>(a, s) : launch_decay_scan_any<float, false>(a, s);
  }
  return check_launch("decay_scan");
}

extern "C" BASED_API int based_decay_step(const void* q, const void* k, const void* v, const float* head_decay, const void* bonus,
                                          const void* hidden, const void* w2, const void* w0, const void* gate, const void* norm_w,
                                          float* state, void* o, const int32_t* pos, int64_t pos_host, int64_t B, int64_t H, int64_t D,
                                          int64_t DV, int64_t state_row, int64_t R, int64_t q_sb, int64_t k_sb, int64_t v_sb,
                                          int64_t h_sb, int64_t g_sb, int64_t o_sb, int activation, float eps, int io_dtype,
                                          void* stream) {
  using namespace based;
  const bool channel = hidden != nullptr;
  BASED_REQUIRE(q && k && v && state && o, BASED_ERR_ARG, "decay_step: null pointer argument");
  BASED_REQUIRE(channel ? (bonus && w2 && w0 && gate && norm_w && R > 0) : head_decay != nullptr, BASED_ERR_ARG,
                "decay_step: decays are missing");
  BASED_REQUIRE(B >= 0 && H > 0 && D > 0 && DV > 0 && pos_host >= 0 && pos_host < (1ll << 31), BASED_ERR_ARG, "decay_step: bad sizes");
  BASED_REQUIRE(D <= 256 && DV <= 256 && R <= 1024, BASED_ERR_SHAPE, "decay_step: sizes %ld x %ld, rank %ld (at most 256, 256, 1024)",
                (long)D, (long)DV, (long)R);
  BASED_REQUIRE(state_row >= D && state_row % 4 == 0 && aligned_to(state, 16), BASED_ERR_ALIGN,
                "decay_step: state rows must be whole 16-byte pieces");
  BASED_REQUIRE(activation == BASED_ACT_NONE || activation == BASED_ACT_SILU, BASED_ERR_ARG, "decay_step: unknown activation");
  BASED_REQUIRE(io_dtype == BASED_BF16 || io_dtype == BASED_F32, BASED_ERR_DTYPE, "decay_step: bad dtype");
  BASED_REQUIRE(B * H < (1ll << 31), BASED_ERR_SHAPE, "decay_step: grid too large");
  if (B == 0) return BASED_OK;
  const DecayStepArgs a{q,   k,   v,    head_decay, bonus, hidden, w2, w0, gate, norm_w, state, o, pos, (int)pos_host, (int)B, (int)H,
                        (int)D, (int)DV, (int)state_row, (int)R, q_sb, k_sb, v_sb, h_sb, g_sb, o_sb, activation == BASED_ACT_SILU, eps};
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (io_dtype == BASED_BF16)
    channel ? launch_decay_step<__bf16, true>(a, s) : launch_decay_step<__bf16, false>(a, s);
  else
    channel ? launch_decay_step<float, true>(a, s) : launch_decay_step<float, false>(a, s);
  return check_launch("decay_step");
}

extern "C" BASED_API int based_group_norm_gate(const void* o, const void* weight, const void* gate, void* y, int64_t B, int64_t L,
                                               int64_t G, int64_t n, int64_t o_sb, int64_t o_sl, int64_t g_sb, int64_t g_sl,
                                               int64_t y_sb, int64_t y_sl, float eps, float scale, int activation, int io_dtype,
                                               void* stream) {
  using namespace based;
  BASED_REQUIRE(o && weight && gate && y, BASED_ERR_ARG, "group_norm_gate: null pointer argument");
  BASED_REQUIRE(B >= 0 && L >= 0 && G > 0 && n > 0, BASED_ERR_ARG, "group_norm_gate: bad sizes");
  BASED_REQUIRE(activation == BASED_ACT_SILU || activation == BASED_ACT_SIGMOID, BASED_ERR_ARG, "group_norm_gate: unknown activation");
  BASED_REQUIRE(io_dtype == BASED_BF16 || io_dtype == BASED_F32, BASED_ERR_DTYPE, "group_norm_gate: bad dtype");
  const int64_t rows = B * L * G;
  BASED_REQUIRE(rows < (1ll << 33), BASED_ERR_SHAPE, "group_norm_gate: grid too large");
  if (rows == 0) return BASED_OK;
  const GroupNormArgs a{o,    weight, gate, y,    (long)rows, (int)L, (int)G, (int)n, o_sb, o_sl, g_sb, g_sl, y_sb, y_sl, eps, scale,
                        activation == BASED_ACT_SIGMOID};
  const int p = io_dtype == BASED_BF16 ? 8 : 4;
  const bool vec = n % p == 0 && o_sb % p == 0 && o_sl % p == 0 && g_sb % p == 0 && g_sl % p == 0 && y_sb % p == 0 && y_sl % p == 0 &&
                   aligned_to(o, 16) && aligned_to(weight, 16) && aligned_to(gate, 16) && aligned_to(y, 16);
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (io_dtype == BASED_BF16)
    vec ? launch_group_norm<__bf16, true>(a, s) : launch_group_norm<__bf16, false>(a, s);
  else
    vec ? launch_group_norm<float, true>(a, s) : launch_group_norm<float, false>(a, s);
  return check_launch("group_norm_gate");
}
