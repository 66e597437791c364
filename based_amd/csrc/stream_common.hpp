// Helpers shared by the kernels of the streaming layers (norms with a scaled residual, causal
// convolutions on a ring of past inputs, grouped window attention, gated delta rule, gated linear
// recurrent unit).  Everything that enters a norm, a softmax or a recurrence is evaluated in 32 bits;
// exponentials, reciprocals and square roots are the hardware's (1 ulp) where a value per element and
// token is needed.
#pragma once

#include "common.hpp"

namespace based {

template <typename T> struct Pack;  // 16 bytes of T
template <> struct Pack<__bf16> {
  static constexpr int kN = 8;
  typedef bf16x8 type;
};
template <> struct Pack<float> {
  static constexpr int kN = 4;
  typedef f32x4 type;
};

// exp of an argument whose rounding to a power of two may cost |z| ulps: callers have |z| small, or a result
// that is far from the scale of what it is added to.
__device__ __forceinline__ float exp_f(float z) { return __builtin_amdgcn_exp2f(z * 1.4426950408889634f); }
__device__ __forceinline__ float sigmoid_f(float z) { return __builtin_amdgcn_rcpf(1.0f + exp_f(-z)); }
__device__ __forceinline__ float silu_exact(float z) { return z * sigmoid_f(z); }
__device__ __forceinline__ float softplus_f(float z) { return log1pf(expf(-fabsf(z))) + fmaxf(z, 0.0f); }
// 0.5 z (1 + tanh(t)) = z sigmoid(2 t)
__device__ __forceinline__ float gelu_tanh_f(float z) {
  return z * sigmoid_f(1.5957691216057308f * (z + 0.044715f * z * z * z));
}
// exp(2z) overflows to infinity and 1 - 0 is left; near zero, where that form cancels, the series (the next term is
// 1e-9 of the sum)
__device__ __forceinline__ float tanh_f(float z) {
  const float e = expf(2.0f * z), q = z * z;
  const float far = 1.0f - 2.0f / (e + 1.0f);
  const float near = z * (1.0f - q * (1.0f / 3.0f - q * (2.0f / 15.0f)));
  return fabsf(z) < 0.05f ? near : far;
}
// 1 - a^2 for a = exp(log_a) <= 1 without cancellation: the series of 1 - exp(x), x = 2 log_a, above -1/4 (the
// next term is 5e-8 of the sum)
__device__ __forceinline__ float one_minus_square(float a, float log_a) {
  const float x = 2.0f * log_a, p = x * (1.f / 720.f) + 1.f / 120.f;
  const float series = -x * (1.f + x * (0.5f + x * (1.f / 6.f + x * (1.f / 24.f + x * p))));
  return x > -0.25f ? series : __builtin_fmaf(-a, a, 1.0f);
}
// x as the element type would keep it
template <typename T> __device__ __forceinline__ float round_to(float x) { return to_f32(from_f32<T>(x)); }

// N consecutive elements as floats; N elements of T are whole 16-byte pieces (N a multiple of
// Pack<T>::kN) and p is 16-byte aligned.
template <typename T, int N> __device__ __forceinline__ void load_vec(const T* p, float (&out)[N]) {
  constexpr int V = Pack<T>::kN;
  static_assert(N % V == 0, "whole 16-byte pieces");
  typedef typename Pack<T>::type vec_t;
#pragma unroll
  for (int i = 0; i < N / V; ++i) {
    const vec_t x = reinterpret_cast<const vec_t*>(p)[i];
#pragma unroll
    for (int j = 0; j < V; ++j) out[i * V + j] = to_f32(x[j]);
  }
}
template <typename T, int N> __device__ __forceinline__ void store_vec(T* p, const float (&in)[N]) {
  constexpr int V = Pack<T>::kN;
  static_assert(N % V == 0, "whole 16-byte pieces");
  typedef typename Pack<T>::type vec_t;
#pragma unroll
  for (int i = 0; i < N / V; ++i) {
    vec_t x;
#pragma unroll
    for (int j = 0; j < V; ++j) x[j] = from_f32<T>(in[i * V + j]);
    reinterpret_cast<vec_t*>(p)[i] = x;
  }
}

template <int CTRL> __device__ __forceinline__ float dpp_move_add(float v) {
  const int moved = __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xf, 0xf, false);
  return v + __builtin_bit_cast(float, moved);
}
// Sum over each aligned group of 8 lanes, in every lane of the group.
__device__ __forceinline__ float sum8(float v) {
  v = dpp_move_add<0xB1>(v);   // quad_perm [1,0,3,2]
  v = dpp_move_add<0x4E>(v);   // quad_perm [2,3,0,1]
  return dpp_move_add<0x141>(v);  // row_half_mirror
}
// Sum over each aligned group of 16 lanes, in every lane of the group.
__device__ __forceinline__ float sum16(float v) {
  v = sum8(v);
  return dpp_move_add<0x140>(v);  // row_mirror
}

inline bool aligned_to(const void* p, uintptr_t n) { return (reinterpret_cast<uintptr_t>(p) & (n - 1)) == 0; }

// Sum of w_j x_{t - taps + 1 + j} over the past inputs of one channel of a ring (taps slots, `stride` elements
// apart; w likewise): three at a time, those before position 0 fetched from slot 0 and left out.
template <typename T>
__device__ __forceinline__ float ring_dot(const T* ring, const T* w, long stride, int taps, int pos) {
  float acc = 0.f;
  for (int j0 = 0; j0 < taps - 1; j0 += 3) {
    T x[3], c[3];
    bool ok[3];
#pragma unroll
    for (int j = 0; j < 3; ++j) {
      const int p = pos - (taps - 1) + j0 + j;
      ok[j] = j0 + j < taps - 1 && p >= 0;
      x[j] = ring[(ok[j] ? p % taps : 0) * stride];
      c[j] = w[(ok[j] ? j0 + j : 0) * stride];
    }
#pragma unroll
    for (int j = 0; j < 3; ++j) acc = ok[j] ? __builtin_fmaf(to_f32(c[j]), to_f32(x[j]), acc) : acc;
  }
  return acc;
}

// What a residual sum may receive besides mult * x: x divided by its RMS (post_eps) and multiplied by post_w
// first, a vector for every row, and rows of a table (by index, or one per row).
struct StreamAddends {
  const void* post_w;
  const void* vec;
  const void* rows;
  const int64_t* rows_index;
  long rows_sr, rows_n;
  float post_eps;
};

// A barrier between wavefronts that only exchange data through LDS: a fence over global memory as well would wait
// for loads that are meant to stay on their way.
__device__ __forceinline__ void lds_barrier() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "workgroup", "local");
  __builtin_amdgcn_s_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "workgroup", "local");
}

// Position of the token a single-token launch brings for batch row b: from the device when there is
// an array of positions, otherwise the one the host passed.
__device__ __forceinline__ int row_pos(const int32_t* pos, int pos_host, int b) { return pos != nullptr ? pos[b] : pos_host; }

}  // namespace based
