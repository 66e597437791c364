// Helpers shared by the kernels of the streaming layers (norms with a scaled residual, causal
// convolutions on a ring of past inputs, grouped window attention, gated delta rule, gated linear
// recurrent unit).  Transcendentals are the library's full-precision fp32 functions: everything
// that enters a norm, a softmax or a recurrence is evaluated in 32 bits.
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

__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu_exact(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplus_f(float z) { return log1pf(expf(-fabsf(z))) + fmaxf(z, 0.0f); }
__device__ __forceinline__ float gelu_tanh_f(float z) {
  const float t = 0.7978845608028654f * (z + 0.044715f * z * z * z);
  return 0.5f * z * (1.0f + tanhf(t));
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

// Position of the token a single-token launch brings for batch row b: from the device when there is
// an array of positions, otherwise the one the host passed.
__device__ __forceinline__ int row_pos(const int32_t* pos, int pos_host, int b) { return pos != nullptr ? pos[b] : pos_host; }

}  // namespace based
