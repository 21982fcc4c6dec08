// Device helpers shared by the kernels of mixed-layer decoders.
#pragma once

#include "common.hpp"

#include <type_traits>

namespace qllm {

// The words a pass reads its place from (include/qllm_kernels.h).
constexpr int kStepPosition = 0;
constexpr int kStepSlot = 1;

__device__ __forceinline__ f32x4 mfma_bf16(i32x4 a, i32x4 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a),
                                                 __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
}

// Two bf16 values in a dword (v_cvt_pk_bf16_f32, nearest even).
__device__ __forceinline__ uint32_t pack_bf16(float low, float high) {
  const bf16x2 pair = {static_cast<__bf16>(low), static_cast<__bf16>(high)};
  return __builtin_bit_cast(uint32_t, pair);
}

// Element types: float, or bf16 as its bit pattern.
__device__ __forceinline__ float load_element(const float* p) { return *p; }
__device__ __forceinline__ float load_element(const uint16_t* p) {
  return bf16_bits_to_f32(*p);
}
__device__ __forceinline__ void store_element(float* p, float value) { *p = value; }
__device__ __forceinline__ void store_element(uint16_t* p, float value) {
  *p = static_cast<uint16_t>(f32_to_bf16_bits(value));
}

__device__ __forceinline__ float sigmoid_f32(float x) { return 1.0f / (1.0f + expf(-x)); }

__device__ __forceinline__ float activate(uint32_t activation, float z) {
  if (activation == QLLM_ACTIVATION_SILU) return z * sigmoid_f32(z);
  // 0.5 (1 + tanh(y)) = sigmoid(2 y)
  const float y = 0.7978845608028654f * (z + 0.044715f * z * z * z);
  return z * sigmoid_f32(2.0f * y);
}

// Sum over the 16 lanes of a row (every lane gets it).
__device__ __forceinline__ float row16_sum(float value) {
  const auto rotated = [](float v, auto control) {
    return __builtin_bit_cast(
        float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v),
                                           decltype(control)::value, 0xf, 0xf, true));
  };
  value += rotated(value, std::integral_constant<int, 0x121>{});   // row_ror:1
  value += rotated(value, std::integral_constant<int, 0x122>{});   // row_ror:2
  value += rotated(value, std::integral_constant<int, 0x124>{});   // row_ror:4
  value += rotated(value, std::integral_constant<int, 0x128>{});   // row_ror:8
  return value;
}

// Sixteen values per lane, sixteen lanes per row: lane i of a row returns the
// row's sum of value[i].  Halves of the values change hands with a partner
// lane in four steps (partners that differ in lane bit 3, 2, 1, 0; together
// they reach every lane of the row), so it costs 15 additions instead of 64.
__device__ __forceinline__ float row16_transposed_sum(float (&value)[16]) {
  const uint32_t lane = threadIdx.x % 16u;
  const auto exchange = [&](auto half, auto control) __attribute__((always_inline)) {
    constexpr int H = decltype(half)::value;
    const bool upper = (lane & H) != 0u;
#pragma unroll
    for (int i = 0; i < H; ++i) {
      const float mine = upper ? value[i + H] : value[i];
      const float theirs = upper ? value[i] : value[i + H];
      value[i] = mine + __builtin_bit_cast(
                            float, __builtin_amdgcn_update_dpp(
                                       0, __builtin_bit_cast(int, theirs),
                                       decltype(control)::value, 0xf, 0xf, true));
    }
  };
  exchange(std::integral_constant<int, 8>{}, std::integral_constant<int, 0x128>{});
  exchange(std::integral_constant<int, 4>{}, std::integral_constant<int, 0x141>{});
  exchange(std::integral_constant<int, 2>{}, std::integral_constant<int, 0x1b>{});
  exchange(std::integral_constant<int, 1>{}, std::integral_constant<int, 0xb1>{});
  return value[0];
}

}  // namespace qllm
