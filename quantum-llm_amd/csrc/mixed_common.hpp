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

}  // namespace qllm
