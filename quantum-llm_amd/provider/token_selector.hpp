// Token selection from rows of logits, shared by the providers' heads: presence
// penalty, arg-max at temperature zero, otherwise top-k on the device (or the
// whole row on the host) and the sampling rules of speculative_sampling.
#pragma once

#include "expert/runtime/program_executor.hpp"
#include "expert/runtime/speculative_sampling.hpp"

#include "host_support.hpp"

#include <cstddef>
#include <cstdint>
#include <span>
#include <vector>

namespace qllm {

class TokenSelector final {
 public:
  static constexpr std::uint32_t kMaximumTopK = 64U;  // provider.cpp:8359

  // `workspace`: device memory of at least workspace_bytes(), shared with the
  // caller's own arg-max launches on the same stream.
  TokenSelector(void* stream, std::uint32_t vocabulary, void* workspace,
                std::size_t workspace_bytes);
  ~TokenSelector();
  TokenSelector(const TokenSelector&) = delete;
  TokenSelector& operator=(const TokenSelector&) = delete;
  [[nodiscard]] static std::size_t workspace_bytes(std::uint32_t vocabulary,
                                                   std::uint32_t rows);

  // The head's token for a request (dense_fp4_provider.cpp:8433-8517) from one
  // row of logits whose arg-max lies in `argmax_tokens`; an output token is
  // marked as emitted in `presence`.
  [[nodiscard]] std::uint32_t select(float* logits, std::uint8_t* presence,
                                     std::uint32_t* argmax_tokens,
                                     const er::ProgramRequestContext& request,
                                     std::uint32_t sample_position);
  [[nodiscard]] er::SamplingDistribution distribution(
      float* row_logits, std::uint32_t vocabulary, std::uint32_t* device_argmax,
      const er::ProgramRequestContext& request, const std::uint8_t* presence);
  [[nodiscard]] std::vector<er::SamplingDistribution> top_k_distributions(
      const float* logits, std::uint32_t vocabulary, std::size_t stride,
      std::uint32_t rows, const er::ProgramRequestContext& request);
  // emitted[token] = 1 for every token (one upload, one launch)
  void mark(std::uint8_t* emitted, std::span<const std::uint32_t> tokens);

  [[nodiscard]] std::uint64_t gpu_calls() const noexcept { return gpu_calls_; }
  [[nodiscard]] std::uint64_t logit_transfer_bytes() const noexcept {
    return logit_transfer_bytes_;
  }

 private:
  struct Staging final {
    float top_logits[8 * kMaximumTopK];            // top-k readback: logits of all
    std::uint32_t top_tokens[8 * kMaximumTopK];    // rows, then their tokens
    std::uint32_t marks[8];                        // tokens whose byte is set
  };
  void* stream_{};
  std::uint32_t vocabulary_{};
  void* workspace_{};
  std::size_t workspace_bytes_{};
  DeviceBuffer device_;
  float* top_logits_{};
  std::uint32_t* top_tokens_{};
  std::uint32_t* mark_tokens_{};
  Staging* staging_{};
  std::uint64_t gpu_calls_{};
  std::uint64_t logit_transfer_bytes_{};
};

}  // namespace qllm
