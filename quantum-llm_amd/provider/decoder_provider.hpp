// What the worker and the trace runner need from a provider beyond the common
// boundary (expert/runtime/program_executor.hpp): how prompts are fed, which
// rows' logits a batch is asked for, service facts and telemetry.
#pragma once

#include "expert/runtime/program_executor.hpp"

#include <cstdint>
#include <map>
#include <memory>
#include <span>
#include <string>
#include <vector>

namespace qllm {

namespace er = expert::runtime;

// Program output of a head that hands out logits: f32 [rows][vocabulary] in
// host memory, the rows asked for through set_logit_rows(), in that order.
inline constexpr std::string_view kLogitsAbi = "batch.logits.f32.host.v1";

class DecoderProvider : public er::IOperationProvider {
 public:
  // A prompt in one call, outside the program's batches.
  struct PrefillResult final {
    er::Status status;
    std::uint32_t predicted{};
  };
  [[nodiscard]] virtual bool supports_tall_prefill() const noexcept { return false; }
  [[nodiscard]] virtual PrefillResult prefill(
      const std::shared_ptr<er::IOperationProviderRequestState>&,
      std::span<const std::uint32_t>, std::uint32_t,
      const er::ProgramRequestContext&) {
    return {{er::ErrorCode::invalid_argument,
             "operation provider has no separate prompt path"},
            0U};
  }
  // Rows of the next batch whose logits the program's logits output shall hold
  // (ascending); without a call none are copied (the output is a
  // placeholder).
  [[nodiscard]] virtual er::Status set_logit_rows(
      const std::shared_ptr<er::IOperationProviderRequestState>&,
      std::vector<std::uint32_t>) {
    return {er::ErrorCode::invalid_argument,
            "operation provider does not hand out logits"};
  }
  [[nodiscard]] virtual bool profiles_gpu_phases() const noexcept { return false; }
  [[nodiscard]] virtual std::map<std::string, std::uint64_t, std::less<>> telemetry()
      const = 0;
  [[nodiscard]] virtual er::ExecutionProviderModule::ServiceContract
  service_contract() const = 0;
};

}  // namespace qllm
