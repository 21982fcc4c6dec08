// A model opened and ready to serve, whatever it was stored as: a published
// artifact directory or a model folder.  Picks the provider module whose
// capabilities cover the model's program, binds and prepares it, and runs
// batches of a session's tokens through the program.  The worker, the trace
// runner and the C interface all stand on this.
#pragma once

#include "artifact_provider.hpp"
#include "decoder_provider.hpp"
#include "program_session.hpp"

#include <cstdint>
#include <filesystem>
#include <memory>
#include <span>
#include <string>
#include <string_view>
#include <vector>

namespace qllm {

class ModelHost final {
 public:
  [[nodiscard]] static er::Status open(const std::filesystem::path& path,
                                       const ArtifactProviderOptions& options,
                                       std::unique_ptr<ModelHost>& host);
  ModelHost(const ModelHost&) = delete;
  ModelHost& operator=(const ModelHost&) = delete;

  [[nodiscard]] const er::ModelDescriptor& model() const noexcept { return model_; }
  [[nodiscard]] const er::ExecutionProviderModule& module() const noexcept {
    return module_;
  }
  [[nodiscard]] const PreparedProgram& prepared() const noexcept { return prepared_; }
  [[nodiscard]] DecoderProvider& provider() const noexcept { return *provider_; }
  // rows one program batch may hold
  [[nodiscard]] std::uint32_t batch_limit() const noexcept {
    return module_.service.prefill_chunk_tokens;
  }

  [[nodiscard]] er::Status begin(er::ProgramRequestContext request,
                                 std::unique_ptr<ProgramSession>& session) const;
  // One batch of the program over `tokens` at first_position, first_position +
  // 1, ...: the token the head selected for the last row, and - when `logits`
  // is given - the logits of the wanted rows appended to it.
  struct BatchResult final {
    er::Status status;
    std::uint32_t token{};
  };
  [[nodiscard]] BatchResult run(ProgramSession& session,
                                std::span<const std::uint32_t> tokens,
                                std::uint32_t first_position,
                                std::span<const std::uint32_t> wanted = {},
                                std::vector<float>* logits = nullptr) const;
  // Any number of tokens, cut into batches of at most batch_limit().
  [[nodiscard]] BatchResult run_all(ProgramSession& session,
                                    std::span<const std::uint32_t> tokens,
                                    std::uint32_t first_position,
                                    std::span<const std::uint32_t> wanted = {},
                                    std::vector<float>* logits = nullptr) const;

 private:
  ModelHost() = default;
  [[nodiscard]] er::Status find_ports();
  std::shared_ptr<er::ModelArtifact> artifact_;
  er::ModelDescriptor model_;
  er::ExecutionProviderModule module_;
  PreparedProgram prepared_;
  std::shared_ptr<DecoderProvider> provider_;
  std::string token_input_, position_input_, token_output_, logits_output_;
};

// Request parameters of a greedy request (moe_vm_runner.cpp:318-347).
[[nodiscard]] er::ProgramRequestContext greedy_request(std::uint64_t id);

}  // namespace qllm
