#include "model_host.hpp"

#include "host_support.hpp"
#include "model_folder.hpp"

#include <algorithm>
#include <cstring>
#include <stdexcept>

namespace qllm {
namespace {

er::Status invalid(std::string message) {
  return {er::ErrorCode::invalid_argument, std::move(message)};
}

// What was opened: the described program and where its tensors are.
struct ModelSource final {
  std::shared_ptr<er::ModelArtifact> artifact;   // null for a model folder
  er::ModelDescriptor model;
  std::shared_ptr<er::IModelTensorStore> tensors;
};

// The callable modules of this build, in the order they are asked.
struct CallableModule final {
  er::WorkerProviderDefinition (*definition)();
  er::CreateExecutionProviderModuleResult (*create)(const ModelSource&,
                                                    const ArtifactProviderOptions&);
};

constexpr CallableModule kModules[]{
    {&make_mi355_dense_fp4_provider,
     [](const ModelSource& source, const ArtifactProviderOptions& options)
         -> er::CreateExecutionProviderModuleResult {
       if (!source.artifact)
         return {invalid("dense FP4 models are served from an artifact directory"), {}};
       return make_mi355_dense_fp4_module(source.artifact, options);
     }},
    {&make_mi355_mixed_provider,
     [](const ModelSource& source, const ArtifactProviderOptions& options)
         -> er::CreateExecutionProviderModuleResult {
       auto tensors = source.tensors;
       if (!tensors) {
         auto store = std::make_shared<er::MappedModelTensorStore>();
         if (auto status = er::MappedModelTensorStore::create(*source.artifact, *store);
             !status.ok())
           return {status, {}};
         tensors = std::move(store);
       }
       return make_mi355_mixed_module(source.model, std::move(tensors), options);
     }},
};

er::Status open_source(const std::filesystem::path& path,
                       const ArtifactProviderOptions& options, ModelSource& source) {
  if (is_model_folder(path)) {
    if (options.mtp_draft_depth)
      return invalid("artifact cannot apply the requested MTP depth");
    ModelFolder folder;
    if (auto status = open_model_folder(path, folder); !status.ok()) return status;
    source.model = std::move(folder.model);
    source.tensors = std::move(folder.tensors);
    return er::Status::success();
  }
  source.artifact = std::make_shared<er::ModelArtifact>();
  if (auto status = er::ModelArtifact::load(path, *source.artifact); !status.ok())
    return status;
  if (options.mtp_draft_depth)
    if (auto status = source.artifact->configure_mtp_draft_depth(options.mtp_draft_depth);
        !status.ok())
      return status;
  source.model = source.artifact->model();
  return er::Status::success();
}

er::ExecutionValue words(std::span<const std::uint32_t> values, std::string_view abi) {
  auto storage =
      std::make_shared<std::vector<std::uint32_t>>(values.begin(), values.end());
  const auto* bytes = reinterpret_cast<const std::byte*>(storage->data());
  return {std::string(abi), "host", storage, bytes,
          storage->size() * sizeof(std::uint32_t)};
}

}  // namespace

er::Status ModelHost::open(const std::filesystem::path& path,
                           const ArtifactProviderOptions& options,
                           std::unique_ptr<ModelHost>& host) {
  try {
    ModelSource source;
    if (auto status = open_source(path, options, source); !status.ok()) return status;
    if (source.model.schema_version < 3U)
      return invalid("callable VM service requires a schema v3 artifact");
    // exactly one module must cover the program (moe_vm_runner.cpp:431-497)
    const CallableModule* chosen = nullptr;
    for (const auto& candidate : kModules)
      if (er::provider_supports_model(source.model, candidate.definition().capabilities)
              .ok()) {
        if (chosen) return invalid("several callable providers implement the program");
        chosen = &candidate;
      }
    if (!chosen) return invalid("no callable provider implements the artifact program");
    auto created = chosen->create(source, options);
    if (!created.status.ok()) return created.status;
    std::unique_ptr<ModelHost> fresh(new ModelHost());
    fresh->artifact_ = std::move(source.artifact);
    fresh->model_ = std::move(source.model);
    fresh->module_ = std::move(created.module);
    fresh->provider_ =
        std::dynamic_pointer_cast<DecoderProvider>(fresh->module_.definition.implementation);
    if (!fresh->provider_)
      return invalid("callable provider module has no implementation");
    if (auto status = prepare_program(fresh->model_, fresh->module_, fresh->prepared_);
        !status.ok())
      return status;
    if (fresh->module_.finalize_service)
      if (auto status = fresh->module_.finalize_service(fresh->module_.service);
          !status.ok())
        return status;
    if (auto status = fresh->find_ports(); !status.ok()) return status;
    host = std::move(fresh);
    return er::Status::success();
  } catch (const std::exception& error) {
    return {er::ErrorCode::internal, error.what()};
  }
}

// The token-step service ABI (moe_vm_runner.cpp:297-316): exactly a token and a
// position input and one token output; a logits output is optional.
er::Status ModelHost::find_ports() {
  const auto claim = [](std::string& port, const std::string& role) {
    if (!port.empty()) return false;
    port = role;
    return true;
  };
  for (const auto& [role, endpoint] : model_.program_inputs) {
    if (endpoint.abi == kTokenAbi && !claim(token_input_, role))
      return invalid("multiple token program inputs");
    if (endpoint.abi == kPositionAbi && !claim(position_input_, role))
      return invalid("multiple position program inputs");
  }
  for (const auto& [role, endpoint] : model_.program_outputs) {
    if (endpoint.abi == kTokenAbi && !claim(token_output_, role))
      return invalid("multiple token program outputs");
    if (endpoint.abi == kLogitsAbi && !claim(logits_output_, role))
      return invalid("multiple logits program outputs");
  }
  if (model_.program_inputs.size() != 2U || token_input_.empty() ||
      position_input_.empty() || token_output_.empty())
    return invalid("artifact does not implement the token-step service ABI");
  return er::Status::success();
}

er::Status ModelHost::begin(er::ProgramRequestContext request,
                            std::unique_ptr<ProgramSession>& session) const {
  return ProgramSession::begin(model_, module_, prepared_, std::move(request), session);
}

ModelHost::BatchResult ModelHost::run(ProgramSession& session,
                                      std::span<const std::uint32_t> tokens,
                                      std::uint32_t first_position,
                                      std::span<const std::uint32_t> wanted,
                                      std::vector<float>* logits) const {
  if (logits) {
    if (logits_output_.empty()) return {invalid("model program publishes no logits"), 0U};
    if (auto status = provider_->set_logit_rows(
            session.state(), std::vector<std::uint32_t>(wanted.begin(), wanted.end()));
        !status.ok())
      return {status, 0U};
  }
  std::vector<std::uint32_t> positions(tokens.size());
  for (std::uint32_t row = 0U; row < positions.size(); ++row)
    positions[row] = first_position + row;
  std::map<std::string, er::ExecutionValue, std::less<>> inputs;
  inputs.emplace(token_input_, words(tokens, kTokenAbi));
  inputs.emplace(position_input_, words(positions, kPositionAbi));
  auto outputs = session.execute(std::move(inputs));
  if (!outputs.status.ok()) return {outputs.status, 0U};
  const auto found = outputs.values.find(token_output_);
  if (found == outputs.values.end())
    return {invalid("model program did not publish its token output"), 0U};
  const er::ExecutionValue& value = found->second;
  if (!value.valid() || value.abi != kTokenAbi || value.memory_domain != "host" ||
      value.bytes == 0U || value.bytes % sizeof(std::uint32_t) != 0U)
    return {invalid("callable VM returned an invalid token value"), 0U};
  BatchResult result{er::Status::success(), 0U};
  std::memcpy(&result.token, value.data + (value.bytes - sizeof(result.token)),
              sizeof(result.token));
  if (logits && !wanted.empty()) {
    const auto& rows = outputs.values.at(logits_output_);
    const std::size_t count = wanted.size() * model_.vocab_size;
    if (rows.memory_domain != "host" || rows.bytes < count * sizeof(float))
      return {invalid("callable VM returned an invalid logits value"), 0U};
    const auto* data = reinterpret_cast<const float*>(rows.data);
    logits->insert(logits->end(), data, data + count);
  }
  return result;
}

ModelHost::BatchResult ModelHost::run_all(ProgramSession& session,
                                          std::span<const std::uint32_t> tokens,
                                          std::uint32_t first_position,
                                          std::span<const std::uint32_t> wanted,
                                          std::vector<float>* logits) const {
  BatchResult result{invalid("batch is empty"), 0U};
  const std::size_t limit = std::max<std::uint32_t>(batch_limit(), 1U);
  for (std::size_t done = 0U; done < tokens.size(); done += limit) {
    const auto rows = tokens.subspan(done, std::min(limit, tokens.size() - done));
    std::vector<std::uint32_t> here;
    for (const auto row : wanted)
      if (row >= done && row < done + rows.size())
        here.push_back(row - static_cast<std::uint32_t>(done));
    result = run(session, rows, first_position + static_cast<std::uint32_t>(done), here,
                 logits);
    if (!result.status.ok()) return result;
  }
  return result;
}

er::ProgramRequestContext greedy_request(std::uint64_t id) {
  er::ProgramRequestContext request;
  request.request_id = id;
  request.parameters = {{"exact_decode_enabled", 0U},
                        {"sampling_first_output_position", 0U},
                        {"sampling_temperature_ppm", 0U},
                        {"sampling_top_p_ppm", 1'000'000U},
                        {"sampling_top_k", 0U},
                        {"sampling_min_p_ppm", 0U},
                        {"sampling_presence_penalty_biased_ppm", 2'000'000U},
                        {"sampling_seed", 0U}};
  return request;
}

}  // namespace qllm
