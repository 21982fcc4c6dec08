// extern "C" surface of opened models (include/qllm_provider.h).
#include "qllm_provider.h"

#include "host_support.hpp"
#include "mixed_provider.hpp"
#include "model_host.hpp"

#include <algorithm>
#include <map>
#include <memory>
#include <stdexcept>
#include <string>
#include <vector>

namespace er = expert::runtime;

namespace qllm {
// defined with the provider's C surface: records the thread's last error
int32_t provider_fail(int32_t code, const std::string& message);
}  // namespace qllm

struct qllm_model {
  struct Request final {
    std::unique_ptr<qllm::ProgramSession> session;
    std::uint32_t position{};
  };
  std::unique_ptr<qllm::ModelHost> host;
  std::map<std::uint64_t, Request> requests;
  std::uint64_t next_id{1};
};

namespace {

int32_t from_status(const er::Status& status) {
  if (status.ok()) return QLLM_OK;
  return qllm::provider_fail(static_cast<int32_t>(status.code()),
                             std::string(status.message()));
}

template <typename Body>
int32_t guarded(Body&& body) {
  try {
    return body();
  } catch (const std::exception& error) {
    return qllm::provider_fail(QLLM_INTERNAL, error.what());
  }
}

qllm_model::Request& request_of(qllm_model* model, std::uint64_t id) {
  if (!model) throw std::runtime_error("model is null");
  const auto found = model->requests.find(id);
  if (found == model->requests.end()) throw std::runtime_error("unknown active request");
  return found->second;
}

}  // namespace

extern "C" qllm_model* qllm_model_open(const char* path, uint32_t max_context,
                                       uint32_t capacity, uint32_t kv_page_tokens,
                                       const char* kv_cache_dtype, uint32_t chunk_rows) {
  if (!path) {
    qllm::provider_fail(QLLM_INVALID_ARGUMENT, "model path is null");
    return nullptr;
  }
  qllm::ArtifactProviderOptions options;
  options.max_context = max_context;
  options.capacity = std::max(1U, capacity);
  if (kv_page_tokens) options.kv_page_tokens = kv_page_tokens;
  if (kv_cache_dtype) options.kv_cache_dtype = kv_cache_dtype;
  options.chunk_rows = chunk_rows;
  auto model = std::make_unique<qllm_model>();
  const auto status = qllm::ModelHost::open(path, options, model->host);
  if (from_status(status) != QLLM_OK) return nullptr;
  return model.release();
}

extern "C" void qllm_model_close(qllm_model* model) { delete model; }

extern "C" uint32_t qllm_model_vocabulary(const qllm_model* model) {
  return model ? model->host->model().vocab_size : 0U;
}

extern "C" uint32_t qllm_model_hidden(const qllm_model* model) {
  return model ? model->host->model().hidden_size : 0U;
}

extern "C" uint32_t qllm_model_batch_limit(const qllm_model* model) {
  return model ? model->host->batch_limit() : 0U;
}

extern "C" int32_t qllm_model_begin(qllm_model* model, uint32_t temperature_ppm,
                                    uint32_t top_p_ppm, uint32_t top_k, uint32_t min_p_ppm,
                                    int32_t presence_ppm, uint64_t seed,
                                    uint32_t first_output_position, uint64_t* request) {
  return guarded([&] {
    if (!model || !request)
      return qllm::provider_fail(QLLM_INVALID_ARGUMENT, "invalid model request");
    auto context = qllm::greedy_request(model->next_id);
    context.parameters["sampling_temperature_ppm"] = temperature_ppm;
    context.parameters["sampling_top_p_ppm"] = top_p_ppm;
    context.parameters["sampling_top_k"] = top_k;
    context.parameters["sampling_min_p_ppm"] = min_p_ppm;
    context.parameters["sampling_presence_penalty_biased_ppm"] =
        static_cast<std::uint64_t>(std::int64_t{presence_ppm} + 2'000'000);
    context.parameters["sampling_seed"] = seed;
    context.parameters["sampling_first_output_position"] = first_output_position;
    qllm_model::Request fresh;
    const auto status = model->host->begin(std::move(context), fresh.session);
    if (!status.ok()) return from_status(status);
    *request = model->next_id++;
    model->requests.emplace(*request, std::move(fresh));
    return int32_t{QLLM_OK};
  });
}

extern "C" int32_t qllm_model_end(qllm_model* model, uint64_t request) {
  return guarded([&] {
    request_of(model, request);
    model->requests.erase(request);
    return int32_t{QLLM_OK};
  });
}

extern "C" int32_t qllm_model_step(qllm_model* model, uint64_t request,
                                   const uint32_t* tokens, uint32_t count,
                                   const uint32_t* wanted, uint32_t wanted_count,
                                   float* logits, uint32_t* next_token) {
  return guarded([&] {
    auto& entry = request_of(model, request);
    if (!tokens || !count || (wanted_count && (!wanted || !logits)))
      return qllm::provider_fail(QLLM_INVALID_ARGUMENT, "invalid model step");
    std::vector<float> rows;
    const auto result = model->host->run_all(
        *entry.session, {tokens, count}, entry.position, {wanted, wanted_count},
        wanted_count ? &rows : nullptr);
    if (!result.status.ok()) return from_status(result.status);
    entry.position += count;
    if (wanted_count) std::copy(rows.begin(), rows.end(), logits);
    if (next_token) *next_token = result.token;
    return int32_t{QLLM_OK};
  });
}

extern "C" int32_t qllm_model_trace_layers(qllm_model* model, uint64_t request,
                                           const uint32_t* tokens, uint32_t count,
                                           float* hidden, uint32_t* next_token) {
  return guarded([&] {
    auto& entry = request_of(model, request);
    auto* provider =
        dynamic_cast<qllm::Mi355MixedProvider*>(&model->host->provider());
    if (!provider || !tokens || !count || !hidden || count > model->host->batch_limit())
      return qllm::provider_fail(QLLM_INVALID_ARGUMENT, "invalid layer trace");
    // the program one operation at a time, as ProgramSession walks it
    const auto& prepared = model->host->prepared();
    const auto& program = prepared.bound.program;
    std::vector<std::uint32_t> positions(count);
    for (std::uint32_t row = 0; row < count; ++row) positions[row] = entry.position + row;
    std::vector<er::ExecutionValue> values(program.values.size());
    const auto host_words = [](const std::uint32_t* data, std::size_t words,
                               std::string_view abi) {
      auto storage = std::make_shared<std::vector<std::uint32_t>>(data, data + words);
      const auto* bytes = reinterpret_cast<const std::byte*>(storage->data());
      return er::ExecutionValue{std::string(abi), "host", storage, bytes, words * 4U};
    };
    for (const auto& endpoint : program.inputs) {
      const auto& abi = program.values.at(endpoint.value_index).abi;
      values[endpoint.value_index] = abi == qllm::kTokenAbi
                                         ? host_words(tokens, count, abi)
                                         : host_words(positions.data(), count, abi);
    }
    std::size_t layer = 0;
    for (std::size_t index = 0; index < program.operations.size(); ++index) {
      const auto& compiled = program.operations[index];
      std::vector<er::ExecutionValue> operands;
      for (const auto& binding : compiled.input_values)
        operands.push_back(values.at(binding.value_index));
      auto handle = provider->execute(
          *prepared.operations[index], entry.session->state(),
          er::OperationInvocation{entry.session->request(), compiled, operands});
      auto result = handle.poll();
      if (!result) throw std::runtime_error("operation did not complete");
      if (!result->status.ok()) return from_status(result->status);
      for (std::size_t port = 0; port < compiled.output_values.size(); ++port)
        values[compiled.output_values[port].value_index] = result->outputs.at(port);
      if (compiled.logical_layer != er::kModelLevelOperationLayer) {
        const auto status = provider->copy_hidden(
            count, hidden + layer++ * count * model->host->model().hidden_size);
        if (!status.ok()) return from_status(status);
      }
    }
    entry.position += count;
    for (const auto& endpoint : program.outputs)
      if (next_token && program.values.at(endpoint.value_index).abi == qllm::kTokenAbi)
        *next_token =
            *reinterpret_cast<const std::uint32_t*>(values[endpoint.value_index].data);
    return int32_t{QLLM_OK};
  });
}

extern "C" uint64_t qllm_model_telemetry(const qllm_model* model, const char* name) {
  if (!model || !name) return 0U;
  const auto figures = model->host->provider().telemetry();
  const auto found = figures.find(name);
  return found == figures.end() ? 0U : found->second;
}
