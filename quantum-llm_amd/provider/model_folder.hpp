// Model folders: config.json beside model.safetensors.  The configuration names
// an architecture; the table of known designs turns it into the same model
// descriptor a published artifact carries - operations with their parameters,
// tensor roles and values - so that everything after (capability check,
// registry, preparation, sessions) is shared.
#pragma once

#include "expert/runtime/model_descriptor.hpp"
#include "expert/runtime/program_executor.hpp"
#include "json_reader.hpp"

#include <filesystem>
#include <memory>
#include <span>
#include <string>
#include <string_view>

namespace qllm {

namespace er = expert::runtime;

// Read-only memory mapping of one safetensors file: an 8-byte little-endian
// header length, a JSON header (name -> dtype, shape, data_offsets), the data.
// A scalar is handed out with shape {1}.
class SafetensorsStore final : public er::IModelTensorStore {
 public:
  [[nodiscard]] static er::Status open(const std::filesystem::path& path,
                                       std::shared_ptr<SafetensorsStore>& store);
  [[nodiscard]] er::ResolveModelTensorResult resolve(std::string_view name) override;

 private:
  class Mapping;
  std::shared_ptr<const Mapping> mapping_;
  std::map<std::string, std::shared_ptr<const er::ImmutableModelTensor>, std::less<>>
      tensors_;
};

// One entry of the design table: the architecture string of config.json and the
// function that describes a model of it.
struct ModelDesign final {
  std::string_view architecture;
  er::ModelDescriptor (*describe)(const json::Object& config,
                                  er::IModelTensorStore& tensors);
};
[[nodiscard]] std::span<const ModelDesign> model_designs();

struct ModelFolder final {
  er::ModelDescriptor model;
  std::shared_ptr<er::IModelTensorStore> tensors;
};
[[nodiscard]] bool is_model_folder(const std::filesystem::path& root);
[[nodiscard]] er::Status open_model_folder(const std::filesystem::path& root,
                                           ModelFolder& folder);

}  // namespace qllm
