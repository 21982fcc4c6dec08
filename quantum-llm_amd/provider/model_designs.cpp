// The designs a model folder can name.  A design lists its layers as operations
// of the mixed-layer provider; mechanisms are capabilities with parameters, so
// another design combines the same ones.
#include "host_support.hpp"
#include "decoder_provider.hpp"
#include "mixed_provider.hpp"
#include "model_folder.hpp"

#include "qllm_kernels.h"

#include <algorithm>
#include <bit>
#include <cmath>
#include <limits>
#include <stdexcept>

namespace qllm {
namespace {

// What a folder without a declared maximum is served up to.
constexpr std::uint32_t kDefaultMaximumContext = 1U << 20U;

std::uint32_t u32(const json::Object& object, std::string_view key,
                  std::string_view where) {
  const auto value = json::required(object, key, where).u64(key);
  if (value > std::numeric_limits<std::uint32_t>::max())
    throw std::runtime_error(std::string(key) + " is out of range");
  return static_cast<std::uint32_t>(value);
}

std::uint32_t positive(const json::Object& object, std::string_view key,
                       std::string_view where) {
  const auto value = u32(object, key, where);
  if (!value) throw std::runtime_error(std::string(key) + " must be positive");
  return value;
}

std::uint64_t f32_bits(double value) {
  return std::bit_cast<std::uint32_t>(static_cast<float>(value));
}

std::uint64_t number_bits(const json::Object& object, std::string_view key,
                          std::string_view where) {
  return f32_bits(json::required(object, key, where).number(key));
}

const json::Object* optional_object(const json::Object& object, std::string_view key) {
  const auto found = object.find(key);
  return found == object.end() || found->second.null() ? nullptr
                                                       : &found->second.object(key);
}

bool flag(const json::Object& object, std::string_view key) {
  const auto found = object.find(key);
  return found != object.end() && !found->second.null() && found->second.boolean(key);
}

// Collects the program while a design walks its layers: operation order, value
// names, required kernels.
class ProgramBuilder final {
 public:
  explicit ProgramBuilder(er::ModelDescriptor& model) : model_(model) {
    model_.schema_version = 3U;
    model_.program_inputs.emplace(
        "token_ids", er::ProgramEndpointDescriptor{"tokens", std::string(kTokenAbi)});
    model_.program_inputs.emplace(
        "positions",
        er::ProgramEndpointDescriptor{"positions", std::string(kPositionAbi)});
  }

  void embedding(std::string capability, er::ParameterMap parameters,
                 er::BindingMap tensors) {
    using Value = er::OperationProgramDescriptor::ValueBinding;
    append(er::kModelLevelOperationLayer, std::move(capability), std::move(parameters),
           std::move(tensors), {{"token_ids", Value{"tokens", std::string(kTokenAbi)}}},
           {{"hidden", Value{"hidden.0", std::string(kHiddenAbi)}}});
  }

  void block(std::string capability, er::ParameterMap parameters,
             er::BindingMap tensors) {
    using Value = er::OperationProgramDescriptor::ValueBinding;
    const auto layer = static_cast<std::uint32_t>(model_.layer_program.size());
    er::LayerProgramDescriptor described;
    described.logical_layer = layer;
    described.block_capability = capability;
    model_.layer_program.push_back(std::move(described));
    append(layer, std::move(capability), std::move(parameters), std::move(tensors),
           {{"hidden", Value{hidden(layer), std::string(kHiddenAbi)}},
            {"positions", Value{"positions", std::string(kPositionAbi)}}},
           {{"hidden", Value{hidden(layer + 1U), std::string(kHiddenAbi)}}});
  }

  void head(std::string capability, er::ParameterMap parameters, er::BindingMap tensors) {
    using Value = er::OperationProgramDescriptor::ValueBinding;
    const auto layers = static_cast<std::uint32_t>(model_.layer_program.size());
    append(er::kModelLevelOperationLayer, std::move(capability), std::move(parameters),
           std::move(tensors), {{"hidden", Value{hidden(layers), std::string(kHiddenAbi)}}},
           {{"logits", Value{"logits", std::string(kLogitsAbi)}},
            {"token_ids", Value{"next", std::string(kTokenAbi)}}});
    model_.program_outputs.emplace(
        "token_ids", er::ProgramEndpointDescriptor{"next", std::string(kTokenAbi)});
    model_.program_outputs.emplace(
        "logits", er::ProgramEndpointDescriptor{"logits", std::string(kLogitsAbi)});
  }

 private:
  static std::string hidden(std::uint32_t layer) {
    return "hidden." + std::to_string(layer);
  }
  void append(
      std::uint32_t layer, std::string capability, er::ParameterMap parameters,
      er::BindingMap tensors,
      std::map<std::string, er::OperationProgramDescriptor::ValueBinding, std::less<>> in,
      std::map<std::string, er::OperationProgramDescriptor::ValueBinding, std::less<>>
          out) {
    const bool known = std::any_of(
        model_.required_kernels.begin(), model_.required_kernels.end(),
        [&](const er::KernelRequirement& kernel) { return kernel.capability == capability; });
    if (!known) model_.required_kernels.push_back({capability, 1U});
    model_.operation_program.emplace_back(
        static_cast<std::uint32_t>(model_.operation_program.size()), layer,
        std::move(capability), 1U, std::string{}, 0U, std::move(parameters),
        std::move(tensors), std::move(in), std::move(out));
  }

  er::ModelDescriptor& model_;
};

void bind(er::BindingMap& tensors, const std::string& prefix,
          std::initializer_list<std::pair<const char*, const char*>> roles) {
  for (const auto& [role, name] : roles) tensors.emplace(role, prefix + name);
}

std::uint64_t f64_bits(const json::Object& object, std::string_view key,
                       std::string_view where) {
  return std::bit_cast<std::uint64_t>(json::required(object, key, where).number(key));
}

// A rotation's dimensions, base and - when there is one - stretched frequencies.
void rotary(const json::Object& rot, er::ParameterMap& parameters) {
  parameters["rotary_dims"] = u32(rot, "dims", "mixer.rot");
  parameters["rotary_base_f64_bits"] = f64_bits(rot, "base", "mixer.rot");
  if (const auto* scaling = optional_object(rot, "scaling"))
    for (const auto& [name, key] : std::initializer_list<std::pair<const char*, const char*>>{
             {"rotary_factor_f64_bits", "factor"},
             {"rotary_original_f64_bits", "original"},
             {"rotary_fast_f64_bits", "fast"},
             {"rotary_slow_f64_bits", "slow"}})
      parameters[name] = f64_bits(*scaling, key, "mixer.rot.scaling");
}

// A dense gated feed-forward behind its norm.
void dense_feed_forward(const json::Object& mlp, std::uint32_t activation,
                        const std::string& prefix, er::ParameterMap& parameters,
                        er::BindingMap& tensors) {
  const auto& kind = json::required(mlp, "kind", "layer.mlp").string("mlp.kind");
  if (kind != "dense")
    throw std::runtime_error("feed-forward kind is not supported: " + kind);
  parameters["intermediate"] = positive(mlp, "ff", "layer.mlp");
  parameters["activation"] = activation;
  bind(tensors, prefix,
       {{"ffn_norm", "norm2"},
        {"gate_projection", "mlp.gate"},
        {"up_projection", "mlp.up"},
        {"down_projection", "mlp.down"}});
}

// ---- Zatupel -----------------------------------------------------------------
// Parallel layers with two norms: a mixer (windowed attention with mixed heads,
// generalised delta rule, or bonus recurrence over token-shifted inputs) and a
// gated feed-forward read the same residual row.

er::ModelDescriptor describe_zatupel(const json::Object& config,
                                     er::IModelTensorStore&) {
  er::ModelDescriptor model;
  model.architecture_id = "zatupel";
  model.vocab_size = positive(config, "vocab", "config");
  model.hidden_size = positive(config, "width", "config");
  model.max_context_tokens = kDefaultMaximumContext;
  const auto& norm = json::required(config, "norm", "config").object("config.norm");
  const auto epsilon = number_bits(norm, "eps", "config.norm");
  const auto& embedding =
      json::required(config, "embedding", "config").object("config.embedding");

  ProgramBuilder program(model);
  program.embedding(kEmbeddingBf16,
                    {{"scale_f32_bits", number_bits(embedding, "scale", "embedding")}},
                    {{"weight", "embed"}});
  bool values_kept = false;
  std::size_t index = 0U;
  for (const auto& entry : json::required(config, "layers", "config").array("layers")) {
    const auto& layer = entry.object("layer");
    const auto& mixer = json::required(layer, "mixer", "layer").object("layer.mixer");
    const auto& type = json::required(layer, "type", "layer").string("layer.type");
    const std::string prefix = "l" + std::to_string(index++) + ".";
    const std::string mix = prefix + "mix.";
    er::ParameterMap parameters{{"norm_epsilon_f32_bits", epsilon}};
    er::BindingMap tensors;
    bind(tensors, prefix, {{"mixer_norm", "norm1"}});

    if (const auto* mlp = optional_object(layer, "mlp")) {
      dense_feed_forward(*mlp, QLLM_ACTIVATION_GELU_TANH, prefix, parameters, tensors);
    }

    parameters["heads"] = positive(mixer, "heads", "layer.mixer");
    parameters["dim"] = positive(mixer, "dim", "layer.mixer");
    bind(tensors, mix, {{"output_projection", "o"}});
    if (type == "attention") {
      parameters["kv_heads"] = positive(mixer, "kv_heads", "layer.mixer");
      parameters["vdim"] = positive(mixer, "vdim", "layer.mixer");
      parameters["score_scale_f32_bits"] = number_bits(mixer, "scale", "layer.mixer");
      if (const auto* turned = optional_object(mixer, "rot")) {
        rotary(*turned, parameters);
      }
      if (const auto* mask = optional_object(mixer, "mask")) {
        parameters["window"] = positive(*mask, "size", "mixer.mask");
        parameters["sinks"] = u32(*mask, "keep_first", "mixer.mask");
      }
      bind(tensors, mix,
           {{"query_projection", "q"},
            {"key_projection", "k"},
            {"value_projection", "v"},
            {"head_gate", "g"},
            {"head_mix", "talk"}});
      if (flag(mixer, "v_mix")) {
        // the first such layer keeps its values, the others blend them in
        parameters["value_blend"] = values_kept ? kValuesBlended : kValuesKept;
        if (values_kept) bind(tensors, mix, {{"value_share", "vmix"}});
        values_kept = true;
      }
      program.block(kBlockWindowedAttention, std::move(parameters), std::move(tensors));
    } else if (type == "general_delta") {
      parameters["unit_epsilon_f32_bits"] = f32_bits(1.0e-6);
      parameters["decay_scale_f32_bits"] = f32_bits(-std::exp(-0.5));
      bind(tensors, mix,
           {{"read_projection", "r"},
            {"key_projection", "k"},
            {"value_projection", "v"},
            {"gate_projection_mixer", "g"},
            {"rate_projection", "a"},
            {"rate_bias", "a.b"},
            {"decay_down", "w1"},
            {"decay_up", "w2"},
            {"decay_base", "w0"},
            {"output_norm", "norm"}});
      program.block(kBlockDelta, std::move(parameters), std::move(tensors));
    } else if (type == "wkv") {
      bind(tensors, mix,
           {{"read_projection", "r"},
            {"key_projection", "k"},
            {"value_projection", "v"},
            {"gate_projection_mixer", "g"},
            {"read_shift", "mu.r"},
            {"key_shift", "mu.k"},
            {"value_shift", "mu.v"},
            {"gate_shift", "mu.g"},
            {"decay_shift", "mu.w"},
            {"decay_down", "w1"},
            {"decay_up", "w2"},
            {"decay_base", "w0"},
            {"bonus", "u"},
            {"output_norm", "norm"}});
      program.block(kBlockBonus, std::move(parameters), std::move(tensors));
    } else {
      throw std::runtime_error("mixer type is not supported: " + type);
    }
  }
  program.head(kHeadBf16, {{"norm_epsilon_f32_bits", epsilon}},
               {{"norm", "final.norm"}, {"weight", "head"}});
  return model;
}

// ---- Nametar -----------------------------------------------------------------
// Sandwich layers, a norm on either side of a sublayer: a mixer (latent attention
// without positions and with an output gate, windowed latent attention with a
// query latent and a rotated shared key part, or gated linear attention), then a
// gated feed-forward or none.

er::ModelDescriptor describe_nametar(const json::Object& config,
                                     er::IModelTensorStore&) {
  er::ModelDescriptor model;
  model.architecture_id = "nametar";
  model.vocab_size = positive(config, "vocab", "config");
  model.hidden_size = positive(config, "width", "config");
  model.max_context_tokens = kDefaultMaximumContext;
  const auto& norm = json::required(config, "norm", "config").object("config.norm");
  const auto epsilon = number_bits(norm, "eps", "config.norm");
  const auto residual_scale = number_bits(config, "residual_mult", "config");
  const auto& embedding =
      json::required(config, "embedding", "config").object("config.embedding");

  ProgramBuilder program(model);
  program.embedding(kEmbeddingBf16,
                    {{"scale_f32_bits", number_bits(embedding, "scale", "embedding")}},
                    {{"weight", "embed"}});
  std::size_t index = 0U;
  for (const auto& entry : json::required(config, "layers", "config").array("layers")) {
    const auto& layer = entry.object("layer");
    const auto& mixer = json::required(layer, "mixer", "layer").object("layer.mixer");
    const auto& type = json::required(layer, "type", "layer").string("layer.type");
    const std::string prefix = "l" + std::to_string(index++) + ".";
    const std::string mix = prefix + "mix.";
    er::ParameterMap parameters{{"norm_epsilon_f32_bits", epsilon},
                                {"residual_scale_f32_bits", residual_scale}};
    er::BindingMap tensors;
    bind(tensors, prefix, {{"mixer_norm", "norm1"}, {"mixer_post_norm", "norm1b"}});
    if (const auto* mlp = optional_object(layer, "mlp")) {
      dense_feed_forward(*mlp, QLLM_ACTIVATION_SILU, prefix, parameters, tensors);
      bind(tensors, prefix, {{"ffn_post_norm", "norm2b"}});
    }

    const auto dim = positive(mixer, "dim", "layer.mixer");
    parameters["heads"] = positive(mixer, "heads", "layer.mixer");
    parameters["dim"] = dim;
    parameters["vdim"] = positive(mixer, "vdim", "layer.mixer");
    bind(tensors, mix, {{"output_projection", "o"}});
    if (type == "latent_attention" || type == "latent_attention_2") {
      parameters["latent_rank"] = positive(mixer, "kv_rank", "layer.mixer");
      parameters["score_scale_f32_bits"] = number_bits(mixer, "scale", "layer.mixer");
      bind(tensors, mix,
           {{"latent_down", "dkv"},
            {"latent_norm", "dkv.norm"},
            {"key_up", "uk"},
            {"value_up", "uv"}});
      if (type == "latent_attention") {
        bind(tensors, mix, {{"query_projection", "q"}, {"output_gate", "g"}});
      } else {
        bind(tensors, mix,
             {{"query_down", "dq"}, {"query_latent_norm", "dq.norm"}, {"query_up", "uq"}});
        parameters["rotary_part"] = positive(mixer, "rot_dim", "layer.mixer");
        rotary(json::required(mixer, "rot", "layer.mixer").object("mixer.rot"), parameters);
        const auto& mask = json::required(mixer, "mask", "layer.mixer").object("mixer.mask");
        parameters["window"] = positive(mask, "size", "mixer.mask");
      }
      program.block(kBlockLatentAttention, std::move(parameters), std::move(tensors));
    } else if (type == "gla") {
      const double tau = json::required(mixer, "tau", "layer.mixer").number("mixer.tau");
      if (!(tau > 0.0)) throw std::runtime_error("tau must be positive");
      parameters["decay_scale_f32_bits"] = f32_bits(1.0 / tau);
      parameters["read_scale_f32_bits"] = f32_bits(1.0 / std::sqrt(double(dim)));
      bind(tensors, mix,
           {{"read_projection", "q"},
            {"key_projection", "k"},
            {"value_projection", "v"},
            {"gate_projection_mixer", "g"},
            {"decay_down", "a1"},
            {"decay_up", "a2"},
            {"decay_base", "a2.b"},
            {"output_norm", "norm"}});
      program.block(kBlockGatedLinear, std::move(parameters), std::move(tensors));
    } else {
      throw std::runtime_error("mixer type is not supported: " + type);
    }
  }
  program.head(kHeadBf16, {{"norm_epsilon_f32_bits", epsilon}},
               {{"norm", "final.norm"}, {"weight", "head"}});
  return model;
}

constexpr ModelDesign kDesigns[]{{"Zatupel", &describe_zatupel},
                                 {"Nametar", &describe_nametar}};

}  // namespace

std::span<const ModelDesign> model_designs() { return kDesigns; }

}  // namespace qllm
