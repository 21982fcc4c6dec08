#include "mixed_provider.hpp"

#include <hip/hip_runtime.h>

#include <algorithm>
#include <bit>
#include <cmath>
#include <cstdlib>
#include <cstring>
#include <stdexcept>

namespace qllm {
namespace {

constexpr std::uint32_t kSmallBatch = 64U;   // rows that stream the weights once
constexpr std::uint32_t kStepWords = 4U;     // ahead of the tokens

std::uint32_t round_up(std::uint32_t value, std::uint32_t to) {
  return (value + to - 1U) / to * to;
}

// Key and value rows are stored in one of three widths the kernels are built
// for; wider heads keep their own (the general kernel takes any).
std::uint32_t cache_stride(std::uint32_t dim) {
  for (const std::uint32_t stride : {64U, 128U, 256U})
    if (dim <= stride) return stride;
  return round_up(dim, 32U);
}

std::uint64_t parameter(const er::ParameterMap& parameters, std::string_view name) {
  const auto found = parameters.find(name);
  if (found == parameters.end())
    throw std::runtime_error("operation parameter is absent: " + std::string(name));
  return found->second;
}

std::uint32_t parameter_or(const er::ParameterMap& parameters, std::string_view name,
                           std::uint32_t otherwise) {
  const auto found = parameters.find(name);
  return found == parameters.end() ? otherwise
                                   : static_cast<std::uint32_t>(found->second);
}

float parameter_f32(const er::ParameterMap& parameters, std::string_view name) {
  const float value =
      std::bit_cast<float>(static_cast<std::uint32_t>(parameter(parameters, name)));
  if (!std::isfinite(value))
    throw std::runtime_error("operation parameter is not finite: " + std::string(name));
  return value;
}

double parameter_f64(const er::ParameterMap& parameters, std::string_view name) {
  const double value = std::bit_cast<double>(parameter(parameters, name));
  if (!(value > 0.0) || !std::isfinite(value))
    throw std::runtime_error("operation parameter is not positive: " + std::string(name));
  return value;
}

// Angles per position of `dims` rotated dimensions, and the factor on their cosine
// and sine.  With a scaling, slow dimensions are stretched by `factor` and fast ones
// stay, with a ramp between those that turn `slow` and `fast` times over the
// original length (YaRN).
struct Rotation final {
  std::vector<double> frequencies;
  double magnitude{1.0};
};

Rotation rotation_of(const er::ParameterMap& parameters, std::uint32_t dims) {
  Rotation out;
  const double base = parameter_f64(parameters, "rotary_base_f64_bits");
  for (std::uint32_t i = 0; i < dims / 2U; ++i)
    out.frequencies.push_back(std::pow(base, -2.0 * i / dims));
  if (!parameters.contains("rotary_factor_f64_bits")) return out;
  const double factor = parameter_f64(parameters, "rotary_factor_f64_bits");
  const double original = parameter_f64(parameters, "rotary_original_f64_bits");
  constexpr double kPi = 3.14159265358979323846;
  const auto turning = [&](double turns) {
    return dims * std::log(original / (2.0 * kPi * turns)) / (2.0 * std::log(base));
  };
  const double low = std::max(
      std::floor(turning(parameter_f64(parameters, "rotary_fast_f64_bits"))), 0.0);
  const double high = std::min(
      std::ceil(turning(parameter_f64(parameters, "rotary_slow_f64_bits"))), dims - 1.0);
  for (std::size_t i = 0; i < out.frequencies.size(); ++i) {
    const double ramp = std::clamp(
        (static_cast<double>(i) - low) / std::max(high - low, 0.001), 0.0, 1.0);
    out.frequencies[i] *= ramp / factor + (1.0 - ramp);
  }
  out.magnitude = 0.1 * std::log(factor) + 1.0;
  return out;
}

std::uint64_t elements_of(const er::ImmutableModelTensor& tensor) {
  std::uint64_t count = 1U;
  for (const auto size : tensor.shape) count *= size;
  return count;
}

void require_matrix(const er::ImmutableModelTensor& tensor, std::uint64_t rows,
                    std::uint64_t columns) {
  if (tensor.encoding != "BF16" || tensor.shape.size() != 2U || tensor.shape[0] != rows ||
      tensor.shape[1] != columns || tensor.data_bytes != rows * columns * 2U ||
      !tensor.value.valid())
    throw std::runtime_error("weight matrix has the wrong type or shape: " + tensor.name);
}

// Enough workgroups for the chip where the rows alone are too few, each with a few
// KiB per wave left to stream.
std::uint32_t k_splits(std::uint32_t rows, std::uint32_t columns) {
  const std::uint32_t tiles = rows / 16U;
  return std::clamp(std::min((768U + tiles - 1U) / tiles, columns / 32U / 16U), 1U, 8U);
}

}  // namespace

// One layer: its norms and matrices, and what its mixer needs.
struct Mi355MixedProvider::Block final {
  Kind kind{};
  float epsilon{};
  DeviceBuffer mixer_norm, ffn_norm;
  // all projections of the mixer that share an input are one matrix; token
  // shift gives every projection its own
  struct Projection final {
    Matrix matrix;
    std::uint32_t input{};     // which mixer input it reads
    std::uint32_t column{};    // first column in the projection rows
  };
  std::vector<Projection> projections;
  std::uint32_t projection_columns{};
  Matrix gate_up;              // interleaved tiles
  std::uint32_t intermediate{};
  std::uint32_t activation{};
  Matrix output;               // mixer columns, then feed-forward columns
  std::uint32_t mixer_columns{};   // padded
  std::uint32_t splits{1};

  // sandwich: the output projection ends with the mixer's columns
  bool sandwich{};
  DeviceBuffer mixer_post_norm, ffn_post_norm;
  float residual_scale{1.0F};
  Matrix down;
  std::uint32_t down_splits{1};

  // attention
  qllm_windowed_attention attention{};
  std::uint32_t rotary_dims{};
  std::uint32_t query_column{}, key_column{}, value_column{}, gate_column{};
  std::uint64_t value_blend{};
  DeviceBuffer frequencies, value_share, head_mix;

  // latent attention
  qllm_latent_attention latent{};
  std::uint32_t latent_column{};
  std::uint32_t query_rank{};      // 0 = queries straight from the input
  Matrix query_up;
  DeviceBuffer latent_norm, query_norm, key_up, key_up_transposed, value_up;

  // recurrence
  qllm_recurrence recurrence{};
  std::uint32_t r_column{}, rate_column{}, low_column{};
  DeviceBuffer decay_up, decay_base, rate_bias, bonus, output_norm;
  std::uint64_t state_offset{}, carry_offset{};   // floats into the slot's state
  std::vector<DeviceBuffer> shifts;
};

struct Mi355MixedProvider::PreparedOperation final : er::IPreparedOperation {
  Kind kind{};
  std::uint32_t block{};
  std::map<std::string, std::size_t, std::less<>> input_indices;
  std::vector<std::pair<std::string, std::string>> outputs;
};

er::Status validate_mixed_descriptor(const er::ModelDescriptor& model) {
  if (model.schema_version < 3U || !model.routed_components.empty() ||
      model.operation_program.empty() || model.exact_decode_program.has_value())
    return {er::ErrorCode::invalid_argument,
            "mixed-layer provider runs schema-v3 programs without routed experts or an "
            "exact-decode service"};
  return er::Status::success();
}

er::WorkerProviderDefinition make_mi355_mixed_provider() {
  const auto validator = [](const er::ModelDescriptor& model) {
    return validate_mixed_descriptor(model);
  };
  return {"mi355-mixed-bf16",
          150U,
          {{kEmbeddingBf16, 1U, 1U, validator},
           {kBlockWindowedAttention, 1U, 1U, validator},
           {kBlockDelta, 1U, 1U, validator},
           {kBlockBonus, 1U, 1U, validator},
           {kBlockLatentAttention, 1U, 1U, validator},
           {kBlockGatedLinear, 1U, 1U, validator},
           {kHeadBf16, 1U, 1U, validator}},
          nullptr};
}

Mi355MixedProvider::Mi355MixedProvider(const MixedGeometry& geometry) : g_(geometry) {
  if (!g_.hidden || !g_.vocabulary || !g_.max_context || !g_.capacity ||
      !g_.kv_page_tokens || g_.kv_page_tokens % 32U || g_.element > QLLM_ELEMENT_F32)
    throw std::invalid_argument("mixed-layer geometry is not supported");
  if (!g_.chunk_rows) g_.chunk_rows = std::min(4096U, g_.max_context);
  g_.chunk_rows = std::min(g_.chunk_rows, g_.max_context);
  if (const char* eager = std::getenv("QLLM_PROVIDER_EAGER")) use_graphs_ = eager[0] == '0';
  hipStream_t stream{};
  hip_check(hipStreamCreate(&stream), "create provider stream");
  stream_ = stream;
  lifetime_ = std::make_shared<std::uint8_t>(std::uint8_t{0});
}

Mi355MixedProvider::~Mi355MixedProvider() { release(); }

void Mi355MixedProvider::release() {
  if (stream_) (void)hipStreamSynchronize(static_cast<hipStream_t>(stream_));
  if (step_graph_) (void)hipGraphExecDestroy(static_cast<hipGraphExec_t>(step_graph_));
  step_graph_ = nullptr;
  selector_.reset();
  if (staging_) (void)hipHostFree(staging_);
  staging_ = nullptr;
  if (stream_) (void)hipStreamDestroy(static_cast<hipStream_t>(stream_));
  stream_ = nullptr;
}

// ---- loading -------------------------------------------------------------------

DeviceBuffer Mi355MixedProvider::upload_raw(const er::ImmutableModelTensor& tensor) {
  DeviceBuffer buffer(tensor.data_bytes, "allocate weights");
  hip_check(hipMemcpy(buffer.get(), tensor.value.data + tensor.data_offset,
                      tensor.data_bytes, hipMemcpyHostToDevice),
            "upload weights");
  weight_bytes_ += tensor.data_bytes;
  return buffer;
}

DeviceBuffer Mi355MixedProvider::upload_f32(const er::ImmutableModelTensor& tensor,
                                            std::uint64_t elements) {
  if (elements_of(tensor) != elements || !tensor.value.valid())
    throw std::runtime_error("weight vector has the wrong shape: " + tensor.name);
  std::vector<float> values(elements);
  const std::byte* data = tensor.value.data + tensor.data_offset;
  if (tensor.encoding == "F32") {
    std::memcpy(values.data(), data, elements * 4U);
  } else if (tensor.encoding == "BF16") {
    for (std::uint64_t i = 0; i < elements; ++i) {
      std::uint16_t bits{};
      std::memcpy(&bits, data + i * 2U, 2U);
      values[i] = std::bit_cast<float>(std::uint32_t{bits} << 16U);
    }
  } else {
    throw std::runtime_error("weight vector has an unsupported type: " + tensor.name);
  }
  DeviceBuffer buffer(elements * 4U, "allocate weight vector");
  hip_check(hipMemcpy(buffer.get(), values.data(), elements * 4U, hipMemcpyHostToDevice),
            "upload weight vector");
  weight_bytes_ += elements * 4U;
  return buffer;
}

Mi355MixedProvider::Matrix Mi355MixedProvider::pack(std::uint32_t rows,
                                                    std::uint32_t columns,
                                                    std::span<const Part> parts) {
  const std::size_t bytes = qllm_linear_packed_bytes(rows, columns);
  Matrix matrix{DeviceBuffer(bytes, "allocate packed weights"), round_up(rows, 16U),
                round_up(columns, 64U)};
  hip_check(hipMemset(matrix.data.get(), 0, bytes), "clear packed weights");
  hip_check(hipDeviceSynchronize(), "clear packed weights");
  for (const auto& part : parts) {
    const auto& tensor = *part.tensor;
    DeviceBuffer source(tensor.data_bytes, "allocate row-major weights");
    hip_check(hipMemcpy(source.get(), tensor.value.data + tensor.data_offset,
                        tensor.data_bytes, hipMemcpyHostToDevice),
              "upload weights");
    status_check(qllm_linear_pack(source.get(), tensor.shape[0], tensor.shape[1],
                                  matrix.data.get(), matrix.columns, part.first_tile,
                                  part.tile_stride, part.first_column, stream_));
    hip_check(hipStreamSynchronize(static_cast<hipStream_t>(stream_)), "pack weights");
  }
  weight_bytes_ += bytes;
  return matrix;
}

DeviceBuffer Mi355MixedProvider::pack_heads(const er::ImmutableModelTensor& tensor,
                                            std::uint32_t heads, std::uint32_t size,
                                            std::uint32_t padded, bool transposed) {
  const std::uint32_t width = tensor.shape.at(1);
  const std::uint32_t rows = transposed ? width : size;
  const std::uint32_t columns = transposed ? size : width;
  const std::size_t bytes = qllm_linear_packed_bytes(heads * padded, columns);
  DeviceBuffer packed(bytes, "allocate packed weights");
  DeviceBuffer source(tensor.data_bytes, "allocate row-major weights");
  hip_check(hipMemset(packed.get(), 0, bytes), "clear packed weights");
  hip_check(hipMemcpy(source.get(), tensor.value.data + tensor.data_offset,
                      tensor.data_bytes, hipMemcpyHostToDevice),
            "upload weights");
  hip_check(hipDeviceSynchronize(), "clear packed weights");
  for (std::uint32_t head = 0; head < heads; ++head)
    status_check(qllm_linear_pack_strided(
        source.as<std::uint16_t>() + std::size_t{head} * size * width, rows, columns,
        transposed ? 1U : width, transposed ? width : 1U, packed.get(),
        round_up(columns, 64U), head * (padded / 16U), 1U, 0U, stream_));
  hip_check(hipStreamSynchronize(static_cast<hipStream_t>(stream_)), "pack weights");
  weight_bytes_ += bytes;
  return packed;
}

void Mi355MixedProvider::prepare_block(Block& block,
                                       const er::OperationPreparationContext& context) {
  const auto& parameters = context.operation.parameters;
  const auto tensor = [&](std::string_view role) -> const er::ImmutableModelTensor& {
    return tensor_for(context.tensors, role);
  };
  block.epsilon = parameter_f32(parameters, "norm_epsilon_f32_bits");
  block.mixer_norm = upload_f32(tensor("mixer_norm"), g_.hidden);
  block.intermediate = parameter_or(parameters, "intermediate", 0U);
  block.sandwich = block.kind == Kind::latent || block.kind == Kind::gated;
  std::uint32_t mixer_width{};
  if (block.kind == Kind::attention) {
    prepare_attention(block, context);
    mixer_width = block.attention.query_heads * block.attention.vdim;
  } else if (block.kind == Kind::latent) {
    prepare_latent(block, context);
    mixer_width = block.latent.heads * block.latent.vdim;
  } else {
    prepare_recurrence(block, context);
    mixer_width = block.recurrence.heads * block.recurrence.vdim;
  }

  const auto& output = tensor("output_projection");
  require_matrix(output, g_.hidden, mixer_width);
  block.mixer_columns = round_up(mixer_width, 64U);
  std::vector<Part> joined{{&output, 0U, 1U, 0U}};
  std::uint32_t columns = block.mixer_columns;
  if (block.sandwich) {
    block.mixer_post_norm = upload_f32(tensor("mixer_post_norm"), g_.hidden);
    block.residual_scale = parameter_f32(parameters, "residual_scale_f32_bits");
  }
  if (block.intermediate) {
    block.activation = static_cast<std::uint32_t>(parameter(parameters, "activation"));
    block.ffn_norm = upload_f32(tensor("ffn_norm"), g_.hidden);
    const auto& gate = tensor("gate_projection");
    const auto& up = tensor("up_projection");
    const auto& down = tensor("down_projection");
    require_matrix(gate, block.intermediate, g_.hidden);
    require_matrix(up, block.intermediate, g_.hidden);
    require_matrix(down, g_.hidden, block.intermediate);
    const Part halves[]{{&gate, 0U, 2U, 0U}, {&up, 1U, 2U, 0U}};
    block.gate_up = pack(round_up(block.intermediate, 16U) * 2U, g_.hidden, halves);
    if (block.sandwich) {
      const Part alone[]{{&down, 0U, 1U, 0U}};
      block.ffn_post_norm = upload_f32(tensor("ffn_post_norm"), g_.hidden);
      block.down = pack(g_.hidden, block.intermediate, alone);
      block.down_splits = k_splits(block.down.rows, block.down.columns);
    } else {
      joined.push_back({&down, 0U, 1U, block.mixer_columns});
      columns += round_up(block.intermediate, 64U);
    }
  }
  block.output = pack(g_.hidden, columns, joined);
  block.splits = k_splits(block.output.rows, block.output.columns);
}

DeviceBuffer Mi355MixedProvider::upload_frequencies(const er::ParameterMap& parameters,
                                                    std::uint32_t dims) {
  const auto frequencies = rotation_of(parameters, dims).frequencies;
  DeviceBuffer table(frequencies.size() * 8U, "allocate rotary table");
  hip_check(hipMemcpy(table.get(), frequencies.data(), frequencies.size() * 8U,
                      hipMemcpyHostToDevice),
            "upload rotary table");
  return table;
}

void Mi355MixedProvider::prepare_attention(Block& block,
                                           const er::OperationPreparationContext& context) {
  const auto& parameters = context.operation.parameters;
  auto& a = block.attention;
  a.query_heads = static_cast<std::uint32_t>(parameter(parameters, "heads"));
  a.kv_heads = static_cast<std::uint32_t>(parameter(parameters, "kv_heads"));
  a.dim = static_cast<std::uint32_t>(parameter(parameters, "dim"));
  a.vdim = static_cast<std::uint32_t>(parameter(parameters, "vdim"));
  if (!a.kv_heads || a.query_heads % a.kv_heads)
    throw std::runtime_error("query heads are not a multiple of key/value heads");
  a.key_stride = cache_stride(a.dim);
  a.value_stride = cache_stride(a.vdim);
  a.window = parameter_or(parameters, "window", 0U);
  a.sinks = parameter_or(parameters, "sinks", 0U);
  a.scale = parameter_f32(parameters, "score_scale_f32_bits");
  a.page_tokens = g_.kv_page_tokens;
  a.element = g_.element;
  block.rotary_dims = parameter_or(parameters, "rotary_dims", 0U);
  if (block.rotary_dims % 2U || block.rotary_dims > a.dim)
    throw std::runtime_error("rotary dimensions do not fit the head");
  if (block.rotary_dims)
    block.frequencies = upload_frequencies(parameters, block.rotary_dims);
  if (const auto* mix = optional_tensor(context.tensors, "head_mix")) {
    block.head_mix = upload_f32(*mix, std::uint64_t{a.query_heads} * a.query_heads);
    a.head_mix = block.head_mix.as<float>();
  }
  block.value_blend = parameter_or(parameters, "value_blend", 0U);
  if (block.value_blend == kValuesBlended) {
    block.value_share = upload_f32(tensor_for(context.tensors, "value_share"), 1U);
    for (const auto& earlier : blocks_)
      if (earlier->value_blend == kValuesKept &&
          earlier->attention.kv_heads * earlier->attention.vdim != a.kv_heads * a.vdim)
        throw std::runtime_error("blended values differ in width between layers");
  }

  std::vector<Part> parts;
  std::uint32_t rows = 0U;
  const auto place = [&](const char* role, std::uint32_t count) {
    const auto& tensor = tensor_for(context.tensors, role);
    require_matrix(tensor, count, g_.hidden);
    const std::uint32_t column = rows;
    parts.push_back({&tensor, rows / 16U, 1U, 0U});
    rows += round_up(count, 16U);
    return column;
  };
  block.query_column = place("query_projection", a.query_heads * a.dim);
  block.key_column = place("key_projection", a.kv_heads * a.dim);
  block.value_column = place("value_projection", a.kv_heads * a.vdim);
  if (optional_tensor(context.tensors, "head_gate"))
    block.gate_column = place("head_gate", a.query_heads);
  block.projections.push_back({pack(rows, g_.hidden, parts), 0U, 0U});
  block.projection_columns = rows;
}

void Mi355MixedProvider::prepare_latent(Block& block,
                                        const er::OperationPreparationContext& context) {
  const auto& parameters = context.operation.parameters;
  auto& a = block.latent;
  a.heads = static_cast<std::uint32_t>(parameter(parameters, "heads"));
  a.dim = static_cast<std::uint32_t>(parameter(parameters, "dim"));
  a.vdim = static_cast<std::uint32_t>(parameter(parameters, "vdim"));
  a.rank = static_cast<std::uint32_t>(parameter(parameters, "latent_rank"));
  a.rot_dim = parameter_or(parameters, "rotary_part", 0U);
  a.rotary_dims = parameter_or(parameters, "rotary_dims", 0U);
  if (a.rotary_dims % 2U || a.rotary_dims > a.rot_dim)
    throw std::runtime_error("rotary dimensions do not fit the shared key part");
  a.window = parameter_or(parameters, "window", 0U);
  a.scale = parameter_f32(parameters, "score_scale_f32_bits");
  a.epsilon = block.epsilon;
  a.rotary_magnitude = 1.0F;
  if (a.rotary_dims) {
    block.frequencies = upload_frequencies(parameters, a.rotary_dims);
    a.frequencies = block.frequencies.as<double>();
    a.rotary_magnitude = static_cast<float>(rotation_of(parameters, a.rotary_dims).magnitude);
  }
  a.page_tokens = g_.kv_page_tokens;
  a.element = g_.element;
  block.latent_norm = upload_f32(tensor_for(context.tensors, "latent_norm"), a.rank);
  a.latent_norm = block.latent_norm.as<float>();
  const auto& key_up = tensor_for(context.tensors, "key_up");
  const auto& value_up = tensor_for(context.tensors, "value_up");
  require_matrix(key_up, std::uint64_t{a.heads} * a.dim, a.rank);
  require_matrix(value_up, std::uint64_t{a.heads} * a.vdim, a.rank);
  block.key_up = pack_heads(key_up, a.heads, a.dim, round_up(a.dim, 32U), false);
  block.key_up_transposed = pack_heads(key_up, a.heads, a.dim, round_up(a.rank, 32U), true);
  block.value_up = pack_heads(value_up, a.heads, a.vdim, round_up(a.vdim, 16U), false);
  a.key_up = block.key_up.get();
  a.key_up_transposed = block.key_up_transposed.get();
  a.value_up = block.value_up.get();

  std::vector<Part> parts;
  std::uint32_t rows = 0U;
  const auto place = [&](const char* role, std::uint32_t count) {
    const auto& tensor = tensor_for(context.tensors, role);
    require_matrix(tensor, count, g_.hidden);
    const std::uint32_t column = rows;
    parts.push_back({&tensor, rows / 16U, 1U, 0U});
    rows += round_up(count, 16U);
    return column;
  };
  const std::uint32_t query_width = a.heads * (a.dim + a.rot_dim);
  if (const auto* down = optional_tensor(context.tensors, "query_down")) {
    block.query_rank = down->shape.at(0);
    block.query_column = place("query_down", block.query_rank);
    block.query_norm =
        upload_f32(tensor_for(context.tensors, "query_latent_norm"), block.query_rank);
    const auto& up = tensor_for(context.tensors, "query_up");
    require_matrix(up, query_width, block.query_rank);
    const Part alone[]{{&up, 0U, 1U, 0U}};
    block.query_up = pack(query_width, block.query_rank, alone);
  } else {
    block.query_column = place("query_projection", query_width);
  }
  block.latent_column = place("latent_down", a.rank + a.rot_dim);
  if (optional_tensor(context.tensors, "output_gate"))
    block.gate_column = place("output_gate", a.heads * a.vdim);
  block.projections.push_back({pack(rows, g_.hidden, parts), 0U, 0U});
  block.projection_columns = rows;
}

void Mi355MixedProvider::prepare_recurrence(
    Block& block, const er::OperationPreparationContext& context) {
  const auto& parameters = context.operation.parameters;
  auto& r = block.recurrence;
  const bool delta = block.kind == Kind::delta;
  const bool gated = block.kind == Kind::gated;
  r.kind = delta   ? QLLM_RECURRENCE_DELTA
           : gated ? QLLM_RECURRENCE_GATED
                   : QLLM_RECURRENCE_BONUS;
  r.gate_kind = delta ? QLLM_GATE_SIGMOID : QLLM_GATE_SILU;
  r.heads = static_cast<std::uint32_t>(parameter(parameters, "heads"));
  r.dim = static_cast<std::uint32_t>(parameter(parameters, "dim"));
  r.vdim = parameter_or(parameters, "vdim", r.dim);
  r.element = g_.element;
  r.epsilon = block.epsilon;
  const std::uint32_t channels = r.heads * r.dim;
  const std::uint32_t values = r.heads * r.vdim;
  if (delta) {
    r.unit_epsilon = parameter_f32(parameters, "unit_epsilon_f32_bits");
    r.decay_scale = parameter_f32(parameters, "decay_scale_f32_bits");
    block.rate_bias = upload_f32(tensor_for(context.tensors, "rate_bias"), channels);
    r.rate_bias = block.rate_bias.as<float>();
  } else if (gated) {
    r.decay_scale = parameter_f32(parameters, "decay_scale_f32_bits");
    r.read_scale = parameter_f32(parameters, "read_scale_f32_bits");
  } else {
    block.bonus = upload_f32(tensor_for(context.tensors, "bonus"), channels);
    r.bonus = block.bonus.as<float>();
  }
  const auto& down = tensor_for(context.tensors, "decay_down");
  const auto& up = tensor_for(context.tensors, "decay_up");
  if (down.shape.size() != 2U)
    throw std::runtime_error("weight matrix has the wrong shape: " + down.name);
  r.rank = down.shape[0];
  require_matrix(down, r.rank, g_.hidden);
  require_matrix(up, channels, r.rank);
  block.decay_up = upload_raw(up);
  block.decay_base = upload_f32(tensor_for(context.tensors, "decay_base"), channels);
  block.output_norm =
      upload_f32(tensor_for(context.tensors, "output_norm"), gated ? r.vdim : channels);
  r.decay_up_bf16 = block.decay_up.get();
  r.decay_base = block.decay_base.as<float>();
  r.norm_weight = block.output_norm.as<float>();

  struct Wanted final {
    const char* role;
    const char* shift;
    std::uint32_t rows;
    std::uint32_t* column;
  };
  std::vector<Wanted> wanted{
      {"read_projection", "read_shift", channels, &block.r_column},
      {"key_projection", "key_shift", channels, &block.key_column},
      {"value_projection", "value_shift", values, &block.value_column},
      {"gate_projection_mixer", "gate_shift", values, &block.gate_column},
      {"decay_down", "decay_shift", r.rank, &block.low_column}};
  if (delta)
    wanted.push_back({"rate_projection", nullptr, channels, &block.rate_column});
  const bool shifted = block.kind == Kind::bonus;
  std::vector<Part> parts;
  std::uint32_t rows = 0U;
  for (const auto& item : wanted) {
    const auto& tensor = tensor_for(context.tensors, item.role);
    require_matrix(tensor, item.rows, g_.hidden);
    *item.column = rows;
    if (shifted) {
      const Part alone[]{{&tensor, 0U, 1U, 0U}};
      block.projections.push_back(
          {pack(item.rows, g_.hidden, alone),
           static_cast<std::uint32_t>(block.shifts.size()), rows});
      block.shifts.push_back(upload_f32(tensor_for(context.tensors, item.shift), g_.hidden));
    } else {
      parts.push_back({&tensor, rows / 16U, 1U, 0U});
    }
    rows += round_up(item.rows, 16U);
  }
  if (!shifted) block.projections.push_back({pack(rows, g_.hidden, parts), 0U, 0U});
  block.projection_columns = rows;
}

er::PrepareOperationResult Mi355MixedProvider::prepare(
    const er::OperationPreparationContext& context) {
  try {
    std::lock_guard lock(mutex_);
    if (finalized_) throw std::runtime_error("provider has already served a request");
    const std::string& capability = context.operation.capability;
    auto prepared = std::make_shared<PreparedOperation>();
    for (std::size_t index = 0; index < context.compiled.input_values.size(); ++index)
      prepared->input_indices.emplace(context.compiled.input_values[index].port, index);
    for (const auto& binding : context.compiled.output_values) {
      const auto output = context.operation.output_bindings.find(binding.port);
      if (output == context.operation.output_bindings.end())
        throw std::runtime_error("compiled output port is absent");
      prepared->outputs.emplace_back(binding.port, output->second.abi);
    }
    if (capability == kEmbeddingBf16) {
      prepared->kind = Kind::embedding;
      const auto& table = tensor_for(context.tensors, "weight");
      require_matrix(table, g_.vocabulary, g_.hidden);
      embedding_ = upload_raw(table);
      embedding_scale_ = parameter_f32(context.operation.parameters, "scale_f32_bits");
    } else if (capability == kHeadBf16) {
      prepared->kind = Kind::head;
      const auto& weight = tensor_for(context.tensors, "weight");
      require_matrix(weight, g_.vocabulary, g_.hidden);
      const Part alone[]{{&weight, 0U, 1U, 0U}};
      head_ = pack(g_.vocabulary, g_.hidden, alone);
      final_norm_ = upload_f32(tensor_for(context.tensors, "norm"), g_.hidden);
      final_epsilon_ =
          parameter_f32(context.operation.parameters, "norm_epsilon_f32_bits");
    } else {
      auto block = std::make_unique<Block>();
      if (capability == kBlockWindowedAttention)
        block->kind = Kind::attention;
      else if (capability == kBlockDelta)
        block->kind = Kind::delta;
      else if (capability == kBlockBonus)
        block->kind = Kind::bonus;
      else if (capability == kBlockLatentAttention)
        block->kind = Kind::latent;
      else if (capability == kBlockGatedLinear)
        block->kind = Kind::gated;
      else
        return {{er::ErrorCode::invalid_argument,
                 "capability is not provided: " + capability},
                {}};
      prepare_block(*block, context);
      prepared->kind = block->kind;
      prepared->block = static_cast<std::uint32_t>(blocks_.size());
      blocks_.push_back(std::move(block));
    }
    return {er::Status::success(), std::move(prepared)};
  } catch (const std::exception& error) {
    return {{er::ErrorCode::internal, error.what()}, {}};
  }
}

er::Status Mi355MixedProvider::finalize() {
  try {
    std::lock_guard lock(mutex_);
    finalize_locked();
    return er::Status::success();
  } catch (const std::exception& error) {
    return {er::ErrorCode::internal, error.what()};
  }
}

void Mi355MixedProvider::finalize_locked() {
  if (finalized_) return;
  if (!embedding_.get() || !head_.data.get() || blocks_.empty())
    throw std::runtime_error("program is not fully prepared");
  mixer_stride_ = round_up(g_.hidden, 64U);
  pages_expire_ = true;
  for (auto& item : blocks_) {
    Block& block = *item;
    projection_stride_ = std::max(projection_stride_, block.projection_columns);
    joined_stride_ = std::max({joined_stride_, block.output.columns, block.down.columns});
    shift_inputs_ = std::max(shift_inputs_, static_cast<std::uint32_t>(block.shifts.size()));
    if (block.kind == Kind::attention) {
      auto& a = block.attention;
      a.layer_offset = page_bytes_;
      page_bytes_ += qllm_windowed_layer_bytes(g_.kv_page_tokens, a.kv_heads, a.key_stride,
                                               a.value_stride, g_.element);
      if (!a.window) pages_expire_ = false;
      widest_window_ = std::max(widest_window_, a.window);
      most_sinks_ = std::max(most_sinks_, a.sinks);
    } else if (block.kind == Kind::latent) {
      auto& a = block.latent;
      a.layer_offset = page_bytes_;
      page_bytes_ +=
          qllm_latent_layer_bytes(g_.kv_page_tokens, a.rank, a.rot_dim, g_.element);
      if (!a.window) pages_expire_ = false;
      widest_window_ = std::max(widest_window_, a.window);
    } else {
      block.state_offset = state_floats_;
      state_floats_ += std::uint64_t{block.recurrence.heads} * block.recurrence.dim *
                       block.recurrence.vdim;
      state_floats_ = (state_floats_ + 3U) / 4U * 4U;
      if (!block.shifts.empty()) {
        block.carry_offset = state_floats_;
        state_floats_ += round_up(g_.hidden, 4U);
      }
    }
  }
  page_bytes_ = std::max<std::uint64_t>(page_bytes_, 16U);
  const std::size_t pages = (g_.max_context + g_.kv_page_tokens - 1U) / g_.kv_page_tokens;
  slots_ = RequestSlots(g_.capacity, pages, page_bytes_);
  page_table_ = DeviceBuffer(g_.capacity * pages * sizeof(void*), "allocate page table");
  hip_check(hipMemset(page_table_.get(), 0, g_.capacity * pages * sizeof(void*)),
            "clear page table");
  states_ = DeviceBuffer(std::max<std::uint64_t>(state_floats_, 4U) * 4U * g_.capacity,
                         "allocate recurrent states");
  presence_ = DeviceBuffer(std::size_t{g_.capacity} * g_.vocabulary,
                           "allocate presence bytes");
  select_workspace_bytes_ = TokenSelector::workspace_bytes(g_.vocabulary, 1U);
  select_workspace_ = DeviceBuffer(select_workspace_bytes_, "allocate token selection");
  argmax_ = DeviceBuffer(4U, "allocate arg-max");
  selector_ = std::make_unique<TokenSelector>(stream_, g_.vocabulary,
                                              select_workspace_.get(),
                                              select_workspace_bytes_);
  const std::uint32_t element_bytes = g_.element == QLLM_ELEMENT_F32 ? 4U : 2U;
  head_input_ = DeviceBuffer(std::size_t{kLogitRows} * mixer_stride_ * element_bytes,
                             "allocate head input");
  gather_ = DeviceBuffer(kLogitRows * 4U, "allocate head rows");
  logits_ = DeviceBuffer(std::size_t{kLogitRows} * round_up(g_.vocabulary, 4U) * 4U,
                         "allocate logits");
  staging_words_ = kStepWords + g_.chunk_rows;
  hip_check(hipHostMalloc(&staging_, (staging_words_ + kLogitRows) * 4U,
                          hipHostMallocDefault),
            "allocate pinned staging");
  step_ = DeviceBuffer(staging_words_ * 4U, "allocate step words");
  for (auto& item : blocks_) {
    Block& block = *item;
    auto* step = step_.as<std::uint32_t>();
    if (block.kind == Kind::attention) {
      block.attention.page_table = page_table_.as<void*>();
      block.attention.pages_per_slot = static_cast<std::uint32_t>(pages);
      block.attention.step = step;
    } else if (block.kind == Kind::latent) {
      block.latent.page_table = page_table_.as<void*>();
      block.latent.pages_per_slot = static_cast<std::uint32_t>(pages);
      block.latent.step = step;
    } else {
      block.recurrence.state = states_.as<float>() + block.state_offset;
      block.recurrence.slot_stride = state_floats_;
      block.recurrence.step = step;
    }
  }
  finalized_ = true;
}

std::size_t Mi355MixedProvider::scratch_bytes_for(std::uint32_t rows,
                                                  std::uint32_t last_position) const {
  std::size_t bytes = 16U;
  for (const auto& item : blocks_) {
    const Block& block = *item;
    if (block.kind == Kind::attention)
      bytes = std::max(bytes, qllm_windowed_attention_workspace_bytes(&block.attention, rows,
                                                                      last_position));
    else if (block.kind == Kind::latent)
      bytes = std::max(bytes, qllm_latent_attention_workspace_bytes(&block.latent, rows,
                                                                    last_position));
    else
      bytes = std::max(bytes, qllm_recurrence_workspace_bytes(&block.recurrence, rows));
  }
  return bytes;
}

// Buffers for batches of up to `rows` rows that end at or before last_position; they
// only grow.  A few rows find room wherever they stand.
void Mi355MixedProvider::ensure_workspace(std::uint32_t rows, std::uint32_t last_position) {
  if (rows <= workspace_rows_ && scratch_bytes_for(rows, last_position) <= scratch_bytes_)
    return;
  std::uint32_t size = 64U;
  while (size < rows) size *= 2U;
  size = std::min(std::max({size, rows, workspace_rows_}), std::max(g_.chunk_rows, 64U));
  if (step_graph_) {   // it addresses the buffers that are about to go
    (void)hipGraphExecDestroy(static_cast<hipGraphExec_t>(step_graph_));
    step_graph_ = nullptr;
  }
  hip_check(hipStreamSynchronize(static_cast<hipStream_t>(stream_)), "grow workspace");
  const std::size_t element = g_.element == QLLM_ELEMENT_F32 ? 4U : 2U;
  const auto zeroed = [](std::size_t bytes, const char* what) {
    DeviceBuffer buffer(std::max<std::size_t>(bytes, 16U), what);
    hip_check(hipMemset(buffer.get(), 0, std::max<std::size_t>(bytes, 16U)), what);
    return buffer;
  };
  const std::uint32_t last = g_.max_context - 1U;
  // room for the context to double
  const std::uint32_t ahead = static_cast<std::uint32_t>(
      std::min<std::uint64_t>(last, std::uint64_t{2U} * std::max(last_position, size)));
  std::size_t scratch = std::max(scratch_bytes_, scratch_bytes_for(size, ahead));
  for (std::uint32_t few = 1U; few <= std::min(size, kSmallBatch); ++few)
    scratch = std::max(scratch, scratch_bytes_for(few, last));
  std::size_t query = 0U;
  std::size_t kept = 0U;
  std::size_t query_rank = 0U;
  std::size_t query_width = 0U;
  std::size_t partial_rows = 0U;
  for (const auto& item : blocks_) {
    const Block& block = *item;
    partial_rows = std::max<std::size_t>(
        partial_rows, std::max(block.splits, block.down_splits) * kSmallBatch);
    if (block.sandwich) partial_rows = std::max<std::size_t>(partial_rows, size);
    if (block.kind == Kind::attention) {
      const auto& a = block.attention;
      query = std::max(query, std::size_t{a.query_heads} * a.key_stride);
      kept = std::max(kept, std::size_t{a.kv_heads} * a.vdim);
      scratch = std::max(scratch, qllm_windowed_attention_workspace_bytes(&a, size, last));
    } else if (block.kind == Kind::latent && block.query_rank) {
      query_rank = std::max<std::size_t>(query_rank, block.query_up.columns);
      query_width = std::max<std::size_t>(query_width, block.query_up.rows);
    }
  }
  workspace_rows_ = 0U;
  for (auto& hidden : hidden_)
    hidden = zeroed(std::size_t{size} * g_.hidden * 4U, "allocate residual stream");
  inputs_ = zeroed((std::max(shift_inputs_, 1U) + 1U) * std::size_t{size} * mixer_stride_ *
                       element,
                   "allocate layer inputs");
  projections_ = zeroed(std::size_t{size} * projection_stride_ * 4U,
                        "allocate projections");
  joined_ = zeroed(std::size_t{size} * joined_stride_ * element, "allocate layer outputs");
  query_ = zeroed(std::size_t{size} * query * element, "allocate queries");
  query_latents_ = zeroed(std::size_t{size} * query_rank * element, "allocate query latents");
  queries_ = zeroed(std::size_t{size} * query_width * 4U, "allocate latent queries");
  kept_values_ = zeroed(std::size_t{size} * kept * 4U, "allocate kept values");
  shift_last_ = zeroed(std::size_t{round_up(g_.hidden, 4U)} * 4U, "allocate shifted row");
  partials_ = zeroed(partial_rows * round_up(g_.hidden, 4U) * 4U,
                     "allocate partial sums");
  scratch_ = zeroed(scratch, "allocate mixer scratch");
  scratch_bytes_ = scratch;
  hip_check(hipDeviceSynchronize(), "clear workspace");
  workspace_rows_ = size;
}

// ---- requests ------------------------------------------------------------------

er::CreateOperationRequestStateResult Mi355MixedProvider::create_request_state(
    const er::ProgramRequestContext& request) {
  try {
    std::lock_guard lock(mutex_);
    finalize_locked();
    require_sampling_profile(request, g_.max_context);
    const auto grant = slots_.take();
    if (!grant)
      return {{er::ErrorCode::backpressure,
               "mixed-layer provider has no free request slot"},
              {}};
    auto state = std::make_shared<MixedRequestState>();
    state->slot = grant->slot;
    state->lease = grant->lease;
    const auto stream = static_cast<hipStream_t>(stream_);
    if (state_floats_)
      hip_check(hipMemsetAsync(states_.as<float>() + state->slot * state_floats_, 0,
                               state_floats_ * 4U, stream),
                "clear recurrent state");
    hip_check(hipMemsetAsync(presence_.as<std::uint8_t>() +
                                 std::size_t{state->slot} * g_.vocabulary,
                             0, g_.vocabulary, stream),
              "clear presence bytes");
    return {er::Status::success(), std::move(state)};
  } catch (const std::exception& error) {
    return {{er::ErrorCode::internal, error.what()}, {}};
  }
}

er::Status Mi355MixedProvider::rebind_request_state(
    const std::shared_ptr<er::IOperationProviderRequestState>& opaque,
    const er::ProgramRequestContext& request) {
  try {
    std::lock_guard lock(mutex_);
    const auto state = std::dynamic_pointer_cast<MixedRequestState>(opaque);
    if (!state) throw std::runtime_error("request state is not this provider's");
    require_sampling_profile(request, g_.max_context);
    hip_check(hipMemsetAsync(presence_.as<std::uint8_t>() +
                                 std::size_t{state->slot} * g_.vocabulary,
                             0, g_.vocabulary, static_cast<hipStream_t>(stream_)),
              "reset presence bytes");
    return er::Status::success();
  } catch (const std::exception& error) {
    return {er::ErrorCode::internal, error.what()};
  }
}

er::Status Mi355MixedProvider::set_logit_rows(
    const std::shared_ptr<er::IOperationProviderRequestState>& opaque,
    std::vector<std::uint32_t> rows) {
  std::lock_guard lock(mutex_);
  const auto state = std::dynamic_pointer_cast<MixedRequestState>(opaque);
  if (!state || !std::is_sorted(rows.begin(), rows.end()))
    return {er::ErrorCode::invalid_argument, "logit rows are invalid"};
  state->logit_rows = std::move(rows);
  return er::Status::success();
}

// Pages no later token can see: past the kept first tokens and behind the
// widest window.
void Mi355MixedProvider::release_pages(const MixedRequestState& state) {
  if (!pages_expire_ || state.position <= widest_window_) return;
  const std::uint64_t oldest = std::uint64_t{state.position} + 1U - widest_window_;
  const std::uint64_t tokens = g_.kv_page_tokens;
  slots_.recycle(state.slot, [&](std::size_t page) {
    return page * tokens >= most_sinks_ && (page + 1U) * tokens <= oldest;
  });
}

// ---- execution -----------------------------------------------------------------

// Uploads a batch's words and makes its pages exist.  The pinned words are
// free: every batch ends with a wait.
void Mi355MixedProvider::begin_batch(MixedRequestState& state,
                                     std::span<const std::uint32_t> tokens,
                                     std::uint32_t first_position) {
  const auto rows = static_cast<std::uint32_t>(tokens.size());
  if (!rows || rows > g_.chunk_rows)
    throw std::runtime_error("program batch holds too many or no tokens");
  if (first_position != state.position)
    throw std::runtime_error("batch does not continue its request");
  if (rows > g_.max_context - first_position)
    throw std::runtime_error("KV position exceeds the configured context");
  for (const auto token : tokens)
    if (token >= g_.vocabulary)
      throw std::runtime_error("embedding token exceeds vocabulary");
  for (const auto row : state.logit_rows)
    if (row >= rows) throw std::runtime_error("logit row exceeds the batch");
  ensure_workspace(rows, first_position + rows - 1U);
  const auto stream = static_cast<hipStream_t>(stream_);
  void** table =
      page_table_.as<void*>() + std::size_t{state.slot} * slots_.pages_per_slot();
  slots_.ensure(state.slot, first_position / g_.kv_page_tokens,
                (first_position + rows - 1U) / g_.kv_page_tokens,
                [&](std::size_t page, void* pointer) {
                  // a pageable source: the copy has read it when the call returns
                  hip_check(hipMemcpyAsync(table + page, &pointer, sizeof(pointer),
                                           hipMemcpyHostToDevice, stream),
                            "publish KV page");
                });
  auto* words = static_cast<std::uint32_t*>(staging_);
  words[0] = first_position;
  words[1] = state.slot;
  words[2] = rows;
  words[3] = 0U;
  std::copy(tokens.begin(), tokens.end(), words + kStepWords);
  hip_check(hipMemcpyAsync(step_.get(), words, (kStepWords + rows) * 4U,
                           hipMemcpyHostToDevice, stream),
            "upload batch words");
  batch_rows_ = rows;
}

void Mi355MixedProvider::enqueue_embedding(std::uint32_t rows) {
  stream_index_ = 0U;
  pending_partials_ = 0U;
  pending_branch_ = {};
  status_check(qllm_embedding_bf16_batch(
      embedding_.get(), g_.vocabulary, step_.as<std::uint32_t>() + kStepWords,
      hidden_[0].as<float>(), rows, g_.hidden, embedding_scale_, stream_));
}

void Mi355MixedProvider::enqueue_attention(Block& block, std::uint32_t rows,
                                           std::uint32_t last_position) {
  qllm_rope_store_launch store{};
  store.projections = projections_.as<float>();
  store.stride = projection_stride_;
  store.query_column = block.query_column;
  store.key_column = block.key_column;
  store.value_column = block.value_column;
  store.rotary_dims = block.rotary_dims;
  store.frequencies = block.frequencies.as<double>();
  if (block.value_blend == kValuesBlended) {
    store.first_values = kept_values_.as<float>();
    store.value_share = block.value_share.as<float>();
  } else if (block.value_blend == kValuesKept) {
    store.values_out = kept_values_.as<float>();
  }
  store.query_out = query_.get();
  store.rows = rows;
  status_check(qllm_windowed_rope_store(&block.attention, &store, stream_));

  qllm_attention_launch launch{};
  launch.query = query_.get();
  launch.gate =
      block.gate_column ? projections_.as<float>() + block.gate_column : nullptr;
  launch.gate_stride = projection_stride_;
  launch.output = joined_.get();
  launch.output_stride = block.output.columns;
  launch.rows = rows;
  launch.maximum_position = last_position;
  launch.workspace = scratch_.get();
  launch.workspace_bytes = scratch_bytes_;
  status_check(qllm_windowed_attention_rows(&block.attention, &launch, stream_));
}

void Mi355MixedProvider::enqueue_recurrence(Block& block, std::uint32_t rows) {
  qllm_recurrence_launch launch{};
  launch.projections = projections_.as<float>();
  launch.stride = projection_stride_;
  launch.r_column = block.r_column;
  launch.k_column = block.key_column;
  launch.v_column = block.value_column;
  launch.gate_column = block.gate_column;
  launch.rate_column = block.rate_column;
  launch.low_column = block.low_column;
  launch.output = joined_.get();
  launch.output_stride = block.output.columns;
  launch.rows = rows;
  if (!block.shifts.empty()) {
    launch.carry_from = shift_last_.as<float>();
    launch.carry_to = states_.as<float>() + block.carry_offset;
    launch.carry_width = g_.hidden;
  }
  launch.workspace = scratch_.get();
  launch.workspace_bytes = scratch_bytes_;
  status_check(qllm_recurrence_rows(&block.recurrence, &launch, stream_));
}

void Mi355MixedProvider::enqueue_latent(Block& block, std::uint32_t rows,
                                        std::uint32_t last_position) {
  auto& a = block.latent;
  qllm_latent_store_launch store{};
  store.projections = projections_.as<float>();
  store.stride = projection_stride_;
  store.latent_column = block.latent_column;
  store.rows = rows;
  if (block.query_rank) {
    store.query_column = block.query_column;
    store.query_rank = block.query_rank;
    store.query_norm = block.query_norm.as<float>();
    store.query_out = query_latents_.get();
    store.query_stride = block.query_up.columns;
  }
  status_check(qllm_latent_store(&a, &store, stream_));

  qllm_latent_launch launch{};
  launch.query = projections_.as<float>() + block.query_column;
  launch.query_stride = projection_stride_;
  if (block.query_rank) {
    qllm_linear_segment s{};
    s.weights = block.query_up.data.get();
    s.input = query_latents_.get();
    s.output = queries_.get();
    s.rows = block.query_up.rows;
    s.columns = block.query_up.columns;
    s.input_stride = block.query_up.columns;
    s.output_stride = block.query_up.rows;
    s.output_columns = a.heads * (a.dim + a.rot_dim);
    s.epilogue = QLLM_LINEAR_STORE;
    status_check(qllm_linear_batch(&s, 1U, rows, g_.element, stream_));
    launch.query = queries_.as<float>();
    launch.query_stride = block.query_up.rows;
  }
  launch.gate =
      block.gate_column ? projections_.as<float>() + block.gate_column : nullptr;
  launch.gate_stride = projection_stride_;
  launch.output = joined_.get();
  launch.output_stride = block.output.columns;
  launch.rows = rows;
  launch.maximum_position = last_position;
  launch.workspace = scratch_.get();
  launch.workspace_bytes = scratch_bytes_;
  status_check(qllm_latent_attention_rows(&a, &launch, stream_));
}

void Mi355MixedProvider::enqueue_mixer(Block& block, std::uint32_t rows,
                                       std::uint32_t last_position) {
  if (block.kind == Kind::attention)
    enqueue_attention(block, rows, last_position);
  else if (block.kind == Kind::latent)
    enqueue_latent(block, rows, last_position);
  else
    enqueue_recurrence(block, rows);
}

qllm_stream_norm_launch Mi355MixedProvider::stream_norm(std::uint32_t rows, float epsilon) {
  qllm_stream_norm_launch norm{};
  norm.input = hidden_[stream_index_].as<float>();
  norm.rows = rows;
  norm.width = g_.hidden;
  norm.epsilon = epsilon;
  norm.element = g_.element;
  norm.step = step_.as<std::uint32_t>();
  if (pending_partials_) {
    norm.partials = partials_.as<float>();
    norm.partial_count = pending_partials_;
    norm.partial_stride = round_up(g_.hidden, 4U);
    norm.branch_weight = pending_branch_.weight;
    norm.branch_scale = pending_branch_.scale;
    norm.branch_epsilon = pending_branch_.epsilon;
    stream_index_ = 1U - stream_index_;
    norm.stream_out = hidden_[stream_index_].as<float>();
    pending_partials_ = 0U;
    pending_branch_ = {};
  }
  return norm;
}

// Mixer and feed-forward one after the other; each leaves its output as partial
// sums (a single one, from a tall batch) that the next norm takes.
void Mi355MixedProvider::enqueue_sandwich(Block& block, std::uint32_t rows,
                                          std::uint32_t last_position) {
  const auto normed = [&](const DeviceBuffer& weight) {
    auto norm = stream_norm(rows, block.epsilon);
    norm.weight[0] = weight.as<float>();
    norm.output[0] = inputs_.get();
    norm.stride[0] = mixer_stride_;
    status_check(qllm_stream_norm(&norm, stream_));
  };
  const auto project = [&](const Matrix& matrix, std::uint32_t splits,
                           const DeviceBuffer& post_norm) {
    const bool split = g_.element == QLLM_ELEMENT_BF16 && rows <= kSmallBatch;
    qllm_linear_segment s{};
    s.weights = matrix.data.get();
    s.input = joined_.get();
    s.output = partials_.get();
    s.rows = matrix.rows;
    s.columns = matrix.columns;
    s.input_stride = matrix.columns;
    s.output_stride = round_up(g_.hidden, 4U);
    s.output_columns = g_.hidden;
    s.epilogue = split ? QLLM_LINEAR_PARTIALS : QLLM_LINEAR_STORE;
    s.splits = split ? splits : 0U;
    status_check(qllm_linear_batch(&s, 1U, rows, g_.element, stream_));
    pending_partials_ = split ? splits : 1U;
    pending_branch_ = {post_norm.as<float>(), block.residual_scale, block.epsilon};
  };
  qllm_linear_segment s{};
  s.input = inputs_.get();
  s.input_stride = mixer_stride_;

  normed(block.mixer_norm);
  const auto& projection = block.projections.front();
  s.weights = projection.matrix.data.get();
  s.output = projections_.get();
  s.rows = projection.matrix.rows;
  s.columns = projection.matrix.columns;
  s.output_stride = projection_stride_;
  s.output_columns = projection.matrix.rows;
  s.epilogue = QLLM_LINEAR_STORE;
  status_check(qllm_linear_batch(&s, 1U, rows, g_.element, stream_));
  enqueue_mixer(block, rows, last_position);
  project(block.output, block.splits, block.mixer_post_norm);
  if (!block.intermediate) return;

  normed(block.ffn_norm);
  s.weights = block.gate_up.data.get();
  s.output = joined_.get();
  s.rows = block.gate_up.rows;
  s.columns = block.gate_up.columns;
  s.output_stride = block.down.columns;
  s.output_columns = block.intermediate;
  s.epilogue = QLLM_LINEAR_GATED;
  s.activation = block.activation;
  status_check(qllm_linear_batch(&s, 1U, rows, g_.element, stream_));
  project(block.down, block.down_splits, block.ffn_post_norm);
}

void Mi355MixedProvider::enqueue_block(Block& block, std::uint32_t rows,
                                       std::uint32_t last_position) {
  if (block.sandwich) return enqueue_sandwich(block, rows, last_position);
  const std::size_t element = g_.element == QLLM_ELEMENT_F32 ? 4U : 2U;
  const auto input = [&](std::uint32_t index) {
    return static_cast<void*>(inputs_.as<std::uint8_t>() +
                              std::size_t{index} * workspace_rows_ * mixer_stride_ * element);
  };
  const std::uint32_t ffn_input = std::max(shift_inputs_, 1U);

  qllm_token_shift shift{};
  auto norm = stream_norm(rows, block.epsilon);
  norm.weight[0] = block.mixer_norm.as<float>();
  norm.output[0] = input(0U);
  norm.stride[0] = mixer_stride_;
  if (block.intermediate) {
    norm.weight[1] = block.ffn_norm.as<float>();
    norm.output[1] = input(ffn_input);
    norm.stride[1] = mixer_stride_;
  }
  if (!block.shifts.empty()) {
    shift.count = static_cast<std::uint32_t>(block.shifts.size());
    for (std::uint32_t i = 0; i < shift.count; ++i) {
      shift.mu[i] = block.shifts[i].as<float>();
      shift.output[i] = input(i);
    }
    shift.previous = states_.as<float>() + block.carry_offset;
    shift.slot_stride = state_floats_;
    shift.last = shift_last_.as<float>();
    norm.shift = &shift;
  }
  status_check(qllm_stream_norm(&norm, stream_));

  std::vector<qllm_linear_segment> segments;
  for (const auto& projection : block.projections) {
    qllm_linear_segment s{};
    s.weights = projection.matrix.data.get();
    s.input = input(projection.input);
    s.output = projections_.as<float>() + projection.column;
    s.rows = projection.matrix.rows;
    s.columns = projection.matrix.columns;
    s.input_stride = mixer_stride_;
    s.output_stride = projection_stride_;
    s.output_columns = projection.matrix.rows;
    s.epilogue = QLLM_LINEAR_STORE;
    segments.push_back(s);
  }
  if (block.intermediate) {
    qllm_linear_segment s{};
    s.weights = block.gate_up.data.get();
    s.input = input(ffn_input);
    s.output = joined_.as<std::uint8_t>() + block.mixer_columns * element;
    s.rows = block.gate_up.rows;
    s.columns = block.gate_up.columns;
    s.input_stride = mixer_stride_;
    s.output_stride = block.output.columns;
    s.output_columns = block.intermediate;
    s.epilogue = QLLM_LINEAR_GATED;
    s.activation = block.activation;
    segments.push_back(s);
  }
  status_check(qllm_linear_batch(segments.data(), static_cast<std::uint32_t>(segments.size()),
                                 rows, g_.element, stream_));
  enqueue_mixer(block, rows, last_position);

  qllm_linear_segment s{};
  s.weights = block.output.data.get();
  s.input = joined_.get();
  s.rows = block.output.rows;
  s.columns = block.output.columns;
  s.input_stride = block.output.columns;
  s.output_columns = g_.hidden;
  if (g_.element == QLLM_ELEMENT_BF16 && rows <= kSmallBatch) {
    s.output = partials_.get();
    s.output_stride = round_up(g_.hidden, 4U);
    s.epilogue = QLLM_LINEAR_PARTIALS;
    s.splits = block.splits;
    pending_partials_ = block.splits;
  } else {
    s.output = hidden_[stream_index_].get();
    s.output_stride = g_.hidden;
    s.epilogue = QLLM_LINEAR_ADD;
  }
  status_check(qllm_linear_batch(&s, 1U, rows, g_.element, stream_));
}

void Mi355MixedProvider::settle_stream(std::uint32_t rows) {
  if (!pending_partials_) return;
  const auto norm = stream_norm(rows, final_epsilon_);
  status_check(qllm_stream_norm(&norm, stream_));
}

// Final norm and head on `count` rows: those from `first` on, or with `gather`
// the rows listed in gather_.
void Mi355MixedProvider::enqueue_head(std::uint32_t batch_rows, std::uint32_t first,
                                      std::uint32_t count, bool gather) {
  if (batch_rows != 1U) settle_stream(batch_rows);
  auto norm = stream_norm(count, final_epsilon_);
  norm.input += std::size_t{first} * g_.hidden;
  norm.weight[0] = final_norm_.as<float>();
  norm.output[0] = head_input_.get();
  norm.stride[0] = mixer_stride_;
  norm.gather = gather ? gather_.as<std::uint32_t>() : nullptr;
  status_check(qllm_stream_norm(&norm, stream_));
  qllm_linear_segment s{};
  s.weights = head_.data.get();
  s.input = head_input_.get();
  s.output = logits_.get();
  s.rows = head_.rows;
  s.columns = head_.columns;
  s.input_stride = mixer_stride_;
  s.output_stride = round_up(g_.vocabulary, 4U);
  s.output_columns = g_.vocabulary;
  s.epilogue = QLLM_LINEAR_STORE;
  status_check(qllm_linear_batch(&s, 1U, count, g_.element, stream_));
}

// Logits of the rows asked for and the token of the last row.  The request has
// advanced when this returns.
Mi355MixedProvider::HeadResult Mi355MixedProvider::finish_batch(
    MixedRequestState& state, std::uint32_t rows, const er::ProgramRequestContext& request,
    bool head_enqueued) {
  const auto stream = static_cast<hipStream_t>(stream_);
  const std::uint32_t stride = round_up(g_.vocabulary, 4U);
  HeadResult result;
  result.logits = std::make_shared<std::vector<float>>();
  const auto wanted = std::move(state.logit_rows);
  state.logit_rows.clear();
  result.logits->resize(std::max<std::size_t>(wanted.size() * g_.vocabulary, 1U));
  const auto copy_rows = [&](std::size_t first, std::size_t count) {
    if (!count) return;
    hip_check(hipMemcpy2DAsync(result.logits->data() + first * g_.vocabulary,
                               std::size_t{g_.vocabulary} * 4U, logits_.get(),
                               std::size_t{stride} * 4U, std::size_t{g_.vocabulary} * 4U,
                               count, hipMemcpyDeviceToHost, stream),
              "copy logits");
    hip_check(hipStreamSynchronize(stream), "copy logits");
  };
  // the last row, asked for or not, is the one the token comes from
  const bool last_wanted = !wanted.empty() && wanted.back() == rows - 1U;
  const std::size_t before = wanted.size() - (last_wanted ? 1U : 0U);
  auto* listed = static_cast<std::uint32_t*>(staging_) + staging_words_;
  for (std::size_t first = 0U; first < before; first += kLogitRows) {
    const auto count =
        static_cast<std::uint32_t>(std::min<std::size_t>(kLogitRows, before - first));
    std::copy_n(wanted.begin() + static_cast<std::ptrdiff_t>(first), count, listed);
    hip_check(hipMemcpyAsync(gather_.get(), listed, count * 4U, hipMemcpyHostToDevice,
                             stream),
              "upload logit rows");
    enqueue_head(rows, 0U, count, true);
    copy_rows(first, count);
  }
  if (!head_enqueued) {
    enqueue_head(rows, rows - 1U, 1U, false);
    status_check(qllm_argmax_batch(logits_.as<float>(), g_.vocabulary, 1U,
                                   argmax_.as<std::uint32_t>(), select_workspace_.get(),
                                   select_workspace_bytes_, stream_));
  }
  if (last_wanted) copy_rows(before, 1U);
  const std::uint32_t last_position = state.position + rows - 1U;
  state.position += rows;
  result.token = selector_->select(
      logits_.as<float>(),
      presence_.as<std::uint8_t>() + std::size_t{state.slot} * g_.vocabulary,
      argmax_.as<std::uint32_t>(), request, last_position);
  release_pages(state);
  program_steps_ += rows;
  if (rows > 1U) prompt_rows_ += rows;
  return result;
}

// One token through the whole program, captured once: token, position and slot
// come from the step words.
void Mi355MixedProvider::launch_step_graph() {
  const auto stream = static_cast<hipStream_t>(stream_);
  const auto enqueue = [this] {
    enqueue_embedding(1U);
    for (auto& block : blocks_) enqueue_block(*block, 1U, g_.max_context - 1U);
    enqueue_head(1U, 0U, 1U, false);
    status_check(qllm_argmax_batch(logits_.as<float>(), g_.vocabulary, 1U,
                                   argmax_.as<std::uint32_t>(), select_workspace_.get(),
                                   select_workspace_bytes_, stream_));
  };
  // the first token runs uncaptured: it loads every kernel it needs
  if (!use_graphs_ || !step_warm_) {
    enqueue();
    step_warm_ = true;
    return;
  }
  if (!step_graph_) {
    hipGraph_t graph{};
    hip_check(hipStreamBeginCapture(stream, hipStreamCaptureModeThreadLocal),
              "begin step capture");
    try {
      enqueue();
    } catch (...) {
      (void)hipStreamEndCapture(stream, &graph);
      if (graph) (void)hipGraphDestroy(graph);
      throw;
    }
    hip_check(hipStreamEndCapture(stream, &graph), "end step capture");
    hipGraphExec_t executable{};
    const auto status = hipGraphInstantiate(&executable, graph, nullptr, nullptr, 0);
    (void)hipGraphDestroy(graph);
    hip_check(status, "instantiate step graph");
    step_graph_ = executable;
    step_stream_index_ = stream_index_;
  }
  stream_index_ = step_stream_index_;
  hip_check(hipGraphLaunch(static_cast<hipGraphExec_t>(step_graph_), stream),
            "launch step graph");
  ++graph_launches_;
}

er::ExecutionValue Mi355MixedProvider::hidden_value(std::uint32_t rows) const {
  return {std::string(kHiddenAbi), std::string(kDeviceDomain), lifetime_,
          reinterpret_cast<const std::byte*>(hidden_[0].get()),
          std::uint64_t{rows} * g_.hidden * 4U};
}

er::OperationExecutionResult Mi355MixedProvider::outputs_for(
    const PreparedOperation& operation,
    std::map<std::string, er::ExecutionValue, std::less<>> values) const {
  er::OperationExecutionResult result;
  result.status = er::Status::success();
  for (const auto& [port, abi] : operation.outputs) {
    const auto found = values.find(port);
    if (found == values.end() || found->second.abi != abi)
      throw std::runtime_error("mixed-layer output ABI mismatch");
    result.outputs.push_back(std::move(found->second));
  }
  return result;
}

namespace {

std::map<std::string, er::ExecutionValue, std::less<>> head_values(
    std::shared_ptr<std::vector<float>> logits, std::uint32_t token) {
  auto chosen = std::make_shared<std::vector<std::uint32_t>>(1U, token);
  const auto* logit_bytes = reinterpret_cast<const std::byte*>(logits->data());
  const std::uint64_t logit_size = logits->size() * 4U;
  const auto* token_bytes = reinterpret_cast<const std::byte*>(chosen->data());
  std::map<std::string, er::ExecutionValue, std::less<>> values;
  values.emplace("logits", er::ExecutionValue{std::string(kLogitsAbi), "host",
                                              std::move(logits), logit_bytes, logit_size});
  values.emplace("token_ids", er::ExecutionValue{std::string(kTokenAbi), "host",
                                                 std::move(chosen), token_bytes, 4U});
  return values;
}

std::uint32_t contiguous_first(std::span<const std::uint32_t> positions,
                               std::size_t rows) {
  if (positions.size() != rows || positions.empty())
    throw std::runtime_error("position batch does not match its tokens");
  for (std::size_t row = 1; row < rows; ++row)
    if (positions[row] != positions[0] + row)
      throw std::runtime_error("position batch is not contiguous");
  return positions[0];
}

}  // namespace

er::OperationExecutionHandle Mi355MixedProvider::execute(
    const er::IPreparedOperation& opaque_operation,
    const std::shared_ptr<er::IOperationProviderRequestState>& opaque_state,
    const er::OperationInvocation& invocation) {
  try {
    std::lock_guard lock(mutex_);
    const auto* operation = dynamic_cast<const PreparedOperation*>(&opaque_operation);
    const auto state = std::dynamic_pointer_cast<MixedRequestState>(opaque_state);
    if (!operation || !state)
      throw std::runtime_error("mixed-layer invocation state is invalid");
    const auto input = [&](std::string_view port) -> const er::ExecutionValue& {
      const auto found = operation->input_indices.find(port);
      if (found == operation->input_indices.end() ||
          found->second >= invocation.inputs.size())
        throw std::runtime_error("operation input port is absent");
      return invocation.inputs[found->second];
    };
    const auto require_rows = [&] {
      const auto& value = input("hidden");
      const std::uint64_t row_bytes = std::uint64_t{g_.hidden} * 4U;
      if (value.abi != kHiddenAbi || value.memory_domain != kDeviceDomain ||
          value.data != reinterpret_cast<const std::byte*>(hidden_[0].get()) ||
          value.bytes != batch_rows_ * row_bytes)
        throw std::runtime_error("hidden-state execution ABI mismatch");
      return batch_rows_;
    };
    std::map<std::string, er::ExecutionValue, std::less<>> values;
    if (operation->kind == Kind::embedding) {
      const auto tokens = host_u32_batch(input("token_ids"), kTokenAbi,
                                         "embedding token batch", g_.chunk_rows);
      begin_batch(*state, tokens, state->position);
      enqueue_embedding(batch_rows_);
      values.emplace("hidden", hidden_value(batch_rows_));
    } else if (operation->kind == Kind::head) {
      const auto rows = require_rows();
      const auto result = finish_batch(*state, rows, invocation.request, false);
      values = head_values(result.logits, result.token);
    } else {
      const auto rows = require_rows();
      const auto positions = host_u32_batch(input("positions"), kPositionAbi,
                                            "position batch", g_.chunk_rows);
      if (contiguous_first(positions, rows) != state->position)
        throw std::runtime_error("batch does not continue its request");
      enqueue_block(*blocks_.at(operation->block), rows, positions.back());
      settle_stream(rows);
      values.emplace("hidden", hidden_value(rows));
    }
    return completed_operation(outputs_for(*operation, std::move(values)));
  } catch (const std::exception& error) {
    return completed_operation({{er::ErrorCode::internal, error.what()}, {}});
  }
}

bool Mi355MixedProvider::supports_program_sequence(
    const er::CompiledModelProgram& program) const noexcept {
  return program.operations.size() == blocks_.size() + 2U;
}

er::OperationExecutionHandle Mi355MixedProvider::execute_program_sequence(
    const std::shared_ptr<er::IOperationProviderRequestState>& opaque_state,
    const er::ProgramSequenceInvocation& invocation) {
  try {
    std::lock_guard lock(mutex_);
    const auto state = std::dynamic_pointer_cast<MixedRequestState>(opaque_state);
    if (!state || invocation.operations.empty() ||
        invocation.inputs.size() != invocation.program.inputs.size())
      throw std::runtime_error("mixed-layer invocation state is invalid");
    const auto input = [&](std::string_view role) -> const er::ExecutionValue& {
      for (std::size_t index = 0; index < invocation.program.inputs.size(); ++index)
        if (invocation.program.inputs[index].role == role) return invocation.inputs[index];
      throw std::runtime_error("program input is absent");
    };
    const auto tokens = host_u32_batch(input("token_ids"), kTokenAbi,
                                       "embedding token batch", g_.chunk_rows);
    const auto positions =
        host_u32_batch(input("positions"), kPositionAbi, "position batch", g_.chunk_rows);
    const auto first = contiguous_first(positions, tokens.size());
    begin_batch(*state, tokens, first);
    const bool single = batch_rows_ == 1U;
    if (single) {
      launch_step_graph();
    } else {
      enqueue_embedding(batch_rows_);
      for (auto& block : blocks_) enqueue_block(*block, batch_rows_, positions.back());
    }
    auto result = finish_batch(*state, batch_rows_, invocation.request, single);
    auto values = head_values(std::move(result.logits), result.token);
    // outputs in the program's order
    er::OperationExecutionResult outputs;
    outputs.status = er::Status::success();
    for (const auto& endpoint : invocation.program.outputs) {
      const auto found = values.find(endpoint.role);
      if (found == values.end()) throw std::runtime_error("program output is unknown");
      outputs.outputs.push_back(std::move(found->second));
    }
    return completed_operation(std::move(outputs));
  } catch (const std::exception& error) {
    return completed_operation({{er::ErrorCode::internal, error.what()}, {}});
  }
}

er::Status Mi355MixedProvider::copy_hidden(std::uint32_t rows, float* host) {
  try {
    std::lock_guard lock(mutex_);
    if (!host || !rows || rows > batch_rows_)
      throw std::runtime_error("hidden rows are not available");
    hip_check(hipStreamSynchronize(static_cast<hipStream_t>(stream_)),
              "copy hidden rows");
    hip_check(hipMemcpy(host, hidden_[stream_index_].get(),
                        std::size_t{rows} * g_.hidden * 4U, hipMemcpyDeviceToHost),
              "copy hidden rows");
    return er::Status::success();
  } catch (const std::exception& error) {
    return {er::ErrorCode::internal, error.what()};
  }
}

std::map<std::string, std::uint64_t, std::less<>> Mi355MixedProvider::telemetry() const {
  std::lock_guard lock(mutex_);
  std::map<std::string, std::uint64_t, std::less<>> values;
  values["provider_program_steps"] = program_steps_;
  values["provider_prompt_rows"] = prompt_rows_;
  values["provider_graph_launches"] = graph_launches_;
  values["provider_weight_bytes"] = weight_bytes_;
  values["provider_kv_page_bytes"] = page_bytes_;
  values["provider_state_bytes"] = state_floats_ * 4U;
  values["kv_allocated_pages"] = slots_.live_pages();
  if (selector_) {
    values["provider_sampling_gpu_calls"] = selector_->gpu_calls();
    values["provider_sampling_logit_transfer_bytes"] = selector_->logit_transfer_bytes();
  }
  return values;
}

er::ExecutionProviderModule::ServiceContract Mi355MixedProvider::service_contract() const {
  er::ExecutionProviderModule::ServiceContract contract;
  contract.prefill_mode = "causal_layer_major";
  contract.prefill_chunk_tokens = g_.chunk_rows;
  contract.request_stream_mode = "per_request_nonblocking";
  contract.rope_mode = "artifact";
  contract.kv_dtype = g_.element == QLLM_ELEMENT_F32 ? "fp32" : "bf16";
  contract.kv_allocation = "paged_on_demand";
  contract.kv_page_tokens = g_.kv_page_tokens;
  contract.kv_page_bytes = std::max<std::uint64_t>(page_bytes_, 1U);
  contract.kv_page_capacity =
      std::uint64_t{g_.capacity} *
      ((g_.max_context + g_.kv_page_tokens - 1U) / g_.kv_page_tokens);
  contract.placement_mode = "resident";
  contract.placement_profile = "resident";
  contract.vram_cache_bytes = std::max<std::uint64_t>(weight_bytes_, 1U);
  contract.placement_prefetch_state = "disabled";
  contract.sampling_supported = true;
  return contract;
}

}  // namespace qllm
