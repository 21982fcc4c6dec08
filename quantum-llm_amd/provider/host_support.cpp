#include "host_support.hpp"

#include "qllm_kernels.h"

#include <hip/hip_runtime.h>

#include <stdexcept>
#include <string>

namespace qllm {

void hip_check(int error, const char* what) {
  if (error != hipSuccess)
    throw std::runtime_error(std::string(what) + ": " +
                             hipGetErrorString(static_cast<hipError_t>(error)));
}

void status_check(std::int32_t status) {
  if (status != QLLM_OK) throw std::runtime_error(qllm_last_error());
}

DeviceBuffer::DeviceBuffer(std::size_t bytes, const char* what) {
  hip_check(hipMalloc(&pointer_, bytes), what);
}

DeviceBuffer::~DeviceBuffer() {
  if (pointer_) (void)hipFree(pointer_);
}

DeviceBuffer& DeviceBuffer::operator=(DeviceBuffer&& other) noexcept {
  if (this != &other) {
    if (pointer_) (void)hipFree(pointer_);
    pointer_ = other.release();
  }
  return *this;
}

std::uint64_t request_parameter(const er::ProgramRequestContext& request,
                                std::string_view name) {
  const auto found = request.parameters.find(name);
  if (found == request.parameters.end())
    throw std::runtime_error("request parameter is absent: " +
                             std::string(name));
  return found->second;
}

double presence_penalty_of(const er::ProgramRequestContext& request) {
  const auto biased =
      request_parameter(request, "sampling_presence_penalty_biased_ppm");
  if (biased > 4'000'000U)
    throw std::runtime_error("sampling presence penalty is invalid");
  return (static_cast<double>(biased) - 2'000'000.0) / 1'000'000.0;
}

void require_sampling_profile(const er::ProgramRequestContext& request,
                              std::uint32_t max_context) {
  const auto temperature = request.parameters.find("sampling_temperature_ppm");
  if (temperature == request.parameters.end() || temperature->second == 0U) return;
  const auto first = request.parameters.find("sampling_first_output_position");
  const auto presence =
      request.parameters.find("sampling_presence_penalty_biased_ppm");
  if (first == request.parameters.end() || first->second >= max_context ||
      presence == request.parameters.end() || presence->second > 4'000'000U)
    throw std::runtime_error("request has an invalid sampling profile");
}

// :5605-5620
er::OperationExecutionHandle completed_operation(
    er::OperationExecutionResult result) {
  auto shared = std::make_shared<std::optional<er::OperationExecutionResult>>(
      std::move(result));
  return er::OperationExecutionHandle::from_callbacks(
      [shared]() {
        auto value = std::move(*shared);
        shared->reset();
        return value;
      },
      [shared]() { shared->reset(); });
}

// :550-564
std::span<const std::uint32_t> host_u32_batch(const er::ExecutionValue& value,
                                              std::string_view abi,
                                              std::string_view description,
                                              std::size_t limit) {
  if (!value.valid() || value.abi != abi || value.memory_domain != "host" ||
      value.bytes % sizeof(std::uint32_t) != 0U ||
      value.bytes / sizeof(std::uint32_t) > limit ||
      reinterpret_cast<std::uintptr_t>(value.data) % alignof(std::uint32_t) != 0U)
    throw std::runtime_error(std::string(description) + " ABI mismatch");
  return {reinterpret_cast<const std::uint32_t*>(value.data),
          static_cast<std::size_t>(value.bytes / sizeof(std::uint32_t))};
}

const er::ImmutableModelTensor* optional_tensor(
    std::span<const er::PreparedTensorBinding> tensors, std::string_view role) {
  for (const auto& binding : tensors)
    if (binding.role == role && binding.tensor) return binding.tensor.get();
  return nullptr;
}

const er::ImmutableModelTensor& tensor_for(
    std::span<const er::PreparedTensorBinding> tensors, std::string_view role) {
  if (const auto* tensor = optional_tensor(tensors, role)) return *tensor;
  throw std::runtime_error("tensor role is not bound: " + std::string(role));
}

}  // namespace qllm
