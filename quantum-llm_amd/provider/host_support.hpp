// Small host-side helpers every provider uses: status plumbing, owned device
// memory, request parameters.
#pragma once

#include "expert/runtime/program_executor.hpp"

#include <cstddef>
#include <cstdint>
#include <string_view>

namespace qllm {

namespace er = expert::runtime;

// hipError_t as int: this header stays free of the HIP runtime
void hip_check(int error, const char* what);
void status_check(std::int32_t status);

// A device allocation that is freed unless release() hands it on.
class DeviceBuffer final {
 public:
  DeviceBuffer() = default;
  DeviceBuffer(std::size_t bytes, const char* what);
  ~DeviceBuffer();
  DeviceBuffer(const DeviceBuffer&) = delete;
  DeviceBuffer& operator=(const DeviceBuffer&) = delete;
  DeviceBuffer(DeviceBuffer&& other) noexcept : pointer_(other.release()) {}
  DeviceBuffer& operator=(DeviceBuffer&& other) noexcept;
  [[nodiscard]] void* get() const noexcept { return pointer_; }
  template <typename T>
  [[nodiscard]] T* as() const noexcept {
    return static_cast<T*>(pointer_);
  }
  [[nodiscard]] void* release() noexcept {
    void* pointer = pointer_;
    pointer_ = nullptr;
    return pointer;
  }

 private:
  void* pointer_{};
};

[[nodiscard]] std::uint64_t request_parameter(const er::ProgramRequestContext& request,
                                              std::string_view name);
// The penalty a request asks for: the parameter is biased by 2,000,000 ppm so
// that negative penalties travel as unsigned values
// (runtime/tools/moe_vm_runner.cpp:318-347, dense_fp4_provider.cpp:8336-8341).
[[nodiscard]] double presence_penalty_of(const er::ProgramRequestContext& request);
// The sampling profile check of dense_fp4_provider.cpp:5502-5513: throws when a
// sampled request's profile is unusable.
void require_sampling_profile(const er::ProgramRequestContext& request,
                              std::uint32_t max_context);

[[nodiscard]] er::OperationExecutionHandle completed_operation(
    er::OperationExecutionResult result);
// token ids or positions of a batch, at most `limit` of them
[[nodiscard]] std::span<const std::uint32_t> host_u32_batch(
    const er::ExecutionValue& value, std::string_view abi,
    std::string_view description, std::size_t limit);

// Value ABIs between operations as an artifact declares them
// (dense_fp4_provider.cpp:59-74).  The hidden-state ABI string names F32 rows
// in device memory; the memory domain says whose device.
inline constexpr std::string_view kHiddenAbi = "batch.hidden.f32.cuda.v1";
inline constexpr std::string_view kTokenAbi = "batch.token-id.u32.host.v1";
inline constexpr std::string_view kPositionAbi = "batch.position.u32.host.v1";
inline constexpr std::string_view kDeviceDomain = "hip.device";

[[nodiscard]] const er::ImmutableModelTensor* optional_tensor(
    std::span<const er::PreparedTensorBinding> tensors, std::string_view role);
[[nodiscard]] const er::ImmutableModelTensor& tensor_for(
    std::span<const er::PreparedTensorBinding> tensors, std::string_view role);

}  // namespace qllm
