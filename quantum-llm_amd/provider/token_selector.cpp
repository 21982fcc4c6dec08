#include "token_selector.hpp"

#include "host_support.hpp"
#include "qllm_kernels.h"

#include <hip/hip_runtime.h>

#include <algorithm>
#include <cmath>
#include <numeric>
#include <stdexcept>

namespace qllm {

TokenSelector::TokenSelector(void* stream, std::uint32_t vocabulary, void* workspace,
                             std::size_t workspace_bytes)
    : stream_(stream), vocabulary_(vocabulary), workspace_(workspace),
      workspace_bytes_(workspace_bytes),
      device_(8U * kMaximumTopK * (4U + 4U) + 8U * 4U, "allocate token selection") {
  // top-k logits of up to 8 rows, then their tokens: one buffer, one readback;
  // the marks follow
  top_logits_ = device_.as<float>();
  top_tokens_ = reinterpret_cast<std::uint32_t*>(top_logits_ + 8U * kMaximumTopK);
  mark_tokens_ = top_tokens_ + 8U * kMaximumTopK;
  void* pinned = nullptr;
  hip_check(hipHostMalloc(&pinned, sizeof(Staging), hipHostMallocDefault),
            "allocate pinned staging");
  staging_ = static_cast<Staging*>(pinned);
  *staging_ = Staging{};
}

TokenSelector::~TokenSelector() {
  if (staging_) (void)hipHostFree(staging_);
}

std::size_t TokenSelector::workspace_bytes(std::uint32_t vocabulary,
                                           std::uint32_t rows) {
  return std::max({qllm_argmax_workspace_bytes(vocabulary, rows),
                   qllm_topk_workspace_bytes(vocabulary, kMaximumTopK),
                   qllm_topk_batch_workspace_bytes(vocabulary, kMaximumTopK, rows)});
}

void TokenSelector::mark(
    std::uint8_t* emitted, std::span<const std::uint32_t> tokens) {
  if (tokens.empty()) return;
  if (tokens.size() > 8U) throw std::runtime_error("too many presence marks");
  const auto stream = static_cast<hipStream_t>(stream_);
  // the pinned words are free: every pass that used them ended with a wait
  std::copy(tokens.begin(), tokens.end(), staging_->marks);
  hip_check(hipMemcpyAsync(mark_tokens_, staging_->marks, tokens.size() * 4U,
                           hipMemcpyHostToDevice, stream),
            "upload presence marks");
  status_check(qllm_mark_presence(emitted, mark_tokens_,
                                  static_cast<std::uint32_t>(tokens.size()),
                                  vocabulary_, stream_));
}


// The head's token for a request (run_head with a request, :8433-8517): the
// presence penalty from the first output position on, arg-max at temperature
// zero, otherwise top-k or whole-row candidates ordered on the host and one
// draw from stream 0; an output token is marked as emitted.  One row of
// logits.
std::uint32_t TokenSelector::select(float* logits, std::uint8_t* presence,
                                    std::uint32_t* argmax_tokens,
                                    const er::ProgramRequestContext& request,
                                    std::uint32_t sample_position) {
  const auto stream = static_cast<hipStream_t>(stream_);
  const auto first_output =
      request_parameter(request, "sampling_first_output_position");
  const bool output_sampling = sample_position >= first_output;
  const auto penalty = presence_penalty_of(request);
  if (output_sampling && penalty != 0.0) {
    status_check(qllm_apply_presence_penalty(logits, presence, vocabulary_,
                                             static_cast<float>(penalty),
                                             stream_));
    status_check(qllm_argmax_batch(logits, vocabulary_, 1U, argmax_tokens,
                                   workspace_, workspace_bytes_,
                                   stream_));
  }
  const auto temperature = request_parameter(request, "sampling_temperature_ppm");
  std::uint32_t selected{};
  if (temperature == 0U) {
    hip_check(hipMemcpyAsync(&selected, argmax_tokens, sizeof(selected),
                             hipMemcpyDeviceToHost, stream),
              "copy greedy token");
    hip_check(hipStreamSynchronize(stream), "copy greedy token");
    // a row without a finite logit selects nothing (0xffffffff): reported
    // before the presence bytes or the caller's state change
    if (selected >= vocabulary_)
      throw std::runtime_error("head logits have no finite maximum");
  } else {
    // the penalty, if any, has been applied: the distribution is taken from
    // the row as it stands
    er::ProgramRequestContext unpenalised = request;
    unpenalised.parameters["sampling_presence_penalty_biased_ppm"] = 2'000'000U;
    const auto top_k = request_parameter(request, "sampling_top_k");
    if (top_k > kMaximumTopK) {
      // the scalar sampler orders that many candidates on the host
      // (sample_token, :773-799)
      std::vector<float> row(vocabulary_);
      hip_check(hipMemcpyAsync(row.data(), logits, row.size() * 4U,
                               hipMemcpyDeviceToHost, stream),
                "copy sampling logits");
      hip_check(hipStreamSynchronize(stream), "copy sampling logits");
      if (top_k > row.size())
        throw std::runtime_error("invalid token sampling contract");
      std::vector<std::uint32_t> candidates(row.size());
      std::iota(candidates.begin(), candidates.end(), 0U);
      const auto before = [&](std::uint32_t left, std::uint32_t right) {
        const float a = row[left];
        const float b = row[right];
        if (std::isnan(a)) return false;
        if (std::isnan(b)) return true;
        return a == b ? left < right : a > b;
      };
      std::partial_sort(candidates.begin(), candidates.begin() + top_k,
                        candidates.end(), before);
      candidates.resize(top_k);
      std::vector<float> ordered;
      for (const auto candidate : candidates) ordered.push_back(row[candidate]);
      logit_transfer_bytes_ += row.size() * 4U;
      const auto distribution = er::make_sampling_distribution(
          ordered, candidates, static_cast<std::uint32_t>(temperature),
          static_cast<std::uint32_t>(
              request_parameter(request, "sampling_top_p_ppm")),
          static_cast<std::uint32_t>(
              request_parameter(request, "sampling_min_p_ppm")));
      selected = er::sample_distribution(
          distribution,
          er::counter_uniform(request_parameter(request, "sampling_seed"),
                              sample_position, 0U));
    } else {
      const auto chosen = this->distribution(
          logits, vocabulary_, argmax_tokens, unpenalised, nullptr);
      selected = er::sample_distribution(
          chosen,
          er::counter_uniform(request_parameter(request, "sampling_seed"),
                              sample_position, 0U));
    }
  }
  if (output_sampling) {
    const std::uint32_t token[1] = {selected};
    mark(presence, token);
  }
  return selected;
}


// distribution_from_logits, dense_fp4_provider.cpp:8331-8391.  top_k == 0
// selects the whole-vocabulary path of the scalar sampler (sample_token,
// :773-799): the row is copied to the host and ordered there.
er::SamplingDistribution TokenSelector::distribution(
    float* row_logits, std::uint32_t vocabulary, std::uint32_t* device_argmax,
    const er::ProgramRequestContext& request, const std::uint8_t* presence) {
  const auto stream = static_cast<hipStream_t>(stream_);
  const auto penalty = presence_penalty_of(request);
  const auto temperature = request_parameter(request, "sampling_temperature_ppm");
  if (penalty != 0.0) {
    if (!presence) throw std::runtime_error("sampling presence state is absent");
    status_check(qllm_apply_presence_penalty(row_logits, presence, vocabulary,
                                             static_cast<float>(penalty),
                                             stream_));
    // the arg-max the pass left behind was taken before the penalty
    if (temperature == 0U)
      status_check(qllm_argmax_batch(row_logits, vocabulary, 1U, device_argmax,
                                     workspace_, workspace_bytes_,
                                     stream_));
  }
  if (temperature == 0U) {
    std::uint32_t token{};
    hip_check(hipMemcpyAsync(&token, device_argmax, sizeof(token),
                             hipMemcpyDeviceToHost, stream),
              "copy exact greedy token");
    hip_check(hipStreamSynchronize(stream), "copy exact greedy token");
    return {{{token, 1.0}}};
  }
  const auto top_p = static_cast<std::uint32_t>(
      request_parameter(request, "sampling_top_p_ppm"));
  const auto min_p = static_cast<std::uint32_t>(
      request_parameter(request, "sampling_min_p_ppm"));
  const auto top_k = request_parameter(request, "sampling_top_k");
  if (top_k > kMaximumTopK || top_k > vocabulary)
    throw std::runtime_error(
        "sampled exact decode requires top-k of at most 64 (0 = whole row)");
  std::vector<float> host_logits;
  std::vector<std::uint32_t> host_tokens;
  if (top_k == 0U) {
    std::vector<float> full(vocabulary);
    hip_check(hipMemcpyAsync(full.data(), row_logits, full.size() * 4U,
                             hipMemcpyDeviceToHost, stream),
              "copy logit row");
    hip_check(hipStreamSynchronize(stream), "copy logit row");
    host_tokens.resize(vocabulary);
    std::iota(host_tokens.begin(), host_tokens.end(), 0U);
    std::sort(host_tokens.begin(), host_tokens.end(),
              [&](std::uint32_t left, std::uint32_t right) {
                const float a = full[left];
                const float b = full[right];
                if (std::isnan(a)) return false;
                if (std::isnan(b)) return true;
                return a == b ? left < right : a > b;
              });
    host_logits.reserve(vocabulary);
    for (const auto token : host_tokens) host_logits.push_back(full[token]);
    logit_transfer_bytes_ += full.size() * 4U;
  } else {
    return std::move(top_k_distributions(row_logits, vocabulary, vocabulary,
                                              1U, request)
                         .front());
  }
  return er::make_sampling_distribution(
      host_logits, host_tokens, static_cast<std::uint32_t>(temperature), top_p,
      min_p);
}

// The distributions of `rows` rows of logits (row r at logits + r * stride)
// for a sampled request with 1 <= top_k <= 64: one selection launch for all
// rows, one readback, then make_sampling_distribution per row
// (distribution_from_logits, dense_fp4_provider.cpp:8331-8391, which selects
// and reads back row by row).
std::vector<er::SamplingDistribution>
TokenSelector::top_k_distributions(
    const float* logits, std::uint32_t vocabulary, std::size_t stride,
    std::uint32_t rows, const er::ProgramRequestContext& request) {
  const auto stream = static_cast<hipStream_t>(stream_);
  const auto temperature = request_parameter(request, "sampling_temperature_ppm");
  const auto top_p = static_cast<std::uint32_t>(
      request_parameter(request, "sampling_top_p_ppm"));
  const auto min_p = static_cast<std::uint32_t>(
      request_parameter(request, "sampling_min_p_ppm"));
  const auto top_k =
      static_cast<std::uint32_t>(request_parameter(request, "sampling_top_k"));
  if (!rows || rows > 8U || !top_k || top_k > kMaximumTopK ||
      top_k > vocabulary)
    throw std::runtime_error(
        "sampled exact decode requires top-k of at most 64 (0 = whole row)");
  status_check(qllm_topk_logits_batch(logits, vocabulary, stride, top_k, rows,
                                      top_logits_, top_tokens_, workspace_,
                                      workspace_bytes_, stream_));
  // logits of all rows, then tokens of all rows (the device buffers are
  // adjacent with room for 8 rows of 64)
  constexpr std::size_t kCapacity = 8U * kMaximumTopK;
  hip_check(hipMemcpyAsync(staging_->top_logits, top_logits_,
                           kCapacity * 4U + std::size_t{rows} * top_k * 4U,
                           hipMemcpyDeviceToHost, stream),
            "copy speculative top-k");
  hip_check(hipStreamSynchronize(stream), "copy speculative top-k");
  ++gpu_calls_;
  logit_transfer_bytes_ += std::size_t{rows} * top_k * 8U;
  std::vector<er::SamplingDistribution> result;
  result.reserve(rows);
  for (std::uint32_t row = 0; row < rows; ++row) {
    const std::span<const float> row_logits(
        staging_->top_logits + std::size_t{row} * top_k, top_k);
    const std::span<const std::uint32_t> row_tokens(
        staging_->top_tokens + std::size_t{row} * top_k, top_k);
    result.push_back(er::make_sampling_distribution(
        row_logits, row_tokens, static_cast<std::uint32_t>(temperature), top_p,
        min_p));
  }
  return result;
}

}  // namespace qllm
