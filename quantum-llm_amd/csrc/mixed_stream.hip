// The residual stream of mixed-layer decoders: embedding lookup and the norm
// kernel every layer starts with - the partial sums of the projection before
// it added to the stream, the row's root mean square taken once, up to two
// normalised copies written (a parallel layer feeds its mixer and its
// feed-forward from the same row), or the token-shift blends of a mixer that
// reads the previous token's normalised input as well.
#include "mixed_common.hpp"

namespace qllm {
namespace {

constexpr int kHeld = 4;   // 16-byte pieces of a row a thread keeps in registers

struct NormArgs {
  qllm_stream_norm_launch launch;
  qllm_token_shift shift;
};

// The stream with the partial sums added; with a branch norm the sums alone.
__device__ __forceinline__ f32x4 stream_value4(const qllm_stream_norm_launch& l,
                                               uint32_t row, uint32_t piece) {
  f32x4 value = l.branch_weight
                    ? f32x4{}
                    : reinterpret_cast<const f32x4*>(l.input + size_t{row} * l.width)[piece];
  // eight loads in flight at a time
  for (uint32_t first = 0; first < l.partial_count; first += 8u) {
    f32x4 part[8];
#pragma unroll
    for (uint32_t i = 0; i < 8u; ++i)
      part[i] = first + i < l.partial_count
                    ? reinterpret_cast<const f32x4*>(
                          l.partials +
                          (size_t{first + i} * l.rows + row) * l.partial_stride)[piece]
                    : f32x4{};
#pragma unroll
    for (uint32_t i = 0; i < 8u; ++i) value += part[i];
  }
  return value;
}

__device__ __forceinline__ float stream_value(const qllm_stream_norm_launch& l,
                                              uint32_t row, uint32_t column) {
  float value = l.branch_weight ? 0.0f : l.input[size_t{row} * l.width + column];
  for (uint32_t p = 0; p < l.partial_count; ++p)
    value += l.partials[(size_t{p} * l.rows + row) * l.partial_stride + column];
  return value;
}

__device__ __forceinline__ float inverse_rms(float squares, uint32_t width, float epsilon) {
  return 1.0f / sqrtf(squares / static_cast<float>(width) + epsilon);
}

template <typename T>
__device__ __forceinline__ void put4(void* output, size_t index, f32x4 value) {
  if constexpr (sizeof(T) == 4) {
    *reinterpret_cast<f32x4*>(static_cast<float*>(output) + index) = value;
  } else {
    const uint32_t low = f32_to_bf16_bits(value[0]) | f32_to_bf16_bits(value[1]) << 16;
    const uint32_t high = f32_to_bf16_bits(value[2]) | f32_to_bf16_bits(value[3]) << 16;
    *reinterpret_cast<i32x2*>(static_cast<uint16_t*>(output) + index) =
        i32x2{static_cast<int>(low), static_cast<int>(high)};
  }
}

template <typename T>
__device__ __forceinline__ void pad_row(void* output, uint32_t row, uint32_t width,
                                        uint32_t stride) {
  for (uint32_t c = width + threadIdx.x; c < stride; c += blockDim.x)
    store_element(static_cast<T*>(output) + size_t{row} * stride + c, 0.0f);
}

// Rows whose width is a multiple of 4 and fits kHeld pieces per thread.
template <typename T>
__global__ __launch_bounds__(1024) void stream_norm_wide_kernel(NormArgs args) {
  __shared__ float scratch[16];
  const qllm_stream_norm_launch& l = args.launch;
  const uint32_t row = blockIdx.x;
  const uint32_t source = l.gather ? l.gather[row] : row;
  const uint32_t pieces = l.width / 4u;
  f32x4 held[kHeld];
  float squares = 0.0f;
#pragma unroll
  for (int i = 0; i < kHeld; ++i) {
    const uint32_t piece = threadIdx.x + i * blockDim.x;
    held[i] = f32x4{};
    if (piece >= pieces) continue;
    held[i] = stream_value4(l, source, piece);
    if (l.partial_count && !l.branch_weight)
      reinterpret_cast<f32x4*>(l.stream_out + size_t{row} * l.width)[piece] = held[i];
#pragma unroll
    for (int c = 0; c < 4; ++c) squares = fmaf(held[i][c], held[i][c], squares);
  }
  if (l.branch_weight) {
    f32x4 before[kHeld], weight[kHeld];
#pragma unroll
    for (int i = 0; i < kHeld; ++i) {
      const uint32_t piece = threadIdx.x + i * blockDim.x;
      if (piece >= pieces) continue;
      before[i] = reinterpret_cast<const f32x4*>(l.input + size_t{row} * l.width)[piece];
      weight[i] = reinterpret_cast<const f32x4*>(l.branch_weight)[piece];
    }
    const float unit =
        inverse_rms(block_sum(squares, scratch), l.width, l.branch_epsilon);
    squares = 0.0f;
#pragma unroll
    for (int i = 0; i < kHeld; ++i) {
      const uint32_t piece = threadIdx.x + i * blockDim.x;
      if (piece >= pieces) continue;
      held[i] = before[i] + held[i] * unit * weight[i] * l.branch_scale;
      reinterpret_cast<f32x4*>(l.stream_out + size_t{row} * l.width)[piece] = held[i];
#pragma unroll
      for (int c = 0; c < 4; ++c) squares = fmaf(held[i][c], held[i][c], squares);
    }
  }
  const float inverse = inverse_rms(block_sum(squares, scratch), l.width, l.epsilon);
  const bool shifted = l.shift != nullptr;
#pragma unroll
  for (int output = 0; output < 2; ++output) {
    if (!l.weight[output] || (shifted && output == 0)) continue;
#pragma unroll
    for (int i = 0; i < kHeld; ++i) {
      const uint32_t piece = threadIdx.x + i * blockDim.x;
      if (piece >= pieces) continue;
      const f32x4 weight = reinterpret_cast<const f32x4*>(l.weight[output])[piece];
      put4<T>(l.output[output], size_t{row} * l.stride[output] + piece * 4u,
              held[i] * inverse * weight);
    }
    pad_row<T>(l.output[output], row, l.width, l.stride[output]);
  }
  if (!shifted) return;

  const qllm_token_shift& shift = args.shift;
  f32x4 before[kHeld];
  float before_squares = 0.0f;
#pragma unroll
  for (int i = 0; i < kHeld; ++i) {
    const uint32_t piece = threadIdx.x + i * blockDim.x;
    before[i] = f32x4{};
    if (piece >= pieces) continue;
    before[i] = row == 0u
                    ? reinterpret_cast<const f32x4*>(
                          shift.previous + l.step[kStepSlot] * shift.slot_stride)[piece]
                    : stream_value4(l, row - 1u, piece);
#pragma unroll
    for (int c = 0; c < 4; ++c)
      before_squares = fmaf(before[i][c], before[i][c], before_squares);
  }
  // row 0 takes the norm the request carries, already weighted
  const float before_inverse =
      inverse_rms(block_sum(before_squares, scratch), l.width, l.epsilon);
#pragma unroll
  for (int i = 0; i < kHeld; ++i) {
    const uint32_t piece = threadIdx.x + i * blockDim.x;
    if (piece >= pieces) continue;
    const f32x4 weight = reinterpret_cast<const f32x4*>(l.weight[0])[piece];
    const f32x4 here = held[i] * inverse * weight;
    const f32x4 there = row == 0u ? before[i] : before[i] * before_inverse * weight;
    for (uint32_t s = 0; s < shift.count; ++s) {
      const f32x4 mu = reinterpret_cast<const f32x4*>(shift.mu[s])[piece];
      put4<T>(shift.output[s], size_t{row} * l.stride[0] + piece * 4u,
              here + (there - here) * mu);
    }
    if (row + 1u == l.rows) reinterpret_cast<f32x4*>(shift.last)[piece] = here;
  }
  for (uint32_t s = 0; s < shift.count; ++s)
    pad_row<T>(shift.output[s], row, l.width, l.stride[0]);
}

template <typename T>
__global__ __launch_bounds__(256) void stream_norm_narrow_kernel(NormArgs args) {
  __shared__ float scratch[16];
  const qllm_stream_norm_launch& l = args.launch;
  const uint32_t row = blockIdx.x;
  const uint32_t source = l.gather ? l.gather[row] : row;
  const bool shifted = l.shift != nullptr;
  const float* carried =
      shifted && row == 0u ? args.shift.previous + l.step[kStepSlot] * args.shift.slot_stride
                           : nullptr;
  float squares = 0.0f;
  float before_squares = 0.0f;
  float unit_branch = 0.0f;
  if (l.branch_weight) {
    float branch_squares = 0.0f;
    for (uint32_t c = threadIdx.x; c < l.width; c += blockDim.x) {
      const float value = stream_value(l, source, c);
      branch_squares = fmaf(value, value, branch_squares);
    }
    unit_branch = inverse_rms(block_sum(branch_squares, scratch), l.width, l.branch_epsilon) *
                  l.branch_scale;
  }
  const auto here_value = [&](uint32_t c) {
    const float value = stream_value(l, source, c);
    return l.branch_weight ? l.input[size_t{row} * l.width + c] +
                                 value * unit_branch * l.branch_weight[c]
                           : value;
  };
  for (uint32_t c = threadIdx.x; c < l.width; c += blockDim.x) {
    const float value = here_value(c);
    if (l.partial_count) l.stream_out[size_t{row} * l.width + c] = value;
    squares = fmaf(value, value, squares);
    if (shifted && !carried) {
      const float before = stream_value(l, row - 1u, c);
      before_squares = fmaf(before, before, before_squares);
    }
  }
  const float inverse = inverse_rms(block_sum(squares, scratch), l.width, l.epsilon);
  const float before_inverse =
      inverse_rms(block_sum(before_squares, scratch), l.width, l.epsilon);
  for (uint32_t c = threadIdx.x; c < l.width; c += blockDim.x) {
    const float unit = here_value(c) * inverse;
    for (int output = 0; output < 2; ++output)
      if (l.weight[output] && !(shifted && output == 0))
        store_element(static_cast<T*>(l.output[output]) +
                          size_t{row} * l.stride[output] + c,
                      unit * l.weight[output][c]);
    if (!shifted) continue;
    const float here = unit * l.weight[0][c];
    const float there =
        carried ? carried[c]
                : stream_value(l, row - 1u, c) * before_inverse * l.weight[0][c];
    for (uint32_t s = 0; s < args.shift.count; ++s)
      store_element(static_cast<T*>(args.shift.output[s]) + size_t{row} * l.stride[0] + c,
                    here + (there - here) * args.shift.mu[s][c]);
    if (row + 1u == l.rows) args.shift.last[c] = here;
  }
  for (int output = 0; output < 2; ++output)
    if (l.weight[output] && !(shifted && output == 0))
      pad_row<T>(l.output[output], row, l.width, l.stride[output]);
  if (shifted)
    for (uint32_t s = 0; s < args.shift.count; ++s)
      pad_row<T>(args.shift.output[s], row, l.width, l.stride[0]);
}

__global__ void embedding_bf16_kernel(const uint16_t* table, uint32_t vocabulary,
                                      const uint32_t* tokens, float* output,
                                      uint32_t width, float scale) {
  const uint32_t token = tokens[blockIdx.x];
  for (uint32_t c = threadIdx.x; c < width; c += blockDim.x)
    output[size_t{blockIdx.x} * width + c] =
        token < vocabulary
            ? bf16_bits_to_f32(table[size_t{token} * width + c]) * scale
            : 0.0f;
}

bool aligned16(const void* pointer) {
  return (reinterpret_cast<uintptr_t>(pointer) & 15u) == 0u;
}

}  // namespace
}  // namespace qllm

using namespace qllm;

extern "C" int32_t qllm_embedding_bf16_batch(const void* table_bf16, uint32_t vocabulary,
                                             const uint32_t* tokens, float* output,
                                             uint32_t rows, uint32_t width, float scale,
                                             void* stream) {
  if (!table_bf16 || !tokens || !output || !rows || !width || !vocabulary)
    return fail(QLLM_INVALID_ARGUMENT, "invalid bf16 embedding lookup");
  embedding_bf16_kernel<<<rows, 256, 0, as_stream(stream)>>>(
      static_cast<const uint16_t*>(table_bf16), vocabulary, tokens, output, width, scale);
  return launched("bf16 embedding lookup");
}

extern "C" int32_t qllm_stream_norm(const qllm_stream_norm_launch* launch, void* stream) {
  if (!launch || !launch->input || !launch->rows || !launch->width ||
      launch->element > QLLM_ELEMENT_F32 ||
      (launch->partial_count &&
       (!launch->partials || !launch->stream_out || launch->stream_out == launch->input ||
        launch->partial_stride < launch->width || launch->gather)) ||
      (launch->branch_weight && (!launch->partial_count || launch->shift)))
    return fail(QLLM_INVALID_ARGUMENT, "invalid stream norm");
  bool wide = launch->width % 4u == 0u && launch->partial_stride % 4u == 0u &&
              aligned16(launch->input) && aligned16(launch->stream_out) &&
              aligned16(launch->partials) && aligned16(launch->branch_weight);
  for (int i = 0; i < 2; ++i) {
    if (!launch->weight[i]) continue;
    const bool blended = i == 0 && launch->shift;
    if ((!launch->output[i] && !blended) || launch->stride[i] < launch->width)
      return fail(QLLM_INVALID_ARGUMENT, "invalid stream norm output");
    wide = wide && aligned16(launch->weight[i]) && aligned16(launch->output[i]) &&
           launch->stride[i] % 4u == 0u;
  }
  NormArgs args{*launch, {}};
  if (const auto* shift = launch->shift) {
    if (!shift->count || shift->count > 6u || !shift->previous || !shift->last ||
        !launch->step || launch->gather || !launch->weight[0])
      return fail(QLLM_INVALID_ARGUMENT, "invalid token shift");
    for (uint32_t s = 0; s < shift->count; ++s) {
      if (!shift->mu[s] || !shift->output[s])
        return fail(QLLM_INVALID_ARGUMENT, "invalid token shift");
      wide = wide && aligned16(shift->mu[s]) && aligned16(shift->output[s]);
    }
    wide = wide && aligned16(shift->previous) && aligned16(shift->last) &&
           shift->slot_stride % 4u == 0u;
    args.shift = *shift;
  }
  const uint32_t pieces = launch->width / 4u;
  uint32_t threads = launch->rows <= 16u ? 1024u : 256u;
  while (threads > 64u && threads / 2u >= pieces) threads /= 2u;
  if (pieces > threads * kHeld) threads = 1024u;
  wide = wide && pieces <= threads * kHeld;
  const auto hip_stream = as_stream(stream);
  const bool f32 = launch->element == QLLM_ELEMENT_F32;
  if (wide && f32)
    stream_norm_wide_kernel<float><<<launch->rows, threads, 0, hip_stream>>>(args);
  else if (wide)
    stream_norm_wide_kernel<uint16_t><<<launch->rows, threads, 0, hip_stream>>>(args);
  else if (f32)
    stream_norm_narrow_kernel<float><<<launch->rows, 256, 0, hip_stream>>>(args);
  else
    stream_norm_narrow_kernel<uint16_t><<<launch->rows, 256, 0, hip_stream>>>(args);
  return launched("stream norm");
}
