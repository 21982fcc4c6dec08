// Recurrent mixers with a matrix state per head: the generalised delta rule and
// the bonus recurrence (include/qllm_kernels.h has the equations).  State,
// decays, unit keys and rates are F32.
//
// The columns of a state (its value dimension) never meet: column j is a
// vector recurrence driven by the token's r, k, u, a u, w and the one number
// v_j.  The scan therefore gives sixteen lanes to a column - a lane holds
// KPL = dim / 16 of its rows in registers for the whole prompt, dot products
// end in four DPP rotations - and sixteen columns to a workgroup, so heads x
// dim / 16 workgroups walk the tokens side by side; the token vectors come
// through LDS in chunks of 4 KiB per vector, the next chunk's loads in flight
// meanwhile.  What depends on the token alone (unit keys, decays with their
// low-rank projection, rates) is prepared before, the output norm and gate
// follow after, both over all tokens at once.  One token (decode) is one
// launch that does all of it with a workgroup per head.
#include "mixed_common.hpp"

namespace qllm {
namespace {

struct RecurrenceArgs {
  qllm_recurrence layer;
  qllm_recurrence_launch launch;
  float* prepared;   // [head][row][slots][padded dim]
  float* scalars;    // BONUS: [head][row] sum of r * bonus * k
  float* outputs;    // [row][heads * dim]
  uint32_t padded;   // dim padded to 16, 32, 64, 128 or 256
};

__host__ __device__ constexpr uint32_t vectors_of(uint32_t kind) {
  return kind == QLLM_RECURRENCE_DELTA ? 5u : 3u;
}

uint32_t padded_dim(uint32_t dim) {
  uint32_t padded = 16u;
  while (padded < dim) padded *= 2u;
  return padded;
}

__device__ __forceinline__ float gate_value(uint32_t kind, float x) {
  return kind == QLLM_GATE_SILU ? x * sigmoid_f32(x) : sigmoid_f32(x);
}

__device__ __forceinline__ float decay_of(const qllm_recurrence& l, float inner) {
  return l.kind == QLLM_RECURRENCE_DELTA ? expf(l.decay_scale * sigmoid_f32(inner))
                                         : expf(-expf(inner));
}

__device__ __forceinline__ void copy_carry(const RecurrenceArgs& args) {
  const auto& run = args.launch;
  if (blockIdx.x != 0 || blockIdx.y != 0 || !run.carry_to) return;
  float* carry = run.carry_to + args.layer.step[kStepSlot] * args.layer.slot_stride;
  for (uint32_t c = threadIdx.x; c < run.carry_width; c += blockDim.x)
    carry[c] = run.carry_from[c];
}

// ---- one token -------------------------------------------------------------------

// KPT = state rows per thread: 1024 / dim groups of threads share the rows of a
// column.
template <typename T, int KPT>
__global__ __launch_bounds__(1024) void recurrence_step_kernel(RecurrenceArgs args) {
  __shared__ float r[256], k[256], u[256], au[256], w[256], low[256];
  __shared__ float part[1024];
  __shared__ float scratch[16];
  const qllm_recurrence& l = args.layer;
  const auto& run = args.launch;
  const uint32_t head = blockIdx.x;
  const uint32_t dim = l.dim;
  const uint32_t first = head * dim;
  const bool delta = l.kind == QLLM_RECURRENCE_DELTA;
  const float* p = run.projections;

  for (uint32_t j = threadIdx.x; j < l.rank; j += blockDim.x)
    low[j] = tanhf(p[run.low_column + j]);
  float key = 0.0f;
  float product = 0.0f;
  if (threadIdx.x < dim) {
    const uint32_t c = first + threadIdx.x;
    key = p[run.k_column + c];
    k[threadIdx.x] = key;
    const float read = p[run.r_column + c];
    r[threadIdx.x] = read;
    product = delta ? key * key : read * l.bonus[c] * key;
  }
  const float total = block_sum(product, scratch);   // synchronises
  // the low-rank products: 1024 / 256 = 4 threads per channel
  {
    const uint32_t channel = threadIdx.x / 4u;
    float inner = 0.0f;
    if (channel < dim) {
      const uint16_t* up = static_cast<const uint16_t*>(l.decay_up_bf16) +
                           size_t{first + channel} * l.rank;
      for (uint32_t j = threadIdx.x % 4u; j < l.rank; j += 4u)
        inner = fmaf(bf16_bits_to_f32(up[j]), low[j], inner);
    }
    inner += __shfl_xor(inner, 1, kWave);
    inner += __shfl_xor(inner, 2, kWave);
    if (channel < dim && threadIdx.x % 4u == 0u)
      w[channel] = decay_of(l, inner + l.decay_base[first + channel]);
  }
  if (delta && threadIdx.x < dim) {
    const uint32_t c = first + threadIdx.x;
    const float unit = key / sqrtf(total + l.unit_epsilon);
    u[threadIdx.x] = unit;
    au[threadIdx.x] = unit * sigmoid_f32(p[run.rate_column + c] + l.rate_bias[c]);
  }
  __syncthreads();

  const uint32_t groups = 1024u / dim;
  const uint32_t group = threadIdx.x / dim;
  const uint32_t column = threadIdx.x - group * dim;
  const bool active = group < groups;
  const uint32_t per_group = (dim + groups - 1u) / groups;
  const uint32_t row0 = group * per_group;
  const uint32_t rows = active && row0 < dim ? min(per_group, dim - row0) : 0u;
  float* state = l.state + l.step[kStepSlot] * l.slot_stride +
                 (size_t{head} * dim + row0) * dim + column;
  float s[KPT];
#pragma unroll
  for (int i = 0; i < KPT; ++i)
    s[i] = static_cast<uint32_t>(i) < rows ? state[size_t{static_cast<uint32_t>(i)} * dim] : 0.0f;
  const float value = active ? p[run.v_column + first + column] : 0.0f;

  const auto column_sum = [&](float mine) {
    part[threadIdx.x] = mine;
    __syncthreads();
    float sum = 0.0f;
    if (active)
      for (uint32_t g = 0; g < groups; ++g) sum += part[g * dim + column];
    __syncthreads();
    return sum;
  };
  float out = 0.0f;
  if (delta) {
    float dot = 0.0f;
#pragma unroll
    for (int i = 0; i < KPT; ++i)
      if (static_cast<uint32_t>(i) < rows) dot = fmaf(u[row0 + i], s[i], dot);
    dot = column_sum(dot);
    float read = 0.0f;
#pragma unroll
    for (int i = 0; i < KPT; ++i)
      if (static_cast<uint32_t>(i) < rows) {
        s[i] = fmaf(k[row0 + i], value, fmaf(-au[row0 + i], dot, w[row0 + i] * s[i]));
        read = fmaf(r[row0 + i], s[i], read);
      }
    out = column_sum(read);
  } else {
    float read = 0.0f;
#pragma unroll
    for (int i = 0; i < KPT; ++i)
      if (static_cast<uint32_t>(i) < rows) {
        read = fmaf(r[row0 + i], s[i], read);
        s[i] = fmaf(k[row0 + i], value, w[row0 + i] * s[i]);
      }
    out = fmaf(total, value, column_sum(read));
  }
#pragma unroll
  for (int i = 0; i < KPT; ++i)
    if (static_cast<uint32_t>(i) < rows) state[size_t{static_cast<uint32_t>(i)} * dim] = s[i];

  const bool owner = threadIdx.x < dim;
  const float squares = block_sum(owner ? out * out : 0.0f, scratch);
  if (owner) {
    const uint32_t c = first + threadIdx.x;
    const float unit = out / sqrtf(squares / static_cast<float>(dim) + l.epsilon);
    store_element(static_cast<T*>(run.output) + c,
                  unit * l.norm_weight[c] * gate_value(l.gate_kind, p[run.gate_column + c]));
  }
  copy_carry(args);
}

// ---- prompts ---------------------------------------------------------------------

constexpr uint32_t kPrepareRows = 8;

// Token vectors of kPrepareRows tokens of one head.
__global__ __launch_bounds__(256) void recurrence_prepare_kernel(RecurrenceArgs args) {
  __shared__ float low[kPrepareRows][256];
  __shared__ float products[kPrepareRows][256];
  __shared__ float sums[kPrepareRows];
  const qllm_recurrence& l = args.layer;
  const auto& run = args.launch;
  const uint32_t head = blockIdx.y;
  const uint32_t dim = l.dim;
  const uint32_t first = head * dim;
  const uint32_t row0 = blockIdx.x * kPrepareRows;
  const uint32_t rows = min(kPrepareRows, run.rows - row0);
  const bool delta = l.kind == QLLM_RECURRENCE_DELTA;

  for (uint32_t i = threadIdx.x; i < rows * l.rank; i += blockDim.x) {
    const uint32_t row = i / l.rank;
    const uint32_t j = i % l.rank;
    low[row][j] = tanhf(run.projections[size_t{row0 + row} * run.stride + run.low_column + j]);
  }
  for (uint32_t i = threadIdx.x; i < rows * dim; i += blockDim.x) {
    const uint32_t row = i / dim;
    const uint32_t c = i % dim;
    const float* p = run.projections + size_t{row0 + row} * run.stride;
    const float key = p[run.k_column + first + c];
    products[row][c] =
        delta ? key * key : p[run.r_column + first + c] * l.bonus[first + c] * key;
  }
  __syncthreads();
  for (uint32_t row = threadIdx.x / kWave; row < rows; row += blockDim.x / kWave) {
    float sum = 0.0f;
    for (uint32_t c = threadIdx.x % kWave; c < dim; c += kWave) sum += products[row][c];
    sum = wave_sum(sum);
    if (threadIdx.x % kWave == 0u) {
      sums[row] = sum;
      if (!delta) args.scalars[size_t{head} * run.rows + row0 + row] = sum;
    }
  }
  __syncthreads();

  const uint32_t padded = args.padded;
  const uint32_t vectors = vectors_of(l.kind);
  const uint32_t lanes = min(blockDim.x, padded);   // threads side by side on channels
  const uint32_t groups = blockDim.x / lanes;
  const uint32_t c = threadIdx.x % lanes;
  const uint32_t group = threadIdx.x / lanes;
  float inner[kPrepareRows] = {};
  if (c < dim) {
    const uint16_t* up =
        static_cast<const uint16_t*>(l.decay_up_bf16) + size_t{first + c} * l.rank;
    for (uint32_t j = 0; j < l.rank; ++j) {
      const float weight = bf16_bits_to_f32(up[j]);
#pragma unroll
      for (uint32_t i = 0; i < kPrepareRows; ++i)
        if (i * groups + group < rows)
          inner[i] = fmaf(weight, low[i * groups + group][j], inner[i]);
    }
  }
#pragma unroll
  for (uint32_t i = 0; i < kPrepareRows; ++i) {
    const uint32_t row = i * groups + group;
    if (row >= rows) break;
    float* out = args.prepared +
                 (size_t{head} * run.rows + row0 + row) * vectors * padded + c;
    const float* p = run.projections + size_t{row0 + row} * run.stride + first + c;
    const bool real = c < dim;
    const float key = real ? p[run.k_column] : 0.0f;
    out[0] = real ? p[run.r_column] : 0.0f;
    out[padded] = key;
    out[2u * padded] =
        real ? decay_of(l, inner[i] + l.decay_base[first + c]) : 0.0f;
    if (delta) {
      const float unit = key / sqrtf(sums[row] + l.unit_epsilon);
      out[3u * padded] = unit;
      out[4u * padded] =
          real ? unit * sigmoid_f32(p[run.rate_column] + l.rate_bias[first + c]) : 0.0f;
    }
  }
}

// Four waves, sixteen columns of one head; tokens in chunks of 1024 / padded.
template <bool DELTA, int KPL>
__global__ __launch_bounds__(256) void recurrence_scan_kernel(RecurrenceArgs args) {
  constexpr uint32_t kPadded = KPL * 16u;
  constexpr uint32_t kVectors = DELTA ? 5u : 3u;
  constexpr uint32_t kTokens = 1024u / kPadded;
  constexpr uint32_t kChunk = 1024u * kVectors;        // floats
  __shared__ float4 chunk[2][kChunk / 4u];
  __shared__ float values[2][kTokens][16];
  __shared__ float bonus[2][kTokens];
  const qllm_recurrence& l = args.layer;
  const auto& run = args.launch;
  const uint32_t head = blockIdx.y;
  const uint32_t dim = l.dim;
  const uint32_t part = threadIdx.x % 16u;             // rows part * KPL ..
  const uint32_t column = blockIdx.x * 16u + threadIdx.x / 16u;
  const bool real = column < dim;

  float* state = l.state + l.step[kStepSlot] * l.slot_stride + size_t{head} * dim * dim;
  float s[KPL];
#pragma unroll
  for (int i = 0; i < KPL; ++i) {
    const uint32_t row = part * KPL + i;
    s[i] = real && row < dim ? state[size_t{row} * dim + column] : 0.0f;
  }

  const float4* source = reinterpret_cast<const float4*>(
      args.prepared + size_t{head} * run.rows * kVectors * kPadded);
  const uint32_t all_pieces = run.rows * kVectors * kPadded / 4u;
  const uint32_t chunks = (run.rows + kTokens - 1u) / kTokens;
  float4 next[kVectors];
  float next_values[(kTokens * 16u + 255u) / 256u];
  float next_bonus = 0.0f;
  const auto fetch = [&](uint32_t which) {
#pragma unroll
    for (uint32_t i = 0; i < kVectors; ++i)
      next[i] = source[min(which * (kChunk / 4u) + i * 256u + threadIdx.x, all_pieces - 1u)];
#pragma unroll
    for (uint32_t i = 0; i < sizeof(next_values) / 4u; ++i) {
      const uint32_t index = i * 256u + threadIdx.x;
      const uint32_t row = min(which * kTokens + index / 16u, run.rows - 1u);
      const uint32_t c = min(blockIdx.x * 16u + index % 16u, dim - 1u);
      next_values[i] =
          run.projections[size_t{row} * run.stride + run.v_column + head * dim + c];
    }
    if (!DELTA)
      next_bonus = args.scalars[size_t{head} * run.rows +
                                min(which * kTokens + threadIdx.x % kTokens, run.rows - 1u)];
  };
  const auto publish = [&](uint32_t slot) {
#pragma unroll
    for (uint32_t i = 0; i < kVectors; ++i) chunk[slot][i * 256u + threadIdx.x] = next[i];
#pragma unroll
    for (uint32_t i = 0; i < sizeof(next_values) / 4u; ++i) {
      const uint32_t index = i * 256u + threadIdx.x;
      if (index < kTokens * 16u) values[slot][index / 16u][index % 16u] = next_values[i];
    }
    if (!DELTA && threadIdx.x < kTokens) bonus[slot][threadIdx.x] = next_bonus;
  };

  fetch(0u);
  publish(0u);
  __syncthreads();
  for (uint32_t which = 0; which < chunks; ++which) {
    const uint32_t slot = which & 1u;
    if (which + 1u < chunks) fetch(which + 1u);
    const uint32_t first_row = which * kTokens;
    const uint32_t tokens = min(kTokens, run.rows - first_row);
    const float* base = reinterpret_cast<const float*>(chunk[slot]) + part * KPL;
    float kept = 0.0f;
    for (uint32_t t = 0; t < tokens; ++t) {
      const float* at = base + t * kVectors * kPadded;
      float r[KPL], k[KPL], w[KPL];
#pragma unroll
      for (int i = 0; i < KPL; ++i) {
        r[i] = at[i];
        k[i] = at[kPadded + i];
        w[i] = at[2u * kPadded + i];
      }
      const float value = values[slot][t][threadIdx.x / 16u];
      float out;
      if constexpr (DELTA) {
        float u[KPL], au[KPL];
#pragma unroll
        for (int i = 0; i < KPL; ++i) {
          u[i] = at[3u * kPadded + i];
          au[i] = at[4u * kPadded + i];
        }
        float dot = u[0] * s[0];
#pragma unroll
        for (int i = 1; i < KPL; ++i) dot = fmaf(u[i], s[i], dot);
        // while the dot product travels: the part that does not need it
#pragma unroll
        for (int i = 0; i < KPL; ++i) s[i] = fmaf(k[i], value, w[i] * s[i]);
        dot = row16_sum(dot);
#pragma unroll
        for (int i = 0; i < KPL; ++i) s[i] = fmaf(-au[i], dot, s[i]);
        out = r[0] * s[0];
#pragma unroll
        for (int i = 1; i < KPL; ++i) out = fmaf(r[i], s[i], out);
        out = row16_sum(out);
      } else {
        out = r[0] * s[0];
#pragma unroll
        for (int i = 1; i < KPL; ++i) out = fmaf(r[i], s[i], out);
#pragma unroll
        for (int i = 0; i < KPL; ++i) s[i] = fmaf(k[i], value, w[i] * s[i]);
        out = fmaf(bonus[slot][t], value, row16_sum(out));
      }
      // every lane of the sixteen has the sum: lane t keeps token t's until
      // sixteen tokens are stored at once
      kept = t % 16u == part ? out : kept;
      if (t % 16u == 15u || t + 1u == tokens) {
        const uint32_t token = first_row + t / 16u * 16u + part;
        if (real && token < first_row + tokens)
          args.outputs[size_t{token} * l.heads * dim + head * dim + column] = kept;
      }
    }
    if (which + 1u < chunks) publish(1u - slot);
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < KPL; ++i) {
    const uint32_t row = part * KPL + i;
    if (real && row < dim) state[size_t{row} * dim + column] = s[i];
  }
  copy_carry(args);
}

// Output norm and gate: a wave per (token, head).
template <typename T>
__global__ __launch_bounds__(256) void recurrence_finish_kernel(RecurrenceArgs args) {
  const qllm_recurrence& l = args.layer;
  const auto& run = args.launch;
  const uint32_t item = blockIdx.x * 4u + threadIdx.x / kWave;
  if (item >= run.rows * l.heads) return;
  const uint32_t row = item / l.heads;
  const uint32_t first = item % l.heads * l.dim;
  const uint32_t lane = threadIdx.x % kWave;
  const float* o = args.outputs + size_t{row} * l.heads * l.dim + first;
  float held[4];
  float squares = 0.0f;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const uint32_t c = lane + i * kWave;
    held[i] = c < l.dim ? o[c] : 0.0f;
    squares = fmaf(held[i], held[i], squares);
  }
  squares = wave_sum(squares);
  const float inverse = 1.0f / sqrtf(squares / static_cast<float>(l.dim) + l.epsilon);
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const uint32_t c = lane + i * kWave;
    if (c >= l.dim) continue;
    const float gate = run.projections[size_t{row} * run.stride + run.gate_column + first + c];
    store_element(static_cast<T*>(run.output) + size_t{row} * run.output_stride + first + c,
                  held[i] * inverse * l.norm_weight[first + c] *
                      gate_value(l.gate_kind, gate));
  }
}

template <bool DELTA>
void launch_scan(const RecurrenceArgs& args, hipStream_t stream) {
  const dim3 grid((args.layer.dim + 15u) / 16u, args.layer.heads);
  switch (args.padded) {
    case 16u: recurrence_scan_kernel<DELTA, 1><<<grid, 256, 0, stream>>>(args); break;
    case 32u: recurrence_scan_kernel<DELTA, 2><<<grid, 256, 0, stream>>>(args); break;
    case 64u: recurrence_scan_kernel<DELTA, 4><<<grid, 256, 0, stream>>>(args); break;
    case 128u: recurrence_scan_kernel<DELTA, 8><<<grid, 256, 0, stream>>>(args); break;
    default: recurrence_scan_kernel<DELTA, 16><<<grid, 256, 0, stream>>>(args); break;
  }
}

template <typename T>
void launch_step(const RecurrenceArgs& args, hipStream_t stream) {
  const uint32_t groups = 1024u / args.layer.dim;
  const uint32_t per_group = (args.layer.dim + groups - 1u) / groups;
  if (per_group <= 4u)
    recurrence_step_kernel<T, 4><<<args.layer.heads, 1024, 0, stream>>>(args);
  else if (per_group <= 16u)
    recurrence_step_kernel<T, 16><<<args.layer.heads, 1024, 0, stream>>>(args);
  else
    recurrence_step_kernel<T, 64><<<args.layer.heads, 1024, 0, stream>>>(args);
}

size_t prepared_bytes(const qllm_recurrence& l, uint32_t rows) {
  return size_t{l.heads} * rows * vectors_of(l.kind) * padded_dim(l.dim) * 4u;
}

size_t scalar_bytes(const qllm_recurrence& l, uint32_t rows) {
  return (size_t{l.heads} * rows * 4u + 15u) / 16u * 16u;
}

}  // namespace
}  // namespace qllm

using namespace qllm;

extern "C" size_t qllm_recurrence_workspace_bytes(const qllm_recurrence* recurrence,
                                                  uint32_t rows) {
  if (!recurrence || rows <= 1u) return 0u;
  return prepared_bytes(*recurrence, rows) + scalar_bytes(*recurrence, rows) +
         size_t{rows} * recurrence->heads * recurrence->dim * 4u;
}

extern "C" int32_t qllm_recurrence_rows(const qllm_recurrence* recurrence,
                                        const qllm_recurrence_launch* launch,
                                        void* stream) {
  if (!recurrence || !launch) return fail(QLLM_INVALID_ARGUMENT, "invalid recurrence");
  const qllm_recurrence& l = *recurrence;
  const bool delta = l.kind == QLLM_RECURRENCE_DELTA;
  if (l.kind > QLLM_RECURRENCE_BONUS || !l.heads || !l.dim || l.dim > 256u || !l.rank ||
      l.rank > 256u || l.gate_kind > QLLM_GATE_SILU || l.element > QLLM_ELEMENT_F32 ||
      !l.decay_up_bf16 || !l.decay_base || !l.norm_weight || !l.state || !l.step ||
      (delta ? !l.rate_bias : !l.bonus) || !launch->projections || !launch->output ||
      !launch->rows || launch->output_stride < l.heads * l.dim ||
      (launch->carry_to && (!launch->carry_from || !launch->carry_width)))
    return fail(QLLM_INVALID_ARGUMENT, "invalid recurrence");
  for (const uint32_t column : {launch->r_column, launch->k_column, launch->v_column,
                                launch->gate_column, delta ? launch->rate_column : 0u})
    if (column + l.heads * l.dim > launch->stride)
      return fail(QLLM_INVALID_ARGUMENT, "recurrence columns exceed the projection rows");
  if (launch->low_column + l.rank > launch->stride)
    return fail(QLLM_INVALID_ARGUMENT, "recurrence columns exceed the projection rows");
  const auto hip_stream = as_stream(stream);
  RecurrenceArgs args{l, *launch, nullptr, nullptr, nullptr, padded_dim(l.dim)};
  const bool f32 = l.element == QLLM_ELEMENT_F32;
  if (launch->rows == 1u) {
    if (f32)
      launch_step<float>(args, hip_stream);
    else
      launch_step<uint16_t>(args, hip_stream);
    return launched("recurrence step");
  }
  if (!launch->workspace ||
      (reinterpret_cast<uintptr_t>(launch->workspace) & 15u) != 0u ||
      launch->workspace_bytes < qllm_recurrence_workspace_bytes(recurrence, launch->rows))
    return fail(QLLM_INVALID_ARGUMENT, "recurrence workspace is too small");
  auto* bytes = static_cast<uint8_t*>(launch->workspace);
  args.prepared = reinterpret_cast<float*>(bytes);
  args.scalars = reinterpret_cast<float*>(bytes + prepared_bytes(l, launch->rows));
  args.outputs = reinterpret_cast<float*>(bytes + prepared_bytes(l, launch->rows) +
                                          scalar_bytes(l, launch->rows));
  recurrence_prepare_kernel<<<dim3((launch->rows + kPrepareRows - 1u) / kPrepareRows,
                                   l.heads),
                              256, 0, hip_stream>>>(args);
  if (delta)
    launch_scan<true>(args, hip_stream);
  else
    launch_scan<false>(args, hip_stream);
  const uint32_t blocks = (launch->rows * l.heads + 3u) / 4u;
  if (f32)
    recurrence_finish_kernel<float><<<blocks, 256, 0, hip_stream>>>(args);
  else
    recurrence_finish_kernel<uint16_t><<<blocks, 256, 0, hip_stream>>>(args);
  return launched("recurrence");
}
