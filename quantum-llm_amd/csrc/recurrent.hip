// Recurrent mixers with a matrix state per head: the generalised delta rule, the
// bonus recurrence and gated linear attention (include/qllm_kernels.h has the
// equations).  State,
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
//
// Where the state only decays by rows and takes up outer products (bonus, gated),
// prompts go through F32 matrix products in chunks of sixteen tokens instead.  With
// D(j, i) the product of the decays of tokens j + 1 .. i, a chunk that starts from S
// has the outputs
//   o_i = (r_i * D(start, i))^T S + sum over j <= i of (r_i . (k_j * D(j, i))) v_j
// and leaves D(start, end) S + sum of (k_j * D(j, end)) v_j^T.  The decays are
// multiplied up pair by pair and none divides, so no product exceeds one: nothing
// overflows, and what underflows is gone token by token as well.  The chunks' own
// matrices are made for all chunks at once; a wave then walks them with sixteen
// columns of the state in its accumulators, which stand as the next product's
// operand as they are.  Long prompts are cut into segments walked side by side:
// once for the states they add, which are then joined, and once for the outputs.
#include "mixed_common.hpp"

namespace qllm {
namespace {

struct RecurrenceArgs {
  qllm_recurrence layer;
  qllm_recurrence_launch launch;
  float* prepared;   // [head][row][slots][padded dim]
  float* scalars;    // BONUS: [head][row] sum of r * bonus * k
  float* outputs;    // [row][heads * vdim]
  // chunks of sixteen tokens:
  float* chunks;     // [head][chunk]: chunk_floats(padded)
  float* starts;     // [segment][head][dim][vdim]
  float* totals;     // [segment][head][padded dim]: all decays of the segment
  uint32_t chunk_count;      // of a head
  uint32_t segments;
  uint32_t segment_chunks;
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
  if (l.kind == QLLM_RECURRENCE_DELTA) return expf(l.decay_scale * sigmoid_f32(inner));
  if (l.kind == QLLM_RECURRENCE_BONUS) return expf(-expf(inner));
  // a power of the sigmoid, through its logarithm
  return expf(l.decay_scale * (fminf(inner, 0.0f) - log1pf(expf(-fabsf(inner)))));
}

// What the decay's low-rank product takes of its projection.
__device__ __forceinline__ float low_value(const qllm_recurrence& l, float x) {
  return l.kind == QLLM_RECURRENCE_GATED ? x : tanhf(x);
}

__device__ __forceinline__ void copy_carry(const RecurrenceArgs& args) {
  const auto& run = args.launch;
  if (blockIdx.x != 0 || blockIdx.y != 0 || blockIdx.z != 0 || !run.carry_to) return;
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

  // everything that depends on nothing is on its way before the first barrier
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

  const bool owner = threadIdx.x < dim;
  float base = 0.0f;
  float rate = 0.0f;
  float gate = 0.0f;
  float weight = 0.0f;
  if (owner) {
    const uint32_t c = first + threadIdx.x;
    base = l.decay_base[c];
    gate = p[run.gate_column + c];
    weight = l.norm_weight[c];
    if (delta) rate = p[run.rate_column + c] + l.rate_bias[c];
  }

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
#pragma unroll 8
      for (uint32_t j = threadIdx.x % 4u; j < l.rank; j += 4u)
        inner = fmaf(bf16_bits_to_f32(up[j]), low[j], inner);
    }
    inner += __shfl_xor(inner, 1, kWave);
    inner += __shfl_xor(inner, 2, kWave);
    if (channel < dim && threadIdx.x % 4u == 0u) w[channel] = inner;
  }
  if (delta && owner) {
    const float unit = key / sqrtf(total + l.unit_epsilon);
    u[threadIdx.x] = unit;
    au[threadIdx.x] = unit * sigmoid_f32(rate);
  }
  __syncthreads();
  if (owner) w[threadIdx.x] = decay_of(l, w[threadIdx.x] + base);
  __syncthreads();

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

  const float squares = block_sum(owner ? out * out : 0.0f, scratch);
  if (owner) {
    const float unit = out / sqrtf(squares / static_cast<float>(dim) + l.epsilon);
    store_element(static_cast<T*>(run.output) + first + threadIdx.x,
                  unit * weight * gate_value(l.gate_kind, gate));
  }
  copy_carry(args);
}

// The same for gated linear attention, whose state may have more columns than
// rows: a row group of threads per `vdim` columns, rows dealt in turn.  KPT = 0
// streams the state instead of holding it.
template <typename T, int KPT>
__global__ __launch_bounds__(1024) void gated_step_kernel(RecurrenceArgs args) {
  __shared__ float r[256], k[256], w[256], low[256];
  __shared__ float part[1024];
  __shared__ float scratch[16];
  const qllm_recurrence& l = args.layer;
  const auto& run = args.launch;
  const uint32_t head = blockIdx.x;
  const uint32_t dim = l.dim;
  const uint32_t vdim = l.vdim;
  const float* p = run.projections;
  const uint32_t groups = 1024u / vdim;
  const uint32_t group = threadIdx.x / vdim;
  const uint32_t column = threadIdx.x - group * vdim;
  const bool active = group < groups;
  float* state = l.state + l.step[kStepSlot] * l.slot_stride + size_t{head} * dim * vdim +
                 column;
  constexpr int kHeld = KPT ? KPT : 1;
  float s[kHeld];
#pragma unroll
  for (int i = 0; i < KPT; ++i) {
    const uint32_t row = group + groups * i;
    s[i] = active && row < dim ? state[size_t{row} * vdim] : 0.0f;
  }
  const float value = active ? p[run.v_column + head * vdim + column] : 0.0f;
  const bool owner = threadIdx.x < vdim;
  const float gate = owner ? p[run.gate_column + head * vdim + threadIdx.x] : 0.0f;
  const float weight = owner ? l.norm_weight[threadIdx.x] : 0.0f;
  for (uint32_t j = threadIdx.x; j < l.rank; j += blockDim.x)
    low[j] = low_value(l, p[run.low_column + j]);
  if (threadIdx.x < dim) {
    r[threadIdx.x] = p[run.r_column + head * dim + threadIdx.x] * l.read_scale;
    k[threadIdx.x] = p[run.k_column + head * dim + threadIdx.x];
  }
  __syncthreads();
  // the low-rank products: 1024 / 256 = 4 threads per channel
  const uint32_t channel = threadIdx.x / 4u;
  float inner = 0.0f;
  if (channel < dim) {
    const uint16_t* up = static_cast<const uint16_t*>(l.decay_up_bf16) +
                         (size_t{head} * dim + channel) * l.rank;
#pragma unroll 8
    for (uint32_t j = threadIdx.x % 4u; j < l.rank; j += 4u)
      inner = fmaf(bf16_bits_to_f32(up[j]), low[j], inner);
  }
  inner += __shfl_xor(inner, 1, kWave);
  inner += __shfl_xor(inner, 2, kWave);
  if (channel < dim && threadIdx.x % 4u == 0u)
    w[channel] = decay_of(l, inner + l.decay_base[head * dim + channel]);
  __syncthreads();
  float read = 0.0f;
  if constexpr (KPT) {
#pragma unroll
    for (int i = 0; i < KPT; ++i) {
      const uint32_t row = group + groups * i;
      if (!active || row >= dim) continue;
      s[i] = fmaf(k[row], value, w[row] * s[i]);
      read = fmaf(r[row], s[i], read);
      state[size_t{row} * vdim] = s[i];
    }
  } else if (active) {
#pragma unroll 8
    for (uint32_t row = group; row < dim; row += groups) {
      const float fresh = fmaf(k[row], value, w[row] * state[size_t{row} * vdim]);
      read = fmaf(r[row], fresh, read);
      state[size_t{row} * vdim] = fresh;
    }
  }
  part[threadIdx.x] = read;
  __syncthreads();
  float out = 0.0f;
  if (owner)
    for (uint32_t g = 0; g < groups; ++g) out += part[g * vdim + threadIdx.x];
  const float squares = block_sum(owner ? out * out : 0.0f, scratch);
  if (owner)
    store_element(static_cast<T*>(run.output) + head * vdim + threadIdx.x,
                  out / sqrtf(squares / static_cast<float>(vdim) + l.epsilon) * weight *
                      gate_value(l.gate_kind, gate));
  copy_carry(args);
}

// ---- prompts ---------------------------------------------------------------------

constexpr uint32_t kRowsPerThread = 8;    // tokens a thread prepares
constexpr uint32_t kRankChunk = 32;

// Token vectors of one head.  Threads lie side by side on channels, in groups
// of kRowsPerThread tokens each; the low-rank product runs over LDS tiles of
// kRankChunk columns.
__global__ __launch_bounds__(256) void recurrence_prepare_kernel(RecurrenceArgs args) {
  constexpr uint32_t kMostRows = 256u / 16u * kRowsPerThread;
  __shared__ float up_tile[kRankChunk][257];
  __shared__ __attribute__((aligned(16))) float low_tile[kMostRows][kRankChunk];
  __shared__ float sums[kMostRows][4];
  const qllm_recurrence& l = args.layer;
  const auto& run = args.launch;
  const uint32_t head = blockIdx.y;
  const uint32_t dim = l.dim;
  const uint32_t first = head * dim;
  const uint32_t padded = args.padded;
  const uint32_t groups = 256u / padded;
  const uint32_t block_rows = groups * kRowsPerThread;
  const uint32_t row0 = blockIdx.x * block_rows;
  const uint32_t rows = min(block_rows, run.rows - row0);
  const bool delta = l.kind == QLLM_RECURRENCE_DELTA;
  const bool gated = l.kind == QLLM_RECURRENCE_GATED;
  const float* block_projections = run.projections + size_t{row0} * run.stride;
  const uint32_t c = threadIdx.x % padded;
  const uint32_t group = threadIdx.x / padded;
  const bool real = c < dim;
  const uint32_t channel = first + min(c, dim - 1u);

  // this thread's tokens: all loads in flight together
  float key[kRowsPerThread], read[kRowsPerThread], rate[kRowsPerThread];
#pragma unroll
  for (uint32_t i = 0; i < kRowsPerThread; ++i) {
    const float* p = block_projections +
                     size_t{min(group * kRowsPerThread + i, rows - 1u)} * run.stride + channel;
    key[i] = p[run.k_column];
    read[i] = gated ? p[run.r_column] * l.read_scale : p[run.r_column];
    rate[i] = delta ? p[run.rate_column] : 0.0f;
  }
  // per token: sum of k^2, or of r * bonus * k
  const float bonus = delta || gated || !real ? 0.0f : l.bonus[channel];
#pragma unroll
  for (uint32_t i = 0; i < kRowsPerThread; ++i) {
    key[i] = real ? key[i] : 0.0f;
    read[i] = real ? read[i] : 0.0f;
    float sum = delta ? key[i] * key[i] : read[i] * bonus * key[i];
    sum = row16_sum(sum);
    for (uint32_t offset = 16u; offset < min(padded, 64u); offset *= 2u)
      sum += __shfl_xor(sum, static_cast<int>(offset), kWave);
    if (c % 64u == 0u) sums[group * kRowsPerThread + i][c / 64u] = sum;
  }

  float inner[kRowsPerThread] = {};
  for (uint32_t j0 = 0; j0 < l.rank; j0 += kRankChunk) {
    __syncthreads();
#pragma unroll 8
    for (uint32_t i = threadIdx.x; i < padded * kRankChunk; i += 256u) {
      const uint32_t at = i / kRankChunk;
      const uint32_t j = i % kRankChunk;
      const float weight = bf16_bits_to_f32(static_cast<const uint16_t*>(
          l.decay_up_bf16)[size_t{first + min(at, dim - 1u)} * l.rank +
                           min(j0 + j, l.rank - 1u)]);
      up_tile[j][at] = j0 + j < l.rank ? weight : 0.0f;
    }
#pragma unroll 4
    for (uint32_t i = threadIdx.x; i < block_rows * kRankChunk; i += 256u) {
      const uint32_t row = i / kRankChunk;
      const uint32_t j = i % kRankChunk;
      const float value =
          low_value(l, block_projections[size_t{min(row, rows - 1u)} * run.stride +
                                         run.low_column + min(j0 + j, l.rank - 1u)]);
      low_tile[row][j] = j0 + j < l.rank ? value : 0.0f;
    }
    __syncthreads();
#pragma unroll 2
    for (uint32_t j = 0; j < kRankChunk; j += 4u) {
      float weight[4];
#pragma unroll
      for (uint32_t e = 0; e < 4u; ++e) weight[e] = up_tile[j + e][c];
#pragma unroll
      for (uint32_t i = 0; i < kRowsPerThread; ++i) {
        const f32x4 low =
            *reinterpret_cast<const f32x4*>(&low_tile[group * kRowsPerThread + i][j]);
#pragma unroll
        for (uint32_t e = 0; e < 4u; ++e) inner[i] = fmaf(weight[e], low[e], inner[i]);
      }
    }
  }

  const uint32_t vectors = vectors_of(l.kind);
  const float base = real ? l.decay_base[channel] : 0.0f;
  const float bias = real && delta ? l.rate_bias[channel] : 0.0f;
#pragma unroll
  for (uint32_t i = 0; i < kRowsPerThread; ++i) {
    const uint32_t row = group * kRowsPerThread + i;
    if (row >= rows) break;
    float sum = sums[row][0];
    for (uint32_t wave = 1; wave < padded / 64u; ++wave) sum += sums[row][wave];
    if (!delta && c == 0u) args.scalars[size_t{head} * run.rows + row0 + row] = sum;
    float* out = args.prepared +
                 (size_t{head} * run.rows + row0 + row) * vectors * padded + c;
    out[0] = read[i];
    out[padded] = key[i];
    out[2u * padded] = real ? decay_of(l, inner[i] + base) : 0.0f;
    if (delta) {
      const float unit = key[i] / sqrtf(sum + l.unit_epsilon);
      out[3u * padded] = unit;
      out[4u * padded] = real ? unit * sigmoid_f32(rate[i] + bias) : 0.0f;
    }
  }
}

// Four waves, sixteen columns of one head; tokens in chunks of 1024 / padded.
template <uint32_t KIND, int KPL>
__global__ __launch_bounds__(256) void recurrence_scan_kernel(RecurrenceArgs args) {
  constexpr bool DELTA = KIND == QLLM_RECURRENCE_DELTA;
  constexpr bool BONUS = KIND == QLLM_RECURRENCE_BONUS;
  constexpr uint32_t kPadded = KPL * 16u;
  constexpr uint32_t kVectors = vectors_of(KIND);
  constexpr uint32_t kTokens = 1024u / kPadded;
  constexpr uint32_t kChunk = 1024u * kVectors;        // floats
  __shared__ f32x4 chunk[2][kChunk / 4u];
  __shared__ float values[2][kTokens][16];
  __shared__ float bonus[2][kTokens];
  const qllm_recurrence& l = args.layer;
  const auto& run = args.launch;
  const uint32_t head = blockIdx.y;
  const uint32_t dim = l.dim;
  const uint32_t vdim = l.vdim;
  const uint32_t part = threadIdx.x % 16u;             // rows part * KPL ..
  const uint32_t column = blockIdx.x * 16u + threadIdx.x / 16u;
  const bool real = column < vdim;

  float* state = l.state + l.step[kStepSlot] * l.slot_stride + size_t{head} * dim * vdim;
  float s[KPL];
#pragma unroll
  for (int i = 0; i < KPL; ++i) {
    const uint32_t row = part * KPL + i;
    s[i] = real && row < dim ? state[size_t{row} * vdim + column] : 0.0f;
  }

  const f32x4* source = reinterpret_cast<const f32x4*>(
      args.prepared + size_t{head} * run.rows * kVectors * kPadded);
  const uint32_t all_pieces = run.rows * kVectors * kPadded / 4u;
  const uint32_t chunks = (run.rows + kTokens - 1u) / kTokens;
  constexpr uint32_t kValueLoads = (kTokens * 16u + 255u) / 256u;
  f32x4 next[kVectors];
  float next_values[kValueLoads];
  float next_bonus = 0.0f;
  // Loads of a chunk, and their way into LDS.
  const auto fetch = [&](uint32_t which) __attribute__((always_inline)) {
#pragma unroll
    for (uint32_t i = 0; i < kVectors; ++i)
      next[i] = source[min(which * (kChunk / 4u) + i * 256u + threadIdx.x, all_pieces - 1u)];
#pragma unroll
    for (uint32_t i = 0; i < kValueLoads; ++i) {
      const uint32_t index = i * 256u + threadIdx.x;
      const uint32_t row = min(which * kTokens + index / 16u, run.rows - 1u);
      const uint32_t c = min(blockIdx.x * 16u + index % 16u, vdim - 1u);
      next_values[i] =
          run.projections[size_t{row} * run.stride + run.v_column + head * vdim + c];
    }
    if (BONUS)
      next_bonus = args.scalars[size_t{head} * run.rows +
                                min(which * kTokens + threadIdx.x % kTokens, run.rows - 1u)];
  };
  const auto publish = [&](uint32_t slot, uint32_t which) __attribute__((always_inline)) {
#pragma unroll
    for (uint32_t i = 0; i < kVectors; ++i) {
      // tokens past the last one: decays of 1 and zeros, which change nothing
      const uint32_t in_chunk = i * 256u + threadIdx.x;
      const float idle = in_chunk / (kPadded / 4u) % kVectors == 2u ? 1.0f : 0.0f;
      const bool there = which * (kChunk / 4u) + in_chunk < all_pieces;
      f32x4 piece;
#pragma unroll
      for (int e = 0; e < 4; ++e) piece[e] = there ? next[i][e] : idle;
      chunk[slot][in_chunk] = piece;
    }
#pragma unroll
    for (uint32_t i = 0; i < kValueLoads; ++i) {
      const uint32_t index = i * 256u + threadIdx.x;
      if (index < kTokens * 16u) values[slot][index / 16u][index % 16u] = next_values[i];
    }
    if (BONUS && threadIdx.x < kTokens) bonus[slot][threadIdx.x] = next_bonus;
  };

  // What a token brings to this lane, read from LDS one token ahead of its use.
  struct Token {
    float vector[kVectors][KPL];
    float value;
  };
  const auto read = [&](Token& token, uint32_t slot, uint32_t t)
      __attribute__((always_inline)) {
    constexpr int kAlignment = KPL >= 4 ? 16 : KPL * 4;
    const float* at = static_cast<const float*>(__builtin_assume_aligned(
        reinterpret_cast<const float*>(chunk[slot]) + t * kVectors * kPadded + part * KPL,
        kAlignment));
#pragma unroll
    for (uint32_t v = 0; v < kVectors; ++v)
#pragma unroll
      for (int i = 0; i < KPL; ++i) token.vector[v][i] = at[v * kPadded + i];
    token.value = values[slot][t][threadIdx.x / 16u];
  };
  const auto dot_with = [&](const float (&vector)[KPL]) __attribute__((always_inline)) {
    float even = vector[0] * s[0];
    float odd = 0.0f;
#pragma unroll
    for (int i = 1; i < KPL; ++i)
      if (i % 2 == 1)
        odd = i == 1 ? vector[i] * s[i] : fmaf(vector[i], s[i], odd);
      else
        even = fmaf(vector[i], s[i], even);
    return even + odd;
  };
  // Moves the state past a token; returns this lane's part of the output.
  const auto advance = [&](const Token& token) __attribute__((always_inline)) {
    const auto& r = token.vector[0];
    const auto& k = token.vector[1];
    const auto& w = token.vector[2];
    if constexpr (DELTA) {
      const auto& u = token.vector[3];
      const auto& au = token.vector[4];
      float dot = dot_with(u);
      // while the dot product travels: the part that does not need it
#pragma unroll
      for (int i = 0; i < KPL; ++i) s[i] = fmaf(k[i], token.value, w[i] * s[i]);
      dot = row16_sum(dot);
#pragma unroll
      for (int i = 0; i < KPL; ++i) s[i] = fmaf(-au[i], dot, s[i]);
      return dot_with(r);
    } else if constexpr (BONUS) {
      const float out = dot_with(r);
#pragma unroll
      for (int i = 0; i < KPL; ++i) s[i] = fmaf(k[i], token.value, w[i] * s[i]);
      return out;
    } else {
#pragma unroll
      for (int i = 0; i < KPL; ++i) s[i] = fmaf(k[i], token.value, w[i] * s[i]);
      return dot_with(r);
    }
  };

  fetch(0u);
  publish(0u, 0u);
  __syncthreads();
  // a block of tokens' outputs is summed over the lanes at once: lane t of a
  // column ends with token t's
  constexpr uint32_t kBlock = kTokens < 16u ? kTokens : 16u;
  for (uint32_t which = 0; which < chunks; ++which) {
    const uint32_t slot = which & 1u;
    fetch(min(which + 1u, chunks - 1u));
    for (uint32_t first = 0; first < kTokens; first += kBlock) {
      float parts[16] = {};
      Token token[2];
      read(token[0], slot, first);
#pragma unroll
      for (uint32_t t = 0; t < kBlock; ++t) {
        if (t + 1u < kBlock) read(token[(t + 1u) % 2u], slot, first + t + 1u);
        parts[t] = advance(token[t % 2u]);
      }
      float out = row16_transposed_sum(parts);
      const uint32_t mine = first + part;
      if (BONUS && part < kBlock)
        out = fmaf(bonus[slot][mine], values[slot][mine][threadIdx.x / 16u], out);
      const uint32_t row = which * kTokens + mine;
      if (real && part < kBlock && row < run.rows)
        args.outputs[size_t{row} * l.heads * vdim + head * vdim + column] = out;
    }
    publish(1u - slot, which + 1u);
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < KPL; ++i) {
    const uint32_t row = part * KPL + i;
    if (real && row < dim) state[size_t{row} * vdim + column] = s[i];
  }
  copy_carry(args);
}

// ---- prompts in chunks of sixteen tokens ---------------------------------------

constexpr uint32_t kChunk = 16;
constexpr uint32_t kMaximumSegments = 16;

// A chunk's matrices: reads times the decays so far [token][padded], keys times the
// decays to come, transposed [padded][token], weights [token][earlier token], all
// decays [padded].
__host__ __device__ constexpr uint32_t chunk_floats(uint32_t padded) {
  return 2u * kChunk * padded + kChunk * kChunk + padded;
}

// Sixteen lanes per token j of a chunk, KPL channels each.
template <uint32_t KIND, int KPL>
__global__ __launch_bounds__(256) void recurrence_chunk_kernel(RecurrenceArgs args) {
  constexpr bool BONUS = KIND == QLLM_RECURRENCE_BONUS;
  constexpr uint32_t kPadded = KPL * 16u;
  constexpr uint32_t kVectors = vectors_of(KIND);
  __shared__ float reads[kChunk][kPadded];
  __shared__ float decays[kChunk][kPadded];
  const auto& run = args.launch;
  const uint32_t head = blockIdx.y;
  const uint32_t j = threadIdx.x / 16u;
  const uint32_t part = threadIdx.x % 16u;
  const uint32_t row = blockIdx.x * kChunk + j;
  const bool there = row < run.rows;
  const float* source =
      args.prepared + (size_t{head} * run.rows + min(row, run.rows - 1u)) * kVectors * kPadded +
      part * KPL;
  float read[KPL], key[KPL];
#pragma unroll
  for (int i = 0; i < KPL; ++i) {
    // tokens past the last one: decays of 1 and zeros, which change nothing
    read[i] = there ? source[i] : 0.0f;
    key[i] = there ? source[kPadded + i] : 0.0f;
    reads[j][part * KPL + i] = read[i];
    decays[j][part * KPL + i] = there ? source[2u * kPadded + i] : 1.0f;
  }
  const float own = BONUS && there ? args.scalars[size_t{head} * run.rows + row] : 0.0f;
  __syncthreads();
  float weight[kChunk];
  float all[KPL];
#pragma unroll
  for (int i = 0; i < KPL; ++i) all[i] = 1.0f;
#pragma unroll
  for (uint32_t t = 0; t < kChunk; ++t) {
    // BONUS reads before token t's decay, GATED after it
    float dot = 0.0f;
#pragma unroll
    for (int i = 0; i < KPL; ++i) {
      const float decay = decays[t][part * KPL + i];
      const float faded = t > j ? key[i] * decay : key[i];
      dot = fmaf(reads[t][part * KPL + i], BONUS ? key[i] : faded, dot);
      key[i] = faded;
      read[i] *= BONUS ? (t < j ? decay : 1.0f) : (t <= j ? decay : 1.0f);
      all[i] *= decay;
    }
    weight[t] = (BONUS ? t > j : t >= j) ? dot : 0.0f;
  }
  // lane t of token j: what output t takes of value j
  float mine = row16_transposed_sum(weight);
  if (BONUS && part == j) mine = own;
  float* out = args.chunks +
               (size_t{head} * args.chunk_count + blockIdx.x) * chunk_floats(kPadded);
  float* transposed = out + kChunk * kPadded;
#pragma unroll
  for (int i = 0; i < KPL; ++i) {
    out[j * kPadded + part * KPL + i] = read[i];
    transposed[(part * KPL + i) * kChunk + j] = key[i];
    if (j == 0u) transposed[kChunk * kPadded + kChunk * kChunk + part * KPL + i] = all[i];
  }
  transposed[kChunk * kPadded + part * kChunk + j] = mine;
}

// A wave per sixteen columns of one head's state, TILES = padded dim / 16.  With
// OUTPUTS the segment's outputs from its starting state; without, the state it ends
// with when it starts from zero (the first one: from the request's).
template <bool OUTPUTS, int TILES>
__global__ __launch_bounds__(256, 1) void recurrence_walk_kernel(RecurrenceArgs args) {
  constexpr uint32_t kPadded = TILES * 16u;
  constexpr uint32_t kPieces = chunk_floats(kPadded) / 4u;
  const qllm_recurrence& l = args.layer;
  const auto& run = args.launch;
  const uint32_t head = blockIdx.y;
  const uint32_t segment = blockIdx.z;
  const uint32_t dim = l.dim;
  const uint32_t vdim = l.vdim;
  const uint32_t lane = threadIdx.x % kWave;
  const uint32_t quarter = lane / 16u;
  const uint32_t first_column = (blockIdx.x * 4u + threadIdx.x / kWave) * 16u;
  const uint32_t column = first_column + lane % 16u;
  const bool real = column < vdim;
  if (OUTPUTS) copy_carry(args);
  if (first_column >= vdim) return;

  const bool several = args.segments > 1u;
  float* const request =
      l.state + l.step[kStepSlot] * l.slot_stride + size_t{head} * dim * vdim;
  float* const kept = args.starts + (size_t{segment} * l.heads + head) * dim * vdim;
  const float* const from = OUTPUTS && several ? kept : request;
  f32x4 state[TILES];
#pragma unroll
  for (int d = 0; d < TILES; ++d)
#pragma unroll
    for (uint32_t i = 0; i < 4u; ++i) {
      const uint32_t row = d * 16u + 4u * quarter + i;
      state[d][i] = real && row < dim && (OUTPUTS || segment == 0u)
                        ? from[size_t{row} * vdim + column]
                        : 0.0f;
    }
  f32x4 faded[TILES];
#pragma unroll
  for (int d = 0; d < TILES; ++d) faded[d] = f32x4{1.0f, 1.0f, 1.0f, 1.0f};

  struct Chunk {
    f32x4 reads[OUTPUTS ? TILES : 1];
    f32x4 keys[TILES];
    f32x4 weights;
    f32x4 decays[TILES];
    float values[4];
  };
  const f32x4* const source =
      reinterpret_cast<const f32x4*>(args.chunks) + size_t{head} * args.chunk_count * kPieces;
  const float* const value_column = run.projections + run.v_column + head * vdim +
                                    min(column, vdim - 1u);
  const auto fetch = [&](Chunk& c, uint32_t which) __attribute__((always_inline)) {
    const f32x4* at = source + size_t{which} * kPieces;
    if constexpr (OUTPUTS) {
#pragma unroll
      for (int d = 0; d < TILES; ++d)
        c.reads[d] = at[(lane % 16u) * (kPadded / 4u) + d * 4u + quarter];
      c.weights = at[2u * kChunk * kPadded / 4u + lane % 16u * (kChunk / 4u) + quarter];
    }
#pragma unroll
    for (int d = 0; d < TILES; ++d) {
      c.keys[d] = at[kChunk * kPadded / 4u + (d * 16u + lane % 16u) * (kChunk / 4u) + quarter];
      c.decays[d] = at[(2u * kChunk * kPadded + kChunk * kChunk) / 4u + d * 4u + quarter];
    }
#pragma unroll
    for (uint32_t e = 0; e < 4u; ++e) {
      const uint32_t row = min(which * kChunk + 4u * quarter + e, run.rows - 1u);
      c.values[e] = value_column[size_t{row} * run.stride];
    }
  };
  const auto advance = [&](const Chunk& c, uint32_t which) __attribute__((always_inline)) {
    if constexpr (OUTPUTS) {
      f32x4 sum[4] = {};
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        sum[e] = __builtin_amdgcn_mfma_f32_16x16x4f32(c.weights[e], c.values[e], sum[e], 0, 0, 0);
#pragma unroll
        for (int d = 0; d < TILES; ++d)
          sum[e] = __builtin_amdgcn_mfma_f32_16x16x4f32(c.reads[d][e], state[d][e], sum[e], 0,
                                                        0, 0);
      }
      const f32x4 out = (sum[0] + sum[1]) + (sum[2] + sum[3]);
#pragma unroll
      for (uint32_t i = 0; i < 4u; ++i) {
        const uint32_t row = which * kChunk + 4u * quarter + i;
        if (real && row < run.rows)
          args.outputs[(size_t{row} * l.heads + head) * vdim + column] = out[i];
      }
    }
#pragma unroll
    for (int d = 0; d < TILES; ++d) {
      state[d] *= c.decays[d];
      if constexpr (!OUTPUTS) faded[d] *= c.decays[d];
    }
#pragma unroll
    for (int e = 0; e < 4; ++e)
#pragma unroll
      for (int d = 0; d < TILES; ++d)
        state[d] = __builtin_amdgcn_mfma_f32_16x16x4f32(c.keys[d][e], c.values[e], state[d], 0,
                                                        0, 0);
  };
  const uint32_t begin = segment * args.segment_chunks;
  const uint32_t end = min(begin + args.segment_chunks, args.chunk_count);
  Chunk even, odd;
  fetch(even, begin);
  uint32_t which = begin;
  while (which < end) {
    fetch(odd, min(which + 1u, end - 1u));
    advance(even, which);
    if (++which >= end) break;
    fetch(even, min(which + 1u, end - 1u));
    advance(odd, which);
    ++which;
  }
  if (OUTPUTS && segment + 1u != args.segments) return;
  float* const to = OUTPUTS ? request : kept;
#pragma unroll
  for (int d = 0; d < TILES; ++d)
#pragma unroll
    for (uint32_t i = 0; i < 4u; ++i) {
      const uint32_t row = d * 16u + 4u * quarter + i;
      if (real && row < dim) to[size_t{row} * vdim + column] = state[d][i];
    }
  if (OUTPUTS || first_column || lane % 16u) return;
#pragma unroll
  for (int d = 0; d < TILES; ++d)
    reinterpret_cast<f32x4*>(args.totals)[(size_t{segment} * l.heads + head) * (kPadded / 4u) +
                                          d * 4u + quarter] = faded[d];
}

// The states that segments end with become the states they start from.
__global__ __launch_bounds__(256) void recurrence_join_kernel(RecurrenceArgs args) {
  const qllm_recurrence& l = args.layer;
  const uint32_t elements = l.heads * l.dim * l.vdim;
  const uint32_t at = blockIdx.x * blockDim.x + threadIdx.x;
  if (at >= elements) return;
  const uint32_t row = at / l.vdim;      // over all heads
  const float* total = args.totals + size_t{row / l.dim} * args.padded + row % l.dim;
  float end[kMaximumSegments], fade[kMaximumSegments];
#pragma unroll
  for (uint32_t z = 0; z + 1u < kMaximumSegments; ++z) {
    const bool there = z + 1u < args.segments;
    end[z] = there ? args.starts[size_t{z} * elements + at] : 0.0f;
    fade[z] = z && there ? total[size_t{z} * l.heads * args.padded] : 0.0f;
  }
  args.starts[at] = l.state[l.step[kStepSlot] * l.slot_stride + at];
  float state = 0.0f;
#pragma unroll
  for (uint32_t z = 0; z + 1u < kMaximumSegments; ++z) {
    if (z + 1u >= args.segments) continue;
    state = fmaf(fade[z], state, end[z]);
    args.starts[size_t{z + 1u} * elements + at] = state;
  }
}

// Output norm and gate: a wave per (token, head).
template <typename T>
__global__ __launch_bounds__(256) void recurrence_finish_kernel(RecurrenceArgs args) {
  const qllm_recurrence& l = args.layer;
  const auto& run = args.launch;
  const uint32_t item = blockIdx.x * 4u + threadIdx.x / kWave;
  if (item >= run.rows * l.heads) return;
  const uint32_t row = item / l.heads;
  const uint32_t vdim = l.vdim;
  const uint32_t first = item % l.heads * vdim;
  const uint32_t lane = threadIdx.x % kWave;
  const float* o = args.outputs + size_t{row} * l.heads * vdim + first;
  const float* gates = run.projections + size_t{row} * run.stride + run.gate_column + first;
  const float* norm = l.norm_weight + (l.kind == QLLM_RECURRENCE_GATED ? 0u : first);
  T* out = static_cast<T*>(run.output) + size_t{row} * run.output_stride + first;
  constexpr uint32_t kHeld = 4;
  float held[kHeld];
  float squares = 0.0f;
#pragma unroll
  for (uint32_t i = 0; i < kHeld; ++i) {
    const uint32_t c = lane + i * kWave;
    held[i] = c < vdim ? o[c] : 0.0f;
    squares = fmaf(held[i], held[i], squares);
  }
  for (uint32_t c = lane + kHeld * kWave; c < vdim; c += kWave)
    squares = fmaf(o[c], o[c], squares);
  squares = wave_sum(squares);
  const float inverse = 1.0f / sqrtf(squares / static_cast<float>(vdim) + l.epsilon);
  const auto finish = [&](uint32_t c, float value) {
    store_element(out + c, value * inverse * norm[c] * gate_value(l.gate_kind, gates[c]));
  };
#pragma unroll
  for (uint32_t i = 0; i < kHeld; ++i)
    if (lane + i * kWave < vdim) finish(lane + i * kWave, held[i]);
  for (uint32_t c = lane + kHeld * kWave; c < vdim; c += kWave) finish(c, o[c]);
}

template <uint32_t KIND>
void launch_scan(const RecurrenceArgs& args, hipStream_t stream) {
  const dim3 grid((args.layer.vdim + 15u) / 16u, args.layer.heads);
  switch (args.padded) {
    case 16u: recurrence_scan_kernel<KIND, 1><<<grid, 256, 0, stream>>>(args); break;
    case 32u: recurrence_scan_kernel<KIND, 2><<<grid, 256, 0, stream>>>(args); break;
    case 64u: recurrence_scan_kernel<KIND, 4><<<grid, 256, 0, stream>>>(args); break;
    case 128u: recurrence_scan_kernel<KIND, 8><<<grid, 256, 0, stream>>>(args); break;
    default: recurrence_scan_kernel<KIND, 16><<<grid, 256, 0, stream>>>(args); break;
  }
}

template <uint32_t KIND, int TILES>
void launch_chunks(const RecurrenceArgs& args, hipStream_t stream) {
  const qllm_recurrence& l = args.layer;
  recurrence_chunk_kernel<KIND, TILES>
      <<<dim3(args.chunk_count, l.heads), 256, 0, stream>>>(args);
  const uint32_t columns = (l.vdim + 63u) / 64u;
  if (args.segments > 1u) {
    // the last segment's own end comes with its outputs
    recurrence_walk_kernel<false, TILES>
        <<<dim3(columns, l.heads, args.segments - 1u), 256, 0, stream>>>(args);
    recurrence_join_kernel<<<(l.heads * l.dim * l.vdim + 255u) / 256u, 256, 0, stream>>>(args);
  }
  recurrence_walk_kernel<true, TILES>
      <<<dim3(columns, l.heads, args.segments), 256, 0, stream>>>(args);
}

template <uint32_t KIND>
void launch_chunks_of(const RecurrenceArgs& args, hipStream_t stream) {
  switch (args.padded) {
    case 16u: launch_chunks<KIND, 1>(args, stream); break;
    case 32u: launch_chunks<KIND, 2>(args, stream); break;
    case 64u: launch_chunks<KIND, 4>(args, stream); break;
    default: launch_chunks<KIND, 8>(args, stream); break;
  }
}

template <typename T>
void launch_gated_step(const RecurrenceArgs& args, hipStream_t stream) {
  const uint32_t groups = 1024u / args.layer.vdim;
  const uint32_t rows = (args.layer.dim + groups - 1u) / groups;
  if (rows <= 4u)
    gated_step_kernel<T, 4><<<args.layer.heads, 1024, 0, stream>>>(args);
  else if (rows <= 16u)
    gated_step_kernel<T, 16><<<args.layer.heads, 1024, 0, stream>>>(args);
  else
    gated_step_kernel<T, 0><<<args.layer.heads, 1024, 0, stream>>>(args);
}

template <typename T>
void launch_step(const RecurrenceArgs& args, hipStream_t stream) {
  if (args.layer.kind == QLLM_RECURRENCE_GATED) {
    launch_gated_step<T>(args, stream);
    return;
  }
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

size_t output_bytes(const qllm_recurrence& l, uint32_t rows) {
  return (size_t{rows} * l.heads * l.vdim * 4u + 15u) / 16u * 16u;
}

constexpr uint32_t kChunkedRows = 64;        // shorter batches go token by token
constexpr uint32_t kSegmentRows = 256;       // at least

bool goes_in_chunks(const qllm_recurrence& l, uint32_t rows) {
  return l.kind != QLLM_RECURRENCE_DELTA && l.dim <= 128u && rows >= kChunkedRows;
}

// Segments of a prompt: a few waves for every SIMD of the chip.
uint32_t segments_for(const qllm_recurrence& l, uint32_t rows) {
  const uint32_t waves = l.heads * ((l.vdim + 15u) / 16u);
  const uint32_t wanted = (2048u + waves - 1u) / waves;
  const uint32_t most = rows / kSegmentRows;
  const uint32_t segments = wanted < most ? wanted : most;
  return segments > kMaximumSegments ? kMaximumSegments : segments ? segments : 1u;
}

size_t chunk_bytes(const qllm_recurrence& l, uint32_t rows) {
  return size_t{l.heads} * ((rows + kChunk - 1u) / kChunk) * chunk_floats(padded_dim(l.dim)) *
         4u;
}

size_t start_bytes(const qllm_recurrence& l, uint32_t segments) {
  return (size_t{segments} * l.heads * l.dim * l.vdim * 4u + 15u) / 16u * 16u;
}

size_t total_bytes(const qllm_recurrence& l, uint32_t segments) {
  return size_t{segments} * l.heads * padded_dim(l.dim) * 4u;
}

}  // namespace
}  // namespace qllm

using namespace qllm;

extern "C" size_t qllm_recurrence_workspace_bytes(const qllm_recurrence* recurrence,
                                                  uint32_t rows) {
  if (!recurrence || rows <= 1u) return 0u;
  qllm_recurrence l = *recurrence;
  if (!l.vdim) l.vdim = l.dim;
  size_t bytes = prepared_bytes(l, rows) + scalar_bytes(l, rows) + output_bytes(l, rows);
  if (goes_in_chunks(l, rows)) {
    const uint32_t segments = segments_for(l, rows);
    bytes += chunk_bytes(l, rows) + start_bytes(l, segments) + total_bytes(l, segments);
  }
  return bytes;
}

extern "C" int32_t qllm_recurrence_rows(const qllm_recurrence* recurrence,
                                        const qllm_recurrence_launch* launch,
                                        void* stream) {
  if (!recurrence || !launch) return fail(QLLM_INVALID_ARGUMENT, "invalid recurrence");
  qllm_recurrence l = *recurrence;
  if (!l.vdim) l.vdim = l.dim;
  const bool delta = l.kind == QLLM_RECURRENCE_DELTA;
  const bool gated = l.kind == QLLM_RECURRENCE_GATED;
  if (l.kind > QLLM_RECURRENCE_GATED || l.vdim > 1024u || (!gated && l.vdim != l.dim) || !l.heads || !l.dim || l.dim > 256u || !l.rank ||
      l.rank > 256u || l.gate_kind > QLLM_GATE_SILU || l.element > QLLM_ELEMENT_F32 ||
      !l.decay_up_bf16 || !l.decay_base || !l.norm_weight || !l.state || !l.step ||
      (delta ? !l.rate_bias : !gated && !l.bonus) || !launch->projections ||
      !launch->output || !launch->rows || launch->output_stride < l.heads * l.vdim ||
      (launch->carry_to && (!launch->carry_from || !launch->carry_width)))
    return fail(QLLM_INVALID_ARGUMENT, "invalid recurrence");
  for (const uint32_t column : {launch->v_column, launch->gate_column})
    if (column + l.heads * l.vdim > launch->stride)
      return fail(QLLM_INVALID_ARGUMENT, "recurrence columns exceed the projection rows");
  for (const uint32_t column :
       {launch->r_column, launch->k_column, delta ? launch->rate_column : 0u})
    if (column + l.heads * l.dim > launch->stride)
      return fail(QLLM_INVALID_ARGUMENT, "recurrence columns exceed the projection rows");
  if (launch->low_column + l.rank > launch->stride)
    return fail(QLLM_INVALID_ARGUMENT, "recurrence columns exceed the projection rows");
  const auto hip_stream = as_stream(stream);
  RecurrenceArgs args{};
  args.layer = l;
  args.launch = *launch;
  args.padded = padded_dim(l.dim);
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
  bytes += prepared_bytes(l, launch->rows) + scalar_bytes(l, launch->rows);
  args.outputs = reinterpret_cast<float*>(bytes);
  bytes += output_bytes(l, launch->rows);
  const uint32_t prepare_rows = 256u / args.padded * kRowsPerThread;
  recurrence_prepare_kernel<<<dim3((launch->rows + prepare_rows - 1u) / prepare_rows,
                                   l.heads),
                              256, 0, hip_stream>>>(args);
  if (goes_in_chunks(l, launch->rows)) {
    const uint32_t segments = segments_for(l, launch->rows);
    args.chunks = reinterpret_cast<float*>(bytes);
    bytes += chunk_bytes(l, launch->rows);
    args.starts = reinterpret_cast<float*>(bytes);
    bytes += start_bytes(l, segments);
    args.totals = reinterpret_cast<float*>(bytes);
    args.chunk_count = (launch->rows + kChunk - 1u) / kChunk;
    args.segment_chunks = (args.chunk_count + segments - 1u) / segments;
    // none is empty
    args.segments = (args.chunk_count + args.segment_chunks - 1u) / args.segment_chunks;
    if (gated)
      launch_chunks_of<QLLM_RECURRENCE_GATED>(args, hip_stream);
    else
      launch_chunks_of<QLLM_RECURRENCE_BONUS>(args, hip_stream);
  } else if (delta)
    launch_scan<QLLM_RECURRENCE_DELTA>(args, hip_stream);
  else if (gated)
    launch_scan<QLLM_RECURRENCE_GATED>(args, hip_stream);
  else
    launch_scan<QLLM_RECURRENCE_BONUS>(args, hip_stream);
  const uint32_t blocks = (launch->rows * l.heads + 3u) / 4u;
  if (f32)
    recurrence_finish_kernel<float><<<blocks, 256, 0, hip_stream>>>(args);
  else
    recurrence_finish_kernel<uint16_t><<<blocks, 256, 0, hip_stream>>>(args);
  return launched("recurrence");
}
