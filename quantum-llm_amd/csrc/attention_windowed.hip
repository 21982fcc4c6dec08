// Windowed attention with kept first tokens and mixed heads, over paged bf16
// (or F32) keys and values.
//
// The heads' softmax weights are mixed before they meet the values, so no head
// can finish on its own: the mix needs every head's normalised weights.  Three
// forms:
//
//  * split (one to four rows, decode): scores of all visible keys once, 16 keys
//    per wave, with each workgroup's maximum and sum; then, per key/value head,
//    normalise, mix (F32) and multiply with the values, the visible tiles dealt
//    over workgroups; then the partial outputs are added and gated.
//  * prompt: a first walk over the visible keys takes every row's softmax
//    denominator.  In a second, a workgroup owns 16 query rows and all heads: it
//    recomputes the scores, leaves the normalised weights in LDS as bf16 high
//    and low halves (together 16 bits of mantissa), lets the matrix cores mix
//    them over heads - the mix matrix is bf16 as stored, so both products are
//    exact and added in F32 - and multiplies the mixed weights with the values.
//  * general: one workgroup per row, any size, bf16 or F32 arithmetic.
//
// Keys lie in fragments of 16 tokens x 32 dimensions and values, transposed, in
// fragments of 16 dimensions x 32 tokens: every operand load of a wave is one
// contiguous KiB.
#include "mixed_common.hpp"

#include <cmath>

namespace qllm {
namespace {

constexpr uint32_t kTileKeys = 32;
constexpr uint32_t kMaximumScoreSplits = 64;
constexpr uint32_t kMaximumValueSplits = 16;
constexpr uint32_t kSplitRows = 4;        // rows of the split form
constexpr uint32_t kPromptHeads = 32;
constexpr uint32_t kMaximumLds = 160u * 1024u;

using Attention = qllm_windowed_attention;

// The 32-key tiles that rows first .. last can see: those of the kept first
// tokens, then those of the windows.
struct TileRange {
  uint32_t sink_tiles;
  uint32_t window_tile;   // first tile of the second part
  uint32_t count;
  __device__ __forceinline__ uint32_t tile(uint32_t ordinal) const {
    return ordinal < sink_tiles ? ordinal : window_tile + (ordinal - sink_tiles);
  }
};

__device__ __forceinline__ TileRange tiles_for(const Attention& a, uint32_t first,
                                               uint32_t last) {
  TileRange range;
  const uint32_t kept = min(a.sinks, last + 1u);
  range.sink_tiles = (kept + kTileKeys - 1u) / kTileKeys;
  const uint32_t low = a.window && first + 1u > a.window ? first + 1u - a.window : 0u;
  range.window_tile = max(low / kTileKeys, range.sink_tiles);
  const uint32_t last_tile = last / kTileKeys;
  range.count = range.sink_tiles + (last_tile >= range.window_tile
                                        ? last_tile - range.window_tile + 1u
                                        : 0u);
  return range;
}

__device__ __forceinline__ bool visible(const Attention& a, uint32_t position,
                                        uint32_t key) {
  return key <= position && (!a.window || position - key < a.window || key < a.sinks);
}

// The request's row of the page table, and the layer's part of a page.
__device__ __forceinline__ void* const* pages_of(const Attention& a) {
  return a.page_table + size_t{a.step[kStepSlot]} * a.pages_per_slot;
}
template <typename T>
__device__ __forceinline__ T* page_of(const Attention& a, void* const* pages,
                                      uint32_t position) {
  return reinterpret_cast<T*>(static_cast<uint8_t*>(pages[position / a.page_tokens]) +
                              a.layer_offset);
}
template <typename T>
__device__ __forceinline__ T* page_of(const Attention& a, uint32_t position) {
  return page_of<T>(a, pages_of(a), position);
}

// Element offsets of fragment rows inside a layer of a page.
__device__ __forceinline__ size_t key_block(const Attention& a, uint32_t kv, uint32_t slot) {
  return size_t{kv * (a.page_tokens / 16u) + slot / 16u} * 16u * a.key_stride;
}
__device__ __forceinline__ size_t value_block(const Attention& a, uint32_t kv,
                                              uint32_t slot) {
  return size_t{a.kv_heads} * a.page_tokens * a.key_stride +
         size_t{kv * (a.page_tokens / 32u) + slot / 32u} * 32u * a.value_stride;
}

// ---- rotary, value blend, store ------------------------------------------------

struct RopeArgs {
  Attention attention;
  qllm_rope_store_launch launch;
  uint32_t rows_per_block;
};

// A wave walks the rows of a block for one query, key or value head.
template <typename T>
__global__ __launch_bounds__(256) void rope_store_kernel(RopeArgs args) {
  const Attention& a = args.attention;
  const auto& run = args.launch;
  const uint32_t unit = blockIdx.y * 4u + threadIdx.x / kWave;
  const uint32_t lane = threadIdx.x % kWave;
  if (unit >= a.query_heads + 2u * a.kv_heads) return;
  const uint32_t first_row = blockIdx.x * args.rows_per_block;
  const uint32_t last_row = min(first_row + args.rows_per_block, run.rows);
  const uint32_t first_position = a.step[kStepPosition];

  if (unit >= a.query_heads + a.kv_heads) {
    const uint32_t kv = unit - a.query_heads - a.kv_heads;
    const float share = run.first_values ? *run.value_share : 0.0f;
    for (uint32_t row = first_row; row < last_row; ++row) {
      const uint32_t position = first_position + row;
      T* page = page_of<T>(a, position);
      const uint32_t slot = position % a.page_tokens;
      T* out = page + value_block(a, kv, slot) + slot % 32u;
      const float* source =
          run.projections + size_t{row} * run.stride + run.value_column + kv * a.vdim;
      const size_t at = size_t{row} * a.kv_heads * a.vdim + kv * a.vdim;
      for (uint32_t d = lane; d < a.vdim; d += kWave) {
        float value = source[d];
        if (run.values_out) run.values_out[at + d] = value;
        if (run.first_values)
          value = (1.0f - share) * value + share * run.first_values[at + d];
        store_element(out + size_t{d} * 32u, value);
      }
    }
    return;
  }

  const bool is_key = unit >= a.query_heads;
  const uint32_t head = is_key ? unit - a.query_heads : unit;
  const uint32_t column = (is_key ? run.key_column : run.query_column) + head * a.dim;
  for (uint32_t pair = lane; pair < a.key_stride / 2u; pair += kWave) {
    const uint32_t d = 2u * pair;
    const bool turns = d < run.rotary_dims;
    const double frequency = turns ? run.frequencies[pair] : 0.0;
    for (uint32_t row = first_row; row < last_row; ++row) {
      const uint32_t position = first_position + row;
      const float* source = run.projections + size_t{row} * run.stride + column;
      float u = d < a.dim ? source[d] : 0.0f;
      float v = d + 1u < a.dim ? source[d + 1u] : 0.0f;
      if (turns) {
        // the angle is reduced to one turn before it becomes F32
        constexpr double kTurn = 6.283185307179586476925286766559;
        double angle = static_cast<double>(position) * frequency;
        angle -= kTurn * rint(angle / kTurn);
        float sine, cosine;
        sincosf(static_cast<float>(angle), &sine, &cosine);
        const float turned = u * cosine - v * sine;
        v = v * cosine + u * sine;
        u = turned;
      }
      T* out;
      if (is_key) {
        const uint32_t slot = position % a.page_tokens;
        out = page_of<T>(a, position) + key_block(a, head, slot) +
              size_t{d / 32u} * 512u + slot % 16u * 32u + d % 32u;
      } else {
        out = static_cast<T*>(run.query_out) +
              (size_t{row} * a.query_heads + head) * a.key_stride + d;
      }
      store_element(out, u);
      store_element(out + 1, v);
    }
  }
}

// ---- general form ----------------------------------------------------------------

struct AttentionArgs {
  Attention attention;
  qllm_attention_launch launch;
  float* scores;          // split form: [row][head][capacity]
  float* maxima;          // [row][split][head] (maximum, sum)
  float* partials;        // [row][split][head][vdim]
  uint32_t capacity;      // score slots per head
  uint32_t score_splits;
  uint32_t value_splits;
};

template <typename T>
__global__ __launch_bounds__(256) void general_attention_kernel(AttentionArgs args) {
  extern __shared__ float shared[];
  const Attention& a = args.attention;
  const auto& run = args.launch;
  const uint32_t heads = a.query_heads;
  const uint32_t group = heads / a.kv_heads;
  float* q = shared;                                   // [heads][dim]
  float* weights = q + heads * a.dim;                  // [heads][32]
  float* mixed = weights + heads * kTileKeys;          // [heads][32]
  float* out = mixed + heads * kTileKeys;              // [heads][vdim]
  float* maximum = out + heads * a.vdim;               // [heads]
  float* sum = maximum + heads;                        // [heads]
  const uint32_t row = blockIdx.x;
  const uint32_t position = a.step[kStepPosition] + row;
  const TileRange range = tiles_for(a, position, position);

  const T* query = static_cast<const T*>(run.query) + size_t{row} * heads * a.key_stride;
  for (uint32_t i = threadIdx.x; i < heads * a.dim; i += blockDim.x)
    q[i] = load_element(query + size_t{i / a.dim} * a.key_stride + i % a.dim);
  for (uint32_t i = threadIdx.x; i < heads * a.vdim; i += blockDim.x) out[i] = 0.0f;
  for (uint32_t h = threadIdx.x; h < heads; h += blockDim.x) {
    maximum[h] = -INFINITY;
    sum[h] = 0.0f;
  }
  __syncthreads();

  const auto score_tile = [&](uint32_t tile, const T* page) {
    for (uint32_t i = threadIdx.x; i < heads * kTileKeys; i += blockDim.x) {
      const uint32_t head = i / kTileKeys;
      const uint32_t key = tile * kTileKeys + i % kTileKeys;
      float score = -INFINITY;
      if (visible(a, position, key)) {
        const uint32_t slot = key % a.page_tokens;
        const T* k = page + key_block(a, head / group, slot) + slot % 16u * 32u;
        score = 0.0f;
        for (uint32_t d = 0; d < a.dim; ++d)
          score = fmaf(q[head * a.dim + d],
                       load_element(k + size_t{d / 32u} * 512u + d % 32u), score);
        score *= a.scale;
      }
      weights[i] = score;
    }
    __syncthreads();
  };

  for (uint32_t ordinal = 0; ordinal < range.count; ++ordinal) {
    const uint32_t tile = range.tile(ordinal);
    score_tile(tile, page_of<const T>(a, tile * kTileKeys));
    for (uint32_t h = threadIdx.x; h < heads; h += blockDim.x) {
      float m = maximum[h];
      for (uint32_t j = 0; j < kTileKeys; ++j) m = fmaxf(m, weights[h * kTileKeys + j]);
      if (m > -INFINITY) {
        float s = sum[h] * expf(maximum[h] - m);
        for (uint32_t j = 0; j < kTileKeys; ++j) s += expf(weights[h * kTileKeys + j] - m);
        sum[h] = s;
        maximum[h] = m;
      }
    }
    __syncthreads();
  }
  for (uint32_t ordinal = 0; ordinal < range.count; ++ordinal) {
    const uint32_t tile = range.tile(ordinal);
    const T* page = page_of<const T>(a, tile * kTileKeys);
    score_tile(tile, page);
    for (uint32_t i = threadIdx.x; i < heads * kTileKeys; i += blockDim.x) {
      const uint32_t h = i / kTileKeys;
      weights[i] = expf(weights[i] - maximum[h]) / sum[h];
    }
    __syncthreads();
    for (uint32_t i = threadIdx.x; i < heads * kTileKeys; i += blockDim.x) {
      if (!a.head_mix) {
        mixed[i] = weights[i];
        continue;
      }
      const float* mix = a.head_mix + size_t{i / kTileKeys} * heads;
      float total = 0.0f;
      for (uint32_t g = 0; g < heads; ++g)
        total = fmaf(mix[g], weights[g * kTileKeys + i % kTileKeys], total);
      mixed[i] = total;
    }
    __syncthreads();
    const uint32_t slot = tile * kTileKeys % a.page_tokens;
    for (uint32_t i = threadIdx.x; i < heads * a.vdim; i += blockDim.x) {
      const uint32_t h = i / a.vdim;
      const T* v = page + value_block(a, h / group, slot) + size_t{i % a.vdim} * 32u;
      float total = out[i];
      // slots past the row's position may hold anything: their weight is zero
      for (uint32_t j = 0; j < kTileKeys; ++j)
        total = fmaf(mixed[h * kTileKeys + j], load_element(v + j), total);
      out[i] = total;
    }
    __syncthreads();
  }
  for (uint32_t i = threadIdx.x; i < heads * a.vdim; i += blockDim.x) {
    const float gate =
        run.gate ? sigmoid_f32(run.gate[size_t{row} * run.gate_stride + i / a.vdim]) : 1.0f;
    store_element(static_cast<T*>(run.output) + size_t{row} * run.output_stride + i,
                  out[i] * gate);
  }
}

// ---- split form (decode) -----------------------------------------------------------

// NK = key_stride / 32.
template <int NK>
__global__ __launch_bounds__(256) void split_scores_kernel(AttentionArgs args) {
  __shared__ float wave_maximum[4][16];
  __shared__ float wave_total[4][16];
  const Attention& a = args.attention;
  const uint32_t row = blockIdx.z;
  const uint32_t kv = blockIdx.y;
  const uint32_t position = a.step[kStepPosition] + row;
  const TileRange range = tiles_for(a, position, position);
  const uint32_t group = a.query_heads / a.kv_heads;
  const uint32_t wave = threadIdx.x / kWave;
  const uint32_t lane = threadIdx.x % kWave;
  const uint32_t in_group = lane % 16u;
  const uint32_t head = kv * group + min(in_group, group - 1u);

  i32x4 q[NK];
  const uint16_t* query = static_cast<const uint16_t*>(args.launch.query) +
                          (size_t{row} * a.query_heads + head) * a.key_stride +
                          8u * (lane / 16u);
#pragma unroll
  for (int c = 0; c < NK; ++c) q[c] = *reinterpret_cast<const i32x4*>(query + c * 32);

  const uint32_t units = range.count * 2u;   // of 16 keys
  const uint32_t begin = static_cast<uint32_t>(uint64_t{units} * blockIdx.x / gridDim.x);
  const uint32_t end = static_cast<uint32_t>(uint64_t{units} * (blockIdx.x + 1u) / gridDim.x);
  float maximum = -INFINITY;
  float total = 0.0f;
  float* scores =
      args.scores + (size_t{row} * a.query_heads + head) * args.capacity + 4u * (lane / 16u);
  for (uint32_t unit = begin + wave; unit < end; unit += 4u) {
    const uint32_t key0 = range.tile(unit / 2u) * kTileKeys + unit % 2u * 16u;
    const uint32_t slot = key0 % a.page_tokens;
    const i32x4* keys = reinterpret_cast<const i32x4*>(page_of<const uint16_t>(a, key0) +
                                                       key_block(a, kv, slot)) +
                        lane % 16u * 4u + lane / 16u;
    i32x4 k[NK];
#pragma unroll
    for (int c = 0; c < NK; ++c) k[c] = keys[c * kWave];
    f32x4 s = {};
#pragma unroll
    for (int c = 0; c < NK; ++c) s = mfma_bf16(k[c], q[c], s);
    float top = -INFINITY;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const uint32_t key = key0 + 4u * (lane / 16u) + i;
      s[i] = visible(a, position, key) ? s[i] * a.scale : -INFINITY;
      top = fmaxf(top, s[i]);
    }
    if (in_group < group) *reinterpret_cast<f32x4*>(scores + size_t{unit} * 16u) = s;
    if (top > -INFINITY) {
      const float fresh = fmaxf(maximum, top);
      total *= expf(maximum - fresh);
#pragma unroll
      for (int i = 0; i < 4; ++i) total += expf(s[i] - fresh);
      maximum = fresh;
    }
  }
  // the four lanes of a head, then the four waves
  const auto merge = [](float& m, float& t, float other_m, float other_t) {
    const float fresh = fmaxf(m, other_m);
    if (fresh == -INFINITY) return;
    t = t * expf(m - fresh) + other_t * expf(other_m - fresh);
    m = fresh;
  };
  merge(maximum, total, __shfl_xor(maximum, 16, kWave), __shfl_xor(total, 16, kWave));
  merge(maximum, total, __shfl_xor(maximum, 32, kWave), __shfl_xor(total, 32, kWave));
  if (lane < 16u) {
    wave_maximum[wave][lane] = maximum;
    wave_total[wave][lane] = total;
  }
  __syncthreads();
  if (threadIdx.x < group) {
    float m = wave_maximum[0][threadIdx.x];
    float t = wave_total[0][threadIdx.x];
    for (int other = 1; other < 4; ++other)
      merge(m, t, wave_maximum[other][threadIdx.x], wave_total[other][threadIdx.x]);
    float* out = args.maxima + ((size_t{row} * args.score_splits + blockIdx.x) *
                                    a.query_heads +
                                kv * group + threadIdx.x) * 2u;
    out[0] = m;
    out[1] = t;
  }
}

constexpr uint32_t kMixRow = 40;   // bf16 values per LDS row of mixed weights (32 + pad)

// NV = value_stride / 16, GROUP = query heads per key/value head at most.
template <int NV, int GROUP>
__global__ __launch_bounds__(256) void split_values_kernel(AttentionArgs args) {
  __shared__ float row_maximum[64], row_inverse[64];
  __shared__ __attribute__((aligned(16))) float mix[64][GROUP];
  __shared__ __attribute__((aligned(16))) uint16_t mixed[4][16 * kMixRow];
  __shared__ f32x4 gathered[NV * kWave];
  const Attention& a = args.attention;
  const uint32_t row = blockIdx.z;
  const uint32_t kv = blockIdx.y;
  const uint32_t position = a.step[kStepPosition] + row;
  const TileRange range = tiles_for(a, position, position);
  const uint32_t heads = a.query_heads;
  const uint32_t group = heads / a.kv_heads;
  const uint32_t wave = threadIdx.x / kWave;
  const uint32_t lane = threadIdx.x % kWave;

  // a wave per head, a lane per score split (at most 64)
#pragma unroll 4
  for (uint32_t h = wave; h < heads; h += 4u) {
    float m = -INFINITY;
    float t = 0.0f;
    if (lane < args.score_splits) {
      const float* pair =
          args.maxima + ((size_t{row} * args.score_splits + lane) * heads + h) * 2u;
      m = pair[0];
      t = pair[1];
    }
    const float top = wave_max(m);
    t = wave_sum(t * expf(m - top));
    if (lane == 0u) {
      row_maximum[h] = top;
      row_inverse[h] = 1.0f / t;
    }
  }
  for (uint32_t i = threadIdx.x; i < heads * GROUP; i += blockDim.x) {
    const uint32_t g = i / GROUP;
    const uint32_t in_group = i % GROUP;
    const uint32_t h = kv * group + min(in_group, group - 1u);
    const float value = a.head_mix ? a.head_mix[size_t{h} * heads + g] : (h == g ? 1.0f : 0.0f);
    mix[g][in_group] = in_group < group ? value : 0.0f;
  }
  for (uint32_t i = threadIdx.x; i < 4u * 16u * kMixRow; i += blockDim.x)
    mixed[0][i] = 0u;
  __syncthreads();

  f32x4 sum[NV] = {};
  const uint32_t begin = static_cast<uint32_t>(uint64_t{range.count} * blockIdx.x / gridDim.x);
  const uint32_t end =
      static_cast<uint32_t>(uint64_t{range.count} * (blockIdx.x + 1u) / gridDim.x);
  for (uint32_t ordinal = begin + wave; ordinal < end; ordinal += 4u) {
    const uint32_t key0 = range.tile(ordinal) * kTileKeys;
    const i32x4* values = reinterpret_cast<const i32x4*>(
                              page_of<const uint16_t>(a, key0) +
                              value_block(a, kv, key0 % a.page_tokens)) +
                          lane % 16u * 4u + lane / 16u;
    i32x4 v[NV];
#pragma unroll
    for (int t = 0; t < NV; ++t) v[t] = values[t * kWave];
    // lane: key lane % 32, heads of parity lane / 32
    const float* scores = args.scores + size_t{row} * heads * args.capacity +
                          size_t{ordinal} * kTileKeys + lane % 32u;
    float share[GROUP] = {};
    for (uint32_t g0 = lane / 32u; g0 < heads; g0 += 16u) {
      float raw[8];
#pragma unroll
      for (uint32_t i = 0; i < 8u; ++i)
        raw[i] = scores[size_t{min(g0 + 2u * i, heads - 1u)} * args.capacity];
#pragma unroll
      for (uint32_t i = 0; i < 8u; ++i) {
        const uint32_t g = min(g0 + 2u * i, heads - 1u);
        const float p = g0 + 2u * i < heads
                            ? expf(raw[i] - row_maximum[g]) * row_inverse[g]
                            : 0.0f;
#pragma unroll
        for (int h = 0; h < GROUP; ++h) share[h] = fmaf(mix[g][h], p, share[h]);
      }
    }
#pragma unroll
    for (int h = 0; h < GROUP; ++h) {
      const float both = share[h] + __shfl_xor(share[h], 32, kWave);
      if (lane < 32u)
        mixed[wave][h * kMixRow + lane] = static_cast<uint16_t>(f32_to_bf16_bits(both));
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
    const i32x4 w = *reinterpret_cast<const i32x4*>(
        &mixed[wave][lane % 16u * kMixRow + 8u * (lane / 16u)]);
#pragma unroll
    for (int t = 0; t < NV; ++t) sum[t] = mfma_bf16(w, v[t], sum[t]);
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
  }
  // the waves' sums in order
  for (uint32_t turn = 0; turn < 4u; ++turn) {
    if (wave == turn)
#pragma unroll
      for (int t = 0; t < NV; ++t)
        gathered[t * kWave + lane] = turn == 0u ? sum[t] : gathered[t * kWave + lane] + sum[t];
    __syncthreads();
  }
  for (uint32_t i = threadIdx.x; i < NV * kWave; i += blockDim.x) {
    const uint32_t d = i / kWave * 16u + i % 16u;
    if (d >= a.vdim) continue;
    for (uint32_t j = 0; j < 4u; ++j) {
      const uint32_t h = 4u * (i % kWave / 16u) + j;
      if (h < group)
        args.partials[((size_t{row} * args.value_splits + blockIdx.x) * heads + kv * group +
                       h) * a.vdim + d] = gathered[i][j];
    }
  }
}

__global__ void split_combine_kernel(AttentionArgs args) {
  const Attention& a = args.attention;
  const auto& run = args.launch;
  const uint32_t head = blockIdx.x;
  const uint32_t row = blockIdx.y;
  const float gate =
      run.gate ? sigmoid_f32(run.gate[size_t{row} * run.gate_stride + head]) : 1.0f;
  for (uint32_t d = threadIdx.x; d < a.vdim; d += blockDim.x) {
    float part[kMaximumValueSplits];
#pragma unroll
    for (uint32_t s = 0; s < kMaximumValueSplits; ++s)
      part[s] = s < args.value_splits
                    ? args.partials[((size_t{row} * args.value_splits + s) * a.query_heads +
                                     head) * a.vdim + d]
                    : 0.0f;
    float total = 0.0f;
#pragma unroll
    for (uint32_t s = 0; s < kMaximumValueSplits; ++s) total += part[s];
    store_element(static_cast<uint16_t*>(run.output) + size_t{row} * run.output_stride +
                      head * a.vdim + d,
                  total * gate);
  }
}

// ---- prompt form -------------------------------------------------------------------

// Sixteen-byte slots of a 64-byte LDS row, permuted by the row so that sixteen
// rows touched at the same slot fall on different banks.
__device__ __forceinline__ uint32_t swizzled(uint32_t row, uint32_t slot) {
  return row * 64u + ((slot ^ (row >> 2 & 3u)) * 16u);
}

// The bf16 halves of two non-negative weights: the upper 16 bits of each as
// they stand, and the rest, rounded.
__device__ __forceinline__ void split_pair(float a, float b, uint32_t& high,
                                           uint32_t& low) {
  const uint32_t a_bits = __float_as_uint(a);
  const uint32_t b_bits = __float_as_uint(b);
  high = __builtin_amdgcn_perm(b_bits, a_bits, 0x07060302u);
  low = pack_bf16(a - __uint_as_float(a_bits & 0xffff0000u),
                  b - __uint_as_float(b_bits & 0xffff0000u));
}

// Row blocks of the prompt kernels: contiguous ranges per XCD (consecutive
// workgroups go round the XCDs), since neighbours share their keys.
__device__ __forceinline__ uint32_t xcd_range(uint32_t block, uint32_t blocks) {
  const uint32_t per_xcd = blocks / 8u;
  return block < per_xcd * 8u ? block % 8u * per_xcd + block / 8u : block;
}

// Keys of one tile as matrix operands: 16 tokens x 32 dimensions each.
template <int NK>
__device__ __forceinline__ void fetch_tile_keys(i32x4 (&k)[2][NK], const Attention& a,
                                                void* const* pages, uint32_t tile,
                                                uint32_t kv_head) {
  const uint32_t lane = threadIdx.x % kWave;
  const uint32_t key0 = tile * kTileKeys;
  const i32x4* keys = reinterpret_cast<const i32x4*>(
                          page_of<const uint16_t>(a, pages, key0) +
                          key_block(a, kv_head, key0 % a.page_tokens)) +
                      lane % 16u * 4u + lane / 16u;
#pragma unroll
  for (int half = 0; half < 2; ++half)
#pragma unroll
    for (int c = 0; c < NK; ++c) k[half][c] = keys[(half * NK + c) * kWave];
}

// s[half][i] = product of key 16 half + 4 quarter + i with query row column.
template <int NK>
__device__ __forceinline__ void tile_products(const i32x4 (&k)[2][NK],
                                              const i32x4 (&query)[NK], f32x4 (&s)[2]) {
#pragma unroll
  for (int half = 0; half < 2; ++half) {
    s[half] = f32x4{};
#pragma unroll
    for (int c = 0; c < NK; ++c) s[half] = mfma_bf16(k[half][c], query[c], s[half]);
  }
}

__device__ __forceinline__ void hide_keys(const Attention& a, uint32_t position,
                                          uint32_t tile, f32x4 (&s)[2]) {
  const uint32_t key0 = tile * kTileKeys + 4u * (threadIdx.x % kWave / 16u);
#pragma unroll
  for (int half = 0; half < 2; ++half)
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (!visible(a, position, key0 + half * 16u + i)) s[half][i] = -INFINITY;
}

// Rows first .. first + 15 all see every key of the tile.
__device__ __forceinline__ bool tile_open(const Attention& a, uint32_t first,
                                          uint32_t tile) {
  const uint32_t first_key = tile * kTileKeys;
  const uint32_t last_key = first_key + kTileKeys - 1u;
  return last_key <= first &&
         (!a.window || first + 15u - first_key < a.window || last_key < a.sinks);
}

template <int NK>
__device__ __forceinline__ void load_query(i32x4 (&q)[NK], const AttentionArgs& args,
                                           uint32_t row, uint32_t head) {
  const Attention& a = args.attention;
  const uint16_t* query = static_cast<const uint16_t*>(args.launch.query) +
                          (size_t{row} * a.query_heads + head) * a.key_stride +
                          8u * (threadIdx.x % kWave / 16u);
#pragma unroll
  for (int c = 0; c < NK; ++c) q[c] = *reinterpret_cast<const i32x4*>(query + c * 32);
}

// First walk: for every row and head the logarithm of the softmax denominator,
// in units of the base-2 exponent (maximum + log2 of the sum), so that
// exp2(score - it) is the normalised weight.  A workgroup owns 16 rows and up
// to HP heads of one key/value head; its waves deal the tiles among them.
template <int HP, int NK>
__global__ __launch_bounds__(256, 2) void prompt_denominators_kernel(AttentionArgs args) {
  __shared__ float wave_maximum[4][HP][16];
  __shared__ float wave_total[4][HP][16];
  const Attention& a = args.attention;
  const auto& run = args.launch;
  const uint32_t heads = a.query_heads;
  const uint32_t group = heads / a.kv_heads;
  const uint32_t wave = threadIdx.x / kWave;
  const uint32_t lane = threadIdx.x % kWave;
  const uint32_t column = lane % 16u;
  const uint32_t row0 = xcd_range(blockIdx.x, gridDim.x) * 16u;
  const uint32_t kv = blockIdx.y;
  const uint32_t head0 = kv * group + blockIdx.z * HP;
  const uint32_t count = min(uint32_t{HP}, group - blockIdx.z * HP);
  const uint32_t first = a.step[kStepPosition] + row0;
  const uint32_t position = first + column;
  const uint32_t last = first + min(16u, run.rows - row0) - 1u;
  const TileRange range = tiles_for(a, first, last);
  void* const* const pages = pages_of(a);
  const float unit = a.scale * 1.4426950408889634f;

  i32x4 q[HP][NK];
#pragma unroll
  for (int i = 0; i < HP; ++i)
    load_query<NK>(q[i], args, min(row0 + column, run.rows - 1u),
                   head0 + min(static_cast<uint32_t>(i), count - 1u));
  float maximum[HP], total[HP];
#pragma unroll
  for (int i = 0; i < HP; ++i) {
    maximum[i] = -INFINITY;
    total[i] = 0.0f;
  }
  const auto survey = [&](i32x4 (&k)[2][NK], uint32_t ordinal) __attribute__((always_inline)) {
    const uint32_t tile = range.tile(ordinal);
    const bool all = tile_open(a, first, tile);
    f32x4 s[HP][2];
#pragma unroll
    for (int i = 0; i < HP; ++i) tile_products<NK>(k, q[i], s[i]);
    fetch_tile_keys<NK>(k, a, pages, range.tile(min(ordinal + 8u, range.count - 1u)), kv);
#pragma unroll
    for (int i = 0; i < HP; ++i) {
#pragma unroll
      for (int half = 0; half < 2; ++half) s[i][half] *= unit;
      if (!all) hide_keys(a, position, tile, s[i]);
      float top = maximum[i];
#pragma unroll
      for (int half = 0; half < 2; ++half)
#pragma unroll
        for (int j = 0; j < 4; ++j) top = fmaxf(top, s[i][half][j]);
      // a row that has seen nothing yet: keep the exponents' argument finite
      const float base = top == -INFINITY ? 0.0f : top;
      float sum = total[i] * __builtin_amdgcn_exp2f(maximum[i] - base);
#pragma unroll
      for (int half = 0; half < 2; ++half)
#pragma unroll
        for (int j = 0; j < 4; ++j) sum += __builtin_amdgcn_exp2f(s[i][half][j] - base);
      total[i] = sum;
      maximum[i] = top;
    }
  };
  if (wave < range.count) {
    i32x4 even[2][NK], odd[2][NK];
    fetch_tile_keys<NK>(even, a, pages, range.tile(wave), kv);
    fetch_tile_keys<NK>(odd, a, pages, range.tile(min(wave + 4u, range.count - 1u)), kv);
    uint32_t ordinal = wave;
    for (; ordinal + 4u < range.count; ordinal += 8u) {
      survey(even, ordinal);
      survey(odd, ordinal + 4u);
    }
    if (ordinal < range.count) survey(even, ordinal);
  }
  const auto merge = [](float& m, float& t, float other, float other_total) {
    const float top = fmaxf(m, other);
    const float base = top == -INFINITY ? 0.0f : top;
    t = t * __builtin_amdgcn_exp2f(m - base) +
        other_total * __builtin_amdgcn_exp2f(other - base);
    m = top;
  };
#pragma unroll
  for (int i = 0; i < HP; ++i) {
#pragma unroll
    for (int offset = 16; offset <= 32; offset *= 2)
      merge(maximum[i], total[i], __shfl_xor(maximum[i], offset, kWave),
            __shfl_xor(total[i], offset, kWave));
    if (lane < 16u) {
      wave_maximum[wave][i][lane] = maximum[i];
      wave_total[wave][i][lane] = total[i];
    }
  }
  __syncthreads();
  for (uint32_t i = threadIdx.x; i < 16u * count; i += blockDim.x) {
    const uint32_t row = row0 + i % 16u;
    if (row >= run.rows) continue;
    float m = wave_maximum[0][i / 16u][i % 16u];
    float t = wave_total[0][i / 16u][i % 16u];
    for (uint32_t other = 1; other < 4u; ++other)
      merge(m, t, wave_maximum[other][i / 16u][i % 16u], wave_total[other][i / 16u][i % 16u]);
    args.maxima[size_t{row} * heads + head0 + i / 16u] = m + log2f(t);
  }
}

// Second walk: HPW score heads and OPW output heads per wave (OPW <= HPW),
// NK = key_stride / 32, NV = value_stride / 16.
//
// Every wave leaves its heads' normalised weights of a tile in LDS, the waves
// mix them (four keys each) on the matrix cores, and every wave multiplies its
// output heads' mixed weights with their values.  With up to 16 heads the high
// and the low halves of the weights share one matrix operand - the mix matrix
// stands in it twice; with up to 32 they take one each, and two workgroups
// share the output heads of a row block (their accumulators would not fit the
// registers of one).  The wave's keys are fetched one tile ahead: their
// registers are free as soon as the tile's scores are out, and the fetch then
// has the rest of the iteration to arrive.
template <int HPW, int OPW, int NK, int NV, bool SHARED>
__global__ __launch_bounds__(512, 2) void prompt_attention_kernel(AttentionArgs args) {
  constexpr bool kFolded = HPW <= 2;
  constexpr int kMixHeads = kFolded ? 16 : 32;
  constexpr int kPairs = (HPW + 1) / 2;
  // normalised weights [key][query row][64 bytes of heads]
  __shared__ __attribute__((aligned(16))) uint8_t high[2][512 * 64];
  __shared__ __attribute__((aligned(16))) uint8_t low[kFolded ? 1 : 2][kFolded ? 16 : 512 * 64];
  // mixed weights [output head][query row][key]
  __shared__ __attribute__((aligned(16))) uint8_t mixed[2][16 * 16 * 64];
  constexpr uint32_t kLowSlot = kFolded ? 2u : 0u;
  const Attention& a = args.attention;
  const auto& run = args.launch;
  const uint32_t heads = a.query_heads;
  const uint32_t group = heads / a.kv_heads;
  const uint32_t wave = threadIdx.x / kWave;
  const uint32_t waves = blockDim.x / kWave;
  const uint32_t lane = threadIdx.x % kWave;
  const uint32_t column = lane % 16u;
  const uint32_t quarter = lane / 16u;
  const uint32_t row0 = xcd_range(blockIdx.x, gridDim.x) * 16u;
  const uint32_t first_output = blockIdx.y * 16u;      // of this workgroup's heads
  const uint32_t first = a.step[kStepPosition] + row0;
  const uint32_t position = first + column;            // of this lane's query row
  const uint32_t last = first + min(16u, run.rows - row0) - 1u;
  const TileRange range = tiles_for(a, first, last);
  void* const* const pages = pages_of(a);
  const float unit = a.scale * 1.4426950408889634f;

  for (uint32_t i = threadIdx.x; i < sizeof(high) / 16u; i += blockDim.x) {
    reinterpret_cast<i32x4*>(high)[i] = i32x4{};
    if (!kFolded) reinterpret_cast<i32x4*>(low)[i] = i32x4{};
  }

  uint32_t kv[HPW], value_kv[OPW];
  i32x4 q[HPW][NK];
  float denominator[HPW];
  const uint32_t query_row = min(row0 + column, run.rows - 1u);
#pragma unroll
  for (int i = 0; i < HPW; ++i) {
    const uint32_t head = min(wave * HPW + i, heads - 1u);
    kv[i] = head / group;
    load_query<NK>(q[i], args, query_row, head);
    denominator[i] = args.maxima[size_t{query_row} * heads + head];
  }
#pragma unroll
  for (int i = 0; i < OPW; ++i)
    value_kv[i] = min(first_output + wave * OPW + i, heads - 1u) / group;
  // rows output head, columns head of the mix matrix
  i32x4 mix;
  {
    uint32_t packed[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      float pair[2];
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        const uint32_t h = first_output + column;
        const uint32_t g = (8u * quarter + 2u * i + j) % kMixHeads;
        const float stored =
            a.head_mix ? a.head_mix[size_t{min(h, heads - 1u)} * heads + min(g, heads - 1u)]
                       : (h == g ? 1.0f : 0.0f);
        pair[j] = h < heads && g < heads ? stored : 0.0f;
      }
      packed[i] = pack_bf16(pair[0], pair[1]);
    }
    mix = i32x4{static_cast<int>(packed[0]), static_cast<int>(packed[1]),
                static_cast<int>(packed[2]), static_cast<int>(packed[3])};
  }
  __syncthreads();   // the weight buffers are clear

  f32x4 out[OPW][NV] = {};
  i32x4 k[2][NK];
  fetch_tile_keys<NK>(k, a, pages, range.tile(0u), kv[0]);

  // weights of a tile into its buffer; the keys of the next one on their way
  const auto weigh = [&](uint32_t ordinal) __attribute__((always_inline)) {
    const uint32_t tile = range.tile(ordinal);
    const bool all = tile_open(a, first, tile);
    uint8_t* const upper_plane = high[ordinal & 1u];
    uint8_t* const lower_plane = kFolded ? upper_plane : low[kFolded ? 0u : ordinal & 1u];
#pragma unroll
    for (int pair = 0; pair < kPairs; ++pair) {
      f32x4 s[2][2];
#pragma unroll
      for (int j = 0; j < 2 && 2 * pair + j < HPW; ++j) {
        const int i = 2 * pair + j;
        if (!SHARED && i > 0 && kv[i] != kv[i - 1])
          fetch_tile_keys<NK>(k, a, pages, tile, kv[i]);
        tile_products<NK>(k, q[i], s[j]);
      }
      if (pair + 1 == kPairs)
        fetch_tile_keys<NK>(k, a, pages, range.tile(min(ordinal + 1u, range.count - 1u)),
                            kv[0]);
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        if (2 * pair + j >= HPW) {
          s[j][0] = s[j][1] = f32x4{};
          continue;
        }
        const float offset = denominator[2 * pair + j];
#pragma unroll
        for (int e = 0; e < 8; ++e)
          s[j][e / 4][e % 4] = fmaf(s[j][e / 4][e % 4], unit, -offset);
        if (!all) hide_keys(a, position, tile, s[j]);
#pragma unroll
        for (int e = 0; e < 8; ++e)
          s[j][e / 4][e % 4] = __builtin_amdgcn_exp2f(s[j][e / 4][e % 4]);
      }
      const uint32_t g = wave * HPW + 2u * pair;
      if (g < heads) {
        const bool second = HPW > 1 && g + 1u < heads;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const uint32_t row = (e / 4 * 16u + 4u * quarter + e % 4) * 16u + column;
          uint32_t upper, lower;
          split_pair(s[0][e / 4][e % 4], second ? s[1][e / 4][e % 4] : 0.0f, upper, lower);
          uint8_t* const upper_at = upper_plane + swizzled(row, g / 8u) + g % 8u * 2u;
          uint8_t* const lower_at = lower_plane + swizzled(row, kLowSlot + g / 8u) + g % 8u * 2u;
          if constexpr (HPW == 1) {
            *reinterpret_cast<uint16_t*>(upper_at) = static_cast<uint16_t>(upper);
            *reinterpret_cast<uint16_t*>(lower_at) = static_cast<uint16_t>(lower);
          } else {
            *reinterpret_cast<uint32_t*>(upper_at) = upper;
            *reinterpret_cast<uint32_t*>(lower_at) = lower;
          }
        }
      }
    }
  };
  // mix: four keys at a time, all query rows, this workgroup's output heads
  const auto blend = [&](uint32_t ordinal) __attribute__((always_inline)) {
    const uint8_t* const upper_plane = high[ordinal & 1u];
    const uint8_t* const lower_plane = low[kFolded ? 0u : ordinal & 1u];
    uint8_t* const target = mixed[ordinal & 1u];
    for (uint32_t four = wave; four < 8u; four += waves) {
      f32x4 m[4] = {};
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const uint32_t at = swizzled((four * 4u + j) * 16u + column, quarter);
        if constexpr (!kFolded)
          m[j] = mfma_bf16(mix, *reinterpret_cast<const i32x4*>(lower_plane + at), m[j]);
        m[j] = mfma_bf16(mix, *reinterpret_cast<const i32x4*>(upper_plane + at), m[j]);
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)
        *reinterpret_cast<i32x2*>(target + (4u * quarter + i) * 1024u +
                                  swizzled(column, four / 2u) + four % 2u * 8u) =
            i32x2{static_cast<int>(pack_bf16(m[0][i], m[1][i])),
                  static_cast<int>(pack_bf16(m[2][i], m[3][i]))};
    }
  };
  const auto values_at = [&](uint32_t tile, uint32_t kv_head) __attribute__((always_inline)) {
    const uint32_t key0 = tile * kTileKeys;
    return reinterpret_cast<const i32x4*>(page_of<const uint16_t>(a, pages, key0) +
                                          value_block(a, kv_head, key0 % a.page_tokens)) +
           column * 4u + quarter;
  };

  // Three tiles are under way between two barriers: the weights of one, the
  // mix of the one before, the values of the one before that.
  weigh(0u);
  __syncthreads();
  blend(0u);
  if (range.count > 1u) weigh(1u);
  __syncthreads();
  for (uint32_t ordinal = 0; ordinal < range.count; ++ordinal) {
    const uint32_t tile = range.tile(ordinal);
    i32x4 v[NV];
    const i32x4* const values = values_at(tile, value_kv[0]);
    const auto load_values = [&]() __attribute__((always_inline)) {
#pragma unroll
      for (int t = 0; t < NV; ++t) v[t] = values[t * kWave];
    };
    // the values early, where registers hold them across the other two stages
    if constexpr (kFolded) {
      load_values();
      if (ordinal + 1u < range.count) blend(ordinal + 1u);
      if (ordinal + 2u < range.count) weigh(ordinal + 2u);
    } else {
      if (ordinal + 2u < range.count) weigh(ordinal + 2u);
      __builtin_amdgcn_sched_barrier(0);
      load_values();
      if (ordinal + 1u < range.count) blend(ordinal + 1u);
    }
#pragma unroll
    for (int i = 0; i < OPW; ++i) {
      const uint32_t at = wave * OPW + i;
      const i32x4 w = *reinterpret_cast<const i32x4*>(
          mixed[ordinal & 1u] + min(at, 15u) * 1024u + swizzled(column, quarter));
      if (!SHARED && i > 0 && value_kv[i] != value_kv[i - 1]) {
        const i32x4* const other = values_at(tile, value_kv[i]);
#pragma unroll
        for (int t = 0; t < NV; ++t) v[t] = other[t * kWave];
      }
#pragma unroll
      for (int t = 0; t < NV; ++t) out[i][t] = mfma_bf16(w, v[t], out[i][t]);
    }
    __syncthreads();
  }

  float gate[OPW][4];
#pragma unroll
  for (int i = 0; i < OPW; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const uint32_t row = min(row0 + 4u * quarter + j, run.rows - 1u);
      const uint32_t head = min(first_output + wave * OPW + i, heads - 1u);
      gate[i][j] = run.gate ? run.gate[size_t{row} * run.gate_stride + head] : 0.0f;
    }
#pragma unroll
  for (int i = 0; i < OPW; ++i) {
    const uint32_t head = first_output + wave * OPW + i;
    if (wave * OPW + i >= 16u || head >= heads) continue;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const uint32_t row = row0 + 4u * quarter + j;
      if (row >= run.rows) continue;
      const float open_gate = run.gate ? sigmoid_f32(gate[i][j]) : 1.0f;
      uint16_t* const output = static_cast<uint16_t*>(run.output) +
                               size_t{row} * run.output_stride + head * a.vdim;
#pragma unroll
      for (int t = 0; t < NV; ++t) {
        const uint32_t d = t * 16u + column;
        if (d < a.vdim) store_element(output + d, out[i][t][j] * open_gate);
      }
    }
  }
}

template <int NK>
void launch_denominators(const AttentionArgs& args, hipStream_t stream) {
  const Attention& a = args.attention;
  const uint32_t group = a.query_heads / a.kv_heads;
  const uint32_t blocks = (args.launch.rows + 15u) / 16u;
  if (group == 1u)
    prompt_denominators_kernel<1, NK><<<dim3(blocks, a.kv_heads), 256, 0, stream>>>(args);
  else if (group == 2u)
    prompt_denominators_kernel<2, NK><<<dim3(blocks, a.kv_heads), 256, 0, stream>>>(args);
  else
    prompt_denominators_kernel<4, NK>
        <<<dim3(blocks, a.kv_heads, (group + 3u) / 4u), 256, 0, stream>>>(args);
}

template <int HPW, int OPW, int NK, int NV>
void launch_prompt_form(const AttentionArgs& args, hipStream_t stream) {
  const uint32_t heads = args.attention.query_heads;
  const uint32_t group = heads / args.attention.kv_heads;
  const uint32_t waves = HPW == 4 ? 8u : (heads + HPW - 1u) / HPW;
  const dim3 grid((args.launch.rows + 15u) / 16u, HPW == 4 ? 2u : 1u);
  // a wave's heads read one key/value head unless the groups are cut unevenly
  if (HPW == 1 || group % HPW == 0u)
    prompt_attention_kernel<HPW, OPW, NK, NV, true>
        <<<grid, waves * kWave, 0, stream>>>(args);
  else
    prompt_attention_kernel<HPW, OPW, NK, NV, HPW == 1>
        <<<grid, waves * kWave, 0, stream>>>(args);
}

template <int HPW, int OPW>
void launch_prompt(const AttentionArgs& args, hipStream_t stream) {
  const bool narrow_keys = args.attention.key_stride == 64u;
  const bool narrow_values = args.attention.value_stride == 64u;
  if (narrow_keys)
    launch_denominators<2>(args, stream);
  else
    launch_denominators<4>(args, stream);
  if (narrow_keys && narrow_values)
    launch_prompt_form<HPW, OPW, 2, 4>(args, stream);
  else if (narrow_keys)
    launch_prompt_form<HPW, OPW, 2, 8>(args, stream);
  else if (narrow_values)
    launch_prompt_form<HPW, OPW, 4, 4>(args, stream);
  else
    launch_prompt_form<HPW, OPW, 4, 8>(args, stream);
}

bool valid_geometry(const Attention& a) {
  return a.query_heads && a.kv_heads && a.query_heads % a.kv_heads == 0u && a.dim &&
         a.vdim && a.dim <= a.key_stride && a.vdim <= a.value_stride &&
         a.key_stride % 32u == 0u && a.value_stride % 16u == 0u && a.page_tokens &&
         a.page_tokens % 32u == 0u && a.layer_offset % 16u == 0u && a.page_table && a.step &&
         a.pages_per_slot && a.element <= QLLM_ELEMENT_F32;
}

// Most tiles a row at or below maximum_position sees.
uint32_t maximum_tiles(const Attention& a, uint32_t maximum_position) {
  const uint64_t all = maximum_position / kTileKeys + 1u;
  if (!a.window) return static_cast<uint32_t>(all);
  const uint64_t seen = (uint64_t{a.sinks} + kTileKeys - 1u) / kTileKeys +
                        (uint64_t{a.window} + kTileKeys - 1u) / kTileKeys + 1u;
  return static_cast<uint32_t>(seen < all ? seen : all);
}

uint32_t score_splits_for(uint32_t tiles) {
  const uint32_t wanted = (tiles * 2u + 3u) / 4u;
  return wanted < kMaximumScoreSplits ? wanted : kMaximumScoreSplits;
}

uint32_t value_splits_for(uint32_t tiles) {
  const uint32_t wanted = (tiles + 3u) / 4u;
  return wanted < kMaximumValueSplits ? wanted : kMaximumValueSplits;
}

size_t general_bytes(const Attention& a) {
  return size_t{a.query_heads} * (a.dim + 2u * kTileKeys + a.vdim + 2u) * 4u;
}

bool split_stride(uint32_t stride) {
  return stride == 64u || stride == 128u || stride == 256u;
}

}  // namespace
}  // namespace qllm

using namespace qllm;

extern "C" size_t qllm_windowed_layer_bytes(uint32_t page_tokens, uint32_t kv_heads,
                                            uint32_t key_stride, uint32_t value_stride,
                                            uint32_t element) {
  return size_t{page_tokens} * kv_heads * (key_stride + value_stride) *
         (element == QLLM_ELEMENT_F32 ? 4u : 2u);
}

extern "C" int32_t qllm_windowed_rope_store(const qllm_windowed_attention* attention,
                                            const qllm_rope_store_launch* launch,
                                            void* stream) {
  if (!attention || !launch || !valid_geometry(*attention) || !launch->projections ||
      !launch->query_out || !launch->rows || launch->rotary_dims % 2u ||
      launch->rotary_dims > attention->dim ||
      (launch->rotary_dims && !launch->frequencies) ||
      (launch->first_values && !launch->value_share) ||
      launch->query_column + attention->query_heads * attention->dim > launch->stride ||
      launch->key_column + attention->kv_heads * attention->dim > launch->stride ||
      launch->value_column + attention->kv_heads * attention->vdim > launch->stride)
    return fail(QLLM_INVALID_ARGUMENT, "invalid windowed rotary store");
  RopeArgs args{*attention, *launch, launch->rows > 64u ? 8u : 1u};
  const uint32_t units = attention->query_heads + 2u * attention->kv_heads;
  const dim3 grid((launch->rows + args.rows_per_block - 1u) / args.rows_per_block,
                  (units + 3u) / 4u);
  if (attention->element == QLLM_ELEMENT_F32)
    rope_store_kernel<float><<<grid, 256, 0, as_stream(stream)>>>(args);
  else
    rope_store_kernel<uint16_t><<<grid, 256, 0, as_stream(stream)>>>(args);
  return launched("windowed rotary store");
}

extern "C" uint32_t qllm_windowed_attention_form(const qllm_windowed_attention* attention,
                                                 uint32_t rows) {
  if (!attention || attention->element != QLLM_ELEMENT_BF16 ||
      !split_stride(attention->key_stride) || !split_stride(attention->value_stride))
    return QLLM_ATTENTION_GENERAL;
  if (rows <= kSplitRows)
    return attention->query_heads <= 64u &&
                   attention->query_heads / attention->kv_heads <= 16u
               ? QLLM_ATTENTION_SPLIT
               : QLLM_ATTENTION_GENERAL;
  return attention->query_heads <= kPromptHeads && attention->key_stride <= 128u &&
                 attention->value_stride <= 128u
             ? QLLM_ATTENTION_PROMPT
             : QLLM_ATTENTION_GENERAL;
}

extern "C" size_t qllm_windowed_attention_workspace_bytes(
    const qllm_windowed_attention* attention, uint32_t rows, uint32_t maximum_position) {
  if (!attention || !attention->kv_heads || !attention->query_heads) return 0u;
  const uint32_t tiles = maximum_tiles(*attention, maximum_position);
  const size_t heads = attention->query_heads;
  const size_t split = kSplitRows * heads * 4u *
                       (size_t{tiles} * kTileKeys + size_t{score_splits_for(tiles)} * 2u +
                        size_t{value_splits_for(tiles)} * attention->vdim);
  const size_t prompt = size_t{rows} * heads * 4u;   // denominators
  return split > prompt ? split : prompt;
}

extern "C" int32_t qllm_windowed_attention_rows(const qllm_windowed_attention* attention,
                                                const qllm_attention_launch* launch,
                                                void* stream) {
  if (!attention || !launch || !valid_geometry(*attention) || !launch->query ||
      !launch->output || !launch->rows ||
      launch->output_stride < attention->query_heads * attention->vdim)
    return fail(QLLM_INVALID_ARGUMENT, "invalid windowed attention");
  const auto hip_stream = as_stream(stream);
  const Attention& a = *attention;
  AttentionArgs args{a, *launch, nullptr, nullptr, nullptr, 0u, 0u, 0u};
  const uint32_t form = qllm_windowed_attention_form(attention, launch->rows);
  if (form == QLLM_ATTENTION_GENERAL) {
    if (general_bytes(a) > kMaximumLds)
      return fail(QLLM_INVALID_ARGUMENT,
                  "windowed attention: heads and dimensions exceed the general kernel");
    if (general_bytes(a) > 65536u) {
      const void* kernel = a.element == QLLM_ELEMENT_F32
                               ? reinterpret_cast<const void*>(general_attention_kernel<float>)
                               : reinterpret_cast<const void*>(
                                     general_attention_kernel<uint16_t>);
      const auto raised = hipFuncSetAttribute(
          kernel, hipFuncAttributeMaxDynamicSharedMemorySize, kMaximumLds);
      if (raised != hipSuccess) return checked(raised, "windowed attention LDS");
    }
    if (a.element == QLLM_ELEMENT_F32)
      general_attention_kernel<float>
          <<<launch->rows, 256, general_bytes(a), hip_stream>>>(args);
    else
      general_attention_kernel<uint16_t>
          <<<launch->rows, 256, general_bytes(a), hip_stream>>>(args);
    return launched("windowed attention");
  }
  if (form == QLLM_ATTENTION_PROMPT) {
    if (!launch->workspace ||
        launch->workspace_bytes < size_t{launch->rows} * a.query_heads * 4u)
      return fail(QLLM_INVALID_ARGUMENT, "windowed attention workspace is too small");
    args.maxima = static_cast<float*>(launch->workspace);
    if (a.query_heads > 16u)
      launch_prompt<4, 2>(args, hip_stream);
    else if (a.query_heads > 8u)
      launch_prompt<2, 2>(args, hip_stream);
    else
      launch_prompt<1, 1>(args, hip_stream);
    return launched("windowed prompt attention");
  }
  if (!launch->workspace || (reinterpret_cast<uintptr_t>(launch->workspace) & 15u) != 0u ||
      launch->workspace_bytes <
          qllm_windowed_attention_workspace_bytes(attention, launch->rows,
                                                  launch->maximum_position))
    return fail(QLLM_INVALID_ARGUMENT, "windowed attention workspace is too small");
  const uint32_t tiles = maximum_tiles(a, launch->maximum_position);
  args.capacity = tiles * kTileKeys;
  args.score_splits = score_splits_for(tiles);
  args.value_splits = value_splits_for(tiles);
  args.scores = static_cast<float*>(launch->workspace);
  args.maxima = args.scores + size_t{launch->rows} * a.query_heads * args.capacity;
  args.partials = args.maxima + size_t{launch->rows} * args.score_splits * a.query_heads * 2u;
  const dim3 score_grid(args.score_splits, a.kv_heads, launch->rows);
  if (a.key_stride == 64u)
    split_scores_kernel<2><<<score_grid, 256, 0, hip_stream>>>(args);
  else if (a.key_stride == 128u)
    split_scores_kernel<4><<<score_grid, 256, 0, hip_stream>>>(args);
  else
    split_scores_kernel<8><<<score_grid, 256, 0, hip_stream>>>(args);
  const dim3 value_grid(args.value_splits, a.kv_heads, launch->rows);
  const bool narrow = a.query_heads / a.kv_heads <= 4u;
  const auto values = [&](auto nv) {
    constexpr int NV = decltype(nv)::value;
    if (narrow)
      split_values_kernel<NV, 4><<<value_grid, 256, 0, hip_stream>>>(args);
    else
      split_values_kernel<NV, 16><<<value_grid, 256, 0, hip_stream>>>(args);
  };
  if (a.value_stride == 64u)
    values(std::integral_constant<int, 4>{});
  else if (a.value_stride == 128u)
    values(std::integral_constant<int, 8>{});
  else
    values(std::integral_constant<int, 16>{});
  split_combine_kernel<<<dim3(a.query_heads, launch->rows), 64, 0, hip_stream>>>(args);
  return launched("windowed split attention");
}
