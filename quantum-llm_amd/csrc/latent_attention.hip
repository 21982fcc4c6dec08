// Attention over a cached latent: a token's cache row is one normed latent and
// one rotated key part shared by all heads; keys and values are linear maps of
// the latent (include/qllm_kernels.h has the layout and the equations).
//
//  * split (few rows, decode): a head's query goes through its transposed key
//    map once, so scores are products with the cached latents themselves and
//    the softmax-weighted sum is a latent again; all heads read one cache row.
//    Sixteen (row, head) pairs are one matrix tile.  The tiles of 32 tokens are
//    dealt over workgroups; the four waves of a workgroup share a tile in LDS,
//    split the score product along the dimensions and the weighted sum by
//    columns, reading the tile transposed for it.  A last launch adds the parts
//    and takes the sums through the value map.
//  * prompt: keys and values of the visible context are expanded once into
//    operand fragments, then a workgroup owns 128 query rows of a head and
//    walks the tiles with a running maximum.  Queries lie along matrix columns
//    in both products, so weights go from the first to the second in registers
//    (the value fragments hold their tokens in the order that comes out).
//  * general: one workgroup per row and head, any size, bf16 or F32.
#include "mixed_common.hpp"

#include <cmath>

namespace qllm {
namespace {

constexpr uint32_t kTile = 32;               // tokens
constexpr uint32_t kFragment = 512;          // elements, 16 x 32
constexpr uint32_t kSplitRows = 32;          // rows of the split form
constexpr uint32_t kMaximumSplits = 128;      // two for a lane when the parts are added
constexpr uint32_t kSplitsFirst = 64;         // of one tile each, before they take several
constexpr uint32_t kValueThreads = 1024;
constexpr float kLog2e = 1.4426950408889634f;

using Latent = qllm_latent_attention;

__host__ __device__ __forceinline__ uint32_t chunks_of(uint32_t size) {
  return (size + 31u) / 32u;
}
// Chunks of a cache row: latent, then shared key part.
__host__ __device__ __forceinline__ uint32_t row_chunks(const Latent& a) {
  return chunks_of(a.rank) + chunks_of(a.rot_dim);
}
// Columns of packed weights, in chunks of 32 (columns are padded to 64).
__host__ __device__ __forceinline__ uint32_t packed_chunks(uint32_t columns) {
  return (columns + 63u) / 64u * 2u;
}
__host__ __device__ __forceinline__ uint32_t value_tiles(const Latent& a) {
  return (a.vdim + 15u) / 16u;
}

// Element offset in a fragment.
__device__ __forceinline__ uint32_t in_fragment(uint32_t row, uint32_t column) {
  return (column / 8u * 16u + row) * 8u + column % 8u;
}

__device__ __forceinline__ uint32_t first_tile(const Latent& a, uint32_t position) {
  return a.window && position + 1u > a.window ? (position + 1u - a.window) / kTile : 0u;
}

__device__ __forceinline__ bool visible(const Latent& a, uint32_t position, uint32_t key) {
  return key <= position && (!a.window || position - key < a.window);
}

// The request's row of the page table, and the fragments of the 16 tokens that
// start at `token`.
__device__ __forceinline__ void* const* pages_of(const Latent& a) {
  return a.page_table + size_t{a.step[kStepSlot]} * a.pages_per_slot;
}
template <typename T>
__device__ __forceinline__ T* cache_block(const Latent& a, void* const* pages,
                                          uint32_t token) {
  void* const page = pages[token / a.page_tokens];
  return reinterpret_cast<T*>(static_cast<uint8_t*>(page) + a.layer_offset) +
         size_t{token % a.page_tokens / 16u} * row_chunks(a) * kFragment;
}
template <typename T>
__device__ __forceinline__ T* cache_block(const Latent& a, uint32_t token) {
  return cache_block<T>(a, pages_of(a), token);
}

// Pieces of a page for operand loads.  A pointer read from memory could point
// anywhere; said to be global, its loads count on their own and complete in order.
typedef const __attribute__((address_space(1))) i32x4 global_piece;
__device__ __forceinline__ global_piece* as_global(const void* pieces) {
  return (global_piece*)(pieces);
}

// Value d of a rotated vector x (its dimensions from rotary_dims on stay).
__device__ __forceinline__ float rotated(const Latent& a, const float* x, uint32_t d,
                                         uint32_t position) {
  if (d >= a.rotary_dims) return x[d];
  const uint32_t half = a.rotary_dims / 2u;
  const uint32_t pair = d < half ? d : d - half;
  // the angle is reduced to one turn before it becomes F32
  constexpr double kTurn = 6.283185307179586476925286766559;
  double angle = static_cast<double>(position) * a.frequencies[pair];
  angle -= kTurn * rint(angle / kTurn);
  float sine, cosine;
  sincosf(static_cast<float>(angle), &sine, &cosine);
  sine *= a.rotary_magnitude;
  cosine *= a.rotary_magnitude;
  const float u = x[pair];
  const float v = x[pair + half];
  return d < half ? u * cosine - v * sine : v * cosine + u * sine;
}

// ---- latents into the pages ------------------------------------------------------

struct StoreArgs {
  Latent attention;
  qllm_latent_store_launch launch;
};

// A workgroup per row and task: the cache row, or the query latent.
template <typename T>
__global__ __launch_bounds__(256) void latent_store_kernel(StoreArgs args) {
  __shared__ float scratch[16];
  const Latent& a = args.attention;
  const auto& run = args.launch;
  const uint32_t row = blockIdx.x;
  const bool query = blockIdx.y == 1u;
  const float* source = run.projections + size_t{row} * run.stride +
                        (query ? run.query_column : run.latent_column);
  const uint32_t rank = query ? run.query_rank : a.rank;
  const float* norm = query ? run.query_norm : a.latent_norm;
  constexpr uint32_t kHeld = 8;
  float held[kHeld], weight[kHeld];
  float squares = 0.0f;
#pragma unroll
  for (uint32_t i = 0; i < kHeld; ++i) {
    const uint32_t d = i * blockDim.x + threadIdx.x;
    held[i] = d < rank ? source[d] : 0.0f;
    weight[i] = d < rank ? norm[d] : 0.0f;
  }
  const uint32_t position = a.step[kStepPosition] + row;
  T* const block = cache_block<T>(a, position);
  const uint32_t n = position % 16u;
  if (!query) {
    // threads from the far end: the latent's own fall to the first ones
    const uint32_t d = blockDim.x - 1u - threadIdx.x;
    T* const shared = block + size_t{chunks_of(a.rank)} * kFragment;
    for (uint32_t at = d; at < chunks_of(a.rot_dim) * 32u; at += blockDim.x)
      store_element(shared + size_t{at / 32u} * kFragment + in_fragment(n, at % 32u),
                    at < a.rot_dim ? rotated(a, source + a.rank, at, position) : 0.0f);
  }
#pragma unroll
  for (uint32_t i = 0; i < kHeld; ++i) squares = fmaf(held[i], held[i], squares);
  for (uint32_t d = kHeld * blockDim.x + threadIdx.x; d < rank; d += blockDim.x)
    squares = fmaf(source[d], source[d], squares);
  const float inverse =
      1.0f / sqrtf(block_sum(squares, scratch) / static_cast<float>(rank) + a.epsilon);
  const auto put_all = [&](auto put, uint32_t padded) {
#pragma unroll
    for (uint32_t i = 0; i < kHeld; ++i) {
      const uint32_t d = i * blockDim.x + threadIdx.x;
      if (d < padded) put(d, held[i] * inverse * weight[i]);
    }
    for (uint32_t d = kHeld * blockDim.x + threadIdx.x; d < padded; d += blockDim.x)
      put(d, d < rank ? source[d] * inverse * norm[d] : 0.0f);
  };
  if (query) {
    T* out = static_cast<T*>(run.query_out) + size_t{row} * run.query_stride;
    put_all([&](uint32_t d, float value) { store_element(out + d, value); },
            run.query_stride);
  } else {
    put_all(
        [&](uint32_t d, float value) {
          store_element(block + size_t{d / 32u} * kFragment + in_fragment(n, d % 32u), value);
        },
        chunks_of(a.rank) * 32u);
  }
}

struct AttentionArgs {
  Latent attention;
  qllm_latent_launch launch;
  uint16_t* query;       // split: [row][head][row chunks * 32]; prompt: [row][head][chunks * 32]
  float* sums;           // split: [split][row * head][latent chunks * 32]
  float* maxima;         // split: [split][row * head] (maximum, total)
  uint16_t* keys;        // prompt: [head][tile][half][key chunks] fragments
  uint16_t* values;      // prompt: [head][tile][value tiles] fragments
  uint32_t splits;
  uint32_t tile0, tiles; // prompt: expanded tiles
};

__device__ __forceinline__ float gate_of(const qllm_latent_launch& run, uint32_t row,
                                         uint32_t column) {
  return run.gate ? sigmoid_f32(run.gate[size_t{row} * run.gate_stride + column]) : 1.0f;
}

// Rows of outputs and gates can be taken four values at a time.
__device__ __forceinline__ bool in_fours(const Latent& a, const qllm_latent_launch& run) {
  return (a.vdim | run.output_stride | run.gate_stride) % 4u == 0u &&
         (reinterpret_cast<uintptr_t>(run.gate) & 15u) == 0u &&
         (reinterpret_cast<uintptr_t>(run.output) & 7u) == 0u;
}

// Gates of N times four values of a head, the first four from n on, the others 16
// apart; no load depends on whether they exist.
template <int N>
__device__ __forceinline__ void take_gates(f32x4 (&gate)[N], const Latent& a,
                                           const qllm_latent_launch& run, uint32_t row,
                                           uint32_t head, uint32_t n) {
  if (!run.gate) {
#pragma unroll
    for (int t = 0; t < N; ++t) gate[t] = f32x4{1.0f, 1.0f, 1.0f, 1.0f};
    return;
  }
  const float* source = run.gate + size_t{row} * run.gate_stride + head * a.vdim;
  if (in_fours(a, run)) {
#pragma unroll
    for (int t = 0; t < N; ++t)
      gate[t] = *reinterpret_cast<const f32x4*>(source + min(n + t * 16u, a.vdim - 4u));
  } else {
#pragma unroll
    for (int t = 0; t < N; ++t)
#pragma unroll
      for (uint32_t i = 0; i < 4u; ++i)
        gate[t][i] = source[min(n + t * 16u + i, a.vdim - 1u)];
  }
#pragma unroll
  for (int t = 0; t < N; ++t)
#pragma unroll
    for (uint32_t i = 0; i < 4u; ++i) gate[t][i] = sigmoid_f32(gate[t][i]);
}

__device__ __forceinline__ void store_four(const Latent& a, const qllm_latent_launch& run,
                                           uint32_t row, uint32_t head, uint32_t n,
                                           f32x4 value) {
  if (n >= a.vdim) return;
  uint16_t* out = static_cast<uint16_t*>(run.output) + size_t{row} * run.output_stride +
                  head * a.vdim + n;
  if (in_fours(a, run)) {
    *reinterpret_cast<i32x2*>(out) =
        i32x2{static_cast<int>(pack_bf16(value[0], value[1])),
              static_cast<int>(pack_bf16(value[2], value[3]))};
  } else {
    for (uint32_t i = 0; i < 4u && n + i < a.vdim; ++i) store_element(out + i, value[i]);
  }
}

// ---- general form ----------------------------------------------------------------

template <typename T>
__global__ __launch_bounds__(256) void latent_general_kernel(AttentionArgs args) {
  extern __shared__ float shared[];
  const Latent& a = args.attention;
  const auto& run = args.launch;
  const uint32_t row = blockIdx.x;
  const uint32_t head = blockIdx.y;
  const uint32_t position = a.step[kStepPosition] + row;
  const uint32_t width = a.dim + a.rot_dim;
  float* query = shared;                     // [dim + rot_dim], rotated
  float* latent = query + width;             // [rank]: the query in latent space
  float* sum = latent + a.rank;              // [rank]
  float* scores = sum + a.rank;              // [32]
  const float* source = run.query + size_t{row} * run.query_stride + size_t{head} * width;
  for (uint32_t d = threadIdx.x; d < width; d += blockDim.x)
    query[d] = d < a.dim ? source[d] : rotated(a, source + a.dim, d - a.dim, position);
  __syncthreads();
  const uint32_t dim_chunks = packed_chunks(a.dim);
  const uint32_t rank_chunks = packed_chunks(a.rank);
  const auto* up = static_cast<const uint16_t*>(a.key_up_transposed) +
                   size_t{head} * chunks_of(a.rank) * 2u * dim_chunks * kFragment;
  for (uint32_t r = threadIdx.x; r < a.rank; r += blockDim.x) {
    float total = 0.0f;
    for (uint32_t d = 0; d < a.dim; ++d)
      total = fmaf(bf16_bits_to_f32(up[(size_t{r / 16u} * dim_chunks + d / 32u) * kFragment +
                                       in_fragment(r % 16u, d % 32u)]),
                   query[d], total);
    latent[r] = total;
    sum[r] = 0.0f;
  }
  __syncthreads();
  float maximum = -INFINITY;
  float total = 0.0f;
  const uint32_t chunks = row_chunks(a);
  for (uint32_t tile = first_tile(a, position); tile <= position / kTile; ++tile) {
    // eight threads per token
    const T* blocks = cache_block<T>(a, tile * kTile);
    const uint32_t token = threadIdx.x / 8u;
    const T* block = blocks + size_t{token / 16u} * chunks * kFragment;
    float score = 0.0f;
    for (uint32_t d = threadIdx.x % 8u; d < a.rank; d += 8u)
      score = fmaf(latent[d],
                   load_element(block + size_t{d / 32u} * kFragment +
                                in_fragment(token % 16u, d % 32u)),
                   score);
    const T* part = block + size_t{chunks_of(a.rank)} * kFragment;
    for (uint32_t d = threadIdx.x % 8u; d < a.rot_dim; d += 8u)
      score = fmaf(query[a.dim + d],
                   load_element(part + size_t{d / 32u} * kFragment +
                                in_fragment(token % 16u, d % 32u)),
                   score);
#pragma unroll
    for (int offset = 1; offset < 8; offset *= 2) score += __shfl_xor(score, offset, kWave);
    if (threadIdx.x % 8u == 0u)
      scores[token] = visible(a, position, tile * kTile + token) ? score * a.scale : -INFINITY;
    __syncthreads();
    float top = maximum;
    for (uint32_t j = 0; j < kTile; ++j) top = fmaxf(top, scores[j]);
    const float base = top == -INFINITY ? 0.0f : top;
    const float fade = expf(maximum - base);
    total *= fade;
    for (uint32_t j = 0; j < kTile; ++j) total += expf(scores[j] - base);
    for (uint32_t r = threadIdx.x; r < a.rank; r += blockDim.x) {
      float value = sum[r] * fade;
      for (uint32_t j = 0; j < kTile; ++j)
        value = fmaf(expf(scores[j] - base),
                     load_element(blocks + (size_t{j / 16u} * chunks + r / 32u) * kFragment +
                                  in_fragment(j % 16u, r % 32u)),
                     value);
      sum[r] = value;
    }
    maximum = top;
    __syncthreads();
  }
  const auto* value_up = static_cast<const uint16_t*>(a.value_up) +
                         size_t{head} * value_tiles(a) * rank_chunks * kFragment;
  for (uint32_t n = threadIdx.x; n < a.vdim; n += blockDim.x) {
    float value = 0.0f;
    for (uint32_t r = 0; r < a.rank; ++r)
      value = fmaf(bf16_bits_to_f32(value_up[(size_t{n / 16u} * rank_chunks + r / 32u) *
                                                 kFragment +
                                             in_fragment(n % 16u, r % 32u)]),
                   sum[r], value);
    const uint32_t column = head * a.vdim + n;
    store_element(static_cast<T*>(run.output) + size_t{row} * run.output_stride + column,
                  value / total * gate_of(run, row, column));
  }
}

// ---- queries -----------------------------------------------------------------------

// Eight query values as a matrix operand, zeros from `end` on.
__device__ __forceinline__ i32x4 query_operand(const float* source, uint32_t d, uint32_t end) {
  uint32_t packed[4];
#pragma unroll
  for (uint32_t i = 0; i < 4u; ++i)
    packed[i] = pack_bf16(d + 2u * i < end ? source[d + 2u * i] : 0.0f,
                          d + 2u * i + 1u < end ? source[d + 2u * i + 1u] : 0.0f);
  return i32x4{static_cast<int>(packed[0]), static_cast<int>(packed[1]),
               static_cast<int>(packed[2]), static_cast<int>(packed[3])};
}

// Split form: the queries of 16 rows and one head through the transposed key
// map (a wave per 16 latent values), or, in the last workgroup along x, their
// rotated parts.
__global__ __launch_bounds__(256) void latent_query_kernel(AttentionArgs args) {
  const Latent& a = args.attention;
  const auto& run = args.launch;
  const uint32_t head = blockIdx.y;
  const uint32_t row0 = blockIdx.z * 16u;
  const uint32_t rows = min(16u, run.rows - row0);
  const uint32_t width = a.dim + a.rot_dim;
  const uint32_t stride = row_chunks(a) * 32u;
  const uint32_t latent_chunks = chunks_of(a.rank);
  const uint32_t tiles = latent_chunks * 2u;
  const float* source = run.query + size_t{row0} * run.query_stride + size_t{head} * width;
  uint16_t* out = args.query + (size_t{row0} * a.heads + head) * stride;
  const size_t out_row = size_t{a.heads} * stride;
  if (blockIdx.x * 4u >= tiles) {
    const uint32_t padded = chunks_of(a.rot_dim) * 32u;
    const uint32_t first = a.step[kStepPosition] + row0;
    for (uint32_t i = threadIdx.x; i < rows * padded; i += blockDim.x) {
      const uint32_t row = i / padded;
      const uint32_t d = i % padded;
      const float value = d < a.rot_dim ? rotated(a, source + size_t{row} * run.query_stride + a.dim,
                                                  d, first + row)
                                        : 0.0f;
      store_element(out + row * out_row + latent_chunks * 32u + d, value);
    }
    return;
  }
  const uint32_t tile = blockIdx.x * 4u + threadIdx.x / kWave;
  if (tile >= tiles) return;
  const uint32_t lane = threadIdx.x % kWave;
  const uint32_t column = lane % 16u;
  const uint32_t quarter = lane / 16u;
  const uint32_t chunks = packed_chunks(a.dim);
  const i32x4* weights = static_cast<const i32x4*>(a.key_up_transposed) +
                         (size_t{head} * tiles + tile) * chunks * kWave + lane;
  const float* q = source + size_t{min(column, rows - 1u)} * run.query_stride;
  f32x4 sum = {};
  for (uint32_t c = 0; c < chunks_of(a.dim); ++c)
    sum = mfma_bf16(weights[c * kWave], query_operand(q, c * 32u + 8u * quarter, a.dim), sum);
  if (column < rows)
    *reinterpret_cast<i32x2*>(out + column * out_row + tile * 16u + 4u * quarter) =
        i32x2{static_cast<int>(pack_bf16(sum[0], sum[1])),
              static_cast<int>(pack_bf16(sum[2], sum[3]))};
}

// Prompt form: queries rounded, their rotated part turned, each part padded to
// 32 with zeros.  A wave per row and head.
__global__ __launch_bounds__(256) void latent_prompt_query_kernel(AttentionArgs args) {
  const Latent& a = args.attention;
  const auto& run = args.launch;
  const uint32_t item = blockIdx.x * 4u + threadIdx.x / kWave;
  if (item >= run.rows * a.heads) return;
  const uint32_t row = item / a.heads;
  const uint32_t head = item % a.heads;
  const uint32_t lane = threadIdx.x % kWave;
  const uint32_t width = a.dim + a.rot_dim;
  const uint32_t plain = chunks_of(a.dim) * 32u;
  const uint32_t padded = plain + chunks_of(a.rot_dim) * 32u;
  const float* source = run.query + size_t{row} * run.query_stride + size_t{head} * width;
  uint16_t* out = args.query + size_t{item} * padded;
  const uint32_t position = a.step[kStepPosition] + row;
  const auto value = [&](uint32_t d) {
    if (d < a.dim) return source[d];
    return d >= plain && d - plain < a.rot_dim ? rotated(a, source + a.dim, d - plain, position)
                                               : 0.0f;
  };
  for (uint32_t d = 2u * lane; d < padded; d += 2u * kWave)
    *reinterpret_cast<uint32_t*>(out + d) = pack_bf16(value(d), value(d + 1u));
}

// ---- split form --------------------------------------------------------------------

__device__ __forceinline__ i32x2 read_transposed(const uint16_t* at) {
  typedef __attribute__((ext_vector_type(4))) short s16x4;
  return __builtin_bit_cast(
      i32x2, __builtin_amdgcn_ds_read_tr16_b64_v4i16(
                 (__attribute__((address_space(3))) s16x4*)(at)));
}

// Lane 16 g + i of a group of sixteen lanes takes part in a transposed read with
// the address of token i / 4, dimensions 4 (i % 4) .. + 3, and gets dimension i
// of the four tokens.
//
// R: latents of up to 64 R values, shared key parts of up to 64.
template <int R>
__global__ __launch_bounds__(256) void latent_split_kernel(AttentionArgs args) {
  constexpr int kChunks = 2 * R + 2;                 // at most
  constexpr int kQuery = (kChunks + 3) / 4;          // chunks per wave
  constexpr int kLoads = (kChunks + 1) / 2;          // 16-byte pieces per thread and tile
  __shared__ __attribute__((aligned(16))) uint16_t tile[2 * kChunks * kFragment];
  __shared__ f32x4 parts[4][2][kWave];
  static_assert(kLoads * 256 == 2 * kChunks * kWave);
  const Latent& a = args.attention;
  const uint32_t wave = __builtin_amdgcn_readfirstlane(threadIdx.x / kWave);
  const uint32_t lane = threadIdx.x % kWave;
  const uint32_t quarter = lane / 16u;
  const uint32_t items = args.launch.rows * a.heads;
  const uint32_t item = blockIdx.y * 16u + lane % 16u;
  const uint32_t first_position = a.step[kStepPosition];
  const uint32_t position = first_position + min(item, items - 1u) / a.heads;
  const uint32_t latent_chunks = chunks_of(a.rank);
  const uint32_t chunks = row_chunks(a);

  const uint32_t low = first_position + blockIdx.y * 16u / a.heads;
  const uint32_t high =
      first_position + min(blockIdx.y * 16u + 15u, items - 1u) / a.heads;
  const uint32_t begin = first_tile(a, low);
  const uint32_t end = high / kTile + 1u;

  // No load or matrix product below depends on a condition - places past the end
  // are clamped to one that exists - so that a wait for one tile's loads leaves the
  // next one's in flight.  Chunks of the query past the last one are zero.
  i32x4 q[kQuery];
  uint32_t key_at[kQuery];
  const uint16_t* query =
      args.query + size_t{min(item, items - 1u)} * chunks * 32u + 8u * quarter;
#pragma unroll
  for (int i = 0; i < kQuery; ++i) {
    const uint32_t c = min(wave + 4u * i, chunks - 1u);
    const i32x4 stored = *reinterpret_cast<const i32x4*>(query + c * 32u);
    q[i] = wave + 4u * i < chunks ? stored : i32x4{};
    key_at[i] = c * kWave + lane;
  }
  void* const* const pages = pages_of(a);
  const uint32_t last_piece = 2u * chunks * kWave - 1u;
  const auto page_for = [&](uint32_t t) {
    return as_global(cache_block<const uint16_t>(a, pages, min(t, end - 1u) * kTile));
  };
  global_piece* ahead = page_for(begin + blockIdx.x);   // of the next fetch
  const auto fetch = [&](i32x4 (&staged)[kLoads], uint32_t t) __attribute__((always_inline)) {
    global_piece* const source = ahead;
    ahead = page_for(t + gridDim.x);
#pragma unroll
    for (int i = 0; i < kLoads; ++i)
      staged[i] = source[min(i * 256u + threadIdx.x, last_piece)];
    __builtin_amdgcn_sched_barrier(0);   // in this order
  };
  const float unit = a.scale * kLog2e;
  float maximum = -INFINITY;
  float total = 0.0f;
  f32x4 sum[R] = {};
  // `staged` holds tile `at` and takes the one after next
  const auto take = [&](i32x4 (&staged)[kLoads], uint32_t at) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < kLoads; ++i)
      reinterpret_cast<i32x4*>(tile)[i * 256u + threadIdx.x] = staged[i];
    __syncthreads();
    fetch(staged, at + 2u * gridDim.x);
    f32x4 s[2] = {};
#pragma unroll
    for (int i = 0; i < kQuery; ++i)
#pragma unroll
      for (int half = 0; half < 2; ++half)
        s[half] = mfma_bf16(
            reinterpret_cast<const i32x4*>(tile)[half * chunks * kWave + key_at[i]], q[i],
            s[half]);
    parts[wave][0][lane] = s[0];
    parts[wave][1][lane] = s[1];
    __syncthreads();
#pragma unroll
    for (int half = 0; half < 2; ++half)
      s[half] = (parts[0][half][lane] + parts[1][half][lane]) +
                (parts[2][half][lane] + parts[3][half][lane]);
    float top = maximum;
#pragma unroll
    for (int half = 0; half < 2; ++half)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const uint32_t key = at * kTile + half * 16u + 4u * quarter + i;
        s[half][i] = visible(a, position, key) ? s[half][i] * unit : -INFINITY;
        top = fmaxf(top, s[half][i]);
      }
    top = fmaxf(top, __shfl_xor(top, 16, kWave));
    top = fmaxf(top, __shfl_xor(top, 32, kWave));
    const float base = top == -INFINITY ? 0.0f : top;
    const float fade = __builtin_amdgcn_exp2f(maximum - base);
    maximum = top;
    total *= fade;
#pragma unroll
    for (int half = 0; half < 2; ++half)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        s[half][i] = __builtin_amdgcn_exp2f(s[half][i] - base);
        total += s[half][i];
      }
    const i32x4 weights{static_cast<int>(pack_bf16(s[0][0], s[0][1])),
                        static_cast<int>(pack_bf16(s[0][2], s[0][3])),
                        static_cast<int>(pack_bf16(s[1][0], s[1][1])),
                        static_cast<int>(pack_bf16(s[1][2], s[1][3]))};
    const uint32_t token = 4u * quarter + lane % 16u / 4u;
#pragma unroll
    for (int j = 0; j < R; ++j) {
      const uint32_t t = min(wave + 4u * j, latent_chunks * 2u - 1u);   // sixteen values
      const uint32_t column = t % 2u * 16u + lane % 4u * 4u;
      const uint16_t* fragment = tile + t / 2u * kFragment + in_fragment(token, column);
      const i32x2 left = read_transposed(fragment);
      const i32x2 right = read_transposed(fragment + chunks * kFragment);
      sum[j] *= fade;
      sum[j] = mfma_bf16(i32x4{left[0], left[1], right[0], right[1]}, weights, sum[j]);
    }
    __syncthreads();
  };
  i32x4 even[kLoads], odd[kLoads];
  uint32_t next = begin + blockIdx.x;
  fetch(even, next);
  fetch(odd, next + gridDim.x);
  while (next < end) {
    take(even, next);
    next += gridDim.x;
    if (next >= end) break;
    take(odd, next);
    next += gridDim.x;
  }
  if (item >= items) return;
  total += __shfl_xor(total, 16, kWave);
  total += __shfl_xor(total, 32, kWave);
  const size_t place = size_t{blockIdx.x} * items + item;
  if (wave == 0u && quarter == 0u) {
    args.maxima[place * 2u] = maximum;
    args.maxima[place * 2u + 1u] = total;
  }
  if (begin + blockIdx.x >= end) return;
  float* out = args.sums + place * latent_chunks * 32u + 4u * quarter;
#pragma unroll
  for (int j = 0; j < R; ++j) {
    const uint32_t t = wave + 4u * j;
    if (t < latent_chunks * 2u) *reinterpret_cast<f32x4*>(out + t * 16u) = sum[j];
  }
}

// Groups of threads that add the parts, a thread four latent values.
__host__ __device__ __forceinline__ uint32_t value_groups(const Latent& a) {
  return kValueThreads / (chunks_of(a.rank) * 8u);
}

// Their sums in LDS, later the sums that cross from wave to wave.
__host__ __device__ __forceinline__ uint32_t added_quads(const Latent& a) {
  const uint32_t groups = value_groups(a) > 16u ? value_groups(a) : 16u;
  const uint32_t quads = groups * chunks_of(a.rank) * 8u;
  return quads > kValueThreads ? quads : kValueThreads;
}

// The parts of one head and up to 16 rows added, then through the value map: a
// wave per 16 values and half of the latent.
__global__ __launch_bounds__(kValueThreads) void latent_value_kernel(AttentionArgs args) {
  extern __shared__ f32x4 dynamic[];
  __shared__ float share[16][kMaximumSplits];
  const Latent& a = args.attention;
  const auto& run = args.launch;
  const uint32_t head = blockIdx.x;
  const uint32_t row0 = blockIdx.y * 16u;
  const uint32_t rows = min(16u, run.rows - row0);
  const uint32_t items = run.rows * a.heads;
  const uint32_t latent = chunks_of(a.rank) * 32u;
  const uint32_t quads = latent / 4u;
  const uint32_t stride = latent + 8u;                        // LDS row, elements
  const uint32_t groups = value_groups(a);
  f32x4* const added = dynamic;                               // [row][part][quads]
  uint16_t* const mean =
      reinterpret_cast<uint16_t*>(added + added_quads(a));         // [16][stride]
  const uint32_t wave = threadIdx.x / kWave;
  const uint32_t lane = threadIdx.x % kWave;

  // this wave's first weights, on their way meanwhile
  const uint32_t column = lane % 16u;
  const uint32_t quarter = lane / 16u;
  const uint32_t chunks = packed_chunks(a.rank);
  const uint32_t half_chunks = (chunks_of(a.rank) + 1u) / 2u;
  const uint32_t units = value_tiles(a) * 2u;
  constexpr uint32_t kAhead = 8;
  i32x4 ahead[kAhead];
  const auto weights_of = [&](uint32_t unit) {
    return static_cast<const i32x4*>(a.value_up) +
           ((size_t{head} * value_tiles(a) + unit / 2u) * chunks + unit % 2u * half_chunks) *
               kWave + lane;
  };
  const auto count_of = [&](uint32_t unit) {
    return unit % 2u ? chunks_of(a.rank) - half_chunks : half_chunks;
  };
  if (wave < units)
#pragma unroll
    for (uint32_t c = 0; c < kAhead; ++c)
      if (c < count_of(wave)) ahead[c] = weights_of(wave)[c * kWave];

  if (wave < rows) {
    const uint32_t item = (row0 + wave) * a.heads + head;
    constexpr uint32_t kEach = kMaximumSplits / kWave;
    float m[kEach], t[kEach];
    float top = -INFINITY;
#pragma unroll
    for (uint32_t i = 0; i < kEach; ++i) {
      const uint32_t split = i * kWave + lane;
      const float* pair =
          args.maxima + (size_t{min(split, args.splits - 1u)} * items + item) * 2u;
      m[i] = split < args.splits ? pair[0] : -INFINITY;
      t[i] = split < args.splits ? pair[1] : 0.0f;
      top = fmaxf(top, m[i]);
    }
    top = wave_max(top);
    float total = 0.0f;
#pragma unroll
    for (uint32_t i = 0; i < kEach; ++i) {
      m[i] = __builtin_amdgcn_exp2f(m[i] - top);
      total = fmaf(m[i], t[i], total);
    }
    total = wave_sum(total);
#pragma unroll
    for (uint32_t i = 0; i < kEach; ++i) share[wave][i * kWave + lane] = m[i] / total;
  }
  __syncthreads();
  // a row's parts over as many groups as there are; every group a row if not
  const uint32_t per_row = max(groups / rows, 1u);
  const uint32_t group = threadIdx.x / quads;
  const uint32_t quad = threadIdx.x % quads;
  if (group < groups)
    for (uint32_t row = group / per_row; row < rows; row += groups / per_row) {
      const uint32_t mine = group % per_row;
      const f32x4* part = reinterpret_cast<const f32x4*>(args.sums) +
                          size_t{(row0 + row) * a.heads + head} * quads + quad;
      f32x4 sum = {};
      for (uint32_t first = mine; first < args.splits; first += 8u * per_row) {
        f32x4 piece[8];
        // a part whose share is zero may never have been written
#pragma unroll
        for (uint32_t s = 0; s < 8u; ++s) {
          const uint32_t split = first + s * per_row;
          const float weight = split < args.splits ? share[row][split] : 0.0f;
          piece[s] = weight > 0.0f ? part[size_t{split} * items * quads] * weight : f32x4{};
        }
#pragma unroll
        for (uint32_t s = 0; s < 8u; ++s) sum += piece[s];
      }
      added[(row * per_row + mine) * quads + quad] = sum;
    }
  __syncthreads();
  for (uint32_t i = threadIdx.x; i < 16u * quads; i += blockDim.x) {
    const uint32_t row = i / quads;
    const uint32_t at = i % quads;
    f32x4 sum = {};
    if (row < rows)
      for (uint32_t p = 0; p < per_row; ++p) sum += added[(row * per_row + p) * quads + at];
    *reinterpret_cast<i32x2*>(mean + row * stride + at * 4u) =
        i32x2{static_cast<int>(pack_bf16(sum[0], sum[1])),
              static_cast<int>(pack_bf16(sum[2], sum[3]))};
  }
  __syncthreads();
  for (uint32_t base = 0; base < units; base += kValueThreads / kWave) {
    const uint32_t unit = base + wave;
    f32x4 sum = {};
    if (unit < units) {
      const uint16_t* operand =
          mean + column * stride + unit % 2u * half_chunks * 32u + 8u * quarter;
      const uint32_t count = count_of(unit);
#pragma unroll
      for (uint32_t c = 0; c < kAhead; ++c) {
        if (c >= count) continue;
        const i32x4 w = base ? weights_of(unit)[c * kWave] : ahead[c];
        sum = mfma_bf16(w, *reinterpret_cast<const i32x4*>(operand + c * 32u), sum);
      }
      for (uint32_t c = kAhead; c < count; ++c)
        sum = mfma_bf16(weights_of(unit)[c * kWave],
                        *reinterpret_cast<const i32x4*>(operand + c * 32u), sum);
      if (unit % 2u) added[wave * kWave + lane] = sum;
    }
    __syncthreads();
    if (unit < units && unit % 2u == 0u && column < rows) {
      sum += added[(wave + 1u) * kWave + lane];
      const uint32_t n = unit / 2u * 16u + 4u * quarter;
      f32x4 gate[1];
      take_gates(gate, a, run, row0 + column, head, n);
      store_four(a, run, row0 + column, head, n, sum * gate[0]);
    }
    __syncthreads();
  }
}

// ---- prompt form -------------------------------------------------------------------

constexpr uint32_t kExpandBlocks = 8;        // sixteen tokens each, per workgroup
constexpr uint32_t kExpandTiles = 16;        // of weights, per workgroup

// Keys or values of the expanded tiles: four waves side by side along the weight
// tiles, four tiles each, the latents of 128 tokens shared through LDS a chunk of
// 32 at a time.
template <bool VALUES>
__device__ __forceinline__ void expand_unit(const AttentionArgs& args, uint32_t unit_tiles,
                                            uint32_t unit_tokens,
                                            i32x4 (&shared)[2][kExpandBlocks * kWave]) {
  constexpr uint32_t WT = kExpandTiles / 4u;
  constexpr uint32_t MB = kExpandBlocks;
  const Latent& a = args.attention;
  const uint32_t wave = threadIdx.x / kWave;
  const uint32_t lane = threadIdx.x % kWave;
  const uint32_t column = lane % 16u;
  const uint32_t quarter = lane / 16u;
  const uint32_t per_head = VALUES ? value_tiles(a) : chunks_of(a.dim) * 2u;
  const uint32_t weight_tiles = a.heads * per_head;
  const uint32_t first_weight = unit_tiles * kExpandTiles + wave * WT;
  const uint32_t first_block = unit_tokens * MB;
  const uint32_t blocks = args.tiles * 2u;
  const uint32_t chunks = packed_chunks(a.rank);
  const uint32_t latent_chunks = chunks_of(a.rank);
  const i32x4* weights[WT];
#pragma unroll
  for (uint32_t i = 0; i < WT; ++i)
    weights[i] = static_cast<const i32x4*>(VALUES ? a.value_up : a.key_up) +
                 size_t{min(first_weight + i, weight_tiles - 1u)} * chunks * kWave + lane;
  // a wave fetches two of the eight token blocks
  global_piece* latents[2];
#pragma unroll
  for (uint32_t i = 0; i < 2u; ++i)
    latents[i] =
        as_global(cache_block<const uint16_t>(
            a, args.tile0 * kTile + min(first_block + wave * 2u + i, blocks - 1u) * 16u)) +
        lane;
  f32x4 sum[WT][MB] = {};
  i32x4 w[2][WT], x[2];
  const auto load = [&](uint32_t c, auto parity) __attribute__((always_inline)) {
    constexpr int P = decltype(parity)::value;
#pragma unroll
    for (uint32_t i = 0; i < WT; ++i) w[P][i] = weights[i][c * kWave];
#pragma unroll
    for (uint32_t i = 0; i < 2u; ++i) x[i] = latents[i][c * kWave];
  };
  const auto publish = [&](auto parity) __attribute__((always_inline)) {
    constexpr int P = decltype(parity)::value;
#pragma unroll
    for (uint32_t i = 0; i < 2u; ++i) shared[P][(wave * 2u + i) * kWave + lane] = x[i];
    __syncthreads();
  };
  const auto multiply = [&](auto parity) __attribute__((always_inline)) {
    constexpr int P = decltype(parity)::value;
#pragma unroll
    for (uint32_t j = 0; j < MB; ++j) {
      const i32x4 tokens = shared[P][j * kWave + lane];
#pragma unroll
      for (uint32_t i = 0; i < WT; ++i)
        sum[i][j] = VALUES ? mfma_bf16(tokens, w[P][i], sum[i][j])
                           : mfma_bf16(w[P][i], tokens, sum[i][j]);
    }
  };
  constexpr std::integral_constant<int, 0> even{};
  constexpr std::integral_constant<int, 1> odd{};
  load(0u, even);
  publish(even);
  uint32_t c = 0;
  for (; c + 2u <= latent_chunks; c += 2u) {
    load(c + 1u, odd);
    multiply(even);
    publish(odd);
    load(min(c + 2u, latent_chunks - 1u), even);
    multiply(odd);
    publish(even);
  }
  if (c < latent_chunks) multiply(even);

#pragma unroll
  for (uint32_t i = 0; i < WT; ++i) {
    const uint32_t at = first_weight + i;
    if (at >= weight_tiles) break;
    const uint32_t head = at / per_head;
    const uint32_t part = at % per_head;
#pragma unroll
    for (uint32_t j = 0; j < MB; ++j) {
      const uint32_t block = first_block + j;
      if (block >= blocks) break;
      const i32x2 four{static_cast<int>(pack_bf16(sum[i][j][0], sum[i][j][1])),
                       static_cast<int>(pack_bf16(sum[i][j][2], sum[i][j][3]))};
      uint16_t* out;
      if constexpr (VALUES) {
        // dimension `column`, tokens 4 quarter .. of this half of the tile: the
        // order in which the scores' registers hold them
        out = args.values +
              ((size_t{head} * args.tiles + block / 2u) * per_head + part) * kFragment +
              (quarter * 16u + column) * 8u + block % 2u * 4u;
      } else {
        out = args.keys +
              ((size_t{head} * args.tiles * 2u + block) * (per_head / 2u) + part / 2u) *
                  kFragment +
              in_fragment(column, part % 2u * 16u + 4u * quarter);
      }
      *reinterpret_cast<i32x2*>(out) = four;
    }
  }
}

__global__ __launch_bounds__(256, 2) void latent_expand_kernel(AttentionArgs args,
                                                               uint32_t key_units) {
  __shared__ i32x4 shared[2][kExpandBlocks * kWave];
  if (blockIdx.x < key_units)
    expand_unit<false>(args, blockIdx.x, blockIdx.y, shared);
  else
    expand_unit<true>(args, blockIdx.x - key_units, blockIdx.y, shared);
}

constexpr uint32_t kPromptRows = 128;

// NK: key chunks (unrotated and shared part), NV: value tiles, both at most.
template <int NK, int NV>
__global__ __launch_bounds__(256, 2) void latent_prompt_kernel(AttentionArgs args) {
  constexpr int MT = 2;                                   // sixteen rows each, per wave
  constexpr int kFragments = 2 * NK + NV;
  constexpr int kLoads = kFragments / 4;                  // fragments per wave and tile
  static_assert(kFragments % 4 == 0);
  __shared__ i32x4 staged[2][kFragments * kWave];
  const Latent& a = args.attention;
  const auto& run = args.launch;
  const uint32_t wave = __builtin_amdgcn_readfirstlane(threadIdx.x / kWave);
  const uint32_t lane = threadIdx.x % kWave;
  const uint32_t column = lane % 16u;
  const uint32_t quarter = lane / 16u;
  // contiguous ranges of (head, row block) per XCD; the longest blocks of one head
  // beside the shortest of the next
  const uint32_t row_blocks = (run.rows + kPromptRows - 1u) / kPromptRows;
  const uint32_t per_xcd = gridDim.x / 8u;
  const uint32_t work = blockIdx.x < per_xcd * 8u
                            ? blockIdx.x % 8u * per_xcd + blockIdx.x / 8u
                            : blockIdx.x;
  const uint32_t head = work / row_blocks;
  const uint32_t ordinal = work % row_blocks;
  const uint32_t block0 = (head % 2u ? ordinal : row_blocks - 1u - ordinal) * kPromptRows;
  const uint32_t row0 = block0 + wave * 16u * MT;         // of this wave
  const uint32_t first = a.step[kStepPosition];
  const uint32_t dim_chunks = chunks_of(a.dim);
  const uint32_t rot_chunks = chunks_of(a.rot_dim);
  const uint32_t latent_chunks = chunks_of(a.rank);
  const uint32_t key_chunks = dim_chunks + rot_chunks;
  const uint32_t tiles_v = value_tiles(a);
  const uint32_t last_row = min(block0 + kPromptRows, run.rows) - 1u;
  const uint32_t begin = first_tile(a, first + block0);
  const uint32_t end = (first + last_row) / kTile + 1u;

  // No load depends on a condition - places past the end are clamped to one that
  // exists - so that a wait for one tile's loads leaves the next one's in flight.
  // Key chunks past the last one meet zeros of the query; value tiles past the last
  // one end in sums that nobody reads.
  i32x4 q[MT][NK];
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    const uint16_t* query =
        args.query +
        (size_t{min(row0 + m * 16u + column, run.rows - 1u)} * a.heads + head) * key_chunks *
            32u +
        8u * quarter;
#pragma unroll
    for (int c = 0; c < NK; ++c) {
      const i32x4 stored = *reinterpret_cast<const i32x4*>(
          query + min(static_cast<uint32_t>(c), key_chunks - 1u) * 32u);
      q[m][c] = static_cast<uint32_t>(c) < key_chunks ? stored : i32x4{};
    }
  }

  // fragment f of a tile: half, key chunk; then value tiles.  A wave fetches every
  // fourth: where it lies for the first tile (or in a tile's cache rows) and how far
  // the next tile's is.
  global_piece* source[kLoads];
  uint32_t stride[kLoads];
  uint32_t in_cache[kLoads];
#pragma unroll
  for (int i = 0; i < kLoads; ++i) {
    const uint32_t f = wave + 4u * i;
    const bool key = f < 2u * NK;
    const uint32_t half = f / NK;
    const uint32_t c = key ? min(f % NK, key_chunks - 1u) : 0u;
    const uint32_t v = key ? 0u : min(f - 2u * NK, tiles_v - 1u);
    const bool cached = key && c >= dim_chunks;
    stride[i] = key ? 2u * dim_chunks * kWave : tiles_v * kWave;
    const uint16_t* base = key ? args.keys : args.values;
    source[i] = as_global(base) + size_t{head} * args.tiles * stride[i] +
                (key ? (half * dim_chunks + (cached ? 0u : c)) * kWave : v * kWave) + lane;
    in_cache[i] = cached ? (half * (latent_chunks + rot_chunks) + latent_chunks + c -
                            dim_chunks) * kWave + lane
                         : ~0u;
  }
  void* const* const pages = pages_of(a);
  const auto page_for = [&](uint32_t tile) {
    return as_global(cache_block<const uint16_t>(a, pages, min(tile, end - 1u) * kTile));
  };
  global_piece* ahead = page_for(begin);     // of the next fetch
  const auto fetch = [&](i32x4 (&loads)[kLoads], uint32_t tile) __attribute__((always_inline)) {
    global_piece* const rows = ahead;
    ahead = page_for(tile + 1u);
    const size_t ordinal = min(tile, end - 1u) - args.tile0;
#pragma unroll
    for (int i = 0; i < kLoads; ++i)
      loads[i] = *(in_cache[i] == ~0u ? source[i] + ordinal * stride[i] : rows + in_cache[i]);
    __builtin_amdgcn_sched_barrier(0);   // in this order
  };
  const auto publish = [&](const i32x4 (&loads)[kLoads], uint32_t slot)
      __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < kLoads; ++i) staged[slot][(wave + 4u * i) * kWave + lane] = loads[i];
  };
  const float unit = a.scale * kLog2e;
  // weights are taken relative to `base`, a maximum that may be out of date by
  // kSlack (a factor of 2^kSlack at most); it starts below every score
  constexpr float kSlack = 8.0f;
  float base[MT], total[MT];
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    base[m] = -INFINITY;
    total[m] = 0.0f;
  }
  f32x4 out[MT][NV] = {};
  const uint32_t wave_first = first + row0;
  const uint32_t wave_last = first + min(row0 + 16u * MT, run.rows) - 1u;
  const bool idle = row0 >= run.rows;
  const auto compute = [&](uint32_t tile) __attribute__((always_inline)) {
    const uint32_t slot = (tile - begin) & 1u;
    const uint32_t key0 = tile * kTile;
    // no row of the wave sees any key
    if (idle || key0 > wave_last || (a.window && key0 + kTile - 1u + a.window <= wave_first))
      return;
    const bool open =
        key0 + kTile - 1u <= wave_first && (!a.window || wave_last - key0 < a.window);
    f32x4 s[MT][2] = {};
#pragma unroll
    for (int c = 0; c < NK; ++c)
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        const i32x4 k = staged[slot][(half * NK + c) * kWave + lane];
#pragma unroll
        for (int m = 0; m < MT; ++m) s[m][half] = mfma_bf16(k, q[m][c], s[m][half]);
      }
    float top[MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) {
#pragma unroll
      for (int half = 0; half < 2; ++half) s[m][half] *= unit;
      if (!open) {
        const uint32_t position = wave_first + m * 16u + column;
#pragma unroll
        for (int half = 0; half < 2; ++half)
#pragma unroll
          for (int i = 0; i < 4; ++i)
            if (!visible(a, position, key0 + half * 16u + 4u * quarter + i))
              s[m][half][i] = -INFINITY;
      }
      top[m] = fmaxf(fmaxf(fmaxf(s[m][0][0], s[m][0][1]), fmaxf(s[m][0][2], s[m][0][3])),
                     fmaxf(fmaxf(s[m][1][0], s[m][1][1]), fmaxf(s[m][1][2], s[m][1][3])));
    }
    i32x4 weights[MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) {
      if (__any(top[m] > base[m] + kSlack)) {
        float fresh = fmaxf(top[m], __shfl_xor(top[m], 16, kWave));
        fresh = fmaxf(fresh, __shfl_xor(fresh, 32, kWave));
        fresh = fmaxf(fresh, base[m]);
        // a row that has seen nothing yet keeps its sums, which are zero
        const float fade =
            base[m] == -INFINITY ? 0.0f : __builtin_amdgcn_exp2f(base[m] - fresh);
        base[m] = fresh;
        total[m] *= fade;
#pragma unroll
        for (int t = 0; t < NV; ++t) out[m][t] *= fade;
      }
      const float offset = base[m] == -INFINITY ? 0.0f : base[m];
      float fresh = 0.0f;
#pragma unroll
      for (int half = 0; half < 2; ++half)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          s[m][half][i] = __builtin_amdgcn_exp2f(s[m][half][i] - offset);
          fresh += s[m][half][i];
        }
      total[m] += fresh;
      weights[m] = i32x4{static_cast<int>(pack_bf16(s[m][0][0], s[m][0][1])),
                         static_cast<int>(pack_bf16(s[m][0][2], s[m][0][3])),
                         static_cast<int>(pack_bf16(s[m][1][0], s[m][1][1])),
                         static_cast<int>(pack_bf16(s[m][1][2], s[m][1][3]))};
    }
#pragma unroll
    for (int t = 0; t < NV; ++t) {
      const i32x4 v = staged[slot][(2 * NK + t) * kWave + lane];
#pragma unroll
      for (int m = 0; m < MT; ++m) out[m][t] = mfma_bf16(v, weights[m], out[m][t]);
    }
  };
  // a tile is fetched two iterations and published one before its turn
  i32x4 even[kLoads], odd[kLoads];
  fetch(even, begin);
  fetch(odd, begin + 1u);
  publish(even, 0u);
  fetch(even, begin + 2u);
  __syncthreads();
  const auto turn = [&](i32x4 (&loads)[kLoads], uint32_t tile) __attribute__((always_inline)) {
    compute(tile);
    publish(loads, (tile + 1u - begin) & 1u);
    fetch(loads, tile + 3u);
    __syncthreads();
  };
  for (uint32_t tile = begin; tile < end; tile += 2u) {
    turn(odd, tile);
    if (tile + 1u < end) turn(even, tile + 1u);
  }
  if (idle) return;
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    const uint32_t row = row0 + m * 16u + column;
    total[m] += __shfl_xor(total[m], 16, kWave);
    total[m] += __shfl_xor(total[m], 32, kWave);
    if (row >= run.rows) continue;
    const float inverse = 1.0f / total[m];
    f32x4 gate[NV];
    take_gates(gate, a, run, row, head, 4u * quarter);
#pragma unroll
    for (int t = 0; t < NV; ++t)
      store_four(a, run, row, head, t * 16u + 4u * quarter, out[m][t] * inverse * gate[t]);
  }
}

template <int NK>
void launch_prompt(const AttentionArgs& args, hipStream_t stream) {
  const uint32_t blocks =
      (args.launch.rows + kPromptRows - 1u) / kPromptRows * args.attention.heads;
  if (value_tiles(args.attention) <= 4u)
    latent_prompt_kernel<NK, 4><<<blocks, 256, 0, stream>>>(args);
  else
    latent_prompt_kernel<NK, 8><<<blocks, 256, 0, stream>>>(args);
}

bool valid_geometry(const Latent& a) {
  return a.heads && a.dim && a.vdim && a.rank && a.rotary_dims <= a.rot_dim &&
         a.rotary_dims % 2u == 0u && (!a.rotary_dims || a.frequencies) && a.latent_norm &&
         a.key_up && a.key_up_transposed && a.value_up && a.page_tokens &&
         a.page_tokens % 32u == 0u && a.layer_offset % 16u == 0u && a.page_table && a.step &&
         a.pages_per_slot && a.element <= QLLM_ELEMENT_F32;
}

uint32_t maximum_tiles(const Latent& a, uint32_t rows, uint32_t maximum_position) {
  const uint64_t all = maximum_position / kTile + 1u;
  if (!a.window) return static_cast<uint32_t>(all);
  const uint64_t seen = (uint64_t{a.window} + rows + kTile - 2u) / kTile + 1u;
  return static_cast<uint32_t>(seen < all ? seen : all);
}

uint32_t item_tiles(const Latent& a, uint32_t rows) { return (rows * a.heads + 15u) / 16u; }

uint32_t splits_for(const Latent& a, uint32_t rows, uint32_t maximum_position) {
  const uint32_t most = 256u / item_tiles(a, rows);
  const uint32_t bound = most < 1u ? 1u : most < kMaximumSplits ? most : kMaximumSplits;
  const uint32_t tiles = maximum_tiles(a, rows, maximum_position);
  const uint32_t wanted =
      tiles <= kSplitsFirst ? tiles : tiles / 4u > kSplitsFirst ? tiles / 4u : kSplitsFirst;
  return wanted < bound ? wanted : bound;
}

size_t align16(size_t bytes) { return (bytes + 15u) / 16u * 16u; }

struct Workspace {
  size_t query, sums, maxima, keys, values;
};

Workspace split_workspace(const Latent& a, uint32_t rows, uint32_t maximum_position) {
  const size_t items = size_t{rows} * a.heads;
  const size_t splits = splits_for(a, rows, maximum_position);
  return {align16(items * row_chunks(a) * 64u), splits * items * chunks_of(a.rank) * 128u,
          align16(splits * items * 8u), 0u, 0u};
}

Workspace prompt_workspace(const Latent& a, uint32_t rows, uint32_t maximum_position) {
  const size_t tiles = maximum_tiles(a, rows, maximum_position);
  return {align16(size_t{rows} * a.heads * (chunks_of(a.dim) + chunks_of(a.rot_dim)) * 64u),
          0u, 0u, a.heads * tiles * 2u * chunks_of(a.dim) * kFragment * 2u,
          a.heads * tiles * value_tiles(a) * kFragment * 2u};
}

size_t bytes_of(const Workspace& w) { return w.query + w.sums + w.maxima + w.keys + w.values; }

size_t general_bytes(const Latent& a) {
  return (size_t{a.dim} + a.rot_dim + 2u * a.rank + kTile) * 4u;
}

size_t value_bytes(const Latent& a) {
  return size_t{added_quads(a)} * 16u + size_t{16u} * (chunks_of(a.rank) * 32u + 8u) * 2u;
}

}  // namespace
}  // namespace qllm

using namespace qllm;

extern "C" size_t qllm_latent_layer_bytes(uint32_t page_tokens, uint32_t rank,
                                          uint32_t rot_dim, uint32_t element) {
  return size_t{page_tokens} * (chunks_of(rank) + chunks_of(rot_dim)) * 32u *
         (element == QLLM_ELEMENT_F32 ? 4u : 2u);
}

extern "C" int32_t qllm_latent_store(const qllm_latent_attention* attention,
                                     const qllm_latent_store_launch* launch, void* stream) {
  if (!attention || !launch || !valid_geometry(*attention) || !launch->projections ||
      !launch->rows ||
      launch->latent_column + attention->rank + attention->rot_dim > launch->stride ||
      (launch->query_rank &&
       (!launch->query_norm || !launch->query_out ||
        launch->query_stride < launch->query_rank ||
        launch->query_column + launch->query_rank > launch->stride)))
    return fail(QLLM_INVALID_ARGUMENT, "invalid latent store");
  const StoreArgs args{*attention, *launch};
  const dim3 grid(launch->rows, launch->query_rank ? 2u : 1u);
  if (attention->element == QLLM_ELEMENT_F32)
    latent_store_kernel<float><<<grid, 256, 0, as_stream(stream)>>>(args);
  else
    latent_store_kernel<uint16_t><<<grid, 256, 0, as_stream(stream)>>>(args);
  return launched("latent store");
}

extern "C" uint32_t qllm_latent_attention_form(const qllm_latent_attention* attention,
                                               uint32_t rows) {
  if (!attention || attention->element != QLLM_ELEMENT_BF16) return QLLM_ATTENTION_GENERAL;
  const Latent& a = *attention;
  if (rows > kSplitRows && chunks_of(a.dim) + chunks_of(a.rot_dim) <= 8u &&
      value_tiles(a) <= 8u)
    return QLLM_ATTENTION_PROMPT;
  return chunks_of(a.rank) <= 16u && chunks_of(a.rot_dim) <= 2u ? QLLM_ATTENTION_SPLIT
                                                                : QLLM_ATTENTION_GENERAL;
}

extern "C" size_t qllm_latent_attention_workspace_bytes(
    const qllm_latent_attention* attention, uint32_t rows, uint32_t maximum_position) {
  if (!attention || !rows) return 0u;
  switch (qllm_latent_attention_form(attention, rows)) {
    case QLLM_ATTENTION_SPLIT:
      return bytes_of(split_workspace(*attention, rows, maximum_position));
    case QLLM_ATTENTION_PROMPT:
      return bytes_of(prompt_workspace(*attention, rows, maximum_position));
    default:
      return 0u;
  }
}

extern "C" int32_t qllm_latent_attention_rows(const qllm_latent_attention* attention,
                                              const qllm_latent_launch* launch,
                                              void* stream) {
  if (!attention || !launch || !valid_geometry(*attention) || !launch->query ||
      !launch->output || !launch->rows ||
      launch->query_stride < attention->heads * (attention->dim + attention->rot_dim) ||
      launch->output_stride < attention->heads * attention->vdim ||
      (launch->gate && launch->gate_stride < attention->heads * attention->vdim) ||
      launch->maximum_position < launch->rows - 1u)
    return fail(QLLM_INVALID_ARGUMENT, "invalid latent attention");
  const Latent& a = *attention;
  const auto hip_stream = as_stream(stream);
  AttentionArgs args{a, *launch, nullptr, nullptr, nullptr, nullptr, nullptr, 0u, 0u, 0u};
  const uint32_t rows = launch->rows;
  const uint32_t form = qllm_latent_attention_form(attention, rows);
  if (form == QLLM_ATTENTION_GENERAL) {
    if (general_bytes(a) > 65536u)
      return fail(QLLM_INVALID_ARGUMENT, "latent attention: dimensions exceed the kernel");
    const dim3 grid(rows, a.heads);
    if (a.element == QLLM_ELEMENT_F32)
      latent_general_kernel<float><<<grid, 256, general_bytes(a), hip_stream>>>(args);
    else
      latent_general_kernel<uint16_t><<<grid, 256, general_bytes(a), hip_stream>>>(args);
    return launched("latent attention");
  }
  if (!launch->workspace || (reinterpret_cast<uintptr_t>(launch->workspace) & 15u) != 0u ||
      launch->workspace_bytes <
          qllm_latent_attention_workspace_bytes(attention, rows, launch->maximum_position))
    return fail(QLLM_INVALID_ARGUMENT, "latent attention workspace is too small");
  auto* bytes = static_cast<uint8_t*>(launch->workspace);
  const Workspace parts = form == QLLM_ATTENTION_SPLIT
                              ? split_workspace(a, rows, launch->maximum_position)
                              : prompt_workspace(a, rows, launch->maximum_position);
  args.query = reinterpret_cast<uint16_t*>(bytes);
  bytes += parts.query;
  args.sums = reinterpret_cast<float*>(bytes);
  bytes += parts.sums;
  args.maxima = reinterpret_cast<float*>(bytes);
  bytes += parts.maxima;
  args.keys = reinterpret_cast<uint16_t*>(bytes);
  bytes += parts.keys;
  args.values = reinterpret_cast<uint16_t*>(bytes);

  if (form == QLLM_ATTENTION_PROMPT) {
    const uint32_t first = launch->maximum_position + 1u - rows;
    args.tile0 = a.window && first + 1u > a.window ? (first + 1u - a.window) / kTile : 0u;
    args.tiles = launch->maximum_position / kTile + 1u - args.tile0;
    latent_prompt_query_kernel<<<(rows * a.heads + 3u) / 4u, 256, 0, hip_stream>>>(args);
    const auto units = [](uint32_t count, uint32_t each) { return (count + each - 1u) / each; };
    const uint32_t key_units = units(a.heads * chunks_of(a.dim) * 2u, kExpandTiles);
    const uint32_t value_units = units(a.heads * value_tiles(a), kExpandTiles);
    latent_expand_kernel<<<dim3(key_units + value_units, units(args.tiles * 2u, kExpandBlocks)),
                           256, 0, hip_stream>>>(args, key_units);
    const uint32_t chunks = chunks_of(a.dim) + chunks_of(a.rot_dim);
    if (chunks <= 2u)
      launch_prompt<2>(args, hip_stream);
    else if (chunks <= 4u)
      launch_prompt<4>(args, hip_stream);
    else if (chunks <= 6u)
      launch_prompt<6>(args, hip_stream);
    else
      launch_prompt<8>(args, hip_stream);
    return launched("latent prompt attention");
  }
  args.splits = splits_for(a, rows, launch->maximum_position);
  const uint32_t row_tiles = (rows + 15u) / 16u;
  latent_query_kernel<<<dim3((chunks_of(a.rank) * 2u + 3u) / 4u + (a.rot_dim ? 1u : 0u),
                             a.heads, row_tiles),
                        256, 0, hip_stream>>>(args);
  const dim3 grid(args.splits, item_tiles(a, rows));
  if (a.rank <= 64u)
    latent_split_kernel<1><<<grid, 256, 0, hip_stream>>>(args);
  else if (a.rank <= 128u)
    latent_split_kernel<2><<<grid, 256, 0, hip_stream>>>(args);
  else if (a.rank <= 256u)
    latent_split_kernel<4><<<grid, 256, 0, hip_stream>>>(args);
  else
    latent_split_kernel<8><<<grid, 256, 0, hip_stream>>>(args);
  latent_value_kernel<<<dim3(a.heads, row_tiles), kValueThreads, value_bytes(a),
                        hip_stream>>>(args);
  return launched("latent split attention");
}
