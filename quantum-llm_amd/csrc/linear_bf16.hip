// Linear layers with bf16 weights: several matrices per launch, each with its
// own input rows and epilogue (store, residual add, gated activation, K-split
// partial sums).
//
// The weights lie in fragment order: 16 rows x 32 columns are one contiguous
// KiB in which lane 16g + n finds row n, columns 8g .. 8g + 7 - its operand of
// v_mfma_f32_16x16x32_bf16.  Every weight load of a wave is one contiguous
// KiB and goes straight to the matrix cores, whatever the batch:
//
//  * up to 64 rows (decode): a workgroup owns one 16-row tile (two for the
//    gated epilogue), its eight waves split K and add their accumulators
//    through LDS in a fixed order.  All of a wave's loads are in flight at
//    once; a small batch costs one matrix instruction per KiB of weights.
//  * more rows (prompts): four waves side by side along the weight rows, each
//    with NT x MT accumulator tiles; the activation tile of 64 columns is
//    shared through LDS (double-buffered, one barrier per step, 16-byte pieces
//    swizzled by row so that a fragment read touches every bank), weights are
//    prefetched one step ahead in registers.  An XCD gets a contiguous range
//    of the grid walked in bands of activation tiles, so operands are shared
//    in its L2.
//  * F32 mode: plain 32-bit multiply-adds from the same packed weights.
#include "common.hpp"
#include "mixed_common.hpp"

namespace qllm {
namespace {

constexpr uint32_t kMaximumSegments = 8;
constexpr uint32_t kSmallWaves = 8;
constexpr uint32_t kBandTiles = 8;       // activation tiles per band of the grid

struct LinearArgs {
  qllm_linear_segment segment[kMaximumSegments];
  uint32_t first_unit[kMaximumSegments + 1];   // workgroups before segment s
  uint32_t count;
  uint32_t batch;
};

__device__ __forceinline__ uint32_t segment_of(const LinearArgs& args, uint32_t unit) {
  uint32_t index = 0;
  while (index + 1u < args.count && unit >= args.first_unit[index + 1u]) ++index;
  return index;
}

// Four consecutive output columns n .. n + 3 of batch row m.
__device__ __forceinline__ void store_four(const qllm_linear_segment& s, float* base,
                                           uint32_t m, uint32_t n, f32x4 value,
                                           bool add) {
  if (n >= s.output_columns) return;
  float* out = base + size_t{m} * s.output_stride + n;
  if (n + 4u <= s.output_columns && s.output_stride % 4u == 0u) {
    f32x4* vector = reinterpret_cast<f32x4*>(out);
    *vector = add ? *vector + value : value;
  } else {
    for (uint32_t i = 0; i < 4u && n + i < s.output_columns; ++i)
      out[i] = add ? out[i] + value[i] : value[i];
  }
}

template <typename T>
__device__ __forceinline__ void store_gated(const qllm_linear_segment& s, uint32_t m,
                                            uint32_t n, f32x4 gate, f32x4 up) {
  T* out = static_cast<T*>(s.output) + size_t{m} * s.output_stride + n;
  for (uint32_t i = 0; i < 4u && n + i < s.output_columns; ++i)
    store_element(out + i, activate(s.activation, gate[i]) * up[i]);
}

// ---- up to 64 rows ------------------------------------------------------------

template <int MT, int TILES, int UNROLL>
__device__ __forceinline__ void small_unit(const qllm_linear_segment& s, uint32_t unit,
                                           uint32_t batch, f32x4* scratch) {
  const uint32_t wave = threadIdx.x / kWave;
  const uint32_t lane = threadIdx.x % kWave;
  const uint32_t tiles = s.rows / (16u * TILES);
  const uint32_t parts = s.epilogue == QLLM_LINEAR_PARTIALS ? s.splits : 1u;
  const uint32_t part = unit / tiles;
  const uint32_t tile = unit % tiles;
  const uint32_t chunks = s.columns / 32u;
  const uint32_t part_begin = chunks * part / parts;
  const uint32_t span = chunks * (part + 1u) / parts - part_begin;
  const uint32_t begin = part_begin + span * wave / kSmallWaves;
  const uint32_t end = part_begin + span * (wave + 1u) / kSmallWaves;

  const i32x4* weights = static_cast<const i32x4*>(s.weights) +
                         size_t{tile} * TILES * chunks * kWave + lane;
  const uint16_t* input[MT];
#pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    const uint32_t row = min(mt * 16u + lane % 16u, batch - 1u);
    input[mt] = static_cast<const uint16_t*>(s.input) + size_t{row} * s.input_stride +
                8u * (lane / 16u);
  }
  f32x4 sum[TILES][MT] = {};
  uint32_t chunk = begin;
  for (; chunk + UNROLL <= end; chunk += UNROLL) {
    i32x4 w[UNROLL][TILES];
    i32x4 x[UNROLL][MT];
#pragma unroll
    for (int u = 0; u < UNROLL; ++u)
#pragma unroll
      for (int t = 0; t < TILES; ++t)
        w[u][t] = __builtin_nontemporal_load(
            weights + (size_t{static_cast<uint32_t>(t)} * chunks + chunk + u) * kWave);
#pragma unroll
    for (int u = 0; u < UNROLL; ++u)
#pragma unroll
      for (int mt = 0; mt < MT; ++mt)
        x[u][mt] = *reinterpret_cast<const i32x4*>(input[mt] + (chunk + u) * 32u);
#pragma unroll
    for (int u = 0; u < UNROLL; ++u)
#pragma unroll
      for (int t = 0; t < TILES; ++t)
#pragma unroll
        for (int mt = 0; mt < MT; ++mt)
          sum[t][mt] = mfma_bf16(w[u][t], x[u][mt], sum[t][mt]);
  }
  for (; chunk < end; ++chunk)
#pragma unroll
    for (int t = 0; t < TILES; ++t) {
      const i32x4 w = weights[(size_t{static_cast<uint32_t>(t)} * chunks + chunk) * kWave];
#pragma unroll
      for (int mt = 0; mt < MT; ++mt)
        sum[t][mt] = mfma_bf16(
            w, *reinterpret_cast<const i32x4*>(input[mt] + chunk * 32u), sum[t][mt]);
    }

#pragma unroll
  for (int t = 0; t < TILES; ++t)
#pragma unroll
    for (int mt = 0; mt < MT; ++mt)
      scratch[((t * MT + mt) * kSmallWaves + wave) * kWave + lane] = sum[t][mt];
  __syncthreads();
  for (uint32_t index = threadIdx.x; index < MT * kWave; index += kSmallWaves * kWave) {
    const uint32_t mt = index / kWave;
    const uint32_t at = index % kWave;
    f32x4 total[TILES];
#pragma unroll
    for (int t = 0; t < TILES; ++t) {
      total[t] = scratch[(t * MT + mt) * kSmallWaves * kWave + at];
      for (uint32_t other = 1; other < kSmallWaves; ++other)
        total[t] += scratch[((t * MT + mt) * kSmallWaves + other) * kWave + at];
    }
    const uint32_t m = mt * 16u + at % 16u;
    const uint32_t n = tile * 16u + 4u * (at / 16u);
    if (m >= batch) continue;
    if constexpr (TILES == 2) {
      store_gated<uint16_t>(s, m, n, total[0], total[1]);
    } else {
      float* base = static_cast<float*>(s.output) +
                    size_t{part} * batch * s.output_stride;
      store_four(s, base, m, n, total[0], s.epilogue == QLLM_LINEAR_ADD);
    }
  }
}

template <int MT>
__global__ __launch_bounds__(kSmallWaves* kWave) void linear_small_kernel(LinearArgs args) {
  __shared__ f32x4 scratch[2 * MT * kSmallWaves * kWave];
  const uint32_t index = segment_of(args, blockIdx.x);
  const qllm_linear_segment& s = args.segment[index];
  const uint32_t unit = blockIdx.x - args.first_unit[index];
  if (s.epilogue == QLLM_LINEAR_GATED)
    small_unit<MT, 2, (MT > 1 ? 2 : 4)>(s, unit, args.batch, scratch);
  else
    small_unit<MT, 1, (MT > 1 ? 4 : 8)>(s, unit, args.batch, scratch);
}

// ---- tall batches --------------------------------------------------------------

template <int NT, int MT>
__global__ __launch_bounds__(256, 2) void linear_tall_kernel(LinearArgs args) {
  constexpr uint32_t kRowsM = MT * 16u;
  constexpr uint32_t kPieces = kRowsM * 8u;           // 16-byte pieces of a tile
  constexpr uint32_t kLoads = kPieces / 256u;
  static_assert(kPieces % 256u == 0u);
  __shared__ i32x4 tile[2][kPieces];

  const uint32_t m_tiles = (args.batch + kRowsM - 1u) / kRowsM;
  // contiguous ranges of workgroups per XCD (consecutive ids go round the XCDs)
  uint32_t work = blockIdx.x;
  {
    const uint32_t per_xcd = gridDim.x / 8u;
    if (work < per_xcd * 8u) work = (work % 8u) * per_xcd + work / 8u;
  }
  const uint32_t index = segment_of(args, work);
  const qllm_linear_segment& s = args.segment[index];
  const uint32_t unit = work - args.first_unit[index];
  const uint32_t n_tiles = (s.rows + 64u * NT - 1u) / (64u * NT);
  // bands of kBandTiles activation tiles, walked column by column
  const uint32_t band = unit / (kBandTiles * n_tiles);
  const uint32_t band_rows = min(kBandTiles, m_tiles - band * kBandTiles);
  const uint32_t in_band = unit - band * kBandTiles * n_tiles;
  const uint32_t m_tile = band * kBandTiles + in_band % band_rows;
  const uint32_t n_tile = in_band / band_rows;

  const uint32_t wave = threadIdx.x / kWave;
  const uint32_t lane = threadIdx.x % kWave;
  const uint32_t chunks = s.columns / 32u;
  const uint32_t steps = s.columns / 64u;
  const uint32_t weight_tiles = s.rows / 16u;
  const uint32_t first_tile = (n_tile * 4u + wave) * NT;

  const i32x4* weights[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t)
    weights[t] = static_cast<const i32x4*>(s.weights) +
                 size_t{min(first_tile + t, weight_tiles - 1u)} * chunks * kWave + lane;

  // piece p of the tile: row p / 8, swizzled slot p % 8
  const i32x4* source[kLoads];
#pragma unroll
  for (uint32_t i = 0; i < kLoads; ++i) {
    const uint32_t piece = i * 256u + threadIdx.x;
    const uint32_t row = piece / 8u;
    const uint32_t column = (piece % 8u) ^ (row % 8u);
    const uint32_t batch_row = min(m_tile * kRowsM + row, args.batch - 1u);
    source[i] = reinterpret_cast<const i32x4*>(
        static_cast<const uint16_t*>(s.input) + size_t{batch_row} * s.input_stride +
        column * 8u);
  }

  f32x4 sum[NT][MT] = {};
  i32x4 staged[kLoads];
  i32x4 held[2][2][NT];   // [step parity][half of 32 columns][tile]
#pragma unroll
  for (uint32_t i = 0; i < kLoads; ++i) staged[i] = source[i][0];
#pragma unroll
  for (int half = 0; half < 2; ++half)
#pragma unroll
    for (int t = 0; t < NT; ++t) held[0][half][t] = weights[t][half * kWave];
#pragma unroll
  for (uint32_t i = 0; i < kLoads; ++i) tile[0][i * 256u + threadIdx.x] = staged[i];
  __syncthreads();

  const auto step_at = [&](uint32_t step, auto parity) {
    constexpr int P = decltype(parity)::value;
    const uint32_t next = min(step + 1u, steps - 1u);   // the last step re-reads itself
#pragma unroll
    for (uint32_t i = 0; i < kLoads; ++i) staged[i] = source[i][next * 8u];
#pragma unroll
    for (int half = 0; half < 2; ++half)
#pragma unroll
      for (int t = 0; t < NT; ++t)
        held[1 - P][half][t] = weights[t][(next * 2u + half) * kWave];
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int half = 0; half < 2; ++half) {
      i32x4 x[MT];
#pragma unroll
      for (int mt = 0; mt < MT; ++mt) {
        const uint32_t row = mt * 16u + lane % 16u;
        const uint32_t column = half * 4u + lane / 16u;
        x[mt] = tile[P][row * 8u + (column ^ (row % 8u))];
      }
#pragma unroll
      for (int mt = 0; mt < MT; ++mt)
#pragma unroll
        for (int t = 0; t < NT; ++t)
          sum[t][mt] = mfma_bf16(held[P][half][t], x[mt], sum[t][mt]);
    }
#pragma unroll
    for (uint32_t i = 0; i < kLoads; ++i) tile[1 - P][i * 256u + threadIdx.x] = staged[i];
    __syncthreads();
  };
  uint32_t step = 0;
  for (; step + 2u <= steps; step += 2u) {
    step_at(step, std::integral_constant<int, 0>{});
    step_at(step + 1u, std::integral_constant<int, 1>{});
  }
  if (step < steps) step_at(step, std::integral_constant<int, 0>{});

#pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    const uint32_t m = m_tile * kRowsM + mt * 16u + lane % 16u;
    if (m >= args.batch) continue;
    if (s.epilogue == QLLM_LINEAR_GATED) {
      if constexpr (NT % 2 == 0) {
#pragma unroll
        for (int t = 0; t < NT; t += 2) {
          const uint32_t at = first_tile + t;
          if (at >= weight_tiles) continue;
          const uint32_t n = at / 2u * 16u + 4u * (lane / 16u);
          if (n + 4u <= s.output_columns && s.output_stride % 4u == 0u) {
            const f32x4 gate = sum[t][mt];
            const f32x4 up = sum[t + 1][mt];
            uint32_t bits[4];
#pragma unroll
            for (int i = 0; i < 4; ++i)
              bits[i] = f32_to_bf16_bits(activate(s.activation, gate[i]) * up[i]);
            *reinterpret_cast<i32x2*>(static_cast<uint16_t*>(s.output) +
                                      size_t{m} * s.output_stride + n) =
                i32x2{static_cast<int>(bits[0] | bits[1] << 16),
                      static_cast<int>(bits[2] | bits[3] << 16)};
          } else {
            store_gated<uint16_t>(s, m, n, sum[t][mt], sum[t + 1][mt]);
          }
        }
      }
    } else {
#pragma unroll
      for (int t = 0; t < NT; ++t)
        if (first_tile + t < weight_tiles)
          store_four(s, static_cast<float*>(s.output), m,
                     (first_tile + t) * 16u + 4u * (lane / 16u), sum[t][mt],
                     s.epilogue == QLLM_LINEAR_ADD);
    }
  }
}

// ---- F32 mode --------------------------------------------------------------------

// 64 batch rows x 64 packed weight rows per workgroup, 4 x 4 products per
// thread; a thread's weight rows are 16 apart, so the two tiles of a gated
// pair meet in it.
__global__ __launch_bounds__(256) void linear_f32_kernel(LinearArgs args) {
  __shared__ float x_tile[32][65];
  __shared__ float w_tile[32][65];
  const uint32_t index = segment_of(args, blockIdx.x);
  const qllm_linear_segment& s = args.segment[index];
  const uint32_t unit = blockIdx.x - args.first_unit[index];
  const uint32_t n_tiles = (s.rows + 63u) / 64u;
  const uint32_t m_tiles = (args.batch + 63u) / 64u;
  const uint32_t parts = s.epilogue == QLLM_LINEAR_PARTIALS ? s.splits : 1u;
  const uint32_t part = unit / (n_tiles * m_tiles);
  const uint32_t rest = unit % (n_tiles * m_tiles);
  const uint32_t m0 = rest / n_tiles * 64u;
  const uint32_t n0 = rest % n_tiles * 64u;
  const uint32_t chunks = s.columns / 32u;
  const uint32_t begin = chunks * part / parts;
  const uint32_t end = chunks * (part + 1u) / parts;
  const auto* weights = static_cast<const uint16_t*>(s.weights);
  const auto* input = static_cast<const float*>(s.input);
  const uint32_t tx = threadIdx.x % 16u;
  const uint32_t ty = threadIdx.x / 16u;
  float sum[4][4] = {};
  for (uint32_t chunk = begin; chunk < end; ++chunk) {
    __syncthreads();
    for (uint32_t i = threadIdx.x; i < 64u * 32u; i += 256u) {
      const uint32_t k = i % 32u;
      const uint32_t row = i / 32u;
      const uint32_t m = min(m0 + row, args.batch - 1u);
      x_tile[k][row] = input[size_t{m} * s.input_stride + chunk * 32u + k];
      const uint32_t n = n0 + row;
      w_tile[k][row] =
          n < s.rows ? bf16_bits_to_f32(weights[(size_t{n / 16u} * chunks + chunk) * 512u +
                                                (k / 8u * 16u + n % 16u) * 8u + k % 8u])
                     : 0.0f;
    }
    __syncthreads();
    for (uint32_t k = 0; k < 32u; ++k) {
      float x[4], w[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        x[i] = x_tile[k][ty * 4u + i];
        w[i] = w_tile[k][tx + 16u * i];
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) sum[i][j] = fmaf(x[i], w[j], sum[i][j]);
    }
  }
  for (int i = 0; i < 4; ++i) {
    const uint32_t m = m0 + ty * 4u + i;
    if (m >= args.batch) continue;
    if (s.epilogue == QLLM_LINEAR_GATED) {
      for (int j = 0; j < 4; j += 2) {
        const uint32_t n = n0 / 2u + j * 8u + tx;
        if (n0 + j * 16u + tx < s.rows && n < s.output_columns)
          static_cast<float*>(s.output)[size_t{m} * s.output_stride + n] =
              activate(s.activation, sum[i][j]) * sum[i][j + 1];
      }
      continue;
    }
    float* out = static_cast<float*>(s.output) +
                 (size_t{part} * args.batch + m) * s.output_stride;
    for (int j = 0; j < 4; ++j) {
      const uint32_t n = n0 + tx + 16u * j;
      if (n >= s.rows || n >= s.output_columns) continue;
      out[n] = s.epilogue == QLLM_LINEAR_ADD ? out[n] + sum[i][j] : sum[i][j];
    }
  }
}

__global__ void linear_pack_kernel(const uint16_t* source, uint32_t rows, uint32_t columns,
                                   uint64_t row_stride, uint64_t column_stride,
                                   uint16_t* packed, uint32_t packed_chunks,
                                   uint32_t first_tile, uint32_t tile_stride,
                                   uint32_t first_chunk, uint32_t chunks,
                                   uint64_t elements) {
  for (uint64_t i = uint64_t{blockIdx.x} * blockDim.x + threadIdx.x; i < elements;
       i += uint64_t{gridDim.x} * blockDim.x) {
    const uint32_t in_fragment = static_cast<uint32_t>(i % 512u);
    const uint64_t fragment = i / 512u;
    const uint32_t chunk = static_cast<uint32_t>(fragment % chunks);
    const uint32_t tile = static_cast<uint32_t>(fragment / chunks);
    const uint32_t lane = in_fragment / 8u;
    const uint32_t row = tile * 16u + lane % 16u;
    const uint32_t column = chunk * 32u + lane / 16u * 8u + in_fragment % 8u;
    const uint16_t value = row < rows && column < columns
                               ? source[row * row_stride + column * column_stride]
                               : uint16_t{0};
    packed[(uint64_t{first_tile + tile * tile_stride} * packed_chunks + first_chunk +
            chunk) * 512u + in_fragment] = value;
  }
}

bool aligned16(const void* pointer) {
  return (reinterpret_cast<uintptr_t>(pointer) & 15u) == 0u;
}

template <int NT, int MT>
uint32_t tall_units(const qllm_linear_segment& s, uint32_t batch) {
  return (s.rows + 64u * NT - 1u) / (64u * NT) * ((batch + 16u * MT - 1u) / (16u * MT));
}

template <int NT, int MT>
int32_t launch_tall(LinearArgs& args, hipStream_t stream) {
  args.first_unit[0] = 0;
  for (uint32_t i = 0; i < args.count; ++i)
    args.first_unit[i + 1] = args.first_unit[i] + tall_units<NT, MT>(args.segment[i], args.batch);
  linear_tall_kernel<NT, MT><<<args.first_unit[args.count], 256, 0, stream>>>(args);
  return launched("tall bf16 linear");
}

template <int NT, int MT>
uint32_t all_tall_units(const LinearArgs& args) {
  uint32_t units = 0;
  for (uint32_t i = 0; i < args.count; ++i)
    units += tall_units<NT, MT>(args.segment[i], args.batch);
  return units;
}

}  // namespace
}  // namespace qllm

using namespace qllm;

extern "C" size_t qllm_linear_packed_bytes(uint32_t rows, uint32_t columns) {
  return size_t{(rows + 15u) / 16u * 16u} * ((size_t{columns} + 63u) / 64u * 64u) * 2u;
}

extern "C" int32_t qllm_linear_pack(const void* source_bf16, uint32_t rows, uint32_t columns,
                                    void* packed, uint32_t packed_columns,
                                    uint32_t first_tile, uint32_t tile_stride,
                                    uint32_t first_column, void* stream) {
  return qllm_linear_pack_strided(source_bf16, rows, columns, columns, 1u, packed,
                                  packed_columns, first_tile, tile_stride, first_column,
                                  stream);
}

extern "C" int32_t qllm_linear_pack_strided(const void* source_bf16, uint32_t rows,
                                            uint32_t columns, uint64_t row_stride,
                                            uint64_t column_stride, void* packed,
                                            uint32_t packed_columns, uint32_t first_tile,
                                            uint32_t tile_stride, uint32_t first_column,
                                            void* stream) {
  const uint32_t padded = (columns + 63u) / 64u * 64u;
  if (!source_bf16 || !packed || !rows || !columns || !tile_stride ||
      packed_columns % 64u || first_column % 64u || !aligned16(packed) ||
      packed_columns < padded || first_column > packed_columns - padded)
    return fail(QLLM_INVALID_ARGUMENT, "invalid linear pack");
  const uint32_t chunks = padded / 32u;
  const uint64_t elements = uint64_t{(rows + 15u) / 16u} * chunks * 512u;
  const uint32_t blocks =
      static_cast<uint32_t>(elements / 256u < 65536u ? (elements + 255u) / 256u : 65536u);
  linear_pack_kernel<<<blocks, 256, 0, as_stream(stream)>>>(
      static_cast<const uint16_t*>(source_bf16), rows, columns, row_stride, column_stride,
      static_cast<uint16_t*>(packed), packed_columns / 32u, first_tile, tile_stride,
      first_column / 32u, chunks, elements);
  return launched("linear pack");
}

extern "C" int32_t qllm_linear_batch(const qllm_linear_segment* segments, uint32_t count,
                                     uint32_t batch, uint32_t element, void* stream) {
  if (!segments || !count || count > kMaximumSegments || !batch ||
      element > QLLM_ELEMENT_F32)
    return fail(QLLM_INVALID_ARGUMENT, "invalid linear batch");
  LinearArgs args{};
  args.count = count;
  args.batch = batch;
  for (uint32_t i = 0; i < count; ++i) {
    const qllm_linear_segment& s = segments[i];
    const bool gated = s.epilogue == QLLM_LINEAR_GATED;
    const bool partials = s.epilogue == QLLM_LINEAR_PARTIALS;
    const uint32_t outputs = gated ? s.rows / 2u : s.rows;
    if (!s.weights || !s.input || !s.output || !s.rows || !s.columns ||
        s.rows % (gated ? 32u : 16u) || s.columns % 64u || s.input_stride < s.columns ||
        s.input_stride % 8u || !s.output_columns ||
        s.output_columns > outputs || s.output_stride < s.output_columns ||
        s.epilogue > QLLM_LINEAR_PARTIALS || s.activation > QLLM_ACTIVATION_SILU ||
        (partials && (!s.splits || s.splits > 16u || batch > 64u)) ||
        !aligned16(s.weights) || !aligned16(s.input) || !aligned16(s.output))
      return fail(QLLM_INVALID_ARGUMENT, "invalid linear segment");
    args.segment[i] = s;
  }
  const auto hip_stream = as_stream(stream);
  if (element == QLLM_ELEMENT_F32) {
    for (uint32_t i = 0; i < count; ++i) {
      const qllm_linear_segment& s = segments[i];
      const uint32_t parts = s.epilogue == QLLM_LINEAR_PARTIALS ? s.splits : 1u;
      args.first_unit[i + 1] = args.first_unit[i] +
                               (s.rows + 63u) / 64u * ((batch + 63u) / 64u) * parts;
    }
    linear_f32_kernel<<<args.first_unit[count], 256, 0, hip_stream>>>(args);
    return launched("F32 linear");
  }
  if (batch <= 64u) {
    for (uint32_t i = 0; i < count; ++i) {
      const qllm_linear_segment& s = segments[i];
      const uint32_t parts = s.epilogue == QLLM_LINEAR_PARTIALS ? s.splits : 1u;
      const uint32_t tile_rows = s.epilogue == QLLM_LINEAR_GATED ? 32u : 16u;
      args.first_unit[i + 1] = args.first_unit[i] + s.rows / tile_rows * parts;
    }
    const uint32_t units = args.first_unit[count];
    const uint32_t threads = kSmallWaves * kWave;
    if (batch <= 16u)
      linear_small_kernel<1><<<units, threads, 0, hip_stream>>>(args);
    else if (batch <= 32u)
      linear_small_kernel<2><<<units, threads, 0, hip_stream>>>(args);
    else
      linear_small_kernel<4><<<units, threads, 0, hip_stream>>>(args);
    return launched("small-batch bf16 linear");
  }
  // the largest tiles that still give every CU two workgroups to hold
  if (all_tall_units<4, 8>(args) >= 512u) return launch_tall<4, 8>(args, hip_stream);
  if (all_tall_units<2, 8>(args) >= 384u) return launch_tall<2, 8>(args, hip_stream);
  return launch_tall<2, 4>(args, hip_stream);
}
