// MI355X provider for mixed-layer decoders: layers of different kinds on one
// F32 residual stream, bf16 weights, bf16 or F32 arithmetic.
//
// Every layer is one operation.  A parallel block: one norm launch (which also
// adds the partial sums of the layer before), one launch for all projections
// of mixer and feed-forward with the activation in its epilogue, the mixer,
// and one launch for both output projections, laid side by side along K.
// A sandwich block runs its mixer and its feed-forward one after the other,
// each between a norm of its input and a norm of its output; the latter is taken
// by the norm launch that follows, with the sublayer's partial sums.
// Five mixers: windowed attention with mixed heads and latent attention over the
// paged cache, and the generalised delta rule, the bonus recurrence over
// token-shifted inputs and gated linear attention, whose states live beside the
// pages in their request's slot.
//
// A batch is any run of consecutive tokens of one request.  A single token is
// replayed from a captured graph: kernels read token, position and slot from
// device words.
#pragma once

#include "decoder_provider.hpp"
#include "host_support.hpp"
#include "request_slots.hpp"
#include "token_selector.hpp"

#include "expert/runtime/worker_provider.hpp"
#include "qllm_kernels.h"

#include <atomic>
#include <cstdint>
#include <map>
#include <memory>
#include <mutex>
#include <span>
#include <string>
#include <vector>

namespace qllm {

inline constexpr char kEmbeddingBf16[] = "embedding.lookup.bf16.v1";
inline constexpr char kBlockWindowedAttention[] =
    "block.parallel.windowed-attention.mixed-heads.v1";
inline constexpr char kBlockDelta[] = "block.parallel.general-delta.v1";
inline constexpr char kBlockBonus[] = "block.parallel.bonus-recurrence.token-shift.v1";
inline constexpr char kBlockLatentAttention[] = "block.sandwich.latent-attention.v1";
inline constexpr char kBlockGatedLinear[] = "block.sandwich.gated-linear-attention.v1";
inline constexpr char kHeadBf16[] = "head.rmsnorm.logits.bf16.v1";

// Parameter value_blend of a windowed attention block.
inline constexpr std::uint64_t kValuesKept = 1U;      // its values are kept for others
inline constexpr std::uint64_t kValuesBlended = 2U;   // the kept ones are blended in

struct MixedGeometry final {
  std::uint32_t hidden{};
  std::uint32_t vocabulary{};
  std::uint32_t max_context{};
  std::uint32_t kv_page_tokens{256};
  std::uint32_t capacity{1};
  // rows one program batch may hold (0 = 4096 or the context, if shorter)
  std::uint32_t chunk_rows{};
  std::uint32_t element{QLLM_ELEMENT_BF16};
};

class MixedRequestState final : public er::IOperationProviderRequestState {
 public:
  ~MixedRequestState() override {
    if (lease) lease->store(false, std::memory_order_release);
  }
  std::uint32_t slot{};
  std::shared_ptr<std::atomic<bool>> lease;
  std::uint32_t position{};                 // of the next token
  std::vector<std::uint32_t> logit_rows;    // asked for in the next batch
};

class Mi355MixedProvider final : public DecoderProvider {
 public:
  explicit Mi355MixedProvider(const MixedGeometry& geometry);
  ~Mi355MixedProvider() override;
  Mi355MixedProvider(const Mi355MixedProvider&) = delete;
  Mi355MixedProvider& operator=(const Mi355MixedProvider&) = delete;

  [[nodiscard]] er::PrepareOperationResult prepare(
      const er::OperationPreparationContext& context) override;
  [[nodiscard]] er::CreateOperationRequestStateResult create_request_state(
      const er::ProgramRequestContext& request) override;
  // One operation at a time ...
  [[nodiscard]] er::OperationExecutionHandle execute(
      const er::IPreparedOperation& operation,
      const std::shared_ptr<er::IOperationProviderRequestState>& request_state,
      const er::OperationInvocation& invocation) override;
  // ... or the whole program, with the partial sums of a layer left to the next
  // and a single token replayed from a captured graph.
  [[nodiscard]] bool supports_program_sequence(
      const er::CompiledModelProgram& program) const noexcept override;
  [[nodiscard]] er::OperationExecutionHandle execute_program_sequence(
      const std::shared_ptr<er::IOperationProviderRequestState>& state,
      const er::ProgramSequenceInvocation& invocation) override;
  [[nodiscard]] er::Status rebind_request_state(
      const std::shared_ptr<er::IOperationProviderRequestState>& state,
      const er::ProgramRequestContext& request) override;

  [[nodiscard]] er::Status set_logit_rows(
      const std::shared_ptr<er::IOperationProviderRequestState>& state,
      std::vector<std::uint32_t> rows) override;
  [[nodiscard]] std::map<std::string, std::uint64_t, std::less<>> telemetry()
      const override;
  [[nodiscard]] er::ExecutionProviderModule::ServiceContract service_contract()
      const override;
  // Allocates what depends on all operations: pages, states, workspaces.  The
  // module's finalize hook; the first request does it otherwise.
  [[nodiscard]] er::Status finalize();

  // Copies the residual stream of the last batch, F32 [rows][hidden].
  [[nodiscard]] er::Status copy_hidden(std::uint32_t rows, float* host);

 private:
  enum class Kind { embedding, attention, latent, delta, bonus, gated, head };
  struct Matrix final {
    DeviceBuffer data;
    std::uint32_t rows{};      // packed
    std::uint32_t columns{};   // packed
  };
  struct Block;
  struct PreparedOperation;

  // loading
  struct Part final {
    const er::ImmutableModelTensor* tensor{};
    std::uint32_t first_tile{};
    std::uint32_t tile_stride{1};
    std::uint32_t first_column{};
  };
  Matrix pack(std::uint32_t rows, std::uint32_t columns, std::span<const Part> parts);
  DeviceBuffer upload_raw(const er::ImmutableModelTensor& tensor);
  DeviceBuffer upload_f32(const er::ImmutableModelTensor& tensor, std::uint64_t elements);
  // Packed per-head matrices: rows of the tensor cut into `heads` parts of `size`
  // rows, each padded to `padded` rows of the packed matrix (of its columns, when
  // transposed).
  DeviceBuffer pack_heads(const er::ImmutableModelTensor& tensor, std::uint32_t heads,
                          std::uint32_t size, std::uint32_t padded, bool transposed);
  DeviceBuffer upload_frequencies(const er::ParameterMap& parameters, std::uint32_t dims);
  void prepare_block(Block& block, const er::OperationPreparationContext& context);
  void prepare_attention(Block& block, const er::OperationPreparationContext& context);
  void prepare_latent(Block& block, const er::OperationPreparationContext& context);
  void prepare_recurrence(Block& block, const er::OperationPreparationContext& context);

  // execution
  void finalize_locked();
  std::size_t scratch_bytes_for(std::uint32_t rows, std::uint32_t last_position) const;
  void ensure_workspace(std::uint32_t rows, std::uint32_t last_position);
  void begin_batch(MixedRequestState& state, std::span<const std::uint32_t> tokens,
                   std::uint32_t first_position);
  void enqueue_embedding(std::uint32_t rows);
  void enqueue_block(Block& block, std::uint32_t rows, std::uint32_t last_position);
  void enqueue_sandwich(Block& block, std::uint32_t rows, std::uint32_t last_position);
  void enqueue_mixer(Block& block, std::uint32_t rows, std::uint32_t last_position);
  // Norm launch over the stream with what partial sums are pending.
  [[nodiscard]] qllm_stream_norm_launch stream_norm(std::uint32_t rows, float epsilon);
  void enqueue_latent(Block& block, std::uint32_t rows, std::uint32_t last_position);
  void enqueue_attention(Block& block, std::uint32_t rows, std::uint32_t last_position);
  void enqueue_recurrence(Block& block, std::uint32_t rows);
  void settle_stream(std::uint32_t rows);   // adds what partial sums are pending
  // Logits of rows of the batch, into logits_ (at most kLogitRows).
  void enqueue_head(std::uint32_t batch_rows, std::uint32_t first, std::uint32_t count,
                    bool gather);
  struct HeadResult final {
    std::shared_ptr<std::vector<float>> logits;
    std::uint32_t token{};
  };
  HeadResult finish_batch(MixedRequestState& state, std::uint32_t rows,
                          const er::ProgramRequestContext& request, bool head_enqueued);
  void launch_step_graph();
  void release_pages(const MixedRequestState& state);
  [[nodiscard]] er::OperationExecutionResult outputs_for(
      const PreparedOperation& operation,
      std::map<std::string, er::ExecutionValue, std::less<>> values) const;
  [[nodiscard]] er::ExecutionValue hidden_value(std::uint32_t rows) const;
  void release();

  static constexpr std::uint32_t kLogitRows = 64U;

  MixedGeometry g_;
  mutable std::mutex mutex_;
  void* stream_{};
  std::shared_ptr<const void> lifetime_;
  std::uint64_t weight_bytes_{};
  bool finalized_{};

  DeviceBuffer embedding_;
  float embedding_scale_{1.0F};
  std::vector<std::unique_ptr<Block>> blocks_;
  Matrix head_;
  DeviceBuffer final_norm_;
  float final_epsilon_{};

  // requests
  RequestSlots slots_;
  std::uint64_t page_bytes_{};
  DeviceBuffer page_table_;      // [slots][pages per slot]
  std::uint64_t state_floats_{}; // per slot
  DeviceBuffer states_;
  DeviceBuffer presence_;        // [slots][vocabulary]
  bool pages_expire_{};          // every attention layer has a window
  std::uint32_t widest_window_{};
  std::uint32_t most_sinks_{};

  // workspace
  std::uint32_t workspace_rows_{};
  std::uint32_t mixer_stride_{}, projection_stride_{}, joined_stride_{};
  std::uint32_t shift_inputs_{};
  DeviceBuffer step_;            // position, slot, rows, spare; then tokens
  DeviceBuffer hidden_[2];
  DeviceBuffer inputs_;          // mixer inputs (several for token shift), then ffn's
  DeviceBuffer projections_;
  DeviceBuffer joined_;          // mixer output | activation
  DeviceBuffer query_;
  DeviceBuffer query_latents_;   // normed, element
  DeviceBuffer queries_;         // F32, from query latents
  DeviceBuffer kept_values_;
  DeviceBuffer shift_last_;
  DeviceBuffer partials_;
  DeviceBuffer scratch_;         // attention splits, recurrence preparation
  std::size_t scratch_bytes_{};
  DeviceBuffer head_input_;
  DeviceBuffer gather_;
  DeviceBuffer logits_;
  DeviceBuffer argmax_;
  DeviceBuffer select_workspace_;
  std::size_t select_workspace_bytes_{};
  std::unique_ptr<TokenSelector> selector_;
  void* staging_{};              // pinned: step words and tokens
  std::size_t staging_words_{};

  std::uint32_t stream_index_{}; // which of hidden_ holds the stream
  std::uint32_t pending_partials_{};
  // the norm pending partial sums pass on their way into the stream, if any
  struct Branch final {
    const float* weight{};
    float scale{};
    float epsilon{};
  };
  Branch pending_branch_;
  std::uint32_t batch_rows_{};
  void* step_graph_{};
  bool use_graphs_{true};
  bool step_warm_{};
  std::uint32_t step_stream_index_{};   // where a replayed step leaves the stream

  std::uint64_t program_steps_{};
  std::uint64_t prompt_rows_{};
  std::uint64_t graph_launches_{};
};

[[nodiscard]] er::WorkerProviderDefinition make_mi355_mixed_provider();
[[nodiscard]] er::Status validate_mixed_descriptor(const er::ModelDescriptor& model);

}  // namespace qllm
