// Request slots and their KV pages, shared by the providers: a request state
// leases one slot for its life and the slot owns the pages the request has
// filled.  Pages come from a pool that grows by allocation; a page is cleared
// once, when it is allocated.
#pragma once

#include <atomic>
#include <cstddef>
#include <cstdint>
#include <functional>
#include <memory>
#include <optional>
#include <vector>

namespace qllm {

class RequestSlots final {
 public:
  RequestSlots() = default;
  RequestSlots(std::uint32_t capacity, std::size_t pages_per_slot,
               std::uint64_t page_bytes);
  ~RequestSlots();
  RequestSlots(const RequestSlots&) = delete;
  RequestSlots& operator=(const RequestSlots&) = delete;
  RequestSlots(RequestSlots&& other) noexcept;
  RequestSlots& operator=(RequestSlots&& other) noexcept;

  struct Grant final {
    std::uint32_t slot{};
    // true while the request lives; whoever holds the grant clears it
    std::shared_ptr<std::atomic<bool>> lease;
  };
  // The lowest free slot, marked as leased; nothing when every slot is taken.
  [[nodiscard]] std::optional<Grant> take();

  [[nodiscard]] std::uint32_t capacity() const noexcept {
    return static_cast<std::uint32_t>(slots_.size());
  }
  [[nodiscard]] std::size_t pages_per_slot() const noexcept { return pages_per_slot_; }
  // Page pointers of a slot, in position order (null = none).
  [[nodiscard]] const std::vector<void*>& pages(std::uint32_t slot) const {
    return slots_.at(slot).pages;
  }
  // Makes pages first .. last of a slot exist; `publish` sees every page that
  // is new to it.
  using Publish = std::function<void(std::size_t page, void* pointer)>;
  void ensure(std::uint32_t slot, std::size_t first, std::size_t last,
              const Publish& publish);
  // Returns the pages of a slot for which `gone` holds to the pool.
  void recycle(std::uint32_t slot, const std::function<bool(std::size_t page)>& gone);
  [[nodiscard]] std::size_t live_pages() const noexcept;

 private:
  struct Slot final {
    std::shared_ptr<std::atomic<bool>> leased;
    std::vector<void*> pages;
  };
  void* obtain(std::uint32_t for_slot);
  void release() noexcept;
  std::vector<Slot> slots_;
  std::vector<void*> pool_;
  std::size_t pages_per_slot_{};
  std::uint64_t page_bytes_{};
};

}  // namespace qllm
