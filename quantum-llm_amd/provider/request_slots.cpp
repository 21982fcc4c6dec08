#include "request_slots.hpp"

#include "host_support.hpp"

#include <hip/hip_runtime.h>

#include <algorithm>
#include <stdexcept>
#include <utility>

namespace qllm {

RequestSlots::RequestSlots(std::uint32_t capacity, std::size_t pages_per_slot,
                           std::uint64_t page_bytes)
    : slots_(std::max(1U, capacity)), pages_per_slot_(pages_per_slot),
      page_bytes_(page_bytes) {
  for (auto& slot : slots_) {
    slot.leased = std::make_shared<std::atomic<bool>>(false);
    slot.pages.assign(pages_per_slot, nullptr);
  }
}

RequestSlots::~RequestSlots() { release(); }

RequestSlots::RequestSlots(RequestSlots&& other) noexcept
    : slots_(std::exchange(other.slots_, {})), pool_(std::exchange(other.pool_, {})),
      pages_per_slot_(other.pages_per_slot_), page_bytes_(other.page_bytes_) {}

RequestSlots& RequestSlots::operator=(RequestSlots&& other) noexcept {
  if (this != &other) {
    release();
    slots_ = std::exchange(other.slots_, {});
    pool_ = std::exchange(other.pool_, {});
    pages_per_slot_ = other.pages_per_slot_;
    page_bytes_ = other.page_bytes_;
  }
  return *this;
}

void RequestSlots::release() noexcept {
  for (auto& slot : slots_)
    for (void* page : slot.pages)
      if (page) (void)hipFree(page);
  for (void* page : pool_) (void)hipFree(page);
  slots_.clear();
  pool_.clear();
}

std::optional<RequestSlots::Grant> RequestSlots::take() {
  for (std::uint32_t index = 0; index < slots_.size(); ++index) {
    auto& lease = slots_[index].leased;
    if (lease->load(std::memory_order_acquire)) continue;
    lease->store(true, std::memory_order_release);
    return Grant{index, lease};
  }
  return std::nullopt;
}

// The pool, else a page of a slot nobody leases, else fresh memory.
void* RequestSlots::obtain(std::uint32_t for_slot) {
  if (pool_.empty())
    for (std::uint32_t index = 0; index < slots_.size(); ++index)
      if (index != for_slot && !slots_[index].leased->load(std::memory_order_acquire))
        recycle(index, [](std::size_t) { return true; });
  if (!pool_.empty()) {
    void* page = pool_.back();
    pool_.pop_back();
    return page;
  }
  DeviceBuffer page(page_bytes_, "allocate KV page");
  hip_check(hipMemset(page.get(), 0, page_bytes_), "clear KV page");
  return page.release();
}

void RequestSlots::ensure(std::uint32_t slot, std::size_t first, std::size_t last,
                          const Publish& publish) {
  auto& pages = slots_.at(slot).pages;
  if (last >= pages.size())
    throw std::runtime_error("KV position exceeds the configured context");
  for (std::size_t page = first; page <= last; ++page) {
    if (pages[page]) continue;
    pages[page] = obtain(slot);
    publish(page, pages[page]);
  }
}

void RequestSlots::recycle(std::uint32_t slot,
                           const std::function<bool(std::size_t page)>& gone) {
  auto& pages = slots_.at(slot).pages;
  for (std::size_t page = 0; page < pages.size(); ++page) {
    if (!pages[page] || !gone(page)) continue;
    pool_.push_back(pages[page]);
    pages[page] = nullptr;
  }
}

std::size_t RequestSlots::live_pages() const noexcept {
  std::size_t count = 0;
  for (const auto& slot : slots_)
    count += static_cast<std::size_t>(
        std::count_if(slot.pages.begin(), slot.pages.end(),
                      [](const void* page) { return page != nullptr; }));
  return count;
}

}  // namespace qllm
