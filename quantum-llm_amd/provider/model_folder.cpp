#include "model_folder.hpp"

#include "expert/runtime/sha256.hpp"

#include <cerrno>
#include <cstring>
#include <fstream>
#include <limits>
#include <sstream>
#include <stdexcept>

#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

namespace qllm {

class SafetensorsStore::Mapping final {
 public:
  explicit Mapping(const std::filesystem::path& path) {
    const int file = ::open(path.c_str(), O_RDONLY);
    if (file < 0)
      throw std::runtime_error("cannot open " + path.string() + ": " +
                               std::strerror(errno));
    struct stat facts {};
    if (::fstat(file, &facts) == 0 && facts.st_size > 0) {
      bytes_ = static_cast<std::size_t>(facts.st_size);
      data_ = ::mmap(nullptr, bytes_, PROT_READ, MAP_PRIVATE, file, 0);
    }
    (void)::close(file);
    if (!bytes_ || data_ == MAP_FAILED) {
      data_ = MAP_FAILED;
      throw std::runtime_error("cannot map " + path.string());
    }
  }
  ~Mapping() {
    if (data_ != MAP_FAILED) ::munmap(data_, bytes_);
  }
  Mapping(const Mapping&) = delete;
  Mapping& operator=(const Mapping&) = delete;
  [[nodiscard]] const std::byte* data() const noexcept {
    return static_cast<const std::byte*>(data_);
  }
  [[nodiscard]] std::size_t bytes() const noexcept { return bytes_; }

 private:
  void* data_{MAP_FAILED};
  std::size_t bytes_{};
};

namespace {

std::uint64_t element_bytes(std::string_view dtype) {
  if (dtype == "BF16" || dtype == "F16") return 2U;
  if (dtype == "F32" || dtype == "I32") return 4U;
  if (dtype == "I64" || dtype == "F64") return 8U;
  if (dtype == "I8" || dtype == "U8" || dtype == "BOOL") return 1U;
  throw std::runtime_error("safetensors dtype is not supported: " + std::string(dtype));
}

std::string read_text(const std::filesystem::path& path) {
  std::ifstream input(path, std::ios::binary);
  if (!input) throw std::runtime_error("cannot open " + path.string());
  std::ostringstream text;
  text << input.rdbuf();
  return text.str();
}

}  // namespace

er::Status SafetensorsStore::open(const std::filesystem::path& path,
                                  std::shared_ptr<SafetensorsStore>& store) {
  try {
    auto mapping = std::make_shared<const Mapping>(path);
    std::uint64_t header_bytes{};
    if (mapping->bytes() < sizeof(header_bytes))
      throw std::runtime_error("safetensors file has no header");
    std::memcpy(&header_bytes, mapping->data(), sizeof(header_bytes));
    if (header_bytes > mapping->bytes() - sizeof(header_bytes))
      throw std::runtime_error("safetensors header exceeds the file");
    const std::string_view text(reinterpret_cast<const char*>(mapping->data()) + 8U,
                                static_cast<std::size_t>(header_bytes));
    const std::byte* const data = mapping->data() + 8U + header_bytes;
    const std::uint64_t data_bytes = mapping->bytes() - 8U - header_bytes;
    const auto document = json::parse(text);
    auto fresh = std::make_shared<SafetensorsStore>();
    for (const auto& [name, value] : document.object("safetensors header")) {
      if (name == "__metadata__") continue;
      const auto& entry = value.object(name);
      auto tensor = std::make_shared<er::ImmutableModelTensor>();
      tensor->name = name;
      tensor->encoding = json::required(entry, "dtype", name).string(name);
      std::uint64_t elements = 1U;
      for (const auto& dimension : json::required(entry, "shape", name).array(name)) {
        const auto size = dimension.u64(name);
        if (!size || size > std::numeric_limits<std::uint32_t>::max() ||
            elements > std::numeric_limits<std::uint64_t>::max() / size)
          throw std::runtime_error("safetensors shape is invalid: " + name);
        tensor->shape.push_back(static_cast<std::uint32_t>(size));
        elements *= size;
      }
      if (tensor->shape.empty()) tensor->shape.push_back(1U);
      const auto& offsets = json::required(entry, "data_offsets", name).array(name);
      if (offsets.size() != 2U)
        throw std::runtime_error("safetensors offsets are invalid: " + name);
      const auto begin = offsets[0].u64(name);
      const auto end = offsets[1].u64(name);
      if (begin > end || end > data_bytes ||
          end - begin != elements * element_bytes(tensor->encoding))
        throw std::runtime_error("safetensors data range is invalid: " + name);
      tensor->data_bytes = end - begin;
      tensor->value = {"safetensors.tensor.v1", "host.mmap.readonly", mapping,
                       data + begin, end - begin};
      fresh->tensors_.emplace(name, std::move(tensor));
    }
    fresh->mapping_ = std::move(mapping);
    store = std::move(fresh);
    return er::Status::success();
  } catch (const std::exception& error) {
    return {er::ErrorCode::open_failed, error.what()};
  }
}

er::ResolveModelTensorResult SafetensorsStore::resolve(std::string_view name) {
  const auto found = tensors_.find(name);
  if (found == tensors_.end())
    return {{er::ErrorCode::invalid_argument,
             "model folder has no tensor: " + std::string(name)},
            {}};
  return {er::Status::success(), found->second};
}

bool is_model_folder(const std::filesystem::path& root) {
  return !std::filesystem::is_regular_file(root / "manifest.json") &&
         std::filesystem::is_regular_file(root / "config.json");
}

er::Status open_model_folder(const std::filesystem::path& root, ModelFolder& folder) {
  try {
    const auto text = read_text(root / "config.json");
    const auto document = json::parse(text);
    const auto& config = document.object("config");
    const auto& architecture =
        json::required(config, "architecture", "config").string("config.architecture");
    const ModelDesign* design = nullptr;
    for (const auto& known : model_designs())
      if (known.architecture == architecture) design = &known;
    if (!design)
      return {er::ErrorCode::invalid_argument,
              "no model design implements the architecture: " + architecture};
    std::shared_ptr<SafetensorsStore> store;
    if (auto status = SafetensorsStore::open(root / "model.safetensors", store);
        !status.ok())
      return status;
    folder.model = design->describe(config, *store);
    folder.model.content_hash =
        er::sha256({reinterpret_cast<const std::byte*>(text.data()), text.size()});
    folder.tensors = std::move(store);
    return er::validate_model_descriptor(folder.model);
  } catch (const std::exception& error) {
    return {er::ErrorCode::invalid_argument,
            std::string("invalid model folder: ") + error.what()};
  }
}

}  // namespace qllm
