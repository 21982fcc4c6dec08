// Replays a trace: token ids in, logits out, through the same opened model,
// program and provider the worker serves from.
//
//   usage: qllm-trace --model DIR --dtype bfloat16|float32 --out DIR
//            --max-tokens N
//
// Reads one JSON object a line from standard input:
//   {"step": n, "entries": [{"id": "a", "tokens": [..], "want": [..]}], "end": [..]}
// An entry brings a request's next tokens; `want` lists the places among them
// whose logits are asked for.  They go to DIR/<n>.f32 in the order of the
// entries (little-endian F32, [wanted, vocabulary]), and "done <n>" is printed.
// Requests under "end" are finished after the step and give back what they
// hold.
#include "json_reader.hpp"
#include "model_host.hpp"
#include "wire.hpp"

#include <algorithm>
#include <cstdint>
#include <cstdio>
#include <filesystem>
#include <fstream>
#include <iostream>
#include <map>
#include <memory>
#include <stdexcept>
#include <string>
#include <string_view>
#include <vector>

namespace qllm {
namespace {

void require(bool holds, std::string_view message) {
  if (!holds) throw std::runtime_error(std::string(message));
}

void require_ok(const er::Status& status) { require(status.ok(), status.message()); }

struct Options final {
  std::filesystem::path model, out;
  std::string dtype;
  std::uint32_t max_tokens{};
};

Options parse(int argc, char** argv) {
  std::map<std::string, std::string, std::less<>> given;
  for (int index = 1; index + 1 < argc; index += 2) given[argv[index]] = argv[index + 1];
  require(argc % 2 == 1, "every option takes a value");
  const auto value = [&](const char* name) {
    const auto found = given.find(name);
    require(found != given.end(), std::string("missing option ") + name);
    return found->second;
  };
  Options options;
  options.model = value("--model");
  options.out = value("--out");
  options.dtype = value("--dtype");
  options.max_tokens = wire::decimal<std::uint32_t>(value("--max-tokens"));
  require(options.dtype == "bfloat16" || options.dtype == "float32",
          "--dtype is bfloat16 or float32");
  return options;
}

std::vector<std::uint32_t> integers(const json::Value& value, std::string_view where) {
  std::vector<std::uint32_t> out;
  for (const auto& item : value.array(where)) {
    const auto number = item.u64(where);
    require(number <= 0xffffffffU, "integer is out of range");
    out.push_back(static_cast<std::uint32_t>(number));
  }
  return out;
}

class Replay final {
 public:
  Replay(const ModelHost& host, std::filesystem::path out)
      : host_(host), out_(std::move(out)) {}

  void step(std::string_view line) {
    const auto document = json::parse(line);
    const auto& step = document.object("step");
    const auto number = json::required(step, "step", "step").u64("step.step");
    std::vector<float> logits;
    bool wanted = false;
    for (const auto& item : json::required(step, "entries", "step").array("entries")) {
      const auto& entry = item.object("entry");
      const auto& id = json::required(entry, "id", "entry").string("entry.id");
      const auto tokens =
          integers(json::required(entry, "tokens", "entry"), "entry.tokens");
      const auto want = integers(json::required(entry, "want", "entry"), "entry.want");
      wanted = wanted || !want.empty();
      run(id, tokens, want, logits);
    }
    if (wanted) {
      std::ofstream file(out_ / (std::to_string(number) + ".f32"), std::ios::binary);
      file.write(reinterpret_cast<const char*>(logits.data()),
                 static_cast<std::streamsize>(logits.size() * sizeof(float)));
      file.close();
      require(static_cast<bool>(file), "cannot write logits");
    }
    for (const auto& id : json::required(step, "end", "step").array("end"))
      requests_.erase(id.string("end"));
    std::cout << "done " << number << std::endl;
  }

 private:
  struct Request final {
    std::unique_ptr<ProgramSession> session;
    std::uint32_t position{};
  };

  void run(const std::string& id, const std::vector<std::uint32_t>& tokens,
           const std::vector<std::uint32_t>& want, std::vector<float>& logits) {
    require(!tokens.empty(), "entry brings no tokens");
    auto& request = requests_[id];
    if (!request.session)
      require_ok(host_.begin(greedy_request(++last_id_), request.session));
    // rows come back in ascending order: asked for once each, handed out as listed
    std::vector<std::uint32_t> rows(want);
    std::sort(rows.begin(), rows.end());
    rows.erase(std::unique(rows.begin(), rows.end()), rows.end());
    require(rows.empty() || rows.back() < tokens.size(), "wanted place exceeds the entry");
    std::vector<float> computed;
    require_ok(host_.run_all(*request.session, tokens, request.position, rows, &computed)
                   .status);
    request.position += static_cast<std::uint32_t>(tokens.size());
    const std::size_t width = host_.model().vocab_size;
    for (const auto place : want) {
      const auto at = static_cast<std::size_t>(
          std::lower_bound(rows.begin(), rows.end(), place) - rows.begin());
      logits.insert(logits.end(), computed.begin() + static_cast<std::ptrdiff_t>(at * width),
                    computed.begin() + static_cast<std::ptrdiff_t>((at + 1U) * width));
    }
  }

  const ModelHost& host_;
  std::filesystem::path out_;
  std::map<std::string, Request, std::less<>> requests_;
  std::uint64_t last_id_{};
};

int run(int argc, char** argv) {
  const Options options = parse(argc, argv);
  ArtifactProviderOptions provider;
  // whole pages, and room for what a request may hold beyond the count
  provider.max_context = (options.max_tokens + 256U + 255U) / 256U * 256U;
  provider.capacity = 8U;
  provider.kv_cache_dtype = options.dtype == "float32" ? "fp32" : "bf16";
  std::unique_ptr<ModelHost> host;
  require_ok(ModelHost::open(options.model, provider, host));
  Replay replay(*host, options.out);
  std::string line;
  while (std::getline(std::cin, line))
    if (!line.empty()) replay.step(line);
  return 0;
}

}  // namespace
}  // namespace qllm

int main(int argc, char** argv) {
  try {
    return qllm::run(argc, argv);
  } catch (const std::exception& error) {
    std::cerr << "qllm trace: " << error.what() << '\n';
    return 1;
  }
}
