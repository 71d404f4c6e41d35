// model_runner.hpp -- what every model this backend serves can do, whatever step function stands behind it: one sequence, prompt in,
// logits or greedy tokens out.
#pragma once
#include <cstdint>
#include <string>
#include <vector>

namespace crabml_host {

class ModelRunner {
 public:
  virtual ~ModelRunner() = default;
  virtual const std::string& architecture() const = 0;
  virtual size_t vocab_size() const = 0;
  virtual size_t kv_cache_len() const = 0;
  virtual void reset() = 0;
  // the prompt (or its next portion) as batched passes; the last token's logits
  virtual std::vector<float> prefill(const std::vector<uint32_t>& tokens) = 0;
  // one token at cache position pos
  virtual std::vector<float> forward(size_t token, size_t pos) = 0;
  // `steps` greedy steps on the device, starting with `token`
  virtual std::vector<uint32_t> decode_greedy(size_t token, size_t steps) = 0;
};

}  // namespace crabml_host
