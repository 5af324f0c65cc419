// model_folder.h -- a model as files: config.json and model.safetensors (8-byte
// little-endian header length, JSON header of name -> dtype, shape, data_offsets,
// then the data).  The tensor file is mapped, not read.
#pragma once

#include "common.h"
#include "json.h"

#include <map>
#include <memory>
#include <string>
#include <vector>

namespace bh {

struct TensorView {
  std::string dtype;          // as in the file: "BF16", "I32", ...
  std::vector<int64_t> shape;
  const void *data = nullptr; // host, inside the mapping
  size_t bytes = 0;
  int64_t count() const {
    int64_t n = 1;
    for (int64_t d : shape)
      n *= d;
    return n;
  }
};

class ModelFolder {
public:
  explicit ModelFolder(const std::string &path); // throws std::runtime_error
  ~ModelFolder();
  ModelFolder(const ModelFolder &) = delete;
  ModelFolder &operator=(const ModelFolder &) = delete;

  const Json &config() const { return config_; }
  std::string architecture() const { return config_.at("architecture").string(); }
  bool has(const std::string &name) const { return tensors_.count(name) != 0; }
  // a size that only the tensor's shape gives
  int size(const std::string &name, size_t axis) const;
  // the tensor, which must be bfloat16 of exactly this shape
  const TensorView &bf16(const std::string &name, const std::vector<int64_t> &shape) const;
  // a bfloat16 tensor of one element
  float scalar(const std::string &name) const;
  // the values of a bfloat16 tensor
  std::vector<float> values(const std::string &name, const std::vector<int64_t> &shape) const;

private:
  Json config_;
  std::map<std::string, TensorView> tensors_;
  void *map_ = nullptr;
  size_t map_bytes_ = 0;
};

} // namespace bh
