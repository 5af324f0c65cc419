// model_folder.cpp -- config.json and model.safetensors of a model folder.
#include "model_folder.h"

#include <cstring>
#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

namespace bh {
namespace {

std::string read_text(const std::string &path) {
  FILE *f = fopen(path.c_str(), "rb");
  if (!f)
    throw std::runtime_error("cannot open " + path);
  std::string s;
  char buf[1 << 16];
  size_t n;
  while ((n = fread(buf, 1, sizeof(buf), f)) > 0)
    s.append(buf, n);
  fclose(f);
  return s;
}

std::string shape_text(const std::vector<int64_t> &shape) {
  std::string s = "[";
  for (size_t i = 0; i < shape.size(); ++i)
    s += (i ? ", " : "") + std::to_string(shape[i]);
  return s + "]";
}

} // namespace

ModelFolder::ModelFolder(const std::string &path) {
  config_ = Json::parse(read_text(path + "/config.json"));
  const std::string file = path + "/model.safetensors";
  const int fd = open(file.c_str(), O_RDONLY | O_CLOEXEC);
  if (fd < 0)
    throw std::runtime_error("cannot open " + file);
  struct stat st;
  if (fstat(fd, &st) != 0 || st.st_size < 8) {
    close(fd);
    throw std::runtime_error(file + " is not a safetensors file");
  }
  map_bytes_ = (size_t)st.st_size;
  map_ = mmap(nullptr, map_bytes_, PROT_READ, MAP_PRIVATE, fd, 0);
  close(fd);
  if (map_ == MAP_FAILED) {
    map_ = nullptr;
    throw std::runtime_error("cannot map " + file);
  }
  try {
    const unsigned char *base = static_cast<const unsigned char *>(map_);
    uint64_t head = 0;
    for (int i = 7; i >= 0; --i)
      head = head << 8 | base[i];
    if (head > map_bytes_ - 8)
      throw std::runtime_error(file + ": the header is longer than the file");
    const Json j = Json::parse(reinterpret_cast<const char *>(base) + 8, (size_t)head);
    const size_t data = 8 + (size_t)head, room = map_bytes_ - data;
    for (const auto &m : j.object()) {
      if (m.first == "__metadata__")
        continue;
      TensorView t;
      t.dtype = m.second.at("dtype").string();
      for (const Json &d : m.second.at("shape").array()) {
        if (d.integer() < 0)
          throw std::runtime_error(file + ": negative size in " + m.first);
        t.shape.push_back(d.integer());
      }
      const auto &off = m.second.at("data_offsets").array();
      if (off.size() != 2 || off[0].integer() < 0 || off[1].integer() < off[0].integer() ||
          (uint64_t)off[1].integer() > room)
        throw std::runtime_error(file + ": bad offsets of " + m.first);
      t.bytes = (size_t)(off[1].integer() - off[0].integer());
      t.data = base + data + off[0].integer();
      tensors_.emplace(m.first, std::move(t));
    }
  } catch (...) {
    munmap(map_, map_bytes_);
    throw;
  }
}

ModelFolder::~ModelFolder() {
  if (map_)
    munmap(map_, map_bytes_);
}

int ModelFolder::size(const std::string &name, size_t axis) const {
  const auto it = tensors_.find(name);
  if (it == tensors_.end())
    throw std::runtime_error("no tensor " + name);
  if (axis >= it->second.shape.size() || it->second.shape[axis] <= 0 || it->second.shape[axis] > (1 << 24))
    throw std::runtime_error("tensor " + name + " has shape " + shape_text(it->second.shape));
  return (int)it->second.shape[axis];
}

const TensorView &ModelFolder::bf16(const std::string &name, const std::vector<int64_t> &shape) const {
  const auto it = tensors_.find(name);
  if (it == tensors_.end())
    throw std::runtime_error("no tensor " + name);
  const TensorView &t = it->second;
  if (t.dtype != "BF16" || t.shape != shape || t.bytes != (size_t)t.count() * 2)
    throw std::runtime_error("tensor " + name + " is " + t.dtype + " " + shape_text(t.shape) +
                             ", expected BF16 " + shape_text(shape));
  return t;
}

std::vector<float> ModelFolder::values(const std::string &name,
                                       const std::vector<int64_t> &shape) const {
  const TensorView &t = bf16(name, shape);
  std::vector<float> v((size_t)t.count());
  const unsigned char *p = static_cast<const unsigned char *>(t.data);
  for (size_t i = 0; i < v.size(); ++i) {
    const uint32_t u = (uint32_t)(p[2 * i] | p[2 * i + 1] << 8) << 16;
    std::memcpy(&v[i], &u, 4);
  }
  return v;
}

float ModelFolder::scalar(const std::string &name) const {
  const auto it = tensors_.find(name);
  if (it == tensors_.end())
    throw std::runtime_error("no tensor " + name);
  if (it->second.count() != 1)
    throw std::runtime_error("tensor " + name + " is not a single number");
  return values(name, it->second.shape)[0];
}

} // namespace bh
