// safetensors.h -- read-only view of a model.safetensors file: an 8-byte
// little-endian length, that many bytes of JSON (name -> dtype, shape,
// data_offsets), then the data.
#pragma once
#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <string>
#include <vector>

#include "json.h"

namespace ffmi {

class SafeTensors {
 public:
  struct Tensor {
    std::string dtype;
    std::vector<long> shape;
    const char *data = nullptr;
    size_t bytes = 0;
  };
  ~SafeTensors() {
    if (map_) munmap(map_, size_);
  }
  bool open(const std::string &path) {
    const int fd = ::open(path.c_str(), O_RDONLY);
    if (fd < 0) return false;
    struct stat st;
    bool ok = fstat(fd, &st) == 0 && st.st_size >= 8;
    if (ok) {
      size_ = (size_t)st.st_size;
      void *m = mmap(nullptr, size_, PROT_READ, MAP_PRIVATE, fd, 0);
      if ((ok = m != MAP_FAILED)) map_ = m;
    }
    ::close(fd);
    return ok && parse();
  }
  const Tensor *find(const std::string &name) const {
    auto it = tensors_.find(name);
    return it == tensors_.end() ? nullptr : &it->second;
  }

 private:
  bool parse() {
    const char *p = (const char *)map_;
    uint64_t n;
    memcpy(&n, p, 8);
    if (n > size_ - 8) return false;
    Json h;
    if (!Json::parse(p + 8, n, &h) || h.type != Json::OBJ) return false;
    const size_t base = 8 + n;
    for (const auto &kv : h.obj) {
      if (kv.first == "__metadata__") continue;
      const Json *off = kv.second.find("data_offsets"), *shape = kv.second.find("shape");
      if (!off || off->arr.size() != 2 || !shape) return false;
      Tensor t;
      t.dtype = kv.second.text("dtype");
      for (const Json &d : shape->arr) t.shape.push_back((long)d.num);
      const double a = off->arr[0].num, b = off->arr[1].num;
      if (a < 0 || b < a || b > (double)(size_ - base)) return false;
      t.data = p + base + (size_t)a;
      t.bytes = (size_t)b - (size_t)a;
      tensors_[kv.first] = t;
    }
    return true;
  }
  void *map_ = nullptr;
  size_t size_ = 0;
  std::map<std::string, Tensor> tensors_;
};

}  // namespace ffmi
