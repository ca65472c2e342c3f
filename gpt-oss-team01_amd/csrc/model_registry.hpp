// Model registry: a model file registers its architecture and how to open a checkpoint of it; a
// checkpoint is a folder with config.json ("architecture" names the class) and model.safetensors, or
// a flat .bin file.
#pragma once
#include <stdint.h>

#include <string>
#include <vector>

#include "common.hpp"
#include "json.hpp"

namespace gptoss {

// Read-only view of a safetensors file.
class SafeTensors {
 public:
  struct Tensor {
    std::string name, dtype;
    std::vector<long long> shape;
    const unsigned char *data;
    size_t bytes, elems;
  };
  ~SafeTensors();
  int open(const std::string &path);
  const Tensor *find(const std::string &name) const;
  // The tensor's elements as floats (BF16 and F32 files); an error unless its shape is the one given.
  int read(const std::string &name, const std::vector<long long> &shape, std::vector<float> *out) const;

 private:
  void *map_ = nullptr;
  size_t size_ = 0;
  std::vector<Tensor> tensors_;
};

struct ModelSource {
  std::string path;
  const Json *config = nullptr;          // folders: config.json
  const SafeTensors *weights = nullptr;  // folders: model.safetensors (nullptr with GPTOSS_ENGINE_SYNTHETIC)
};

struct OpenOptions {
  int max_batch, max_seq, flags;   // max_seq <= 0: as long as the model allows
  uint64_t seed;
};

using OpenModel = int (*)(const ModelSource &, const OpenOptions &, gptoss_engine **);

struct ModelClass {
  ModelClass(const char *architecture, OpenModel open, bool flat_file = false);
  const char *architecture;
  OpenModel open;
  bool flat_file;   // opens flat .bin files
};

}  // namespace gptoss
