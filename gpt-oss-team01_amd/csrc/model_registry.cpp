#include "model_registry.hpp"

#include <fcntl.h>
#include <stdio.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

namespace gptoss {

static std::vector<const ModelClass *> &classes() {
  static std::vector<const ModelClass *> list;   // filled by static constructors of the model files
  return list;
}

ModelClass::ModelClass(const char *architecture, OpenModel open, bool flat_file)
    : architecture(architecture), open(open), flat_file(flat_file) {
  classes().push_back(this);
}

SafeTensors::~SafeTensors() {
  if (map_) munmap(map_, size_);
}

int SafeTensors::open(const std::string &path) {
  const int fd = ::open(path.c_str(), O_RDONLY);
  GPTOSS_REQUIRE(fd >= 0, GPTOSS_ERR_IO, "cannot open %s", path.c_str());
  struct stat st;
  void *m = MAP_FAILED;
  if (fstat(fd, &st) == 0 && st.st_size >= 8) m = mmap(nullptr, st.st_size, PROT_READ, MAP_PRIVATE, fd, 0);
  ::close(fd);
  GPTOSS_REQUIRE(m != MAP_FAILED, GPTOSS_ERR_IO, "cannot map %s", path.c_str());
  map_ = m;
  size_ = st.st_size;
  const unsigned char *p = (const unsigned char *)m;
  uint64_t head = 0;
  for (int i = 0; i < 8; i++) head |= (uint64_t)p[i] << (8 * i);
  Json j;
  GPTOSS_REQUIRE(head <= size_ - 8 && Json::parse((const char *)p + 8, head, &j) && j.is(Json::OBJECT), GPTOSS_ERR_IO,
                 "%s: not a safetensors file", path.c_str());
  const unsigned char *data = p + 8 + head;
  const size_t data_bytes = size_ - 8 - head;
  for (const auto &f : j.fields) {
    if (f.first == "__metadata__") continue;
    const Json *dt = f.second.find("dtype"), *shape = f.second.find("shape"), *off = f.second.find("data_offsets");
    GPTOSS_REQUIRE(dt && shape && off && off->items.size() == 2, GPTOSS_ERR_IO, "%s: bad entry %s", path.c_str(),
                   f.first.c_str());
    Tensor t;
    t.name = f.first;
    t.dtype = dt->text;
    t.elems = 1;
    for (const Json &d : shape->items) {
      t.shape.push_back((long long)d.number);
      t.elems *= (size_t)d.number;
    }
    const size_t lo = (size_t)off->items[0].number, hi = (size_t)off->items[1].number;
    const size_t width = (t.dtype == "BF16" || t.dtype == "F16") ? 2 : (t.dtype == "F32" || t.dtype == "I32") ? 4 : 0;
    GPTOSS_REQUIRE(lo <= hi && hi <= data_bytes && (width == 0 || hi - lo == t.elems * width), GPTOSS_ERR_IO,
                   "%s: tensor %s lies outside the file", path.c_str(), f.first.c_str());
    t.data = data + lo;
    t.bytes = hi - lo;
    tensors_.push_back(std::move(t));
  }
  return GPTOSS_OK;
}

const SafeTensors::Tensor *SafeTensors::find(const std::string &name) const {
  for (const Tensor &t : tensors_)
    if (t.name == name) return &t;
  return nullptr;
}

int SafeTensors::read(const std::string &name, const std::vector<long long> &shape, std::vector<float> *out) const {
  const Tensor *t = find(name);
  GPTOSS_REQUIRE(t, GPTOSS_ERR_IO, "model.safetensors has no tensor %s", name.c_str());
  std::string want, got;
  for (long long d : shape) want += std::to_string(d) + " ";
  for (long long d : t->shape) got += std::to_string(d) + " ";
  GPTOSS_REQUIRE(t->shape == shape, GPTOSS_ERR_IO, "tensor %s has shape [ %s], expected [ %s]", name.c_str(), got.c_str(),
                 want.c_str());
  out->resize(t->elems);
  if (t->dtype == "F32") {
    memcpy(out->data(), t->data, t->bytes);
    return GPTOSS_OK;
  }
  GPTOSS_REQUIRE(t->dtype == "BF16", GPTOSS_ERR_IO, "tensor %s has dtype %s (BF16 or F32 expected)", name.c_str(),
                 t->dtype.c_str());
  for (size_t i = 0; i < t->elems; i++) {
    const uint32_t bits = ((uint32_t)t->data[2 * i] | (uint32_t)t->data[2 * i + 1] << 8) << 16;
    memcpy(&(*out)[i], &bits, 4);
  }
  return GPTOSS_OK;
}

static int open_folder(const std::string &path, const OpenOptions &o, gptoss_engine **out) {
  FILE *f = fopen((path + "/config.json").c_str(), "rb");
  GPTOSS_REQUIRE(f, GPTOSS_ERR_IO, "cannot open %s/config.json", path.c_str());
  std::string text;
  char buf[1 << 14];
  for (size_t n; (n = fread(buf, 1, sizeof(buf), f)) > 0;) text.append(buf, n);
  fclose(f);
  Json config;
  GPTOSS_REQUIRE(Json::parse(text.data(), text.size(), &config) && config.is(Json::OBJECT), GPTOSS_ERR_IO,
                 "%s/config.json is not a JSON object", path.c_str());
  const Json *arch = config.find("architecture");
  GPTOSS_REQUIRE(arch && arch->is(Json::STRING), GPTOSS_ERR_IO, "%s/config.json names no architecture", path.c_str());
  for (const ModelClass *c : classes())
    if (!c->flat_file && arch->text == c->architecture) {
      SafeTensors weights;
      if (!(o.flags & GPTOSS_ENGINE_SYNTHETIC)) {
        const int rc = weights.open(path + "/model.safetensors");
        if (rc != GPTOSS_OK) return rc;
      }
      ModelSource src;
      src.path = path;
      src.config = &config;
      src.weights = (o.flags & GPTOSS_ENGINE_SYNTHETIC) ? nullptr : &weights;
      return c->open(src, o, out);
    }
  return fail(GPTOSS_ERR_IO, "%s: no model class for architecture \"%s\"", path.c_str(), arch->text.c_str());
}

}  // namespace gptoss

using namespace gptoss;

extern "C" int gptoss_engine_open(const char *path, int max_batch, int max_seq, int flags, uint64_t seed,
                                  gptoss_engine **out) {
  GPTOSS_REQUIRE(path && out, GPTOSS_ERR_NULL, "engine_open: null pointer");
  *out = nullptr;
  GPTOSS_REQUIRE(max_batch >= 1, GPTOSS_ERR_DIM, "engine_open: max_batch must be at least 1");
  const OpenOptions o{max_batch, max_seq, flags, seed};
  struct stat st;
  GPTOSS_REQUIRE(stat(path, &st) == 0, GPTOSS_ERR_IO, "engine_open: %s does not exist", path);
  if (S_ISDIR(st.st_mode)) return open_folder(path, o, out);
  for (const ModelClass *c : classes())
    if (c->flat_file) {
      ModelSource src;
      src.path = path;
      return c->open(src, o, out);
    }
  return fail(GPTOSS_ERR_IO, "engine_open: no model class opens flat files (%s)", path);
}

extern "C" const char *gptoss_model_name(int i) {
  return i >= 0 && i < (int)classes().size() ? classes()[i]->architecture : nullptr;
}
