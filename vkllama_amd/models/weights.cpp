#include "models/weights.h"
#include "absl/strings/str_format.h"
#include "models/json.h"
#include <cmath>
#include <fcntl.h>
#include <string.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

namespace vkllama
{
namespace
{
std::vector<float>
widen (const uint8_t *data, size_t n)
{
  std::vector<float> out (n);
  for (size_t i = 0; i < n; ++i)
    {
      uint16_t h;
      memcpy (&h, data + 2 * i, 2);
      const uint32_t u = (uint32_t)h << 16;
      memcpy (&out[i], &u, 4);
    }
  return out;
}
}

absl::StatusOr<WeightView>
WeightSource::find (const std::string &name) const
{
  const auto it = views_.find (name);
  if (it == views_.end ())
    return absl::NotFoundError ("model tensor " + name + " is missing");
  return it->second;
}

absl::StatusOr<const uint16_t *>
WeightSource::matrix (const std::string &name, size_t rows, size_t cols) const
{
  auto v = find (name);
  VKLLAMA_STATUS_OK (v);
  if (v->dtype != BF16 || v->shape.size () != 2 || v->shape[0] != rows || v->shape[1] != cols
      || v->bytes != rows * cols * 2)
    return absl::InvalidArgumentError (
        absl::StrFormat ("model tensor %s: a bf16 matrix [%zu, %zu] is needed", name, rows, cols));
  return (const uint16_t *)v->data;
}

absl::StatusOr<std::vector<float> >
WeightSource::vector (const std::string &name, size_t n) const
{
  auto v = find (name);
  VKLLAMA_STATUS_OK (v);
  if (v->dtype != BF16 || v->shape.size () != 1 || v->shape[0] != n || v->bytes != n * 2)
    return absl::InvalidArgumentError (
        absl::StrFormat ("model tensor %s: a bf16 vector of %zu is needed", name, n));
  return widen (v->data, n);
}

absl::StatusOr<float>
WeightSource::scalar (const std::string &name) const
{
  auto v = find (name);
  VKLLAMA_STATUS_OK (v);
  if (v->dtype != BF16 || v->bytes != 2)
    return absl::InvalidArgumentError (absl::StrFormat ("model tensor %s: one bf16 value is needed", name));
  return widen (v->data, 1)[0];
}

SafetensorsFile::~SafetensorsFile ()
{
  if (map_)
    munmap (map_, size_);
}

absl::StatusOr<std::shared_ptr<SafetensorsFile> >
SafetensorsFile::open (const std::string &path)
{
  std::shared_ptr<SafetensorsFile> f (new SafetensorsFile ());
  const int fd = ::open (path.c_str (), O_RDONLY | O_CLOEXEC);
  if (fd < 0)
    return absl::NotFoundError ("cannot open " + path);
  struct stat st;
  void *p = MAP_FAILED;
  if (fstat (fd, &st) == 0 && st.st_size >= 8)
    p = mmap (nullptr, (size_t)st.st_size, PROT_READ, MAP_PRIVATE, fd, 0);
  ::close (fd);
  if (p == MAP_FAILED)
    return absl::InvalidArgumentError ("not a safetensors file: " + path);
  f->map_ = p, f->size_ = (size_t)st.st_size;
  const uint8_t *base = (const uint8_t *)p;
  uint64_t hn = 0;
  for (int i = 7; i >= 0; --i)
    hn = hn << 8 | base[i];
  if (hn > f->size_ - 8)
    return absl::InvalidArgumentError ("not a safetensors file: " + path);
  auto head = Json::parse ((const char *)base + 8, (size_t)hn);
  VKLLAMA_STATUS_OK (head);
  const size_t room = f->size_ - 8 - (size_t)hn;
  for (const auto &kv : head->members ())
    {
      if (kv.first == "__metadata__")
        continue;
      const Json &t = kv.second, &off = t["data_offsets"];
      const std::string &dt = t["dtype"].string ();
      WeightView v;
      if (dt == "BF16")
        v.dtype = BF16;
      else if (dt == "F32")
        v.dtype = FP32;
      else if (dt == "F16")
        v.dtype = FP16;
      else if (dt == "I32" || dt == "U32")
        v.dtype = UINT32;
      else
        continue; // (a type no model here reads; a model that needs the tensor reports it missing)
      size_t n = v.dtype == FP32 || v.dtype == UINT32 ? 4 : 2;
      for (const Json &d : t["shape"].items ())
        {
          const double x = d.number ();
          if (d.kind () != Json::Number || x < 0 || x != std::floor (x) || x > 1e12)
            return absl::InvalidArgumentError ("safetensors: bad shape of " + kv.first);
          v.shape.push_back ((size_t)x);
          if (x > 0 && n > (size_t)1 << 50)
            return absl::InvalidArgumentError ("safetensors: bad shape of " + kv.first);
          n *= (size_t)x;
        }
      if (off.items ().size () != 2)
        return absl::InvalidArgumentError ("safetensors: bad offsets of " + kv.first);
      const double lo = off.items ()[0].number (), hi = off.items ()[1].number ();
      if (!(lo >= 0 && lo <= hi && hi <= (double)room) || (size_t)(hi - lo) != n)
        return absl::InvalidArgumentError ("safetensors: bad offsets of " + kv.first);
      v.data = base + 8 + hn + (size_t)lo;
      v.bytes = n;
      f->add (kv.first, v);
    }
  return f;
}
}
