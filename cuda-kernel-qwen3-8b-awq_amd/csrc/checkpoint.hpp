// A model folder's files: config.json as a small JSON tree, model.safetensors as named tensors in a mapped file.
#pragma once
#include <stdint.h>

#include <map>
#include <string>
#include <utility>
#include <vector>

// One JSON value.  Numbers are binary64; object members keep their order.
struct Json {
  enum Type { Null, Bool, Number, String, Array, Object } type = Null;
  bool boolean = false;
  double number = 0.0;
  std::string str;
  std::vector<Json> items;
  std::vector<std::pair<std::string, Json>> members;

  const Json* find(const std::string& key) const;  // nullptr: not an object, or no such member
  bool is(Type t) const { return type == t; }
};
// the whole text must be one value; false: `err` says where it is not
bool json_parse(const char* text, size_t n, Json* out, std::string* err);
int awq_read_json(const std::string& path, Json* out);
// "architecture" of dir/config.json
int awq_config_architecture(const std::string& dir, std::string* out);

struct Tensor {
  std::string dtype;  // as the file names it: BF16, F32, I32, ...
  std::vector<int64_t> shape;
  const void* data = nullptr;
  int64_t bytes = 0;
};

// model.safetensors: an 8-byte length, that many bytes of JSON (name -> dtype, shape, data_offsets), the data
class Safetensors {
 public:
  Safetensors() = default;
  ~Safetensors();
  Safetensors(const Safetensors&) = delete;
  Safetensors& operator=(const Safetensors&) = delete;
  int open(const std::string& path);
  const Tensor* find(const std::string& name) const;
  const std::map<std::string, Tensor>& tensors() const { return tensors_; }

 private:
  void* map_ = nullptr;
  size_t size_ = 0;
  std::map<std::string, Tensor> tensors_;
};
