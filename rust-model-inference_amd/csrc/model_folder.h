// A model folder (config.json and model.safetensors) as a decoder session reads it.
#pragma once

#include <string>
#include <unordered_map>
#include <vector>

#include "json.h"
#include "rmi_internal.h"

struct RmiTensor {
    enum Dtype { kBf16, kF16, kF32, kI32, kOther } dtype = kOther;
    std::vector<uint64_t> shape;
    const uint8_t *data = nullptr;  // into the mapping
    uint64_t count = 0;
};

class RmiSafetensors {
  public:
    ~RmiSafetensors();
    bool open(const char *path);  // false + error text
    const RmiTensor *find(const std::string &name) const;
    size_t size() const { return tensors_.size(); }

  private:
    void *map_ = nullptr;
    size_t bytes_ = 0;
    std::unordered_map<std::string, RmiTensor> tensors_;
};

struct RmiModelFolder {
    RmiJson config;
    RmiSafetensors tensors;
    bool open(const char *dir);  // false + error text
};
// only config.json; false + error text
bool rmi_read_config(const char *dir, RmiJson *out);
// element i of a bf16 / f16 / f32 tensor's data as f32
float rmi_tensor_f32(const RmiTensor &t, uint64_t i);
// elements at .. at + n - 1 as bf16, to nearest even
void rmi_tensor_bf16(const RmiTensor &t, uint64_t at, uint64_t n, uint16_t *dst);
