// Declarations shared by the host-side translation units of libpuppygrad_hip.so
// (not part of the public contract in include/puppygrad_hip.h).
#pragma once

#include <string>
#include <vector>

#include "../../include/puppygrad_hip.h"

namespace pgh {

// Vectors a kernel stages in LDS (a LayerNorm row, the input of a matrix-vector product, the
// scores of the generic attention kernel) take this many floats at most: 64 KiB of dynamic LDS
// less the kernels' small static blocks.
constexpr unsigned long long kMaxStagedFloats = 16320;

// Records `msg` as the calling thread's last error message and returns `s`.
__attribute__((visibility("hidden"))) pg_status fail(pg_status s, const std::string& msg);

// Gpt2Config::validate (src/models/gpt2/rust.rs:60-95) plus this backend's limits.
__attribute__((visibility("hidden"))) pg_status validate_config(const pg_gpt2_config& c);

// One tensor of a store as it lies in the file.
struct TensorView {
  enum Dtype { F32, BF16, I32 } dtype = F32;
  const unsigned char* data = nullptr;
  std::vector<uint64_t> shape;
  uint64_t count = 0;
};
// PG_ASSET when the tensor is missing or has another dtype.
__attribute__((visibility("hidden"))) pg_status find_tensor(const pg_tensor_store& store, const std::string& name,
                                                            TensorView* out);

// Architecture name of a model ("gpt2" or the name config.json gives a stack model).
__attribute__((visibility("hidden"))) const char* architecture_of(const pg_model* m);

}  // namespace pgh
