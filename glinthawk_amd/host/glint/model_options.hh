// Options of a model driver that are not part of the reference's settings.
#pragma once

#include <cstdint>

namespace glint {

constexpr uint64_t MAX_BATCH_SIZE = 1024; // models/llama2/base.hh:26

struct ModelOptions
{
  bool fused_attention { true };  // false: the reference's three unfused ops + score buffer
  bool fused_projections { true }; // with fused_attention: projections fused with the ops that follow them
  int balanced_attention { 0 };   // fused decode attention over equal runs of keys: 0 where the step's lengths call for it, 1 always (shapes that have it), -1 never
  bool allocate_logits { true };  // only needed when the classifier is hosted
  uint64_t seed { 1 };            // random initialisation of weights
  float weight_std { 0.02f };     // N(0, std) for every tensor, as the benchmark configurations say
  bool randomize { true };        // false: leave the weights for load() / set_*_tensor()
};

} // namespace glint
