// Loads layered models into the GPU-resident runtime: a model directory (config.json, model.safetensors), or seeded random weights
// of a configuration for measurements and tests.
#pragma once

#include <memory>
#include <string>

#include "../layered_runtime.h"
#include "model_support.h"

namespace esp {

// The engine-level description of a layered model directory (architecture layered; the context length is the caller's choice).
int layered_model_config(const std::string &model_dir, int max_seq, MultiModelConfig *out);
int load_layered_model(const std::string &model_dir, const LayeredOptions &options, std::unique_ptr<LayeredRuntime> *out);
// Weights ~ uniform with standard deviation `std_dev` (matrices), norms around 1, sinks around 0.
int make_synthetic_layered_model(const LayeredConfig &config, const LayeredOptions &options, uint64_t seed, float std_dev, std::unique_ptr<LayeredRuntime> *out);

}  // namespace esp
