// Runtime families: which loader serves a model's architecture, and the draft/verify generation where a family has one.  Every family
// registers itself (static objects in llama_loader.cpp, layered_loader.cpp, two_token.cpp), so the engine names none of them.
#pragma once

#include <map>
#include <memory>
#include <string>
#include <vector>

#include "../generation.h"
#include "model_support.h"

namespace esp {

using Environment = std::map<std::string, std::string>;

// Loads the model directory into a ready runtime.
using RuntimeLoader = int (*)(const MultiModelConfig &config, const std::string &modelDir, const Environment &environment, std::unique_ptr<DecoderRuntime> *out);
struct RuntimeFamilyRegistration {
    RuntimeFamilyRegistration(MultiModelConfig::Architecture architecture, RuntimeLoader loader);
};
RuntimeLoader find_runtime_loader(MultiModelConfig::Architecture architecture);   // nullptr: nothing runs this architecture

using DraftedGeneration = int (*)(DecoderRuntime &target, DecoderRuntime &draft, const uint32_t *prompt, int prompt_count, int max_tokens, std::vector<uint32_t> *out,
                                  TwoTokenStats *stats, GenerationTiming *timing);
struct DraftedGenerationRegistration {
    explicit DraftedGenerationRegistration(DraftedGeneration run);
};
DraftedGeneration find_drafted_generation();                                      // nullptr: the library was built without it

}  // namespace esp
