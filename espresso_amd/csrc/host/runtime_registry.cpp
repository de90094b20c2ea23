#include "runtime_registry.h"

namespace esp {
namespace {
std::map<MultiModelConfig::Architecture, RuntimeLoader> &families() {
    static std::map<MultiModelConfig::Architecture, RuntimeLoader> table;
    return table;
}
DraftedGeneration &drafted() {
    static DraftedGeneration run = nullptr;
    return run;
}
}  // namespace

RuntimeFamilyRegistration::RuntimeFamilyRegistration(MultiModelConfig::Architecture architecture, RuntimeLoader loader) { families()[architecture] = loader; }
RuntimeLoader find_runtime_loader(MultiModelConfig::Architecture architecture) {
    auto it = families().find(architecture);
    return it == families().end() ? nullptr : it->second;
}
DraftedGenerationRegistration::DraftedGenerationRegistration(DraftedGeneration run) { drafted() = run; }
DraftedGeneration find_drafted_generation() { return drafted(); }

}  // namespace esp
