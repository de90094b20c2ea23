// What the generation loops share: clocks, captured passes, device arrays, the budget of a batch.
#pragma once

#include <chrono>

#include "decoder_runtime.h"

namespace esp {
namespace loop {

using Clock = std::chrono::steady_clock;
inline double ms_since(Clock::time_point t0) { return std::chrono::duration<double, std::milli>(Clock::now() - t0).count(); }

// A pass of a generation loop as a captured graph: the first pass runs as plain launches (whatever a kernel configures on its first
// use happens outside the capture), later ones replay.
struct PassGraph {
    hipGraphExec_t exec = nullptr;
    ~PassGraph() { if (exec) (void)hipGraphExecDestroy(exec); }
    template <class Enqueue>
    int capture(Enqueue enqueue) {
        hipStream_t s = context().stream;
        hipGraph_t graph = nullptr;
        hipError_t e = hipStreamBeginCapture(s, hipStreamCaptureModeThreadLocal);
        if (e != hipSuccess) return fail_hip(e, "hipStreamBeginCapture");
        int rc = enqueue();
        e = hipStreamEndCapture(s, &graph);
        if (rc == ESP_OK && e != hipSuccess) rc = fail_hip(e, "hipStreamEndCapture");
        if (rc == ESP_OK && (e = hipGraphInstantiate(&exec, graph, nullptr, nullptr, 0)) != hipSuccess) rc = fail_hip(e, "hipGraphInstantiate");
        if (graph) (void)hipGraphDestroy(graph);
        return rc;
    }
    int launch(int times) {
        for (int i = 0; i < times; i++) {
            const hipError_t e = hipGraphLaunch(exec, context().stream);
            if (e != hipSuccess) return fail_hip(e, "hipGraphLaunch");
        }
        return ESP_OK;
    }
};
template <class T>
struct DeviceArray {
    T *p = nullptr;
    ~DeviceArray() { if (p) (void)hipFree(p); }
    int alloc(size_t count) { return device_alloc(&p, count); }
};
inline int hip_ok(hipError_t e, const char *what) { return e == hipSuccess ? ESP_OK : fail_hip(e, what); }

// Sequence s of `n_seq` uses KV cache s of both runtimes.  Greedy, no EOS handling (the batched configs
// decode a fixed budget); every sequence produces exactly `eff` tokens.
int batch_budget(const DecoderRuntime &a, const DecoderRuntime *b, const int *prompt_counts, int n_seq, int max_tokens, int *eff);

}  // namespace loop
}  // namespace esp
