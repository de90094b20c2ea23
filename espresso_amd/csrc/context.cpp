#include "context.h"

#include <cstdarg>
#include <cstdio>
#include <cstring>
#include <mutex>
#include <vector>

namespace esp {
namespace {
thread_local std::string t_last_error;
std::mutex g_init_mutex;
Context g_context;
std::vector<int (*)(int)> &setup_hooks() {
    static std::vector<int (*)(int)> hooks;
    return hooks;
}
}  // namespace

DeviceSetup::DeviceSetup(int (*setup)(int device)) { setup_hooks().push_back(setup); }

Context &context() { return g_context; }

void clear_error() { t_last_error.clear(); }

int fail(int code, const char *fmt, ...) {
    char buf[512];
    va_list ap;
    va_start(ap, fmt);
    vsnprintf(buf, sizeof(buf), fmt, ap);
    va_end(ap);
    t_last_error = buf;
    return code;
}

int fail_hip(hipError_t e, const char *what) {
    int code = e == hipErrorOutOfMemory ? ESP_ERR_OUT_OF_MEMORY
               : (e == hipErrorNoDevice || e == hipErrorInvalidDevice) ? ESP_ERR_NO_DEVICE
                                                                        : ESP_ERR_LAUNCH_FAILED;
    return fail(code, "%s: %s", what, hipGetErrorString(e));
}

const char *last_error_text() { return t_last_error.c_str(); }

int ensure_init() {
    std::lock_guard<std::mutex> lock(g_init_mutex);
    if (g_context.ready) return ESP_OK;
    int count = 0;
    hipError_t e = hipGetDeviceCount(&count);
    if (e != hipSuccess || count <= 0) {
        (void)hipGetLastError();
        return fail(ESP_ERR_NO_DEVICE, "no HIP device available (%s); this library has no CPU fallback",
                    e == hipSuccess ? "device count is 0" : hipGetErrorString(e));
    }
    ESP_HIP_TRY(hipSetDevice(0));
    ESP_HIP_TRY(hipGetDeviceProperties(&g_context.props, 0));
    ESP_HIP_TRY(hipStreamCreateWithFlags(&g_context.stream, hipStreamNonBlocking));
    g_context.device = 0;
    for (int (*setup)(int) : setup_hooks()) {
        const int rc = setup(0);
        if (rc != ESP_OK) return rc;
    }
    g_context.ready = true;
    return ESP_OK;
}

}  // namespace esp

extern "C" {

using namespace esp;

const char *esp_last_error(void) { return last_error_text(); }

int esp_init(void) { return ensure_init(); }

int esp_device_info(char *name, size_t name_capacity, int *compute_units, size_t *hbm_bytes) {
    int rc = ensure_init();
    if (rc != ESP_OK) return rc;
    const Context &c = context();
    if (name && name_capacity) {
        std::strncpy(name, c.props.gcnArchName, name_capacity - 1);
        name[name_capacity - 1] = 0;
    }
    if (compute_units) *compute_units = c.props.multiProcessorCount;
    if (hbm_bytes) *hbm_bytes = c.props.totalGlobalMem;
    return ESP_OK;
}

}  // extern "C"
