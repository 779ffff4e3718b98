// base.hip -- what every entry point of the C ABI leans on: the thread-local error string, the knob table, version and device queries.
#include <cstring>

#include "common.hpp"

namespace {
thread_local std::string g_last_error;
int g_knobs[PIE_KNOB_COUNT] = {-1, -1, -1, -1, -1, -1, -1, -1, -1, -1, -1};
}
int pie_knob(int knob) { return knob >= 0 && knob < PIE_KNOB_COUNT ? g_knobs[knob] : PIE_KNOB_DEFAULT; }
namespace pie {
void set_error(const std::string &msg) { g_last_error = msg; }
int fail(int code, const std::string &msg) {
    g_last_error = msg;
    return code;
}
}  // namespace pie

extern "C" {

const char *pie_hello(void) { return "pie_core \xe2\x9c\x93"; }
#ifndef PIE_BUILD_HASH
#define PIE_BUILD_HASH "unhashed"
#endif
const char *pie_version(void) { return "pie_hip 0.3.0 (gfx950) " PIE_BUILD_HASH; }  // the hash of the sources: proxy_inference_engine_amd/build.py
const char *pie_last_error(void) { return g_last_error.c_str(); }

int pie_set_knob(int knob, int value) {
    PIE_REQUIRE(knob >= 0 && knob < PIE_KNOB_COUNT, PIE_E_ARG, "pie_set_knob: unknown knob");
    g_knobs[knob] = value < 0 ? PIE_KNOB_DEFAULT : value;
    return PIE_OK;
}
int pie_get_knob(int knob) { return pie_knob(knob); }

int pie_device_info(char *name, int name_len, int *n_cus, size_t *hbm_bytes) {
    int dev = 0;
    PIE_HIP_TRY(hipGetDevice(&dev));
    hipDeviceProp_t p;
    PIE_HIP_TRY(hipGetDeviceProperties(&p, dev));
    if (name && name_len > 0) {
        strncpy(name, p.gcnArchName, (size_t)name_len - 1);
        name[name_len - 1] = 0;
    }
    if (n_cus) *n_cus = p.multiProcessorCount;
    if (hbm_bytes) *hbm_bytes = p.totalGlobalMem;
    return PIE_OK;
}

}  // extern "C"
