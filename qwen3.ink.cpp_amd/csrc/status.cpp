// Status codes and the calling thread's last error message, shared by every library of this directory.
#include "../../include/a81w41.h"

#include <cstdio>

#include "decoder_session.h"

namespace {
thread_local char g_err[512] = "";
}

namespace a81w41 {
int report_failure(int status, const char* message) {
    snprintf(g_err, sizeof(g_err), "%s", message);
    return status;
}
int failf(int status, const char* fmt, ...) {
    va_list ap;
    va_start(ap, fmt);
    vsnprintf(g_err, sizeof(g_err), fmt, ap);
    va_end(ap);
    return status;
}
}  // namespace a81w41

extern "C" {

const char* a81w41_status_string(int status) {
    switch (status) {
        case A81W41_OK: return "ok";
        case A81W41_ERR_INVALID_ARG: return "invalid argument";
        case A81W41_ERR_HIP: return "HIP runtime error";
        case A81W41_ERR_IO: return "weight file error";
        case A81W41_ERR_NO_DEVICE: return "no gfx950 device";
        case A81W41_ERR_UNSUPPORTED: return "not supported by this model";
        default: return "unknown status";
    }
}

const char* a81w41_last_error(void) { return g_err; }

}  // extern "C"
