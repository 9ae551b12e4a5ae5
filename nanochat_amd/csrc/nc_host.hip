// What every library of the package needs on the host: the error channel of the C ABI (the message of the last failure on the calling
// thread) and the number of compute units of the current device.
#include <atomic>
#include <stdarg.h>
#include <stdio.h>
#include "nc_common.h"
#include "nc_kernels.h"

static thread_local char g_error[512] = "";

void nc_set_error(const char* fmt, ...) {
    va_list ap;
    va_start(ap, fmt);
    vsnprintf(g_error, sizeof(g_error), fmt, ap);
    va_end(ap);
}

extern "C" const char* nc_last_error(void) { return g_error; }

int nc_cu_count() {
    constexpr int MAX_DEVICES = 64;
    static std::atomic<int> cached[MAX_DEVICES];
    int dev = 0;
    if (hipGetDevice(&dev) != hipSuccess || dev < 0 || dev >= MAX_DEVICES) dev = 0;
    int cus = cached[dev].load(std::memory_order_relaxed);
    if (cus == 0) {
        cus = 256;
        (void)hipDeviceGetAttribute(&cus, hipDeviceAttributeMultiprocessorCount, dev);
        cached[dev].store(cus, std::memory_order_relaxed);
    }
    return cus;
}
