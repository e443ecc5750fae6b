// Error plumbing and ABI version, shared by every library of the package.
#include <stdarg.h>
#include <stdio.h>

#include "common.cuh"

static thread_local char g_err[512] = "";
void omni_set_error(const char* fmt, ...) {
    va_list ap;
    va_start(ap, fmt);
    vsnprintf(g_err, sizeof(g_err), fmt, ap);
    va_end(ap);
}
extern "C" const char* omni_last_error(void) { return g_err; }
extern "C" int omni_abi_version(void) { return 7; }
