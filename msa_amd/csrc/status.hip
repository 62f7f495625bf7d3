// Error plumbing shared by the libraries (host code only).
#include <stdarg.h>

#include "common.h"

static thread_local char g_err[512] = "";

void msa_set_error(const char* fmt, ...) {
  va_list ap;
  va_start(ap, fmt);
  vsnprintf(g_err, sizeof(g_err), fmt, ap);
  va_end(ap);
}

extern "C" const char* msa_last_error(void) { return g_err; }
extern "C" int msa_abi_version(void) { return 1; }
