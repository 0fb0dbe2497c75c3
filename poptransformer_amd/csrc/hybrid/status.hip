// Per-thread message of the last failing call of this library.
#include "hybrid.h"
#include <cstdarg>
#include <cstdio>

static thread_local char g_error[512] = "";

void pta_set_error(const char* fmt, ...) {
  va_list ap;
  va_start(ap, fmt);
  vsnprintf(g_error, sizeof(g_error), fmt, ap);
  va_end(ap);
}

extern "C" const char* pta_hybrid_last_error(void) { return g_error; }
