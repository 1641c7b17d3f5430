// Version and error text of the kernel library.
#include "common.h"

namespace nf {

static thread_local char g_err[512] = "";

void set_error(const char* fmt, ...) {
  va_list ap;
  va_start(ap, fmt);
  vsnprintf(g_err, sizeof(g_err), fmt, ap);
  va_end(ap);
}

}  // namespace nf

extern "C" {

int nf_abi_version(void) { return 1; }
const char* nf_last_error(void) { return nf::g_err; }

}  // extern "C"
