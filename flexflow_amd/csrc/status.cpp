// status.cpp -- error state and version of the C ABI.
#include <stdio.h>
#include <stdlib.h>

#include <string>

#include "ffmi_internal.h"

static thread_local std::string g_last_error;

void ffmi_set_last_error(const char *msg, const char *file, int line) {
  char buf[512];
  snprintf(buf, sizeof(buf), "%s (%s:%d)", msg, file, line);
  g_last_error = buf;
  if (getenv("FFMI_VERBOSE_ERRORS")) fprintf(stderr, "[ffmi] error: %s\n", buf);
}

extern "C" const char *ffmi_last_error(void) { return g_last_error.c_str(); }

extern "C" const char *ffmi_status_str(ffmi_status s) {
  switch (s) {
    case FFMI_OK: return "ok";
    case FFMI_ERR_INVALID: return "invalid argument";
    case FFMI_ERR_HIP: return "hip error";
    case FFMI_ERR_NCCL: return "rccl error";
    case FFMI_ERR_OOM: return "out of device memory";
    case FFMI_ERR_UNSUPPORTED: return "unsupported";
    case FFMI_ERR_NO_DEVICE: return "no gfx950 device";
  }
  return "unknown";
}

// 0.2: ffmi_attn_cfg.full_precision and ffmi_model_opts.full_precision
// appended (struct sizes changed), the *_f32 entry points added
// 0.3: ffmi_rm_config.spec_extensions
// 0.4: ffmi_model_opts.kv_pool_tokens, models by config.json, replay steps
extern "C" const char *ffmi_version(void) { return "ffmi 0.4 (gfx950)"; }
