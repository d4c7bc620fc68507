// device_buf.h -- device memory of one call.
#pragma once
#include <hip/hip_runtime.h>

namespace ffmi {

struct DeviceBuf {
  void *p = nullptr;
  ~DeviceBuf() {
    if (p) (void)hipFree(p);
  }
  bool get(size_t bytes) { return hipMalloc(&p, bytes ? bytes : 16) == hipSuccess; }
};

}  // namespace ffmi
