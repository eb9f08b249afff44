// lv_common.h — what every translation unit of libllava_hip.so shares on the host side: error text and status macros.
#pragma once

#include <hip/hip_runtime.h>
#include <stdint.h>

#include "../../include/llava_hip.h"

namespace lv {

// records the calling thread's error text (lv_last_error) and returns `code`
int fail(int code, const char *fmt, ...) __attribute__((format(printf, 2, 3)));

// zero fill by a kernel on the stream (usable inside graph capture, unlike a memset node); bytes a multiple of 4
int zero_async(void *p, uint64_t bytes, hipStream_t st);

}  // namespace lv

#define HIP_TRY(expr)                                                                                         \
    do {                                                                                                      \
        hipError_t e_ = (expr);                                                                               \
        if (e_ != hipSuccess) return lv::fail(LV_ERR_HIP, "%s failed: %s (%s:%d)", #expr, hipGetErrorString(e_), \
                                              __FILE__, __LINE__);                                            \
    } while (0)

#define LV_TRY(expr)              \
    do {                          \
        int rc_ = (expr);         \
        if (rc_ != LV_OK) return rc_; \
    } while (0)
