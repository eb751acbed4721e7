// docqa_bind.h -- argument checks and error reporting shared by the operator bindings
// (bindings.cpp, bindings_hybrid.cpp).
#pragma once
#include <torch/library.h>
#include <ATen/ATen.h>
#include <c10/hip/HIPStream.h>
#include <c10/core/DeviceGuard.h>
#include <stdlib.h>

namespace {

hipStream_t stream() { return c10::hip::getCurrentHIPStream().stream(); }

#define CHECK_GPU(t) TORCH_CHECK((t).is_cuda(), #t " must be a GPU tensor")
#define CHECK_BF16(t) TORCH_CHECK((t).scalar_type() == at::kBFloat16, #t " must be bfloat16")
#define CHECK_I32(t) TORCH_CHECK((t).scalar_type() == at::kInt, #t " must be int32")
#define CHECK_CONTIG(t) TORCH_CHECK((t).is_contiguous(), #t " must be contiguous")
#define CHECK_ALIGN16(t) \
  TORCH_CHECK((reinterpret_cast<uintptr_t>((t).data_ptr()) & 15u) == 0, \
              #t " must be 16-byte aligned (storage offset a multiple of 16 bytes)")
// DOCQA_KERNEL_DEBUG=1: synchronous kernel checking (the HIP_LAUNCH_BLOCKING of this
// extension): after every op that is not being graph-captured, the stream
// is synchronised and any asynchronous fault is reported with the op's name -- a
// faulting kernel is named by the op that launched it, not by a later unrelated sync.
static bool kernel_debug() {
  static const bool on = [] {
    const char* e = getenv("DOCQA_KERNEL_DEBUG");
    return e && atoi(e) != 0;
  }();
  return on;
}

static void debug_sync(const char* name) {
  hipStream_t s = stream();
  hipStreamCaptureStatus cs = hipStreamCaptureStatusNone;
  if (hipStreamIsCapturing(s, &cs) != hipSuccess || cs != hipStreamCaptureStatusNone) return;
  const hipError_t e = hipStreamSynchronize(s);
  TORCH_CHECK(e == hipSuccess, "docqa kernel ", name, " faulted (DOCQA_KERNEL_DEBUG): ", hipGetErrorString(e));
}

#define CHECK_RC(rc, name)                                                                 \
  do {                                                                                     \
    const int rc__ = (rc);                                                                 \
    TORCH_CHECK(rc__ == 0, "docqa kernel " name " failed with code ", rc__);               \
    if (kernel_debug()) debug_sync(name);                                                  \
  } while (0)

}  // namespace
