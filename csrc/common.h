// Common helpers for the scaffold's CDNA4 (gfx950) HIP kernels.
// Target: MI355X only — wave64, 256 CUs / 8 XCDs, 160 KiB LDS/CU.
#pragma once

#include "device.h"

#include <torch/extension.h>
#include <c10/hip/HIPStream.h>

// torch's current stream for this device (ROCm-native name; avoids the
// hipify rewrite of at::cuda::getCurrentCUDAStream)
inline hipStream_t scaffold_stream() {
  return c10::hip::getCurrentHIPStream().stream();
}

#define HIP_CHECK(expr)                                                        \
  do {                                                                         \
    hipError_t _e = (expr);                                                    \
    TORCH_CHECK(_e == hipSuccess, "HIP error: ", hipGetErrorString(_e));       \
  } while (0)

#define CHECK_CUDA(x) TORCH_CHECK(x.is_cuda(), #x " must be a HIP tensor")
#define CHECK_CONTIG(x) TORCH_CHECK(x.is_contiguous(), #x " must be contiguous")

// Element strides of a logical (B,H,S,D) tensor with contiguous D —
// lets attention/RoPE consume permuted views (e.g. the (B,S,H,D)
// physical layout of a QKV projection) without transpose copies.
struct Strides4 {
  long sb, sh, ss;
};

inline Strides4 strides_of(const torch::Tensor& t) {
  TORCH_CHECK(t.dim() == 4 && t.stride(3) == 1,
              "expected 4-D tensor with contiguous last dim");
  return {t.stride(0), t.stride(1), t.stride(2)};
}
