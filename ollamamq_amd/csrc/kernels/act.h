// Activations that several kernels share.
#pragma once
#include <hip/hip_runtime.h>

// 0.5 z (1 + tanh(sqrt(2/pi) (z + 0.044715 z^3))) is z times the sigmoid of
// this
static __device__ __forceinline__ float gelu_arg(float z) {
    return 1.5957691216057308f * (z + 0.044715f * z * z * z);
}
