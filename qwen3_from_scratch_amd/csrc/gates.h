// What the gate of a gated unit passes: ACT 0: silu(g) = g / (1 + exp(-g)); 1: the tanh form of gelu,
// 0.5 g (1 + tanh(sqrt(2/pi) (g + 0.044715 g^3))); 2: the exact gelu, 0.5 g (1 + erf(g / sqrt 2)).
// float32. Shared by the activation kernels and the products that carry an activation in their epilogues,
// so that both give the same bits.
#pragma once

#include <hip/hip_runtime.h>

template <int ACT>
__device__ inline float gate_value(float g) {
  if (ACT == 0) return g / (1.f + expf(-g));
  if (ACT == 1) return 0.5f * g * (1.f + tanhf(0.79788456080286536f * (g + 0.044715f * g * g * g)));
  return 0.5f * g * (1.f + erff(g * 0.70710678118654752f));
}
