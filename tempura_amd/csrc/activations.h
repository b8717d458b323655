// Activations of ungated feed-forwards, on float32 sums.
#pragma once
#include <math.h>
#include "common.h"

// kind 0: the tanh form of GELU, 0.5 z (1 + tanh(sqrt(2 / pi) (z + 0.044715 z^3))); kind 1: SiLU; kind 2: the exact
// GELU, 0.5 z (1 + erf(z / sqrt(2))); kind 3: the square of ReLU, max(z, 0)^2.
__device__ inline float act_f(float z, int kind) {
  if (kind == 0) return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
  if (kind == 2) return 0.5f * z * (1.0f + erff(z * 0.7071067811865476f));
  if (kind == 3) return relu_squared(z);
  return z * (1.0f / (1.0f + expf(-z)));
}
