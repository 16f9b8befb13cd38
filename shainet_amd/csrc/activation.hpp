// Activations that ride in a product's epilogue, with their constants as parameters.
#pragma once
#include <hip/hip_runtime.h>

namespace shainet {

enum { kActNone = 0, kActXielu = 1 };
// kActXielu: pos z^2 + z / 2 for z > 0, neg (exp(z) - 1 - z) + z / 2 otherwise
struct Activation {
  int kind = kActNone;
  float pos = 0.f, neg = 0.f;
};

__device__ __forceinline__ float activate(const Activation &a, float z) {
  if (a.kind == kActXielu) return (z > 0.f ? a.pos * z * z : a.neg * (expm1f(z) - z)) + 0.5f * z;
  return z;
}

}  // namespace shainet
