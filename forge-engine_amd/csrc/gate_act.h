// The activation of a gated product, act(gate) * up: z * sigmoid(z * (linear + cubic * z^2)).
//   silu: (1, 0); the tanh form of gelu, 0.5 z (1 + tanh(sqrt(2/pi) (z + 0.044715 z^3))): since
//   0.5 (1 + tanh(y)) = sigmoid(2 y), linear = 2 sqrt(2/pi) and cubic = 0.044715 times that.
// With cubic = 0 the arithmetic is that of z / (1 + exp(-z)), bit for bit.
#pragma once
#include "common.h"

struct GateAct {
  float linear, cubic;
};

#define FE_GATE_SILU 0
#define FE_GATE_GELU_TANH 1

static inline bool gate_act(int code, GateAct* act) {
  if (code == FE_GATE_SILU) *act = GateAct{1.f, 0.f};
  else if (code == FE_GATE_GELU_TANH) *act = GateAct{1.5957691216057308f, 0.0713548162726009f};
  else return false;
  return true;
}

__device__ __forceinline__ float gate_exponent(float g, GateAct act) { return -g * __fmaf_rn(act.cubic * g, g, act.linear); }
// with the fast exponential, where the result is rounded to bfloat16
__device__ __forceinline__ float gate_times(float g, float u, GateAct act) { return g / (1.f + __expf(gate_exponent(g, act))) * u; }
__device__ __forceinline__ float gate_times_exact(float g, float u, GateAct act) { return g / (1.f + expf(gate_exponent(g, act))) * u; }
