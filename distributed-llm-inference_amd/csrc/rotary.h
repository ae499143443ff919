// The angle of a rotary pair in 32-bit.
#pragma once
#include "common.h"

// cos and sin of position * freq with the product's rounding error taken back: the product's low
// half (one fused multiply-add) turns the functions by their own derivatives.
__device__ __forceinline__ void rotary_cos_sin(float position, float freq, float* c, float* s) {
  const float hi = position * freq;
  const float lo = fmaf(position, freq, -hi);
  float sh, ch;
  sincosf(hi, &sh, &ch);
  *c = fmaf(-lo, sh, ch);
  *s = fmaf(lo, ch, sh);
}
