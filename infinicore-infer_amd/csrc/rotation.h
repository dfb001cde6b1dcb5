// Angles of rotary positions.
#pragma once
#include "common.h"

// cos and sin of position * f, f given as the float32 rounding of its float64 value and what the rounding left: the
// float32 product plus a small rest (the product's own rounding error from an fma, and position * the second
// part), to second order in the rest.
__device__ __forceinline__ void pair_angle(float p, float f_hi, float f_lo, float& cs, float& sn) {
    const float ang = p * f_hi;
    const float rest = fmaf(p, f_hi, -ang) + p * f_lo;
    const float s0 = sinf(ang), c0 = cosf(ang), half = 0.5f * rest * rest;
    sn = (s0 - half * s0) + rest * c0;
    cs = (c0 - half * c0) - rest * s0;
}
