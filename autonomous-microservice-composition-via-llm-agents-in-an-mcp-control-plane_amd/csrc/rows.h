// Vector loads and stores of activation rows (bf16, or float in the 32-bit mode)
// as fp32, and rotation of halves.
#pragma once
#include "common.h"

namespace {

DEV void load8(const bf16* p, float (&v)[8]) {
  const bf16x8 x = *reinterpret_cast<const bf16x8*>(p);
#pragma unroll
  for (int j = 0; j < 8; ++j) v[j] = (float)x[j];
}
DEV void load8(const float* p, float (&v)[8]) {
#pragma unroll
  for (int h = 0; h < 2; ++h) {
    const f32x4 x = reinterpret_cast<const f32x4*>(p)[h];
#pragma unroll
    for (int j = 0; j < 4; ++j) v[4 * h + j] = x[j];
  }
}
DEV void store8(bf16* p, const float (&v)[8]) {
  bf16x8 x;
#pragma unroll
  for (int j = 0; j < 8; ++j) x[j] = (bf16)v[j];
  *reinterpret_cast<bf16x8*>(p) = x;
}
DEV void store8(float* p, const float (&v)[8]) {
#pragma unroll
  for (int h = 0; h < 2; ++h)
    reinterpret_cast<f32x4*>(p)[h] = f32x4{v[4 * h], v[4 * h + 1], v[4 * h + 2], v[4 * h + 3]};
}

// element / elements of a row whose first ``rot`` of 2 pairs + rest rotate as halves:
// d turns with d + pairs by cs[2 d], cs[2 d + 1] (cos, sin); zero from ``rot`` on
template <class T>
DEV float rotated(const T* __restrict__ p, const float* __restrict__ cs, int pairs, int rot, int d) {
  if (d < pairs) return (float)p[d] * cs[2 * d] - (float)p[d + pairs] * cs[2 * d + 1];
  if (d < 2 * pairs) {
    const int e = d - pairs;
    return (float)p[d] * cs[2 * e] + (float)p[e] * cs[2 * e + 1];
  }
  return d < rot ? (float)p[d] : 0.f;
}
// 8 elements from d on; halves that are multiples of 8 go by vectors
template <class T>
DEV void rotated8(const T* __restrict__ p, const float* __restrict__ cs, int pairs, int rot, int d,
                  float (&v)[8]) {
  if (pairs % 8 || d >= 2 * pairs) {
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = rotated(p, cs, pairs, rot, d + j);
    return;
  }
  const bool second = d >= pairs;
  const int e = second ? d - pairs : d;
  float a[8], b[8];
  load8(p + e, a);
  load8(p + e + pairs, b);
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    const float c = cs[2 * (e + j)], s = cs[2 * (e + j) + 1];
    v[j] = second ? b[j] * c + a[j] * s : a[j] * c - b[j] * s;
  }
}

}  // namespace
