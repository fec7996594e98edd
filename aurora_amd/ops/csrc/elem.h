// Element access for kernels that run in bf16 or in float32 throughout.
#pragma once
#include <hip/hip_runtime.h>

#include "common.h"

typedef unsigned short bf16_t;  // raw bf16 bits

template <typename T> struct Elem;
template <> struct Elem<bf16_t> {
  static DEVINL float load(const bf16_t* p) { return bf16_to_f32(*p); }
  static DEVINL void store(bf16_t* p, float v) { *p = f32_to_bf16(v); }
};
template <> struct Elem<float> {
  static DEVINL float load(const float* p) { return *p; }
  static DEVINL void store(float* p, float v) { *p = v; }
};

template <typename T>
DEVINL float ldf(const T* p) { return Elem<T>::load(p); }
template <typename T>
DEVINL void stf(T* p, float v) { Elem<T>::store(p, v); }

// 4 consecutive elements (the pointer is 4-element aligned)
DEVINL floatx4 ld4(const float* p) { return *reinterpret_cast<const floatx4*>(p); }
DEVINL floatx4 ld4(const bf16_t* p) {
  const shortx4 v = *reinterpret_cast<const shortx4*>(p);
  floatx4 r;
#pragma unroll
  for (int i = 0; i < 4; ++i) r[i] = bf16_to_f32((unsigned short)v[i]);
  return r;
}
DEVINL void st4(float* p, floatx4 v) { *reinterpret_cast<floatx4*>(p) = v; }
DEVINL void st4(bf16_t* p, floatx4 v) {
  shortx4 r;
#pragma unroll
  for (int i = 0; i < 4; ++i) r[i] = (short)f32_to_bf16(v[i]);
  *reinterpret_cast<shortx4*>(p) = r;
}

DEVINL float sigmoid_f(float x) { return 1.f / (1.f + expf(-x)); }
DEVINL float silu_f(float x) { return x / (1.f + expf(-x)); }
// max(x, 0) + log(1 + y), y = e^-|x|; a short series where 1 + y would round y
DEVINL float softplus_f(float x) {
  const float y = expf(-fabsf(x));
  const float s = y < 0.015625f ? y * (1.f - y * (0.5f - y * (1.f / 3.f - 0.25f * y)))
                                : logf(1.f + y);
  return fmaxf(x, 0.f) + s;
}

// sum over a workgroup of NW waves; every thread gets it (red: NW floats of LDS)
template <int NW>
DEVINL float block_sum(float x, float* red) {
  x = wave_sum(x);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = x;
  __syncthreads();
  float y = red[0];
#pragma unroll
  for (int i = 1; i < NW; ++i) y += red[i];
  return y;
}
DEVINL float block_sum4(float x, float* red) { return block_sum<4>(x, red); }

#define DISPATCH_ELEM(IS_BF16, ...)                     \
  do {                                                  \
    if (IS_BF16) { using T = bf16_t; __VA_ARGS__; }     \
    else { using T = float; __VA_ARGS__; }              \
  } while (0)
