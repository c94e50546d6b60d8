// Rows of a norm: access in vectors of VEC elements, sums over the TPR threads
// that share a row, and statistics.  Row values stay in registers between the
// mean and the variance pass.
#pragma once

#include "lm.h"
#include "tile.h"

template <int VEC> struct Pack { float v[VEC]; };

template <bool F32, int VEC>
DEVINL Pack<VEC> ldv(const void* base, long i) {
  Pack<VEC> p;
  if constexpr (F32) {
    const float* s = (const float*)base + i;
    if constexpr (VEC == 4) *(f32x4*)p.v = *(const f32x4*)s;
    else p.v[0] = s[0];
  } else {
    const short* s = (const short*)base + i;
    if constexpr (VEC == 4) {
      const bf16x4 t = *(const bf16x4*)s;
      #pragma unroll
      for (int j = 0; j < 4; ++j) p.v[j] = bf2f(t[j]);
    } else {
      p.v[0] = bf2f(s[0]);
    }
  }
  return p;
}

// VEC elements as stored (half the registers of their float form in bf16)
template <bool F32, int VEC> struct Held {
  typename Num<F32>::E e[VEC];
  DEVINL void load(const void* base, long i) {
    const auto* s = (const typename Num<F32>::E*)base + i;
    if constexpr (VEC == 4 && F32) *(f32x4*)e = *(const f32x4*)s;
    else if constexpr (VEC == 4) *(bf16x4*)e = *(const bf16x4*)s;
    else e[0] = s[0];
  }
  // a norm's weights: base[i..], or base[0] everywhere
  DEVINL void load_weight(const void* base, long i, bool one) {
    if (!one) return load(base, i);
    #pragma unroll
    for (int j = 0; j < VEC; ++j) e[j] = *(const typename Num<F32>::E*)base;
  }
  DEVINL Pack<VEC> up() const {
    Pack<VEC> p;
    #pragma unroll
    for (int j = 0; j < VEC; ++j) p.v[j] = Num<F32>::up(e[j]);
    return p;
  }
};

template <bool F32, int VEC>
DEVINL void stv(void* base, long i, const Pack<VEC>& p) {
  if constexpr (F32) {
    float* s = (float*)base + i;
    if constexpr (VEC == 4) *(f32x4*)s = *(const f32x4*)p.v;
    else s[0] = p.v[0];
  } else {
    short* s = (short*)base + i;
    if constexpr (VEC == 4) {
      bf16x4 t;
      #pragma unroll
      for (int j = 0; j < 4; ++j) t[j] = cvt_bf16(p.v[j]);
      *(bf16x4*)s = t;
    } else {
      s[0] = cvt_bf16(p.v[0]);
    }
  }
}

template <int TPR>
DEVINL float row_sum(float v, float* red) {
  v = group_sum<64>(v);
  if constexpr (TPR == 256) {
    const int w = threadIdx.x >> 6;
    __syncthreads();             // the previous use of red is over
    if ((threadIdx.x & 63) == 0) red[w] = v;
    __syncthreads();
    v = red[0] + red[1] + red[2] + red[3];
  }
  return v;
}

// rms: without taking the mean off
template <int TPR, int VEC, int NV>
DEVINL void layer_norm_rows(Pack<VEC> (&v)[NV], int tid, int W, float eps,
                            bool rms, float* red) {
  float mean = 0.f;
  if (!rms) {
    float s = 0.f;
    #pragma unroll
    for (int i = 0; i < NV; ++i)
      #pragma unroll
      for (int j = 0; j < VEC; ++j) s += v[i].v[j];  // lanes past W hold 0
    mean = row_sum<TPR>(s, red) / (float)W;
  }
  float q = 0.f;
  #pragma unroll
  for (int i = 0; i < NV; ++i) {
    const bool ok = (i * TPR + tid) * VEC < W;
    #pragma unroll
    for (int j = 0; j < VEC; ++j) {
      const float d = v[i].v[j] - mean;
      v[i].v[j] = d;
      q += ok ? d * d : 0.f;
    }
  }
  const float inv = 1.0f / sqrtf(row_sum<TPR>(q, red) / (float)W + eps);
  #pragma unroll
  for (int i = 0; i < NV; ++i)
    #pragma unroll
    for (int j = 0; j < VEC; ++j) v[i].v[j] *= inv;
}
