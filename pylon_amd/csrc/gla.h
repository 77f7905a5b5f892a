// The decay of gated linear attention, shared by its recurrent and its chunked form.
#pragma once
#include "common.h"

// log(sigmoid(z)) as min(z, 0) - log1p(e^-|z|), which neither overflows nor loses a decay close to one.  With
// x = e^-|z| and u = 1 + x rounded, log1p(x) = log(u) * x / (u - 1): the quotient takes back what the rounding
// of u moved (u - 1 is exact), and where u is one, log1p(x) is x.
__device__ __forceinline__ float gla_log_sigmoid(float z) {
  const float x = __expf(-fabsf(z));
  const float u = 1.0f + x, du = u - 1.0f;
  const float l = du == 0.f ? x : __logf(u) * (x / du);
  return fminf(z, 0.f) - l;
}

// log(sigmoid(z)^(1/tau)) of one key channel: z = a2_row . low + bias.
template <typename T>
__device__ __forceinline__ float gla_log_decay(const T* __restrict__ low, const float* __restrict__ a2_row, int rank,
                                               float bias, float inv_tau) {
  float z = 0.f;
  for (int r = 0; r < rank; ++r) z = fmaf(to_float(low[r]), a2_row[r], z);
  return gla_log_sigmoid(z + bias) * inv_tau;
}
