// The decay of gated linear attention, shared by its recurrent and its chunked form.
#pragma once
#include "common.h"

// log(sigmoid(z)) as min(z, 0) - log1p(e^-|z|), which neither overflows nor loses a decay close to one.
__device__ __forceinline__ float gla_log_sigmoid(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }

// log(sigmoid(z)^(1/tau)) of one key channel: z = a2_row . low + bias.
template <typename T>
__device__ __forceinline__ float gla_log_decay(const T* __restrict__ low, const float* __restrict__ a2_row, int rank,
                                               float bias, float inv_tau) {
  float z = 0.f;
  for (int r = 0; r < rank; ++r) z = fmaf(to_float(low[r]), a2_row[r], z);
  return gla_log_sigmoid(z + bias) * inv_tau;
}
