// A norm over all heads of a mixer at once, with a gate per element:
//
//   out[t, i] = x[t, i] / sqrt(mean_j(x[t, j]^2) + eps) * w[i] * gate(g[t, i])
//
// gate: sigmoid, or silu.  x is float (a recurrence's outputs), g lies inside the rows of a fused
// projection; everything is computed in float and rounded once on the store.  One workgroup a row, the
// row held in registers between the sum of squares and the product; all of a row's loads are sent for
// before the sum.  The order of the sum depends on the row's length only.
#include "common.h"

__device__ __forceinline__ float4 ng_load4(const float* p, int c) { return reinterpret_cast<const float4*>(p)[c]; }
__device__ __forceinline__ float4 ng_load4(const bf16_t* p, int c) {
  const uint2 raw = reinterpret_cast<const uint2*>(p)[c];
  return float4{__uint_as_float(raw.x << 16), __uint_as_float(raw.x & 0xffff0000u), __uint_as_float(raw.y << 16),
                __uint_as_float(raw.y & 0xffff0000u)};
}
__device__ __forceinline__ void ng_store4(float* p, int c, float4 y) { reinterpret_cast<float4*>(p)[c] = y; }
__device__ __forceinline__ void ng_store4(bf16_t* p, int c, float4 y) {
  uint2 raw;
  raw.x = static_cast<uint32_t>(float_to_bf16_bits(y.x)) | (static_cast<uint32_t>(float_to_bf16_bits(y.y)) << 16);
  raw.y = static_cast<uint32_t>(float_to_bf16_bits(y.z)) | (static_cast<uint32_t>(float_to_bf16_bits(y.w)) << 16);
  reinterpret_cast<uint2*>(p)[c] = raw;
}
__device__ __forceinline__ float ng_gate(float g, int silu) {
  const float s = 1.0f / (1.0f + expf(-g));
  return silu ? g * s : s;
}

// VEC: groups of four elements a thread holds (0: rows that are read twice, element by element).
template <typename T, int VEC>
__global__ __launch_bounds__(1024) void norm_gate_kernel(T* __restrict__ out, const float* __restrict__ x,
                                                         const float* __restrict__ w, const T* __restrict__ g,
                                                         long long ldg, int dim, float eps, int silu) {
  __shared__ float scratch[16];
  const size_t row = blockIdx.x;
  const float* xr = x + row * dim;
  const T* gr = g + row * ldg;
  T* yr = out + row * dim;
  if constexpr (VEC == 0) {
    float ss = 0.f;
    for (int i = threadIdx.x; i < dim; i += blockDim.x) ss += xr[i] * xr[i];
    const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / static_cast<float>(dim) + eps);
    for (int i = threadIdx.x; i < dim; i += blockDim.x)
      yr[i] = from_float<T>((xr[i] * inv) * w[i] * ng_gate(to_float(gr[i]), silu));
  } else {
    const int chunks = dim >> 2;
    float4 held[VEC], gate[VEC], wt[VEC];
#pragma unroll
    for (int n = 0; n < VEC; ++n) {
      const int c = threadIdx.x + n * blockDim.x;
      held[n] = gate[n] = wt[n] = float4{0.f, 0.f, 0.f, 0.f};
      if (c < chunks) {
        held[n] = ng_load4(xr, c);
        gate[n] = ng_load4(gr, c);
        wt[n] = ng_load4(w, c);
      }
    }
    float ss = 0.f;
#pragma unroll
    for (int n = 0; n < VEC; ++n)
      ss += held[n].x * held[n].x + held[n].y * held[n].y + held[n].z * held[n].z + held[n].w * held[n].w;
    const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / static_cast<float>(dim) + eps);
#pragma unroll
    for (int n = 0; n < VEC; ++n) {
      const int c = threadIdx.x + n * blockDim.x;
      if (c < chunks)
        ng_store4(yr, c, float4{(held[n].x * inv) * wt[n].x * ng_gate(gate[n].x, silu),
                                (held[n].y * inv) * wt[n].y * ng_gate(gate[n].y, silu),
                                (held[n].z * inv) * wt[n].z * ng_gate(gate[n].z, silu),
                                (held[n].w * inv) * wt[n].w * ng_gate(gate[n].w, silu)});
    }
  }
}

// out: [rows, dim] of dtype; x: float [rows, dim]; w: dim floats; g: rows of dtype, ldg elements apart, whose
// first dim elements are the gate's logits.  act 0: sigmoid, 1: silu.
extern "C" int pylon_norm_gate(void* out, int dtype, const float* x, const float* w, const void* g, long long ldg,
                               int rows, int dim, float eps, int act, hipStream_t stream) {
  PYLON_REQUIRE(pylon_valid_dtype(dtype), "norm_gate: unknown dtype");
  PYLON_REQUIRE(rows >= 0 && dim > 0 && (rows <= 1 || ldg >= dim), "norm_gate: bad sizes");
  PYLON_REQUIRE(act == 0 || act == 1, "norm_gate: unknown gate %d", act);
  if (rows == 0) return 0;
  const uintptr_t ends = reinterpret_cast<uintptr_t>(out) | reinterpret_cast<uintptr_t>(x) | reinterpret_cast<uintptr_t>(w) |
                         reinterpret_cast<uintptr_t>(g);
  const bool wide = dim % 4 == 0 && ldg % 4 == 0 && (ends & (dtype == PYLON_F32 ? 15 : 7)) == 0 &&
                    ((reinterpret_cast<uintptr_t>(x) | reinterpret_cast<uintptr_t>(w)) & 15) == 0 && dim <= 16384;
  const int threads = dim <= 4096 ? 256 : (dim <= 8192 ? 512 : 1024);
  const int per = (dim / 4 + threads - 1) / threads;
#define GO(T, VEC)                                                                                              \
  hipLaunchKernelGGL((norm_gate_kernel<T, VEC>), dim3(rows), dim3(threads), 0, stream, (T*)out, x, w, (const T*)g, \
                     ldg, dim, eps, act)
#define PICK(T)               \
  do {                        \
    if (!wide) GO(T, 0);      \
    else if (per <= 1) GO(T, 1); \
    else if (per <= 2) GO(T, 2); \
    else GO(T, 4);            \
  } while (0)
  if (dtype == PYLON_F32) PICK(float);
  else PICK(bf16_t);
#undef PICK
#undef GO
  PYLON_LAUNCHED("norm_gate");
}
