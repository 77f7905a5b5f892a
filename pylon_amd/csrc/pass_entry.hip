// What happens to the residual stream ahead of a pass through a stretch of layers: x <- W [x; x0] + step,
// with x0 the embedded tokens.  The product is the engine's own; these two kernels make its input and take
// its output:
//
//   pass_join:  rows [x | x0] in the activation type, x = resid + factor * sum_p delta[p] (the sublayer output
//               that was still to be added)
//   pass_begin: resid = sum_p product[p] + step (float)
#include "common.h"

template <typename TD, typename TO>
__global__ __launch_bounds__(256) void pass_join_kernel(TO* __restrict__ out, const float* __restrict__ resid,
                                                        const TD* __restrict__ delta, int n_delta,
                                                        long long delta_stride, float factor,
                                                        const float* __restrict__ embedded, int dim) {
  const size_t row = blockIdx.x;
  TO* yr = out + row * 2 * dim;
  const TD* dr = delta ? delta + row * dim : nullptr;
  const int i = blockIdx.y * 256 + threadIdx.x;
  if (i < dim) {
    float v = resid[row * dim + i];
    if (dr) {
      float d = to_float(dr[i]);
#pragma unroll 4
      for (int p = 1; p < n_delta; ++p) d += to_float(dr[i + p * delta_stride]);
      v = fmaf(factor, d, v);
    }
    yr[i] = from_float<TO>(v);
    yr[dim + i] = from_float<TO>(embedded[row * dim + i]);
  }
}

// out: [rows, 2 dim] of out_dtype; resid, embedded: float [rows, dim]; delta: null, [rows, dim], or n_delta
// such tensors delta_stride elements apart.
extern "C" int pylon_pass_join(void* out, int out_dtype, const float* resid, const void* delta, int delta_dtype,
                               int n_delta, long long delta_stride, float factor, const float* embedded, int rows,
                               int dim, hipStream_t stream) {
  PYLON_REQUIRE(pylon_valid_dtype(out_dtype) && pylon_valid_dtype(delta_dtype), "pass_join: unknown dtype");
  PYLON_REQUIRE(rows >= 0 && dim > 0 && n_delta >= 1, "pass_join: bad sizes");
  if (rows == 0) return 0;
#define GO(TD, TO)                                                                                                \
  hipLaunchKernelGGL((pass_join_kernel<TD, TO>), dim3(rows, (dim + 255) / 256), dim3(256), 0, stream, (TO*)out, resid, (const TD*)delta, \
                     n_delta, delta_stride, factor, embedded, dim)
  if (delta_dtype == PYLON_F32 && out_dtype == PYLON_F32) GO(float, float);
  else if (delta_dtype == PYLON_F32) GO(float, bf16_t);
  else if (out_dtype == PYLON_F32) GO(bf16_t, float);
  else GO(bf16_t, bf16_t);
#undef GO
  PYLON_LAUNCHED("pass_join");
}

__global__ __launch_bounds__(256) void pass_begin_kernel(float* __restrict__ resid, const float* __restrict__ product,
                                                         int n_parts, long long part_stride,
                                                         const float* __restrict__ step, int dim) {
  const size_t row = blockIdx.x;
  const int i = blockIdx.y * 256 + threadIdx.x;
  if (i < dim) {
    float v = product[row * dim + i];
#pragma unroll 4
    for (int p = 1; p < n_parts; ++p) v += product[row * dim + i + p * part_stride];
    resid[row * dim + i] = step ? v + step[i] : v;
  }
}

// resid: float [rows, dim], overwritten; product: float [rows, dim], or n_parts of them part_stride elements
// apart (added in order); step: null or dim floats.
extern "C" int pylon_pass_begin(float* resid, const float* product, int n_parts, long long part_stride,
                                const float* step, int rows, int dim, hipStream_t stream) {
  PYLON_REQUIRE(rows >= 0 && dim > 0 && n_parts >= 1, "pass_begin: bad sizes");
  if (rows == 0) return 0;
  hipLaunchKernelGGL(pass_begin_kernel, dim3(rows, (dim + 255) / 256), dim3(256), 0, stream, resid, product, n_parts,
                     part_stride, step, dim);
  PYLON_LAUNCHED("pass_begin");
}
