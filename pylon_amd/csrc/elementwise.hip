// Row-wise kernels of the decoder: embedding gather, RMSNorm (alone, or fused with the
// residual sum that precedes it), and the gated activation of the feed-forward.
// All reductions and all arithmetic are in float; only loads and stores see bf16.
#include "common.h"

// ---- embedding ------------------------------------------------------------------
// out[t, :] = table[ids[t], :] * scale, written as float (the residual stream).
// A negative id -(1 + s) stands for "the token that the sampler left in chosen[s]": a
// request's last sampled token can be fed back without a trip through the host.
template <typename T>
__global__ void embed_kernel(float* __restrict__ out, const T* __restrict__ table,
                             const int* __restrict__ ids, const int* __restrict__ chosen, int hidden,
                             int vocab, float scale, int copies) {
  const int t = blockIdx.x;
  int id = ids[t];
  if (id < 0 && chosen != nullptr) id = chosen[-1 - id];
  // The host checks ids; the clamp only keeps a bad id from reading outside the table.
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
  const T* row = table + static_cast<size_t>(id) * hidden;
  float* dst = out + static_cast<size_t>(t) * hidden;
  const size_t apart = static_cast<size_t>(gridDim.x) * hidden;  // from one copy to the next
  for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
    const float v = to_float(row[i]) * scale;
    for (int c = 0; c < copies; ++c) dst[c * apart + i] = v;
  }
}

// chosen may be null; then every id must be a table row.  The host guarantees that a
// negative id -(1 + s) names an entry s inside chosen.  out: [copies, tokens, hidden], all copies equal.
extern "C" int pylon_embed(float* out, const void* table, int table_dtype, const int* ids,
                           const int* chosen, int tokens, int hidden, int vocab, float scale, int copies,
                           hipStream_t stream) {
  PYLON_REQUIRE(pylon_valid_dtype(table_dtype), "embed: unknown table dtype %d", table_dtype);
  PYLON_REQUIRE(tokens >= 0 && hidden > 0 && vocab > 0, "embed: bad sizes tokens=%d hidden=%d vocab=%d",
                tokens, hidden, vocab);
  PYLON_REQUIRE(copies >= 1, "embed: at least one copy");
  if (tokens == 0) return 0;
  dim3 grid(tokens), block(256);
  if (table_dtype == PYLON_F32)
    hipLaunchKernelGGL(embed_kernel<float>, grid, block, 0, stream, out, (const float*)table, ids,
                       chosen, hidden, vocab, scale, copies);
  else
    hipLaunchKernelGGL(embed_kernel<bf16_t>, grid, block, 0, stream, out, (const bf16_t*)table, ids,
                       chosen, hidden, vocab, scale, copies);
  PYLON_LAUNCHED("embed");
}

// Four consecutive elements number 4c .. 4c+3 of a row, as floats.
__device__ __forceinline__ float4 load4(const float* p, long long c) {
  return reinterpret_cast<const float4*>(p)[c];
}
__device__ __forceinline__ float4 load4(const bf16_t* p, long long c) {
  const uint2 raw = reinterpret_cast<const uint2*>(p)[c];
  return float4{__uint_as_float(raw.x << 16), __uint_as_float(raw.x & 0xffff0000u),
                __uint_as_float(raw.y << 16), __uint_as_float(raw.y & 0xffff0000u)};
}
__device__ __forceinline__ void store4(float* p, long long c, float a, float b, float d, float e) {
  reinterpret_cast<float4*>(p)[c] = float4{a, b, d, e};
}
__device__ __forceinline__ void store4(bf16_t* p, long long c, float a, float b, float d, float e) {
  uint2 raw;
  raw.x = static_cast<uint32_t>(float_to_bf16_bits(a)) | (static_cast<uint32_t>(float_to_bf16_bits(b)) << 16);
  raw.y = static_cast<uint32_t>(float_to_bf16_bits(d)) | (static_cast<uint32_t>(float_to_bf16_bits(e)) << 16);
  reinterpret_cast<uint2*>(p)[c] = raw;
}

// ---- RMSNorm ----------------------------------------------------------------------
// y = (x * 1/sqrt(mean(x^2) + eps)) * w, in float, rounded once on the store.
// One workgroup per output row. `row_idx` (optional) picks the input row of each
// output row. With `delta`, the input is resid + factor * delta (float sum); `write_resid`
// stores that sum back into resid (only meaningful without row_idx).
// At most 512 threads per workgroup, so that a thread may hold the eight partial sums of its
// sixteen elements in registers (a kernel that may be launched with 1,024 threads gets 128).
template <typename TX, typename TD, typename TO>
__global__ __launch_bounds__(512) void rmsnorm_kernel(TO* __restrict__ out, TX* x, const TD* __restrict__ delta,
                               int n_delta, long long delta_stride,
                               const float* __restrict__ w, const int* __restrict__ row_idx,
                               int dim, float eps, int write_resid, float factor) {
  __shared__ float scratch[16];
  const int r_out = blockIdx.x;
  const int r_in = row_idx ? row_idx[r_out] : r_out;
  TX* xr = x + static_cast<size_t>(r_in) * dim;
  const TD* dr = delta ? delta + static_cast<size_t>(r_in) * dim : nullptr;
  TO* yr = out + static_cast<size_t>(r_out) * dim;

  // Fast path (float rows whose length is a multiple of 4 and fits the registers): every
  // load of the row is a 16-byte load issued before anything is stored, so the row costs
  // one trip to memory.
  constexpr int VEC = 4;  // float4 chunks per thread
  if (sizeof(TX) == 4 && (dim & 3) == 0 && dim <= 4 * VEC * static_cast<int>(blockDim.x) &&
      (delta_stride & 3) == 0) {
    const int chunks = dim >> 2;
    const float4* x4 = reinterpret_cast<const float4*>(xr);
    const float4* w4 = reinterpret_cast<const float4*>(w);
    float4 held[VEC], wt[VEC];
#pragma unroll
    for (int n = 0; n < VEC; ++n) {
      const int c = threadIdx.x + n * blockDim.x;
      held[n] = (c < chunks) ? x4[c] : float4{0.f, 0.f, 0.f, 0.f};
      wt[n] = (c < chunks) ? w4[c] : float4{0.f, 0.f, 0.f, 0.f};
    }
    if (dr) {
      // Partial sums of the previous matrix product are added in a fixed order.  For the
      // usual counts every load is issued before the first addition: a loop over a count
      // only known at run time would wait for memory once per partial sum.
      const long long stride4 = delta_stride >> 2;
      float4 d[VEC];
#define PYLON_SUM_PARTS(ND)                                                                   \
  do {                                                                                        \
    float4 e[ND][VEC];                                                                        \
    _Pragma("unroll") for (int p = 0; p < ND; ++p) _Pragma("unroll") for (int n = 0; n < VEC; ++n) { \
      const int c = threadIdx.x + n * blockDim.x;                                             \
      e[p][n] = (c < chunks) ? load4(dr, c + p * stride4) : float4{0.f, 0.f, 0.f, 0.f};       \
    }                                                                                         \
    _Pragma("unroll") for (int n = 0; n < VEC; ++n) {                                         \
      d[n] = e[0][n];                                                                         \
      _Pragma("unroll") for (int p = 1; p < ND; ++p) {                                        \
        d[n].x += e[p][n].x; d[n].y += e[p][n].y; d[n].z += e[p][n].z; d[n].w += e[p][n].w;   \
      }                                                                                       \
    }                                                                                         \
  } while (0)
      if (n_delta == 1) {
        PYLON_SUM_PARTS(1);
      } else if (n_delta == 2) {
        PYLON_SUM_PARTS(2);
      } else if (n_delta == 4) {
        PYLON_SUM_PARTS(4);
      } else if (n_delta == 8) {
        PYLON_SUM_PARTS(8);
      } else {
        PYLON_SUM_PARTS(1);
        for (int p = 1; p < n_delta; ++p) {
#pragma unroll
          for (int n = 0; n < VEC; ++n) {
            const int c = threadIdx.x + n * blockDim.x;
            if (c < chunks) {
              const float4 e = load4(dr, c + p * stride4);
              d[n].x += e.x; d[n].y += e.y; d[n].z += e.z; d[n].w += e.w;
            }
          }
        }
      }
#undef PYLON_SUM_PARTS
#pragma unroll
      for (int n = 0; n < VEC; ++n) {
        held[n].x = fmaf(factor, d[n].x, held[n].x);
        held[n].y = fmaf(factor, d[n].y, held[n].y);
        held[n].z = fmaf(factor, d[n].z, held[n].z);
        held[n].w = fmaf(factor, d[n].w, held[n].w);
      }
    }
    float ss = 0.f;
#pragma unroll
    for (int n = 0; n < VEC; ++n)
      ss += held[n].x * held[n].x + held[n].y * held[n].y + held[n].z * held[n].z + held[n].w * held[n].w;
    const float total = block_sum(ss, scratch);
    const float inv = 1.0f / sqrtf(total / static_cast<float>(dim) + eps);
#pragma unroll
    for (int n = 0; n < VEC; ++n) {
      const int c = threadIdx.x + n * blockDim.x;
      if (c < chunks) {
        if (dr && write_resid) reinterpret_cast<float4*>(xr)[c] = held[n];
        const float y0 = (held[n].x * inv) * wt[n].x, y1 = (held[n].y * inv) * wt[n].y;
        const float y2 = (held[n].z * inv) * wt[n].z, y3 = (held[n].w * inv) * wt[n].w;
        store4(yr, c, y0, y1, y2, y3);
      }
    }
    return;
  }

  float ss = 0.f;
  for (int i = threadIdx.x; i < dim; i += blockDim.x) {
    float v = to_float(xr[i]);
    if (dr) {
      float d = to_float(dr[i]);
      for (int p = 1; p < n_delta; ++p) d += to_float(dr[i + p * delta_stride]);
      v = fmaf(factor, d, v);
      if (write_resid) xr[i] = from_float<TX>(v);
    }
    ss += v * v;
  }
  const float total = block_sum(ss, scratch);
  const float inv = 1.0f / sqrtf(total / static_cast<float>(dim) + eps);
  for (int i = threadIdx.x; i < dim; i += blockDim.x) {
    float v = to_float(xr[i]);
    if (dr && !write_resid) {
      float d = to_float(dr[i]);
      for (int p = 1; p < n_delta; ++p) d += to_float(dr[i + p * delta_stride]);
      v = fmaf(factor, d, v);
    }
    yr[i] = from_float<TO>((v * inv) * w[i]);
  }
}

// The same arithmetic, in the same order, for steps of many rows (prompt portions): a
// workgroup takes R rows and issues the loads of all of them before the first sum, so that one
// row's stores travel beside the next row's loads instead of every workgroup of the launch
// reading at one time and writing at another (2,048 rows of 2,560: 19.5 -> 15.8 us on data
// that no cache holds; four rows per workgroup lose again, 19.2 us).  Float residual, one
// delta, rows of a multiple of 4 elements that fit 16 per thread; as many threads as the
// kernel for few rows has at this width, so that a row's sum is formed in the same order.
template <typename TD, typename TO, int R, int THREADS>
__global__ __launch_bounds__(THREADS) void add_rmsnorm_many_kernel(TO* __restrict__ out, float* resid,
                                                               const TD* __restrict__ delta,
                                                               const float* __restrict__ w, int rows, int dim,
                                                               float eps, float factor) {
  __shared__ float scratch[16];
  constexpr int VEC = 4;
  const int chunks = dim >> 2;
  const float4* w4 = reinterpret_cast<const float4*>(w);
  float4 held[R][VEC], wt[VEC];
  const int r0 = blockIdx.x * R;
#pragma unroll
  for (int n = 0; n < VEC; ++n) {
    const int c = threadIdx.x + n * THREADS;
    wt[n] = (c < chunks) ? w4[c] : float4{0.f, 0.f, 0.f, 0.f};
  }
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const bool live = r0 + i < rows;
    const float* xr = resid + static_cast<size_t>(live ? r0 + i : r0) * dim;
    const TD* dr = delta + static_cast<size_t>(live ? r0 + i : r0) * dim;
#pragma unroll
    for (int n = 0; n < VEC; ++n) {
      const int c = threadIdx.x + n * THREADS;
      if (c < chunks) {
        const float4 x = reinterpret_cast<const float4*>(xr)[c];
        const float4 d = load4(dr, c);
        held[i][n] = float4{fmaf(factor, d.x, x.x), fmaf(factor, d.y, x.y), fmaf(factor, d.z, x.z), fmaf(factor, d.w, x.w)};
      } else {
        held[i][n] = float4{0.f, 0.f, 0.f, 0.f};
      }
    }
  }
#pragma unroll
  for (int i = 0; i < R; ++i) {
    if (r0 + i >= rows) break;  // the same for the whole workgroup
    float ss = 0.f;
#pragma unroll
    for (int n = 0; n < VEC; ++n)
      ss += held[i][n].x * held[i][n].x + held[i][n].y * held[i][n].y + held[i][n].z * held[i][n].z +
            held[i][n].w * held[i][n].w;
    const float total = block_sum(ss, scratch);
    const float inv = 1.0f / sqrtf(total / static_cast<float>(dim) + eps);
    float* xr = resid + static_cast<size_t>(r0 + i) * dim;
    TO* yr = out + static_cast<size_t>(r0 + i) * dim;
#pragma unroll
    for (int n = 0; n < VEC; ++n) {
      const int c = threadIdx.x + n * THREADS;
      if (c < chunks) {
        reinterpret_cast<float4*>(xr)[c] = held[i][n];
        store4(yr, c, (held[i][n].x * inv) * wt[n].x, (held[i][n].y * inv) * wt[n].y,
               (held[i][n].z * inv) * wt[n].z, (held[i][n].w * inv) * wt[n].w);
      }
    }
  }
}

#define PYLON_NORM_MANY_ROWS 512  // from this many rows on, a workgroup takes two

template <typename TX, typename TD>
static void launch_rmsnorm_out(void* out, int out_dtype, TX* x, const TD* delta, int n_delta,
                               long long delta_stride, const float* w, const int* row_idx, int rows,
                               int dim, float eps, int write_resid, float factor, hipStream_t stream) {
  if constexpr (sizeof(TX) == 4) {
    if (rows >= PYLON_NORM_MANY_ROWS && delta != nullptr && n_delta == 1 && row_idx == nullptr && write_resid &&
        (dim & 3) == 0 && dim <= 8192) {
      constexpr int R = 2;
      dim3 grid((rows + R - 1) / R);
#define GO(TO, THREADS)                                                                                    \
  hipLaunchKernelGGL((add_rmsnorm_many_kernel<TD, TO, R, THREADS>), grid, dim3(THREADS), 0, stream, (TO*)out, x, \
                     delta, w, rows, dim, eps, factor)
      if (dim > 4096) {
        if (out_dtype == PYLON_F32) GO(float, 512); else GO(bf16_t, 512);
      } else {
        if (out_dtype == PYLON_F32) GO(float, 256); else GO(bf16_t, 256);
      }
#undef GO
      return;
    }
  }
  dim3 grid(rows), block(dim > 4096 ? 512 : 256);
  if (out_dtype == PYLON_F32)
    hipLaunchKernelGGL((rmsnorm_kernel<TX, TD, float>), grid, block, 0, stream, (float*)out, x, delta,
                       n_delta, delta_stride, w, row_idx, dim, eps, write_resid, factor);
  else
    hipLaunchKernelGGL((rmsnorm_kernel<TX, TD, bf16_t>), grid, block, 0, stream, (bf16_t*)out, x,
                       delta, n_delta, delta_stride, w, row_idx, dim, eps, write_resid, factor);
}

// out[r] = rmsnorm(x[idx(r)]) for any input dtype.
extern "C" int pylon_rmsnorm(void* out, int out_dtype, const void* x, int x_dtype, const float* w,
                             const int* row_idx, int rows, int dim, float eps, hipStream_t stream) {
  PYLON_REQUIRE(pylon_valid_dtype(out_dtype) && pylon_valid_dtype(x_dtype), "rmsnorm: unknown dtype");
  PYLON_REQUIRE(rows >= 0 && dim > 0, "rmsnorm: bad sizes rows=%d dim=%d", rows, dim);
  PYLON_REQUIRE(eps >= 0.f, "rmsnorm: eps must not be negative");
  if (rows == 0) return 0;
  if (x_dtype == PYLON_F32)
    launch_rmsnorm_out<float, float>(out, out_dtype, (float*)x, nullptr, 0, 0, w, row_idx, rows, dim,
                                     eps, 0, 1.0f, stream);
  else
    launch_rmsnorm_out<bf16_t, bf16_t>(out, out_dtype, (bf16_t*)x, nullptr, 0, 0, w, row_idx, rows, dim,
                                       eps, 0, 1.0f, stream);
  PYLON_LAUNCHED("rmsnorm");
}

// resid (float) += factor * delta, then out = rmsnorm(resid). With row_idx the sum is formed only
// for the picked rows and resid is left untouched. delta may come as n_delta partial sums,
// delta_stride elements apart, which are added up first.
extern "C" int pylon_add_rmsnorm(void* out, int out_dtype, float* resid, const void* delta,
                                 int delta_dtype, int n_delta, long long delta_stride, const float* w,
                                 const int* row_idx, int rows, int dim, float eps, float factor,
                                 hipStream_t stream) {
  PYLON_REQUIRE(pylon_valid_dtype(out_dtype), "add_rmsnorm: unknown out dtype");
  PYLON_REQUIRE(delta == nullptr || pylon_valid_dtype(delta_dtype), "add_rmsnorm: unknown delta dtype");
  PYLON_REQUIRE(rows >= 0 && dim > 0, "add_rmsnorm: bad sizes rows=%d dim=%d", rows, dim);
  PYLON_REQUIRE(delta == nullptr || (n_delta >= 1 && n_delta <= 64), "add_rmsnorm: 1..64 partial sums");
  if (rows == 0) return 0;
  const int write_resid = (delta != nullptr && row_idx == nullptr) ? 1 : 0;
  if (delta == nullptr || delta_dtype == PYLON_F32)
    launch_rmsnorm_out<float, float>(out, out_dtype, resid, (const float*)delta, n_delta, delta_stride,
                                     w, row_idx, rows, dim, eps, write_resid, factor, stream);
  else
    launch_rmsnorm_out<float, bf16_t>(out, out_dtype, resid, (const bf16_t*)delta, n_delta,
                                      delta_stride, w, row_idx, rows, dim, eps, write_resid, factor, stream);
  PYLON_LAUNCHED("add_rmsnorm");
}

// resid (float) += delta, nothing else (the last residual sum when no norm follows).
template <typename TD>
__global__ void add_kernel(float* __restrict__ resid, const TD* __restrict__ delta, size_t n) {
  size_t i = static_cast<size_t>(blockIdx.x) * blockDim.x + threadIdx.x;
  const size_t step = static_cast<size_t>(gridDim.x) * blockDim.x;
  for (; i < n; i += step) resid[i] += to_float(delta[i]);
}

extern "C" int pylon_residual_add(float* resid, const void* delta, int delta_dtype, long long count,
                                  hipStream_t stream) {
  PYLON_REQUIRE(pylon_valid_dtype(delta_dtype), "residual_add: unknown dtype");
  PYLON_REQUIRE(count >= 0, "residual_add: negative count");
  if (count == 0) return 0;
  long long blocks = (count + 255) / 256;
  if (blocks > 65535 * 16) blocks = 65535 * 16;
  dim3 grid((unsigned)blocks), block(256);
  if (delta_dtype == PYLON_F32)
    hipLaunchKernelGGL(add_kernel<float>, grid, block, 0, stream, resid, (const float*)delta, (size_t)count);
  else
    hipLaunchKernelGGL(add_kernel<bf16_t>, grid, block, 0, stream, resid, (const bf16_t*)delta,
                       (size_t)count);
  PYLON_LAUNCHED("residual_add");
}

// ---- gated activation -----------------------------------------------------------------
// out[t, i] = act(gu[t, i]) * gu[t, inter + i]; act: silu(z) = z / (1 + exp(-z)), or gelu's tanh form.
template <typename TI, typename TO>
__global__ void silu_gate_kernel(TO* __restrict__ out, const TI* __restrict__ gu, int inter, size_t total, int act) {
  size_t i = static_cast<size_t>(blockIdx.x) * blockDim.x + threadIdx.x;
  const size_t step = static_cast<size_t>(gridDim.x) * blockDim.x;
  for (; i < total; i += step) {
    const size_t t = i / inter;
    const size_t c = i - t * inter;
    const float g = to_float(gu[t * 2 * inter + c]);
    const float u = to_float(gu[t * 2 * inter + inter + c]);
    out[i] = from_float<TO>(pylon_gate_act(g, act) * u);
  }
}

// bfloat16 rows whose length is a multiple of 8: eight elements (16 bytes) per thread.
__global__ void silu_gate_bf16x8_kernel(uint4* __restrict__ out, const uint4* __restrict__ gu, int chunks,
                                        size_t total, int act) {
  size_t i = static_cast<size_t>(blockIdx.x) * blockDim.x + threadIdx.x;
  const size_t step = static_cast<size_t>(gridDim.x) * blockDim.x;
  for (; i < total; i += step) {
    const size_t t = i / chunks;
    const size_t c = i - t * chunks;
    const uint4 g = gu[t * 2 * chunks + c];
    const uint4 u = gu[t * 2 * chunks + chunks + c];
    const uint32_t gw[4] = {g.x, g.y, g.z, g.w}, uw[4] = {u.x, u.y, u.z, u.w};
    uint32_t r[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const float g0 = __uint_as_float(gw[j] << 16), g1 = __uint_as_float(gw[j] & 0xffff0000u);
      const float u0 = __uint_as_float(uw[j] << 16), u1 = __uint_as_float(uw[j] & 0xffff0000u);
      const float a0 = pylon_gate_act(g0, act) * u0;
      const float a1 = pylon_gate_act(g1, act) * u1;
      r[j] = static_cast<uint32_t>(float_to_bf16_bits(a0)) | (static_cast<uint32_t>(float_to_bf16_bits(a1)) << 16);
    }
    out[i] = uint4{r[0], r[1], r[2], r[3]};
  }
}

// gate_up: [tokens, 2 * inter] of in_dtype; out: [tokens, inter] of out_dtype (float sums of a
// product may come in as float and leave as bfloat16: one rounding, after the activation).
extern "C" int pylon_silu_gate(void* out, int out_dtype, const void* gate_up, int in_dtype, int tokens, int inter,
                               int act, hipStream_t stream) {
  PYLON_REQUIRE(act == PYLON_ACT_SILU || act == PYLON_ACT_GELU, "silu_gate: unknown activation %d", act);
  PYLON_REQUIRE(pylon_valid_dtype(in_dtype) && pylon_valid_dtype(out_dtype), "silu_gate: unknown dtype");
  PYLON_REQUIRE(tokens >= 0 && inter > 0, "silu_gate: bad sizes tokens=%d inter=%d", tokens, inter);
  const size_t total = static_cast<size_t>(tokens) * inter;
  if (total == 0) return 0;
  if (in_dtype == PYLON_BF16 && out_dtype == PYLON_BF16 && inter % 8 == 0 &&
      (reinterpret_cast<uintptr_t>(out) & 15) == 0 && (reinterpret_cast<uintptr_t>(gate_up) & 15) == 0) {
    const size_t chunks_total = total / 8;
    size_t nblocks = (chunks_total + 255) / 256;
    if (nblocks > 65535u * 16u) nblocks = 65535u * 16u;
    hipLaunchKernelGGL(silu_gate_bf16x8_kernel, dim3((unsigned)nblocks), dim3(256), 0, stream, (uint4*)out,
                       (const uint4*)gate_up, inter / 8, chunks_total, act);
    PYLON_LAUNCHED("silu_gate");
  }
  size_t blocks = (total + 255) / 256;
  if (blocks > 65535u * 16u) blocks = 65535u * 16u;
  dim3 grid((unsigned)blocks), block(256);
#define GO(TI, TO) \
  hipLaunchKernelGGL((silu_gate_kernel<TI, TO>), grid, block, 0, stream, (TO*)out, (const TI*)gate_up, inter, total, act)
  if (in_dtype == PYLON_F32 && out_dtype == PYLON_F32) GO(float, float);
  else if (in_dtype == PYLON_F32) GO(float, bf16_t);
  else if (out_dtype == PYLON_F32) GO(bf16_t, float);
  else GO(bf16_t, bf16_t);
#undef GO
  PYLON_LAUNCHED("silu_gate");
}

// ---- gated activation with constants -----------------------------------------------------
// out[t, i] = a(g) * (u + offset) with g = min(gu[t, i], limit), u = clamp(gu[t, inter + i], -limit,
// limit) and a(g) = g / (1 + exp(-alpha * g)): a sigmoid-gated unit whose steepness, offset of
// the linear branch and cap are the caller's (limit <= 0: no cap).
template <typename TI, typename TO>
__global__ void gated_act_kernel(TO* __restrict__ out, const TI* __restrict__ gu, int inter, size_t total,
                                 float alpha, float offset, float limit, const float* __restrict__ bias) {
  size_t i = static_cast<size_t>(blockIdx.x) * blockDim.x + threadIdx.x;
  const size_t step = static_cast<size_t>(gridDim.x) * blockDim.x;
  for (; i < total; i += step) {
    const size_t t = i / inter;
    const size_t c = i - t * inter;
    float g = to_float(gu[t * 2 * inter + c]);
    float u = to_float(gu[t * 2 * inter + inter + c]);
    if (bias != nullptr) {  // the two projections' biases, [2 inter]
      g += bias[c];
      u += bias[inter + c];
    }
    if (limit > 0.f) {
      g = fminf(g, limit);
      u = fminf(fmaxf(u, -limit), limit);
    }
    out[i] = from_float<TO>((g / (1.0f + expf(-alpha * g))) * (u + offset));
  }
}

// bfloat16 rows whose length is a multiple of 8: eight elements (16 bytes) per thread.
__global__ void gated_act_bf16x8_kernel(uint4* __restrict__ out, const uint4* __restrict__ gu, int chunks, size_t total,
                                        float alpha, float offset, float limit) {
  size_t i = static_cast<size_t>(blockIdx.x) * blockDim.x + threadIdx.x;
  const size_t step = static_cast<size_t>(gridDim.x) * blockDim.x;
  for (; i < total; i += step) {
    const size_t t = i / chunks;
    const size_t c = i - t * chunks;
    const uint4 g = gu[t * 2 * chunks + c];
    const uint4 u = gu[t * 2 * chunks + chunks + c];
    const uint32_t gw[4] = {g.x, g.y, g.z, g.w}, uw[4] = {u.x, u.y, u.z, u.w};
    uint32_t r[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      float gv[2] = {__uint_as_float(gw[j] << 16), __uint_as_float(gw[j] & 0xffff0000u)};
      float uv[2] = {__uint_as_float(uw[j] << 16), __uint_as_float(uw[j] & 0xffff0000u)};
      float a[2];
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        if (limit > 0.f) {
          gv[k] = fminf(gv[k], limit);
          uv[k] = fminf(fmaxf(uv[k], -limit), limit);
        }
        a[k] = (gv[k] / (1.0f + expf(-alpha * gv[k]))) * (uv[k] + offset);
      }
      r[j] = static_cast<uint32_t>(float_to_bf16_bits(a[0])) | (static_cast<uint32_t>(float_to_bf16_bits(a[1])) << 16);
    }
    out[i] = uint4{r[0], r[1], r[2], r[3]};
  }
}

extern "C" int pylon_gated_act(void* out, int out_dtype, const void* gate_up, int in_dtype, int tokens, int inter,
                               float alpha, float offset, float limit, const float* bias, hipStream_t stream) {
  PYLON_REQUIRE(pylon_valid_dtype(in_dtype) && pylon_valid_dtype(out_dtype), "gated_act: unknown dtype");
  PYLON_REQUIRE(tokens >= 0 && inter > 0, "gated_act: bad sizes tokens=%d inter=%d", tokens, inter);
  const size_t total = static_cast<size_t>(tokens) * inter;
  if (total == 0) return 0;
  if (bias == nullptr && in_dtype == PYLON_BF16 && out_dtype == PYLON_BF16 && inter % 8 == 0 &&
      (reinterpret_cast<uintptr_t>(out) & 15) == 0 && (reinterpret_cast<uintptr_t>(gate_up) & 15) == 0) {
    const size_t chunks_total = total / 8;
    size_t nblocks = (chunks_total + 255) / 256;
    if (nblocks > 65535u * 16u) nblocks = 65535u * 16u;
    hipLaunchKernelGGL(gated_act_bf16x8_kernel, dim3((unsigned)nblocks), dim3(256), 0, stream, (uint4*)out,
                       (const uint4*)gate_up, inter / 8, chunks_total, alpha, offset, limit);
    PYLON_LAUNCHED("gated_act");
  }
  size_t blocks = (total + 255) / 256;
  if (blocks > 65535u * 16u) blocks = 65535u * 16u;
  dim3 grid((unsigned)blocks), block(256);
#define GO(TI, TO)                                                                                             \
  hipLaunchKernelGGL((gated_act_kernel<TI, TO>), grid, block, 0, stream, (TO*)out, (const TI*)gate_up, inter, \
                     total, alpha, offset, limit, bias)
  if (in_dtype == PYLON_F32 && out_dtype == PYLON_F32) GO(float, float);
  else if (in_dtype == PYLON_F32) GO(float, bf16_t);
  else if (out_dtype == PYLON_F32) GO(bf16_t, float);
  else GO(bf16_t, bf16_t);
#undef GO
  PYLON_LAUNCHED("gated_act");
}

// ---- the square of relu: out = max(x, 0)^2 -----------------------------------------------------
template <typename TI, typename TO>
__global__ void relu2_kernel(TO* __restrict__ out, const TI* __restrict__ x, size_t total) {
  size_t i = static_cast<size_t>(blockIdx.x) * blockDim.x + threadIdx.x;
  const size_t step = static_cast<size_t>(gridDim.x) * blockDim.x;
  for (; i < total; i += step) {
    const float v = fmaxf(to_float(x[i]), 0.f);
    out[i] = from_float<TO>(v * v);
  }
}

// Eight elements (16 bytes of bfloat16) a thread.
__global__ void relu2_bf16x8_kernel(uint4* __restrict__ out, const uint4* __restrict__ x, size_t total) {
  size_t i = static_cast<size_t>(blockIdx.x) * blockDim.x + threadIdx.x;
  const size_t step = static_cast<size_t>(gridDim.x) * blockDim.x;
  for (; i < total; i += step) {
    const uint4 raw = x[i];
    const uint32_t w[4] = {raw.x, raw.y, raw.z, raw.w};
    uint32_t r[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const float a = fmaxf(__uint_as_float(w[j] << 16), 0.f), b = fmaxf(__uint_as_float(w[j] & 0xffff0000u), 0.f);
      r[j] = static_cast<uint32_t>(float_to_bf16_bits(a * a)) | (static_cast<uint32_t>(float_to_bf16_bits(b * b)) << 16);
    }
    out[i] = uint4{r[0], r[1], r[2], r[3]};
  }
}

// x and out may be the same tensor where their types are.
extern "C" int pylon_relu2(void* out, int out_dtype, const void* x, int in_dtype, long long count, hipStream_t stream) {
  PYLON_REQUIRE(pylon_valid_dtype(in_dtype) && pylon_valid_dtype(out_dtype) && count >= 0, "relu2: bad arguments");
  if (count == 0) return 0;
  const bool wide = in_dtype == PYLON_BF16 && out_dtype == PYLON_BF16 && count % 8 == 0 &&
                    ((reinterpret_cast<uintptr_t>(out) | reinterpret_cast<uintptr_t>(x)) & 15) == 0;
  const size_t total = wide ? static_cast<size_t>(count) / 8 : static_cast<size_t>(count);
  size_t blocks = (total + 255) / 256;
  if (blocks > 65535u * 16u) blocks = 65535u * 16u;
  dim3 grid((unsigned)blocks), block(256);
  if (wide) hipLaunchKernelGGL(relu2_bf16x8_kernel, grid, block, 0, stream, (uint4*)out, (const uint4*)x, total);
  else if (in_dtype == PYLON_F32 && out_dtype == PYLON_F32)
    hipLaunchKernelGGL((relu2_kernel<float, float>), grid, block, 0, stream, (float*)out, (const float*)x, total);
  else if (in_dtype == PYLON_F32)
    hipLaunchKernelGGL((relu2_kernel<float, bf16_t>), grid, block, 0, stream, (bf16_t*)out, (const float*)x, total);
  else if (out_dtype == PYLON_F32)
    hipLaunchKernelGGL((relu2_kernel<bf16_t, float>), grid, block, 0, stream, (float*)out, (const bf16_t*)x, total);
  else
    hipLaunchKernelGGL((relu2_kernel<bf16_t, bf16_t>), grid, block, 0, stream, (bf16_t*)out, (const bf16_t*)x, total);
  PYLON_LAUNCHED("relu2");
}

// ---- scaling in place ------------------------------------------------------------------------
__global__ void scale_kernel(float* __restrict__ x, size_t total, float factor) {
  size_t i = static_cast<size_t>(blockIdx.x) * blockDim.x + threadIdx.x;
  const size_t step = static_cast<size_t>(gridDim.x) * blockDim.x;
  for (; i < total; i += step) x[i] *= factor;
}

extern "C" int pylon_scale(float* x, long long count, float factor, hipStream_t stream) {
  PYLON_REQUIRE(count >= 0, "scale: negative count");
  if (count == 0) return 0;
  size_t blocks = (static_cast<size_t>(count) + 255) / 256;
  if (blocks > 65535u * 16u) blocks = 65535u * 16u;
  hipLaunchKernelGGL(scale_kernel, dim3((unsigned)blocks), dim3(256), 0, stream, x, (size_t)count, factor);
  PYLON_LAUNCHED("scale");
}

// ---- soft cap in place: x <- cap * tanh(x / cap) ----------------------------------------------
__global__ void softcap_kernel(float* __restrict__ x, size_t total, float cap) {
  size_t i = static_cast<size_t>(blockIdx.x) * blockDim.x + threadIdx.x;
  const size_t step = static_cast<size_t>(gridDim.x) * blockDim.x;
  for (; i < total; i += step) x[i] = cap * tanhf(x[i] / cap);
}

extern "C" int pylon_softcap(float* x, long long count, float cap, hipStream_t stream) {
  PYLON_REQUIRE(count >= 0, "softcap: negative count");
  PYLON_REQUIRE(cap > 0.f, "softcap: the cap must be positive");
  if (count == 0) return 0;
  size_t blocks = (static_cast<size_t>(count) + 255) / 256;
  if (blocks > 65535u * 16u) blocks = 65535u * 16u;
  hipLaunchKernelGGL(softcap_kernel, dim3((unsigned)blocks), dim3(256), 0, stream, x, (size_t)count, cap);
  PYLON_LAUNCHED("softcap");
}

// ---- sinusoidal positions ----------------------------------------------------------------------
// x[t, 2i] += sin(p_t * f_i), x[t, 2i + 1] += cos(p_t * f_i): the angle is the float product of the
// token's position and a frequency that the caller formed once; sine and cosine with full range
// reduction.
__global__ void add_sinusoid_kernel(float* __restrict__ x, const int* __restrict__ positions,
                                    const float* __restrict__ freq, int dim, size_t total_pairs, int pairs) {
  size_t i = static_cast<size_t>(blockIdx.x) * blockDim.x + threadIdx.x;
  const size_t step = static_cast<size_t>(gridDim.x) * blockDim.x;
  for (; i < total_pairs; i += step) {
    const size_t t = i / pairs;
    const int k = static_cast<int>(i - t * pairs);
    const float angle = static_cast<float>(positions[t]) * freq[k];
    float* row = x + t * dim;
    row[2 * k] += sinf(angle);
    if (2 * k + 1 < dim) row[2 * k + 1] += cosf(angle);
  }
}

// x: float [tokens, dim]; positions: int [tokens]; freq: float [(dim + 1) / 2].
extern "C" int pylon_add_sinusoid(float* x, const int* positions, const float* freq, int tokens, int dim,
                                  hipStream_t stream) {
  PYLON_REQUIRE(tokens >= 0 && dim > 0, "add_sinusoid: bad sizes");
  if (tokens == 0) return 0;
  const int pairs = (dim + 1) / 2;
  const size_t total = static_cast<size_t>(tokens) * pairs;
  size_t blocks = (total + 255) / 256;
  if (blocks > 65535u * 16u) blocks = 65535u * 16u;
  hipLaunchKernelGGL(add_sinusoid_kernel, dim3((unsigned)blocks), dim3(256), 0, stream, x, positions, freq, dim, total,
                     pairs);
  PYLON_LAUNCHED("add_sinusoid");
}

// ---- a bias per column, in place -----------------------------------------------------------------
template <typename T>
__global__ void add_bias_kernel(T* __restrict__ x, const float* __restrict__ bias, int dim, size_t total) {
  size_t i = static_cast<size_t>(blockIdx.x) * blockDim.x + threadIdx.x;
  const size_t step = static_cast<size_t>(gridDim.x) * blockDim.x;
  for (; i < total; i += step) x[i] = from_float<T>(to_float(x[i]) + bias[i % dim]);
}

// x: [rows, dim] of dtype, contiguous; bias: float [dim].
extern "C" int pylon_add_bias(void* x, int dtype, const float* bias, long long rows, int dim, hipStream_t stream) {
  PYLON_REQUIRE(pylon_valid_dtype(dtype) && rows >= 0 && dim > 0, "add_bias: bad arguments");
  const size_t total = static_cast<size_t>(rows) * dim;
  if (total == 0) return 0;
  size_t blocks = (total + 255) / 256;
  if (blocks > 65535u * 16u) blocks = 65535u * 16u;
  if (dtype == PYLON_F32)
    hipLaunchKernelGGL(add_bias_kernel<float>, dim3((unsigned)blocks), dim3(256), 0, stream, (float*)x, bias, dim, total);
  else
    hipLaunchKernelGGL(add_bias_kernel<bf16_t>, dim3((unsigned)blocks), dim3(256), 0, stream, (bf16_t*)x, bias, dim, total);
  PYLON_LAUNCHED("add_bias");
}

// ---- a sigmoid gate on a mixer's heads, in place ---------------------------------------------------
// x[t, i] *= sigmoid(g[t, i / per]): per = the size of a head for one gate per head, 1 for a gate
// per element.  The gates' logits lie in rows g_stride apart (a slice of a wider projection).
template <typename T>
__global__ void sigmoid_gate_kernel(T* __restrict__ x, const T* __restrict__ g, long long g_stride, int dim, int per,
                                    size_t total) {
  size_t i = static_cast<size_t>(blockIdx.x) * blockDim.x + threadIdx.x;
  const size_t step = static_cast<size_t>(gridDim.x) * blockDim.x;
  for (; i < total; i += step) {
    const size_t t = i / dim;
    const int e = static_cast<int>(i - t * dim);
    const float z = to_float(g[t * g_stride + e / per]);
    x[i] = from_float<T>(to_float(x[i]) / (1.0f + expf(-z)));
  }
}

// Eight bfloat16 elements (16 bytes) a thread; EACH: a gate per element (eight neighbours, 16 bytes as well), else
// one for all eight (a head's size is a multiple of 8).
template <bool EACH>
__global__ void sigmoid_gate_bf16x8_kernel(uint4* __restrict__ x, const bf16_t* __restrict__ g, long long g_stride, int chunks,
                                           int per, size_t total) {
  size_t i = static_cast<size_t>(blockIdx.x) * blockDim.x + threadIdx.x;
  const size_t step = static_cast<size_t>(gridDim.x) * blockDim.x;
  for (; i < total; i += step) {
    const size_t t = i / chunks;
    const int e = static_cast<int>(i - t * chunks) * 8;
    const uint4 raw = x[i];
    const uint32_t w[4] = {raw.x, raw.y, raw.z, raw.w};
    uint32_t gw[4] = {0u, 0u, 0u, 0u};
    float one = 0.f;
    if constexpr (EACH) {
      const uint4 graw = *reinterpret_cast<const uint4*>(g + t * g_stride + e);
      gw[0] = graw.x; gw[1] = graw.y; gw[2] = graw.z; gw[3] = graw.w;
    } else {
      one = 1.0f / (1.0f + __expf(-to_float(g[t * g_stride + e / per])));
    }
    uint32_t r[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const float ga = EACH ? 1.0f / (1.0f + __expf(-__uint_as_float(gw[j] << 16))) : one;
      const float gb = EACH ? 1.0f / (1.0f + __expf(-__uint_as_float(gw[j] & 0xffff0000u))) : one;
      const float a = __uint_as_float(w[j] << 16) * ga, b = __uint_as_float(w[j] & 0xffff0000u) * gb;
      r[j] = static_cast<uint32_t>(float_to_bf16_bits(a)) | (static_cast<uint32_t>(float_to_bf16_bits(b)) << 16);
    }
    x[i] = uint4{r[0], r[1], r[2], r[3]};
  }
}

// x: [rows, dim] of dtype, contiguous; g: [rows, dim / per] of the same dtype, rows g_stride apart.
extern "C" int pylon_sigmoid_gate(void* x, int dtype, const void* g, long long g_stride, long long rows, int dim,
                                  int per, hipStream_t stream) {
  PYLON_REQUIRE(pylon_valid_dtype(dtype) && rows >= 0 && dim > 0 && per > 0 && dim % per == 0,
                "sigmoid_gate: bad arguments");
  PYLON_REQUIRE(g_stride >= dim / per, "sigmoid_gate: rows of gates overlap");
  const size_t total = static_cast<size_t>(rows) * dim;
  if (total == 0) return 0;
  if (dtype == PYLON_BF16 && dim % 8 == 0 && (reinterpret_cast<uintptr_t>(x) & 15) == 0 &&
      (per % 8 == 0 || (per == 1 && g_stride % 8 == 0 && (reinterpret_cast<uintptr_t>(g) & 15) == 0))) {
    size_t wide = (total / 8 + 255) / 256;
    if (wide > 65535u * 16u) wide = 65535u * 16u;
    if (per == 1)
      hipLaunchKernelGGL(sigmoid_gate_bf16x8_kernel<true>, dim3((unsigned)wide), dim3(256), 0, stream, (uint4*)x,
                         (const bf16_t*)g, g_stride, dim / 8, per, total / 8);
    else
      hipLaunchKernelGGL(sigmoid_gate_bf16x8_kernel<false>, dim3((unsigned)wide), dim3(256), 0, stream, (uint4*)x,
                         (const bf16_t*)g, g_stride, dim / 8, per, total / 8);
    PYLON_LAUNCHED("sigmoid_gate");
  }
  size_t blocks = (total + 255) / 256;
  if (blocks > 65535u * 16u) blocks = 65535u * 16u;
  if (dtype == PYLON_F32)
    hipLaunchKernelGGL(sigmoid_gate_kernel<float>, dim3((unsigned)blocks), dim3(256), 0, stream, (float*)x,
                       (const float*)g, g_stride, dim, per, total);
  else
    hipLaunchKernelGGL(sigmoid_gate_kernel<bf16_t>, dim3((unsigned)blocks), dim3(256), 0, stream, (bf16_t*)x,
                       (const bf16_t*)g, g_stride, dim, per, total);
  PYLON_LAUNCHED("sigmoid_gate");
}

// ---- two mixers side by side: out = sa * a + sb * b, float ----------------------------------------
// a and b are each one tensor of n elements, or a stack of float partial sums that are added up in
// order first (parts > 1: the parts lie n elements apart).
template <typename TA, typename TB>
__global__ void scaled_sum_kernel(float* __restrict__ out, const TA* __restrict__ a, int a_parts, float sa,
                                  const TB* __restrict__ b, int b_parts, float sb, size_t n) {
  size_t i = static_cast<size_t>(blockIdx.x) * blockDim.x + threadIdx.x;
  const size_t step = static_cast<size_t>(gridDim.x) * blockDim.x;
  for (; i < n; i += step) {
    float x = to_float(a[i]);
    for (int p = 1; p < a_parts; ++p) x += to_float(a[i + p * n]);
    float y = to_float(b[i]);
    for (int p = 1; p < b_parts; ++p) y += to_float(b[i + p * n]);
    out[i] = fmaf(sa, x, sb * y);
  }
}

extern "C" int pylon_scaled_sum(float* out, const void* a, int a_dtype, int a_parts, float sa, const void* b,
                                int b_dtype, int b_parts, float sb, long long n, hipStream_t stream) {
  PYLON_REQUIRE(pylon_valid_dtype(a_dtype) && pylon_valid_dtype(b_dtype) && n >= 0 && a_parts >= 1 && b_parts >= 1,
                "scaled_sum: bad arguments");
  if (n == 0) return 0;
  size_t blocks = (static_cast<size_t>(n) + 255) / 256;
  if (blocks > 65535u * 16u) blocks = 65535u * 16u;
#define GO(TA, TB)                                                                                          \
  hipLaunchKernelGGL((scaled_sum_kernel<TA, TB>), dim3((unsigned)blocks), dim3(256), 0, stream, out,        \
                     (const TA*)a, a_parts, sa, (const TB*)b, b_parts, sb, static_cast<size_t>(n))
  if (a_dtype == PYLON_F32 && b_dtype == PYLON_F32) GO(float, float);
  else if (a_dtype == PYLON_F32) GO(float, bf16_t);
  else if (b_dtype == PYLON_F32) GO(bf16_t, float);
  else GO(bf16_t, bf16_t);
#undef GO
  PYLON_LAUNCHED("scaled_sum");
}
