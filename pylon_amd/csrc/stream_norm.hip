// A residual stream kept in several copies that a layer's sublayers mix (hyper-connections), fused
// with the norm in front of the next sublayer:
//
//   d = sum_p delta[p]                              (the last sublayer's output, maybe as partial sums)
//   x_t <- sum_s mix[s, t] x_s + write[t] d         (each from what all copies held before)
//   u = sum_t read[t] x_t                           (what the next sublayer, or the output, reads)
//   out = (u - mean(u)) / sqrt(var(u) + eps) * w    (layer norm; without `centre` u / sqrt(mean(u^2) + eps) * w)
//
// all in float, `out` rounded once on the store.  One copy without coefficients is an ordinary
// residual stream: x += d, out = norm(x).  The variance is the mean of the squared deviations, taken
// from the row in registers after its mean.  One workgroup per output row; a thread keeps its
// elements of u between the passes, so that a row costs one trip to memory.  The order of every sum
// depends on the row's length, the number of copies and of partial sums only.
#include "common.h"

#define SN_BATCH 4  // partial sums whose loads are in flight together

template <int VEC>
struct SnVec {
  float v[VEC];
};

template <int VEC>
__device__ __forceinline__ SnVec<VEC> sn_load(const float* p, int c) {
  SnVec<VEC> r;
  if constexpr (VEC == 4) {
    const float4 raw = reinterpret_cast<const float4*>(p)[c];
    r.v[0] = raw.x; r.v[1] = raw.y; r.v[2] = raw.z; r.v[3] = raw.w;
  } else {
    r.v[0] = p[c];
  }
  return r;
}

template <int VEC>
__device__ __forceinline__ SnVec<VEC> sn_load(const bf16_t* p, int c) {
  SnVec<VEC> r;
  if constexpr (VEC == 4) {
    const uint2 raw = reinterpret_cast<const uint2*>(p)[c];
    r.v[0] = __uint_as_float(raw.x << 16); r.v[1] = __uint_as_float(raw.x & 0xffff0000u);
    r.v[2] = __uint_as_float(raw.y << 16); r.v[3] = __uint_as_float(raw.y & 0xffff0000u);
  } else {
    r.v[0] = to_float(p[c]);
  }
  return r;
}

template <int VEC>
__device__ __forceinline__ void sn_store(float* p, int c, const SnVec<VEC>& a) {
  if constexpr (VEC == 4) reinterpret_cast<float4*>(p)[c] = float4{a.v[0], a.v[1], a.v[2], a.v[3]};
  else p[c] = a.v[0];
}

template <int VEC>
__device__ __forceinline__ void sn_store(bf16_t* p, int c, const SnVec<VEC>& a) {
  if constexpr (VEC == 4) {
    uint2 raw;
    raw.x = static_cast<uint32_t>(float_to_bf16_bits(a.v[0])) | (static_cast<uint32_t>(float_to_bf16_bits(a.v[1])) << 16);
    raw.y = static_cast<uint32_t>(float_to_bf16_bits(a.v[2])) | (static_cast<uint32_t>(float_to_bf16_bits(a.v[3])) << 16);
    reinterpret_cast<uint2*>(p)[c] = raw;
  } else {
    p[c] = from_float<bf16_t>(a.v[0]);
  }
}

// S: the most copies this instance takes (`streams` of them are there); PER: pieces of VEC elements a thread.
template <typename TD, typename TO, int S, int PER, int VEC>
__global__ __launch_bounds__(1024) void stream_norm_kernel(
    TO* __restrict__ out, float* resid, long long stream_stride, int streams, const TD* __restrict__ delta,
    int n_delta, long long delta_stride, const float* __restrict__ mix, const float* __restrict__ write,
    const float* __restrict__ read, const float* __restrict__ w, const int* __restrict__ row_idx, int dim,
    float eps, int centre, int store) {
  __shared__ float scratch[16];
  const int r_out = blockIdx.x;
  const int r_in = row_idx ? row_idx[r_out] : r_out;
  float* xr = resid + static_cast<size_t>(r_in) * dim;
  const TD* dr = delta ? delta + static_cast<size_t>(r_in) * dim : nullptr;
  const int pieces = dim / VEC;
  SnVec<VEC> u[PER];
#pragma unroll
  for (int n = 0; n < PER; ++n) {
    const int c = threadIdx.x + n * blockDim.x;
#pragma unroll
    for (int e = 0; e < VEC; ++e) u[n].v[e] = 0.f;
    if (c >= pieces) continue;
    SnVec<VEC> x[S];
#pragma unroll
    for (int s = 0; s < S; ++s)
      if (s < streams) x[s] = sn_load<VEC>(xr + s * stream_stride, c);
    if (dr) {
      SnVec<VEC> d = sn_load<VEC>(dr, c);
      for (int p0 = 1; p0 < n_delta; p0 += SN_BATCH) {
        SnVec<VEC> part[SN_BATCH];
#pragma unroll
        for (int p = 0; p < SN_BATCH; ++p)  // past the last: the last again, unused
          part[p] = sn_load<VEC>(dr + (p0 + p < n_delta ? p0 + p : n_delta - 1) * delta_stride, c);
#pragma unroll
        for (int p = 0; p < SN_BATCH; ++p)
          if (p0 + p < n_delta) {
#pragma unroll
            for (int e = 0; e < VEC; ++e) d.v[e] += part[p].v[e];
          }
      }
      // one new copy from all old ones (a copy index known at compile time stays in registers; with many
      // copies the loop is kept and a missing mix is the identity)
      auto renew = [&](int t, bool identity) {
        SnVec<VEC> y;
        const float wt = write ? write[t] : 1.f;
        const float rt = read ? read[t] : 1.f;
#pragma unroll
        for (int e = 0; e < VEC; ++e) y.v[e] = 0.f;
#pragma unroll
        for (int s = 0; s < S; ++s) {
          if (s >= streams) continue;
          const float m = identity ? (s == t ? 1.f : 0.f) : mix[s * streams + t];
#pragma unroll
          for (int e = 0; e < VEC; ++e) y.v[e] = fmaf(m, x[s].v[e], y.v[e]);
        }
#pragma unroll
        for (int e = 0; e < VEC; ++e) y.v[e] = fmaf(wt, d.v[e], y.v[e]);
        if (store) sn_store<VEC>(xr + t * stream_stride, c, y);
#pragma unroll
        for (int e = 0; e < VEC; ++e) u[n].v[e] = fmaf(rt, y.v[e], u[n].v[e]);
      };
      if constexpr (S <= 4) {
#pragma unroll
        for (int t = 0; t < S; ++t)
          if (t < streams) renew(t, mix == nullptr);
      } else {
        for (int t = 0; t < streams; ++t) renew(t, mix == nullptr);
      }
    } else {
#pragma unroll
      for (int t = 0; t < S; ++t) {
        if (t >= streams) continue;
        const float rt = read ? read[t] : 1.f;
#pragma unroll
        for (int e = 0; e < VEC; ++e) u[n].v[e] = fmaf(rt, x[t].v[e], u[n].v[e]);
      }
    }
  }
  if (centre) {
    float sum = 0.f;
#pragma unroll
    for (int n = 0; n < PER; ++n)
#pragma unroll
      for (int e = 0; e < VEC; ++e) sum += u[n].v[e];
    const float mean = block_sum(sum, scratch) / static_cast<float>(dim);
#pragma unroll
    for (int n = 0; n < PER; ++n)
      if (threadIdx.x + n * blockDim.x < pieces) {
#pragma unroll
        for (int e = 0; e < VEC; ++e) u[n].v[e] -= mean;
      }
  }
  float ss = 0.f;
#pragma unroll
  for (int n = 0; n < PER; ++n)
#pragma unroll
    for (int e = 0; e < VEC; ++e) ss += u[n].v[e] * u[n].v[e];
  const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / static_cast<float>(dim) + eps);
  TO* yr = out + static_cast<size_t>(r_out) * dim;
#pragma unroll
  for (int n = 0; n < PER; ++n) {
    const int c = threadIdx.x + n * blockDim.x;
    if (c >= pieces) continue;
    const SnVec<VEC> g = sn_load<VEC>(w, c);
    SnVec<VEC> y;
#pragma unroll
    for (int e = 0; e < VEC; ++e) y.v[e] = (u[n].v[e] * inv) * g.v[e];
    sn_store<VEC>(yr, c, y);
  }
}

// resid: float [streams, tokens, dim], the copies stream_stride elements apart, updated in place unless
// row_idx picks rows (or delta is null).  delta: null (nothing is added, nothing mixed), [tokens, dim], or
// n_delta such tensors delta_stride elements apart.  mix: float [streams, streams] (from, to) or null
// (every copy stays itself); write, read: float [streams] or null (ones).  w: dim floats.
// out: [rows, dim] of out_dtype.
extern "C" int pylon_stream_norm(void* out, int out_dtype, float* resid, long long stream_stride, int streams,
                                 const void* delta, int delta_dtype, int n_delta, long long delta_stride,
                                 const float* mix, const float* write, const float* read, const float* w,
                                 const int* row_idx, int rows, int dim, float eps, int centre, hipStream_t stream) {
  PYLON_REQUIRE(pylon_valid_dtype(out_dtype) && pylon_valid_dtype(delta_dtype), "stream_norm: unknown dtype");
  PYLON_REQUIRE(rows >= 0 && dim > 0 && dim <= 16384, "stream_norm: rows of 1 to 16384 elements, got %d", dim);
  PYLON_REQUIRE(streams >= 1 && streams <= 16, "stream_norm: 1 to 16 copies of the stream, got %d", streams);
  PYLON_REQUIRE(n_delta >= 1 && out != nullptr && w != nullptr, "stream_norm: bad arguments");
  PYLON_REQUIRE(streams == 1 || stream_stride >= dim, "stream_norm: the copies overlap");
  if (rows == 0) return 0;
  const int store = (delta != nullptr && row_idx == nullptr) ? 1 : 0;
  const uintptr_t bases = reinterpret_cast<uintptr_t>(out) | reinterpret_cast<uintptr_t>(resid) |
                          reinterpret_cast<uintptr_t>(delta) | reinterpret_cast<uintptr_t>(w);
  const bool wide = dim % 4 == 0 && stream_stride % 4 == 0 && delta_stride % 4 == 0 && bases % 16 == 0;
  const int pieces = wide ? dim / 4 : dim;
  const int per = (pieces + 1023) / 1024 <= 1 ? 1 : (pieces + 1023) / 1024 <= 4 ? 4 : 16;
  const int threads = ((pieces + per - 1) / per + PYLON_WAVE - 1) / PYLON_WAVE * PYLON_WAVE;
  dim3 grid(rows), block(threads);
#define GO(TD, TO, S, PER, VEC)                                                                                     \
  hipLaunchKernelGGL((stream_norm_kernel<TD, TO, S, PER, VEC>), grid, block, 0, stream, (TO*)out, resid, stream_stride, \
                     streams, (const TD*)delta, n_delta, delta_stride, mix, write, read, w, row_idx, dim, eps, centre, store)
#define PICK(TD, TO, S)                    \
  do {                                     \
    if (wide && per == 1) GO(TD, TO, S, 1, 4);  \
    else if (wide) GO(TD, TO, S, 4, 4);    \
    else if (per <= 4) GO(TD, TO, S, 4, 1); \
    else GO(TD, TO, S, 16, 1);             \
  } while (0)
#define PICK_MANY(TD, TO)                  \
  do {                                     \
    if (wide) GO(TD, TO, 16, 4, 4);        \
    else GO(TD, TO, 16, 16, 1);            \
  } while (0)
#define STREAMS(TD, TO)                       \
  do {                                        \
    if (streams == 1) PICK(TD, TO, 1);        \
    else if (streams == 2) PICK(TD, TO, 2);   \
    else if (streams <= 4) PICK(TD, TO, 4);   \
    else PICK_MANY(TD, TO);                   \
  } while (0)
  if (delta_dtype == PYLON_F32 && out_dtype == PYLON_F32) STREAMS(float, float);
  else if (delta_dtype == PYLON_F32) STREAMS(float, bf16_t);
  else if (out_dtype == PYLON_F32) STREAMS(bf16_t, float);
  else STREAMS(bf16_t, bf16_t);
#undef STREAMS
#undef PICK_MANY
#undef PICK
#undef GO
  PYLON_LAUNCHED("stream_norm");
}
