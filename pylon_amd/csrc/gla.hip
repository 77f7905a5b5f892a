// Gated linear attention: linear attention whose state forgets by a learned, input-dependent decay per
// key channel.  Per request and head a state S [dim, vdim] of floats goes from token to token:
//
//   z = W_a2 (W_a1 h) + b,   alpha = sigmoid(z)^(1/tau)        (one number per key channel)
//   S_t = diag(alpha_t) S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t  (q times q_scale; a row of S belongs to a key channel)
//   out_t = o_t / sqrt(mean(o_t^2) + eps) * w * silu(g_t)       (w: vdim numbers shared by the heads)
//
// The projection's rows hold q, k, v, g and the low-rank logits W_a1 h; W_a2 is applied here.
// Everything but the loads of the projection and the store of the result is float.
//
// This file holds the recurrent form: one workgroup per (row of the step, head) walks the row's tokens
// in order with S in registers, column j of S in the threads j, j + vdim, ..., each of which keeps every
// ip_count-th row.  The order of every sum is fixed by the head's sizes, so a request's results do not
// depend on how it was cut into steps or on what shared a step.
#include "common.h"
#include "gla.h"

template <typename T, int NI, int THREADS>
__global__ __launch_bounds__(THREADS) void gla_recurrent_kernel(
    T* __restrict__ out, const T* __restrict__ proj, long long ld, int q_off, int k_off, int v_off, int g_off, int a_off,
    int rank, const float* __restrict__ a2, const float* __restrict__ a2_bias, float inv_tau, float* state,
    const float* __restrict__ norm_w, const int* __restrict__ row_start, const int* __restrict__ row_slots, int heads,
    int dim, int vdim, int ip_count, float eps, float q_scale) {
  extern __shared__ float lds[];
  float* qs = lds;                 // [dim]
  float* ks = qs + dim;            // [dim]
  float* al = ks + dim;            // [dim]: the token's decays
  float* part = al + dim;          // [ip_count * vdim]
  float* red = part + ip_count * vdim;  // [16]
  const int row = blockIdx.x, head = blockIdx.y;
  const int tid = threadIdx.x;
  const int j = tid % vdim, ip = tid / vdim;  // column of S, and which rows of it
  const bool owner = ip < ip_count;           // the workgroup is padded to whole wavefronts
  const int begin = row_start[row], end = row_start[row + 1];
  float* st = state + ((static_cast<size_t>(row_slots[row]) * heads + head) * dim) * vdim;
  float s[NI];
#pragma unroll
  for (int n = 0; n < NI; ++n) {
    const int i = ip + n * ip_count;
    s[n] = (owner && i < dim) ? st[static_cast<size_t>(i) * vdim + j] : 0.f;
  }
  for (int t = begin; t < end; ++t) {
    const T* pr = proj + static_cast<size_t>(t) * ld;
    for (int e = tid; e < 3 * dim; e += blockDim.x) {
      const int what = e / dim, d = e - what * dim;
      if (what == 0) {
        al[d] = expf(gla_log_decay(pr + a_off, a2 + static_cast<size_t>(head * dim + d) * rank, rank,
                                   a2_bias[head * dim + d], inv_tau));
      } else if (what == 1) {
        qs[d] = to_float(pr[q_off + head * dim + d]) * q_scale;
      } else {
        ks[d] = to_float(pr[k_off + head * dim + d]);
      }
    }
    const float vj = to_float(pr[v_off + head * vdim + j]);
    const float gj = to_float(pr[g_off + head * vdim + j]);
    __syncthreads();
    float acc = 0.f;
    if (owner) {
#pragma unroll
      for (int n = 0; n < NI; ++n) {
        const int i = ip + n * ip_count;
        if (i < dim) {
          s[n] = fmaf(al[i], s[n], ks[i] * vj);
          acc = fmaf(s[n], qs[i], acc);
        }
      }
      part[ip * vdim + j] = acc;
    }
    __syncthreads();
    float o = 0.f, sq = 0.f;
    if (ip == 0) {
      for (int p = 0; p < ip_count; ++p) o += part[p * vdim + j];
      sq = o * o;
    }
    const float total = block_sum(sq, red);  // two barriers inside: qs, ks, al and part are free again after it
    if (ip == 0) {
      const float inv = 1.0f / sqrtf(total / static_cast<float>(vdim) + eps);
      out[(static_cast<size_t>(t) * heads + head) * vdim + j] =
          from_float<T>(((o * inv) * norm_w[j]) * (gj / (1.0f + expf(-gj))));
    }
  }
#pragma unroll
  for (int n = 0; n < NI; ++n) {
    const int i = ip + n * ip_count;
    if (owner && i < dim) st[static_cast<size_t>(i) * vdim + j] = s[n];
  }
}

// proj: [tokens, ld] of dtype, one row per token holding q (heads * dim elements from q_off), k (from
// k_off), v and the gate g (heads * vdim from v_off and g_off) and the decays' low-rank logits (rank
// elements from a_off).  a2: float [heads * dim, rank]; a2_bias: float [heads * dim]; inv_tau: 1 / tau.
// out: [tokens, heads * vdim] of dtype.  state: float [slots, heads, dim, vdim].  norm_w: float [vdim].
// The host guarantees row_slots < slots and row_start[rows] <= tokens.
extern "C" int pylon_gla_recurrent(void* out, const void* proj, int dtype, long long ld, int q_off, int k_off, int v_off,
                                   int g_off, int a_off, int rank, const float* a2, const float* a2_bias,
                                   float inv_tau, float* state, const float* norm_w, const int* row_start,
                                   const int* row_slots, int rows, int heads, int dim, int vdim, float eps,
                                   float q_scale, hipStream_t stream) {
  PYLON_REQUIRE(pylon_valid_dtype(dtype), "gla: unknown dtype");
  PYLON_REQUIRE(rows >= 0 && heads > 0 && dim > 0 && vdim > 0 && rank > 0, "gla: bad sizes");
  PYLON_REQUIRE(heads <= 65535, "gla: too many heads for one launch");
  PYLON_REQUIRE(vdim <= 1024 && dim <= 1024, "gla: heads of up to 1024 key and value elements, got %d and %d", dim, vdim);
  PYLON_REQUIRE(inv_tau > 0.f, "gla: tau must be positive");
  if (rows == 0) return 0;
  int ip_count = 256 / vdim;
  if (ip_count > dim) ip_count = dim;
  if (ip_count < 1 || (dim + ip_count - 1) / ip_count > 16) {  // a large head: more threads, fewer rows of S each
    ip_count = 1024 / vdim;
    if (ip_count > dim) ip_count = dim;
  }
  const int per = (dim + ip_count - 1) / ip_count;
  PYLON_REQUIRE(per <= 64, "gla: a head of %d x %d does not fit a workgroup's registers", dim, vdim);
  dim3 grid(rows, heads), block((vdim * ip_count + PYLON_WAVE - 1) / PYLON_WAVE * PYLON_WAVE);
  const size_t lds = sizeof(float) * (3 * dim + ip_count * vdim + 16);
#define GO(T, NI, THREADS)                                                                                         \
  hipLaunchKernelGGL((gla_recurrent_kernel<T, NI, THREADS>), grid, block, lds, stream, (T*)out, (const T*)proj, ld, \
                     q_off, k_off, v_off, g_off, a_off, rank, a2, a2_bias, inv_tau, state, norm_w, row_start,       \
                     row_slots, heads, dim, vdim, ip_count, eps, q_scale)
#define PICK(T)                                       \
  do {                                                \
    if (block.x <= 256) GO(T, 16, 256);               \
    else if (per <= 16) GO(T, 16, 1024);              \
    else GO(T, 64, 1024);                             \
  } while (0)
  if (dtype == PYLON_F32) PICK(float);
  else PICK(bf16_t);
#undef PICK
#undef GO
  PYLON_LAUNCHED("gla_recurrent");
}
