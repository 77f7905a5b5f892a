// Kernels of latent attention, in which only a small latent per token is cached and every head's
// keys and values are linear maps of it.  With q'_h = W_uk[h]^T q_h the score q_h . (W_uk[h] c)
// equals q'_h . c, and sum_j p_j W_uv[h] c_j equals W_uv[h] (sum_j p_j c_j): attention runs over
// the cached latents themselves (one key/value head, keys = values = c), between two small
// products per head.
//
// latent_prepare: from the fused down projection's float sums [tokens, q_rank + kv_rank + gates]
//   the normed query latent, the normed key/value latent into its cache slot, and sigmoid of the
//   gate logits.  Norms (root mean square, eps inside the root, times a weight) in float.
// head_project: out[t, h, :] = gate[t, h] * x[t, h, :] @ m[h] with m [heads, n_in, n_out]; a
//   workgroup keeps the inputs of a few tokens in LDS and walks 64 columns of m[h] once for all of
//   them, its four waves a quarter of n_in each; sums in float in one fixed order, whatever the batch.
//   The heads of x and of out may lie apart (parts of wider heads), and the gate may come as raw logits
//   of x's type, one per head or per element, whose sigmoid is taken here.
// head_project_rows: the same for few bfloat16 tokens on the matrix cores, from a matrix that lies output by output.
// gate_heads: x[t, h, :] *= gate[t, h] in place.
//
// Where a part of every key carries positions, the row of a token in the cache is [c | r]: the normed
// latent and one rotated key part r that all heads share; a query in that space is [q' | rotated part of
// q], so that the score is still one product of the two and the values are still the latent's elements.
// latent_rotate: from the projection's rows, c normed and r rotated into the token's cache slot, and the
//   rotated part of every head of q into the places it has in the query rows.
#include "common.h"

#define LP_THREADS 256

template <typename T>
__global__ void __launch_bounds__(LP_THREADS)
latent_prepare_kernel(T* __restrict__ q_latent, T* __restrict__ c_cache, float* __restrict__ gate_out,
                      const float* __restrict__ down, long long row_stride, const float* __restrict__ q_weight,
                      const float* __restrict__ c_weight, float eps, const int* __restrict__ slot_map, int q_rank,
                      int kv_rank, int n_gate, int store) {
  __shared__ float scratch[16];
  const int t = blockIdx.x, tid = threadIdx.x;
  const float* row = down + static_cast<size_t>(t) * row_stride;
  float sq = 0.f;
  for (int i = tid; i < q_rank; i += LP_THREADS) sq = fmaf(row[i], row[i], sq);
  const float inv_q = 1.0f / sqrtf(block_sum(sq, scratch) / static_cast<float>(q_rank > 0 ? q_rank : 1) + eps);
  for (int i = tid; i < q_rank; i += LP_THREADS)
    q_latent[static_cast<size_t>(t) * q_rank + i] = from_float<T>(row[i] * inv_q * q_weight[i]);
  if (store) {
    const float* c = row + q_rank;
    float sc = 0.f;
    for (int i = tid; i < kv_rank; i += LP_THREADS) sc = fmaf(c[i], c[i], sc);
    const float inv_c = 1.0f / sqrtf(block_sum(sc, scratch) / static_cast<float>(kv_rank) + eps);
    T* dst = c_cache + static_cast<size_t>(slot_map[t]) * kv_rank;
    for (int i = tid; i < kv_rank; i += LP_THREADS) dst[i] = from_float<T>(c[i] * inv_c * c_weight[i]);
  }
  const float* g = row + q_rank + kv_rank;
  for (int i = tid; i < n_gate; i += LP_THREADS)
    gate_out[static_cast<size_t>(t) * n_gate + i] = 1.0f / (1.0f + expf(-g[i]));
}

extern "C" int pylon_latent_prepare(void* q_latent, void* c_cache, float* gate_out, const float* down,
                                    long long row_stride, int dtype, const float* q_weight, const float* c_weight,
                                    float eps, const int* slot_map, int tokens, int q_rank, int kv_rank, int n_gate,
                                    int store, hipStream_t stream) {
  PYLON_REQUIRE(pylon_valid_dtype(dtype), "latent_prepare: unknown dtype");
  PYLON_REQUIRE(tokens >= 0 && q_rank > 0 && kv_rank > 0 && n_gate >= 0, "latent_prepare: sizes must be positive");
  PYLON_REQUIRE(row_stride >= static_cast<long long>(q_rank) + kv_rank + n_gate,
                "latent_prepare: rows hold fewer numbers than the latents and gates take");
  PYLON_REQUIRE(q_weight != nullptr && c_weight != nullptr, "latent_prepare: both norms have weights");
  PYLON_REQUIRE(!store || (c_cache != nullptr && slot_map != nullptr), "latent_prepare: storing needs cache and slots");
  PYLON_REQUIRE(n_gate == 0 || gate_out != nullptr, "latent_prepare: gates need a place");
  if (tokens == 0) return 0;
  if (dtype == PYLON_F32)
    hipLaunchKernelGGL((latent_prepare_kernel<float>), dim3(tokens), dim3(LP_THREADS), 0, stream, (float*)q_latent,
                       (float*)c_cache, gate_out, down, row_stride, q_weight, c_weight, eps, slot_map, q_rank,
                       kv_rank, n_gate, store);
  else
    hipLaunchKernelGGL((latent_prepare_kernel<bf16_t>), dim3(tokens), dim3(LP_THREADS), 0, stream,
                       (bf16_t*)q_latent, (bf16_t*)c_cache, gate_out, down, row_stride, q_weight, c_weight, eps,
                       slot_map, q_rank, kv_rank, n_gate, store);
  PYLON_LAUNCHED("latent_prepare");
}

template <typename T>
__global__ void __launch_bounds__(LP_THREADS)
latent_rotate_kernel(T* __restrict__ q_out, T* __restrict__ cache, const T* __restrict__ proj, long long ld, int q_off,
                     int heads, int dim, int rot, int c_off, int rank, const float* __restrict__ c_weight, float eps,
                     const float* __restrict__ inv_freq, float rot_scale, int interleaved,
                     const int* __restrict__ positions, const int* __restrict__ slot_map, int store) {
  extern __shared__ float turn[];  // [2][rot / 2]: cosines and sines of the token's angles, times rot_scale
  __shared__ float scratch[16];
  const int t = blockIdx.x, tid = threadIdx.x;
  const T* row = proj + static_cast<size_t>(t) * ld;
  const int half = rot / 2, width = rank + rot;
  if (inv_freq != nullptr) {
    const float pos = static_cast<float>(positions[t]);
    for (int i = tid; i < half; i += LP_THREADS) {
      float sn, cs;
      sincosf(pos * inv_freq[i], &sn, &cs);
      turn[i] = cs * rot_scale;
      turn[half + i] = sn * rot_scale;
    }
  }
  __syncthreads();
  // pair i of a part: neighbours (2i, 2i + 1), or halves (i, i + rot / 2)
  auto rotate = [&](const T* src, T* dst, int i) {
    const int a = interleaved ? 2 * i : i, b = interleaved ? 2 * i + 1 : i + half;
    const float u = to_float(src[a]), v = to_float(src[b]);
    float x = u, y = v;
    if (inv_freq != nullptr) {
      const float cs = turn[i], sn = turn[half + i];
      x = u * cs - v * sn;
      y = v * cs + u * sn;
    }
    dst[a] = from_float<T>(x);
    dst[b] = from_float<T>(y);
  };
  for (int e = tid; e < heads * half; e += LP_THREADS) {
    const int h = e / half, i = e - h * half;
    rotate(row + q_off + static_cast<size_t>(h) * (dim + rot) + dim,
           q_out + (static_cast<size_t>(t) * heads + h) * width + rank, i);
  }
  if (!store) return;
  const T* c = row + c_off;
  float sq = 0.f;
  for (int i = tid; i < rank; i += LP_THREADS) {
    const float v = to_float(c[i]);
    sq = fmaf(v, v, sq);
  }
  const float inv = 1.0f / sqrtf(block_sum(sq, scratch) / static_cast<float>(rank) + eps);
  T* dst = cache + static_cast<size_t>(slot_map[t]) * width;
  for (int i = tid; i < rank; i += LP_THREADS) dst[i] = from_float<T>(to_float(c[i]) * inv * c_weight[i]);
  for (int i = tid; i < half; i += LP_THREADS) rotate(c + rank, dst + rank, i);
}

// proj: [tokens, ld] of dtype holding, from q_off, the heads of q as [dim | rot] each, and from c_off the
// latent (rank elements) and behind it the shared rotated key part (rot elements).  q_out: [tokens, heads,
// rank + rot], of which only the last rot elements of every head are written.  cache: [slots, rank + rot].
// inv_freq: float [rot / 2], or null (the parts are copied as they are); rot_scale multiplies every cosine
// and sine.
extern "C" int pylon_latent_rotate(void* q_out, void* cache, const void* proj, int dtype, long long ld, int q_off,
                                   int heads, int dim, int rot, int c_off, int rank, const float* c_weight, float eps,
                                   const float* inv_freq, float rot_scale, int interleaved, const int* positions,
                                   const int* slot_map, int tokens, int store, hipStream_t stream) {
  PYLON_REQUIRE(pylon_valid_dtype(dtype), "latent_rotate: unknown dtype");
  PYLON_REQUIRE(tokens >= 0 && heads > 0 && dim > 0 && rot >= 0 && rot % 2 == 0 && rot <= 1024 && rank > 0,
                "latent_rotate: bad sizes");
  PYLON_REQUIRE(q_off >= 0 && c_off >= 0 && q_off + static_cast<long long>(heads) * (dim + rot) <= ld &&
                    c_off + static_cast<long long>(rank) + rot <= ld,
                "latent_rotate: q or the latent lie outside the projection's rows");
  PYLON_REQUIRE(inv_freq == nullptr || positions != nullptr, "latent_rotate: a rotation needs positions");
  PYLON_REQUIRE(!store || (cache != nullptr && slot_map != nullptr && c_weight != nullptr),
                "latent_rotate: storing needs cache, slots and the norm's weight");
  if (tokens == 0) return 0;
  const size_t lds = sizeof(float) * (rot > 0 ? rot : 2);
  if (dtype == PYLON_F32)
    hipLaunchKernelGGL((latent_rotate_kernel<float>), dim3(tokens), dim3(LP_THREADS), lds, stream, (float*)q_out,
                       (float*)cache, (const float*)proj, ld, q_off, heads, dim, rot, c_off, rank, c_weight, eps,
                       inv_freq, rot_scale, interleaved, positions, slot_map, store);
  else
    hipLaunchKernelGGL((latent_rotate_kernel<bf16_t>), dim3(tokens), dim3(LP_THREADS), lds, stream, (bf16_t*)q_out,
                       (bf16_t*)cache, (const bf16_t*)proj, ld, q_off, heads, dim, rot, c_off, rank, c_weight, eps,
                       inv_freq, rot_scale, interleaved, positions, slot_map, store);
  PYLON_LAUNCHED("latent_rotate");
}

// What multiplies an output of the per-head product: a float gate per (token, head), or the sigmoid of
// raw logits (per: outputs that share one, a head's or 1).
template <typename TX>
struct HeadGate {
  const float* heads;
  const TX* logits;
  long long logit_stride;
  int per;
  __device__ __forceinline__ float at(int t, int n_heads, int h, int n_out, int o) const {
    if (logits != nullptr)
      return 1.0f / (1.0f + expf(-to_float(logits[static_cast<size_t>(t) * logit_stride + (h * n_out + o) / per])));
    return heads != nullptr ? heads[static_cast<size_t>(t) * n_heads + h] : 1.f;
  }
};

#define HP_THREADS 256
#define HP_TOKENS 8
#define HP_COLS 64   // outputs of a workgroup
#define HP_SLICES 4  // the waves of a workgroup cut n_in between them

template <typename TX, typename TM>
__global__ void __launch_bounds__(HP_THREADS)
head_project_kernel(TX* __restrict__ out, long long out_stride, int out_hstride, const TX* __restrict__ x,
                    long long x_stride, int x_hstride, const TM* __restrict__ m, HeadGate<TX> gate, int tokens,
                    int heads, int n_in, int n_out) {
  extern __shared__ float xs[];  // [HP_TOKENS, n_in], then the slices' partial sums [HP_SLICES, HP_TOKENS, HP_COLS]
  float* partial = xs + HP_TOKENS * n_in;
  const int t0 = blockIdx.x * HP_TOKENS, h = blockIdx.y, tid = threadIdx.x;
  for (int i = tid; i < HP_TOKENS * n_in; i += HP_THREADS) {
    const int tt = i / n_in, k = i - tt * n_in;
    xs[i] = (t0 + tt < tokens) ? to_float(x[static_cast<size_t>(t0 + tt) * x_stride + static_cast<size_t>(h) * x_hstride + k])
                               : 0.f;
  }
  __syncthreads();
  const int slice = tid / HP_COLS, col = tid % HP_COLS;
  const int o = blockIdx.z * HP_COLS + col;
  const int per = (n_in + HP_SLICES - 1) / HP_SLICES;
  const int k0 = slice * per, k1 = k0 + per < n_in ? k0 + per : n_in;
  float acc[HP_TOKENS];
#pragma unroll
  for (int tt = 0; tt < HP_TOKENS; ++tt) acc[tt] = 0.f;
  if (o < n_out) {
    const TM* mh = m + static_cast<size_t>(h) * n_in * n_out + o;
#pragma unroll 8
    for (int k = k0; k < k1; ++k) {  // unrolled: eight loads of m in flight
      const float w = to_float(mh[static_cast<size_t>(k) * n_out]);
#pragma unroll
      for (int tt = 0; tt < HP_TOKENS; ++tt) acc[tt] = fmaf(xs[tt * n_in + k], w, acc[tt]);
    }
  }
#pragma unroll
  for (int tt = 0; tt < HP_TOKENS; ++tt) partial[(slice * HP_TOKENS + tt) * HP_COLS + col] = acc[tt];
  __syncthreads();
  // the slices' sums are added in their order, whatever the batch
  for (int i = tid; i < HP_TOKENS * HP_COLS; i += HP_THREADS) {
    const int tt = i / HP_COLS, c = i % HP_COLS;
    const int oc = blockIdx.z * HP_COLS + c;
    if (t0 + tt >= tokens || oc >= n_out) continue;
    float sum = partial[tt * HP_COLS + c];
#pragma unroll
    for (int sl = 1; sl < HP_SLICES; ++sl) sum += partial[(sl * HP_TOKENS + tt) * HP_COLS + c];
    const float g = gate.at(t0 + tt, heads, h, n_out, oc);
    out[static_cast<size_t>(t0 + tt) * out_stride + static_cast<size_t>(h) * out_hstride + oc] = from_float<TX>(sum * g);
  }
}

// The same product for bfloat16 matrices whose rows are whole 16-byte pieces: a lane reads eight
// neighbouring columns of a row of m[h] at once, the lanes of a row segment side by side, the groups of
// lanes of a workgroup every 16th row; their sums meet by shuffles inside a
// wave and through LDS between the four waves, always in the same order.
#define HW_COLS 128  // outputs of a workgroup

__global__ void __launch_bounds__(HP_THREADS)
head_project_wide_kernel(bf16_t* __restrict__ out, long long out_stride, int out_hstride, const bf16_t* __restrict__ x,
                         long long x_stride, int x_hstride, const bf16_t* __restrict__ m, HeadGate<bf16_t> gate,
                         int tokens, int heads, int n_in, int n_out) {
  constexpr int CG = HW_COLS / 8;              // lanes side by side on a row segment
  constexpr int KG = HP_THREADS / CG;       // rows of m[h] under way at once
  extern __shared__ float xs[];  // [HP_TOKENS, n_in], then the waves' partial sums [4, HP_TOKENS, HW_COLS]
  float* partial = xs + HP_TOKENS * n_in;
  const int t0 = blockIdx.x * HP_TOKENS, h = blockIdx.y, c0 = blockIdx.z * HW_COLS, tid = threadIdx.x;
  for (int i = tid; i < HP_TOKENS * n_in; i += HP_THREADS) {
    const int tt = i / n_in, k = i - tt * n_in;
    xs[i] = (t0 + tt < tokens) ? to_float(x[static_cast<size_t>(t0 + tt) * x_stride + static_cast<size_t>(h) * x_hstride + k])
                               : 0.f;
  }
  __syncthreads();
  const int lane = tid & (PYLON_WAVE - 1), wave = tid / PYLON_WAVE;
  const int cg = tid % CG, kg = tid / CG;
  float acc[HP_TOKENS][8];
#pragma unroll
  for (int tt = 0; tt < HP_TOKENS; ++tt)
#pragma unroll
    for (int c = 0; c < 8; ++c) acc[tt][c] = 0.f;
  const int col = c0 + 8 * cg;
  if (col < n_out) {  // n_out is a multiple of 8: the lane's eight columns are all inside
    const bf16_t* mh = m + static_cast<size_t>(h) * n_in * n_out + col;
#pragma unroll 4
    for (int k = kg; k < n_in; k += KG) {
      const uint4 raw = *reinterpret_cast<const uint4*>(mh + static_cast<size_t>(k) * n_out);
      const uint32_t words[4] = {raw.x, raw.y, raw.z, raw.w};
      float wv[8];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        wv[2 * j] = __uint_as_float(words[j] << 16);
        wv[2 * j + 1] = __uint_as_float(words[j] & 0xffff0000u);
      }
#pragma unroll
      for (int tt = 0; tt < HP_TOKENS; ++tt) {
        const float xv = xs[tt * n_in + k];
#pragma unroll
        for (int c = 0; c < 8; ++c) acc[tt][c] = fmaf(xv, wv[c], acc[tt][c]);
      }
    }
  }
#pragma unroll
  for (int tt = 0; tt < HP_TOKENS; ++tt)
#pragma unroll
    for (int c = 0; c < 8; ++c) {
      float v = acc[tt][c];
#pragma unroll
      for (int off = CG; off < PYLON_WAVE; off <<= 1) v += __shfl_xor(v, off, PYLON_WAVE);
      if (lane < CG) partial[(wave * HP_TOKENS + tt) * HW_COLS + 8 * cg + c] = v;
    }
  __syncthreads();
  for (int i = tid; i < HP_TOKENS * HW_COLS; i += HP_THREADS) {
    const int tt = i / HW_COLS, c = i % HW_COLS;
    if (t0 + tt >= tokens || c0 + c >= n_out) continue;
    float sum = partial[tt * HW_COLS + c];
#pragma unroll
    for (int wv = 1; wv < 4; ++wv) sum += partial[(wv * HP_TOKENS + tt) * HW_COLS + c];
    const float g = gate.at(t0 + tt, heads, h, n_out, c0 + c);
    out[static_cast<size_t>(t0 + tt) * out_stride + static_cast<size_t>(h) * out_hstride + c0 + c] = from_float<bf16_t>(sum * g);
  }
}

// The same product on the matrix cores for few tokens, from a matrix that lies output by output, mt[h] =
// [n_out, n_in]: a wave owns 16 outputs of one head (the rows of the instruction) and all tokens (its
// columns); every load of a few slabs of 32 inputs is sent for before the first product.  No LDS, no barrier;
// the sums run along n_in in one order, whatever the batch.
typedef __bf16 hp_bf16x8 __attribute__((ext_vector_type(8)));
typedef float hp_floatx4 __attribute__((ext_vector_type(4)));
typedef unsigned int hp_u32x4 __attribute__((ext_vector_type(4)));
#define HM_SLABS 8  // slabs under way together
#define HM_OUTPUTS 64  // outputs of a workgroup

template <int TT>
__global__ void __launch_bounds__(HP_THREADS)
head_project_rows_kernel(bf16_t* __restrict__ out, long long out_stride, int out_hstride, const bf16_t* __restrict__ x,
                         long long x_stride, int x_hstride, const bf16_t* __restrict__ mt, HeadGate<bf16_t> gate, int tokens,
                         int heads, int n_in, int n_out) {
  constexpr int SLABS = TT > 2 ? HM_SLABS / 2 : HM_SLABS;
  const int lane = threadIdx.x & (PYLON_WAVE - 1), wave = threadIdx.x / PYLON_WAVE;
  const int col = lane & 15, grp = lane >> 4;
  const int h = blockIdx.x, o0 = blockIdx.y * HM_OUTPUTS + wave * 16;
  if (o0 >= n_out) return;
  const bf16_t* mrow = mt + (static_cast<size_t>(h) * n_out + (o0 + col < n_out ? o0 + col : n_out - 1)) * n_in;
  const bf16_t* xrow[TT];
  hp_floatx4 acc[TT];
#pragma unroll
  for (int t = 0; t < TT; ++t) {
    const int tok = t * 16 + col;
    xrow[t] = x + static_cast<size_t>(tok < tokens ? tok : tokens - 1) * x_stride + static_cast<size_t>(h) * x_hstride;
    acc[t] = hp_floatx4{0.f, 0.f, 0.f, 0.f};
  }
  for (int k0 = 0; k0 < n_in; k0 += 32 * SLABS) {
    hp_u32x4 a[SLABS], b[SLABS][TT];
#pragma unroll
    for (int s = 0; s < SLABS; ++s) {
      const int k = k0 + s * 32 + grp * 8;
      const bool in = k < n_in;  // n_in is a multiple of 8: the lane's eight inputs are all inside
      a[s] = hp_u32x4{0u, 0u, 0u, 0u};
      if (in) a[s] = *reinterpret_cast<const hp_u32x4*>(mrow + k);
#pragma unroll
      for (int t = 0; t < TT; ++t) {
        b[s][t] = hp_u32x4{0u, 0u, 0u, 0u};
        if (in) b[s][t] = *reinterpret_cast<const hp_u32x4*>(xrow[t] + k);
      }
    }
#pragma unroll
    for (int s = 0; s < SLABS; ++s)
#pragma unroll
      for (int t = 0; t < TT; ++t)
        acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(hp_bf16x8, a[s]),
                                                         __builtin_bit_cast(hp_bf16x8, b[s][t]), acc[t], 0, 0, 0);
  }
#pragma unroll
  for (int t = 0; t < TT; ++t) {
    const int tok = t * 16 + col;
    if (tok >= tokens) continue;
    bf16_t* dst = out + static_cast<size_t>(tok) * out_stride + static_cast<size_t>(h) * out_hstride;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int o = o0 + 4 * grp + i;
      if (o < n_out) dst[o] = from_float<bf16_t>(acc[t][i] * gate.at(tok, heads, h, n_out, o));
    }
  }
}

// x, out and the gates as for pylon_head_project, at most 64 tokens; mt: bf16 [heads, n_out, n_in], n_in a
// multiple of 8, mt and the rows of every head of x 16-byte aligned.
extern "C" int pylon_head_project_rows(void* out, long long out_stride, int out_hstride, const void* x, long long x_stride,
                                       int x_hstride, const void* mt, const float* gate, const void* gate_logits,
                                       long long gate_stride, int gate_per, int tokens, int heads, int n_in, int n_out,
                                       hipStream_t stream) {
  PYLON_REQUIRE(tokens >= 0 && tokens <= 64 && heads > 0 && n_in > 0 && n_out > 0, "head_project_rows: bad sizes");
  PYLON_REQUIRE(n_in % 8 == 0 && x_stride % 8 == 0 && x_hstride % 8 == 0 &&
                    ((reinterpret_cast<uintptr_t>(x) | reinterpret_cast<uintptr_t>(mt)) & 15) == 0,
                "head_project_rows: inputs must be whole 16-byte pieces");
  PYLON_REQUIRE(x_hstride >= n_in && x_stride >= static_cast<long long>(heads - 1) * x_hstride + n_in,
                "head_project_rows: rows of x overlap");
  PYLON_REQUIRE(out_hstride >= n_out && out_stride >= static_cast<long long>(heads - 1) * out_hstride + n_out,
                "head_project_rows: rows of the result overlap");
  PYLON_REQUIRE(gate == nullptr || gate_logits == nullptr, "head_project_rows: gates or their logits, not both");
  PYLON_REQUIRE(gate_logits == nullptr || (gate_per >= 1 && (static_cast<long long>(heads) * n_out) % gate_per == 0 &&
                                           gate_stride >= static_cast<long long>(heads) * n_out / gate_per),
                "head_project_rows: the gates' logits do not match the outputs");
  if (tokens == 0) return 0;
  const dim3 grid(heads, (n_out + HM_OUTPUTS - 1) / HM_OUTPUTS);
  PYLON_REQUIRE(grid.y <= 65535, "head_project_rows: too many outputs per head for one launch");
  const HeadGate<bf16_t> gates = {gate, (const bf16_t*)gate_logits, gate_stride, gate_per};
#define GO(TT)                                                                                                      \
  hipLaunchKernelGGL(head_project_rows_kernel<TT>, grid, dim3(HP_THREADS), 0, stream, (bf16_t*)out, out_stride,     \
                     out_hstride, (const bf16_t*)x, x_stride, x_hstride, (const bf16_t*)mt, gates, tokens, heads, n_in, n_out)
  if (tokens <= 16) GO(1);
  else if (tokens <= 32) GO(2);
  else GO(4);
#undef GO
  PYLON_LAUNCHED("head_project_rows");
}

// x: [tokens, heads, n_in], rows x_stride and heads x_hstride elements apart; m: [heads, n_in, n_out]; gate:
// null or float [tokens, heads]; gate_logits: null (and then at most one of the two) or, of x's type, [tokens,
// heads * n_out / gate_per], rows gate_stride apart; out: [tokens, heads, n_out] of x's type, rows out_stride
// and heads out_hstride apart.  m may be float while x is bfloat16.
extern "C" int pylon_head_project(void* out, long long out_stride, int out_hstride, const void* x, int x_dtype,
                                  long long x_stride, int x_hstride, const void* m, int m_dtype, const float* gate,
                                  const void* gate_logits, long long gate_stride, int gate_per, int tokens, int heads,
                                  int n_in, int n_out, hipStream_t stream) {
  PYLON_REQUIRE(pylon_valid_dtype(x_dtype) && pylon_valid_dtype(m_dtype), "head_project: unknown dtype");
  PYLON_REQUIRE(tokens >= 0 && heads > 0 && n_in > 0 && n_out > 0, "head_project: sizes must be positive");
  PYLON_REQUIRE(heads <= 65535, "head_project: too many heads for one launch");
  PYLON_REQUIRE(x_hstride >= n_in && x_stride >= static_cast<long long>(heads - 1) * x_hstride + n_in,
                "head_project: rows of x overlap");
  PYLON_REQUIRE(out_hstride >= n_out && out_stride >= static_cast<long long>(heads - 1) * out_hstride + n_out,
                "head_project: rows of the result overlap");
  PYLON_REQUIRE(gate == nullptr || gate_logits == nullptr, "head_project: gates or their logits, not both");
  PYLON_REQUIRE(gate_logits == nullptr || (gate_per >= 1 && (static_cast<long long>(heads) * n_out) % gate_per == 0 &&
                                           gate_stride >= static_cast<long long>(heads) * n_out / gate_per),
                "head_project: the gates' logits do not match the outputs");
  const size_t lds = sizeof(float) * (HP_TOKENS * n_in + HP_SLICES * HP_TOKENS * HP_COLS);
  PYLON_REQUIRE(lds <= 64 * 1024, "head_project: %d inputs per head do not fit LDS", n_in);
  PYLON_REQUIRE(!(x_dtype == PYLON_F32 && m_dtype == PYLON_BF16), "head_project: float inputs take a float matrix");
  if (tokens == 0) return 0;
  if (x_dtype == PYLON_BF16 && m_dtype == PYLON_BF16 && n_out % 8 == 0 && reinterpret_cast<uintptr_t>(m) % 16 == 0) {
    const size_t wide_lds = sizeof(float) * (HP_TOKENS * n_in + 4 * HP_TOKENS * HW_COLS);
    const int zw = (n_out + HW_COLS - 1) / HW_COLS;
    if (wide_lds <= 64 * 1024 && zw <= 65535) {
      hipLaunchKernelGGL(head_project_wide_kernel, dim3((tokens + HP_TOKENS - 1) / HP_TOKENS, heads, zw),
                         dim3(HP_THREADS), wide_lds, stream, (bf16_t*)out, out_stride, out_hstride, (const bf16_t*)x,
                         x_stride, x_hstride, (const bf16_t*)m,
                         (HeadGate<bf16_t>{gate, (const bf16_t*)gate_logits, gate_stride, gate_per}), tokens, heads, n_in,
                         n_out);
      PYLON_LAUNCHED("head_project");
    }
  }
  const int zs = (n_out + HP_COLS - 1) / HP_COLS;
  PYLON_REQUIRE(zs <= 65535, "head_project: too many outputs per head for one launch");
  dim3 grid((tokens + HP_TOKENS - 1) / HP_TOKENS, heads, zs), block(HP_THREADS);
#define GO(TX, TM)                                                                                              \
  hipLaunchKernelGGL((head_project_kernel<TX, TM>), grid, block, lds, stream, (TX*)out, out_stride, out_hstride, \
                     (const TX*)x, x_stride, x_hstride, (const TM*)m,                                           \
                     (HeadGate<TX>{gate, (const TX*)gate_logits, gate_stride, gate_per}), tokens, heads, n_in, n_out)
  if (x_dtype == PYLON_F32) GO(float, float);
  else if (m_dtype == PYLON_F32) GO(bf16_t, float);
  else GO(bf16_t, bf16_t);
#undef GO
  PYLON_LAUNCHED("head_project");
}

template <typename T>
__global__ void gate_heads_kernel(T* __restrict__ x, const float* __restrict__ gate, long long total, int n_out) {
  const long long i = static_cast<long long>(blockIdx.x) * blockDim.x + threadIdx.x;
  if (i < total) x[i] = from_float<T>(to_float(x[i]) * gate[i / n_out]);
}

// x: [tokens * heads, n_out] contiguous, multiplied in place by gate[tokens * heads].
extern "C" int pylon_gate_heads(void* x, int dtype, const float* gate, long long rows, int n_out,
                                hipStream_t stream) {
  PYLON_REQUIRE(pylon_valid_dtype(dtype), "gate_heads: unknown dtype");
  PYLON_REQUIRE(rows >= 0 && n_out > 0 && gate != nullptr, "gate_heads: bad sizes");
  const long long total = rows * n_out;
  if (total == 0) return 0;
  PYLON_REQUIRE((total + 255) / 256 < (1ll << 31), "gate_heads: too many elements for one launch");
  dim3 grid((unsigned)((total + 255) / 256)), block(256);
  if (dtype == PYLON_F32)
    hipLaunchKernelGGL((gate_heads_kernel<float>), grid, block, 0, stream, (float*)x, gate, total, n_out);
  else
    hipLaunchKernelGGL((gate_heads_kernel<bf16_t>), grid, block, 0, stream, (bf16_t*)x, gate, total, n_out);
  PYLON_LAUNCHED("gate_heads");
}
