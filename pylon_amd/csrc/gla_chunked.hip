// Gated linear attention of bfloat16 prompt portions on the matrix cores, sixteen tokens at a time.  For the
// tokens 0..n-1 of such a step, with S the state before it and b_t[d] = sum_{s <= t} log2(alpha_s[d]) the
// decays' running logarithms inside the step:
//
//   o_i = sum_d q_i[d] 2^(b_i[d]) S[d, :] + sum_{j <= i} A_ij v_j,   A_ij = sum_d q_i[d] k_j[d] 2^(b_i[d] - b_j[d])
//   S' = diag(2^(b_(n-1))) S + sum_j (k_j 2^(b_(n-1) - b_j)) v_j^T
//
// (q scaled), then out_i = o_i / rms(o_i) * w * silu(g_i) as in the recurrent form.  To be products of
// matrices, both sums split their powers at a reference r[d], q'_i = q_i 2^(b_i - r), k'_j = k_j 2^(r - b_j):
// A = Q' K'^T below its diagonal, S^T q'_i with S's rows times 2^r, and S' from K'^T V with rows times
// 2^(b_(n-1) - r).  r is b at the step's middle, so that no power leaves +-64 as long as a channel keeps
// more than 2^-64 of what it held sixteen tokens ago; for a channel that forgets faster, q' takes r = 0
// and k' takes r = b_(n-1) (no power above one): its share of A then vanishes from the matrix product and is
// added exactly, pair by pair, on the vector unit.
//
// One workgroup of four waves per (row of the step, head) walks the row.  The state stays in float
// accumulators, every wave owning the columns (value elements) of its tiles.  Float operands (q', k', the
// state, A) enter the products as two bfloat16 terms, x = hi + lo, products of two such operands as hi*hi +
// hi*lo + lo*hi; v is the projection's bfloat16 as it is.  Outputs are computed transposed (rows: value
// elements, columns: tokens), so that a token's norm is a sum within its column's lanes; k' and v are kept
// row by row and read across tokens by the transposing LDS read.
//
// Rows too few to fill the chip that way are cut into chunks of 64 tokens with a workgroup each, in three
// launches: what every chunk adds to the state and how much it forgets, a scan over the chunks, every
// chunk's outputs from the state before it.
#include "common.h"
#include "gla.h"

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float floatx4 __attribute__((ext_vector_type(4)));
typedef short s16x4 __attribute__((ext_vector_type(4)));
typedef unsigned int u32x4 __attribute__((ext_vector_type(4)));
typedef unsigned int u32x2 __attribute__((ext_vector_type(2)));

#define GC_STEP 16
#define GC_CHUNK 64      // tokens of a chunk with a workgroup of its own (a whole number of steps)
#define GC_RANGE 64.0f   // how far (as a power of two) a channel may forget inside a step and stay in the products
#define GC_LDS(T) __attribute__((address_space(3))) T
#define GC_MFMA32(a, b, c) \
  __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0, 0)
#define GC_MFMA16(a, b, c) __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(a, b, c, 0, 0, 0)

// Upper halves of two floats side by side (a bfloat16 pair, truncated), and of what is left.
__device__ __forceinline__ void gc_split(float a, float b, uint32_t& hi, uint32_t& lo) {
  const uint32_t ua = __float_as_uint(a), ub = __float_as_uint(b);
  hi = __builtin_amdgcn_perm(ub, ua, 0x07060302u);
  const float ra = a - __uint_as_float(ua & 0xffff0000u), rb = b - __uint_as_float(ub & 0xffff0000u);
  lo = __builtin_amdgcn_perm(__float_as_uint(rb), __float_as_uint(ra), 0x07060302u);
}

// b_t of every token and key channel: the running sum of log2 decays inside its step.  One thread a
// channel, one workgroup 256 channels of one step.
#define GD_RANK 16  // elements of a row of a2 held in registers at a time
__global__ __launch_bounds__(256) void gla_decay_kernel(float* __restrict__ b, const bf16_t* __restrict__ proj, long long ld,
                                                        int a_off, int rank, const float* __restrict__ a2,
                                                        const float* __restrict__ a2_bias, float inv_tau,
                                                        const int* __restrict__ row_start, int channels) {
  extern __shared__ __attribute__((aligned(16))) float low[];  // [GC_STEP][rank rounded up to GD_RANK], zeros behind the rank
  const int row = blockIdx.y, padded = (rank + GD_RANK - 1) / GD_RANK * GD_RANK;
  const int t0 = row_start[row] + blockIdx.x * GC_STEP, end = row_start[row + 1];
  if (t0 >= end) return;
  const int n = end - t0 < GC_STEP ? end - t0 : GC_STEP;
  for (int i = threadIdx.x; i < GC_STEP * padded; i += 256) {
    const int t = i / padded, r = i - t * padded;
    low[i] = (t < n && r < rank) ? to_float(proj[static_cast<size_t>(t0 + t) * ld + a_off + r]) : 0.f;
  }
  __syncthreads();
  const int c = blockIdx.z * 256 + threadIdx.x;
  if (c >= channels) return;
  float z[GC_STEP];
#pragma unroll
  for (int t = 0; t < GC_STEP; ++t) z[t] = 0.f;
  const float* row_a2 = a2 + static_cast<size_t>(c) * rank;
  for (int r0 = 0; r0 < rank; r0 += GD_RANK) {
    float w[GD_RANK];
#pragma unroll
    for (int r = 0; r < GD_RANK; ++r) w[r] = r0 + r < rank ? row_a2[r0 + r] : 0.f;
#pragma unroll
    for (int t = 0; t < GC_STEP; ++t)
#pragma unroll
      for (int r = 0; r < GD_RANK; r += 4) {
        const float4 x = *reinterpret_cast<const float4*>(low + t * padded + r0 + r);
        z[t] = fmaf(x.x, w[r], z[t]);
        z[t] = fmaf(x.y, w[r + 1], z[t]);
        z[t] = fmaf(x.z, w[r + 2], z[t]);
        z[t] = fmaf(x.w, w[r + 3], z[t]);
      }
  }
  const float bias = a2_bias[c];
  float sum = 0.f;
#pragma unroll
  for (int t = 0; t < GC_STEP; ++t) {
    if (t >= n) break;
    sum += gla_log_sigmoid(z[t] + bias) * inv_tau * 1.44269504088896340736f;
    b[static_cast<size_t>(t0 + t) * channels + c] = sum;
  }
}

// KS: slabs of 32 key elements (dim = 32 KS); NVW: tiles of 16 value elements per wave (vdim <= 64 NVW).
// MODE 0: the whole row; MODE 1: what one chunk adds to a state of zero, into chunk_state, and the logarithm
// of how much of a state it leaves, into chunk_log; MODE 2: one chunk's outputs from the state in chunk_state.
template <int KS, int NVW, int MODE>
__global__ __launch_bounds__(256) void gla_chunked_kernel(
    bf16_t* __restrict__ out, const bf16_t* __restrict__ proj, long long ld, int q_off, int k_off, int v_off, int g_off,
    const float* __restrict__ b, float* state, const float* __restrict__ norm_w, const int* __restrict__ row_start,
    const int* __restrict__ row_slots, int heads, int vdim, float eps, float q_scale, float* __restrict__ chunk_state,
    float* __restrict__ chunk_log, int max_chunks) {
  constexpr int dim = 32 * KS, ND = 2 * KS, QSTR = dim + 8;
  constexpr int QKI = (GC_STEP * dim / 8 + 255) / 256;  // pieces of eight elements of q and k a thread stages
  constexpr int VI = (GC_STEP * NVW * 8 + 255) / 256;
  extern __shared__ __attribute__((aligned(16))) uint16_t gc_lds[];
  uint16_t* q_hi = gc_lds;                       // [16][QSTR]: q', then k', as two terms each
  uint16_t* q_lo = q_hi + GC_STEP * QSTR;
  uint16_t* k_hi = q_lo + GC_STEP * QSTR;
  uint16_t* k_lo = k_hi + GC_STEP * QSTR;
  const int vstr = 64 * NVW + 8;
  uint16_t* v_rows = k_lo + GC_STEP * QSTR;      // [16][vstr]
  float* before = reinterpret_cast<float*>(v_rows + GC_STEP * vstr);  // [dim]: 2^(q's reference)
  float* keep = before + dim;                    // [dim]: 2^b_(n-1)
  float* after = keep + dim;                     // [dim]: 2^(b_(n-1) - k's reference)
  float* red = after + dim;                      // [4][16]
  float* exact = red + 64;                       // [16][17]: A's share of the channels that forget fast
  __shared__ unsigned long long fast[4];         // which channels those are

  const int row = blockIdx.x, head = blockIdx.y;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int col = lane & 15, grp = lane >> 4;
  const int row_begin = row_start[row], row_end = row_start[row + 1];
  const int begin = MODE == 0 ? row_begin : row_begin + static_cast<int>(blockIdx.z) * GC_CHUNK;
  const int end = MODE == 0 ? row_end : (begin + GC_CHUNK < row_end ? begin + GC_CHUNK : row_end);
  if (begin >= end) return;
  const size_t chunk_at = (static_cast<size_t>(row) * heads + head) * max_chunks + blockIdx.z;
  float* st = MODE != 0 ? chunk_state + chunk_at * dim * vdim
                        : state + (static_cast<size_t>(row_slots[row]) * heads + head) * dim * vdim;
  const int channels = heads * dim;
  const float* b_head = b + head * dim;
  const int n_vt = (vdim + 15) / 16;
  const bool wide = ld % 8 == 0 && q_off % 8 == 0 && k_off % 8 == 0;  // 16-byte loads of q and k, and of v
  const bool wide_v = wide && vdim % 8 == 0 && v_off % 8 == 0;

  // A step travels global -> registers -> LDS; the registers of the next are filled while this one is computed.
  u32x4 q_raw[QKI], k_raw[QKI], v_raw[VI];
  float b_own[QKI][8], b_mid[QKI][8], b_end[QKI][8];
  auto load8 = [](float (&dst)[8], const float* src) {
    const float4 x = reinterpret_cast<const float4*>(src)[0], y = reinterpret_cast<const float4*>(src)[1];
    dst[0] = x.x; dst[1] = x.y; dst[2] = x.z; dst[3] = x.w;
    dst[4] = y.x; dst[5] = y.y; dst[6] = y.z; dst[7] = y.w;
  };
  auto fetch = [&](int t0, int n) {
    const int mid = n - 1 < 7 ? n - 1 : 7;
#pragma unroll
    for (int it = 0; it < QKI; ++it) {
      const int idx = tid + it * 256;
      const int tok = idx / (dim / 8), d = (idx - tok * (dim / 8)) * 8;
      q_raw[it] = u32x4{0u, 0u, 0u, 0u};
      k_raw[it] = u32x4{0u, 0u, 0u, 0u};
      if (idx < GC_STEP * dim / 8) {
        const int t = t0 + (tok < n ? tok : n - 1);
        if (tok < n) {
          const bf16_t* src = proj + static_cast<size_t>(t) * ld + head * dim + d;
          if (wide) {
            if (MODE != 1) q_raw[it] = *reinterpret_cast<const u32x4*>(src + q_off);
            k_raw[it] = *reinterpret_cast<const u32x4*>(src + k_off);
          } else {
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              if (MODE != 1) q_raw[it][e] = src[q_off + 2 * e].bits | (static_cast<uint32_t>(src[q_off + 2 * e + 1].bits) << 16);
              k_raw[it][e] = src[k_off + 2 * e].bits | (static_cast<uint32_t>(src[k_off + 2 * e + 1].bits) << 16);
            }
          }
        }
        load8(b_own[it], b_head + static_cast<size_t>(t) * channels + d);
        load8(b_mid[it], b_head + static_cast<size_t>(t0 + mid) * channels + d);
        load8(b_end[it], b_head + static_cast<size_t>(t0 + n - 1) * channels + d);
      }
    }
    if (wide_v) {
#pragma unroll
      for (int it = 0; it < VI; ++it) {
        const int idx = tid + it * 256;
        const int tok = idx / (8 * NVW), e = (idx - tok * (8 * NVW)) * 8;
        v_raw[it] = u32x4{0u, 0u, 0u, 0u};
        if (idx < GC_STEP * 8 * NVW && tok < n && e < vdim)
          v_raw[it] = *reinterpret_cast<const u32x4*>(proj + static_cast<size_t>(t0 + tok) * ld + v_off + head * vdim + e);
      }
    }
  };

  // S[d tile][own value tile]: column = value element, rows = key elements 4 grp + i
  floatx4 s[ND][NVW];
#pragma unroll
  for (int n = 0; n < NVW; ++n) {
    const int e = (wave + 4 * n) * 16 + col;
#pragma unroll
    for (int dt = 0; dt < ND; ++dt)
#pragma unroll
      for (int i = 0; i < 4; ++i)
        s[dt][n][i] = (MODE != 1 && e < vdim) ? st[static_cast<size_t>(dt * 16 + 4 * grp + i) * vdim + e] : 0.f;
  }
  float forgotten = 0.f;  // MODE 1: thread d's sum of b_(n-1) over the chunk's steps
  fetch(begin, end - begin < GC_STEP ? end - begin : GC_STEP);

  for (int t0 = begin; t0 < end; t0 += GC_STEP) {
    const int n_tok = end - t0 < GC_STEP ? end - t0 : GC_STEP;
    // ---- stage q', k' and v; the channels' powers
#pragma unroll
    for (int it = 0; it < QKI; ++it) {
      const int idx = tid + it * 256;
      if (idx >= GC_STEP * dim / 8) break;
      const int tok = idx / (dim / 8), d = (idx - tok * (dim / 8)) * 8;
      u32x4 qh, ql, kh, kl;
#pragma unroll
      for (int e = 0; e < 8; e += 2) {
        float qv[2], kv[2];
#pragma unroll
        for (int u = 0; u < 2; ++u) {
          const bool quick = b_end[it][e + u] < -GC_RANGE;
          const float rq = quick ? 0.f : b_mid[it][e + u], rk = quick ? b_end[it][e + u] : b_mid[it][e + u];
          const uint32_t qw = q_raw[it][e >> 1], kw = k_raw[it][e >> 1];
          const float qx = __uint_as_float(u ? (qw & 0xffff0000u) : (qw << 16));
          const float kx = __uint_as_float(u ? (kw & 0xffff0000u) : (kw << 16));
          qv[u] = MODE == 1 ? 0.f : qx * q_scale * __builtin_amdgcn_exp2f(b_own[it][e + u] - rq);
          kv[u] = kx * __builtin_amdgcn_exp2f(rk - b_own[it][e + u]);
        }
        uint32_t h, l;
        if (MODE != 1) {
          gc_split(qv[0], qv[1], h, l);
          qh[e >> 1] = h;
          ql[e >> 1] = l;
        }
        gc_split(kv[0], kv[1], h, l);
        kh[e >> 1] = h;
        kl[e >> 1] = l;
      }
      if (MODE != 1) {
        *reinterpret_cast<u32x4*>(q_hi + tok * QSTR + d) = qh;
        *reinterpret_cast<u32x4*>(q_lo + tok * QSTR + d) = ql;
      }
      *reinterpret_cast<u32x4*>(k_hi + tok * QSTR + d) = kh;
      *reinterpret_cast<u32x4*>(k_lo + tok * QSTR + d) = kl;
    }
    if (wide_v) {
#pragma unroll
      for (int it = 0; it < VI; ++it) {
        const int idx = tid + it * 256;
        if (idx >= GC_STEP * 8 * NVW) break;
        const int tok = idx / (8 * NVW), e = (idx - tok * (8 * NVW)) * 8;
        *reinterpret_cast<u32x4*>(v_rows + tok * vstr + e) = v_raw[it];
      }
    } else {
      for (int idx = tid; idx < GC_STEP * 64 * NVW; idx += 256) {
        const int tok = idx / (64 * NVW), e = idx - tok * (64 * NVW);
        v_rows[tok * vstr + e] =
            tok < n_tok && e < vdim ? proj[static_cast<size_t>(t0 + tok) * ld + v_off + head * vdim + e].bits : 0;
      }
    }
    {
      bool quick = false;
      if (tid < dim) {
        const int mid = n_tok - 1 < 7 ? n_tok - 1 : 7;
        const float bm = b_head[static_cast<size_t>(t0 + mid) * channels + tid];
        const float bn = b_head[static_cast<size_t>(t0 + n_tok - 1) * channels + tid];
        quick = bn < -GC_RANGE;
        before[tid] = __builtin_amdgcn_exp2f(quick ? 0.f : bm);
        keep[tid] = __builtin_amdgcn_exp2f(bn);
        after[tid] = __builtin_amdgcn_exp2f(quick ? 0.f : bn - bm);
        forgotten += bn;
      }
      const unsigned long long which = __ballot(quick);
      if (lane == 0) fast[wave] = which;
    }
    __syncthreads();
    if (t0 + GC_STEP < end) fetch(t0 + GC_STEP, end - t0 - GC_STEP < GC_STEP ? end - t0 - GC_STEP : GC_STEP);

    floatx4 o[NVW];
    if (MODE != 1) {
      const bool any_fast = (fast[0] | fast[1] | fast[2] | fast[3]) != 0;  // the same for the whole workgroup
      if (any_fast) {
        const int i = tid >> 4, j = tid & 15;
        float acc = 0.f;
        if (j <= i && i < n_tok) {
          const bf16_t* qi = proj + static_cast<size_t>(t0 + i) * ld + q_off + head * dim;
          const bf16_t* kj = proj + static_cast<size_t>(t0 + j) * ld + k_off + head * dim;
          const float* bi = b_head + static_cast<size_t>(t0 + i) * channels;
          const float* bj = b_head + static_cast<size_t>(t0 + j) * channels;
          for (int w = 0; w < 4; ++w) {
            for (unsigned long long left = fast[w]; left != 0; left &= left - 1) {
              const int d = w * 64 + __ffsll(static_cast<long long>(left)) - 1;
              acc = fmaf(to_float(qi[d]) * q_scale * __builtin_amdgcn_exp2f(bi[d] - bj[d]), to_float(kj[d]), acc);
            }
          }
        }
        exact[i * 17 + j] = acc;
        __syncthreads();
      }
      // ---- A, transposed: rows = tokens j = 4 grp + r, column = token i = col
      floatx4 a = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        const int at = col * QSTR + ks * 32 + grp * 8;
        const u32x4 kh = *reinterpret_cast<const u32x4*>(k_hi + at), kl = *reinterpret_cast<const u32x4*>(k_lo + at);
        const u32x4 qh = *reinterpret_cast<const u32x4*>(q_hi + at), ql = *reinterpret_cast<const u32x4*>(q_lo + at);
        a = GC_MFMA32(kh, qh, a);
        a = GC_MFMA32(kh, ql, a);
        a = GC_MFMA32(kl, qh, a);
      }
      float p[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int j = 4 * grp + r;
        p[r] = j <= col ? a[r] : 0.f;  // above the diagonal the split powers mean nothing
        if (any_fast && j <= col) p[r] += exact[col * 17 + j];
      }
      uint32_t ph[2], pl[2];
      gc_split(p[0], p[1], ph[0], pl[0]);
      gc_split(p[2], p[3], ph[1], pl[1]);
      const s16x4 p_hi = __builtin_bit_cast(s16x4, u32x2{ph[0], ph[1]}), p_lo = __builtin_bit_cast(s16x4, u32x2{pl[0], pl[1]});

      // ---- outputs, transposed: rows = value elements of the wave's tiles, columns = tokens
#pragma unroll
      for (int n = 0; n < NVW; ++n) {
        o[n] = floatx4{0.f, 0.f, 0.f, 0.f};
        const int vt = wave + 4 * n;
        if (vt >= n_vt) continue;
        // the state's share: S's rows times 2^r, the key elements of a slab in the order the accumulators hold
        // them (4 grp + i, then 16 + 4 grp + i)
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
          u32x4 sh, sl;
#pragma unroll
          for (int half = 0; half < 2; ++half) {
            const float4 f = *reinterpret_cast<const float4*>(before + ks * 32 + half * 16 + 4 * grp);
            const floatx4& x = s[2 * ks + half][n];
            uint32_t h, l;
            gc_split(x[0] * f.x, x[1] * f.y, h, l);
            sh[2 * half] = h;
            sl[2 * half] = l;
            gc_split(x[2] * f.z, x[3] * f.w, h, l);
            sh[2 * half + 1] = h;
            sl[2 * half + 1] = l;
          }
          const uint16_t* qh_row = q_hi + col * QSTR + ks * 32 + 4 * grp;
          const uint16_t* ql_row = q_lo + col * QSTR + ks * 32 + 4 * grp;
          const u32x2 a0 = *reinterpret_cast<const u32x2*>(qh_row), a1 = *reinterpret_cast<const u32x2*>(qh_row + 16);
          const u32x2 b0 = *reinterpret_cast<const u32x2*>(ql_row), b1 = *reinterpret_cast<const u32x2*>(ql_row + 16);
          const u32x4 qh = {a0[0], a0[1], a1[0], a1[1]}, ql = {b0[0], b0[1], b1[0], b1[1]};
          o[n] = GC_MFMA32(sh, qh, o[n]);
          o[n] = GC_MFMA32(sh, ql, o[n]);
          o[n] = GC_MFMA32(sl, qh, o[n]);
        }
      }
      // the step's own tokens' share
      const int at = (4 * grp + (col >> 2)) * vstr + 4 * (col & 3);
#pragma unroll
      for (int n = 0; n < NVW; ++n) {
        const int vt = wave + 4 * n;
        if (vt >= n_vt) continue;
        const s16x4 vf = __builtin_amdgcn_ds_read_tr16_b64_v4i16((GC_LDS(s16x4)*)(v_rows + at + vt * 16));
        o[n] = GC_MFMA16(vf, p_hi, o[n]);
        o[n] = GC_MFMA16(vf, p_lo, o[n]);
      }
    }

    if (MODE != 2 || t0 + GC_STEP < end) {
      // ---- the state after the step: rows of S times what the channel keeps, plus K'^T V's times their power
      s16x4 vf[NVW];
#pragma unroll
      for (int n = 0; n < NVW; ++n)
        vf[n] = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
            (GC_LDS(s16x4)*)(v_rows + (4 * grp + (col >> 2)) * vstr + 4 * (col & 3) + (wave + 4 * n) * 16));
#pragma unroll
      for (int dt = 0; dt < ND; ++dt) {
        const int at = (4 * grp + (col >> 2)) * QSTR + dt * 16 + 4 * (col & 3);
        const s16x4 kh = __builtin_amdgcn_ds_read_tr16_b64_v4i16((GC_LDS(s16x4)*)(k_hi + at));
        const s16x4 kl = __builtin_amdgcn_ds_read_tr16_b64_v4i16((GC_LDS(s16x4)*)(k_lo + at));
        const float4 kp = *reinterpret_cast<const float4*>(keep + dt * 16 + 4 * grp);
        const float4 af = *reinterpret_cast<const float4*>(after + dt * 16 + 4 * grp);
#pragma unroll
        for (int n = 0; n < NVW; ++n) {
          if (wave + 4 * n >= n_vt) continue;
          floatx4 u = {0.f, 0.f, 0.f, 0.f};
          u = GC_MFMA16(kh, vf[n], u);
          u = GC_MFMA16(kl, vf[n], u);
          floatx4 x = s[dt][n];
          x[0] = fmaf(kp.x, x[0], af.x * u[0]);
          x[1] = fmaf(kp.y, x[1], af.y * u[1]);
          x[2] = fmaf(kp.z, x[2], af.z * u[2]);
          x[3] = fmaf(kp.w, x[3], af.w * u[3]);
          s[dt][n] = x;
        }
      }
    }

    if (MODE != 1) {
      // ---- every token's norm over all value elements, the gate, the store
      float sq = 0.f;
#pragma unroll
      for (int n = 0; n < NVW; ++n)
#pragma unroll
        for (int i = 0; i < 4; ++i) sq += o[n][i] * o[n][i];  // elements past vdim are zero (their v and S are)
      sq += __shfl_xor(sq, 16, 64);
      sq += __shfl_xor(sq, 32, 64);
      if (grp == 0) red[wave * 16 + col] = sq;
      __syncthreads();  // also: every wave is done with the step's arrays
      const float total = red[col] + red[16 + col] + red[32 + col] + red[48 + col];
      const float inv = 1.0f / sqrtf(total / static_cast<float>(vdim) + eps);
      if (col < n_tok) {
        const bf16_t* g_row = proj + static_cast<size_t>(t0 + col) * ld + g_off + head * vdim;
        bf16_t* o_row = out + (static_cast<size_t>(t0 + col) * heads + head) * vdim;
#pragma unroll
        for (int n = 0; n < NVW; ++n) {
          const int e0 = (wave + 4 * n) * 16 + 4 * grp;
          if (e0 >= vdim) continue;
          if (wide_v && g_off % 4 == 0) {  // four neighbours: 8-byte loads and stores
            const u32x2 raw = *reinterpret_cast<const u32x2*>(g_row + e0);
            const float4 w = *reinterpret_cast<const float4*>(norm_w + e0);
            const float wv[4] = {w.x, w.y, w.z, w.w};
            float y[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
              const float g = __uint_as_float((i & 1) ? (raw[i >> 1] & 0xffff0000u) : (raw[i >> 1] << 16));
              y[i] = ((o[n][i] * inv) * wv[i]) * (g / (1.0f + __expf(-g)));
            }
            u32x2 packed;
            packed[0] = static_cast<uint32_t>(float_to_bf16_bits(y[0])) | (static_cast<uint32_t>(float_to_bf16_bits(y[1])) << 16);
            packed[1] = static_cast<uint32_t>(float_to_bf16_bits(y[2])) | (static_cast<uint32_t>(float_to_bf16_bits(y[3])) << 16);
            *reinterpret_cast<u32x2*>(o_row + e0) = packed;
          } else {
#pragma unroll
            for (int i = 0; i < 4; ++i) {
              if (e0 + i < vdim) {
                const float g = to_float(g_row[e0 + i]);
                o_row[e0 + i].bits = float_to_bf16_bits(((o[n][i] * inv) * norm_w[e0 + i]) * (g / (1.0f + __expf(-g))));
              }
            }
          }
        }
      }
    } else {
      __syncthreads();  // the step's arrays are read before the next step's are written
    }
  }

  if (MODE == 1 && tid < dim) chunk_log[chunk_at * dim + tid] = forgotten;
#pragma unroll
  for (int n = 0; n < NVW; ++n) {
    const int e = (wave + 4 * n) * 16 + col;
#pragma unroll
    for (int dt = 0; dt < ND; ++dt)
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (MODE != 2 && e < vdim) st[static_cast<size_t>(dt * 16 + 4 * grp + i) * vdim + e] = s[dt][n][i];
  }
}

// chunk_state[.., c] holds what chunk c adds on entry and the state before it on exit, S_(c+1) = 2^log_c S_c + U_c
// row by row; the request's state slot receives the state after the last chunk.  One thread an element; a
// chunk's loads do not wait for the chunk before.
__global__ void gla_scan_kernel(float* __restrict__ chunk_state, const float* __restrict__ chunk_log, float* __restrict__ state,
                                const int* __restrict__ row_start, const int* __restrict__ row_slots, int heads, int dim,
                                int vdim, int max_chunks) {
  const int row = blockIdx.x / heads, head = blockIdx.x - row * heads;
  const int per_head = dim * vdim;
  const int x = blockIdx.y * blockDim.x + threadIdx.x;
  if (x >= per_head) return;
  const int d = x / vdim;
  const int n_chunks = (row_start[row + 1] - row_start[row] + GC_CHUNK - 1) / GC_CHUNK;
  const size_t first = (static_cast<size_t>(row) * heads + head) * max_chunks;
  float* cs = chunk_state + first * per_head + x;
  const float* cl = chunk_log + first * dim + d;
  float* st = state + (static_cast<size_t>(row_slots[row]) * heads + head) * per_head + x;
  float sv = *st;
  for (int c0 = 0; c0 < n_chunks; c0 += 8) {
    float u[8], l[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      u[i] = (c0 + i < n_chunks) ? cs[static_cast<size_t>(c0 + i) * per_head] : 0.f;
      l[i] = (c0 + i < n_chunks) ? cl[static_cast<size_t>(c0 + i) * dim] : 0.f;
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      if (c0 + i >= n_chunks) break;
      cs[static_cast<size_t>(c0 + i) * per_head] = sv;
      sv = fmaf(__builtin_amdgcn_exp2f(l[i]), sv, u[i]);
    }
  }
  *st = sv;
}

// Arguments as for the recurrent form (bfloat16 only); dim a multiple of 32 up to 256, vdim up to 256.  b: float [tokens, heads * dim], scratch.  max_count: the most tokens a row
// brings.  chunk_state and chunk_log: null (one workgroup walks a row), or rows * heads * chunks * dim * vdim
// and rows * heads * chunks * dim floats with chunks = ceil(max_count / 64).
extern "C" int pylon_gla_chunked(void* out, const void* proj, long long ld, int q_off, int k_off, int v_off, int g_off,
                                 int a_off, int rank, const float* a2, const float* a2_bias, float inv_tau, float* b,
                                 float* state, const float* norm_w, const int* row_start, const int* row_slots, int rows,
                                 int heads, int dim, int vdim, float eps, float q_scale, int max_count,
                                 float* chunk_state, long long chunk_floats, float* chunk_log, long long log_floats,
                                 hipStream_t stream) {
  PYLON_REQUIRE(rows >= 0 && rows <= 65535 && heads > 0 && heads <= 65535 && max_count >= 1 && rank >= 1, "gla_chunked: bad sizes");
  PYLON_REQUIRE(dim >= 32 && dim % 32 == 0 && dim <= 256, "gla_chunked: keys of a multiple of 32 up to 256 elements, got %d", dim);
  PYLON_REQUIRE(vdim >= 1 && vdim <= 256, "gla_chunked: values of up to 256 elements, got %d", vdim);
  PYLON_REQUIRE(rank <= 512, "gla_chunked: at most 512 logits of the decays, got %d", rank);
  PYLON_REQUIRE((reinterpret_cast<uintptr_t>(proj) & 15) == 0 && (reinterpret_cast<uintptr_t>(b) & 15) == 0 && (reinterpret_cast<uintptr_t>(norm_w) & 15) == 0 &&
                    (reinterpret_cast<uintptr_t>(out) & 7) == 0, "gla_chunked: operands must be aligned");
  PYLON_REQUIRE(inv_tau > 0.f, "gla_chunked: tau must be positive");
  if (rows == 0) return 0;
  const int max_chunks = (max_count + GC_CHUNK - 1) / GC_CHUNK;
  const long long chunks = static_cast<long long>(rows) * heads * max_chunks;
  PYLON_REQUIRE(chunk_state == nullptr || (chunk_log != nullptr && max_chunks <= 65535 && chunk_floats >= chunks * dim * vdim &&
                                           log_floats >= chunks * dim),
                "gla_chunked: the chunks' states need rows x heads x chunks x dim x vdim floats, their decays x dim");
  const int channels = heads * dim;
  const int steps = (max_count + GC_STEP - 1) / GC_STEP;
  hipLaunchKernelGGL(gla_decay_kernel, dim3(steps, rows, (channels + 255) / 256), dim3(256),
                     sizeof(float) * GC_STEP * ((rank + GD_RANK - 1) / GD_RANK * GD_RANK),
                     stream, b, (const bf16_t*)proj, ld, a_off, rank, a2, a2_bias, inv_tau, row_start, channels);
  const int nvw = vdim <= 64 ? 1 : vdim <= 128 ? 2 : 4;
  const size_t lds = 2 * (4 * static_cast<size_t>(GC_STEP) * (dim + 8) + static_cast<size_t>(GC_STEP) * (64 * nvw + 8)) +
                     sizeof(float) * (3 * dim + 64 + 16 * 17);
  dim3 block(256);
#define LAUNCH(KS, NVW, MODE)                                                                                       \
  hipLaunchKernelGGL((gla_chunked_kernel<KS, NVW, MODE>), dim3(rows, heads, MODE ? max_chunks : 1), block, lds, stream, \
                     (bf16_t*)out, (const bf16_t*)proj, ld, q_off, k_off, v_off, g_off, b, state, norm_w, row_start, \
                     row_slots, heads, vdim, eps, q_scale, chunk_state, chunk_log, max_chunks)
#define GO(KS, NVW)                                                                                                 \
  do {                                                                                                              \
    if (chunk_state == nullptr) {                                                                                   \
      LAUNCH(KS, NVW, 0);                                                                                           \
    } else {                                                                                                        \
      LAUNCH(KS, NVW, 1);                                                                                           \
      hipLaunchKernelGGL(gla_scan_kernel, dim3(rows * heads, (dim * vdim + 255) / 256), block, 0, stream, chunk_state, \
                         chunk_log, state, row_start, row_slots, heads, dim, vdim, max_chunks);                     \
      LAUNCH(KS, NVW, 2);                                                                                           \
    }                                                                                                               \
  } while (0)
#define PICK(KS)                  \
  do {                            \
    if (nvw == 1) GO(KS, 1);      \
    else if (nvw == 2) GO(KS, 2); \
    else GO(KS, 4);               \
  } while (0)
  switch (dim / 32) {
    case 1: PICK(1); break;
    case 2: PICK(2); break;
    case 3: PICK(3); break;
    case 4: PICK(4); break;
    case 5: PICK(5); break;
    case 6: PICK(6); break;
    case 7: PICK(7); break;
    default: PICK(8); break;
  }
#undef PICK
#undef GO
#undef LAUNCH
  PYLON_LAUNCHED("gla_chunked");
}
