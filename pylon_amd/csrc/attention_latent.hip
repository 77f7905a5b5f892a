// Paged causal attention over cached latents, on the matrix cores, for bfloat16: every token has one row
// in the cache, [c | r] of `width` elements, that all query heads share; a key is the whole row, its value
// the row's first `rank` elements:
//
//   s_ij = scale * q_i . row_j,   j <= i inside the mask
//   out_i = sum_j exp(s_ij) c_j / (sum_j exp(s_ij) + exp(sink_h))      (without a sink: no last term)
//
// A block of rows is brought into LDS once and read from there in both roles: as keys along their
// elements, as values across keys by the transposing LDS read of gfx950 (ds_read_b64_tr_b16; lane p of a
// group of 16 names row p / 4, elements 4 * (p % 4) .. + 3; lane i receives element i % 4 of lanes i / 4,
// i / 4 + 4, i / 4 + 8, i / 4 + 12).  Rows travel from memory straight into LDS (global_load_lds, 16 bytes a
// lane).  In LDS a row is P pieces of 16 bytes, P a multiple of 8, and piece c of row r lies at piece c ^
// f(r): with f the keys' reads (16 rows, one piece) and the values' (4 rows, 32 bytes) both fall into
// different banks.  Pieces past the row's end repeat its first one (finite numbers that meet zeros).
//
// Scores are computed transposed (rows: keys, columns: queries), so that a query's maximum lives in the
// lanes of its column and the exponentials are already laid out as the row operand of the value product.
// Scores, maximum, exponentials and sums are float; the weights enter the value product as two bfloat16
// terms, p = hi + lo (sixteen bits of mantissa), and their sums come from a product with ones.
//
// Prompt tiles: a workgroup of four waves takes up to 64 or 128 (token, head) pairs of consecutive tokens
// of one request, 16 or 32 a wave, and walks the visible keys 64 at a time through two buffers.
// Single tokens: a workgroup of four waves takes one token, 16 or 32 of its heads as query columns, and one
// cut of its keys; every wave stages blocks of 32 keys of its own (no barrier in the walk); the waves' partial
// results meet in LDS, and those of several cuts in a second small kernel, in their order.
#include "common.h"

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float floatx4 __attribute__((ext_vector_type(4)));
typedef unsigned int u32x4 __attribute__((ext_vector_type(4)));
typedef short s16x4 __attribute__((ext_vector_type(4)));

#define AL_BK 64       // keys of a block of a prompt tile
#define AL_DK 32       // keys of a block of a single token's wave
#define AL_SLACK 8.0f  // how far (as a power of two) a score may exceed the maximum in use
#define AL_LOG2E 1.44269504088896340736f
#define AL_LDS(T) __attribute__((address_space(3))) T
#define AL_GLOBAL(T) __attribute__((address_space(1))) T

// A row of 32 KS elements in LDS.
template <int KS>
struct LatentRow {
  static constexpr int P = (4 * KS + 7) / 8 * 8;  // pieces of 16 bytes
  static constexpr int BYTES = P * 16;
  static constexpr bool EVEN = P % 16 == 0;       // rows a multiple of 256 bytes
  static constexpr int SPAN = EVEN ? 16 : 8;      // pieces that f permutes among themselves
  static __device__ __forceinline__ unsigned f(unsigned r) {
    return EVEN ? (((r & 7) << 1) | ((r >> 3) & 1)) : ((((r >> 1) & 3) << 1) | ((r >> 3) & 1));
  }
};

// Brings rows 0..ROWS-1 of a block into LDS at `lds` with THREADS lanes of which this one is `lane0` (its wave
// starts at lane0 & ~63); rows past `last` repeat it.  `block` is the first row in memory.
template <int KS, int ROWS, int THREADS>
__device__ __forceinline__ void latent_fetch(const uint16_t* block, int width, unsigned last, uint16_t* lds, int lane0) {
  typedef LatentRow<KS> R;
  static_assert(ROWS * R::P % THREADS == 0, "whole rounds of loads");
  const int wave0 = __builtin_amdgcn_readfirstlane(lane0 & ~(PYLON_WAVE - 1));
  const unsigned pieces = width >> 3;
#pragma unroll
  for (int i = 0; i < ROWS * R::P / THREADS; ++i) {
    const unsigned idx = i * THREADS + lane0;
    const unsigned row = idx / R::P, at = idx - row * R::P;
    const unsigned c = at ^ R::f(row);
    const unsigned src = (row < last ? row : last) * width + (c < pieces ? c : 0) * 8;
    __builtin_amdgcn_global_load_lds((const AL_GLOBAL(void)*)(block + src),
                                     (AL_LDS(void)*)(lds + (i * THREADS + wave0) * 8), 16, 0, 0);
  }
}

// Where a lane reads its operands of a block (bytes from the block's start).
template <int KS>
struct LatentReads {
  typedef LatentRow<KS> R;
  static constexpr int NK = R::SPAN / 4, NV = R::SPAN / 2;
  unsigned k[NK], v[NV];
  __device__ __forceinline__ LatentReads(int col, int grp) {
    const unsigned fk = R::f(col);
#pragma unroll
    for (int i = 0; i < NK; ++i) k[i] = col * R::BYTES + ((4 * i + grp) ^ fk) * 16;
    const unsigned row = 4 * grp + (col >> 2), fv = R::f(row);
#pragma unroll
    for (int i = 0; i < NV; ++i) v[i] = row * R::BYTES + ((2 * i + ((col & 3) >> 1)) ^ fv) * 16 + (col & 1) * 8;
  }
  // keys 16 kt + col, elements 32 ks + 8 grp .. + 7
  __device__ __forceinline__ bf16x8 key(const AL_LDS(char)* tile, int kt, int ks) const {
    return *reinterpret_cast<const AL_LDS(bf16x8)*>(tile + k[ks % NK] + kt * 16 * R::BYTES + (ks / NK) * R::SPAN * 16);
  }
  // element 16 dt + col of keys 32 kg + 4 grp .. + 3 and 32 kg + 16 + 4 grp .. + 3
  __device__ __forceinline__ bf16x8 value(const AL_LDS(char)* tile, int kg, int dt) const {
    const AL_LDS(char)* at = tile + v[dt % NV] + kg * 32 * R::BYTES + (dt / NV) * R::SPAN * 16;
    const s16x4 a = __builtin_amdgcn_ds_read_tr16_b64_v4i16((AL_LDS(s16x4)*)at);
    const s16x4 b = __builtin_amdgcn_ds_read_tr16_b64_v4i16((AL_LDS(s16x4)*)(at + 16 * R::BYTES));
    return __builtin_bit_cast(bf16x8, __builtin_shufflevector(a, b, 0, 1, 2, 3, 4, 5, 6, 7));
  }
};

// Scores (in place: keys kb + 16 kt + 4 grp + r of the lane's query column) masked where asked, the running
// maximum kept and the accumulators (rows 4 grp + r) rescaled when it moves; returns what to add to
// scale_log2 * score before exp2.  The maximum is raised only when a score exceeds it by more than the
// slack: until then weights may reach 2^AL_SLACK instead of 1, which the float sums hold just as well.
template <int KT, int NT>
__device__ __forceinline__ float latent_softmax(floatx4 (&s)[KT], float& m_run, floatx4 (&o)[NT], int last_seen,
                                                int first_seen, bool masked, float scale_log2, float slack) {
  if (masked) {
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (!(kt * 16 + r <= last_seen && kt * 16 + r >= first_seen)) s[kt][r] = -INFINITY;
  }
  float top = -INFINITY;
#pragma unroll
  for (int kt = 0; kt < KT; ++kt)
#pragma unroll
    for (int r = 0; r < 4; ++r) top = fmaxf(top, s[kt][r]);
  if (__ballot(top > m_run + slack) != 0) {  // the same for the whole wave
    top = fmaxf(top, __shfl_xor(top, 16, PYLON_WAVE));
    top = fmaxf(top, __shfl_xor(top, 32, PYLON_WAVE));
    const float m_new = fmaxf(m_run, top);
    const float m_use = (m_new == -INFINITY) ? 0.f : m_new;  // a column that has seen no key yet
    const float corr = __builtin_amdgcn_exp2f((m_run - m_use) * scale_log2);
    m_run = m_new;
    const int grp = (threadIdx.x & (PYLON_WAVE - 1)) >> 4;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float c = __shfl(corr, 4 * grp + r, PYLON_WAVE);
#pragma unroll
      for (int nt = 0; nt < NT; ++nt) o[nt][r] *= c;
    }
  }
  return (m_run == -INFINITY) ? 0.f : -m_run * scale_log2;
}

// The weights of 32 keys as two row operands of the value product (slot j: key 4 grp + j, then 16 + 4 grp + j - 4).
__device__ __forceinline__ void latent_weights(const floatx4& a, const floatx4& b, float scale_log2, float shift,
                                               bf16x8& hi, bf16x8& lo) {
  uint32_t ph[4], pl[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const floatx4& s = e < 2 ? a : b;
    const float p0 = __builtin_amdgcn_exp2f(fmaf(s[2 * (e & 1)], scale_log2, shift));
    const float p1 = __builtin_amdgcn_exp2f(fmaf(s[2 * (e & 1) + 1], scale_log2, shift));
    const uint32_t u0 = __float_as_uint(p0), u1 = __float_as_uint(p1);
    ph[e] = __builtin_amdgcn_perm(u1, u0, 0x07060302u);  // the upper halves side by side
    const float r0 = p0 - __uint_as_float(u0 & 0xffff0000u), r1 = p1 - __uint_as_float(u1 & 0xffff0000u);
    pl[e] = __builtin_amdgcn_perm(__float_as_uint(r1), __float_as_uint(r0), 0x07060302u);
  }
  hi = __builtin_bit_cast(bf16x8, u32x4{ph[0], ph[1], ph[2], ph[3]});
  lo = __builtin_bit_cast(bf16x8, u32x4{pl[0], pl[1], pl[2], pl[3]});
}

template <int KS>
__device__ __forceinline__ void latent_queries(bf16x8 (&qf)[KS], const uint16_t* row, int width, int grp, bool valid) {
#pragma unroll
  for (int ks = 0; ks < KS; ++ks) {
    const int d = ks * 32 + grp * 8;
    u32x4 raw = {0u, 0u, 0u, 0u};
    if (valid && d < width) raw = *reinterpret_cast<const u32x4*>(row + d);
    qf[ks] = __builtin_bit_cast(bf16x8, raw);
  }
}

// KS: steps of 32 elements of a row (width <= 32 KS); NT: tiles of 16 value elements (rank <= 16 NT);
// QT: tiles of 16 query rows a wave.
template <int KS, int NT, int QT>
__global__ __launch_bounds__(256, 1) void latent_prefill_kernel(
    uint16_t* __restrict__ out, const uint16_t* __restrict__ q, const uint16_t* __restrict__ cache,
    const int* __restrict__ block_table, int table_width, const int* __restrict__ tiles, int n_heads, int width,
    int rank, int page_size, int window, float scale, const float* __restrict__ sink) {
  typedef LatentRow<KS> R;
  // two blocks, as two arrays: loads into one must not be taken to touch the other
  __shared__ __attribute__((aligned(16))) uint16_t buf_a[AL_BK * R::P * 8];
  __shared__ __attribute__((aligned(16))) uint16_t buf_b[AL_BK * R::P * 8];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int col = lane & 15, grp = lane >> 4;
  const int* td = tiles + blockIdx.x * 4;
  const int tok0 = td[0], ntok = td[1], pos0 = td[3];
  const int* table = block_table + static_cast<size_t>(td[2]) * table_width;
  const int kv_last = pos0 + ntok - 1;
  const int kb_first = first_visible(pos0, window) / AL_BK * AL_BK;
  const int edge = first_visible(kv_last, window);  // keys from here on are inside every query's window
  const LatentReads<KS> at(col, grp);

  auto fetch = [&](int kb, uint16_t* into) {  // a block lies inside one page
    const int page = kb / page_size;
    const size_t row0 = static_cast<size_t>(table[page]) * page_size + (kb - page * page_size);
    latent_fetch<KS, AL_BK, 256>(cache + row0 * width, width, kv_last - kb, into, tid);
  };
  fetch(kb_first, buf_a);

  int qpos[QT];
  bf16x8 qf[QT][KS];
  floatx4 o[QT][NT + 1];  // the output tiles and, last, the rows' sums of weights
  float m_run[QT];
#pragma unroll
  for (int qt = 0; qt < QT; ++qt) {
    const int rr = wave * (16 * QT) + qt * 16 + col;
    const int ti = rr / n_heads, hh = rr - ti * n_heads;
    const bool valid = ti < ntok;
    qpos[qt] = valid ? pos0 + ti : -1;
    latent_queries<KS>(qf[qt], q + (static_cast<size_t>(tok0 + (valid ? ti : 0)) * n_heads + hh) * width, width, grp, valid);
    m_run[qt] = -INFINITY;
#pragma unroll
    for (int nt = 0; nt <= NT; ++nt) o[qt][nt] = floatx4{0.f, 0.f, 0.f, 0.f};
  }
  const bf16x8 ones = __builtin_bit_cast(bf16x8, u32x4{0x3f803f80u, 0x3f803f80u, 0x3f803f80u, 0x3f803f80u});
  const float scale_log2 = scale * AL_LOG2E;
  const float slack = AL_SLACK / scale_log2;

  auto block = [&](int kb, uint16_t* current, uint16_t* next) __attribute__((always_inline)) {
    __builtin_amdgcn_s_waitcnt(0);  // this wave's loads, then everyone's
    __syncthreads();
    if (kb + AL_BK <= kv_last) fetch(kb + AL_BK, next);
    const AL_LDS(char)* tile = (const AL_LDS(char)*)current;
    floatx4 s[QT][AL_BK / 16];
#pragma unroll
    for (int kt = 0; kt < AL_BK / 16; ++kt) {
#pragma unroll
      for (int qt = 0; qt < QT; ++qt) s[qt][kt] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        const bf16x8 kf = at.key(tile, kt, ks);
#pragma unroll
        for (int qt = 0; qt < QT; ++qt) s[qt][kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[qt][ks], s[qt][kt], 0, 0, 0);
      }
    }
    const bool masked = kb + AL_BK - 1 > pos0 || kb < edge;
    bf16x8 hi[QT][AL_BK / 32], lo[QT][AL_BK / 32];
#pragma unroll
    for (int qt = 0; qt < QT; ++qt) {
      const int qp = qpos[qt];
      const int base = kb + 4 * grp;
      const float shift = latent_softmax<AL_BK / 16, NT + 1>(
          s[qt], m_run[qt], o[qt], qp - base, (qp < 0 ? 0 : first_visible(qp, window)) - base, masked || qp < 0, scale_log2,
          slack);
#pragma unroll
      for (int kg = 0; kg < AL_BK / 32; ++kg)
        latent_weights(s[qt][2 * kg], s[qt][2 * kg + 1], scale_log2, shift, hi[qt][kg], lo[qt][kg]);
    }
#pragma unroll
    for (int kg = 0; kg < AL_BK / 32; ++kg) {
#pragma unroll
      for (int nt = 0; nt < NT; ++nt) {
        const bf16x8 vf = at.value(tile, kg, nt);
#pragma unroll
        for (int qt = 0; qt < QT; ++qt) {
          o[qt][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi[qt][kg], vf, o[qt][nt], 0, 0, 0);
          o[qt][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo[qt][kg], vf, o[qt][nt], 0, 0, 0);
        }
      }
#pragma unroll
      for (int qt = 0; qt < QT; ++qt) {
        o[qt][NT] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi[qt][kg], ones, o[qt][NT], 0, 0, 0);
        o[qt][NT] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo[qt][kg], ones, o[qt][NT], 0, 0, 0);
      }
    }
  };
  for (int kb = kb_first;; kb += 2 * AL_BK) {
    block(kb, buf_a, buf_b);
    if (kb + AL_BK > kv_last) break;
    block(kb + AL_BK, buf_b, buf_a);
    if (kb + 2 * AL_BK > kv_last) break;
  }

#pragma unroll
  for (int qt = 0; qt < QT; ++qt) {
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int rr = wave * (16 * QT) + qt * 16 + 4 * grp + r;
      const int ti = rr / n_heads, hh = rr - ti * n_heads;
      const float m = __shfl(m_run[qt], 4 * grp + r, PYLON_WAVE);
      if (ti >= ntok) continue;
      float l = o[qt][NT][r];
      // the sink on the scale of the running maximum (a sink far above every score: infinity, and the output zero)
      if (sink != nullptr) l += __builtin_amdgcn_exp2f(sink[hh] * AL_LOG2E - m * scale_log2);
      const float inv = 1.0f / l;
      uint16_t* orow = out + (static_cast<size_t>(tok0 + ti) * n_heads + hh) * rank;
#pragma unroll
      for (int nt = 0; nt < NT; ++nt)
        if (nt * 16 + col < rank) orow[nt * 16 + col] = float_to_bf16_bits(o[qt][nt][r] * inv);
    }
  }
}

// One token, up to 16 QT of its heads, one cut of its keys.  partial (cuts > 1): float [token][head][cut]
// [2 + rank]: the maximum as a power of two, the sum, the unnormalised output.
template <int KS, int NT, int QT>
__global__ __launch_bounds__(256, 1) void latent_decode_kernel(
    uint16_t* __restrict__ out, const uint16_t* __restrict__ q, const uint16_t* __restrict__ cache,
    const int* __restrict__ block_table, int table_width, const int* __restrict__ positions, int n_heads, int width,
    int rank, int page_size, int window, float scale, const float* __restrict__ sink, int cuts,
    float* __restrict__ partial) {
  typedef LatentRow<KS> R;
  constexpr int HEADS = 16 * QT, CT = 4;  // tiles of value elements merged at a time
  constexpr int STAGE = AL_DK * R::P * 8;  // elements of a wave's block
  extern __shared__ __attribute__((aligned(16))) uint16_t al_lds[];  // a block a wave; then the merge
  __shared__ float merge_m[4][HEADS], merge_l[4][HEADS];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int col = lane & 15, grp = lane >> 4;
  const int tok = blockIdx.x, head0 = blockIdx.y * HEADS, cut = blockIdx.z;
  const int pos = positions[tok];
  const int* table = block_table + static_cast<size_t>(tok) * table_width;
  const int first = first_visible(pos, window);
  const int b_first = first / AL_DK, n_blocks = pos / AL_DK - b_first + 1;
  const int per_cut = (n_blocks + cuts - 1) / cuts;
  const int b_begin = b_first + cut * per_cut;
  int b_end = b_begin + per_cut;
  if (b_end > b_first + n_blocks) b_end = b_first + n_blocks;
  const LatentReads<KS> at(col, grp);
  uint16_t* mine = al_lds + wave * STAGE;

  auto fetch = [&](int b) {  // a block lies inside one page
    const int kb = b * AL_DK, page = kb / page_size;
    const size_t row0 = static_cast<size_t>(table[page]) * page_size + (kb - page * page_size);
    latent_fetch<KS, AL_DK, PYLON_WAVE>(cache + row0 * width, width, pos - kb, mine, lane);
  };
  if (b_begin + wave < b_end) fetch(b_begin + wave);  // on their way while the queries come

  bf16x8 qf[QT][KS];
  floatx4 o[QT][NT + 1];
  float m_run[QT];
#pragma unroll
  for (int qt = 0; qt < QT; ++qt) {
    const int h = head0 + qt * 16 + col;
    const bool valid = h < n_heads;
    latent_queries<KS>(qf[qt], q + (static_cast<size_t>(tok) * n_heads + (valid ? h : 0)) * width, width, grp, valid);
    m_run[qt] = -INFINITY;
#pragma unroll
    for (int nt = 0; nt <= NT; ++nt) o[qt][nt] = floatx4{0.f, 0.f, 0.f, 0.f};
  }
  const bf16x8 ones = __builtin_bit_cast(bf16x8, u32x4{0x3f803f80u, 0x3f803f80u, 0x3f803f80u, 0x3f803f80u});
  const float scale_log2 = scale * AL_LOG2E;
  const float slack = AL_SLACK / scale_log2;
  const AL_LDS(char)* tile = (const AL_LDS(char)*)mine;

  for (int b = b_begin + wave; b < b_end; b += 4) {
    __builtin_amdgcn_s_waitcnt(0);  // the block has landed (it is this wave's own)
    __builtin_amdgcn_wave_barrier();
    const int kb = b * AL_DK;
    floatx4 s[QT][2];
#pragma unroll
    for (int kt = 0; kt < 2; ++kt) {
#pragma unroll
      for (int qt = 0; qt < QT; ++qt) s[qt][kt] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        const bf16x8 kf = at.key(tile, kt, ks);
#pragma unroll
        for (int qt = 0; qt < QT; ++qt) s[qt][kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[qt][ks], s[qt][kt], 0, 0, 0);
      }
    }
    const bool masked = kb + AL_DK - 1 > pos || kb < first;
    bf16x8 hi[QT], lo[QT];
#pragma unroll
    for (int qt = 0; qt < QT; ++qt) {
      const float shift = latent_softmax<2, NT + 1>(s[qt], m_run[qt], o[qt], pos - kb - 4 * grp, first - kb - 4 * grp, masked,
                                                    scale_log2, slack);
      latent_weights(s[qt][0], s[qt][1], scale_log2, shift, hi[qt], lo[qt]);
    }
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) {
      const bf16x8 vf = at.value(tile, 0, nt);
#pragma unroll
      for (int qt = 0; qt < QT; ++qt) {
        o[qt][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi[qt], vf, o[qt][nt], 0, 0, 0);
        o[qt][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo[qt], vf, o[qt][nt], 0, 0, 0);
      }
    }
#pragma unroll
    for (int qt = 0; qt < QT; ++qt) {
      o[qt][NT] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi[qt], ones, o[qt][NT], 0, 0, 0);
      o[qt][NT] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo[qt], ones, o[qt][NT], 0, 0, 0);
    }
    if (b + 4 < b_end) {
      // every read of the block has returned (its numbers are in registers) before the next one overwrites it
      __builtin_amdgcn_s_waitcnt(0);
      __builtin_amdgcn_wave_barrier();
      fetch(b + 4);
    }
  }

  // the waves' maxima and sums meet: per head the maximum of all, every wave's factor and the whole sum
#pragma unroll
  for (int qt = 0; qt < QT; ++qt) {
    if (grp == 0) merge_m[wave][qt * 16 + col] = m_run[qt];
    if (col == 0) {
#pragma unroll
      for (int r = 0; r < 4; ++r) merge_l[wave][qt * 16 + 4 * grp + r] = o[qt][NT][r];
    }
  }
  __syncthreads();  // also: no wave reads its block any more
  if (tid < HEADS) {
    float m = merge_m[0][tid];
#pragma unroll
    for (int w = 1; w < 4; ++w) m = fmaxf(m, merge_m[w][tid]);
    float l = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      const float mw = merge_m[w][tid];
      const float fac = (mw == -INFINITY) ? 0.f : __builtin_amdgcn_exp2f((mw - m) * scale_log2);
      l = fmaf(merge_l[w][tid], fac, l);
      merge_m[w][tid] = fac;
    }
    if (head0 + tid < n_heads) {
      if (cuts > 1) {
        float* dst = partial + ((static_cast<size_t>(tok) * n_heads + head0 + tid) * cuts + cut) * (2 + rank);
        dst[0] = m * scale_log2;
        dst[1] = l;
      } else if (sink != nullptr) {
        l += __builtin_amdgcn_exp2f(sink[head0 + tid] * AL_LOG2E - m * scale_log2);
      }
    }
    merge_l[0][tid] = 1.0f / l;  // used where the keys are not cut
  }
  __syncthreads();
  float* stage = reinterpret_cast<float*>(al_lds);  // [4 waves][HEADS][16 CT]
#pragma unroll
  for (int qt = 0; qt < QT; ++qt) {
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float fac = merge_m[wave][qt * 16 + 4 * grp + r];
#pragma unroll
      for (int nt = 0; nt < NT; ++nt) o[qt][nt][r] *= fac;
    }
  }
#pragma unroll
  for (int c0 = 0; c0 < NT; c0 += CT) {
    if (c0) __syncthreads();
#pragma unroll
    for (int qt = 0; qt < QT; ++qt)
#pragma unroll
      for (int c = 0; c < CT; ++c)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          stage[(wave * HEADS + qt * 16 + 4 * grp + r) * (16 * CT) + c * 16 + col] = o[qt][c0 + c][r];
    __syncthreads();
#pragma unroll
    for (int j = 0; j < HEADS * 16 * CT / 1024; ++j) {  // four neighbouring elements a thread
      const int i = (j * 256 + tid) * 4;
      const int h = i / (16 * CT), d = c0 * 16 + i % (16 * CT);
      float4 acc = *reinterpret_cast<const float4*>(stage + i);
#pragma unroll
      for (int w = 1; w < 4; ++w) {
        const float4 x = *reinterpret_cast<const float4*>(stage + w * HEADS * 16 * CT + i);
        acc.x += x.x; acc.y += x.y; acc.z += x.z; acc.w += x.w;
      }
      if (head0 + h >= n_heads) continue;
      const float v[4] = {acc.x, acc.y, acc.z, acc.w};
      const size_t item = static_cast<size_t>(tok) * n_heads + head0 + h;
      float* dst = partial + (item * cuts + cut) * (2 + rank) + 2 + d;
      const float inv = merge_l[0][h];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        if (d + e >= rank) continue;
        if (cuts > 1) dst[e] = v[e];
        else out[item * rank + d + e] = float_to_bf16_bits(v[e] * inv);
      }
    }
  }
}

// One workgroup per (token, head) merges the cuts (at most 64) in their order; the sink joins here.  A
// thread takes an element of the values; the loads of eight cuts do not wait for one another.
__global__ __launch_bounds__(256) void latent_merge_kernel(uint16_t* __restrict__ out, const float* __restrict__ partial,
                                                           int n_heads, int cuts, int rank, const float* __restrict__ sink) {
  const int item = blockIdx.x;
  const int lane = threadIdx.x & (PYLON_WAVE - 1);
  const int stride = 2 + rank;
  const float* src = partial + static_cast<size_t>(item) * cuts * stride;
  const float mc = lane < cuts ? src[lane * stride] : -INFINITY;
  const float lc = lane < cuts ? src[lane * stride + 1] : 0.f;
  const float z = sink != nullptr ? sink[item % n_heads] * AL_LOG2E : 0.f;
  const int last = cuts - 1;
  const int d0 = static_cast<int>(threadIdx.x) < rank ? static_cast<int>(threadIdx.x) : rank - 1;
  float v[8];  // the first element's first cuts are on their way while the maxima meet
#pragma unroll
  for (int u = 0; u < 8; ++u) v[u] = src[(u < last ? u : last) * stride + 2 + d0];
  const float m = wave_max(mc);  // finite: some cut holds the token's own key
  const float w = (mc == -INFINITY) ? 0.f : __builtin_amdgcn_exp2f(mc - m);
  float l = wave_sum(lc * w);
  if (sink != nullptr) l += __builtin_amdgcn_exp2f(z - m);
  const float inv = 1.0f / l;
  for (int base = 0; base < rank; base += 256) {  // every lane stays in the loop: its weight is read by the others
    const int d = base + threadIdx.x;
    const int dd = d < rank ? d : rank - 1;
    float acc = 0.f;
    for (int c0 = 0; c0 < cuts; c0 += 8) {
      if (base != 0 || c0 != 0) {
#pragma unroll
        for (int u = 0; u < 8; ++u) v[u] = src[(c0 + u < last ? c0 + u : last) * stride + 2 + dd];
      }
#pragma unroll
      for (int u = 0; u < 8; ++u) {
        const float f = __shfl(w, (c0 + u) & (PYLON_WAVE - 1), PYLON_WAVE);
        if (c0 + u < cuts) acc = fmaf(v[u], f, acc);
      }
    }
    if (d < rank) out[static_cast<size_t>(item) * rank + d] = float_to_bf16_bits(acc * inv);
  }
}

// The instances: (steps of 32 row elements, tiles of 16 value elements), the first that holds a row is taken.
#define AL_SHAPES(X) X(2, 4) X(3, 4) X(4, 8) X(6, 8) X(8, 8) X(10, 16) X(12, 16) X(18, 32)

static int latent_shape(int width, int rank) {
  int index = 0;
#define AL_FITS(KS, NT)                                    \
  if (width <= 32 * KS && rank <= 16 * NT) return index;   \
  ++index;
  AL_SHAPES(AL_FITS)
#undef AL_FITS
  return -1;
}

// 1 if rows of `width` elements with values of `rank` over pages of `page_size` are taken, else 0.
extern "C" int pylon_latent_attention_ok(int width, int rank, int page_size) {
  return width % 8 == 0 && rank >= 1 && rank <= width && page_size > 0 && page_size % AL_BK == 0 &&
         latent_shape(width, rank) >= 0;
}

static int check_latent(const char* name, const void* q, const void* cache, int n_heads, int width, int rank,
                        int page_size, int table_width, float scale) {
  PYLON_REQUIRE(n_heads > 0 && table_width > 0, "%s: bad sizes", name);
  PYLON_REQUIRE(pylon_latent_attention_ok(width, rank, page_size),
                "%s: rows of %d elements with values of %d over pages of %d are not taken", name, width, rank, page_size);
  PYLON_REQUIRE(((reinterpret_cast<uintptr_t>(q) | reinterpret_cast<uintptr_t>(cache)) & 15) == 0,
                "%s: operands must be 16-byte aligned", name);
  PYLON_REQUIRE(scale > 0.f, "%s: the scale must be positive", name);
  return 0;
}

// Prompt tiles.  q: bf16 [tokens, n_heads, width]; cache: bf16 [pages * page_size, width]; out: bf16 [tokens,
// n_heads, rank].  tiles: int [n_tiles, 4] = (first token, count, block-table row, first position) of runs of
// consecutive tokens of one request, at most floor(rows / n_heads) of them; rows: 64 or 128.  window: the
// mask as one integer (first_visible in common.h).  sink: null or float [n_heads].
extern "C" int pylon_latent_prefill(void* out, const void* q, const void* cache, const int* block_table, int table_width,
                                    const int* tiles, int n_tiles, int n_heads, int width, int rank, int page_size,
                                    int window, float scale, const float* sink, int rows, hipStream_t stream) {
  PYLON_REQUIRE(n_tiles >= 0 && (rows == 64 || rows == 128), "latent_prefill: 64 or 128 query rows a workgroup");
  PYLON_REQUIRE(n_heads <= rows, "latent_prefill: at most %d heads", rows);
  if (check_latent("latent_prefill", q, cache, n_heads, width, rank, page_size, table_width, scale)) return 1;
  if (n_tiles == 0) return 0;
  int index = latent_shape(width, rank);
#define AL_GO(KS, NT, QT)                                                                                           \
  hipLaunchKernelGGL((latent_prefill_kernel<KS, NT, QT>), dim3(n_tiles), dim3(256), 0, stream, (uint16_t*)out,      \
                     (const uint16_t*)q, (const uint16_t*)cache, block_table, table_width, tiles, n_heads, width,   \
                     rank, page_size, window, scale, sink)
#define AL_PICK(KS, NT)                   \
  if (index-- == 0) {                     \
    if (rows == 64) AL_GO(KS, NT, 1);     \
    else if constexpr (NT <= 16) AL_GO(KS, NT, 2); \
    else PYLON_REFUSE("latent_prefill: values this wide take 64 query rows a workgroup"); \
  }
  AL_SHAPES(AL_PICK)
#undef AL_PICK
#undef AL_GO
  PYLON_LAUNCHED("latent_prefill");
}

// A step of single tokens: token t on row t of the block table at positions[t]; `cuts` workgroups (at most 64)
// share the keys of a token and a group of heads, and then partial holds tokens * n_heads * cuts * (2 + rank)
// floats.
extern "C" int pylon_latent_decode(void* out, const void* q, const void* cache, const int* block_table, int table_width,
                                   const int* positions, int tokens, int n_heads, int width, int rank, int page_size,
                                   int window, float scale, const float* sink, int cuts, float* partial,
                                   long long partial_floats, hipStream_t stream) {
  PYLON_REQUIRE(tokens >= 0 && cuts >= 1 && cuts <= 64, "latent_decode: 1 to 64 cuts");
  if (check_latent("latent_decode", q, cache, n_heads, width, rank, page_size, table_width, scale)) return 1;
  PYLON_REQUIRE(cuts == 1 || (partial != nullptr &&
                              partial_floats >= static_cast<long long>(tokens) * n_heads * cuts * (2 + rank)),
                "latent_decode: %d cuts need a scratch buffer", cuts);
  if (tokens == 0) return 0;
  int index = latent_shape(width, rank);
#define AL_GO(KS, NT, QT)                                                                                            \
  do {                                                                                                               \
    constexpr size_t stage = 4 * AL_DK * LatentRow<KS>::BYTES, merge = 4 * 16 * QT * 64 * sizeof(float);             \
    constexpr size_t lds = stage > merge ? stage : merge;                                                            \
    if (lds > 48 * 1024)                                                                                             \
      (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&latent_decode_kernel<KS, NT, QT>),                    \
                                hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(lds));                  \
    const int groups = (n_heads + 16 * QT - 1) / (16 * QT);                                                          \
    PYLON_REQUIRE(groups <= 65535, "latent_decode: too many heads");                                                 \
    hipLaunchKernelGGL((latent_decode_kernel<KS, NT, QT>), dim3(tokens, groups, cuts), dim3(256), lds, stream,       \
                       (uint16_t*)out, (const uint16_t*)q, (const uint16_t*)cache, block_table, table_width, positions, \
                       n_heads, width, rank, page_size, window, scale, sink, cuts, partial);                         \
  } while (0)
#define AL_PICK(KS, NT)                                       \
  if (index-- == 0) {                                         \
    if constexpr (NT <= 16 && KS >= 3) {                      \
      if (n_heads > 16) AL_GO(KS, NT, 2);                     \
      else AL_GO(KS, NT, 1);                                  \
    } else {                                                  \
      AL_GO(KS, NT, 1);                                       \
    }                                                         \
  }
  AL_SHAPES(AL_PICK)
#undef AL_PICK
#undef AL_GO
  if (cuts > 1) {
    const long long items = static_cast<long long>(tokens) * n_heads;
    PYLON_REQUIRE(items < (1ll << 31), "latent_decode: too many (token, head) pairs for one launch");
    hipLaunchKernelGGL(latent_merge_kernel, dim3((unsigned)items), dim3(256), 0, stream, (uint16_t*)out, partial, n_heads,
                       cuts, rank, sink);
  }
  PYLON_LAUNCHED("latent_decode");
}
