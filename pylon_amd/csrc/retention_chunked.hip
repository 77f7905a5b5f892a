// Retention and lightning attention of bfloat16 prompt portions: the entry point of the chunked kernels
// (retention_chunked.h), and the launches of retention's form.
#include "retention_chunked.h"

// Arguments as for the recurrent form (bfloat16 only): proj [tokens, ld] with q, k, v and the gate
// at their offsets; state float [slots, heads, dim, vdim].  dim a multiple of 32 up to 256, vdim up to
// 256.  form 0: rot_dims even and at most dim, out bfloat16 [tokens, heads * vdim]; form 1: no rotation,
// no gate, k_scale 1, out float.  chunk_state given: a workgroup takes `span` chunks of 32 tokens, in three
// launches (contributions, scan, outputs).
extern "C" int pylon_retention_chunked(void* out, const void* proj, long long ld, int q_off, int k_off, int v_off,
                                       int g_off, float* state, const float* decay, const float* inv_freq,
                                       int rot_dims, const int* positions, const int* row_start, const int* row_slots,
                                       int rows, int heads, int dim, int vdim, float eps, float k_scale,
                                       int max_count, float* chunk_state, long long chunk_floats, int span, int form,
                                       hipStream_t stream) {
  PYLON_REQUIRE(form == 0 || form == 1, "retention_chunked: unknown form %d", form);
  PYLON_REQUIRE(rows >= 0 && heads > 0, "retention_chunked: bad sizes");
  PYLON_REQUIRE(dim >= 32 && dim % 32 == 0 && dim <= 256, "retention_chunked: keys of a multiple of 32 up to 256 elements, got %d", dim);
  PYLON_REQUIRE(vdim >= 1 && vdim <= 256, "retention_chunked: values of up to 256 elements, got %d", vdim);
  PYLON_REQUIRE(rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= dim && (dim - rot_dims) % 2 == 0,
                "retention_chunked: rot_dims %d does not fit a head of %d", rot_dims, dim);
  PYLON_REQUIRE(rot_dims == 0 || inv_freq != nullptr, "retention_chunked: a rotation needs its frequencies");
  PYLON_REQUIRE(form == 0 || (rot_dims == 0 && k_scale == 1.0f), "retention_chunked: form 1 neither rotates nor scales");
  PYLON_REQUIRE(span >= 1 && span <= 1024, "retention_chunked: a workgroup takes 1 to 1024 chunks, got %d", span);
  if (rows == 0) return 0;
  const int max_chunks = (max_count + RC_CHUNK * span - 1) / (RC_CHUNK * span);
  PYLON_REQUIRE(chunk_state == nullptr ||
                    (max_count >= 1 && chunk_floats >= static_cast<long long>(rows) * heads * max_chunks * dim * vdim),
                "retention_chunked: the stretches' states need rows x heads x stretches x dim x vdim floats");
  if (form == 0)
    retention_chunked_run<0>(out, (const bf16_t*)proj, ld, q_off, k_off, v_off, g_off, state, decay, inv_freq, rot_dims,
                             positions, row_start, row_slots, rows, heads, dim, vdim, eps, k_scale, chunk_state,
                             max_chunks, span, stream);
  else
    pylon_lightning_chunked_run(out, (const bf16_t*)proj, ld, q_off, k_off, v_off, g_off, state, decay, inv_freq,
                                rot_dims, positions, row_start, row_slots, rows, heads, dim, vdim, eps, k_scale,
                                chunk_state, max_chunks, span, stream);
  PYLON_LAUNCHED("retention_chunked");
}
