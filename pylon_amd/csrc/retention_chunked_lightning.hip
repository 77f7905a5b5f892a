// The chunked kernels of lightning attention (retention_chunked.h, FORM 1).
#include "retention_chunked.h"

void pylon_lightning_chunked_run(RC_RUN_ARGS) {
  retention_chunked_run<1>(out, proj, ld, q_off, k_off, v_off, g_off, state, decay, inv_freq, rot_dims, positions,
                           row_start, row_slots, rows, heads, dim, vdim, eps, k_scale, chunk_state, max_chunks, span,
                           stream);
}
