// The extended forms of the windowed paged attention (attn_window.inc, MODE 1 and 2): the query heads of
// a key / value head share a tile, pooled blocks before the window, sigmoid weights, an output gate and
// a strided output. A file of its own so that its instantiations compile beside those of mixers.hip.
#include <algorithm>

#include "bfly_common.h"
#include "bfly_mixers.h"

namespace bfly {

#include "attn_window.inc"

bool launch_attn_window_mfma_ext(const void* q, long q_ld, const void* k_cache, const void* v_cache, const int* tables,
                                 int max_blocks, const int* row_cu, int nseq, const int* positions, float scale,
                                 int window, int keep_first, const float* sink, const float* out_scale, void* out, int T,
                                 int H, int G, int D, int Dv, int block_size, float* part, long part_floats,
                                 hipStream_t s, const AttnMod& md) {
  if (md.sigmoid)
    return attn_mfma_launch<2>(q, q_ld, k_cache, v_cache, tables, max_blocks, row_cu, nseq, positions, scale, window,
                               keep_first, nullptr, out_scale, out, T, H, G, D, Dv, block_size, false, part, part_floats,
                               s, md);
  return attn_mfma_launch<1>(q, q_ld, k_cache, v_cache, tables, max_blocks, row_cu, nseq, positions, scale, window,
                             keep_first, sink, out_scale, out, T, H, G, D, Dv, block_size, false, part, part_floats, s, md);
}

}  // namespace bfly
