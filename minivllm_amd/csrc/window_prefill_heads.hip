// Windowed prefill, tiled kernels for ordinary grouped heads: keys and values of their own, nothing that all heads share.
#include "window_prefill.h"

namespace mvllm {

int launch_window_prefill_heads(const WindowPrefillArgs& a, hipStream_t s) {
  switch (a.dim) {
    case 32: return launch_window_prefill<2, 0, 1, false>(a, s);
    case 64: return launch_window_prefill<4, 0, 2, false>(a, s);
    case 96: return launch_window_prefill<6, 0, 3, false>(a, s);
    case 128: return launch_window_prefill<8, 0, 4, false>(a, s);
    case 192: return launch_window_prefill<12, 0, 6, false>(a, s);
    case 256: return launch_window_prefill<16, 0, 8, false>(a, s);
    default: return kNoTiles;
  }
}

}  // namespace mvllm
