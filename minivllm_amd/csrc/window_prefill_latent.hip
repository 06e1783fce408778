// Windowed prefill, tiled kernels for keys with a part of each head's own and one that all heads share, and values of their own.
#include "window_prefill.h"

namespace mvllm {

template <int KS2>
static int launch_for_dim(const WindowPrefillArgs& a, hipStream_t s) {
  switch (a.dim) {
    case 32: return launch_window_prefill<2, KS2, 1, false>(a, s);
    case 64: return launch_window_prefill<4, KS2, 2, false>(a, s);
    case 96: return launch_window_prefill<6, KS2, 3, false>(a, s);
    case 128: return launch_window_prefill<8, KS2, 4, false>(a, s);
    case 192: return launch_window_prefill<12, KS2, 6, false>(a, s);
    case 256: return launch_window_prefill<16, KS2, 8, false>(a, s);
    default: return kNoTiles;
  }
}

int launch_window_prefill_parts(const WindowPrefillArgs& a, hipStream_t stream) {
  return a.rot == 32 ? launch_for_dim<2>(a, stream) : a.rot == 64 ? launch_for_dim<4>(a, stream) : kNoTiles;
}

}  // namespace mvllm
