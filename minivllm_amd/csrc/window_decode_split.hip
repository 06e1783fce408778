// Windowed decode, tiled kernels for cached rows of a key and behind it a value of the same width.
#include "latent_decode.h"

namespace mvllm {

int launch_decode_split(const LatentDecodeArgs& a, int rows, hipStream_t s) {
  if (a.values != a.padded) return kNotBuilt;
  switch (a.padded) {
    case 32: return launch_decode_as<1, 1, true, true>(a, rows, s);
    case 64: return launch_decode_as<2, 2, true, true>(a, rows, s);
    case 96: return launch_decode_as<3, 3, true, true>(a, rows, s);
    case 128: return launch_decode_as<4, 4, true, true>(a, rows, s);
    case 192: return launch_decode_as<6, 6, true, true>(a, rows, s);
    case 256: return launch_decode_as<8, 8, true, true>(a, rows, s);
    default: return kNotBuilt;
  }
}

}  // namespace mvllm
