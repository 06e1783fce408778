// Stand-ins for the kernel families a partial library leaves out (minivllm_amd/_build.py: build_part): every one of them
// says "not taken".  Weak, so that a family that is linked after all replaces its stand-in; the full library does not
// contain this file.
#include "prefill_mfma.h"

namespace mvllm {

__attribute__((weak)) bool prefill_pp_takes(int, int, int, int, int, int) { return false; }
__attribute__((weak)) int launch_prefill_pp(const PrefillPpArgs&, int, hipStream_t) { return MVLLM_ERR_UNSUPPORTED; }
__attribute__((weak)) bool prefill_mfma_other_dim(int) { return false; }
__attribute__((weak)) int launch_prefill_mfma_other(const PrefillArgs&, int, bool, hipStream_t) { return MVLLM_ERR_UNSUPPORTED; }
__attribute__((weak)) int launch_prefill_mfma_half_step(const PrefillArgs&, int, bool, hipStream_t) { return MVLLM_ERR_UNSUPPORTED; }

}  // namespace mvllm
