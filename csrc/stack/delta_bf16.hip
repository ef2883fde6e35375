// The delta rule over runs of tokens with bf16 activations.
#include "delta_chunk.h"

namespace nls_gla {

int delta_scan_bf16(const GA& p, int nruns, int nt, hipStream_t st) { return delta_d<__bf16>(p, nruns, nt, st); }

}  // namespace nls_gla
