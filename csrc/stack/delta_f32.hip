// The delta rule over runs of tokens with f32 activations.
#include "delta_chunk.h"

namespace nls_gla {

int delta_scan_f32(const GA& p, int nruns, int nt, hipStream_t st) { return delta_d<float>(p, nruns, nt, st); }

}  // namespace nls_gla
