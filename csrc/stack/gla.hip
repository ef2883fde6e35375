// Gated linear attention (gfx950): entry points of its recurrence (scan.h). Keys and values may differ in width.
#include "scan.h"

namespace nls_gla {
using namespace nls_scan;

// cpl: value columns per lane (1: short chains, 4: fewer operand reads); parts: lanes that share a column's keys
template <typename T, int DP>
int scan_d(Scan p, int nruns, int parts, int cpl, hipStream_t st) {
#define NLS_GS(P, C) \
  if (parts == P && cpl == C) { \
    const int wc = 256 / P * C; \
    const dim3 grid(p.H * ((p.V + wc - 1) / wc), nruns, p.nseg - (p.nseg > 1)); \
    hipLaunchKernelGGL((scan_kernel<T, GLA, DP, P, C>), grid, dim3(256), 0, st, p); \
    if (p.nseg > 1) { \
      p.pass = 1; \
      hipLaunchKernelGGL((scan_kernel<T, GLA, DP, P, C>), grid, dim3(256), 0, st, p); \
    } \
    return (int)hipGetLastError(); \
  }
  if constexpr (DP <= 64) { NLS_GS(8, 1) NLS_GS(8, 4) }
  if constexpr (DP >= 64) { NLS_GS(16, 1) NLS_GS(16, 4) }
#undef NLS_GS
  return -1;
}

template <typename T>
int scan_t(const Scan& p, int nruns, int parts, int cpl, hipStream_t st) {
  if (p.D <= 32) return scan_d<T, 32>(p, nruns, parts, cpl, st);
  if (p.D <= 64) return scan_d<T, 64>(p, nruns, parts, cpl, st);
  if (p.D <= 128) return scan_d<T, 128>(p, nruns, parts, cpl, st);
  if (p.D <= 256) return scan_d<T, 256>(p, nruns, parts, cpl, st);
  return -1;
}

}  // namespace nls_gla

extern "C" {
using namespace nls_gla;

// nseg > 1: seg_s [nruns][nseg - 1][H][D][V] and seg_w [nruns][nseg - 1][H][D] scratch. D up to 256 ; parts 8: D up to 64, 16: above 32.
int nls_gla_scan(const void* q, const void* k, const void* v, long ld, const float* a, long lda, float qscale, float* o,
                 long ldo, float* state, long sstride, const int* runs, int nruns, int H, int D, int V, int nseg, float* seg_s,
                 float* seg_w, int parts, int cpl, int f32, void* stream) {
  if (nruns < 1 || H < 1 || D < 1 || V < 1 || nseg < 1 || nseg > 64 || (nseg > 1 && (!seg_s || !seg_w))) return -1;
  const Scan p{q, k, v, a, nullptr, o, state, nullptr, nullptr, runs, seg_s, seg_w, ld, lda, ldo, sstride, 0, 0, H, D, V, 0,
               nseg, 0, qscale};
  return f32 ? scan_t<float>(p, nruns, parts, cpl, (hipStream_t)stream)
             : scan_t<__bf16>(p, nruns, parts, cpl, (hipStream_t)stream);
}

// every run has one token (or none); V a multiple of 4, at most 1024; D at most 256
int nls_gla_step(const void* q, const void* k, const void* v, long ld, const float* a, long lda, float qscale, float* state,
                 long sstride, const int* runs, int nruns, const float* norm, const void* gate, long ldg, void* out, long ldout,
                 int H, int D, int V, float eps, int f32, void* stream) {
  const Scan p{q, k, v, a, nullptr, nullptr, state, nullptr, nullptr, runs, nullptr, nullptr, ld, lda, 0, sstride, 0, 0, H, D,
               V, 0, 1, 0, qscale};
  return f32 ? step_rows<float, GLA>(p, nruns, norm, gate, ldg, out, ldout, eps, (hipStream_t)stream)
             : step_rows<__bf16, GLA>(p, nruns, norm, gate, ldg, out, ldout, eps, (hipStream_t)stream);
}

}  // extern "C"
