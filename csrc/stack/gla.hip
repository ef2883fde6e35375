// Gated linear attention (gfx950): runs of tokens in chunks (gla_chunk.h) and the single-token step (scan.h). Decays come per
// token and channel, or (row stride 0) constant.
#include "gla_chunk.h"

namespace nls_gla {

// the states that the segments of each run start from, in the place of their end states
__global__ __launch_bounds__(256) void gla_chain_kernel(GA p) {
  const int* run = p.runs + 4 * blockIdx.y;
  const int n = run[1], slot = run[2];
  if (slot < 0 || n < 1) return;
  const size_t sst = (size_t)p.H * p.D * p.V, swt = (size_t)p.H * p.D;
  const int m = (n + seg_len(n, p.nseg) - 1) / seg_len(n, p.nseg);
  float* rec = p.rec + (size_t)blockIdx.y * p.nseg * sst;
  const float* rw = p.recw + (size_t)blockIdx.y * p.nseg * swt;
  for (size_t e = (size_t)blockIdx.x * 256 + threadIdx.x; e < sst; e += (size_t)gridDim.x * 256) {
    float s = run[3] > 0 ? p.state[(size_t)slot * p.sstride + e] : 0.f;
    const size_t w = e / p.V;
    for (int z = 0; z + 1 < m; ++z) {
      const float l = rec[z * sst + e];
      rec[z * sst + e] = s;
      s = fmaf(rw[z * swt + w], s, l);
    }
    rec[(size_t)(m - 1) * sst + e] = s;
  }
}

template <typename T, int DP, int NT>
int chunk_t(GA p, int nruns, hipStream_t st) {
  typedef GC<T, DP, NT, false, gc_chunks<T, DP, NT, false>()> C;
  static bool attr = false;
  if (!attr) {
    if (gla_lds<C::LDS>((const void*)gla_chunk_kernel<T, DP, NT, false, false>, (const void*)gla_chunk_kernel<T, DP, NT, true, false>))
      return -1;
    attr = true;
  }
  const int nx = p.H * ((p.V + C::WC - 1) / C::WC);
  if (p.fused && p.V > C::WC) return -1;
  if (p.nseg > 1) {
    hipLaunchKernelGGL((gla_chunk_kernel<T, DP, NT, true, false>), dim3(nx, nruns, p.nseg - 1), dim3(256), C::LDS, st, p);
    const long n = (long)p.H * p.D * p.V;
    hipLaunchKernelGGL(gla_chain_kernel, dim3((int)min((n + 255) / 256, 4096L), nruns), dim3(256), 0, st, p);
  }
  hipLaunchKernelGGL((gla_chunk_kernel<T, DP, NT, false, false>), dim3(nx, nruns, p.nseg), dim3(256), C::LDS, st, p);
  return (int)hipGetLastError();
}

template <typename T>
int chunk_d(const GA& p, int nruns, int nt, hipStream_t st) {
#define NLS_GC(DP) \
  if (p.D <= DP) return nt == 1 ? chunk_t<T, DP, 1>(p, nruns, st) : nt == 2 ? chunk_t<T, DP, 2>(p, nruns, st) : -1;
  NLS_GC(32) NLS_GC(64) NLS_GC(128) NLS_GC(256)
#undef NLS_GC
  return -1;
}

}  // namespace nls_gla

extern "C" {
using namespace nls_gla;

// nt: 64 nt value columns per workgroup (1, 2). norm and gate given: out = (o / rms(o) per head) * norm * gate, for V up to
// 64 nt; else o. nseg > 1: rec [nruns][nseg][H][D][V] and recw [nruns][nseg][H][D] scratch. D up to 256.
int nls_gla_scan(const void* q, const void* k, const void* v, long ld, const float* a, long lda, float qscale, float* o,
                 long ldo, const float* norm, const void* gate, long ldg, void* out, long ldout, float eps, float* state,
                 long sstride, const int* runs, int nruns, int H, int D, int V, int nseg, float* rec, float* recw, int nt,
                 int f32, void* stream) {
  const bool fused = norm && gate && out;
  if (nruns < 1 || H < 1 || D < 1 || V < 1 || nseg < 1 || nseg > 64 || (nseg > 1 && (!rec || !recw)) || (!fused && !o)) return -1;
  const GA p = gla_args(q, k, v, ld, a, lda, qscale, o, ldo, norm, gate, ldg, out, ldout, eps, state, sstride, runs, H, D, V, nseg,
                        rec, recw, f32);
  return f32 ? chunk_d<float>(p, nruns, nt, (hipStream_t)stream) : chunk_d<__bf16>(p, nruns, nt, (hipStream_t)stream);
}

// every run has one token (or none); V a multiple of 4, at most 1024; D at most 256. Decays: a, or (a null) from the low-rank
// gate input `low` (row stride ld, 16-byte aligned rows) with a2 [H * D][rank] in the activation type: sigmoid(a2 low + a2b)^ia
// norm null: the plain outputs o
int nls_gla_step(const void* q, const void* k, const void* v, long ld, const float* a, long lda, const void* low, const void* a2,
                 const float* a2b, int rank, float ia, float qscale, float* state, long sstride, const int* runs, int nruns,
                 const float* norm, const void* gate, long ldg, void* out, long ldout, float* o, long ldo, int H, int D, int V,
                 float eps, int f32, void* stream) {
  if (norm ? !gate || !out : !o) return -1;
  if (!a && (!low || !a2 || !a2b || rank < 1 || ((uintptr_t)low & 15) || ((uintptr_t)a2 & 15) || (ld & 7))) return -1;
  const Scan p{q, k, v, a, nullptr, o, state, nullptr, nullptr, runs, ld, lda, ldo, sstride, 0, 0, H, D, V, 0, qscale,
               low, a2, a2b, rank, ia};
  return f32 ? step_rows<float, GLA>(p, nruns, norm, gate, ldg, out, ldout, eps, (hipStream_t)stream)
             : step_rows<__bf16, GLA>(p, nruns, norm, gate, ldg, out, ldout, eps, (hipStream_t)stream);
}

}  // extern "C"
