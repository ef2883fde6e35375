// Gated delta rule over runs of tokens (gfx950): the launches of gla_chunk.h's kernels with the delta rule, and the chain of the
// segments' states. One source per activation type (delta_bf16.hip, delta_f32.hip) holds its kernels.
#pragma once
#include "gla_chunk.h"

namespace nls_gla {

// ---- the states that the segments of each run start from, in the place of their end states: S_(z + 1) = M_z S_z + S_local,z. A
// workgroup per (run, head, 16 columns); its waves share the rows' tiles, the state is handed over in LDS.
template <int DP>
__global__ __launch_bounds__(256) void delta_chain_kernel(GA p) {
  constexpr int NTD = DP / 16;
  __shared__ float sh[2][DP][17];
  const int* run = p.runs + 4 * blockIdx.y;
  const int n = run[1], slot = run[2];
  if (slot < 0 || n < 1) return;
  const int D = p.D, V = p.V, ncb = (V + 15) / 16, head = blockIdx.x / ncb, c0 = (blockIdx.x % ncb) * 16;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), r = lane & 15, g = lane >> 4;
  const int m = (n + seg_len(n, p.nseg) - 1) / seg_len(n, p.nseg);
  const size_t sst = (size_t)p.H * D * V, smt = (size_t)p.H * D * D;
  float* rec = p.rec + (size_t)blockIdx.y * p.nseg * sst + (size_t)head * D * V;
  const float* rm = p.recm + (size_t)blockIdx.y * p.nseg * smt + (size_t)head * D * D;
  const float* st = p.state + (size_t)slot * p.sstride + (size_t)head * D * V;
  for (int e = threadIdx.x; e < DP * 16; e += 256) {
    const int d = e >> 4, c = c0 + (e & 15);
    const float s = run[3] > 0 && d < D && c < V ? st[(size_t)d * V + c] : 0.f;
    sh[0][d][e & 15] = s;
  }
  __syncthreads();
  for (int z = 0; z < m; ++z) {
    const int cur = z & 1;
    if (z + 1 < m)
      for (int t = wave; t < NTD; t += 4) {
        f32x4 acc;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int d = 16 * t + 4 * g + i;
          const float l = rec[z * sst + (size_t)min(d, D - 1) * V + min(c0 + r, V - 1)];
          acc[i] = d < D && c0 + r < V ? l : 0.f;
        }
        const float* mr = rm + z * smt + (size_t)min(16 * t + r, D - 1) * D;
#pragma unroll
        for (int k = 0; k < NTD; ++k) {
          float a[4];
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int d = 16 * k + 4 * g + i;
            const float x = mr[min(d, D - 1)];
            a[i] = d < D && 16 * t + r < D ? x : 0.f;
          }
#pragma unroll
          for (int i = 0; i < 4; ++i) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], sh[cur][16 * k + 4 * g + i][r], acc, 0, 0, 0);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) sh[cur ^ 1][16 * t + 4 * g + i][r] = acc[i];
      }
    __syncthreads();                         // (every end state that this segment's place holds has been read)
    for (int e = threadIdx.x; e < D * 16; e += 256) {
      const int d = e >> 4, c = c0 + (e & 15);
      if (c < V) rec[z * sst + (size_t)d * V + c] = sh[cur][d][e & 15];
    }
    __syncthreads();
  }
}

template <typename T, int DP, int NT>
int delta_t(const GA& p, int nruns, hipStream_t st) {
  typedef GC<T, DP, NT, true, gc_chunks<T, DP, NT, true>()> C;
  static bool attr = false;
  if (!attr) {
    if (gla_lds<C::LDS>((const void*)gla_chunk_kernel<T, DP, NT, false, true>, (const void*)gla_chunk_kernel<T, DP, NT, true, true>))
      return -1;
    attr = true;
  }
  const int nv = (p.V + C::WC - 1) / C::WC, ni = (p.D + C::WC - 1) / C::WC;
  if (p.fused && p.V > C::WC) return -1;
  if (p.nseg > 1) {
    hipLaunchKernelGGL((gla_chunk_kernel<T, DP, NT, true, true>), dim3(p.H * (nv + ni), nruns, p.nseg - 1), dim3(256), C::LDS, st, p);
    hipLaunchKernelGGL(delta_chain_kernel<DP>, dim3(p.H * ((p.V + 15) / 16), nruns), dim3(256), 0, st, p);
  }
  hipLaunchKernelGGL((gla_chunk_kernel<T, DP, NT, false, true>), dim3(p.H * nv, nruns, p.nseg), dim3(256), C::LDS, st, p);
  return (int)hipGetLastError();
}

template <typename T>
int delta_d(const GA& p, int nruns, int nt, hipStream_t st) {
#define NLS_DD(DP) \
  if (p.D <= DP) return nt == 1 ? delta_t<T, DP, 1>(p, nruns, st) : nt == 2 ? delta_t<T, DP, 2>(p, nruns, st) : -1;
  NLS_DD(32) NLS_DD(64) NLS_DD(128) NLS_DD(256)
#undef NLS_DD
  return -1;
}

}  // namespace nls_gla
