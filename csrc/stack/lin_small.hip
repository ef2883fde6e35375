// Few-row linear layers (decode, small prompt portions, routed experts with few rows): one workgroup per 16 weight
// rows, its waves split K (interleaved 1 KiB sub-tiles, so the workgroup streams the tile's weights sequentially) and
// meet in LDS. The weights are the MFMA's row operand, so a lane ends with 4 consecutive output columns of one row.
#include "lin.h"

namespace nls_lin {

template <typename T, int MT, int NW>
__global__ __launch_bounds__(64 * NW) void lin_small_kernel(LinArgs a) {
  __shared__ f32x4 red[NW][MT][64];
  constexpr int U = 4;                       // sub-tiles in flight per wave
  typedef LT<T> L;
  LinTile t;
  if (!lin_tile<16, 16 * MT>(a, blockIdx.x, t)) return;
  const LinSeg& S = a.s[t.seg];
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int r = lane & 15, g = lane >> 4;
  const int nsub = S.nsub;
  const uint8_t* wp = (const uint8_t*)S.w + (size_t)t.grp * S.wstride + (size_t)(t.n0 >> 4) * nsub * 1024 + lane * 16;
  const T* xp[MT];
#pragma unroll
  for (int i = 0; i < MT; ++i) {
    int xr, yr;
    lin_row(S, t, 16 * i + r, xr, yr);
    xp[i] = (const T*)S.x + (size_t)xr * S.ldx + (size_t)t.grp * S.xgs + L::EL * g;
  }
  f32x4 acc[MT];
#pragma unroll
  for (int i = 0; i < MT; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  int k = wave;
  for (; k + (U - 1) * NW < nsub; k += U * NW) {
    u32x4 w[U], x[U][MT];
#pragma unroll
    for (int u = 0; u < U; ++u) w[u] = ld16_nt(wp + (size_t)(k + u * NW) * 1024);
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int i = 0; i < MT; ++i) x[u][i] = ld16(xp[i] + (size_t)(k + u * NW) * L::KS);
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int i = 0; i < MT; ++i) acc[i] = L::mma(w[u], x[u][i], acc[i]);
  }
  for (; k < nsub; k += NW) {
    const u32x4 w = ld16_nt(wp + (size_t)k * 1024);
#pragma unroll
    for (int i = 0; i < MT; ++i) acc[i] = L::mma(w, ld16(xp[i] + (size_t)k * L::KS), acc[i]);
  }
#pragma unroll
  for (int i = 0; i < MT; ++i) red[wave][i][lane] = acc[i];
  __syncthreads();
  for (int i = wave; i < MT; i += NW) {
    f32x4 v = red[0][i][lane];
#pragma unroll
    for (int w = 1; w < NW; ++w) v += red[w][i][lane];
    if (16 * i + r < t.cnt) {
      int xr, yr;
      lin_row(S, t, 16 * i + r, xr, yr);
      lin_store4<T>(S, t.grp, t.n0 + 4 * g, yr, v);
    }
  }
}

template <typename T, int MT, int NW>
int small_t(LinArgs& a, hipStream_t st) {
  const int n = lin_count(a, 16, 16 * MT);
  if (n < 1) return -1;
  hipLaunchKernelGGL((lin_small_kernel<T, MT, NW>), dim3(n), dim3(64 * NW), 0, st, a);
  return (int)hipGetLastError();
}

template <typename T>
int small_d(LinArgs& a, int mt, int nw, hipStream_t st) {
#define NLS_LS(M, W) \
  if (mt == M && nw == W) return small_t<T, M, W>(a, st);
  NLS_LS(1, 4) NLS_LS(1, 8) NLS_LS(1, 16) NLS_LS(2, 4) NLS_LS(2, 8) NLS_LS(4, 4) NLS_LS(4, 8)
#undef NLS_LS
  return -1;
}

}  // namespace nls_lin

extern "C" {

int nls_lin_args_size() { return (int)sizeof(nls_lin::LinArgs); }

// f32: 1 = f32 operands, 0 = bf16. mt: 16-row tiles per workgroup (1, 2, 4); nw: waves (4, 8, 16)
int nls_lin_small(const void* args, int f32, int mt, int nw, void* stream) {
  nls_lin::LinArgs a = *reinterpret_cast<const nls_lin::LinArgs*>(args);
  return f32 ? nls_lin::small_d<float>(a, mt, nw, (hipStream_t)stream)
             : nls_lin::small_d<__bf16>(a, mt, nw, (hipStream_t)stream);
}

}  // extern "C"
