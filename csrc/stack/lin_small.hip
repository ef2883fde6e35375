// Few-row linear layers (decode, small prompt portions, routed experts with few rows): one workgroup per RT tiles of 16
// weight rows, its waves split K (interleaved 1 KiB sub-tiles, so the workgroup streams the tiles' weights sequentially)
// and meet in LDS. With several activation tiles RT > 1 pays: the activations are read once per RT tiles. The weights are the MFMA's row operand, so a lane ends with 4 consecutive output columns of one row.
#include "lin.h"

namespace nls_lin {

template <typename T, int MT, int NW, int RT>
__global__ __launch_bounds__(64 * NW) void lin_small_kernel(LinArgs a) {
  __shared__ f32x4 red[NW][RT * MT][64];
  constexpr int U = RT * MT >= 8 ? 2 : 4;    // sub-tiles in flight per wave
  typedef LT<T> L;
  LinTile t;
  if (!lin_tile<16 * RT, 16 * MT>(a, blockIdx.x, t)) return;
  const LinSeg& S = a.s[t.seg];
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int r = lane & 15, g = lane >> 4;
  const int nsub = S.nsub, nwt = (S.N + 15) >> 4;
  const int kb = nsub * t.ks / S.ks, ke = nsub * (t.ks + 1) / S.ks;         // this split's sub-tiles
  const uint8_t* wp[RT];
#pragma unroll
  for (int q = 0; q < RT; ++q)               // (a tile past the matrix: its last one again, not stored)
    wp[q] = (const uint8_t*)S.w + (size_t)t.grp * S.wstride + (size_t)min((t.n0 >> 4) + q, nwt - 1) * nsub * 1024 + lane * 16;
  const T* xp[MT];
#pragma unroll
  for (int i = 0; i < MT; ++i) {
    int xr, yr;
    lin_row(S, t, 16 * i + r, xr, yr);
    xp[i] = (const T*)S.x + (size_t)xr * S.ldx + (size_t)t.grp * S.xgs + L::EL * g;
  }
  f32x4 acc[RT][MT];
#pragma unroll
  for (int q = 0; q < RT; ++q)
#pragma unroll
    for (int i = 0; i < MT; ++i) acc[q][i] = f32x4{0.f, 0.f, 0.f, 0.f};
  int k = kb + wave;
  for (; k + (U - 1) * NW < ke; k += U * NW) {
    u32x4 w[U][RT], x[U][MT];
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int q = 0; q < RT; ++q) w[u][q] = ld16_nt(wp[q] + (size_t)(k + u * NW) * 1024);
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int i = 0; i < MT; ++i) x[u][i] = ld16(xp[i] + (size_t)(k + u * NW) * L::KS);
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int q = 0; q < RT; ++q)
#pragma unroll
        for (int i = 0; i < MT; ++i) acc[q][i] = L::mma(w[u][q], x[u][i], acc[q][i]);
  }
  for (; k < ke; k += NW) {
#pragma unroll
    for (int i = 0; i < MT; ++i) {
      const u32x4 x = ld16(xp[i] + (size_t)k * L::KS);
#pragma unroll
      for (int q = 0; q < RT; ++q) acc[q][i] = L::mma(ld16_nt(wp[q] + (size_t)k * 1024), x, acc[q][i]);
    }
  }
#pragma unroll
  for (int q = 0; q < RT; ++q)
#pragma unroll
    for (int i = 0; i < MT; ++i) red[wave][q * MT + i][lane] = acc[q][i];
  __syncthreads();
  for (int j = wave; j < RT * MT; j += NW) {
    const int q = j / MT, i = j % MT;
    f32x4 v = red[0][j][lane];
#pragma unroll
    for (int w = 1; w < NW; ++w) v += red[w][j][lane];
    if (16 * i + r < t.cnt) {
      int xr, yr;
      lin_row(S, t, 16 * i + r, xr, yr);
      lin_store4<T>(S, t.grp, t.ks, t.n0 + 16 * q + 4 * g, yr, v);
    }
  }
}

template <typename T, int MT, int NW, int RT>
int small_t(LinArgs& a, hipStream_t st) {
  const int n = lin_count(a, 16 * RT, 16 * MT);
  if (n < 1) return -1;
  hipLaunchKernelGGL((lin_small_kernel<T, MT, NW, RT>), dim3(n), dim3(64 * NW), 0, st, a);
  return (int)hipGetLastError();
}

template <typename T>
int small_d(LinArgs& a, int mt, int nw, int rt, hipStream_t st) {
#define NLS_LS(M, W, R) \
  if (mt == M && nw == W && rt == R) return small_t<T, M, W, R>(a, st);
  NLS_LS(1, 4, 1) NLS_LS(1, 8, 1) NLS_LS(1, 16, 1) NLS_LS(1, 4, 2) NLS_LS(1, 8, 2)
  NLS_LS(2, 4, 1) NLS_LS(2, 8, 1) NLS_LS(2, 4, 2) NLS_LS(2, 8, 2) NLS_LS(2, 4, 4)
  NLS_LS(4, 4, 1) NLS_LS(4, 8, 1) NLS_LS(4, 4, 2) NLS_LS(4, 8, 2) NLS_LS(4, 4, 4)
#undef NLS_LS
  return -1;
}

}  // namespace nls_lin

extern "C" {

int nls_lin_args_size() { return (int)sizeof(nls_lin::LinArgs); }

// f32: 1 = f32 operands, 0 = bf16. mt: 16-row tiles per workgroup (1, 2, 4); nw: waves (4, 8, 16); rt: 16-row weight
// tiles per workgroup (1, 2, 4)
int nls_lin_small(const void* args, int f32, int mt, int nw, int rt, void* stream) {
  nls_lin::LinArgs a = *reinterpret_cast<const nls_lin::LinArgs*>(args);
  return f32 ? nls_lin::small_d<float>(a, mt, nw, rt, (hipStream_t)stream)
             : nls_lin::small_d<__bf16>(a, mt, nw, rt, (hipStream_t)stream);
}

}  // extern "C"
