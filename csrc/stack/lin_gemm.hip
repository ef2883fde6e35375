// Tiled MFMA GEMM on packed bf16 / f32 weights (prompt chunks, large decode batches, routed experts with many rows).
//
// BN weight rows x BM activation rows per workgroup; K advances two 1 KiB sub-tiles (64 bf16 / 32 f32 values) per
// step. Both operands arrive by LDS-DMA into NST-deep rings: weight sub-tiles verbatim (already in fragment order),
// activation sub-tiles with the 16-byte chunks of a row permuted on the DMA source (chunk ^ swz(row)), so every
// fragment is one conflict-free ds_read_b128. One raw barrier per step with a counted vmcnt leaves the later stages
// in flight. Routed rows (experts) are gathered by the DMA's per-lane source addresses.
// Tile ids are dealt to the 8 XCDs in contiguous ranges, a few m-tiles innermost (lin_tile): the workgroups that run
// together on an XCD form a block of weight and row tiles and read both through its L2.
#include "../kernels/lds_dma.h"
#include "lin.h"

namespace nls_lin {
using nls_dma::glds16;
using nls_dma::lds_addr;
using nls_dma::wait_vm_lgkm0;

DEVI int lin_swz(int r) { return (0x1320 >> (4 * ((r >> 2) & 3))) & 3; }

template <int BN, int BM, int WN, int WM, int NST>
struct LG {
  static constexpr int NWV = WN * WM;
  static constexpr int NTW = BN / 16 / WN;          // weight tiles per wave
  static constexpr int MTW = BM / 16 / WM;          // row tiles per wave
  static constexpr int WST = BN * 128, XST = BM * 128, STG = WST + XST;   // bytes per stage
  static constexpr int NW = BN / 8 / NWV, NX = BM / 8 / NWV;              // DMA instructions per wave per stage
  static constexpr int LDS = NST * STG;
  static_assert(NW >= 1 && NX >= 2 && NX % 2 == 0 && NTW >= 1 && MTW >= 1, "tile too small for the wave count");
  static_assert(LDS <= 160 * 1024, "LDS");
};

template <typename T, int BN, int BM, int WN, int WM, int NST>
__global__ __launch_bounds__(64 * WN * WM) void lin_gemm_kernel(LinArgs a, int ntot) {
  extern __shared__ __attribute__((aligned(16))) uint8_t lglds[];
  typedef LG<BN, BM, WN, WM, NST> G;
  typedef LT<T> L;
  constexpr int NW = G::NW, NX = G::NX, NTW = G::NTW, MTW = G::MTW;
  const int per = gridDim.x >> 3;
  const int id = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
  if (id >= ntot) return;
  LinTile t;
  if (!lin_tile<BN, BM>(a, id, t)) return;
  const LinSeg& S = a.s[t.seg];
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int r = lane & 15, g = lane >> 4;
  const int wn = wave / WM, wm = wave % WM;
  const int nsub = S.nsub;
  const int jb = (nsub >> 1) * t.ks / S.ks, nst = (nsub >> 1) * (t.ks + 1) / S.ks - jb;     // this split's steps
  const int nwt = (S.N + 15) >> 4;

  const uint8_t* wbase = (const uint8_t*)S.w + (size_t)t.grp * S.wstride + lane * 16;
  const uint8_t* wsrc[NW];
#pragma unroll
  for (int i = 0; i < NW; ++i) {
    const int q = NW * wave + i;                     // stage sub-tile: weight tile q >> 1, k half q & 1
    wsrc[i] = wbase + ((size_t)min((t.n0 >> 4) + (q >> 1), nwt - 1) * nsub + (q & 1)) * 1024;
  }
  const T* xsrc[NX / 2];
#pragma unroll
  for (int i = 0; i < NX / 2; ++i) {
    const int row = 16 * ((NX * wave) / 2 + i) + (lane >> 2);
    int xr, yr;
    lin_row(S, t, row, xr, yr);
    xsrc[i] = (const T*)S.x + (size_t)xr * S.ldx + (size_t)t.grp * S.xgs + ((lane & 3) ^ lin_swz(lane >> 2)) * L::EL;
  }
  const uint32_t base = __builtin_amdgcn_readfirstlane(lds_addr(lglds));
  const uint32_t wl = base + (uint32_t)(NW * wave) * 1024u;
  const uint32_t xl = base + G::WST + (uint32_t)(NX * wave) * 1024u;
  auto dma = [&](int j) __attribute__((always_inline)) {     // step j (clamped) -> stage j % NST
    const int jc = jb + min(j, nst - 1);
    const uint32_t so = (uint32_t)(j % NST) * G::STG;
#pragma unroll
    for (int i = 0; i < NW; ++i) glds16(wsrc[i] + (size_t)jc * 2048, wl + so + i * 1024);
#pragma unroll
    for (int i = 0; i < NX; ++i) glds16(xsrc[i >> 1] + (size_t)(2 * jc + (i & 1)) * L::KS, xl + so + i * 1024);
  };
  f32x4 acc[NTW][MTW];
#pragma unroll
  for (int i = 0; i < NTW; ++i)
#pragma unroll
    for (int j = 0; j < MTW; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int xfo = r * 64 + ((g ^ lin_swz(r)) << 4);
  auto step = [&](int j) __attribute__((always_inline)) {
    const uint8_t* wb = lglds + (j % NST) * G::STG + lane * 16;
    const uint8_t* xb = lglds + (j % NST) * G::STG + G::WST + xfo;
#pragma unroll
    for (int h = 0; h < 2; ++h) {
      u32x4 A[NTW], B[MTW];
#pragma unroll
      for (int i = 0; i < NTW; ++i) A[i] = *reinterpret_cast<const u32x4*>(wb + ((wn * NTW + i) * 2 + h) * 1024);
#pragma unroll
      for (int i = 0; i < MTW; ++i) B[i] = *reinterpret_cast<const u32x4*>(xb + ((wm * MTW + i) * 2 + h) * 1024);
#pragma unroll
      for (int i = 0; i < NTW; ++i)
#pragma unroll
        for (int jj = 0; jj < MTW; ++jj) acc[i][jj] = L::mma(A[i], B[jj], acc[i][jj]);
    }
  };
  constexpr int FL = (NST - 2) * (NW + NX);           // DMA instructions left in flight across the barrier
#pragma unroll
  for (int j = 0; j < NST - 1; ++j) dma(j);
  wait_vm_lgkm0<FL>();
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
  for (int j = 0; j < nst; ++j) {
    dma(j + NST - 1);                                 // that stage was last read in step j - 1: retired
    step(j);
    wait_vm_lgkm0<FL>();
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
  }
  wait_vm_lgkm0<0>();                                 // the clamped tail DMAs land before the workgroup's LDS is freed
#pragma unroll
  for (int j = 0; j < MTW; ++j) {
    const int row = 16 * (wm * MTW + j) + r;
    if (row >= t.cnt) continue;
    int xr, yr;
    lin_row(S, t, row, xr, yr);
#pragma unroll
    for (int i = 0; i < NTW; ++i) lin_store4<T>(S, t.grp, t.ks, t.n0 + 16 * (wn * NTW + i) + 4 * g, yr, acc[i][j]);
  }
}

template <typename T, int BN, int BM, int WN, int WM, int NST>
int gemm_t(LinArgs& a, hipStream_t st) {
  typedef LG<BN, BM, WN, WM, NST> G;
  const int n = lin_count(a, BN, BM);
  if (n < 1) return -1;
  static bool attr = false;
  if (!attr) {
    if (hipFuncSetAttribute((const void*)lin_gemm_kernel<T, BN, BM, WN, WM, NST>,
                            hipFuncAttributeMaxDynamicSharedMemorySize, G::LDS) != hipSuccess)
      return -1;
    attr = true;
  }
  hipLaunchKernelGGL((lin_gemm_kernel<T, BN, BM, WN, WM, NST>), dim3((n + 7) / 8 * 8), dim3(64 * G::NWV), G::LDS, st,
                     a, n);
  return (int)hipGetLastError();
}

template <typename T>
int gemm_d(LinArgs& a, int cfg, hipStream_t st) {
  switch (cfg) {
    case 0: return gemm_t<T, 64, 64, 2, 2, 3>(a, st);
    case 1: return gemm_t<T, 128, 64, 4, 1, 2>(a, st);
    case 2: return gemm_t<T, 128, 128, 2, 2, 2>(a, st);
    case 3: return gemm_t<T, 256, 128, 4, 2, 3>(a, st);
    case 4: return gemm_t<T, 256, 256, 4, 2, 2>(a, st);
    case 5: return gemm_t<T, 64, 64, 2, 2, 8>(a, st);
    case 6: return gemm_t<T, 192, 128, 4, 2, 3>(a, st);
  }
  return -1;
}

}  // namespace nls_lin

extern "C" {

// cfg: tile of the launch (BN x BM): 0 = 64 x 64, 1 = 128 x 64, 2 = 128 x 128, 3 = 256 x 128, 4 = 256 x 256,
// 5 = 64 x 64 with 8 stages in flight (launches of at most one workgroup per CU), 6 = 192 x 128
int nls_lin_gemm(const void* args, int f32, int cfg, void* stream) {
  nls_lin::LinArgs a = *reinterpret_cast<const nls_lin::LinArgs*>(args);
  return f32 ? nls_lin::gemm_d<float>(a, cfg, (hipStream_t)stream)
             : nls_lin::gemm_d<__bf16>(a, cfg, (hipStream_t)stream);
}

}  // extern "C"
