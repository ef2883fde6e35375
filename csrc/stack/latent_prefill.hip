// Prompt attention of latent-attention layers (bf16, gfx950): for runs of many tokens the per-head keys and values are
// expanded once from the cached latents (a GEMM over the run's context, ops/stack.py) and this kernel is a causal flash
// attention over them; the rotated key part, shared by all heads, is read from the cache rows themselves. Short runs and
// decoded tokens attend in the latent space instead (latent_attn.hip).
//
// Workgroup = (head, block of 32 * NWV query tokens of one run), one wave per 32 tokens; every 64-key tile staged in LDS
// serves all of them. Per tile and wave, with v_mfma_f32_32x32x16_bf16:
//   S^T = K Q^T: lane l owns token l & 31 and, per 32-key block, keys (r & 3) + 8 (r >> 2) + 4 (l >> 5): the row maximum
//   closes with one lane exchange; P^T goes from those registers straight into O^T += V^T P^T (V^T by transposed LDS
//   reads in the same key order), so a token's rescale is lane-local and skipped when no maximum grew.
// The next tile's loads are in flight in registers while a tile computes; one barrier per tile, two LDS buffers. Rows are
// padded in LDS (K: 16 bytes, V: 64) against bank conflicts. The epilogue applies the head's output gate.
#include "../kernels/common.h"

namespace nls_lpf {

typedef float f32x16 __attribute__((ext_vector_type(16)));
typedef short s16x4 __attribute__((ext_vector_type(4)));
typedef short s16x8 __attribute__((ext_vector_type(8)));

// context rows of the expanded runs: xmap[xoff + p] = cache slot of position p. spans [n][8]: (first row, rows, sequence,
// first position, xoff, context, -, -). actx (optional): the rows' key counts with the spans' rows cleared.
__global__ __launch_bounds__(256) void expand_plan_kernel(const int* __restrict__ spans, const int* __restrict__ bt, int bts,
                                                          int bs, int* __restrict__ xmap, int* __restrict__ actx) {
  const int* s = spans + 8 * blockIdx.x;
  const int* b = bt + (size_t)s[2] * bts;
  for (int p = blockIdx.y * 256 + threadIdx.x; p < s[5]; p += gridDim.y * 256) xmap[s[4] + p] = b[p / bs] * bs + p % bs;
  if (actx)
    for (int i = blockIdx.y * 256 + threadIdx.x; i < s[1]; i += gridDim.y * 256) actx[s[0] + i] = 0;
}

struct LP {
  const __bf16* qn;       // unrotated queries [T][ldqn], head stride qns
  const __bf16* qr;       // rotated queries [T][ldqr], head stride qrs (pointer at the rotated part of head 0)
  const __bf16* kx;       // expanded keys [context rows][H * DKU]
  const __bf16* vx;       // expanded values [context rows][H * DV]
  const __bf16* cache;    // cache rows at their rotated part
  const int* xmap;
  const int* blocks;      // [n][8]: (first row, rows, sequence, first position, xoff, -, -, -), heaviest first
  const float* gate;      // [T][H]
  __bf16* out;            // [T][ldo], head stride vdim
  long ldqn, ldqr, ldc, ldo;
  int qns, qrs, H, vdim, ldg;
  float scale;
};

template <int NKU, int NKR, int NDB, int NWV>      // 32-column units: keys unrotated / rotated, values; waves
__global__ __launch_bounds__(64 * NWV) void latent_prefill_kernel(LP p) {
  constexpr int NT = 64 * NWV, KT = 64;
  constexpr int DKU = 32 * NKU, DR = 32 * NKR, DK = DKU + DR, DV = 32 * NDB;
  constexpr int KROW = DK * 2 + 16, VROW = DV * 2 + (NDB > 1 ? 64 : 0);
  constexpr int TB = KT * (KROW + VROW);
  constexpr int CU = DKU / 8, CR = DR / 8, CV = DV / 8, CPR = CU + CR + CV;   // 16-byte chunks per key
  constexpr int NLD = (KT * CPR + NT - 1) / NT;
  constexpr int NKS = DK / 16;
  extern __shared__ __attribute__((aligned(16))) uint8_t lds[];              // [2][K tile | V tile]

  const int head = blockIdx.x % p.H;
  const int* blk = p.blocks + 8 * (blockIdx.x / p.H);
  const int t0 = blk[0], ntok = blk[1], pos0 = blk[3], xoff = blk[4];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = lane >> 5, tl = lane & 31;
  const int tw0 = 32 * wave;
  const float sl2 = p.scale * 1.4426950408889634f;
  const int nkeys = pos0 + ntok, ntile = (nkeys + KT - 1) / KT;
  const int wlast = pos0 + min(tw0 + 31, ntok - 1);
  const bool wact = tw0 < ntok;
  const int qpos = pos0 + tw0 + tl;

  bf16x8 qf[NKS];
  {
    const size_t row = (size_t)(t0 + min(tw0 + tl, ntok - 1));
    const __bf16* a = p.qn + row * p.ldqn + (size_t)head * p.qns + 8 * h;
    const __bf16* b = p.qr + row * p.ldqr + (size_t)head * p.qrs + 8 * h;
#pragma unroll
    for (int ks = 0; ks < NKS; ++ks)
      qf[ks] = *reinterpret_cast<const bf16x8*>(ks < 2 * NKU ? a + 16 * ks : b + 16 * (ks - 2 * NKU));
  }

  u32x4 st[NLD];
  auto load_tile = [&](int t) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < NLD; ++i) {
      const int e = tid + NT * i;
      u32x4 v = u32x4{0u, 0u, 0u, 0u};
      if (e < KT * CU) {
        const int key = t * KT + e / CU;
        if (key < nkeys) v = ld16(p.kx + ((size_t)(xoff + key) * p.H + head) * DKU + (e % CU) * 8);
      } else if (e < KT * (CU + CR)) {
        const int f = e - KT * CU, key = t * KT + f / CR;
        if (key < nkeys) v = ld16(p.cache + (size_t)p.xmap[xoff + key] * p.ldc + (f % CR) * 8);
      } else if (e < KT * CPR) {
        const int f = e - KT * (CU + CR), key = t * KT + f / CV;
        if (key < nkeys) v = ld16(p.vx + ((size_t)(xoff + key) * p.H + head) * DV + (f % CV) * 8);
      }
      st[i] = v;
    }
  };
  auto store_tile = [&](int buf) __attribute__((always_inline)) {
    uint8_t* kb = lds + buf * TB;
    uint8_t* vb = kb + KT * KROW;
#pragma unroll
    for (int i = 0; i < NLD; ++i) {
      const int e = tid + NT * i;
      uint8_t* d;
      if (e < KT * CU) d = kb + (e / CU) * KROW + (e % CU) * 16;
      else if (e < KT * (CU + CR)) d = kb + ((e - KT * CU) / CR) * KROW + DKU * 2 + ((e - KT * CU) % CR) * 16;
      else d = vb + ((e - KT * (CU + CR)) / CV) * VROW + ((e - KT * (CU + CR)) % CV) * 16;
      if (KT * CPR % NT == 0 || e < KT * CPR) *reinterpret_cast<u32x4*>(d) = st[i];
    }
  };

  f32x16 o[NDB];
#pragma unroll
  for (int i = 0; i < NDB; ++i) o[i] = f32x16{};
  float m = -INFINITY, l = 0.f;
  load_tile(0);
  store_tile(0);
  __syncthreads();
  const int vq = (lane & 15) >> 2, vp = lane & 3, vhalf = (lane >> 4) & 1;
  for (int t = 0; t < ntile; ++t) {
    const int cur = t & 1, k0 = t * KT;
    if (t + 1 < ntile) load_tile(t + 1);
    if (wact && k0 <= wlast) {
      const uint8_t* kb = lds + cur * TB;
      const uint8_t* vb = kb + KT * KROW;
      f32x16 s[2];
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        s[u] = f32x16{};
        const uint8_t* krow = kb + (32 * u + tl) * KROW + 16 * h;
#pragma unroll
        for (int ks = 0; ks < NKS; ++ks)
          s[u] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*reinterpret_cast<const bf16x8*>(krow + 32 * ks), qf[ks], s[u], 0,
                                                         0, 0);
      }
      float mx = -INFINITY;
      if (k0 + KT - 1 > pos0 + tw0) {
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
          for (int r = 0; r < 16; ++r) {
            const int key = k0 + 32 * u + (r & 3) + 8 * (r >> 2) + 4 * h;
            s[u][r] = key <= qpos ? s[u][r] : -INFINITY;
            mx = fmaxf(mx, s[u][r]);
          }
      } else {
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
          for (int r = 0; r < 16; ++r) mx = fmaxf(mx, s[u][r]);
      }
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      const float mn = fmaxf(m, mx);
      if (!__all(mn == m)) {
        const float alpha = mn == -INFINITY ? 1.f : __builtin_amdgcn_exp2f((m - mn) * sl2);
        l *= alpha;
#pragma unroll
        for (int db = 0; db < NDB; ++db) o[db] *= alpha;
        m = mn;
      }
      const float nb = m == -INFINITY ? 0.f : -m * sl2;
#pragma unroll
      for (int ks = 0; ks < 4; ++ks) {
        const int u = ks >> 1, r0 = 8 * (ks & 1);
        bf16x8 pb;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const float e = __builtin_amdgcn_exp2f(fmaf(s[u][r0 + j], sl2, nb));
          l += e;
          pb[j] = (__bf16)e;
        }
        const int kbase = 32 * u + 16 * (ks & 1) + 4 * h;
#pragma unroll
        for (int db = 0; db < NDB; ++db) {
          const int col = 64 * db + 32 * vhalf + 8 * vp;       // bytes
          const s16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
              (__attribute__((address_space(3))) s16x4*)(vb + (kbase + vq) * VROW + col));
          const s16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
              (__attribute__((address_space(3))) s16x4*)(vb + (kbase + 8 + vq) * VROW + col));
          const s16x8 a8 = __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7);
          o[db] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, a8), pb, o[db], 0, 0, 0);
        }
      }
    }
    if (t + 1 < ntile) store_tile(cur ^ 1);                     // that buffer was last read in tile t - 1
    __syncthreads();
  }
  l += __shfl_xor(l, 32, 64);
  const int tok = tw0 + tl;
  if (!wact || tok >= ntok) return;
  // lane holds O[token][32 db + 8 g + 4 h + 0 .. 3] in o[db][4 g ..]
  const float f = (l > 0.f ? 1.f / l : 0.f) * p.gate[(size_t)(t0 + tok) * p.ldg + head];
  __bf16* y = p.out + (size_t)(t0 + tok) * p.ldo + (size_t)head * p.vdim;
  const bool vec = (p.vdim & 3) == 0;
#pragma unroll
  for (int db = 0; db < NDB; ++db)
#pragma unroll
    for (int g = 0; g < 4; ++g) {
      const int c = 32 * db + 8 * g + 4 * h;
      typedef __bf16 bf4 __attribute__((ext_vector_type(4)));
      const bf4 b = {(__bf16)(o[db][4 * g] * f), (__bf16)(o[db][4 * g + 1] * f), (__bf16)(o[db][4 * g + 2] * f),
                     (__bf16)(o[db][4 * g + 3] * f)};
      if (vec) {
        if (c < p.vdim) *reinterpret_cast<bf4*>(y + c) = b;
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (c + e < p.vdim) y[c + e] = b[e];
      }
    }
}

template <int NKU, int NKR, int NDB, int NWV>
int launch_t(const LP& p, int nblocks, hipStream_t st) {
  constexpr int LDS = 2 * 64 * (32 * (NKU + NKR) * 2 + 16 + 32 * NDB * 2 + (NDB > 1 ? 64 : 0));
  static bool attr = false;
  if (!attr) {
    if (hipFuncSetAttribute((const void*)latent_prefill_kernel<NKU, NKR, NDB, NWV>,
                            hipFuncAttributeMaxDynamicSharedMemorySize, LDS) != hipSuccess)
      return -1;
    attr = true;
  }
  hipLaunchKernelGGL((latent_prefill_kernel<NKU, NKR, NDB, NWV>), dim3(nblocks * p.H), dim3(64 * NWV), LDS, st, p);
  return (int)hipGetLastError();
}

}  // namespace nls_lpf

extern "C" {
using namespace nls_lpf;

int nls_expand_plan(const int* spans, int nspans, int maxctx, const int* bt, int bts, int bs, int* xmap, int* actx,
                    void* stream) {
  if (nspans < 1 || maxctx < 1 || bs < 1) return -1;
  hipLaunchKernelGGL(expand_plan_kernel, dim3(nspans, min((maxctx + 255) / 256, 64)), dim3(256), 0, (hipStream_t)stream,
                     spans, bt, bts, bs, xmap, actx);
  return (int)hipGetLastError();
}

// dku, dr, dv: expanded widths per head: dku, dv in {32, 64, 128}, dr in {32, 64}; waves 4 or 8 (blocks of 32 * waves rows)
int nls_latent_prefill(const void* qn, long ldqn, int qns, const void* qr, long ldqr, int qrs, const void* kx,
                       const void* vx, const void* cache, long ldc, const int* xmap, const int* blocks, int nblocks,
                       const float* gate, int ldg, void* out, long ldo, int H, int dku, int dr, int dv, int vdim,
                       int waves, float scale, void* stream) {
  if (nblocks < 1 || H < 1 || vdim < 1 || vdim > dv) return -1;
  LP p{(const __bf16*)qn, (const __bf16*)qr, (const __bf16*)kx, (const __bf16*)vx, (const __bf16*)cache, xmap, blocks,
       gate, (__bf16*)out, ldqn, ldqr, ldc, ldo, qns, qrs, H, vdim, ldg, scale};
  hipStream_t st = (hipStream_t)stream;
#define NLS_LP(U, R, V) \
  if (dku == 32 * U && dr == 32 * R && dv == 32 * V) \
    return waves == 8 ? launch_t<U, R, V, 8>(p, nblocks, st) : waves == 4 ? launch_t<U, R, V, 4>(p, nblocks, st) : -1;
#define NLS_LPV(U, R) NLS_LP(U, R, 1) NLS_LP(U, R, 2) NLS_LP(U, R, 4)
  NLS_LPV(1, 1) NLS_LPV(2, 1) NLS_LPV(4, 1) NLS_LPV(1, 2) NLS_LPV(2, 2) NLS_LPV(4, 2)
#undef NLS_LPV
#undef NLS_LP
  return -1;
}

}  // extern "C"
