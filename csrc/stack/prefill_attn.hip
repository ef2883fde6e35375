// Prompt attention of the config-driven stacks (bf16, gfx950), a causal flash attention in two forms:
//   latent attention: the per-head keys and values of a run are expanded once from the cached latents (a GEMM over the run's
//     context, ops/stack.py); the rotated key part, shared by all heads, is read from the cache rows themselves.
//   grouped-query attention (no rotated part, NKR = 0): keys and values are the paged cache rows; the gs query heads of a key
//     head are rows beside each other (row = token * gs + head of the group), so any group size fills the MFMA tiles and a
//     tile staged in LDS serves the whole group.
// Short runs and decoded tokens attend row by row instead (latent_attn.hip, attn.hip).
//
// Workgroup = (key head, 32 * NWV rows of a block of one run's tokens), one wave per 32 rows; every 64-key tile staged in LDS
// serves all of them. Per tile and wave, with v_mfma_f32_32x32x16_bf16:
//   S^T = K Q^T: lane l owns row l & 31 and, per 32-key block, keys (r & 3) + 8 (r >> 2) + 4 (l >> 5): the row maximum
//   closes with one lane exchange; P^T goes from those registers straight into O^T += V^T P^T (V^T by transposed LDS
//   reads in the same key order), so a row's rescale is lane-local and skipped when no maximum grew.
// The next tile's loads are in flight in registers while a tile computes (its cache slots one tile ahead of that); one
// barrier per tile, two LDS buffers. Rows are padded in LDS (K: 16 bytes, V: 64) against bank conflicts. Under a sliding window
// (with kept first keys) tiles that no row sees are left out. The epilogue applies the head's output gate, if there is one.
#include "../kernels/common.h"

namespace nls_pfa {

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

struct FP {
  const __bf16* qn;       // queries (latent: their unrotated part) [T][ldqn], head stride qns
  const __bf16* qr;       // latent: rotated queries [T][ldqr], head stride qrs (pointer at the rotated part of head 0)
  const __bf16* kx;       // latent: expanded keys [context rows][H * DKU]; grouped: cache rows [slots][ldc], key heads DKU apart
  const __bf16* vx;       // values likewise (DV)
  const __bf16* cache;    // latent: cache rows at their rotated part
  const int* xmap;        // cache slot of every context row
  const int* blocks;      // [n][8]: (first row, rows, sequence, first position, xoff, -, -, -), heaviest first
  const float* gate;      // [T][H] (null: none)
  __bf16* out;            // [T][ldo], head stride vdim
  long ldqn, ldqr, ldc, ldo;
  int qns, qrs, H, vdim, ldg;
  int gs, nsub;           // grouped: query heads per key head; workgroups per block and key head
  float scale;
  int window, keep, sink; // position i sees j <= i if i - j < window or j < keep; sink: one more in the denominator
};
constexpr int NO_WINDOW = 1 << 30;

template <int NKU, int NKR, int NDB, int NWV>      // 32-column units: keys unrotated / rotated, values; waves
__global__ __launch_bounds__(64 * NWV) void flash_prefill_kernel(FP p) {
  constexpr bool PAGED = NKR == 0;
  static_assert(!PAGED || NKU == NDB, "grouped form: equal key and value widths");
  constexpr int NT = 64 * NWV, KT = 64;
  constexpr int DKU = 32 * NKU, DR = 32 * NKR, DK = DKU + DR, DV = 32 * NDB;
  constexpr int KROW = DK * 2 + 16, VROW = DV * 2 + (NDB > 1 ? 64 : 0);
  constexpr int TB = KT * (KROW + VROW);
  constexpr int CU = DKU / 8, CR = DR / 8, CV = DV / 8, CPR = CU + CR + CV;   // 16-byte chunks per key
  constexpr int NLK = (KT * CU + NT - 1) / NT;                               // grouped: chunks per thread of K, and of V
  constexpr int NLD = PAGED ? 2 * NLK : (KT * CPR + NT - 1) / NT;
  constexpr int NKS = DK / 16;
  extern __shared__ __attribute__((aligned(16))) uint8_t lds[];              // [2][K tile | V tile]

  const int HK = PAGED ? p.H / p.gs : p.H, gs = PAGED ? p.gs : 1;
  const int kh = blockIdx.x % HK, rest = blockIdx.x / HK;
  const int row0 = PAGED ? (p.nsub - 1 - rest % p.nsub) * 32 * NWV : 0;      // (later rows see more keys: they go first)
  const int* blk = p.blocks + 8 * (PAGED ? rest / p.nsub : rest);
  const int t0 = blk[0], ntok = blk[1], pos0 = blk[3], xoff = blk[4];
  const int nrow = ntok * gs;
  if (PAGED && row0 >= nrow) return;
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = lane >> 5, tl = lane & 31;
  const int tw0 = row0 + 32 * wave;
  const int myrow = min(tw0 + tl, nrow - 1), mytok = myrow / gs, head = PAGED ? kh * gs + myrow - mytok * gs : kh;
  const float sl2 = p.scale * 1.4426950408889634f;
  const int nkeys = pos0 + (min(row0 + 32 * NWV, nrow) - 1) / gs + 1, lowt = max(pos0 + row0 / gs - p.window + 1, 0) / KT;
  // tiles that no row sees are left out: `skip` of them behind the kept keys' `nkt`
  const int nkt = min((p.keep + KT - 1) / KT, lowt), skip = lowt - nkt, ntile = (nkeys + KT - 1) / KT - skip;
  auto tile = [&](int t) { return t < nkt ? t : t + skip; };
  const int wlast = pos0 + min(tw0 + 31, nrow - 1) / gs, wfirst = pos0 + tw0 / gs;
  const bool wact = tw0 < nrow;
  const int qpos = pos0 + mytok;

  bf16x8 qf[NKS];
  {
    const size_t row = (size_t)(t0 + mytok);
    const __bf16* a = p.qn + row * p.ldqn + (size_t)head * p.qns + 8 * h;
    const __bf16* b = p.qr + row * p.ldqr + (size_t)head * p.qrs + 8 * h;
#pragma unroll
    for (int ks = 0; ks < NKS; ++ks)
      qf[ks] = *reinterpret_cast<const bf16x8*>(ks < 2 * NKU ? a + 16 * ks : b + 16 * (ks - 2 * NKU));
  }
  int sl[PAGED ? NLK : 1];                                      // grouped: cache slots of the next tile's rows
  auto load_slots = [&](int t) __attribute__((always_inline)) {
    if constexpr (PAGED) {
#pragma unroll
      for (int i = 0; i < NLK; ++i) sl[i] = p.xmap[xoff + min(tile(t) * KT + (tid + NT * i) / CU, nkeys - 1)];
    }
  };
  load_slots(0);

  u32x4 st[NLD];
  auto load_tile = [&](int t) __attribute__((always_inline)) {
    if constexpr (PAGED) {
#pragma unroll
      for (int i = 0; i < NLK; ++i) {                           // (rows past the last key repeat it: masked below)
        const size_t o = (size_t)sl[i] * p.ldc + (size_t)kh * DKU + ((tid + NT * i) % CU) * 8;
        st[i] = ld16(p.kx + o);
        st[NLK + i] = ld16(p.vx + o);
      }
      return;
    }
#pragma unroll
    for (int i = 0; i < NLD; ++i) {
      const int e = tid + NT * i;
      u32x4 v = u32x4{0u, 0u, 0u, 0u};
      if (e < KT * CU) {
        const int key = tile(t) * KT + e / CU;
        if (key < nkeys) v = ld16(p.kx + ((size_t)(xoff + key) * p.H + kh) * DKU + (e % CU) * 8);
      } else if (e < KT * (CU + CR)) {
        const int f = e - KT * CU, key = tile(t) * KT + f / max(CR, 1);
        if (key < nkeys) v = ld16(p.cache + (size_t)p.xmap[xoff + key] * p.ldc + (f % max(CR, 1)) * 8);
      } else if (e < KT * CPR) {
        const int f = e - KT * (CU + CR), key = tile(t) * KT + f / CV;
        if (key < nkeys) v = ld16(p.vx + ((size_t)(xoff + key) * p.H + kh) * DV + (f % CV) * 8);
      }
      st[i] = v;
    }
  };
  auto store_tile = [&](int buf) __attribute__((always_inline)) {
    uint8_t* kb = lds + buf * TB;
    uint8_t* vb = kb + KT * KROW;
    if constexpr (PAGED) {
#pragma unroll
      for (int i = 0; i < NLK; ++i) {
        const int e = tid + NT * i;
        if (KT * CU % NT == 0 || e < KT * CU) {
          *reinterpret_cast<u32x4*>(kb + (e / CU) * KROW + (e % CU) * 16) = st[i];
          *reinterpret_cast<u32x4*>(vb + (e / CU) * VROW + (e % CU) * 16) = st[NLK + i];
        }
      }
      return;
    }
#pragma unroll
    for (int i = 0; i < NLD; ++i) {
      const int e = tid + NT * i;
      uint8_t* d;
      if (e < KT * CU) d = kb + (e / CU) * KROW + (e % CU) * 16;
      else if (e < KT * (CU + CR)) d = kb + ((e - KT * CU) / max(CR, 1)) * KROW + DKU * 2 + ((e - KT * CU) % max(CR, 1)) * 16;
      else d = vb + ((e - KT * (CU + CR)) / CV) * VROW + ((e - KT * (CU + CR)) % CV) * 16;
      if (KT * CPR % NT == 0 || e < KT * CPR) *reinterpret_cast<u32x4*>(d) = st[i];
    }
  };

  f32x16 o[NDB];
#pragma unroll
  for (int i = 0; i < NDB; ++i) o[i] = f32x16{};
  float m = p.sink ? 0.f : -INFINITY, l = p.sink && h == 0 ? 1.f : 0.f;       // (l: two lanes' shares of a row)
  load_tile(0);
  load_slots(1);
  store_tile(0);
  __syncthreads();
  const int vq = (lane & 15) >> 2, vp = lane & 3, vhalf = (lane >> 4) & 1;
  for (int t = 0; t < ntile; ++t) {
    const int cur = t & 1, k0 = tile(t) * KT;
    if (t + 1 < ntile) {
      load_tile(t + 1);
      load_slots(t + 2);
    }
    if (wact && k0 <= wlast && (k0 < p.keep || k0 + KT > wfirst - p.window + 1)) {
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
      if (k0 + KT - 1 > wfirst || (k0 <= wlast - p.window && k0 + KT > p.keep)) {
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
          for (int r = 0; r < 16; ++r) {
            const int key = k0 + 32 * u + (r & 3) + 8 * (r >> 2) + 4 * h;
            s[u][r] = key <= qpos && (key > qpos - p.window || key < p.keep) ? s[u][r] : -INFINITY;
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
  if (tw0 + tl >= nrow) return;
  // lane holds O[row][32 db + 8 g + 4 h + 0 .. 3] in o[db][4 g ..]
  const float f = (l > 0.f ? 1.f / l : 0.f) * (p.gate ? p.gate[(size_t)(t0 + mytok) * p.ldg + head] : 1.f);
  __bf16* y = p.out + (size_t)(t0 + mytok) * p.ldo + (size_t)head * p.vdim;
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
int launch_t(const FP& p, int nblocks, hipStream_t st) {
  constexpr int LDS = 2 * 64 * (32 * (NKU + NKR) * 2 + 16 + 32 * NDB * 2 + (NDB > 1 ? 64 : 0));
  static bool attr = false;
  if (!attr) {
    if (hipFuncSetAttribute((const void*)flash_prefill_kernel<NKU, NKR, NDB, NWV>,
                            hipFuncAttributeMaxDynamicSharedMemorySize, LDS) != hipSuccess)
      return -1;
    attr = true;
  }
  hipLaunchKernelGGL((flash_prefill_kernel<NKU, NKR, NDB, NWV>), dim3(nblocks * (p.H / p.gs) * p.nsub), dim3(64 * NWV), LDS,
                     st, p);
  return (int)hipGetLastError();
}

}  // namespace nls_pfa

extern "C" {
using namespace nls_pfa;

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
  FP p{(const __bf16*)qn, (const __bf16*)qr, (const __bf16*)kx, (const __bf16*)vx, (const __bf16*)cache, xmap, blocks,
       gate, (__bf16*)out, ldqn, ldqr, ldc, ldo, qns, qrs, H, vdim, ldg, 1, 1, scale, NO_WINDOW, 0, 0};
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

// Dp: padded head width (32, 64, 128; 256 with 4 waves); k, v: paged [slots][G][Dp]; blocks of up to 32 * waves tokens. window > 0: a
// sliding window with `keep` first keys
int nls_gqa_prefill(const void* q, long ldq, const void* k, const void* v, const int* xmap, const int* blocks, int nblocks,
                    const float* gate, int ldg, void* out, long ldo, int H, int G, int Dp, int waves, float scale,
                    int window, int keep, int sink, void* stream) {
  if (nblocks < 1 || G < 1 || H < 1 || H % G || window < 0 || window > NO_WINDOW || keep < 0 || (ldq & 7) || (ldo & 3))
    return -1;
  FP p{(const __bf16*)q, (const __bf16*)q, (const __bf16*)k, (const __bf16*)v, nullptr, xmap, blocks, gate, (__bf16*)out, ldq, ldq,
       (long)G * Dp, ldo, Dp, Dp, H, Dp, ldg, H / G, H / G, scale, window ? window : NO_WINDOW, keep, sink};
  hipStream_t st = (hipStream_t)stream;
  // (nsub = H / G workgroups of 32 * waves rows cover a block of 32 * waves tokens)
  if (waves == 8 && Dp == 256) {
    p.nsub *= 2;
    return launch_t<8, 0, 8, 4>(p, nblocks, st);
  }
#define NLS_GP(D, N) \
  if (Dp == D) return waves == 8 ? launch_t<N, 0, N, 8>(p, nblocks, st) : waves == 4 ? launch_t<N, 0, N, 4>(p, nblocks, st) : -1;
  NLS_GP(32, 1) NLS_GP(64, 2) NLS_GP(128, 4)
#undef NLS_GP
  return Dp == 256 && waves == 4 ? launch_t<8, 0, 8, 4>(p, nblocks, st) : -1;
}

}  // extern "C"
