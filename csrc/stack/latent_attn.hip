// Attention over the paged latent cache (gfx950): every head's keys and values are linear images of one cached row per
// token, [c (R, padded to Rp) | rotated key part (padded to rp)], so with the up-projections folded into the query and
// applied to the output the cache is read once for all heads: score = q_abs . c + q_rot . k_rot, out = sum p c.
//
// latent_attn_kernel (bf16): workgroup = (token, split of the keys, NHB blocks of 16 heads), 4 waves per head block.
// KT-key tiles of the cache rows arrive by LDS-DMA into two buffers (16-byte chunks swizzled by the key on the DMA
// source), once for all head blocks; a 32-key half is refilled as soon as it is consumed, so loads of the next two tiles
// stay in flight. Each wave forms S^T of 16 keys (A = cache rows, B = its block's queries, held in
// registers), the four waves of a block exchange row maxima and the bf16 weights through LDS, and each owns a quarter of
// the output columns: O^T += C^T P^T with C^T fragments from transposed LDS reads of the same tile. Softmax in base 2, all
// of it f32.
// 32-bit models: one workgroup per (token, head) (attn_plain.h).
#include "../kernels/lds_dma.h"
#include "attn_plain.h"

namespace nls_latent {
using nls_dma::glds16;
using nls_dma::lds_addr;

typedef short s16x4 __attribute__((ext_vector_type(4)));
typedef short s16x8 __attribute__((ext_vector_type(8)));

struct LA {
  const void* q;            // [T][H][Dp]
  const void* cache;        // [slots][Dp]
  void* out;                // [T][H][Rp]
  float* part_o;            // [T][H][ns][Rp]
  float* part_ml;           // [T][H][ns][2]
  const int* bt;            // block tables
  const int* tok_seq;
  const int* ctx_len;       // keys of each token (0: padded row)
  int bts, bs, T, H, ns, Rp, rp, bshift;
  float scale;
};

DEVI void bar_lgkm() {
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
}

// chunk permutation of a cache row in LDS: 16 consecutive rows of one chunk land on distinct banks (a row is an odd or even
// multiple of 128 bytes)
template <int Dp>
DEVI int row_swz(int row) {
  return (Dp / 64) & 1 ? (row >> 1) & 7 : row & 15;
}

constexpr int NBT = 1024;    // block-table entries of one split, kept in LDS

template <int N>
DEVI void wait_vm() {
  asm volatile("s_waitcnt vmcnt(%0)" ::"i"(N) : "memory");
}
// everything but one tile's own DMA instructions of this wave has landed
template <int ND, int NH, int NHB>
DEVI void wait_tile(int hsub) {
  if (NHB == 1) wait_vm<ND * NH>();
  else if (hsub < NH) wait_vm<ND>();
  else wait_vm<0>();
}

template <int NT, int RT, int KT, int NHB>
__global__ __launch_bounds__(256 * NHB, 1) void latent_attn_kernel(LA p) {
  constexpr int Rp = 64 * NT, Dp = Rp + 64 * RT;
  constexpr int CPR = Dp / 8;                  // 16-byte chunks per row
  constexpr int TB = KT * Dp * 2;              // bytes per tile
  constexpr int NH = KT / 32;                  // 32-key halves per tile
  constexpr int ND = Dp / 64;                  // DMA instructions per half and issuing wave (four waves issue a half)
  constexpr int NK = Dp / 32;                  // k-steps of a score
  constexpr int PS = KT + 8;                   // P row stride
  constexpr int PR = (Dp / 64) & 1 ? 8 : 16;   // chunks a row's permutation ranges over
  extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
  const int wv = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int wave = wv & 3, hsub = wv >> 2;     // wave of its head block; head block of the workgroup
  __bf16* P = reinterpret_cast<__bf16*>(lds + 2 * TB) + hsub * 16 * PS;                  // [NHB][16][PS]
  float* mx = reinterpret_cast<float*>(lds + 2 * TB + NHB * 16 * PS * 2) + hsub * 64;    // [NHB][4][16]
  int* btl = reinterpret_cast<int*>(lds + 2 * TB + NHB * (16 * PS * 2 + 256));           // [NBT]

  const int HB = (p.H + 16 * NHB - 1) / (16 * NHB);
  const int ts = ((int)blockIdx.x / (8 * HB)) * 8 + (blockIdx.x & 7);
  const int hb = ((int)blockIdx.x >> 3) % HB;
  if (ts >= p.T * p.ns) return;
  const int t = ts / p.ns, split = ts % p.ns;
  const int ctx = p.ctx_len[t];
  const int tiles = (ctx + KT - 1) / KT;       // dealt to the splits as evenly as whole tiles go
  const int k0 = tiles * split / p.ns * KT, k1 = min(ctx, tiles * (split + 1) / p.ns * KT);
  const int lane = threadIdx.x & 63;
  const int r = lane & 15, g = lane >> 4;
  const int head = (hb * NHB + hsub) * 16 + r;
  const __bf16* cache = reinterpret_cast<const __bf16*>(p.cache);
  const int* bt = p.bt + (size_t)p.tok_seq[t] * p.bts;

  f32x4 o[NT];
#pragma unroll
  for (int c = 0; c < NT; ++c) o[c] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;

  if (k0 < k1) {
    u32x4 qf[NK];
    const __bf16* qr = reinterpret_cast<const __bf16*>(p.q) + ((size_t)t * p.H + min(head, p.H - 1)) * Dp;
#pragma unroll
    for (int kk = 0; kk < NK; ++kk) qf[kk] = ld16(qr + kk * 32 + 8 * g);
    const float sl2 = p.scale * 1.4426950408889634f;
    const uint32_t base = __builtin_amdgcn_readfirstlane(lds_addr(lds));
    const int bmask = p.bs - 1;
    // keys [w0, w1) per pass: as many as the block-table window in LDS holds
    for (int w0 = k0; w0 < k1; w0 += NBT << p.bshift) {
      const int w1 = min(k1, w0 + (NBT << p.bshift));
      const int b0 = w0 >> p.bshift, nb = ((w1 - 1) >> p.bshift) - b0 + 1;
      __syncthreads();
      for (int i = threadIdx.x; i < min(nb, NBT); i += 256 * NHB) btl[i] = bt[b0 + i];
      __syncthreads();
      // half u (32 keys) of tile j -> its place in buffer j & 1; issued by the four waves of head block u % NHB
      auto dma = [&](int j, int u) __attribute__((always_inline)) {
        if (NHB > 1 && hsub != u % NHB) return;
        const uint32_t dst = base + (uint32_t)(j & 1) * TB + (uint32_t)u * (32 * Dp * 2) + (uint32_t)(ND * wave) * 1024u;
        // every source address first (their block lookups overlap), then the copies
        const __bf16* src[ND];
#pragma unroll
        for (int i = 0; i < ND; ++i) {
          const int ci = (ND * wave + i) * 64 + lane;
          const int row = ci / CPR, pc = ci - row * CPR;
          const int key = min(w0 + j * KT + 32 * u + row, w1 - 1);
          src[i] = cache + (uint32_t)((pc ^ row_swz<Dp>(row)) * 8) +
                   (((size_t)btl[min((key >> p.bshift) - b0, NBT - 1)] << p.bshift) + (key & bmask)) * Dp;
        }
#pragma unroll
        for (int i = 0; i < ND; ++i) glds16(src[i], dst + i * 1024);
      };
      const int nt = (w1 - w0 + KT - 1) / KT;
#pragma unroll
      for (int u = 0; u < NH; ++u) dma(0, u);
      if (nt > 1) {
#pragma unroll
        for (int u = 0; u < NH; ++u) dma(1, u);
        wait_tile<ND, NH, NHB>(hsub);
      } else {
        wait_vm<0>();
      }
      bar_lgkm();
      for (int j = 0; j < nt; ++j) {
        const uint8_t* cb = lds + (j & 1) * TB;
        f32x4 s = f32x4{-INFINITY, -INFINITY, -INFINITY, -INFINITY};
        float tm = -INFINITY;
        if (KT == 64 || wave < KT / 16) {
          f32x4 s2[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};     // two chains of dependent products
          const uint8_t* kr = cb + (16 * wave + r) * (2 * Dp);
          const int sw = row_swz<Dp>(r);                                            // (16 rows: one period)
#pragma unroll
          for (int kk = 0; kk < NK; ++kk) {
            const int hi = 4 * kk & ~(PR - 1);
            const bf16x8 a = *reinterpret_cast<const bf16x8*>(kr + (hi << 4) + (((((4 * kk) & (PR - 1)) + g) ^ sw) << 4));
            s2[kk & 1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, __builtin_bit_cast(bf16x8, qf[kk]), s2[kk & 1], 0, 0, 0);
          }
          s = s2[0] + s2[1];
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            s[i] = w0 + j * KT + 16 * wave + 4 * g + i < w1 ? s[i] * sl2 : -INFINITY;
            tm = fmaxf(tm, s[i]);
          }
          tm = fmaxf(tm, __shfl_xor(tm, 16, 64));
          tm = fmaxf(tm, __shfl_xor(tm, 32, 64));
        }
        if (g == 0) mx[wave * 16 + r] = tm;
        bar_lgkm();
        const float mn = fmaxf(fmaxf(fmaxf(mx[r], mx[16 + r]), fmaxf(mx[32 + r], mx[48 + r])), m);
        const float alpha = m == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m - mn);
        if (KT == 64 || wave < KT / 16) {
          typedef __bf16 bf4 __attribute__((ext_vector_type(4)));
          bf4 pb;
          float ps = 0.f;
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const float e = s[i] == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(s[i] - mn);
            ps += e;
            pb[i] = (__bf16)e;
          }
          l = l * alpha + ps;                    // this lane's keys; lanes and waves are summed at the end
          *reinterpret_cast<bf4*>(P + r * PS + 16 * wave + 4 * g) = pb;
        }
        m = mn;
        bar_lgkm();
        const int qq = r >> 2, pp = r & 3;
#pragma unroll
        for (int u = 0; u < KT / 32; ++u) {
          const uint2 p0 = *reinterpret_cast<const uint2*>(P + r * PS + 32 * u + 4 * g);
          const uint2 p1 = *reinterpret_cast<const uint2*>(P + r * PS + 32 * u + 16 + 4 * g);
          const bf16x8 pf = __builtin_bit_cast(bf16x8, u32x4{p0.x, p0.y, p1.x, p1.y});
          const uint8_t* vr = cb + (4 * g + qq) * (2 * Dp) + 8 * (pp & 1);
          const int sw = row_swz<Dp>(4 * g + qq);                                   // same for the rows 16, 32, .. below
#pragma unroll
          for (int c = 0; c < NT; ++c) {
            int off;
            if constexpr (2 * NT % PR == 0) {
              const int hi = 2 * c & ~(PR - 1);
              off = ((2 * wave * NT + hi) << 4) + (((((2 * c) & (PR - 1)) + (pp >> 1)) ^ sw) << 4);
            } else {
              off = ((2 * (wave * NT + c) + (pp >> 1)) ^ sw) << 4;
            }
            const s16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
                (__attribute__((address_space(3))) s16x4*)(vr + off + 32 * u * (2 * Dp)));
            const s16x4 hi4 = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
                (__attribute__((address_space(3))) s16x4*)(vr + off + (32 * u + 16) * (2 * Dp)));
            const s16x8 a8 = __builtin_shufflevector(lo, hi4, 0, 1, 2, 3, 4, 5, 6, 7);
            const f32x4 acc = u == 0 ? o[c] * alpha : o[c];
            o[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a8), pf, acc, 0, 0, 0);
          }
          // the half is free once every wave is done with it: refill it with tile j + 2's
          if (u + 1 < NH) {
            bar_lgkm();
            if (j + 2 < nt) dma(j + 2, u);
          }
        }
        if (j + 2 < nt && NH > 1 && (NHB == 1 || hsub == 0)) wait_vm<ND>();       // tile j + 1 landed, that refill in flight
        else wait_vm<0>();
        bar_lgkm();
        if (j + 2 < nt) dma(j + 2, NH - 1);
      }
    }
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (g == 0) mx[wave * 16 + r] = l;
    bar_lgkm();
    l = mx[r] + mx[16 + r] + mx[32 + r] + mx[48 + r];
  }
  if (head >= p.H) return;
  if (p.ns == 1) {
    const float inv = l > 0.f ? 1.f / l : 0.f;
    typedef __bf16 bf4 __attribute__((ext_vector_type(4)));
    __bf16* y = reinterpret_cast<__bf16*>(p.out) + ((size_t)t * p.H + head) * Rp + wave * NT * 16 + 4 * g;
#pragma unroll
    for (int c = 0; c < NT; ++c)
      *reinterpret_cast<bf4*>(y + 16 * c) =
          bf4{(__bf16)(o[c][0] * inv), (__bf16)(o[c][1] * inv), (__bf16)(o[c][2] * inv), (__bf16)(o[c][3] * inv)};
    return;
  }
  const size_t pi = ((size_t)t * p.H + head) * p.ns + split;
  if (k0 < k1)                                 // (an empty split weighs nothing: only its (m, l) is read)
#pragma unroll
  for (int c = 0; c < NT; ++c)
    *reinterpret_cast<f32x4*>(p.part_o + pi * Rp + wave * NT * 16 + 16 * c + 4 * g) = o[c];
  if (wave == 0 && g == 0) {
    p.part_ml[2 * pi] = m;
    p.part_ml[2 * pi + 1] = l;
  }
}

// few splits: a workgroup per (token, head), 4 columns per thread
__global__ __launch_bounds__(256) void latent_merge_few_kernel(LA p) {
  const size_t th = blockIdx.x;
  const float* ml = p.part_ml + th * p.ns * 2;
  float M = -INFINITY, L = 0.f, w[8];
#pragma unroll
  for (int s = 0; s < 8; ++s) {
    w[s] = s < p.ns ? ml[2 * s] : -INFINITY;
    M = fmaxf(M, w[s]);
  }
#pragma unroll
  for (int s = 0; s < 8; ++s) {
    w[s] = w[s] == -INFINITY ? 0.f : exp2f(w[s] - M);
    if (s < p.ns) L += ml[2 * s + 1] * w[s];
  }
  const float inv = L > 0.f ? 1.f / L : 0.f;
  for (int c = threadIdx.x * 4; c < p.Rp; c += (int)blockDim.x * 4) {
    const float* po = p.part_o + th * p.ns * p.Rp + c;
    f32x4 a = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < 8; ++s)
      if (w[s] != 0.f) a += *reinterpret_cast<const f32x4*>(po + (size_t)s * p.Rp) * (w[s] * inv);
    typedef __bf16 bf4 __attribute__((ext_vector_type(4)));
    *reinterpret_cast<bf4*>(reinterpret_cast<__bf16*>(p.out) + th * p.Rp + c) =
        bf4{(__bf16)a[0], (__bf16)a[1], (__bf16)a[2], (__bf16)a[3]};
  }
}

// splits of one (token, head), 64 output columns: 16 lanes x 4 columns, 16 groups of splits
__global__ __launch_bounds__(256) void latent_merge_kernel(LA p) {
  __shared__ float w[64];
  __shared__ f32x4 red[16][16];
  const size_t th = blockIdx.x;
  const float* ml = p.part_ml + th * p.ns * 2;
  const int lane = threadIdx.x & 63;
  if (threadIdx.x < 64) {
    const float m = lane < p.ns ? ml[2 * lane] : -INFINITY, l = lane < p.ns ? ml[2 * lane + 1] : 0.f;
    float M = m;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) M = fmaxf(M, __shfl_xor(M, o, 64));
    const float e = m == -INFINITY ? 0.f : exp2f(m - M);
    float L = l * e;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) L += __shfl_xor(L, o, 64);
    w[lane] = L > 0.f ? e / L : 0.f;
  }
  __syncthreads();
  const int c = threadIdx.x & 15, g = threadIdx.x >> 4;
  const float* po = p.part_o + th * p.ns * p.Rp + blockIdx.y * 64 + 4 * c;
  f32x4 a = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int s = g; s < p.ns; s += 16)
    if (w[s] != 0.f) a += *reinterpret_cast<const f32x4*>(po + (size_t)s * p.Rp) * w[s];
  red[g][c] = a;
  __syncthreads();
  if (g == 0) {
#pragma unroll
    for (int i = 1; i < 16; ++i) a += red[i][c];
    typedef __bf16 bf4 __attribute__((ext_vector_type(4)));
    *reinterpret_cast<bf4*>(reinterpret_cast<__bf16*>(p.out) + th * p.Rp + blockIdx.y * 64 + 4 * c) =
        bf4{(__bf16)a[0], (__bf16)a[1], (__bf16)a[2], (__bf16)a[3]};
  }
}

template <int NT, int RT, int NHB>
int launch_t(const LA& p, hipStream_t st) {
  constexpr int KT = NT + RT > 9 ? 32 : 64;
  constexpr int LDS = 2 * KT * 128 * (NT + RT) + NHB * (16 * (KT + 8) * 2 + 256) + NBT * 4;
  static_assert(LDS <= 160 * 1024, "LDS");
  static bool attr = false;
  if (!attr) {
    if (hipFuncSetAttribute((const void*)latent_attn_kernel<NT, RT, KT, NHB>,
                            hipFuncAttributeMaxDynamicSharedMemorySize, LDS) != hipSuccess)
      return -1;
    attr = true;
  }
  const int HB = (p.H + 16 * NHB - 1) / (16 * NHB), n = (p.T * p.ns + 7) / 8 * 8 * HB;
  hipLaunchKernelGGL((latent_attn_kernel<NT, RT, KT, NHB>), dim3(n), dim3(256 * NHB), LDS, st, p);
  int rc = (int)hipGetLastError();
  if (rc == 0 && p.ns > 1) {
    if (p.ns <= 8)
      hipLaunchKernelGGL(latent_merge_few_kernel, dim3(p.T * p.H), dim3(min(256, p.Rp / 4)), 0, st, p);
    else
      hipLaunchKernelGGL(latent_merge_kernel, dim3(p.T * p.H, p.Rp / 64), dim3(256), 0, st, p);
    rc = (int)hipGetLastError();
  }
  return rc;
}

template <int NT>
int launch_r(const LA& p, hipStream_t st) {
  // 17 .. 32 heads (and pairs of 16-head blocks beyond) share a workgroup's tiles
  constexpr int PAIR = NT < 16 ? 2 : 1;        // (the widest latents would spill)
  if (p.rp == 64) return p.H > 16 ? launch_t<NT, 1, PAIR>(p, st) : launch_t<NT, 1, 1>(p, st);
  if (p.rp == 128) return p.H > 16 ? launch_t<NT, 2, PAIR>(p, st) : launch_t<NT, 2, 1>(p, st);
  return -1;
}

}  // namespace nls_latent

extern "C" {

// Rp: latent width padded to 64 * {1, 2, 3, 4, 6, 8, 12, 16}; rp: rotated width padded to 64 or 128 (multiples of 4 in
// f32 launches); cache rows and queries are Rp + rp wide, zero in the padding.
int nls_latent_attn(const void* q, const void* cache, void* out, float* part_o, float* part_ml, const int* bt, int bts,
                    int bs, const int* tok_seq, const int* ctx_len, int T, int H, int ns, int Rp, int rp, float scale,
                    int f32, void* stream) {
  using namespace nls_latent;
  if (T < 1 || H < 1 || ns < 1 || ns > 64 || bs < 1 || (bs & (bs - 1)) || (ns > 1 && (!part_o || !part_ml))) return -1;
  int bshift = 0;
  while ((1 << bshift) < bs) ++bshift;
  LA p{q, cache, out, part_o, part_ml, bt, tok_seq, ctx_len, bts, bs, T, H, ns, Rp, rp, bshift, scale};
  hipStream_t st = (hipStream_t)stream;
  if (f32) {
    const long Dp = Rp + rp;
    const nls_plain::PA a{q, cache, cache, out, bt, tok_seq, ctx_len, nullptr, H * Dp, Dp, Dp, 0, (long)H * Rp, Rp, 0,
                          bts, bs, H, (int)Dp, Rp, scale};
    return nls_plain::launch<float>(a, T, H, st);
  }
  switch (Rp / 64 * (Rp % 64 == 0)) {
    case 1: return launch_r<1>(p, st);
    case 2: return launch_r<2>(p, st);
    case 3: return launch_r<3>(p, st);
    case 4: return launch_r<4>(p, st);
    case 6: return launch_r<6>(p, st);
    case 8: return launch_r<8>(p, st);
    case 12: return launch_r<12>(p, st);
    case 16: return launch_r<16>(p, st);
  }
  return -1;
}

}  // extern "C"
