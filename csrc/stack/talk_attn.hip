// Grouped-query attention whose heads' softmax weights are mixed ("talking heads"), bf16, gfx950:
//   w_g(i, j) = softmax over the visible j of scale q_g . k_g,   W_h = sum_g talk[h, g] w_g,   out_h = gate * sum_j W_h v_h(j)
// A mixed weight needs the finished softmax of every head (its denominator), so the keys are scored before any value is used:
//   decoded tokens, short runs  two launches: scores [keys][heads] in f32 with each split's maxima and sums; then mix, values,
//                               gate. Splits of normalised weights add up without a rescale.
//   prompts                     one workgroup per 16 tokens and all heads, two walks over the keys: the first leaves each head's
//                               log-sum-exp in registers, the second scores again, mixes and multiplies with the values.
// Keys come in tiles of 16 slots, [slots / 16][G][Dp / 8][16][8]: the 16 keys of an MFMA operand lie side by side, and a wave's load of
// 32 of their columns is 1 KB in a row. Values are rows.
// The mix itself is on MFMA: a softmax weight goes in as two bf16 parts (16 bits of it), the matrix, which is stored in bf16,
// exactly, and the sums are f32.
#include "../kernels/lds_dma.h"
#include "talk_plain.h"
#include <type_traits>

namespace nls_talk {
using nls_dma::glds16;
using nls_dma::lds_addr;
using nls_dma::wait_vm_lgkm0;

typedef short s16x4 __attribute__((ext_vector_type(4)));
typedef short s16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf4 __attribute__((ext_vector_type(4)));
constexpr float LOG2E = 1.4426950408889634f;
constexpr int KG = 32;        // keys per step

DEVI f32x4 mma(const bf16x8& a, const bf16x8& b, const f32x4& c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }

// byte offset of 16-byte chunk ch of row `row` in a tile of D-column bf16 rows, permuted against bank conflicts
template <int D> DEVI int vswz(int row, int ch) {
  if constexpr (D == 128) return ch ^ (((row & 3) << 2) | ((row >> 2) & 3));
  else return ch ^ (row & (D == 256 ? 15 : D / 8 - 1));
}
template <int D> DEVI int voff(int row, int ch) { return row * (2 * D) + 16 * vswz<D>(row, ch); }

// V^T fragment of columns 16 c .. 16 c + 15 from a 32-row tile: lane (g, r) gets column r of rows 4 g .. + 3 and 16 + 4 g .. + 3
// (at: vfrag_at(tile's LDS address); rows 16 apart are permuted alike, and tiles aligned to their rows, so the column is an xor)
template <int D> DEVI uint32_t vfrag_at(uint32_t tile, int g, int r) {
  const int qq = r >> 2, pp = r & 3;
  return tile + voff<D>(4 * g + qq, pp >> 1) + 8 * (pp & 1);
}
template <int D> DEVI bf16x8 vfrag(uint32_t at, int c) {
  typedef __attribute__((address_space(3))) s16x4* lp;
  const uint32_t x = at ^ (32u * c);
  const s16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lp)x);
  const s16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lp)(x + 32 * D));
  return __builtin_bit_cast(bf16x8, __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7));
}

// out[.. + 0 .. 3] = v * gate of columns d .. d + 3 of a head (V: its columns; the padding past them is not stored)
DEVI bool by_four(const TalkArgs& p) { return !((p.V | p.ldg) & 3); }
template <bool FOUR> DEVI void put_out(const TalkArgs& p, int t, int h, int d, const f32x4& v) {
  const __bf16* ga = p.gate ? (const __bf16*)p.gate + (size_t)t * p.ldg + (size_t)h * p.V + d : nullptr;
  __bf16* y = (__bf16*)p.out + (size_t)t * p.ldo + (size_t)h * p.Dp + d;
  if constexpr (FOUR) {
    if (d >= p.V) return;
    const bf4 g4 = ga ? *reinterpret_cast<const bf4*>(ga) : bf4{(__bf16)1.f, (__bf16)1.f, (__bf16)1.f, (__bf16)1.f};
    *reinterpret_cast<bf4*>(y) = bf4{(__bf16)(v[0] * (float)g4[0]), (__bf16)(v[1] * (float)g4[1]), (__bf16)(v[2] * (float)g4[2]),
                                     (__bf16)(v[3] * (float)g4[3])};
  } else {
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (d + e < p.V) y[e] = (__bf16)(v[e] * (ga ? (float)ga[e] : 1.f));
  }
}

// ---------------------------------------------------------------------------------------------------------------------
// Decode: row by row
// ---------------------------------------------------------------------------------------------------------------------
struct Decode {
  TalkArgs a;
  float* sc;            // [rows][ks][hs]: scores times log2(e), key 32 * (first visible / 32) first
  float* st;            // [rows][ns1][hs][2]: each score split's maximum and sum
  float* part;          // [rows][H][ns][Dp]
  int* cnt;             // [rows][workgroups]
  long ks;
  int hs, ns1, ns, bshift, t0;
};

// the keys of a row: tiles of 32 from the first visible one's
struct Keys {
  int ctx, low, first, ntile;
  DEVI Keys(const Decode& p, int t) {
    ctx = p.a.ctx_len[t];
    low = p.a.window > 0 ? max(0, ctx - p.a.window) : 0;
    first = low & ~(KG - 1);
    ntile = ctx > 0 ? min((ctx - first + KG - 1) / KG, (int)(p.ks / KG)) : 0;
  }
};

// scores: one wave per (row, 16 heads of a key head, split of the keys). S^T = K Q^T: lane (g, r) holds head r, keys 4 g + i.
template <int D>
__global__ __launch_bounds__(64) void talk_score_kernel(Decode p) {
  constexpr int NKK = D / 32;
  const TalkArgs& a = p.a;
  const int tr = blockIdx.x, t = p.t0 + tr, split = blockIdx.z, gq = a.H / a.G, nhb = (gq + 15) >> 4;
  const int kh = blockIdx.y / nhb, hofs = (blockIdx.y - kh * nhb) * 16, n = min(gq - hofs, 16), h0 = kh * gq + hofs;
  const int lane = threadIdx.x, g = lane >> 4, r = lane & 15;
  const Keys key(p, t);
  const int tps = (key.ntile + p.ns1 - 1) / p.ns1, ta = split * tps, tb = min(ta + tps, key.ntile);
  if (ta >= tb) return;
  const int* bt = a.bt + (size_t)a.tok_seq[t] * a.bts;
  const __bf16* kc = (const __bf16*)a.k + (size_t)kh * 16 * D + 128 * g;
  const size_t ldkv = (size_t)a.G * D;
  bf16x8 qf[NKK];
#pragma unroll
  for (int kk = 0; kk < NKK; ++kk) {
    qf[kk] = bf16x8{};
    if (r < n) qf[kk] = *reinterpret_cast<const bf16x8*>((const __bf16*)a.q + (size_t)t * a.ldq + (size_t)(h0 + r) * D + 32 * kk + 8 * g);
  }
  auto load = [&](int tile, u32x4 (&K)[2][NKK]) __attribute__((always_inline)) {
#pragma unroll
    for (int nt = 0; nt < 2; ++nt) {
      const int k = min(key.first + tile * KG + 16 * nt + r, key.ctx - 1);
      const size_t slot = ((size_t)bt[k >> p.bshift] << p.bshift) + (k & ((1 << p.bshift) - 1));
      const size_t o = (slot & ~(size_t)15) * ldkv + (slot & 15) * 8;
#pragma unroll
      for (int kk = 0; kk < NKK; ++kk) K[nt][kk] = ld16(kc + o + 512 * kk);
    }
  };
  u32x4 kr[2][NKK], kn[2][NKK];
  load(ta, kr);
  const float sl2 = a.scale * LOG2E;
  float m = -1e30f, l = 0.f;
  for (int j = ta; j < tb; ++j) {
    if (j + 1 < tb) load(j + 1, kn);
    f32x4 s[2];
    float mn = m;
#pragma unroll
    for (int nt = 0; nt < 2; ++nt) {
      s[nt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < NKK; ++kk) s[nt] = mma(__builtin_bit_cast(bf16x8, kr[nt][kk]), qf[kk], s[nt]);
      const int k0 = j * KG + 16 * nt + 4 * g;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int pos = key.first + k0 + i;
        s[nt][i] = pos >= key.low && pos < key.ctx ? s[nt][i] * sl2 : -INFINITY;
        if (r < n) p.sc[((size_t)tr * p.ks + k0 + i) * p.hs + h0 + r] = s[nt][i];
        mn = fmaxf(mn, s[nt][i]);
      }
    }
    l *= exp2f(m - mn);
    m = mn;
#pragma unroll
    for (int nt = 0; nt < 2; ++nt)
#pragma unroll
      for (int i = 0; i < 4; ++i) l += exp2f(s[nt][i] - m);
#pragma unroll
    for (int nt = 0; nt < 2; ++nt)
#pragma unroll
      for (int kk = 0; kk < NKK; ++kk) kr[nt][kk] = kn[nt][kk];
  }
#pragma unroll
  for (int o = 16; o <= 32; o <<= 1) {
    const float mo = __shfl_xor(m, o, 64), lo = __shfl_xor(l, o, 64), M = fmaxf(m, mo);
    l = l * exp2f(m - M) + lo * exp2f(mo - M);
    m = M;
  }
  if (g == 0 && r < n) {
    float* s = p.st + (((size_t)tr * p.ns1 + split) * p.hs + h0 + r) * 2;
    s[0] = m;
    s[1] = l;
  }
}

// mix and values: W waves per (row, 16 heads of a key head, split). The mix has keys as rows and this workgroup's heads as columns,
// which is the layout of P^T that the product with V^T takes.
template <int D, int KK, int W>
__global__ __launch_bounds__(64 * W) void talk_value_kernel(Decode p) {
  constexpr int NDT = D / 16, LPR = D / 8, RPI = 64 / LPR, NVL = KG / RPI;
  constexpr int HP = 32 * KK, VB = KG * D * 2, RB = W > 1 ? W * 16 * D * 4 : 0;
  __shared__ __attribute__((aligned(512))) uint8_t smem[W * VB > RB ? W * VB : RB];
  __shared__ float lse[HP];
  __shared__ int last;
  const TalkArgs& a = p.a;
  const int tr = blockIdx.x, t = p.t0 + tr, split = blockIdx.z, gq = a.H / a.G, nhb = (gq + 15) >> 4;
  const int kh = blockIdx.y / nhb, hofs = (blockIdx.y - kh * nhb) * 16, n = min(gq - hofs, 16), h0 = kh * gq + hofs;
  const int lane = threadIdx.x & 63, g = lane >> 4, r = lane & 15;
  const int wave = W == 1 ? 0 : __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const Keys key(p, t);
  const int tps = (key.ntile + p.ns - 1) / p.ns, ta = split * tps, tb = min(ta + tps, key.ntile);
  if (ta >= tb) return;
  const int na = (key.ntile + tps - 1) / tps;                                    // active splits
  const int tps1 = (key.ntile + p.ns1 - 1) / p.ns1, na1 = (key.ntile + tps1 - 1) / tps1;
  const int* bt = a.bt + (size_t)a.tok_seq[t] * a.bts;
  const size_t ldkv = (size_t)a.G * D;
  const __bf16* vc = (const __bf16*)a.v + (size_t)kh * D + 8 * (lane % LPR);
  auto load_v = [&](int tile, u32x4 (&V)[NVL]) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < NVL; ++i) {
      const int k = min(key.first + tile * KG + RPI * i + lane / LPR, key.ctx - 1);
      V[i] = ld16(vc + (((size_t)bt[k >> p.bshift] << p.bshift) + (k & ((1 << p.bshift) - 1))) * ldkv);
    }
  };
  // scores of key 16 nt + r, heads 32 kk + 8 g .. + 7
  auto load_s = [&](int tile, f32x4 (&S)[2][KK][2]) __attribute__((always_inline)) {
#pragma unroll
    for (int nt = 0; nt < 2; ++nt) {
      const float* s = p.sc + ((size_t)tr * p.ks + tile * KG + 16 * nt + r) * p.hs + 8 * g;
#pragma unroll
      for (int kk = 0; kk < KK; ++kk)
#pragma unroll
        for (int u = 0; u < 2; ++u)
          S[nt][kk][u] = 32 * kk + 8 * g < p.hs ? *reinterpret_cast<const f32x4*>(s + 32 * kk + 4 * u) : f32x4{0.f, 0.f, 0.f, 0.f};
    }
  };
  u32x4 vr[NVL], vn[NVL];
  f32x4 sr[2][KK][2], sn[2][KK][2];
  const int j0 = ta + wave;
  if (j0 < tb) {
    load_v(j0, vr);
    load_s(j0, sr);
  }
  bf16x8 tf[KK];
#pragma unroll
  for (int kk = 0; kk < KK; ++kk) {
    tf[kk] = bf16x8{};
    if (r < n) tf[kk] = *reinterpret_cast<const bf16x8*>((const __bf16*)a.talk + (size_t)(h0 + r) * HP + 32 * kk + 8 * g);
  }
  for (int h = threadIdx.x; h < HP; h += 64 * W) {                 // log2 of the softmax's denominator (past H: weights of 0)
    float M = -1e30f, L = 0.f;
    if (h < a.H) {
      const float* s = p.st + ((size_t)tr * p.ns1 * p.hs + h) * 2;
#pragma unroll 8
      for (int i = 0; i < na1; ++i) {
        const float2 ml = *reinterpret_cast<const float2*>(s + (size_t)i * p.hs * 2);
        const float mn = fmaxf(M, ml.x);
        L = L * exp2f(M - mn) + ml.y * exp2f(ml.x - mn);
        M = mn;
      }
    }
    lse[h] = h < a.H ? M + log2f(L) : INFINITY;
  }
  __syncthreads();
  uint8_t* vs = smem + wave * VB;
  const uint32_t vat = vfrag_at<D>(lds_addr(vs), g, r);
  auto store_v = [&](u32x4 (&V)[NVL]) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < NVL; ++i) *reinterpret_cast<u32x4*>(vs + voff<D>(RPI * i + lane / LPR, lane % LPR)) = V[i];
  };
  f32x4 o[NDT];
#pragma unroll
  for (int c = 0; c < NDT; ++c) o[c] = f32x4{0.f, 0.f, 0.f, 0.f};
  if (j0 < tb) store_v(vr);
  for (int j = j0; j < tb; j += W) {
    if (j + W < tb) {
      load_v(j + W, vn);
      load_s(j + W, sn);
    }
    f32x4 mx[2];
#pragma unroll
    for (int nt = 0; nt < 2; ++nt) {
      mx[nt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < KK; ++kk) {
        bf16x8 hi, lo;
        const f32x4 c0 = *reinterpret_cast<const f32x4*>(lse + 32 * kk + 8 * g);
        const f32x4 c1 = *reinterpret_cast<const f32x4*>(lse + 32 * kk + 8 * g + 4);
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const float c = e < 4 ? c0[e & 3] : c1[e & 3];
          const float w = c == INFINITY ? 0.f : exp2f(sr[nt][kk][e >> 2][e & 3] - c);
          hi[e] = (__bf16)w;
          lo[e] = (__bf16)(w - (float)hi[e]);
        }
        mx[nt] = mma(hi, tf[kk], mx[nt]);
        mx[nt] = mma(lo, tf[kk], mx[nt]);
      }
    }
    bf16x8 pb;
#pragma unroll
    for (int nt = 0; nt < 2; ++nt)
#pragma unroll
      for (int i = 0; i < 4; ++i) pb[4 * nt + i] = (__bf16)mx[nt][i];
#pragma unroll
    for (int c = 0; c < NDT; ++c) o[c] = mma(vfrag<D>(vat, c), pb, o[c]);
    if (j + W < tb) {
      store_v(vn);
#pragma unroll
      for (int nt = 0; nt < 2; ++nt)
#pragma unroll
        for (int kk = 0; kk < KK; ++kk) {
          sr[nt][kk][0] = sn[nt][kk][0];
          sr[nt][kk][1] = sn[nt][kk][1];
        }
    }
  }
  // lane (g, r): columns 16 c + 4 g + i of head r
  auto finish = [&](int h, int d, const f32x4& v) {                 // head of the workgroup, column
    if (na == 1) {
      if (by_four(a)) put_out<true>(a, t, h0 + h, d, v);
      else put_out<false>(a, t, h0 + h, d, v);
    }
    else *reinterpret_cast<f32x4*>(p.part + (((size_t)tr * a.H + h0 + h) * p.ns + split) * D + d) = v;
  };
  if constexpr (W > 1) {
    float* red = reinterpret_cast<float*>(smem);
    __syncthreads();
#pragma unroll
    for (int c = 0; c < NDT; ++c) *reinterpret_cast<f32x4*>(red + ((size_t)wave * 16 + r) * D + 16 * c + 4 * g) = o[c];
    __syncthreads();
    for (int e = threadIdx.x; e < n * (D / 4); e += 64 * W) {
      const int h = e / (D / 4), d = 4 * (e - h * (D / 4));
      f32x4 v = *reinterpret_cast<const f32x4*>(red + (size_t)h * D + d);
#pragma unroll
      for (int w = 1; w < W; ++w) v += *reinterpret_cast<const f32x4*>(red + ((size_t)w * 16 + h) * D + d);
      finish(h, d, v);
    }
  } else if (r < n) {
#pragma unroll
    for (int c = 0; c < NDT; ++c) finish(r, 16 * c + 4 * g, o[c]);
  }
  if (na == 1) return;
  // the last split to arrive adds them up
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  __syncthreads();
  if (threadIdx.x == 0) {
    int* cp = p.cnt + (size_t)tr * gridDim.y + blockIdx.y;
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "agent");
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    const int old = __hip_atomic_fetch_add(cp, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    last = old == na - 1;
    if (last) {
      __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "agent");
      __hip_atomic_store(cp, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
      asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    }
  }
  __syncthreads();
  if (!last) return;
  for (int e = threadIdx.x; e < n * (D / 4); e += 64 * W) {
    const int h = e / (D / 4), d = 4 * (e - h * (D / 4));
    const float* s = p.part + ((size_t)tr * a.H + h0 + h) * p.ns * D + d;
    f32x4 v = *reinterpret_cast<const f32x4*>(s);
#pragma unroll 8
    for (int i = 1; i < na; ++i) v += *reinterpret_cast<const f32x4*>(s + (size_t)i * D);
    if (by_four(a)) put_out<true>(a, t, h0 + h, d, v);
    else put_out<false>(a, t, h0 + h, d, v);
  }
}

template <int D>
int decode_score(const Decode& p, int rows, int groups, hipStream_t st) {
  hipLaunchKernelGGL(talk_score_kernel<D>, dim3(rows, groups, p.ns1), dim3(64), 0, st, p);
  return (int)hipGetLastError();
}

template <int D, int KK>
int decode_value(const Decode& p, int rows, int groups, int waves, hipStream_t st) {
  if (waves == 1) hipLaunchKernelGGL((talk_value_kernel<D, KK, 1>), dim3(rows, groups, p.ns), dim3(64), 0, st, p);
  else hipLaunchKernelGGL((talk_value_kernel<D, KK, 4>), dim3(rows, groups, p.ns), dim3(256), 0, st, p);
  return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------------------------
// Prompts
// ---------------------------------------------------------------------------------------------------------------------
struct Prefill {
  TalkArgs a;
  const int* blocks;      // [n][8]: (first row, rows, sequence, first position, -, -, -, -)
  int bshift;             // pages of 1 << bshift >= 16 keys
  int nblocks, nsub;      // blocks; workgroups of 16 tokens of each
};

// Eight waves of HW heads each, 16 tokens. Weights of a 32-key tile in LDS, [token][key][head][two bf16 parts]; wave w mixes
// tokens 2 w and 2 w + 1 (rows: keys, columns: heads) and leaves the mixed weights, [token][head][key], in that token's space;
// then each wave multiplies its own heads with the values, whose tile it has fetched by LDS-DMA for itself. Keys are read a tile
// ahead, values while the weights are mixed. 16 keys beside each other lie in one page, so addresses are a wave-uniform base and a
// constant offset per lane.
constexpr int PKS = 144, PTS = 32 * PKS + 16, PW = 16 * PTS, PHS = 80;     // bytes: key row, token, all; row of a mixed head
// behind the value tiles what the registers do not hold through the second walk: the matrix, the denominators, and at the largest
// size some of the last head's queries
template <int D, int HW> struct PL {
  static constexpr int V = PW, T = V + 8 * KG * D * 2, L = T + 2048, Q = L + 2048, NQ = D == 128 && HW == 4 ? 2 : 0;
  static constexpr int BYTES = Q + 8 * NQ * 1024;
  static_assert(BYTES <= 160 * 1024, "LDS");
};

// ONE: a wave's heads share a key head
template <int D, int HW, bool ONE>
__global__ __launch_bounds__(512) void talk_prefill_kernel(Prefill p) {
  constexpr int NKK = D / 32, NDT = D / 16, LPR = D / 8, RPI = 64 / LPR, NVL = KG / RPI, VB = KG * D * 2;
  typedef PL<D, HW> P;
  extern __shared__ __attribute__((aligned(16))) uint8_t lds[];      // [weights | a value tile per wave | PL]
  const TalkArgs& a = p.a;
  // a block's workgroups share most of their keys: they run on one XCD
  const int unit = blockIdx.x >> 3, bi = unit / p.nsub * 8 + (blockIdx.x & 7);
  if (bi >= p.nblocks) return;
  const int* blk = p.blocks + 8 * bi;
  const int row0 = 16 * (p.nsub - 1 - unit % p.nsub), n = min(16, blk[1] - row0);      // (later rows see more keys)
  if (n <= 0) return;
  const int t0 = blk[0] + row0, pos0 = blk[3] + row0, last = pos0 + n - 1;
  const int tid = threadIdx.x, lane = tid & 63, g = lane >> 4, r = lane & 15;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int hb = wave * HW, nh = min(HW, a.H - hb), gq = a.H / a.G;
  // heads past nh (a wave may have none): queries of zeros, columns that the matrix leaves out, nothing stored. They run along: where
  // paths with and without loads meet, the counted waits would become waits for everything.
  const int tok = t0 + min(r, n - 1), qpos = pos0 + min(r, n - 1);
  const int window = a.window > 0 ? a.window : 1 << 30;
  const long ldkv = (long)a.G * D;
  const float sl2 = a.scale * LOG2E;
  for (int i = tid; i < PW / 16; i += 512) reinterpret_cast<u32x4*>(lds)[i] = u32x4{0u, 0u, 0u, 0u};

  bf16x8 qf[HW][NKK];
#pragma unroll
  for (int i = 0; i < HW; ++i)
#pragma unroll
    for (int kk = 0; kk < NKK; ++kk)
      qf[i][kk] = i < nh ? *reinterpret_cast<const bf16x8*>((const __bf16*)a.q + (size_t)tok * a.ldq + (size_t)(hb + i) * D + 32 * kk + 8 * g)
                         : bf16x8{};

  const int first = max(0, pos0 - window + 1) / KG, end = last / KG + 1;
  // cache rows of the two groups of 16 keys of a tile (past the last key: its group again, masked): table entries come from a
  // register window of 64
  const int* bt = a.bt + (size_t)__builtin_amdgcn_readfirstlane(blk[2]) * a.bts;
  const int e0 = first * KG >> p.bshift, elast = last >> p.bshift;
  int btwin = -1, btreg = 0;
  struct Rows { long at[2]; };
  auto rows = [&](int t) __attribute__((always_inline)) {
    Rows s;
#pragma unroll
    for (int nt = 0; nt < 2; ++nt) {
      const int k = min(t * KG + 16 * nt, last & ~15), e = (k >> p.bshift) - e0;
      if (nt == 0 && e >> 6 != btwin) {             // (both groups lie in one window: it starts with a tile)
        btwin = e >> 6;
        const int i = e0 + 64 * btwin + lane;
        btreg = i <= elast ? bt[i] : 0;
        asm volatile("" : "+v"(btreg));             // waited for here, not where the paths meet: there other loads are on their way
      }
      s.at[nt] = (((long)__builtin_amdgcn_readlane(btreg, e & 63) << p.bshift) + (k & ((1 << p.bshift) - 1))) * ldkv;
    }
    return s;
  };
  auto load_k = [&](const Rows& s, int nt, int kh, u32x4 (&K)[NKK]) __attribute__((always_inline)) {
    const __bf16* base = (const __bf16*)a.k + s.at[nt] + kh * 16 * D;
#pragma unroll
    for (int kk = 0; kk < NKK; ++kk) {
      K[kk] = ld16(base + (8u * lane + 512 * kk));
      __builtin_amdgcn_sched_barrier(0);            // (in the order of their use, also ahead of the loops: the waits are counted)
    }
  };
  // The scores' sums start from what hides the keys 4 g .. of a group that the lane's token does not see. No branch over whole and
  // partly seen tiles: where its paths meet, the counted waits would become waits for everything.
  auto hidden = [&](int k0, int g) __attribute__((always_inline)) {
    f32x4 c;
#pragma unroll
    for (int e = 0; e < 4; ++e) c[e] = (uint32_t)(qpos - (k0 + 4 * g + e)) < (uint32_t)window ? 0.f : -INFINITY;
    return c;
  };
  auto score = [&](const u32x4 (&K)[NKK], const bf16x8 (&q)[NKK], f32x4 s) __attribute__((always_inline)) {
#pragma unroll
    for (int kk = 0; kk < NKK; ++kk) s = mma(__builtin_bit_cast(bf16x8, K[kk]), q[kk], s);
    return s;
  };
  const int kh0 = min(hb / gq, a.G - 1);

  // ---- first walk: each head's log2 of the softmax's denominator (lane: token r, its own keys; joined at the end)
  {
    float m[HW], l[HW];
#pragma unroll
    for (int i = 0; i < HW; ++i) {
      m[i] = -1e30f;
      l[i] = 0.f;
    }
    {
      Rows sl = rows(first);
      u32x4 kf[2][NKK];
      load_k(sl, 0, kh0, kf[0]);
      load_k(sl, 1, kh0, kf[1]);
      for (int t = first; t < end; ++t) {
        const Rows s1 = rows(min(t + 1, end - 1));
        f32x4 s[HW][2];
        const f32x4 c[2] = {hidden(t * KG, g), hidden(t * KG + 16, g)};
#pragma unroll
        for (int i = 0; i < HW; ++i) {
          if (!ONE && i > 0 && i < nh && (hb + i) % gq == 0) {
            load_k(sl, 0, (hb + i) / gq, kf[0]);
            load_k(sl, 1, (hb + i) / gq, kf[1]);
          }
#pragma unroll
          for (int nt = 0; nt < 2; ++nt) s[i][nt] = score(kf[nt], qf[i], c[nt]);
        }
        __builtin_amdgcn_sched_barrier(0);
        load_k(s1, 0, kh0, kf[0]);
        load_k(s1, 1, kh0, kf[1]);
#pragma unroll
        for (int i = 0; i < HW; ++i) {
          float mn = m[i];                          // (of the scores as they are: sl2 >= 0)
#pragma unroll
          for (int nt = 0; nt < 2; ++nt)
#pragma unroll
            for (int e = 0; e < 4; ++e) mn = fmaxf(mn, s[i][nt][e]);
          const float nb = -mn * sl2;
          float l2 = l[i] * __builtin_amdgcn_exp2f((m[i] - mn) * sl2);
#pragma unroll
          for (int nt = 0; nt < 2; ++nt)
#pragma unroll
            for (int e = 0; e < 4; ++e) l2 += __builtin_amdgcn_exp2f(fmaf(s[i][nt][e], sl2, nb));
          l[i] = l2;
          m[i] = mn;
        }
        sl = s1;
      }
    }
#pragma unroll
    for (int i = 0; i < HW; ++i) {
#pragma unroll
      for (int o = 16; o <= 32; o <<= 1) {
        const float mo = __shfl_xor(m[i], o, 64), lo = __shfl_xor(l[i], o, 64), M = fmaxf(m[i], mo);
        l[i] = l[i] * __builtin_amdgcn_exp2f((m[i] - M) * sl2) + lo * __builtin_amdgcn_exp2f((mo - M) * sl2);
        m[i] = M;
      }
      if (g == 0) reinterpret_cast<float*>(lds + P::L)[(hb + i) * 16 + r] = m[i] * sl2 + __builtin_amdgcn_logf(l[i]);
    }
  }

  // ---- second walk
  bf4* tl = reinterpret_cast<bf4*>(lds + P::T) + lane;      // [4][64]: rows 16 u + r, columns 16 v + 4 g ..
  if (wave < 4) tl[64 * wave] = *reinterpret_cast<const bf4*>((const __bf16*)a.talk + (16 * (wave >> 1) + r) * 32 + 16 * (wave & 1) + 4 * g);
  bf16x8* ql = reinterpret_cast<bf16x8*>(lds + P::Q + wave * P::NQ * 1024) + lane;
#pragma unroll
  for (int j = 0; j < P::NQ; ++j) ql[64 * j] = qf[HW - 1][NKK - P::NQ + j];
  f32x4 o[HW][NDT];
#pragma unroll
  for (int i = 0; i < HW; ++i)
#pragma unroll
    for (int c = 0; c < NDT; ++c) o[i][c] = f32x4{0.f, 0.f, 0.f, 0.f};
  btwin = -1;
  const uint32_t vdst = __builtin_amdgcn_readfirstlane(lds_addr(lds)) + P::V + wave * VB;
  // the lane's number anew: what follows from it need not live through the loop
  auto again = [](int v) __attribute__((always_inline)) {
    asm volatile("" : "+v"(v));
    return v;
  };
  auto fetch_v = [&](const Rows& s, int kh) __attribute__((always_inline)) {
    const int ln = again(lane);
#pragma unroll
    for (int i = 0; i < NVL; ++i) {
      const int row = RPI * i;
      glds16((const __bf16*)a.v + s.at[row >> 4] + (row & 15) * ldkv + kh * D,
             2 * ((ln / LPR) * (uint32_t)ldkv + 8 * vswz<D>(row + ln / LPR, ln % LPR)), vdst + 1024 * i);
    }
  };
  auto barrier = [&]() __attribute__((always_inline)) {
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
  };
  __syncthreads();
  Rows sl = rows(first);
  u32x4 kf[2][NKK];
  load_k(sl, 0, kh0, kf[0]);
  load_k(sl, 1, kh0, kf[1]);
  auto weigh = [&](int t, const Rows& sl) __attribute__((always_inline)) {
    const int ln = again(lane), g = ln >> 4, r = ln & 15;
    const float* ll = reinterpret_cast<const float*>(lds + P::L) + hb * 16 + r;
    const bf16x8* ql = reinterpret_cast<const bf16x8*>(lds + P::Q + wave * P::NQ * 1024) + ln;
    f32x4 c;
    auto product = [&](int u) __attribute__((always_inline)) {                  // keys 16 nt .., head i
      const int nt = u / HW, i = u % HW;
      if (!ONE && i > 0 && i < nh && (hb + i) % gq == 0) load_k(sl, nt, (hb + i) / gq, kf[nt]);
      if (P::NQ && i == HW - 1) {
#pragma unroll
        for (int j = 0; j < P::NQ; ++j) qf[i][NKK - P::NQ + j] = ql[64 * j];
      }
      if (i == 0) c = hidden(t * KG + 16 * nt, g);
      return score(kf[nt], qf[i], c);
    };
    f32x4 s = product(0);
    float lse = ll[0];
    uint32_t held[4];
#pragma unroll
    for (int u = 0; u < 2 * HW; ++u) {                                          // a product is on its way while the last one's weights are made
      const int nt = u / HW, i = u % HW;
      f32x4 sn = s;
      if (u == HW) fetch_v(sl, kh0);                // (the tile's keys are there: nothing else waits for it)
      if (u + 1 < 2 * HW) sn = product(u + 1);
      const float lsen = ll[16 * ((u + 1) % HW)];
      constexpr int PAIR = HW > 1 ? 2 : 1;          // heads per store
      uint8_t* d = lds + r * PTS + (16 * nt + 4 * g) * PKS + (hb + i / PAIR * PAIR) * 4;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float w = __builtin_amdgcn_exp2f(fmaf(s[e], sl2, -lse));
        // the upper half of w, and of what that leaves: 16 bits of it
        const uint32_t up = __builtin_bit_cast(uint32_t, w) & 0xffff0000u;
        const uint32_t low = __builtin_bit_cast(uint32_t, w - __builtin_bit_cast(float, up));
        const uint32_t both = __builtin_amdgcn_perm(low, up, 0x07060302);
        if constexpr (PAIR == 1) *reinterpret_cast<uint32_t*>(d + e * PKS) = both;
        else if (i & 1) *reinterpret_cast<uint2*>(d + e * PKS) = uint2{held[e], both};
        else held[e] = both;
      }
      s = sn;
      lse = lsen;
      __builtin_amdgcn_sched_barrier(0);            // (heads one by one: registers)
    }
  };
  for (int t = first; t < end; ++t) {
    const Rows s1 = rows(min(t + 1, end - 1));
    weigh(t, sl);
    barrier();
    const int ln = again(lane), g = ln >> 4, r = ln & 15;
    bf4 tf[2][2];
#pragma unroll
    for (int u = 0; u < 4; ++u) tf[u >> 1][u & 1] = reinterpret_cast<const bf4*>(lds + P::T)[64 * u + ln];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      uint8_t* tw = lds + (2 * wave + u) * PTS;
      bf16x8 w[2][2];                              // keys 16 nt + r, both parts of heads 16 v + 4 g ..
#pragma unroll
      for (int nt = 0; nt < 2; ++nt)
#pragma unroll
        for (int v = 0; v < 2; ++v)
          w[nt][v] = *reinterpret_cast<const bf16x8*>(tw + (16 * nt + r) * PKS + 64 * v + 16 * g);
#pragma unroll
      for (int ht = 0; ht < 2; ++ht) {
        bf16x8 pb;
#pragma unroll
        for (int nt = 0; nt < 2; ++nt) {
          f32x4 mx = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int v = 0; v < 2; ++v) mx = mma(w[nt][v], __builtin_shufflevector(tf[ht][v], tf[ht][v], 0, 0, 1, 1, 2, 2, 3, 3), mx);
#pragma unroll
          for (int e = 0; e < 4; ++e) pb[4 * nt + e] = (__bf16)mx[e];
        }
        *reinterpret_cast<bf16x8*>(tw + (16 * ht + r) * PHS + 16 * g) = pb;      // keys 4 g .., 16 + 4 g .. of head 16 ht + r
      }
      __builtin_amdgcn_sched_barrier(0);
    }
    barrier();
    const uint32_t vat = vfrag_at<D>(vdst, g, r);
    const uint8_t* pw = lds + r * PTS + hb * PHS + 16 * g;
    if constexpr (ONE) {
      bf16x8 pb[HW];
#pragma unroll
      for (int i = 0; i < HW; ++i) pb[i] = *reinterpret_cast<const bf16x8*>(pw + i * PHS);
      barrier();                                    // the next tile's weights may come: waves go on at their own pace until they mix
      wait_vm_lgkm0<0>();                           // the values
      load_k(s1, 0, kh0, kf[0]);
      bf16x8 vf = vfrag<D>(vat, 0);
#pragma unroll
      for (int c = 0; c < NDT; ++c) {
        const bf16x8 vn = c + 1 < NDT ? vfrag<D>(vat, c + 1) : vf;
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int i = 0; i < HW; ++i) o[i][c] = mma(vf, pb[i], o[i][c]);
        vf = vn;
      }
    } else {
      wait_vm_lgkm0<0>();
      load_k(s1, 0, kh0, kf[0]);
#pragma unroll
      for (int i = 0; i < HW; ++i) {
        if (i > 0 && i < nh && (hb + i) % gq == 0) {
          asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");                   // the last head's reads are done
          fetch_v(sl, (hb + i) / gq);
          wait_vm_lgkm0<0>();
        }
        const bf16x8 pb = *reinterpret_cast<const bf16x8*>(pw + i * PHS);
#pragma unroll
        for (int c = 0; c < NDT; ++c) o[i][c] = mma(vfrag<D>(vat, c), pb, o[i][c]);
      }
    }
    __builtin_amdgcn_sched_barrier(0);
    load_k(s1, 1, kh0, kf[1]);
    if constexpr (!ONE) barrier();
    sl = s1;
  }
  if (r >= n) return;
  auto store = [&](auto four) {
#pragma unroll
    for (int i = 0; i < HW; ++i)
      if (i < nh) {
#pragma unroll
        for (int c = 0; c < NDT; ++c) put_out<decltype(four)::value>(a, tok, hb + i, 16 * c + 4 * g, o[i][c]);
      }
  };
  if (by_four(a)) store(std::true_type{});
  else store(std::false_type{});
}

template <int D, int HW, bool ONE>
int prefill_o(const Prefill& p, int n, hipStream_t st) {
  constexpr int LDS = PL<D, HW>::BYTES;
  static bool attr = false;
  if (!attr) {
    if (hipFuncSetAttribute((const void*)talk_prefill_kernel<D, HW, ONE>, hipFuncAttributeMaxDynamicSharedMemorySize, LDS) != hipSuccess)
      return -1;
    attr = true;
  }
  hipLaunchKernelGGL((talk_prefill_kernel<D, HW, ONE>), dim3((n + 7) / 8 * 8 * p.nsub), dim3(512), LDS, st, p);
  return (int)hipGetLastError();
}

template <int D, int HW>
int prefill_t(const Prefill& p, int n, hipStream_t st) {
  return p.a.H / p.a.G % HW == 0 ? prefill_o<D, HW, true>(p, n, st) : prefill_o<D, HW, false>(p, n, st);
}

inline bool valid(const TalkArgs& a) {
  return a.q && a.k && a.v && a.out && a.talk && a.G >= 1 && a.H >= 1 && a.H % a.G == 0 && a.Dp >= 1 && a.V >= 1 && a.V <= a.Dp &&
         a.window >= 0 && (long)a.H * a.Dp <= a.ldq && (long)a.H * a.Dp <= a.ldo && (!a.gate || (long)a.H * a.V <= a.ldg);
}

}  // namespace nls_talk

extern "C" {
using namespace nls_talk;

// any shape, f32 arithmetic: talk f32 [H][H]
int nls_talk_plain(const void* q, long ldq, const void* k, const void* v, const int* bt, int bts, int bs, const int* tok_seq,
                   const int* ctx_len, int T, int H, int G, int Dp, int V, float scale, int window, const float* talk,
                   const void* gate, long ldg, void* out, long ldo, int f32, void* stream) {
  const TalkArgs a{q, k, v, out, gate, talk, bt, tok_seq, ctx_len, ldq, ldo, ldg, bts, bs, H, G, Dp, V, scale, window};
  if (T < 1 || bs < 1 || !valid(a)) return -1;
  return f32 ? plain::launch<float>(a, T, (hipStream_t)stream) : plain::launch<__bf16>(a, T, (hipStream_t)stream);
}

// rows t0 .. t0 + rows - 1, bf16; bs a power of two, Dp 32, 64, 128 or 256, H <= 128. talk: bf16 [32 kk][32 kk]. sc [rows][ks][hs], ks
// a multiple of 32 that holds 32 * (first visible / 32) .. the last key, hs = H rounded up to 8; st [rows][ns1][hs][2]; ns > 1:
// part [rows][H][ns][Dp], cnt [rows][workgroups] zeros (left zero). waves: 1 or 4
int nls_talk_decode(const void* q, long ldq, const void* k, const void* v, const int* bt, int bts, int bs, const int* tok_seq,
                    const int* ctx_len, int t0, int rows, int H, int G, int Dp, int V, float scale, int window, const void* talk,
                    const void* gate, long ldg, void* out, long ldo, float* sc, long ks, float* st, float* part, int* cnt, int ns1,
                    int ns, int waves, void* stream) {
  const TalkArgs a{q, k, v, out, gate, talk, bt, tok_seq, ctx_len, ldq, ldo, ldg, bts, bs, H, G, Dp, V, scale, window};
  if (rows < 1 || t0 < 0 || !valid(a) || H > 128 || bs < 1 || (bs & (bs - 1)) || (ldq & 7) || (ldo & 3) || !sc || !st || ks < KG ||
      (ks & (KG - 1)) || ns1 < 1 || ns1 > 64 || ns < 1 || ns > 64 || (ns > 1 && (!part || !cnt)) || (waves != 1 && waves != 4))
    return -1;
  const Decode p{a, sc, st, part, cnt, ks, (H + 7) / 8 * 8, ns1, ns, __builtin_ctz((unsigned)bs), t0};
  const int groups = G * ((H / G + 15) / 16);
  hipStream_t s = (hipStream_t)stream;
  int rc = -1;
#define NLS_TD(D) \
  if (Dp == D) { \
    rc = decode_score<D>(p, rows, groups, s); \
    if (rc) return rc; \
    return H <= 32 ? decode_value<D, 1>(p, rows, groups, waves, s) : H <= 64 ? decode_value<D, 2>(p, rows, groups, waves, s) \
                                                                             : decode_value<D, 4>(p, rows, groups, waves, s); \
  }
  NLS_TD(32) NLS_TD(64) NLS_TD(128) NLS_TD(256)
#undef NLS_TD
  return rc;
}

// query blocks of up to 16 * nsub tokens, bf16; H <= 32, Dp 32, 64 or 128, scale > 0, bs a power of two >= 16. talk: bf16 [32][32]
int nls_talk_prefill(const void* q, long ldq, const void* k, const void* v, const int* bt, int bts, int bs, const int* blocks,
                     int nblocks, int nsub, int H, int G, int Dp, int V, float scale, int window, const void* talk, const void* gate,
                     long ldg, void* out, long ldo, void* stream) {
  const TalkArgs a{q, k, v, out, gate, talk, bt, nullptr, nullptr, ldq, ldo, ldg, bts, bs, H, G, Dp, V, scale, window};
  if (nblocks < 1 || nsub < 1 || !valid(a) || H > 32 || !(scale > 0.f) || (ldq & 7) || (ldo & 3) || !bt || !blocks || bs < 16 ||
      (bs & (bs - 1)))
    return -1;
  const Prefill p{a, blocks, __builtin_ctz((unsigned)bs), nblocks, nsub};
  const int hw = (H + 7) / 8;
  hipStream_t s = (hipStream_t)stream;
#define NLS_TP(D) \
  if (Dp == D) return hw == 1 ? prefill_t<D, 1>(p, nblocks, s) : hw == 2 ? prefill_t<D, 2>(p, nblocks, s) : prefill_t<D, 4>(p, nblocks, s);
  NLS_TP(32) NLS_TP(64) NLS_TP(128)
#undef NLS_TP
  return -1;
}

}  // extern "C"
