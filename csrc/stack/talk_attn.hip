// Grouped-query attention whose heads' softmax weights are mixed ("talking heads"), bf16, gfx950:
//   w_g(i, j) = softmax over the visible j of scale q_g . k_g,   W_h = sum_g talk[h, g] w_g,   out_h = gate * sum_j W_h v_h(j)
// A mixed weight needs the finished softmax of every head (its denominator), so the keys are scored before any value is used:
//   decoded tokens, short runs  two launches: scores [keys][heads] in f32 with each split's maxima and sums; then mix, values,
//                               gate. Splits of normalised weights add up without a rescale.
//   prompts                     one workgroup per 16 tokens and all heads, two walks over the keys: the first leaves each head's
//                               log-sum-exp in registers, the second scores again, mixes and multiplies with the values.
// The mix itself is on MFMA: a softmax weight goes in as two bf16 parts (16 bits of it), the matrix, which is stored in bf16,
// exactly, and the sums are f32.
#include "../kernels/lds_dma.h"
#include "talk_plain.h"

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
  else return ch ^ (row & (D / 8 - 1));
}
template <int D> DEVI int voff(int row, int ch) { return row * (2 * D) + 16 * vswz<D>(row, ch); }

// V^T fragment of columns 16 c .. 16 c + 15 from a 32-row tile: lane (g, r) gets column r of rows 4 g .. + 3 and 16 + 4 g .. + 3
template <int D> DEVI bf16x8 vfrag(const uint8_t* vb, int c, int g, int r) {
  const int qq = r >> 2, pp = r & 3, ch = 2 * c + (pp >> 1);
  const s16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
      (__attribute__((address_space(3))) s16x4*)(vb + voff<D>(4 * g + qq, ch) + 8 * (pp & 1)));
  const s16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
      (__attribute__((address_space(3))) s16x4*)(vb + voff<D>(16 + 4 * g + qq, ch) + 8 * (pp & 1)));
  return __builtin_bit_cast(bf16x8, __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7));
}

// out[.. + 0 .. 3] = v * gate of columns d .. d + 3 of a head (V: its columns; the padding past them is not stored)
DEVI void put_out(const TalkArgs& p, int t, int h, int d, const f32x4& v) {
  const __bf16* ga = p.gate ? (const __bf16*)p.gate + (size_t)t * p.ldg + (size_t)h * p.V + d : nullptr;
  __bf16* y = (__bf16*)p.out + (size_t)t * p.ldo + (size_t)h * p.Dp + d;
  if (!((p.V | p.ldg) & 3)) {
    if (d >= p.V) return;
    const bf4 g4 = ga ? *reinterpret_cast<const bf4*>(ga) : bf4{(__bf16)1.f, (__bf16)1.f, (__bf16)1.f, (__bf16)1.f};
    *reinterpret_cast<bf4*>(y) = bf4{(__bf16)(v[0] * (float)g4[0]), (__bf16)(v[1] * (float)g4[1]), (__bf16)(v[2] * (float)g4[2]),
                                     (__bf16)(v[3] * (float)g4[3])};
    return;
  }
#pragma unroll
  for (int e = 0; e < 4; ++e)
    if (d + e < p.V) y[e] = (__bf16)(v[e] * (ga ? (float)ga[e] : 1.f));
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
  const __bf16* kc = (const __bf16*)a.k + (size_t)kh * D + 8 * g;
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
      const size_t o = (((size_t)bt[k >> p.bshift] << p.bshift) + (k & ((1 << p.bshift) - 1))) * ldkv;
#pragma unroll
      for (int kk = 0; kk < NKK; ++kk) K[nt][kk] = ld16(kc + o + 32 * kk);
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
  __shared__ __attribute__((aligned(16))) uint8_t smem[W * VB > RB ? W * VB : RB];
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
    for (int c = 0; c < NDT; ++c) o[c] = mma(vfrag<D>(vs, c, g, r), pb, o[c]);
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
    if (na == 1) put_out(a, t, h0 + h, d, v);
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
    put_out(a, t, h0 + h, d, v);
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
  const int* xmap;        // cache slot of every context row
  const int* blocks;      // [n][8]: (first row, rows, sequence, first position, xoff, -, -, -)
  int nsub;               // workgroups of 16 tokens per block
};

// Eight waves of HW heads each, 16 tokens. Weights of a 32-key tile in LDS, [token][key][head] as two bf16 planes; wave w mixes
// tokens 2 w and 2 w + 1 (rows: keys, columns: heads) and leaves the mixed weights, [token][head][key], where that token's first
// plane was; then each wave multiplies its own heads with the values, whose tile it has fetched by LDS-DMA for itself.
constexpr int PKS = 80, PTS = 32 * PKS + 16, PPL = 16 * PTS;     // bytes: key (head) row, token, plane

template <int D, int HW>
__global__ __launch_bounds__(512) void talk_prefill_kernel(Prefill p) {
  constexpr int NKK = D / 32, NDT = D / 16, LPR = D / 8, RPI = 64 / LPR, NVL = KG / RPI, VB = KG * D * 2;
  extern __shared__ __attribute__((aligned(16))) uint8_t lds[];      // [hi plane | lo plane | a value tile per wave]
  const TalkArgs& a = p.a;
  const int* blk = p.blocks + 8 * (blockIdx.x / p.nsub);
  const int row0 = 16 * (p.nsub - 1 - blockIdx.x % p.nsub), n = min(16, blk[1] - row0);      // (later rows see more keys)
  if (n <= 0) return;
  const int t0 = blk[0] + row0, pos0 = blk[3] + row0, last = pos0 + n - 1;
  const int* xmap = p.xmap + blk[4];
  const int tid = threadIdx.x, lane = tid & 63, g = lane >> 4, r = lane & 15;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int hb = wave * HW, nh = min(HW, a.H - hb), gq = a.H / a.G;               // (nh <= 0: a wave without heads)
  const bool one = nh > 0 && hb / gq == (hb + nh - 1) / gq;                       // its heads share a key head
  const int tok = t0 + min(r, n - 1), qpos = pos0 + min(r, n - 1);
  const int window = a.window > 0 ? a.window : 1 << 30;
  const size_t ldkv = (size_t)a.G * D;
  const float sl2 = a.scale * LOG2E;
  const __bf16 *kc = (const __bf16*)a.k + 8 * g, *vc = (const __bf16*)a.v;
  for (int i = tid; i < 2 * PPL / 16; i += 512) reinterpret_cast<u32x4*>(lds)[i] = u32x4{0u, 0u, 0u, 0u};

  bf16x8 qf[HW][NKK];
#pragma unroll
  for (int i = 0; i < HW; ++i)
#pragma unroll
    for (int kk = 0; kk < NKK; ++kk)
      qf[i][kk] = i < nh ? *reinterpret_cast<const bf16x8*>((const __bf16*)a.q + (size_t)tok * a.ldq + (size_t)(hb + i) * D + 32 * kk + 8 * g)
                         : bf16x8{};
  bf16x8 tf[2];
#pragma unroll
  for (int u = 0; u < 2; ++u) tf[u] = *reinterpret_cast<const bf16x8*>((const __bf16*)a.talk + (16 * u + r) * 32 + 8 * g);

  const int first = max(0, pos0 - window + 1) / KG, end = last / KG + 1;
  auto slots = [&](int t) { return xmap[min(t * KG + (lane & 31), last)]; };      // lane: slot of key lane % 32
  auto load_k = [&](int sl, int nt, int kh, u32x4 (&K)[NKK]) __attribute__((always_inline)) {
    const __bf16* s = kc + (size_t)__shfl(sl, 16 * nt + r, 64) * ldkv + (size_t)kh * D;
#pragma unroll
    for (int kk = 0; kk < NKK; ++kk) K[kk] = ld16(s + 32 * kk);
  };
  auto score = [&](const u32x4 (&K)[NKK], const bf16x8 (&q)[NKK]) __attribute__((always_inline)) {
    f32x4 s = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kk = 0; kk < NKK; ++kk) s = mma(__builtin_bit_cast(bf16x8, K[kk]), q[kk], s);
    return s;
  };
  auto hide = [&](int k, float s) { return k <= qpos && k > qpos - window ? s : -INFINITY; };
  const int kh0 = min(hb / gq, a.G - 1);

  // ---- first walk: each head's log2 of the softmax's denominator (lane: token r, its own keys; joined at the end)
  float lse[HW];
  {
    float m[HW], l[HW];
#pragma unroll
    for (int i = 0; i < HW; ++i) {
      m[i] = -1e30f;
      l[i] = 0.f;
    }
    if (nh > 0) {
      int sl = slots(first);
      u32x4 kf[2][NKK];
      load_k(sl, 0, kh0, kf[0]);
      load_k(sl, 1, kh0, kf[1]);
      for (int t = first; t < end; ++t) {
        const bool edge = t * KG + KG - 1 > pos0 || t * KG <= last - window;
        const int nx = slots(min(t + 1, end - 1));
        u32x4 kn[2][NKK];
        load_k(nx, 0, kh0, kn[0]);
        load_k(nx, 1, kh0, kn[1]);
#pragma unroll
        for (int i = 0; i < HW; ++i) {
          if (i >= nh) break;
          if (!one && i > 0 && (hb + i) % gq == 0) {
            load_k(sl, 0, (hb + i) / gq, kf[0]);
            load_k(sl, 1, (hb + i) / gq, kf[1]);
          }
          f32x4 s[2] = {score(kf[0], qf[i]), score(kf[1], qf[i])};
          if (edge) {
#pragma unroll
            for (int nt = 0; nt < 2; ++nt)
#pragma unroll
              for (int e = 0; e < 4; ++e) s[nt][e] = hide(t * KG + 16 * nt + 4 * g + e, s[nt][e]);
          }
          float mn = m[i];
#pragma unroll
          for (int nt = 0; nt < 2; ++nt)
#pragma unroll
            for (int e = 0; e < 4; ++e) mn = fmaxf(mn, s[nt][e] * sl2);
          float sum = l[i] * __builtin_amdgcn_exp2f(m[i] - mn);
#pragma unroll
          for (int nt = 0; nt < 2; ++nt)
#pragma unroll
            for (int e = 0; e < 4; ++e) sum += __builtin_amdgcn_exp2f(fmaf(s[nt][e], sl2, -mn));
          l[i] = sum;
          m[i] = mn;
        }
        sl = nx;
#pragma unroll
        for (int nt = 0; nt < 2; ++nt)
#pragma unroll
          for (int kk = 0; kk < NKK; ++kk) kf[nt][kk] = kn[nt][kk];
      }
    }
#pragma unroll
    for (int i = 0; i < HW; ++i) {
#pragma unroll
      for (int o = 16; o <= 32; o <<= 1) {
        const float mo = __shfl_xor(m[i], o, 64), lo = __shfl_xor(l[i], o, 64), M = fmaxf(m[i], mo);
        l[i] = l[i] * __builtin_amdgcn_exp2f(m[i] - M) + lo * __builtin_amdgcn_exp2f(mo - M);
        m[i] = M;
      }
      lse[i] = m[i] + __builtin_amdgcn_logf(l[i]);
    }
  }

  // ---- second walk
  f32x4 o[HW][NDT];
#pragma unroll
  for (int i = 0; i < HW; ++i)
#pragma unroll
    for (int c = 0; c < NDT; ++c) o[i][c] = f32x4{0.f, 0.f, 0.f, 0.f};
  const uint32_t vdst = __builtin_amdgcn_readfirstlane(lds_addr(lds)) + 2 * PPL + wave * VB;
  const uint8_t* vs = lds + 2 * PPL + wave * VB;
  auto fetch_v = [&](int sl, int kh) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < NVL; ++i) {
      const int row = RPI * i + lane / LPR;
      glds16(vc + (size_t)__shfl(sl, row, 64) * ldkv + (size_t)kh * D + 8 * vswz<D>(row, lane % LPR), vdst + 1024 * i);
    }
  };
  auto barrier = [&]() __attribute__((always_inline)) {
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
  };
  __syncthreads();
  int sl = slots(first);
  u32x4 kf[2][NKK];
  if (nh > 0) {
    load_k(sl, 0, kh0, kf[0]);
    load_k(sl, 1, kh0, kf[1]);
  }
  for (int t = first; t < end; ++t) {
    const bool edge = t * KG + KG - 1 > pos0 || t * KG <= last - window;
    const int nx = slots(min(t + 1, end - 1));
    if (nh > 0) {
      fetch_v(sl, kh0);
#pragma unroll
      for (int nt = 0; nt < 2; ++nt) {
        __bf16 hi[4][HW], lo[4][HW];
#pragma unroll
        for (int i = 0; i < HW; ++i) {
          if (!one && i > 0 && i < nh && (hb + i) % gq == 0) load_k(sl, nt, (hb + i) / gq, kf[nt]);
          f32x4 s = score(kf[nt], qf[i]);
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            if (edge) s[e] = hide(t * KG + 16 * nt + 4 * g + e, s[e]);
            const float w = i < nh ? __builtin_amdgcn_exp2f(fmaf(s[e], sl2, -lse[i])) : 0.f;
            hi[e][i] = (__bf16)w;
            lo[e][i] = (__bf16)(w - (float)hi[e][i]);
          }
        }
        load_k(nx, nt, kh0, kf[nt]);
        typedef __bf16 bfw __attribute__((ext_vector_type(HW)));
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          bfw a1, a2;
#pragma unroll
          for (int i = 0; i < HW; ++i) {
            if constexpr (HW == 1) {
              a1 = hi[e][i];
              a2 = lo[e][i];
            } else {
              a1[i] = hi[e][i];
              a2[i] = lo[e][i];
            }
          }
          uint8_t* d = lds + r * PTS + (16 * nt + 4 * g + e) * PKS + hb * 2;
          *reinterpret_cast<bfw*>(d) = a1;
          *reinterpret_cast<bfw*>(d + PPL) = a2;
        }
      }
    }
    barrier();
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      uint8_t* tw = lds + (2 * wave + u) * PTS;
      bf16x8 w[2][2];
#pragma unroll
      for (int nt = 0; nt < 2; ++nt)
#pragma unroll
        for (int pl = 0; pl < 2; ++pl)
          w[nt][pl] = *reinterpret_cast<const bf16x8*>(tw + pl * PPL + (16 * nt + r) * PKS + 16 * g);
#pragma unroll
      for (int ht = 0; ht < 2; ++ht) {
        if (16 * ht >= a.H) break;
        bf16x8 pb;
#pragma unroll
        for (int nt = 0; nt < 2; ++nt) {
          f32x4 mx = f32x4{0.f, 0.f, 0.f, 0.f};
          mx = mma(w[nt][0], tf[ht], mx);
          mx = mma(w[nt][1], tf[ht], mx);
#pragma unroll
          for (int e = 0; e < 4; ++e) pb[4 * nt + e] = (__bf16)mx[e];
        }
        *reinterpret_cast<bf16x8*>(tw + (16 * ht + r) * PKS + 16 * g) = pb;      // keys 4 g .., 16 + 4 g .. of head 16 ht + r
      }
    }
    barrier();
    if (nh > 0) {
      wait_vm_lgkm0<0>();
      const uint8_t* pw = lds + r * PTS + hb * PKS + 16 * g;
      if (one) {
        bf16x8 pb[HW];
#pragma unroll
        for (int i = 0; i < HW; ++i) pb[i] = *reinterpret_cast<const bf16x8*>(pw + (i < nh ? i : 0) * PKS);
#pragma unroll
        for (int c = 0; c < NDT; ++c) {
          const bf16x8 vf = vfrag<D>(vs, c, g, r);
#pragma unroll
          for (int i = 0; i < HW; ++i) o[i][c] = mma(vf, pb[i], o[i][c]);
        }
      } else {
#pragma unroll
        for (int i = 0; i < HW; ++i) {
          if (i >= nh) break;
          if (i > 0 && (hb + i) % gq == 0) {
            asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");                   // the last head's reads are done
            fetch_v(sl, (hb + i) / gq);
            wait_vm_lgkm0<0>();
          }
          const bf16x8 pb = *reinterpret_cast<const bf16x8*>(pw + i * PKS);
#pragma unroll
          for (int c = 0; c < NDT; ++c) o[i][c] = mma(vfrag<D>(vs, c, g, r), pb, o[i][c]);
        }
      }
    }
    barrier();
    sl = nx;
  }
  if (r >= n) return;
#pragma unroll
  for (int i = 0; i < HW; ++i) {
    if (i >= nh) break;
#pragma unroll
    for (int c = 0; c < NDT; ++c) put_out(a, tok, hb + i, 16 * c + 4 * g, o[i][c]);
  }
}

template <int D, int HW>
int prefill_t(const Prefill& p, int n, hipStream_t st) {
  constexpr int LDS = 2 * PPL + 8 * KG * D * 2;
  static_assert(LDS <= 160 * 1024, "LDS");
  static bool attr = false;
  if (!attr) {
    if (hipFuncSetAttribute((const void*)talk_prefill_kernel<D, HW>, hipFuncAttributeMaxDynamicSharedMemorySize, LDS) != hipSuccess)
      return -1;
    attr = true;
  }
  hipLaunchKernelGGL((talk_prefill_kernel<D, HW>), dim3(n * p.nsub), dim3(512), LDS, st, p);
  return (int)hipGetLastError();
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

// query blocks of up to 16 * nsub tokens, bf16; H <= 32, Dp 32, 64 or 128, ceil(H / 8) heads of Dp columns at most 512 columns. talk:
// bf16 [32][32]
int nls_talk_prefill(const void* q, long ldq, const void* k, const void* v, const int* xmap, const int* blocks, int nblocks, int nsub,
                     int H, int G, int Dp, int V, float scale, int window, const void* talk, const void* gate, long ldg, void* out,
                     long ldo, void* stream) {
  const TalkArgs a{q, k, v, out, gate, talk, nullptr, nullptr, nullptr, ldq, ldo, ldg, 0, 0, H, G, Dp, V, scale, window};
  if (nblocks < 1 || nsub < 1 || !valid(a) || H > 32 || (ldq & 7) || (ldo & 3) || !xmap || !blocks) return -1;
  const Prefill p{a, xmap, blocks, nsub};
  const int hw = (H + 7) / 8;
  hipStream_t s = (hipStream_t)stream;
#define NLS_TP(D) \
  if (Dp == D) return hw == 1 ? prefill_t<D, 1>(p, nblocks, s) : hw == 2 ? prefill_t<D, 2>(p, nblocks, s) : prefill_t<D, 4>(p, nblocks, s);
  NLS_TP(32) NLS_TP(64) NLS_TP(128)
#undef NLS_TP
  return -1;
}

}  // extern "C"
