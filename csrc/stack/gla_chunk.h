// Linear recurrences with a decay per key channel over runs of tokens (gfx950), in chunks on f32 MFMA: gated linear attention
// (gla.hip) and the delta rule (delta_chunk.h). Keys and values may differ in width. First the form without the delta rule:
//
// Per head, state S [D][V] in f32: S_t = diag(a_t) S_(t-1) + k_t v_t^T, o_t = rs S_t^T q_t. With the decays' products inside a
// chunk of 16 tokens, P(j, i) = prod of a_t over j < t <= i (per key channel, P from the chunk's start with j = -1):
//   o_i = rs [ (q_i P(-1, i))^T S + sum_(j <= i) A_ij v_j ],  A_ij = sum_d q_i k_j P(j, i)
//   S   = diag(P(-1, 15)) S + sum_j (k_j P(j, 15)) v_j^T
// Only products of decays appear, nothing is divided and no logarithm taken: nothing over- or underflows that would not in
// the plain recurrence, and all of it is 32-bit (v_mfma_f32_16x16x4f32).
//
// Workgroup = (run, segment, head, 64 NT value columns), 4 waves; 16 NCH tokens at a time. Wave w prepares chunk w: the
// scaled queries and keys (a lane per key channel) and A (a lane per key token and quarter of the channels, walking down the
// rows with the running product). Then every wave runs the chunks on its 16 NT columns, the state in accumulators: their
// layout is that of the other product's B operand, so the state never moves. The next tokens' loads are in flight
// meanwhile. Where one workgroup holds a head's columns, it ends with the head's norm, its weight and the gate.
//
// Segments: a long run is cut into `nseg` segments that run in parallel: (1) every segment but the last from a zero state,
// end state and decay product only; (2) chained into the states the segments start from; (3) all segments with outputs.
//
// Delta rule: S_t = diag(a_t) S_(t-1) + k_t u_t^T with u_t = beta_t (v_t - (diag(a_t) S_(t-1))^T k_t). Inside a chunk
//   u_i = beta_i [ v_i - (k_i P(-1, i))^T S ] - sum_(j < i) L_ij u_j,  L_ij = beta_i sum_d k_i k_j P(j, i),
// so the chunk's u = (1 + L)^-1 diag(beta) (V - K' S): L comes from the same walk as A, the inverse of the unit triangular matrix
// from 16 steps of substitution (a lane per column), and u takes the place of v above. The products' accumulators are again the
// next product's operand. Queries and keys come with a 32-bit factor per token and head. A segment's effect on the state it
// starts from is not diagonal: the first pass also runs the columns of the identity (without values), which end as the matrix M
// of S_end = M S_start + S_local, and the chain multiplies by it (delta_chunk.h).
#pragma once
#include "scan.h"

namespace nls_gla {
using namespace nls_scan;

struct GA {
  const void *q, *k, *v;   // activation type, [rows][ld]: [H * D], [H * D], [H * V]
  const float* a;          // decays in [0, 1], f32 [rows][lda]
  float* o;                // f32 [rows][ldo] (unfused)
  const float* norm;       // fused: [H * V]
  const void* gate;        // fused: [rows][ldg]
  void* out;               // fused: [rows][ldout]
  float* state;            // [slots][sstride]: [H][D][V]
  float* rec;              // segments: [run][nseg][H][D][V]
  float* recw;             // their decay products [run][nseg][H][D]
  const int* runs;
  long ld, lda, ldo, ldg, ldout, sstride;
  int H, D, V, nseg, fused, vec, vecq;
  float rs, eps;
  // delta rule
  const float* fac;        // [rows][2 G]: factors of the queries' heads, of the keys'
  const float* beta;       // [rows][ldb]
  float* recm;             // segments: their matrices [run][nseg][H][D][D]
  long ldf, ldb;
  int G;                   // query and key heads
};

// tokens per segment of a run of n
DEVI int seg_len(int n, int nseg) { return ((n + nseg - 1) / nseg + 63) & ~63; }

template <typename T, int DP, int NT, bool DELTA, int N>
struct GC {
  static constexpr int NCH = N, SC = 16 * NCH;                      // chunks and tokens per round
  static constexpr int LQ = DP + 16;                                // row strides: decays / scaled queries (f32),
  static constexpr int LR = DP + 8;                                 // queries (T),
  static constexpr int LK = 20;                                     // scaled keys, transposed (f32),
  static constexpr int LKR = DP == 32 ? 40 : DP + 16;               // keys (in the place of the scaled ones),
  static constexpr int WC = 64 * NT, LV = WC + 8;                   // values (T)
  static constexpr int LO = WC + 4;                                 // outputs (f32, in the place of queries and keys)
  static constexpr int OQ = 0, OK = OQ + SC * LQ * 4, OE = OK + NCH * DP * LK * 4,
                       OA = OE > SC * LO * 4 ? OE : SC * LO * 4, OG = OA + NCH * 16 * LK * 4,
                       OS = OG + NCH * DP * 4, OR = OS + 4 * SC * 4, OV = OR + SC * LR * (int)sizeof(T),
                       OD = OV + SC * LV * (int)sizeof(T),          // delta: decayed keys, L and the inverse, factors
                       OB = OD + (DELTA ? SC * LQ * 4 : 0), OF = OB + (DELTA ? NCH * 16 * LK * 4 : 0),
                       LDS = OF + (DELTA ? 2 * SC * 4 : 0);
  static_assert(16 * LKR <= DP * LK, "keys in the place of the scaled ones");
};
// as many chunks per round as LDS holds
template <typename T, int DP, int NT, bool DELTA>
constexpr int gc_chunks() {
  if (DP <= 128 && GC<T, DP, NT, DELTA, 4>::LDS <= 160 * 1024) return 4;
  return GC<T, DP, NT, DELTA, 2>::LDS <= 160 * 1024 ? 2 : 1;
}

template <typename T> DEVI void ldt4(const T* p, float (&v)[4]) {
  typedef T t4 __attribute__((ext_vector_type(4)));
  const t4 x = *reinterpret_cast<const t4*>(p);
#pragma unroll
  for (int e = 0; e < 4; ++e) v[e] = (float)x[e];
}

template <typename T, int DP, int NT, bool LOCAL, bool DELTA>
__global__ __launch_bounds__(256, DP <= 64 ? 2 : 1) void gla_chunk_kernel(GA p) {
  typedef GC<T, DP, NT, DELTA, gc_chunks<T, DP, NT, DELTA>()> C;
  static_assert(C::LDS <= 160 * 1024, "LDS");
  constexpr int NCH = C::NCH, SC = C::SC, WC = C::WC, NTD = DP / 16, NDP = (DP + 63) / 64;
  constexpr int NVG = SC * (WC / 4) / 256;                          // groups of 4 values per thread
  extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
  float* aq = reinterpret_cast<float*>(lds + C::OQ);                // [SC][LQ]
  float* kt = reinterpret_cast<float*>(lds + C::OK);                // [NCH][DP][LK]
  float* am = reinterpret_cast<float*>(lds + C::OA);                // [NCH][16][LK]
  float* gm = reinterpret_cast<float*>(lds + C::OG);                // [NCH][DP]
  float* sq = reinterpret_cast<float*>(lds + C::OS);                // [4][SC] sums of squares
  T* rq = reinterpret_cast<T*>(lds + C::OR);                        // [SC][LR]
  T* vs = reinterpret_cast<T*>(lds + C::OV);                        // [SC][LV]
  float* kd = reinterpret_cast<float*>(lds + C::OD);                // delta: [SC][LQ] decayed keys, negated
  float* bm = reinterpret_cast<float*>(lds + C::OB);                // delta: [NCH][16][LK] L, then the inverse
  float* qs = reinterpret_cast<float*>(lds + C::OF);                // delta: [SC] factors of the queries
  float* bs = qs + SC;                                              // delta: [SC] beta

  const int* run = p.runs + 4 * blockIdx.y;
  int t0 = run[0], n = run[1];
  const int slot = run[2], pos0 = run[3], z = blockIdx.z;
  if (slot < 0 || n < 1) return;
  bool last = true;
  if (p.nseg > 1) {
    const int sl = seg_len(n, p.nseg);
    if (z * sl >= n) return;
    last = (z + 1) * sl >= n;
    if (LOCAL && last) return;
    t0 += z * sl;
    n = min(sl, n - z * sl);
  }
  const int D = p.D, nvb = (p.V + WC - 1) / WC;                     // column blocks: the values', (delta) the identity's
  const int ncb = nvb + (DELTA && LOCAL ? (D + WC - 1) / WC : 0);
  const int head = blockIdx.x / ncb, cb = blockIdx.x % ncb;
  const bool ident = DELTA && LOCAL && cb >= nvb;
  const int V = ident ? D : p.V, c0 = (ident ? cb - nvb : cb) * WC;
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int r = lane & 15, g = lane >> 4;
  const int wc = c0 + wave * 16 * NT;                               // the wave's first column
  const bool act = wc < V;
  const int hq = DELTA ? head / (p.H / p.G) : head;
  const size_t hb = (size_t)head * D, hv = (size_t)head * V, hk = (size_t)hq * D;
  const size_t sst = (size_t)p.H * D * V, swt = (size_t)p.H * D;
  const size_t seg = (size_t)blockIdx.y * p.nseg + z;
  float* st = p.state + (size_t)slot * p.sstride + hb * V;

  // (loads below are never in a branch of their own: addresses are clamped and the value selected afterwards, so that they
  // all are in flight together)
  f32x4 S[NTD][NT];                                                 // rows 16 t + 4 g + i, column wc + 16 c + r
  f32x4 pw[NTD];
  if (LOCAL || (p.nseg == 1 && pos0 == 0)) {
#pragma unroll
    for (int t = 0; t < NTD; ++t)
#pragma unroll
      for (int c = 0; c < NT; ++c)
#pragma unroll
        for (int i = 0; i < 4; ++i) S[t][c][i] = ident && 16 * t + 4 * g + i == wc + 16 * c + r ? 1.f : 0.f;
  } else {
    const float* src = p.nseg > 1 ? p.rec + seg * sst + hb * V : st;
#pragma unroll
    for (int t = 0; t < NTD; ++t)
#pragma unroll
      for (int c = 0; c < NT; ++c)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int d = 16 * t + 4 * g + i, col = wc + 16 * c + r;
          const float x = src[(size_t)min(d, D - 1) * V + min(col, V - 1)];
          S[t][c][i] = d < D && col < V ? x : 0.f;
        }
  }
#pragma unroll
  for (int t = 0; t < NTD; ++t) pw[t] = f32x4{1.f, 1.f, 1.f, 1.f};

  // loads of one round, in groups of 4 columns: a lane takes the channels 4 cg .. of TPL tokens of chunk `wave`
  typedef T t4 __attribute__((ext_vector_type(4)));
  constexpr int TPL = DP / 16;
  const int cg = 4 * (lane % (DP / 4)), ts = TPL * (lane / (DP / 4));
  t4 fq[TPL], fk[TPL], fv[NVG];
  f32x4 fa[TPL];
  float fqs[TPL], fks[TPL], fb = 0.f;                               // delta: the tokens' factors, beta of token `lane`
  auto fetch = [&](int base) __attribute__((always_inline)) {
    if (wave < NCH) {
      const T *qp = (const T*)p.q + hk, *kp = (const T*)p.k + hk;
      const float* ap = p.a + hb;
#pragma unroll
      for (int e = 0; e < TPL; ++e) {
        const size_t row = (size_t)(t0 + min(base + 16 * wave + ts + e, n - 1));
        if (DELTA) {
          fqs[e] = p.fac[row * p.ldf + hq];
          fks[e] = p.fac[row * p.ldf + p.G + hq];
        }
        if (p.vecq) {
          const int d = min(cg, D - 4);
          if (!LOCAL) fq[e] = *reinterpret_cast<const t4*>(qp + row * p.ld + d);
          fk[e] = *reinterpret_cast<const t4*>(kp + row * p.ld + d);
          fa[e] = *reinterpret_cast<const f32x4*>(ap + row * p.lda + d);
        } else {
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int d = min(cg + i, D - 1);
            if (!LOCAL) fq[e][i] = qp[row * p.ld + d];
            fk[e][i] = kp[row * p.ld + d];
            fa[e][i] = ap[row * p.lda + d];
          }
        }
      }
#pragma unroll
      for (int e = 0; e < TPL; ++e)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const bool in = base + 16 * wave + ts + e < n && cg + i < D;
          if (!LOCAL) fq[e][i] = in ? fq[e][i] : (T)0.f;
          fk[e][i] = in ? fk[e][i] : (T)0.f;
          fa[e][i] = in ? fa[e][i] : 1.f;
        }
      if (DELTA) {
        const int tb = base + 16 * wave + r;
        fb = p.beta[(size_t)(t0 + min(tb, n - 1)) * p.ldb + head];
        fb = tb < n ? fb : 0.f;
      }
    }
    if (ident) {
#pragma unroll
      for (int e = 0; e < NVG; ++e) fv[e] = t4{(T)0.f, (T)0.f, (T)0.f, (T)0.f};
      return;
    }
    const T* vp = (const T*)p.v + hv;
    if (p.vec) {
#pragma unroll
      for (int e = 0; e < NVG; ++e) {
        const int x = tid + 256 * e, col = c0 + (x % (WC / 4)) * 4;
        fv[e] = *reinterpret_cast<const t4*>(vp + (size_t)(t0 + min(base + x / (WC / 4), n - 1)) * p.ld + min(col, V - 4));
      }
    } else {
#pragma unroll
      for (int e = 0; e < NVG; ++e) {
        const int x = tid + 256 * e, col = c0 + (x % (WC / 4)) * 4;
#pragma unroll
        for (int i = 0; i < 4; ++i)
          fv[e][i] = vp[(size_t)(t0 + min(base + x / (WC / 4), n - 1)) * p.ld + min(col + i, V - 1)];
      }
    }
#pragma unroll
    for (int e = 0; e < NVG; ++e) {
      const int x = tid + 256 * e, col = c0 + (x % (WC / 4)) * 4;
#pragma unroll
      for (int i = 0; i < 4; ++i) fv[e][i] = base + x / (WC / 4) < n && col + i < V ? fv[e][i] : (T)0.f;
    }
  };
  fetch(0);
  for (int base = 0; base < n; base += SC) {
    // ---- this round's operands
    if (wave < NCH) {
      float* kr = kt + wave * DP * C::LK;
      // as loaded: decays and keys (f32), queries
#pragma unroll
      for (int e = 0; e < TPL; ++e) {
        *reinterpret_cast<f32x4*>(aq + (16 * wave + ts + e) * C::LQ + cg) = fa[e];
        f32x4 kf = f32x4{(float)fk[e][0], (float)fk[e][1], (float)fk[e][2], (float)fk[e][3]};
        if (DELTA) {
          kf *= fks[e];
          if (cg == 0) qs[16 * wave + ts + e] = fqs[e];
        }
        *reinterpret_cast<f32x4*>(kr + (ts + e) * C::LKR + cg) = kf;
        if (!LOCAL) *reinterpret_cast<t4*>(rq + (16 * wave + ts + e) * C::LR + cg) = fq[e];
      }
      if (DELTA && lane < 16) bs[16 * wave + lane] = fb;
      if (!LOCAL || DELTA) {
        // A (and L): lane = (key token j, channels 16 m + 4 dg ..), down the rows i = j, j + 1, ..; rows past the chunk clear the
        // part above the diagonal
        const int j = lane >> 2, dg = lane & 3;
        float uu[NTD][4];
#pragma unroll
        for (int m = 0; m < NTD; ++m) {
          const f32x4 x = *reinterpret_cast<const f32x4*>(kr + j * C::LKR + 16 * m + 4 * dg);
#pragma unroll
          for (int e = 0; e < 4; ++e) uu[m][e] = x[e];
        }
#pragma unroll 4
        for (int s = 0; s < 16; ++s) {
          const int i = j + s;
          const T* qr = rq + (16 * wave + min(i, 15)) * C::LR + 4 * dg;
          const float* ar = aq + (16 * wave + min(i + 1, 15)) * C::LQ + 4 * dg;
          const float* br = kr + min(i, 15) * C::LKR + 4 * dg;
          float acc = 0.f, acb = 0.f;
#pragma unroll
          for (int m = 0; m < NTD; ++m) {
            float x[4] = {0.f, 0.f, 0.f, 0.f};
            f32x4 y = f32x4{0.f, 0.f, 0.f, 0.f};
            if (!LOCAL) ldt4(qr + 16 * m, x);
            if (DELTA) y = *reinterpret_cast<const f32x4*>(br + 16 * m);
            const f32x4 w = *reinterpret_cast<const f32x4*>(ar + 16 * m);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              if (!LOCAL) acc = fmaf(x[e], uu[m][e], acc);
              if (DELTA) acb = fmaf(y[e], uu[m][e], acb);
              uu[m][e] *= w[e];
            }
          }
          if (!LOCAL) {
            acc = dpp_add<0x4E>(dpp_add<0xB1>(acc));
            if (dg == 0)
              am[(wave * 16 + (i & 15)) * C::LK + j] = i < 16 ? acc * (DELTA ? qs[16 * wave + min(i, 15)] : p.rs) : 0.f;
          }
          if (DELTA) {
            acb = dpp_add<0x4E>(dpp_add<0xB1>(acb));
            if (dg == 0) bm[(wave * 16 + (i & 15)) * C::LK + j] = s > 0 && i < 16 ? acb * bs[16 * wave + min(i, 15)] : 0.f;
          }
        }
      }
      if (DELTA) {
        // (1 + L)^-1 diag(beta): a lane per column
        float x[16];
        const int col = lane & 15;
        float* bw = bm + wave * 16 * C::LK;
        __builtin_amdgcn_wave_barrier();
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
#pragma unroll
        for (int i = 0; i < 16; ++i) {
          float acc = col == i ? bs[16 * wave + i] : 0.f;
#pragma unroll
          for (int j = 0; j < i; j += 4) {
            const f32x4 l = *reinterpret_cast<const f32x4*>(bw + i * C::LK + j);
#pragma unroll
            for (int e = 0; e < 4; ++e)
              if (j + e < i) acc = fmaf(-l[e], x[j + e], acc);
          }
          x[i] = acc;
        }
        __builtin_amdgcn_wave_barrier();
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
        if (lane < 16)
#pragma unroll
          for (int i = 0; i < 16; ++i) bw[i * C::LK + col] = x[i];
      }
      // the products: a lane per channel
      float kx[NDP][16];
#pragma unroll
      for (int u = 0; u < NDP; ++u)
#pragma unroll
        for (int t = 0; t < 16; ++t) kx[u][t] = kr[t * C::LKR + min(lane + 64 * u, DP - 1)];
#pragma unroll
      for (int u = 0; u < NDP; ++u) {
        const int d = lane + 64 * u;
        if (DP >= 64 || d < DP) {
          float ax[16], w = 1.f;
#pragma unroll
          for (int t = 0; t < 16; ++t) ax[t] = aq[(16 * wave + t) * C::LQ + d];
#pragma unroll
          for (int t = 0; t < 16; ++t) {
            w *= ax[t];
            if (DELTA) kd[(16 * wave + t) * C::LQ + d] = -kx[u][t] * w;
            if (!LOCAL)
              aq[(16 * wave + t) * C::LQ + d] = (float)rq[(16 * wave + t) * C::LR + d] * w * (DELTA ? qs[16 * wave + t] : p.rs);
          }
          gm[wave * DP + d] = w;
          w = 1.f;
#pragma unroll
          for (int t = 15; t >= 0; --t) {
            kx[u][t] *= w;
            w *= ax[t];
          }
#pragma unroll
          for (int t = 0; t < 16; t += 4)
            *reinterpret_cast<f32x4*>(kr + d * C::LK + t) = f32x4{kx[u][t], kx[u][t + 1], kx[u][t + 2], kx[u][t + 3]};
        }
      }
    }
#pragma unroll
    for (int e = 0; e < NVG; ++e) {
      const int x = tid + 256 * e;
      *reinterpret_cast<t4*>(vs + (x / (WC / 4)) * C::LV + (x % (WC / 4)) * 4) = fv[e];
    }
    __syncthreads();
    if (base + SC < n) fetch(base + SC);
    // ---- the chunks, one after the other
    f32x4 O[NCH][NT];
#pragma unroll
    for (int ch = 0; ch < NCH; ++ch)
#pragma unroll
      for (int c = 0; c < NT; ++c) O[ch][c] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (act)
#pragma unroll
      for (int ch = 0; ch < NCH; ++ch) {
        if (base + 16 * ch >= n) continue;                          // (uniform)
        float v[NT][4];
#pragma unroll
        for (int c = 0; c < NT; ++c)
#pragma unroll
          for (int s = 0; s < 4; ++s) v[c][s] = (float)vs[(16 * ch + 4 * g + s) * C::LV + wave * 16 * NT + 16 * c + r];
        if (DELTA) {
          f32x4 X[NT], U[NT];
#pragma unroll
          for (int c = 0; c < NT; ++c) {
            X[c] = f32x4{v[c][0], v[c][1], v[c][2], v[c][3]};
            U[c] = f32x4{0.f, 0.f, 0.f, 0.f};
          }
#pragma unroll
          for (int t = 0; t < NTD; ++t) {
            const f32x4 ka = *reinterpret_cast<const f32x4*>(kd + (16 * ch + r) * C::LQ + 16 * t + 4 * g);
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
              for (int c = 0; c < NT; ++c) X[c] = __builtin_amdgcn_mfma_f32_16x16x4f32(ka[i], S[t][c][i], X[c], 0, 0, 0);
          }
          const f32x4 ta = *reinterpret_cast<const f32x4*>(bm + (ch * 16 + r) * C::LK + 4 * g);
#pragma unroll
          for (int s = 0; s < 4; ++s)
#pragma unroll
            for (int c = 0; c < NT; ++c) U[c] = __builtin_amdgcn_mfma_f32_16x16x4f32(ta[s], X[c][s], U[c], 0, 0, 0);
#pragma unroll
          for (int c = 0; c < NT; ++c)
#pragma unroll
            for (int s = 0; s < 4; ++s) v[c][s] = U[c][s];
        }
        if (!LOCAL) {
#pragma unroll
          for (int t = 0; t < NTD; ++t) {
            const f32x4 qa = *reinterpret_cast<const f32x4*>(aq + (16 * ch + r) * C::LQ + 16 * t + 4 * g);
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
              for (int c = 0; c < NT; ++c)
                O[ch][c] = __builtin_amdgcn_mfma_f32_16x16x4f32(qa[i], S[t][c][i], O[ch][c], 0, 0, 0);
          }
          const f32x4 aa = *reinterpret_cast<const f32x4*>(am + (ch * 16 + r) * C::LK + 4 * g);
#pragma unroll
          for (int s = 0; s < 4; ++s)
#pragma unroll
            for (int c = 0; c < NT; ++c) O[ch][c] = __builtin_amdgcn_mfma_f32_16x16x4f32(aa[s], v[c][s], O[ch][c], 0, 0, 0);
        }
#pragma unroll
        for (int t = 0; t < NTD; ++t) {
          const f32x4 w = *reinterpret_cast<const f32x4*>(gm + ch * DP + 16 * t + 4 * g);
          const f32x4 ka = *reinterpret_cast<const f32x4*>(kt + (ch * DP + 16 * t + r) * C::LK + 4 * g);
          if (LOCAL && !DELTA) pw[t] *= w;
#pragma unroll
          for (int c = 0; c < NT; ++c) S[t][c] *= w;
#pragma unroll
          for (int s = 0; s < 4; ++s)
#pragma unroll
            for (int c = 0; c < NT; ++c) S[t][c] = __builtin_amdgcn_mfma_f32_16x16x4f32(ka[s], v[c][s], S[t][c], 0, 0, 0);
        }
      }
    // ---- outputs: lane holds tokens 16 ch + 4 g + i, columns wc + 16 c + r
    if (!LOCAL && !p.fused && act) {
#pragma unroll
      for (int ch = 0; ch < NCH; ++ch)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int tt = base + 16 * ch + 4 * g + i;
#pragma unroll
          for (int c = 0; c < NT; ++c)
            if (tt < n && wc + 16 * c + r < V) p.o[(size_t)(t0 + tt) * p.ldo + hv + wc + 16 * c + r] = O[ch][c][i];
        }
    }
    if (!LOCAL && p.fused) {
      // head norm, weight and gate: the outputs pass through LDS, so that rows are read and written in groups of 4 columns
      float* ob = aq;                                               // [SC][LO]
      t4 gt[NVG];
#pragma unroll
      for (int e = 0; e < NVG; ++e) {
        const int x = tid + 256 * e, col = (x % (WC / 4)) * 4;
        const T* gp = (const T*)p.gate + (size_t)(t0 + min(base + x / (WC / 4), n - 1)) * p.ldg + hv;
        if (p.vec) gt[e] = *reinterpret_cast<const t4*>(gp + min(col, V - 4));
        else
#pragma unroll
          for (int i = 0; i < 4; ++i) gt[e][i] = gp[min(col + i, V - 1)];
      }
#pragma unroll
      for (int ch = 0; ch < NCH; ++ch)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          float s = 0.f;                                            // (columns past V hold zeros)
#pragma unroll
          for (int c = 0; c < NT; ++c) s += O[ch][c][i] * O[ch][c][i];
          s = dpp_add<0x140>(dpp_add<0x141>(dpp_add<0x4E>(dpp_add<0xB1>(s))));
          if (r == 0) sq[wave * SC + 16 * ch + 4 * g + i] = s;
        }
      __syncthreads();
#pragma unroll
      for (int ch = 0; ch < NCH; ++ch)
#pragma unroll
        for (int c = 0; c < NT; ++c)
#pragma unroll
          for (int i = 0; i < 4; ++i) ob[(16 * ch + 4 * g + i) * C::LO + wave * 16 * NT + 16 * c + r] = O[ch][c][i];
      __syncthreads();
#pragma unroll
      for (int e = 0; e < NVG; ++e) {
        const int x = tid + 256 * e, tr = x / (WC / 4), col = (x % (WC / 4)) * 4, tt = base + tr;
        const float s = sq[tr] + sq[SC + tr] + sq[2 * SC + tr] + sq[3 * SC + tr];
        const float inv = 1.f / sqrtf(s / (float)V + p.eps);
        const f32x4 o = *reinterpret_cast<const f32x4*>(ob + tr * C::LO + col);
        T* op = (T*)p.out + (size_t)(t0 + tt) * p.ldout + hv + col;
        if (tt >= n) continue;
        if (p.vec) {
          if (col < V) {
            const f32x4 nw = *reinterpret_cast<const f32x4*>(p.norm + hv + col);
            *reinterpret_cast<t4*>(op) = t4{(T)(o[0] * inv * nw[0] * (float)gt[e][0]), (T)(o[1] * inv * nw[1] * (float)gt[e][1]),
                                            (T)(o[2] * inv * nw[2] * (float)gt[e][2]), (T)(o[3] * inv * nw[3] * (float)gt[e][3])};
          }
        } else {
#pragma unroll
          for (int i = 0; i < 4; ++i)
            if (col + i < V) op[i] = (T)(o[i] * inv * p.norm[hv + col + i] * (float)gt[e][i]);
        }
      }
    }
    __syncthreads();
  }
  // ---- the state of the run, or of a segment that another one follows
  if (!act || !(last || LOCAL)) return;
  float* dst = ident ? p.recm + seg * sst + hb * V : LOCAL ? p.rec + seg * sst + hb * V : st;
#pragma unroll
  for (int t = 0; t < NTD; ++t)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 16 * t + 4 * g + i;
#pragma unroll
      for (int c = 0; c < NT; ++c)
        if (d < D && wc + 16 * c + r < V) dst[(size_t)d * V + wc + 16 * c + r] = S[t][c][i];
      if (LOCAL && !DELTA && wc + r == 0 && d < D) p.recw[seg * swt + hb + d] = pw[t][i];
    }
}

// LDS of a kernel beyond the default limit
template <int LDS>
inline int gla_lds(const void* a, const void* b) {
  for (const void* f : {a, b})
    if (hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, LDS) != hipSuccess) return -1;
  return 0;
}

inline GA gla_args(const void* q, const void* k, const void* v, long ld, const float* a, long lda, float qscale, float* o, long ldo,
                   const float* norm, const void* gate, long ldg, void* out, long ldout, float eps, float* state, long sstride,
                   const int* runs, int H, int D, int V, int nseg, float* rec, float* recw, int f32) {
  const bool fused = norm && gate && out;
  const long al = f32 ? 16 : 8;
  const int vec = V % 4 == 0 && ld % 4 == 0 && (long)((uintptr_t)v % al) == 0 &&
                  (!fused || (ldg % 4 == 0 && ldout % 4 == 0 && (long)(((uintptr_t)gate | (uintptr_t)out) % al) == 0 &&
                              (uintptr_t)norm % 16 == 0));
  const int vecq = D % 4 == 0 && ld % 4 == 0 && lda % 4 == 0 && (long)(((uintptr_t)q | (uintptr_t)k) % al) == 0 &&
                   (uintptr_t)a % 16 == 0;
  GA p{};
  p.q = q, p.k = k, p.v = v, p.a = a, p.o = o, p.norm = norm, p.gate = gate, p.out = out, p.state = state, p.rec = rec;
  p.recw = recw, p.runs = runs, p.ld = ld, p.lda = lda, p.ldo = ldo, p.ldg = ldg, p.ldout = ldout, p.sstride = sstride;
  p.H = H, p.D = D, p.V = V, p.nseg = nseg, p.fused = fused, p.vec = vec, p.vecq = vecq, p.rs = qscale, p.eps = eps, p.G = H;
  return p;
}

}  // namespace nls_gla
