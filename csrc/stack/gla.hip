// Gated linear attention (gfx950): the recurrence over runs of tokens in chunks on f32 MFMA, and the entry point of its
// single-token step (scan.h). Keys and values may differ in width.
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
};

// tokens per segment of a run of n
DEVI int seg_len(int n, int nseg) { return ((n + nseg - 1) / nseg + 63) & ~63; }

template <typename T, int DP, int NT>
struct GC {
  static constexpr int NCH = DP <= 128 ? 4 : 2, SC = 16 * NCH;      // chunks and tokens per round
  static constexpr int LQ = DP + 16;                                // row strides: decays / scaled queries (f32),
  static constexpr int LR = DP + 8;                                 // queries (T),
  static constexpr int LK = 20;                                     // scaled keys, transposed (f32),
  static constexpr int LKR = DP == 32 ? 40 : DP + 16;               // keys (in the place of the scaled ones),
  static constexpr int WC = 64 * NT, LV = WC + 8;                   // values (T)
  static constexpr int LO = WC + 4;                                 // outputs (f32, in the place of queries and keys)
  static constexpr int OQ = 0, OK = OQ + SC * LQ * 4, OE = OK + NCH * DP * LK * 4,
                       OA = OE > SC * LO * 4 ? OE : SC * LO * 4, OG = OA + NCH * 16 * LK * 4,
                       OS = OG + NCH * DP * 4, OR = OS + 4 * SC * 4, OV = OR + SC * LR * (int)sizeof(T),
                       LDS = OV + SC * LV * (int)sizeof(T);
  static_assert(16 * LKR <= DP * LK && LDS <= 160 * 1024, "LDS");
};

template <typename T> DEVI void ldt4(const T* p, float (&v)[4]) {
  typedef T t4 __attribute__((ext_vector_type(4)));
  const t4 x = *reinterpret_cast<const t4*>(p);
#pragma unroll
  for (int e = 0; e < 4; ++e) v[e] = (float)x[e];
}

template <typename T, int DP, int NT, bool LOCAL>
__global__ __launch_bounds__(256, DP <= 64 ? 2 : 1) void gla_chunk_kernel(GA p) {
  typedef GC<T, DP, NT> C;
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
  const int D = p.D, V = p.V, ncb = (V + WC - 1) / WC;
  const int head = blockIdx.x / ncb, c0 = (blockIdx.x % ncb) * WC;
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int r = lane & 15, g = lane >> 4;
  const int wc = c0 + wave * 16 * NT;                               // the wave's first column
  const bool act = wc < V;
  const size_t hb = (size_t)head * D, hv = (size_t)head * V;
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
      for (int c = 0; c < NT; ++c) S[t][c] = f32x4{0.f, 0.f, 0.f, 0.f};
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
  auto fetch = [&](int base) __attribute__((always_inline)) {
    if (wave < NCH) {
      const T *qp = (const T*)p.q + hb, *kp = (const T*)p.k + hb;
      const float* ap = p.a + hb;
#pragma unroll
      for (int e = 0; e < TPL; ++e) {
        const size_t row = (size_t)(t0 + min(base + 16 * wave + ts + e, n - 1));
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
        *reinterpret_cast<f32x4*>(kr + (ts + e) * C::LKR + cg) =
            f32x4{(float)fk[e][0], (float)fk[e][1], (float)fk[e][2], (float)fk[e][3]};
        if (!LOCAL) *reinterpret_cast<t4*>(rq + (16 * wave + ts + e) * C::LR + cg) = fq[e];
      }
      if (!LOCAL) {
        // A: lane = (key token j, channels 16 m + 4 dg ..), down the rows i = j, j + 1, ..; rows past the chunk clear the
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
          float acc = 0.f;
#pragma unroll
          for (int m = 0; m < NTD; ++m) {
            float x[4];
            ldt4(qr + 16 * m, x);
            const f32x4 w = *reinterpret_cast<const f32x4*>(ar + 16 * m);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              acc = fmaf(x[e], uu[m][e], acc);
              uu[m][e] *= w[e];
            }
          }
          acc = dpp_add<0x4E>(dpp_add<0xB1>(acc));
          if (dg == 0) am[(wave * 16 + (i & 15)) * C::LK + j] = i < 16 ? acc * p.rs : 0.f;
        }
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
            if (!LOCAL) aq[(16 * wave + t) * C::LQ + d] = (float)rq[(16 * wave + t) * C::LR + d] * w * p.rs;
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
          if (LOCAL) pw[t] *= w;
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
  float* dst = LOCAL ? p.rec + seg * sst + hb * V : st;
#pragma unroll
  for (int t = 0; t < NTD; ++t)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 16 * t + 4 * g + i;
#pragma unroll
      for (int c = 0; c < NT; ++c)
        if (d < D && wc + 16 * c + r < V) dst[(size_t)d * V + wc + 16 * c + r] = S[t][c][i];
      if (LOCAL && wc + r == 0 && d < D) p.recw[seg * swt + hb + d] = pw[t][i];
    }
}

// the states that the segments of each run start from, in the place of their end states
__global__ __launch_bounds__(256) void gla_chain_kernel(GA p) {
  const int* run = p.runs + 4 * blockIdx.y;
  const int n = run[1], slot = run[2];
  if (slot < 0 || n < 1) return;
  const size_t sst = (size_t)p.H * p.D * p.V, swt = (size_t)p.H * p.D;
  const int m = (n + seg_len(n, p.nseg) - 1) / seg_len(n, p.nseg);
  float* rec = p.rec + (size_t)blockIdx.y * p.nseg * sst;
  const float* rw = p.recw + (size_t)blockIdx.y * p.nseg * swt;
  for (size_t e = (size_t)blockIdx.x * 256 + threadIdx.x; e < sst; e += (size_t)gridDim.x * 256) {
    float s = run[3] > 0 ? p.state[(size_t)slot * p.sstride + e] : 0.f;
    const size_t w = e / p.V;
    for (int z = 0; z + 1 < m; ++z) {
      const float l = rec[z * sst + e];
      rec[z * sst + e] = s;
      s = fmaf(rw[z * swt + w], s, l);
    }
    rec[(size_t)(m - 1) * sst + e] = s;
  }
}

template <typename T, int DP, int NT>
int chunk_t(GA p, int nruns, hipStream_t st) {
  typedef GC<T, DP, NT> C;
  static bool attr = false;
  if (!attr) {
    for (const void* f : {(const void*)gla_chunk_kernel<T, DP, NT, false>, (const void*)gla_chunk_kernel<T, DP, NT, true>})
      if (hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, C::LDS) != hipSuccess) return -1;
    attr = true;
  }
  const int nx = p.H * ((p.V + C::WC - 1) / C::WC);
  if (p.fused && p.V > C::WC) return -1;
  if (p.nseg > 1) {
    hipLaunchKernelGGL((gla_chunk_kernel<T, DP, NT, true>), dim3(nx, nruns, p.nseg - 1), dim3(256), C::LDS, st, p);
    const long n = (long)p.H * p.D * p.V;
    hipLaunchKernelGGL(gla_chain_kernel, dim3((int)min((n + 255) / 256, 4096L), nruns), dim3(256), 0, st, p);
  }
  hipLaunchKernelGGL((gla_chunk_kernel<T, DP, NT, false>), dim3(nx, nruns, p.nseg), dim3(256), C::LDS, st, p);
  return (int)hipGetLastError();
}

template <typename T>
int chunk_d(const GA& p, int nruns, int nt, hipStream_t st) {
#define NLS_GC(DP) \
  if (p.D <= DP) return nt == 1 ? chunk_t<T, DP, 1>(p, nruns, st) : nt == 2 ? chunk_t<T, DP, 2>(p, nruns, st) : -1;
  NLS_GC(32) NLS_GC(64) NLS_GC(128) NLS_GC(256)
#undef NLS_GC
  return -1;
}

}  // namespace nls_gla

extern "C" {
using namespace nls_gla;

// nt: 64 nt value columns per workgroup (1, 2). norm and gate given: out = (o / rms(o) per head) * norm * gate, for V up to
// 64 nt; else o. nseg > 1: rec [nruns][nseg][H][D][V] and recw [nruns][nseg][H][D] scratch. D up to 256.
int nls_gla_scan(const void* q, const void* k, const void* v, long ld, const float* a, long lda, float qscale, float* o,
                 long ldo, const float* norm, const void* gate, long ldg, void* out, long ldout, float eps, float* state,
                 long sstride, const int* runs, int nruns, int H, int D, int V, int nseg, float* rec, float* recw, int nt,
                 int f32, void* stream) {
  const bool fused = norm && gate && out;
  if (nruns < 1 || H < 1 || D < 1 || V < 1 || nseg < 1 || nseg > 64 || (nseg > 1 && (!rec || !recw)) || (!fused && !o)) return -1;
  const long al = f32 ? 16 : 8;
  const int vec = V % 4 == 0 && ld % 4 == 0 && (long)((uintptr_t)v % al) == 0 &&
                  (!fused || (ldg % 4 == 0 && ldout % 4 == 0 && (long)(((uintptr_t)gate | (uintptr_t)out) % al) == 0 &&
                              (uintptr_t)norm % 16 == 0));
  const int vecq = D % 4 == 0 && ld % 4 == 0 && lda % 4 == 0 && (long)(((uintptr_t)q | (uintptr_t)k) % al) == 0 &&
                   (uintptr_t)a % 16 == 0;
  const GA p{q, k, v, a, o, norm, gate, out, state, rec, recw, runs, ld, lda, ldo, ldg, ldout, sstride, H, D, V, nseg, fused, vec,
             vecq, qscale, eps};
  return f32 ? chunk_d<float>(p, nruns, nt, (hipStream_t)stream) : chunk_d<__bf16>(p, nruns, nt, (hipStream_t)stream);
}

// every run has one token (or none); V a multiple of 4, at most 1024; D at most 256. Decays: a, or (a null) from the low-rank
// gate input `low` (row stride ld, 16-byte aligned rows) with a2 [H * D][rank] in the activation type: sigmoid(a2 low + a2b)^ia
int nls_gla_step(const void* q, const void* k, const void* v, long ld, const float* a, long lda, const void* low, const void* a2,
                 const float* a2b, int rank, float ia, float qscale, float* state, long sstride, const int* runs, int nruns,
                 const float* norm, const void* gate, long ldg, void* out, long ldout, int H, int D, int V, float eps, int f32,
                 void* stream) {
  if (!a && (!low || !a2 || !a2b || rank < 1 || ((uintptr_t)low & 15) || ((uintptr_t)a2 & 15) || (ld & 7))) return -1;
  const Scan p{q, k, v, a, nullptr, nullptr, state, nullptr, nullptr, runs, ld, lda, 0, sstride, 0, 0, H, D, V, 0, qscale,
               low, a2, a2b, rank, ia};
  return f32 ? step_rows<float, GLA>(p, nruns, norm, gate, ldg, out, ldout, eps, (hipStream_t)stream)
             : step_rows<__bf16, GLA>(p, nruns, norm, gate, ldg, out, ldout, eps, (hipStream_t)stream);
}

}  // extern "C"
