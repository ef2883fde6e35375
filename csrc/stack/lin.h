// Linear layers on packed bf16 / f32 weights (gfx950): the operand layout, launch descriptors and epilogues shared
// by the few-row kernel (lin_small.hip) and the tiled MFMA GEMM (lin_gemm.hip).
//
//   y[m, n] = epi(sum_k x[m, k] * W[n, k])        x, W: bf16 (f32 accumulate) or f32 (f32 MFMA throughout)
//
// Packed weights: [N / 16 tiles][K / KS sub-tiles] of 1 KiB. A sub-tile is 16 rows x 64 bytes (KS = 32 bf16 or 16
// f32 values) in MFMA fragment order: lane 16 g + r owns bytes 16 (16 g + r) .. +16 = row r, k = EL g .. EL g + EL - 1
// (EL = 8 or 4). Few-row launches stream it with 1 KiB wave loads, the GEMM's LDS-DMA copies sub-tiles verbatim and
// reads them back lane-linearly. N is padded to 16 and K to 2 KS * (1 or 2) with zeros; activation rows are readable
// (and finite) up to the padded K. For f32 the four k of a lane are the j-th operands of four 16x16x4 MFMAs: both
// operands use the same k order, so the sum is over the same products.
//
// A segment without an epilogue may split K over `ks` workgroups per tile: each writes an f32 slab of its own (`yks` apart), which
// the caller's next kernel adds.
// A launch holds up to LIN_SEGS segments (own x, W, y, epilogue), so independent projections share one grid. A segment
// may be a batch of `ng` groups (per-head products: column offsets xgs / ygs per group), or routed: its (group, rows)
// tiles come from a device list written by moe_plan_kernel and its rows from the routed-entry list.
#pragma once
#include "../kernels/common.h"

namespace nls_lin {

constexpr int LIN_SEGS = 6;
constexpr int LIN_GM = 4;      // row tiles that are walked together down the weights (lin_tile)

enum LinEpi : int {
  LE_NONE = 0, LE_SILU = 1, LE_TANH = 2, LE_SIGMOID = 3, LE_RELU2 = 4,
  LE_DECAY = 5,     // exp(-exp(v + bias[n]))
  LE_GATE = 6,      // v * gate[m * ldg + group]
  LE_ROPE = 7,      // rotate the pairs (n, n + 1), n % cb < 2 * half, with cs[pos[m]]
  LE_GEGLU = 8,     // gelu_tanh(v[n]) * v[n + 1] -> column n / 2 (gate and up rows of the weights alternate)
  LE_SIGPOW = 9,    // sigmoid(v + bias[n]) ^ alpha, or (gate given) ^ gate[n]
  LE_SOFTCAP = 10,  // alpha * tanh(v / alpha)
  LE_SWIGLU = 11,   // g = min(v[n], alpha), u = v[n + 1] clamped to +- alpha: g sigmoid(1.702 g) (u + 1) -> column n / 2
  LE_SILUGLU = 12,  // silu(v[n]) * v[n + 1] -> column n / 2
};                  // LE_SIGMOID: alpha * sigmoid(v)

struct LinSeg {
  const void* w;        // packed weights of group 0
  const void* x;
  void* y;
  const float* bias;
  const float* gate;
  const float* cs;      // [positions][half][2] cos, sin
  const int* pos;
  const int* rows;      // routed entries (null: rows 0 .. M - 1)
  const int* xmap;      // x row of row m (null: m); identity segments only
  long wstride;         // bytes between the groups' packed weights
  long ldx, ldy;        // elements
  long xgs, ygs;        // column offset per group (elements)
  long yks;             // elements between the slabs of a split K
  int N, nsub;          // output columns; 1 KiB sub-tiles per 16-row tile
  int M, ng;
  int epi, yact;        // yact: store the activation type (bf16; f32 in f32 launches), else f32
  int cb, cstep;        // output column n -> (n / cb) * cstep + n % cb
  int xdiv, ldg;        // routed: x row = entry / xdiv
  int half;
  float alpha;          // constant of the epilogue
  int ks, pad0;         // K splits (identity segments without an epilogue; 1: none)
};

struct LinArgs {
  LinSeg s[LIN_SEGS];
  const int* tiles;     // routed: [max][4] (group, first entry of the list, rows, 0)
  const int* ntiles;    // routed: tiles in the list
  int nseg, maxtiles;
  int begin[LIN_SEGS + 1];   // first tile id of each segment (filled by the launcher)
  int nmt[LIN_SEGS];         // m-tiles of each segment
};

template <typename T> struct LT;
template <> struct LT<__bf16> {
  static constexpr int KS = 32, EL = 8;
  static DEVI f32x4 mma(const u32x4& a, const u32x4& b, const f32x4& c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0,
                                                   0, 0);
  }
};
template <> struct LT<float> {
  static constexpr int KS = 16, EL = 4;
  static DEVI f32x4 mma(const u32x4& a, const u32x4& b, f32x4 c) {
    const f32x4 x = __builtin_bit_cast(f32x4, a), y = __builtin_bit_cast(f32x4, b);
#pragma unroll
    for (int j = 0; j < 4; ++j) c = __builtin_amdgcn_mfma_f32_16x16x4f32(x[j], y[j], c, 0, 0, 0);
    return c;
  }
};

// one workgroup's tile: segment, group, split of K, first weight row, first row, rows
struct LinTile {
  int seg, grp, ks, n0, m0, cnt;
  const int* rows;      // routed: entries of this tile
};

// tile id -> tile (BN weight rows x BM rows); false: past the routed list
template <int BN, int BM>
DEVI bool lin_tile(const LinArgs& a, int id, LinTile& t) {
  int s = 0;
#pragma unroll
  for (int i = 1; i < LIN_SEGS; ++i)
    if (i < a.nseg && id >= a.begin[i]) s = i;
  const LinSeg& S = a.s[s];
  int q = id - a.begin[s];
  const int nmt = a.nmt[s];
  const int nnt = (S.N + BN - 1) / BN;
  int mi = q % nmt, ni = q / nmt;
  if (nmt > LIN_GM && !S.rows && S.ng == 1 && S.ks == 1) {
    // LIN_GM row tiles at a time: the workgroups that an XCD runs together share weight tiles and row tiles in its L2
    const int first = q / (LIN_GM * nnt) * LIN_GM, gm = min(LIN_GM, nmt - first), r = q - first * nnt;
    mi = first + r % gm;
    ni = r / gm;
  }
  q = ni;
  t.seg = s;
  t.n0 = (q % nnt) * BN;
  t.ks = 0;
  if (S.rows) {
    if (mi >= *a.ntiles) return false;
    t.grp = a.tiles[4 * mi];
    t.rows = S.rows + a.tiles[4 * mi + 1];
    t.cnt = a.tiles[4 * mi + 2];
    t.m0 = 0;
  } else {
    q /= nnt;
    t.grp = S.ng == 1 ? 0 : q % S.ng;
    t.ks = S.ng == 1 ? q : q / S.ng;
    t.rows = nullptr;
    t.m0 = mi * BM;
    t.cnt = min(BM, S.M - t.m0);
  }
  return true;
}

// x row and y row of tile row i (clamped to the tile's rows)
DEVI void lin_row(const LinSeg& S, const LinTile& t, int i, int& xr, int& yr) {
  i = min(i, t.cnt - 1);
  if (t.rows) {
    yr = t.rows[i];
    xr = yr / S.xdiv;
  } else {
    yr = t.m0 + i;
    xr = S.xmap ? S.xmap[yr] : yr;
  }
}

constexpr float LOG2E = 1.4426950408889634f;
DEVI float lin_sigmoid(float v) { return __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-v * LOG2E)); }
// z / 2 (1 + tanh(y)) = z sigmoid(2 y), y = sqrt(2 / pi) (z + 0.044715 z^3)
DEVI float lin_gelu(float z) { return z * lin_sigmoid(1.5957691216057308f * fmaf(0.044715f * z * z, z, z)); }

// clamped gate and up: g sigmoid(1.702 g) (u + 1)
DEVI float lin_swiglu(float g, float u, float lim) {
  g = fminf(g, lim);
  return g * lin_sigmoid(1.702f * g) * (fminf(fmaxf(u, -lim), lim) + 1.f);
}

DEVI float lin_glu(const LinSeg& S, float g, float u) {
  return S.epi == LE_SWIGLU ? lin_swiglu(g, u, S.alpha) : (S.epi == LE_SILUGLU ? g * lin_sigmoid(g) : lin_gelu(g)) * u;
}

// sigmoid(z)^a = 2^(-a (max(-z, 0) log2(e) + log2(1 + u))), u = e^-|z|; log2(w) u / (w - 1) with w = fl(1 + u) keeps the
// digits of a small u
DEVI float lin_sigpow(float z, float a) {
  const float u = __builtin_amdgcn_exp2f(-fabsf(z) * LOG2E), w = 1.f + u;
  const float l = w == 1.f ? u * LOG2E : __builtin_amdgcn_logf(w) * (u * __builtin_amdgcn_rcpf(w - 1.f));
  return __builtin_amdgcn_exp2f(-a * fmaf(fmaxf(-z, 0.f), LOG2E, l));
}

// epilogue of 4 consecutive output columns n .. n + 3 of one row
template <typename T>
DEVI void lin_store4(const LinSeg& S, int grp, int ks, int n, int yr, f32x4 v) {
  if (n >= S.N) return;
  const int nb = S.cb < S.N ? n / S.cb : 0, nr = n - nb * S.cb;      // (no division where columns are not blocked)
  switch (S.epi) {
    case LE_SILU:
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = v[e] * lin_sigmoid(v[e]);
      break;
    case LE_TANH:
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = tanhf(v[e]);
      break;
    case LE_SIGMOID:
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = S.alpha * lin_sigmoid(v[e]);
      break;
    case LE_RELU2:
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float r = fmaxf(v[e], 0.f);
        v[e] = r * r;
      }
      break;
    case LE_DECAY:
#pragma unroll
      for (int e = 0; e < 4; ++e)
        v[e] = expf(-expf(v[e] + S.bias[min(n + e, S.N - 1)]));
      break;
    case LE_SIGPOW:
#pragma unroll
      for (int e = 0; e < 4; ++e)
        v[e] = lin_sigpow(v[e] + S.bias[min(n + e, S.N - 1)], S.gate ? S.gate[min(n + e, S.N - 1)] : S.alpha);
      break;
    case LE_SOFTCAP:
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = S.alpha * tanhf(v[e] / S.alpha);
      break;
    case LE_GEGLU:
    case LE_SWIGLU:
    case LE_SILUGLU: {                  // N is even: both pairs or the first one lie inside
      const size_t o = (size_t)yr * S.ldy + (size_t)grp * S.ygs + (n >> 1);
      const float a = lin_glu(S, v[0], v[1]), b = lin_glu(S, v[2], v[3]);
      if (S.yact && sizeof(T) == 2) {
        __bf16* y = reinterpret_cast<__bf16*>(S.y) + o;
        typedef __bf16 bf2 __attribute__((ext_vector_type(2)));
        if (n + 4 <= S.N && (o & 1) == 0) *reinterpret_cast<bf2*>(y) = bf2{(__bf16)a, (__bf16)b};
        else {
          y[0] = (__bf16)a;
          if (n + 4 <= S.N) y[1] = (__bf16)b;
        }
      } else {
        float* y = reinterpret_cast<float*>(S.y) + o;
        y[0] = a;
        if (n + 4 <= S.N) y[1] = b;
      }
      return;
    }
    case LE_GATE: {
      const float gt = S.gate[(size_t)yr * S.ldg + grp];
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] *= gt;
      break;
    }
    case LE_ROPE: {
      const float* cs = S.cs + (size_t)S.pos[yr] * S.half * 2;
#pragma unroll
      for (int e = 0; e < 4; e += 2) {
        const int i = (nr + e) >> 1;
        if (i < S.half) {
          const float c = cs[2 * i], s = cs[2 * i + 1];
          const float p = v[e], q = v[e + 1];
          v[e] = p * c - q * s;
          v[e + 1] = q * c + p * s;
        }
      }
      break;
    }
    default: break;
  }
  const size_t o = (size_t)yr * S.ldy + (size_t)grp * S.ygs + (size_t)nb * S.cstep + nr + (size_t)ks * S.yks;
  const bool full = n + 4 <= S.N && (o & 3) == 0;
  if (S.yact && sizeof(T) == 2) {
    __bf16* y = reinterpret_cast<__bf16*>(S.y) + o;
    typedef __bf16 bf4 __attribute__((ext_vector_type(4)));
    const bf4 b = {(__bf16)v[0], (__bf16)v[1], (__bf16)v[2], (__bf16)v[3]};
    if (full) *reinterpret_cast<bf4*>(y) = b;
    else
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (n + e < S.N) y[e] = b[e];
  } else {
    float* y = reinterpret_cast<float*>(S.y) + o;
    if (full) *reinterpret_cast<f32x4*>(y) = v;
    else
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (n + e < S.N) y[e] = v[e];
  }
}

// Tile ids of a launch with BN x BM tiles; returns the tile count, or -1 for a descriptor the kernels do not take.
inline int lin_count(LinArgs& a, int BN, int BM) {
  if (a.nseg < 1 || a.nseg > LIN_SEGS) return -1;
  int n = 0;
  for (int i = 0; i < a.nseg; ++i) {
    const LinSeg& S = a.s[i];
    if (S.N < 1 || S.nsub < 2 || (S.nsub & 1) || S.ng < 1 || S.cb < 4 || (S.cb & 3) || S.xdiv < 1) return -1;
    if (!S.w || !S.x || !S.y) return -1;
    if (S.epi == LE_ROPE && (!S.cs || !S.pos)) return -1;
    if ((S.epi == LE_DECAY || S.epi == LE_SIGPOW) && !S.bias) return -1;
    if ((S.epi == LE_GEGLU || S.epi == LE_SWIGLU || S.epi == LE_SILUGLU) && ((S.N & 1) || S.cb < S.N)) return -1;
    if (S.epi == LE_GATE && !S.gate) return -1;
    if (S.ks < 1 || S.ks > S.nsub / 2 || (S.ks > 1 && (S.rows || S.yact || S.epi != LE_NONE))) return -1;
    if (S.rows && (!a.tiles || !a.ntiles || a.maxtiles < 1)) return -1;
    if (!S.rows && S.M < 1) return -1;
    a.begin[i] = n;
    a.nmt[i] = S.rows ? a.maxtiles : (S.M + BM - 1) / BM;
    n += ((S.N + BN - 1) / BN) * a.nmt[i] * (S.rows ? 1 : S.ng * S.ks);
  }
  a.begin[a.nseg] = n;
  return n;
}

}  // namespace nls_lin
