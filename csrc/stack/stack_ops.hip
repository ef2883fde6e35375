// Row kernels of the config-driven decoder stacks (models/stack.py): embedding, norms with the residual add,
// routed-expert combine, attention and latent-attention row preparation, expert routing. The residual stream is f32; `xb`
// is its bf16 rounding, the operand of the next projections where sublayers read the residual itself (f32 launches: null).
#include "../kernels/common.h"

namespace nls_stack {

DEVI float wsum(float v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
  return v;
}

// sum over the workgroup's NW waves; sh: NW floats, reusable on return
template <int NW>
DEVI float bsum(float v, float* sh) {
  v = wsum(v);
  if ((threadIdx.x & 63) == 0) sh[threadIdx.x >> 6] = v;
  __syncthreads();
  float t = 0.f;
#pragma unroll
  for (int i = 0; i < NW; ++i) t += sh[i];
  __syncthreads();
  return t;
}

template <typename T> DEVI float ldv(const T* p, long i) { return (float)p[i]; }
template <typename T> DEVI void stv(T* p, long i, float v) { p[i] = (T)v; }

// ---- x[t] = table[id] * scale (+ the row of the token pair, + the position's vector, + a vector), id from the host or (use_prev) the
// previous step's next_ids. The token ahead of a run's first is the slot's; the run's first row, which alone reads it,
// leaves the run's last token there.
struct Embed {
  int* ids;
  const int *next_ids, *use_prev;
  const __bf16* tab;
  float* x;
  __bf16* xb;              // optional bf16 rounding, row stride ldx
  void *c0, *c1;           // optional copies in the activation type (f32: float), row stride ldc
  const __bf16* pairs;     // optional [buckets + 1][D]
  int* prev;               // [slots]
  const int *runs, *tok_seq;
  const __bf16* ptab;      // optional [npos][D]
  const int* pos;
  const float* add;        // optional [D]
  long ldx, ldc;
  int V, D, buckets, mul_prev, mul_cur, npos, f32, vec;
  float scale;
};

DEVI int token_of(const Embed& p, int t) {
  const int a = p.ids[t], n = p.use_prev ? p.next_ids[t] : 0, u = p.use_prev ? p.use_prev[t] : 0;       // (in flight together)
  return min(max(u ? n : a, 0), p.V - 1);
}

template <int N>
DEVI void embed_cols(const Embed& p, int t, const __bf16* row, const __bf16* pair, const __bf16* pv) {
  typedef __bf16 bfn __attribute__((ext_vector_type(N)));
  typedef float fn __attribute__((ext_vector_type(N)));
  for (int i = threadIdx.x * N; i < p.D; i += 256 * N) {
    const bfn none = (bfn)((__bf16)0.f);
    const bfn a = *reinterpret_cast<const bfn*>(row + i), b = pair ? *reinterpret_cast<const bfn*>(pair + i) : none;
    const bfn c = pv ? *reinterpret_cast<const bfn*>(pv + i) : none;
    fn y;
    bfn yb;
#pragma unroll
    for (int e = 0; e < N; ++e) {
      y[e] = (float)a[e] * p.scale + (float)b[e] + (float)c[e];
      if (p.add) y[e] += p.add[i + e];
      yb[e] = (__bf16)y[e];
    }
    *reinterpret_cast<fn*>(p.x + (size_t)t * p.ldx + i) = y;
    if (p.xb) *reinterpret_cast<bfn*>(p.xb + (size_t)t * p.ldx + i) = yb;
    const size_t o = (size_t)t * p.ldc + i;
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      void* d = k ? p.c1 : p.c0;
      if (!d) continue;
      if (p.f32) *reinterpret_cast<fn*>(reinterpret_cast<float*>(d) + o) = y;
      else *reinterpret_cast<bfn*>(reinterpret_cast<__bf16*>(d) + o) = yb;
    }
  }
}

__global__ __launch_bounds__(256) void embed_kernel(Embed p) {
  const int t = blockIdx.x, id = token_of(p, t);
  const __bf16 *pair = nullptr, *pv = nullptr;
  int keep = -1, slot = -1;
  if (p.pairs) {
    const int* run = p.runs + 4 * p.tok_seq[t];
    const int t0 = run[0], n = run[1], pos0 = run[3];
    slot = run[2];
    long r = p.buckets;
    if (slot >= 0 && t >= t0 && t < t0 + n) {
      if (t > t0 || pos0 > 0) {
        const long before = t > t0 ? token_of(p, t - 1) : p.prev[slot];
        r = (before * p.mul_prev + (long)id * p.mul_cur) % p.buckets;
        if (r < 0) r += p.buckets;
      }
      if (t == t0) keep = token_of(p, t0 + n - 1);
    }
    pair = p.pairs + (size_t)r * p.D;
  }
  if (p.ptab) pv = p.ptab + (size_t)min(max(p.pos[t], 0), p.npos - 1) * p.D;
  __syncthreads();
  if (threadIdx.x == 0) {
    if (p.use_prev) p.ids[t] = id;
    if (keep >= 0) p.prev[slot] = keep;
  }
  const __bf16* row = p.tab + (size_t)id * p.D;
  if (p.vec) embed_cols<8>(p, t, row, pair, pv);
  else embed_cols<1>(p, t, row, pair, pv);
}

// ---- x[t] += norm(y) * w (w null: x[t] += y); y = one row (the sum of `nslab` slabs' rows), or (topk)
// sum_j topw[t][j] * ye[t * topk + j] (+ ye[sh0 + t], the shared expert); y null: x is only read. Optional second norm (the
// next sublayers' or the model's last one) of the new x into `on`. norm: (v - mean) / sqrt(var + eps), or (rms)
// v / sqrt(mean(v^2) + eps), of `groups` equal parts of the row each on its own (rms). `add`, a vector, comes on top of the new x;
// without `keep` the old x is left out. The normed x may go out with two weights (`ow` / `ow2`), and (gate) times a gate per column.
// A workgroup per row (`rows`: gathered), 4 consecutive columns x NV per thread in registers.
struct NormAdd {
  const float* y;
  const float* topw;
  const float* w;
  float* x;
  void* xb;             // optional copy of the new x, activation type
  const float* ow;      // optional output norm weight
  void* on;             // its output, activation type
  const int* rows;      // optional: row i of the launch is row rows[i] of x
  long ldy, ldx, ldo;
  long sh0;             // first shared-expert row, -1: none
  int D, topk, f32, rms;
  float eps;
  int nslab;
  long slab;            // elements between slabs
  long ldxb;
  const float* add;     // optional [D], added to the new x
  int keep;
  const float* ow2;     // optional second weight of the output norm
  void* on2;            // its output, row stride ldo
  const void* gate;     // optional [rows][ldg], activation type: on *= gate
  long ldg;
  int groups;           // parts of the row that are normed each on its own
};

// 4 consecutive values, columns i .. i + 3 of a row of D (VEC: D and the row strides are multiples of 4)
template <bool VEC>
DEVI f32x4 row4(const float* p, int i, int D) {
  f32x4 v = f32x4{0.f, 0.f, 0.f, 0.f};
  if (VEC) {
    if (i < D) v = *reinterpret_cast<const f32x4*>(p + i);
  } else {
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (i + e < D) v[e] = p[i + e];
  }
  return v;
}
template <bool VEC>
DEVI f32x4 row4(const __bf16* p, int i, int D) {
  typedef __bf16 bf4 __attribute__((ext_vector_type(4)));
  f32x4 v = f32x4{0.f, 0.f, 0.f, 0.f};
  if (VEC) {
    if (i < D) {
      const bf4 b = *reinterpret_cast<const bf4*>(p + i);
      v = f32x4{(float)b[0], (float)b[1], (float)b[2], (float)b[3]};
    }
  } else {
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (i + e < D) v[e] = (float)p[i + e];
  }
  return v;
}
template <bool VEC>
DEVI void put4(float* p, int i, int D, const f32x4& v) {
  if (VEC) {
    if (i < D) *reinterpret_cast<f32x4*>(p + i) = v;
  } else {
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (i + e < D) p[i + e] = v[e];
  }
}
template <bool VEC>
DEVI void put4(__bf16* p, int i, int D, const f32x4& v) {
  typedef __bf16 bf4 __attribute__((ext_vector_type(4)));
  const bf4 b = {(__bf16)v[0], (__bf16)v[1], (__bf16)v[2], (__bf16)v[3]};
  if (VEC) {
    if (i < D) *reinterpret_cast<bf4*>(p + i) = b;
  } else {
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (i + e < D) p[i + e] = b[e];
  }
}
// RMS norm of `groups` parts of the row each on its own. Parts of whole 256 columns are sums of the waves' sums, others are added up
// from the squares in LDS (sh: D + groups floats).
template <int NV, int NTH>
DEVI void normalise_groups(f32x4 (&v)[NV], int D, float eps, int groups, float* sh) {
  constexpr int NW = NTH / 64;
  const int gs = D / groups, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  if (!(gs & 255)) {
    const int per = gs >> 8;                       // 256-column slots of a part; slot j * NW + wave holds columns 256 slot ..
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const float s = wsum((v[j][0] * v[j][0] + v[j][1] * v[j][1]) + (v[j][2] * v[j][2] + v[j][3] * v[j][3]));
      if (lane == 0) sh[j * NW + wave] = s;
    }
    __syncthreads();
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int s0 = (j * NW + wave) / per * per;
      if (s0 >= D >> 8) continue;
      float s = 0.f;
      for (int i = 0; i < per; ++i) s += sh[s0 + i];
      v[j] *= 1.f / sqrtf(s / (float)gs + eps);
    }
    __syncthreads();
    return;
  }
#pragma unroll
  for (int j = 0; j < NV; ++j)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = (int)(threadIdx.x + j * NTH) * 4 + e;
      if (i < D) sh[i] = v[j][e] * v[j][e];
    }
  __syncthreads();
  for (int g = wave; g < groups; g += NW) {
    float s = 0.f;
    for (int i = lane; i < gs; i += 64) s += sh[g * gs + i];
    s = wsum(s);
    if (lane == 0) sh[D + g] = 1.f / sqrtf(s / (float)gs + eps);
  }
  __syncthreads();
#pragma unroll
  for (int j = 0; j < NV; ++j)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = (int)(threadIdx.x + j * NTH) * 4 + e;
      if (i < D) v[j][e] *= sh[D + i / gs];
    }
}

// the norm over the row's D columns (columns past D hold zeros)
template <int NV, int NTH>
DEVI void normalise(f32x4 (&v)[NV], int D, float eps, int rms, int groups, float* sh) {
  if (groups > 1) {
    normalise_groups<NV, NTH>(v, D, eps, groups, sh);
    return;
  }
  float s = 0.f, mean = 0.f;
  if (!rms) {
#pragma unroll
    for (int j = 0; j < NV; ++j) s += (v[j][0] + v[j][1]) + (v[j][2] + v[j][3]);
    mean = bsum<NTH / 64>(s, sh) / (float)D;
  }
  s = 0.f;
#pragma unroll
  for (int j = 0; j < NV; ++j)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float d = (int)(threadIdx.x + j * NTH) * 4 + e < D ? v[j][e] - mean : 0.f;
      v[j][e] = d;
      s += d * d;
    }
  const float inv = 1.f / sqrtf(bsum<NTH / 64>(s, sh) / (float)D + eps);
#pragma unroll
  for (int j = 0; j < NV; ++j) v[j] *= inv;
}

template <int NV, int NTH, bool VEC>
__global__ __launch_bounds__(NTH) void norm_add_kernel(NormAdd p) {
  extern __shared__ float sh[];
  const int t = p.rows ? p.rows[blockIdx.x] : (int)blockIdx.x, D = p.D;
  float* xr = p.x + (size_t)t * p.ldx;
  f32x4 v[NV], x[NV], w[NV];
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    x[j] = p.keep ? row4<VEC>(xr, (threadIdx.x + j * NTH) * 4, D) : f32x4{0.f, 0.f, 0.f, 0.f};
    if (p.add) x[j] += row4<VEC>(p.add, (threadIdx.x + j * NTH) * 4, D);
  }
  if (p.y) {
#pragma unroll
    for (int j = 0; j < NV; ++j)
      w[j] = p.w ? row4<VEC>(p.w, (threadIdx.x + j * NTH) * 4, D) : f32x4{1.f, 1.f, 1.f, 1.f};
    if (p.topk) {
#pragma unroll
      for (int j = 0; j < NV; ++j)
        v[j] = p.sh0 >= 0 ? row4<VEC>(p.y + (size_t)(p.sh0 + t) * p.ldy, (threadIdx.x + j * NTH) * 4, D)
                          : f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
      for (int k = 0; k < p.topk; ++k) {
        const float wk = p.topw[(size_t)t * p.topk + k];
        const float* yr = p.y + ((size_t)t * p.topk + k) * p.ldy;
#pragma unroll
        for (int j = 0; j < NV; ++j) v[j] += row4<VEC>(yr, (threadIdx.x + j * NTH) * 4, D) * wk;
      }
    } else {
#pragma unroll
      for (int j = 0; j < NV; ++j) v[j] = row4<VEC>(p.y + (size_t)t * p.ldy, (threadIdx.x + j * NTH) * 4, D);
#pragma unroll 4
      for (int s = 1; s < p.nslab; ++s)
#pragma unroll
        for (int j = 0; j < NV; ++j) v[j] += row4<VEC>(p.y + s * p.slab + (size_t)t * p.ldy, (threadIdx.x + j * NTH) * 4, D);
    }
    if (p.w) normalise<NV, NTH>(v, D, p.eps, p.rms, p.groups, sh);
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int i = (threadIdx.x + j * NTH) * 4;
      x[j] += v[j] * w[j];
      put4<VEC>(xr, i, D, x[j]);
      if (p.xb) {
        if (p.f32) put4<VEC>(reinterpret_cast<float*>(p.xb) + (size_t)t * p.ldxb, i, D, x[j]);
        else put4<VEC>(reinterpret_cast<__bf16*>(p.xb) + (size_t)t * p.ldxb, i, D, x[j]);
      }
    }
  }
  if (!p.ow) return;
#pragma unroll
  for (int j = 0; j < NV; ++j) w[j] = row4<VEC>(p.ow, (threadIdx.x + j * NTH) * 4, D);
  normalise<NV, NTH>(x, D, p.eps, p.rms, p.groups, sh);
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int i = (threadIdx.x + j * NTH) * 4;
    f32x4 y = x[j] * w[j];
    if (p.gate)
      y *= p.f32 ? row4<VEC>(reinterpret_cast<const float*>(p.gate) + (size_t)blockIdx.x * p.ldg, i, D)
                 : row4<VEC>(reinterpret_cast<const __bf16*>(p.gate) + (size_t)blockIdx.x * p.ldg, i, D);
    if (p.f32) put4<VEC>(reinterpret_cast<float*>(p.on) + (size_t)blockIdx.x * p.ldo, i, D, y);
    else put4<VEC>(reinterpret_cast<__bf16*>(p.on) + (size_t)blockIdx.x * p.ldo, i, D, y);
  }
  if (!p.ow2) return;
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int i = (threadIdx.x + j * NTH) * 4;
    const f32x4 y = x[j] * row4<VEC>(p.ow2, i, D);
    if (p.f32) put4<VEC>(reinterpret_cast<float*>(p.on2) + (size_t)blockIdx.x * p.ldo, i, D, y);
    else put4<VEC>(reinterpret_cast<__bf16*>(p.on2) + (size_t)blockIdx.x * p.ldo, i, D, y);
  }
}

// LDS of a row's sums: one float per wave and group of 4 columns per thread, or the squares of all columns
inline size_t norm_lds(const NormAdd& p, int slots) {
  return 4 * (size_t)(p.groups > 1 && (p.D / p.groups & 255) ? p.D + p.groups : slots);
}

template <bool VEC>
int norm_add_v(const NormAdd& p, int n, hipStream_t st) {
#define NLS_NA(LIM, NV, NTH) \
  if (p.D <= LIM) { \
    hipLaunchKernelGGL((norm_add_kernel<NV, NTH, VEC>), dim3(n), dim3(NTH), norm_lds(p, NV * NTH / 64), st, p); \
    return (int)hipGetLastError(); \
  }
  NLS_NA(1024, 1, 256) NLS_NA(2048, 2, 256)
  if (n <= 64) { NLS_NA(4096, 1, 1024) NLS_NA(8192, 2, 1024) }      // few rows: shorter per-thread chains
  NLS_NA(4096, 4, 256) NLS_NA(8192, 4, 512) NLS_NA(16384, 4, 1024)
#undef NLS_NA
  return -1;
}

inline int norm_add(const NormAdd& p, int n, hipStream_t st) {
  if (n < 1 || p.D < 1 || p.groups < 1 || p.D % p.groups || (p.groups > 1 && !p.rms) || norm_lds(p, 0) > 65536) return -1;
  const bool vec = !(p.D & 3) && !(p.ldx & 3) && !(p.ldy & 3) && !(p.ldo & 3) && !(p.ldxb & 3) && !(p.ldg & 3) &&
                   !(((uintptr_t)p.gate | (uintptr_t)p.xb | (uintptr_t)p.add) & 15);
  return vec ? norm_add_v<true>(p, n, st) : norm_add_v<false>(p, n, st);
}

// ---- latent attention rows: cq = RMSNorm(dq) * wq -> activation; c = RMSNorm(dkv[:R]) * wc and the rotated key part
// rope(dkv[R:]) -> the paged cache row of the token ([c | zeros to Rp | k_rot | zeros]; slot < 0: not stored)
template <typename T>
__global__ __launch_bounds__(256) void latent_rows_kernel(const float* __restrict__ dq, long lddq, int Q,
                                                          const float* __restrict__ wq, T* __restrict__ cq, long ldcq,
                                                          const float* __restrict__ dkv, long lddkv, int R, int Rp,
                                                          int rot, const float* __restrict__ wc,
                                                          const float* __restrict__ cs, const int* __restrict__ pos,
                                                          const int* __restrict__ slot, T* __restrict__ cache,
                                                          long ldc, float eps) {
  __shared__ float sh[4];
  const int t = blockIdx.x;
  const float* a = dq + (size_t)t * lddq;
  float s = 0.f;
  for (int i = threadIdx.x; i < Q; i += 256) s += a[i] * a[i];
  const float iq = 1.f / sqrtf(bsum<4>(s, sh) / (float)Q + eps);
  for (int i = threadIdx.x; i < Q; i += 256) stv(cq + (size_t)t * ldcq, i, a[i] * iq * wq[i]);
  if (!dkv) return;
  const float* b = dkv + (size_t)t * lddkv;
  s = 0.f;
  for (int i = threadIdx.x; i < R; i += 256) s += b[i] * b[i];
  const float ic = 1.f / sqrtf(bsum<4>(s, sh) / (float)R + eps);
  const int sl = slot[t];
  if (sl < 0) return;
  T* c = cache + (size_t)sl * ldc;
  for (int i = threadIdx.x; i < R; i += 256) stv(c, i, b[i] * ic * wc[i]);
  const float* f = cs + (size_t)pos[t] * rot;
  for (int i = threadIdx.x; i < rot / 2; i += 256) {
    const float u = b[R + 2 * i], v = b[R + 2 * i + 1];
    stv(c, Rp + 2 * i, u * f[2 * i] - v * f[2 * i + 1]);
    stv(c, Rp + 2 * i + 1, v * f[2 * i] + u * f[2 * i + 1]);
  }
}

// ---- attention rows: one workgroup per token. q and k are RMS-normed over all their heads together (norm weights optional),
// rotated on the first `rot` columns of each head (pairs 2i, 2i + 1) and stored in the activation type, heads Dp columns
// apart: q to `qo`, k and v (unnormed, unrotated) to the token's rows of the paged caches. The columns past D of a head
// are never written (zero from the start); slot < 0: no cache row. ktile: 16 slots of the key cache are a tile [G][Dp / 8][16][8]
// instead of rows, in which the 16 keys of an MFMA operand lie side by side.
struct AttnRows {
  const float *q, *k, *v;     // projections, f32
  const float *qn, *kn;       // norm weights (null: no norm)
  const float* cs;            // [positions][rot / 2][2]
  const int *pos, *slot;
  void *qo, *kc, *vc;
  long ldq, ldqo, ldc;        // row strides: projections, qo, caches
  int H, G, D, Dp, rot, V;    // V: columns of a value head
  float eps;
  int hnorm;                  // each rotated head of q and k is RMS-normed on its own, without weights
  int ktile;
  // 16 tokens beside each other, which fill the same lines of a key tile, run on one XCD
  DEVI int token() const {
    const int b = blockIdx.x;
    return ktile && b < ((int)gridDim.x & ~127) ? (b & ~127) | (b & 7) << 4 | (b >> 3 & 15) : b;
  }
  // where column c of a slot's key head h goes
  DEVI size_t key(int slot, int h, int c) const {
    return ktile ? (size_t)(slot & ~15) * ldc + (size_t)h * 16 * Dp + (c >> 3) * 128 + (slot & 15) * 8 + (c & 7)
                 : (size_t)slot * ldc + (size_t)h * Dp + c;
  }
};

template <typename T>
__global__ __launch_bounds__(256) void attn_rows_kernel(AttnRows p) {
  __shared__ float sh[4];
  const int t = p.token(), D = p.D, slot = p.slot[t];
  const float* f = p.rot ? p.cs + (size_t)p.pos[t] * p.rot : nullptr;
  auto norm = [&](const float* a, int n) {
    float s = 0.f;
    for (int i = threadIdx.x; i < n; i += 256) s += a[i] * a[i];
    return 1.f / sqrtf(bsum<4>(s, sh) / (float)n + p.eps);
  };
  auto put = [&](const float* a, const float* w, float inv, int heads, auto at) {
    const int D2 = (D + 1) >> 1;
    for (int e = threadIdx.x; e < heads * D2; e += 256) {
      const int h = e / D2, c = 2 * (e - h * D2), i = h * D + c;
      const bool two = c + 1 < D;
      float u = a[i], v = two ? a[i + 1] : 0.f;
      if (w) {
        u = u * inv * w[i];
        if (two) v = v * inv * w[i + 1];
      }
      if (c < p.rot) {
        const float cc = f[c], ss = f[c + 1], r = u * cc - v * ss;
        v = v * cc + u * ss;
        u = r;
      }
      T* o = at(h, c);                              // (columns c and c + 1, c even, are beside each other)
      o[0] = (T)u;
      if (two) o[1] = (T)v;
    }
  };
  const float *q = p.q + (size_t)t * p.ldq, *k = p.k + (size_t)t * p.ldq, *v = p.v + (size_t)t * p.ldq;
  put(q, p.qn, p.qn ? norm(q, p.H * D) : 1.f, p.H,
      [&](int h, int c) { return (T*)p.qo + (size_t)t * p.ldqo + (size_t)h * p.Dp + c; });
  const float ik = p.kn ? norm(k, p.G * D) : 1.f;
  if (slot < 0) return;
  put(k, p.kn, ik, p.G, [&](int h, int c) { return (T*)p.kc + p.key(slot, h, c); });
  T* vo = (T*)p.vc + (size_t)slot * p.ldc;
  for (int e = threadIdx.x; e < p.G * p.V; e += 256) vo[(size_t)(e / p.V) * p.Dp + e % p.V] = (T)v[e];
}

// the same for heads of a multiple of 4 columns: the row's q and k stay in registers, NV groups of 4 columns per thread. HN (heads
// of 4, 8, 16 .. 256 columns): no norm of the whole rows, but an RMS norm without weights of each rotated head on its own, whose
// columns are lanes beside each other.
template <typename T, int NV, int NTH, bool HN>
__global__ __launch_bounds__(NTH) void attn_rows4_kernel(AttnRows p) {
  __shared__ float sh[2][NTH / 64];
  typedef T t4 __attribute__((ext_vector_type(4)));
  const int t = p.token(), D4 = p.D >> 2, nq = p.H * D4, n = nq + p.G * D4, slot = p.slot[t];
  const float *q = p.q + (size_t)t * p.ldq, *k = p.k + (size_t)t * p.ldq, *v = p.v + (size_t)t * p.ldq;
  const float* f = p.rot ? p.cs + (size_t)p.pos[t] * p.rot : nullptr;
  f32x4 x[NV];
  float sq = 0.f, sk = 0.f;
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int e = threadIdx.x + j * NTH;
    x[j] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (e < n) x[j] = *reinterpret_cast<const f32x4*>(e < nq ? q + 4 * e : k + 4 * (e - nq));
    if constexpr (HN) continue;
    const float s = (x[j][0] * x[j][0] + x[j][1] * x[j][1]) + (x[j][2] * x[j][2] + x[j][3] * x[j][3]);
    if (e < nq) sq += s;
    else sk += s;
  }
  float iq = 1.f, ik = 1.f;
  if constexpr (!HN) {
    sq = wsum(sq);
    sk = wsum(sk);
    if ((threadIdx.x & 63) == 0) {
      sh[0][threadIdx.x >> 6] = sq;
      sh[1][threadIdx.x >> 6] = sk;
    }
    __syncthreads();
    sq = sk = 0.f;
#pragma unroll
    for (int i = 0; i < NTH / 64; ++i) {
      sq += sh[0][i];
      sk += sh[1][i];
    }
    iq = 1.f / sqrtf(sq / (float)(4 * nq) + p.eps);
    ik = 1.f / sqrtf(sk / (float)(4 * (n - nq)) + p.eps);
  }
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int e = threadIdx.x + j * NTH;
    if (e >= n) continue;
    const bool isq = e < nq;
    const int i = isq ? e : e - nq, h = i / D4, c = 4 * (i - h * D4);
    if (!isq && slot < 0) continue;
    f32x4 y = x[j];
    const float* w = isq ? p.qn : p.kn;
    if (w) y = y * (isq ? iq : ik) * *reinterpret_cast<const f32x4*>(w + 4 * i);
#pragma unroll
    for (int u = 0; u < 4; u += 2)
      if (c + u < p.rot) {
        const float cc = f[c + u], ss = f[c + u + 1], a = y[u], b = y[u + 1];
        y[u] = a * cc - b * ss;
        y[u + 1] = b * cc + a * ss;
      }
    if constexpr (HN) {
      float s = (y[0] * y[0] + y[1] * y[1]) + (y[2] * y[2] + y[3] * y[3]);
      for (int m = D4 >> 1; m > 0; m >>= 1) s += __shfl_xor(s, m, 64);
      y *= 1.f / sqrtf(s / (float)p.D + p.eps);
    }
    const t4 o = {(T)y[0], (T)y[1], (T)y[2], (T)y[3]};
    if (isq) {
      *reinterpret_cast<t4*>((T*)p.qo + (size_t)t * p.ldqo + (size_t)h * p.Dp + c) = o;
    } else {
      *reinterpret_cast<t4*>((T*)p.kc + p.key(slot, h, c)) = o;
      if (p.v == p.k) *reinterpret_cast<t4*>((T*)p.vc + (size_t)slot * p.ldc + (size_t)h * p.Dp + c) = t4{(T)x[j][0], (T)x[j][1], (T)x[j][2], (T)x[j][3]};
    }
  }
  if (p.v == p.k || slot < 0) return;
  const int V4 = p.V >> 2;
  for (int e = threadIdx.x; e < p.G * V4; e += NTH) {
    const int h = e / V4;
    const f32x4 z = *reinterpret_cast<const f32x4*>(v + 4 * e);
    *reinterpret_cast<t4*>((T*)p.vc + (size_t)slot * p.ldc + (size_t)h * p.Dp + 4 * (e - h * V4)) =
        t4{(T)z[0], (T)z[1], (T)z[2], (T)z[3]};
  }
}

// the same with an RMS norm without weights of each rotated head of q and k: one wave per head
template <typename T>
__global__ __launch_bounds__(256) void attn_head_rows_kernel(AttnRows p) {
  constexpr int NP = 8;                           // pairs of columns per lane: heads of up to 1024 columns
  const int t = p.token(), D = p.D, D2 = (D + 1) >> 1, lane = threadIdx.x & 63;
  const int slot = p.slot[t], u = blockIdx.y * 4 + (threadIdx.x >> 6);          // a head of q, k or v
  if (u >= p.H + 2 * p.G || (u >= p.H && slot < 0)) return;
  if (u >= p.H + p.G) {
    const int h = u - p.H - p.G;
    const float* a = p.v + (size_t)t * p.ldq + (size_t)h * p.V;
    T* o = (T*)p.vc + (size_t)slot * p.ldc + (size_t)h * p.Dp;
    for (int c = lane; c < p.V; c += 64) o[c] = (T)a[c];
    return;
  }
  const bool isq = u < p.H;
  const int h = isq ? u : u - p.H;
  const float* a = (isq ? p.q : p.k) + (size_t)t * p.ldq + (size_t)h * D;
  auto at = [&](int c) { return isq ? (T*)p.qo + (size_t)t * p.ldqo + (size_t)h * p.Dp + c : (T*)p.kc + p.key(slot, h, c); };
  const float* f = p.rot ? p.cs + (size_t)p.pos[t] * p.rot : nullptr;
  float x[NP], y[NP], s = 0.f;
#pragma unroll
  for (int j = 0; j < NP; ++j) {
    const int i = lane + 64 * j, c = 2 * i;
    x[j] = y[j] = 0.f;
    if (i >= D2) continue;
    x[j] = a[c];
    if (c + 1 < D) y[j] = a[c + 1];
    if (c < p.rot) {
      const float cc = f[c], ss = f[c + 1], v = x[j] * cc - y[j] * ss;
      y[j] = y[j] * cc + x[j] * ss;
      x[j] = v;
    }
    s += x[j] * x[j] + y[j] * y[j];
  }
  const float inv = 1.f / sqrtf(wsum(s) / (float)D + p.eps);
#pragma unroll
  for (int j = 0; j < NP; ++j) {
    const int i = lane + 64 * j, c = 2 * i;
    if (i >= D2) continue;
    T* o = at(c);                                   // (columns c and c + 1, c even, are beside each other)
    o[0] = (T)(x[j] * inv);
    if (c + 1 < D) o[1] = (T)(y[j] * inv);
  }
}

// ---- PolyNorm: out = a N(z) + b N(z^2) + c N(z^3) + e of each row, powers by element, N(v) = v / sqrt(mean(v^2) + eps)
template <typename T, int NTH>
__global__ __launch_bounds__(NTH) void poly_norm_kernel(const T* __restrict__ z, long ldz, const float* __restrict__ act,
                                                        T* __restrict__ out, long ldo, int N, float eps) {
  typedef T t8 __attribute__((ext_vector_type(8)));
  __shared__ float sh[3][NTH / 64];
  const T* a = z + (size_t)blockIdx.x * ldz;
  T* o = out + (size_t)blockIdx.x * ldo;
  float s1 = 0.f, s2 = 0.f, s3 = 0.f;
  const int N8 = N & ~7;
  auto add = [&](float v) {
    const float q = v * v, q2 = q * q;
    s1 += q;
    s2 += q2;
    s3 += q2 * q;
  };
  for (int i = threadIdx.x * 8; i < N8; i += NTH * 8) {
    const t8 v = *reinterpret_cast<const t8*>(a + i);
#pragma unroll
    for (int e = 0; e < 8; ++e) add((float)v[e]);
  }
  if (N8 + (int)threadIdx.x < N) add((float)a[N8 + threadIdx.x]);
  s1 = wsum(s1);
  s2 = wsum(s2);
  s3 = wsum(s3);
  if ((threadIdx.x & 63) == 0) {
    sh[0][threadIdx.x >> 6] = s1;
    sh[1][threadIdx.x >> 6] = s2;
    sh[2][threadIdx.x >> 6] = s3;
  }
  __syncthreads();
  s1 = s2 = s3 = 0.f;
#pragma unroll
  for (int i = 0; i < NTH / 64; ++i) {
    s1 += sh[0][i];
    s2 += sh[1][i];
    s3 += sh[2][i];
  }
  const float n = (float)N, k1 = act[0] / sqrtf(s1 / n + eps), k2 = act[1] / sqrtf(s2 / n + eps), k3 = act[2] / sqrtf(s3 / n + eps);
  const float k0 = act[3];
  auto poly = [&](float v) { return fmaf(fmaf(fmaf(k3, v, k2), v, k1), v, k0); };
  for (int i = threadIdx.x * 8; i < N8; i += NTH * 8) {
    const t8 v = *reinterpret_cast<const t8*>(a + i);
    t8 y;
#pragma unroll
    for (int e = 0; e < 8; ++e) y[e] = (T)poly((float)v[e]);
    *reinterpret_cast<t8*>(o + i) = y;
  }
  if (N8 + (int)threadIdx.x < N) o[N8 + threadIdx.x] = (T)poly((float)a[N8 + threadIdx.x]);
}

template <typename T>
int poly_norm_t(const void* z, long ldz, const float* act, void* out, long ldo, int N, int n, float eps, hipStream_t st) {
  if (N > 8192 || n <= 64)
    hipLaunchKernelGGL((poly_norm_kernel<T, 1024>), dim3(n), dim3(1024), 0, st, (const T*)z, ldz, act, (T*)out, ldo, N, eps);
  else
    hipLaunchKernelGGL((poly_norm_kernel<T, 256>), dim3(n), dim3(256), 0, st, (const T*)z, ldz, act, (T*)out, ldo, N, eps);
  return (int)hipGetLastError();
}

template <typename T>
int attn_rows_t(const AttnRows& p, int n, hipStream_t st) {
  const int cols = (p.H + p.G) * p.D;
  const bool vec = !((p.D | p.V) & 3) && !(p.ldq & 3) && !(p.Dp & 3) && !(p.ldqo & 3) && !(p.ldc & 3) &&
                   !(((uintptr_t)p.q | (uintptr_t)p.k | (uintptr_t)p.v) & 15);
  const bool lanes = p.hnorm && p.D <= 256 && !(p.D & (p.D - 1));
#define NLS_AR(NV, NTH) \
  if (vec && (lanes || !p.hnorm) && cols <= 4 * NV * NTH) { \
    if (lanes) hipLaunchKernelGGL((attn_rows4_kernel<T, NV, NTH, true>), dim3(n), dim3(NTH), 0, st, p); \
    else hipLaunchKernelGGL((attn_rows4_kernel<T, NV, NTH, false>), dim3(n), dim3(NTH), 0, st, p); \
    return (int)hipGetLastError(); \
  }
  NLS_AR(1, 256)
  if (n <= 64) { NLS_AR(1, 1024) NLS_AR(2, 1024) }
  NLS_AR(2, 256) NLS_AR(5, 256) NLS_AR(8, 256) NLS_AR(8, 1024)
#undef NLS_AR
  if (p.hnorm) {
    hipLaunchKernelGGL(attn_head_rows_kernel<T>, dim3(n, (p.H + 2 * p.G + 3) / 4), dim3(256), 0, st, p);
    return (int)hipGetLastError();
  }
  hipLaunchKernelGGL(attn_rows_kernel<T>, dim3(n), dim3(256), 0, st, p);
  return (int)hipGetLastError();
}

// ---- expert choice of one token: scores (sigmoid, or a softmax over all experts), the `keep` groups with the largest sum of their
// two best scores (gbest 2) or the largest score (1), the `topk` best experts of those; weight = score * scale. Ties go to the
// lowest index. One wave per token; scores in LDS.
struct Route {
  int E, topk, groups, keep, softmax, gbest;
  float scale;
};

DEVI void pick_experts(const float* __restrict__ z, const Route& R, int lane, float* sc, float* gs, float* __restrict__ topw,
                       int* __restrict__ sel) {
  const int E = R.E, topk = R.topk, groups = R.groups, keep = R.keep;
  const float scale = R.scale;
  if (R.softmax) {
    float m = -INFINITY, l = 0.f;
    for (int e = lane; e < E; e += 64) m = fmaxf(m, z[e]);
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) m = fmaxf(m, __shfl_xor(m, o, 64));
    for (int e = lane; e < E; e += 64) {
      const float s = expf(z[e] - m);
      sc[e] = s;
      l += s;
    }
    l = wsum(l);
    for (int e = lane; e < E; e += 64) {
      const float s = sc[e] / l;
      sc[e] = s == s ? s : -1.f;
    }
  } else {
    for (int e = lane; e < E; e += 64) {
      const float s = 1.f / (1.f + expf(-z[e]));
      sc[e] = s == s ? s : -1.f;
    }
  }
  __builtin_amdgcn_wave_barrier();
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  const int per = E / groups;
  for (int g = lane; g < groups; g += 64) {
    float a = -2.f, b = -2.f;
    for (int i = 0; i < per; ++i) {
      const float s = sc[g * per + i];
      if (s > a) { b = a; a = s; }
      else if (s > b) b = s;
    }
    gs[g] = per > 1 && R.gbest == 2 ? a + b : a;
  }
  __builtin_amdgcn_wave_barrier();
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  // group g is kept when fewer than `keep` groups beat it
  for (int g = lane; g < groups; g += 64) {
    int better = 0;
    for (int h = 0; h < groups; ++h) better += gs[h] > gs[g] || (gs[h] == gs[g] && h < g);
    if (better >= keep)
      for (int i = 0; i < per; ++i) sc[g * per + i] = -3.f;
  }
  __builtin_amdgcn_wave_barrier();
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  for (int j = 0; j < topk; ++j) {
    float bv = -4.f;
    int be = 0x7fffffff;
    for (int e = lane; e < E; e += 64)
      if (sc[e] > bv) { bv = sc[e]; be = e; }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ov = __shfl_xor(bv, o, 64);
      const int oe = __shfl_xor(be, o, 64);
      if (ov > bv || (ov == bv && oe < be)) { bv = ov; be = oe; }
    }
    if (lane == 0) {
      topw[j] = bv * scale;
      sel[j] = be;
    }
    if (lane == (be & 63)) sc[be] = -4.f;
    __builtin_amdgcn_wave_barrier();
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  }
}

constexpr int ME = 512;       // experts per layer
constexpr int PW = 8;         // waves that choose experts in moe_plan_kernel<true>

__global__ __launch_bounds__(64) void moe_pick_kernel(const float* __restrict__ z, long ldz, Route R, float* __restrict__ topw,
                                                      int* __restrict__ sel) {
  __shared__ float sc[ME], gs[ME];
  const int t = blockIdx.x;
  pick_experts(z + (size_t)t * ldz, R, threadIdx.x, sc, gs, topw + (size_t)t * R.topk, sel + (size_t)t * R.topk);
}

// ---- routed-entry lists of one step: entries (token t, choice j) = t * topk + j grouped by expert (entry order within
// an expert is arbitrary: rows do not interact), and the (expert, <= bm entries) tiles of the grouped products.
// One workgroup. PICK: also choose the experts (small steps: one launch less).
template <bool PICK>
__global__ __launch_bounds__(1024) void moe_plan_kernel(const float* __restrict__ z, long ldz, int T, Route R,
                                                        float* __restrict__ topw, int* __restrict__ sel, int bm,
                                                        int* __restrict__ rows, int* __restrict__ tiles,
                                                        int* __restrict__ ntiles, int maxtiles) {
  __shared__ int cnt[ME], off[ME], pos[ME];
  __shared__ float sc[PICK ? PW : 1][PICK ? ME : 1], gs[PICK ? PW : 1][PICK ? ME : 1];
  const int E = R.E, topk = R.topk, n = T * topk;
  if constexpr (PICK) {
    const int w = threadIdx.x >> 6, lane = threadIdx.x & 63;
    for (int t = w; w < PW && t < T; t += PW)
      pick_experts(z + (size_t)t * ldz, R, lane, sc[w], gs[w], topw + (size_t)t * topk, sel + (size_t)t * topk);
    __threadfence_block();
  }
  for (int e = threadIdx.x; e < E; e += 1024) cnt[e] = 0;
  __syncthreads();
  for (int i = threadIdx.x; i < n; i += 1024) atomicAdd(&cnt[min(max(sel[i], 0), E - 1)], 1);
  __syncthreads();
  if (threadIdx.x < 64) {
    // one wave: exclusive prefix sums of counts and tile counts, 64 experts at a time
    int o = 0, to = 0;
    for (int e0 = 0; e0 < E; e0 += 64) {
      const int e = e0 + threadIdx.x;
      const int c = e < E ? cnt[e] : 0;
      const int nt = (c + bm - 1) / bm;
      int a = c, b = nt;
#pragma unroll
      for (int s = 1; s < 64; s <<= 1) {
        const int ua = __shfl_up(a, s, 64), ub = __shfl_up(b, s, 64);
        if (threadIdx.x >= s) { a += ua; b += ub; }
      }
      if (e < E) {
        off[e] = o + a - c;
        pos[e] = 0;
        for (int i = 0; i < nt; ++i) {
          const int ti = to + b - nt + i;
          if (ti < maxtiles) {
            tiles[4 * ti] = e;
            tiles[4 * ti + 1] = o + a - c + i * bm;
            tiles[4 * ti + 2] = min(bm, c - i * bm);
            tiles[4 * ti + 3] = 0;
          }
        }
      }
      o += __shfl(a, 63, 64);
      to += __shfl(b, 63, 64);
    }
    if (threadIdx.x == 0) *ntiles = min(to, maxtiles);
  }
  __syncthreads();
  for (int i = threadIdx.x; i < n; i += 1024) {
    const int e = min(max(sel[i], 0), E - 1);
    rows[off[e] + atomicAdd(&pos[e], 1)] = i;
  }
}

// ---- greedy pick: lowest index of the row's largest logit
__global__ __launch_bounds__(1024) void argmax_kernel(const float* __restrict__ z, long ldz, int V,
                                                      int* __restrict__ out) {
  __shared__ float bv[16];
  __shared__ int bi[16];
  const float* r = z + (size_t)blockIdx.x * ldz;
  float v = -INFINITY;
  int ix = 0x7fffffff;
  int i = threadIdx.x;
  for (; i + 7 * 1024 < V; i += 8 * 1024) {      // 8 loads in flight
    float a[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) a[j] = r[i + j * 1024];
#pragma unroll
    for (int j = 0; j < 8; ++j)
      if (a[j] > v || ix == 0x7fffffff) { v = a[j]; ix = i + j * 1024; }
  }
  for (; i < V; i += 1024) {
    const float a = r[i];
    if (a > v || ix == 0x7fffffff) { v = a; ix = i; }
  }
  auto take = [&](float ov, int oi) {
    if (ov > v || (ov == v && oi < ix)) { v = ov; ix = oi; }
  };
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) {
    const float ov = __shfl_xor(v, o, 64);
    const int oi = __shfl_xor(ix, o, 64);
    take(ov, oi);
  }
  if ((threadIdx.x & 63) == 0) { bv[threadIdx.x >> 6] = v; bi[threadIdx.x >> 6] = ix; }
  __syncthreads();
  if (threadIdx.x == 0) {
    for (int w = 1; w < 16; ++w) take(bv[w], bi[w]);
    out[blockIdx.x] = ix < V ? ix : 0;
  }
}

}  // namespace nls_stack

extern "C" {
using namespace nls_stack;

// pairs (optional): [buckets + 1][D] with the slots' previous tokens; ptab (optional): [npos][D]
int nls_stack_embed(int* ids, const int* next_ids, const int* use_prev, const void* tab, int V, int D, float scale,
                    float* x, void* xb, long ldx, int T, void* c0, void* c1, long ldc, int f32, const void* pairs, int buckets,
                    int mul_prev, int mul_cur, int* prev, const int* runs, const int* tok_seq, const void* ptab, int npos,
                    const int* pos, const float* add, void* stream) {
  if (T < 1 || D < 1 || V < 1 || (pairs && (buckets < 1 || !prev || !runs || !tok_seq)) || (ptab && (npos < 1 || !pos))) return -1;
  const uintptr_t at = (uintptr_t)tab | (uintptr_t)x | (uintptr_t)xb | (uintptr_t)c0 | (uintptr_t)c1 | (uintptr_t)pairs |
                       (uintptr_t)ptab;
  const int vec = !((D | ldx | ldc) & 7) && !(at & 31);
  const Embed p{ids, next_ids, use_prev, (const __bf16*)tab, x, (__bf16*)xb, c0, c1, (const __bf16*)pairs, prev, runs, tok_seq,
                (const __bf16*)ptab, pos, add, ldx, ldc, V, D, buckets, mul_prev, mul_cur, npos, f32, vec, scale};
  hipLaunchKernelGGL(embed_kernel, dim3(T), dim3(256), 0, (hipStream_t)stream, p);
  return (int)hipGetLastError();
}

int nls_norm_add(const float* y, long ldy, const float* topw, int topk, long sh0, const float* w, float* x, long ldx, void* xb,
                 long ldxb, const float* ow, void* on, const float* ow2, void* on2, long ldo, const float* add, int keep, int D,
                 int T, float eps, int f32, int rms, int groups, int nslab, long slab, void* stream) {
  if (!y || nslab < 1 || (slab & 3) || (ow2 && (!ow || !on2))) return -1;
  return norm_add(NormAdd{y, topw, w, x, xb, ow, on, nullptr, ldy, ldx, ldo, sh0, D, topk, f32, rms, eps, nslab, slab, ldxb, add,
                          keep, ow2, on2, nullptr, 0, groups}, T, (hipStream_t)stream);
}

// out[i] = norm(x[rows ? rows[i] : i]) * w (* gate[i]); w2, out2: the same with another weight
int nls_row_norm(const float* x, long ldx, const int* rows, const float* w, void* out, const float* w2, void* out2, long ldo,
                 const void* gate, long ldg, int D, int n, float eps, int f32, int rms, int groups, void* stream) {
  if (w2 && !out2) return -1;
  return norm_add(NormAdd{nullptr, nullptr, nullptr, const_cast<float*>(x), nullptr, w, out, rows, 0, ldx, ldo, -1, D, 0,
                          f32, rms, eps, 1, 0, 0, nullptr, 1, w2, out2, gate, ldg, groups}, n, (hipStream_t)stream);
}

int nls_latent_rows(const float* dq, long lddq, int Q, const float* wq, void* cq, long ldcq, const float* dkv,
                    long lddkv, int R, int Rp, int rot, const float* wc, const float* cs, const int* pos,
                    const int* slot, void* cache, long ldc, int T, float eps, int f32, void* stream) {
  if (T < 1 || Q < 1 || (dkv && (R < 1 || (rot & 1) || Rp + rot > ldc))) return -1;
  if (f32)
    hipLaunchKernelGGL(latent_rows_kernel<float>, dim3(T), dim3(256), 0, (hipStream_t)stream, dq, lddq, Q, wq,
                       (float*)cq, ldcq, dkv, lddkv, R, Rp, rot, wc, cs, pos, slot, (float*)cache, ldc, eps);
  else
    hipLaunchKernelGGL(latent_rows_kernel<__bf16>, dim3(T), dim3(256), 0, (hipStream_t)stream, dq, lddq, Q, wq,
                       (__bf16*)cq, ldcq, dkv, lddkv, R, Rp, rot, wc, cs, pos, slot, (__bf16*)cache, ldc, eps);
  return (int)hipGetLastError();
}

// heads of D columns (values: V), Dp apart in the outputs; rot even, at most D; hnorm: no weights
int nls_attn_rows(const float* q, const float* k, const float* v, long ldq, const float* qn, const float* kn, const float* cs,
                  const int* pos, const int* slot, void* qo, long ldqo, void* kc, void* vc, long ldc, int T, int H, int G,
                  int D, int V, int Dp, int rot, int hnorm, int ktile, float eps, int f32, void* stream) {
  if (T < 1 || (ktile && ((Dp & 7) || ldc != (long)G * Dp)) || (hnorm && (qn || kn || D > 1024)) || H < 1 || G < 1 || D < 1 || V < 1 || Dp < D || Dp < V || (v == k && V != D) || (rot && !cs) || (rot & 1) || rot < 0 ||
      rot > D || (long)H * Dp > ldqo || (long)G * Dp > ldc)
    return -1;
  AttnRows p{q, k, v, qn, kn, cs, pos, slot, qo, kc, vc, ldq, ldqo, ldc, H, G, D, Dp, rot, V, eps, hnorm, ktile};
  return f32 ? attn_rows_t<float>(p, T, (hipStream_t)stream) : attn_rows_t<__bf16>(p, T, (hipStream_t)stream);
}

// z, out: rows of N values, 16-byte aligned; act: a, b, c, e
int nls_poly_norm(const void* z, long ldz, const float* act, void* out, long ldo, int N, int n, float eps, int f32, void* stream) {
  if (n < 1 || N < 1 || ((ldz | ldo) & 7) || (((uintptr_t)z | (uintptr_t)out) & 15)) return -1;
  return f32 ? poly_norm_t<float>(z, ldz, act, out, ldo, N, n, eps, (hipStream_t)stream)
             : poly_norm_t<__bf16>(z, ldz, act, out, ldo, N, n, eps, (hipStream_t)stream);
}

int nls_stack_argmax(const float* z, long ldz, int V, int* out, int n, void* stream) {
  if (n < 1 || V < 1) return -1;
  hipLaunchKernelGGL(argmax_kernel, dim3(n), dim3(1024), 0, (hipStream_t)stream, z, ldz, V, out);
  return (int)hipGetLastError();
}

// rows: int [T * topk]; tiles: int [maxtiles][4], maxtiles >= min(T * topk, E + T * topk / bm)
int nls_moe_plan(const float* z, long ldz, int T, int E, int topk, int groups, int keep, int softmax, int gbest, float scale,
                 float* topw, int* sel, int bm, int* rows, int* tiles, int* ntiles, int maxtiles, void* stream) {
  if (T < 1 || E < 1 || E > ME || topk < 1 || topk > E || groups < 1 || E % groups || keep < 1 || bm < 1 ||
      (long)min(keep, groups) * (E / groups) < topk || maxtiles < 1 || gbest < 1 || gbest > 2)
    return -1;
  const Route R{E, topk, groups, keep, softmax, gbest, scale};
  hipStream_t st = (hipStream_t)stream;
  if (T <= 32) {
    hipLaunchKernelGGL(moe_plan_kernel<true>, dim3(1), dim3(1024), 0, st, z, ldz, T, R, topw, sel, bm,
                       rows, tiles, ntiles, maxtiles);
    return (int)hipGetLastError();
  }
  hipLaunchKernelGGL(moe_pick_kernel, dim3(T), dim3(64), 0, st, z, ldz, R, topw, sel);
  hipLaunchKernelGGL(moe_plan_kernel<false>, dim3(1), dim3(1024), 0, st, z, ldz, T, R, topw, sel, bm, rows,
                     tiles, ntiles, maxtiles);
  return (int)hipGetLastError();
}

}  // extern "C"
