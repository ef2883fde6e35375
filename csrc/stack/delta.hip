// Gated delta rule with a decay per key channel (gfx950): the short causal convolutions ahead of it, the step of single tokens, and
// the entry points; runs of tokens go in chunks (gla_chunk.h, delta_chunk.h).
//
// Per head, state S [D][V] in f32:  S <- diag(a) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q.
// Queries and keys have G heads (head h uses h / (H / G)). They are kept as the convolutions leave them, with 32-bit factors per
// token and head that make them unit vectors (queries: times D^-1/2).
#include "gla_chunk.h"

namespace nls_gla {

int delta_scan_bf16(const GA& p, int nruns, int nt, hipStream_t st);        // delta_bf16.hip
int delta_scan_f32(const GA& p, int nruns, int nt, hipStream_t st);         // delta_f32.hip

// ---- convolutions: y[t] = silu(sum_j w[j] z[t - (taps - 1) + j]) per channel, channels [q: G D | k: G D | v: H V] of z and y. Tokens
// ahead of a run come from its slot's state [taps - 1][channels] (zeros at position 0). fac [rows][2 G]: D^-1/2 / |q|, 1 / |k| per
// head, |x|^2 = sum(x^2) + 1e-6 of the values as stored. A wave takes a head's columns of TG rows. Runs of one token also move
// their state on (a channel belongs to one lane); conv_tail_kernel does that for the others, once no row reads the old one.
struct CV {
  const void* z;
  void* y;
  const float* w;          // [channels][taps]
  float* fac;
  float* state;            // [slots][sstride]
  const int *runs, *tok_seq;
  long ldz, ldy, ldf, sstride;
  int T, H, G, D, V, taps;
};

template <typename T, int TAPS, int TG, int VC>      // TAPS 0: any number, re-reading the inputs; VC: channels per lane
__global__ __launch_bounds__(256) void conv_kernel(CV p) {
  typedef T tv __attribute__((ext_vector_type(VC)));
  typedef float fv __attribute__((ext_vector_type(VC)));
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int unit = blockIdx.y * 4 + wave, nqk = 2 * p.G;
  if (unit >= nqk + p.H) return;
  const bool qk = unit < nqk;
  const int W = qk ? p.D : p.V, ch0 = qk ? unit * p.D : nqk * p.D + (unit - nqk) * p.V;
  const int nch = nqk * p.D + p.H * p.V, taps = TAPS ? TAPS : p.taps, r0 = blockIdx.x * TG, r1 = min(p.T, r0 + TG);
  float ss[TG];
#pragma unroll
  for (int e = 0; e < TG; ++e) ss[e] = 0.f;
  for (int c = lane * VC; c < W; c += 64 * VC) {
    const int ch = ch0 + c;
    const T* zc = (const T*)p.z + ch;
    auto row = [&](int u) { return __builtin_convertvector(*reinterpret_cast<const tv*>(zc + (size_t)u * p.ldz), fv); };
    auto weight = [&](int j) {
      fv v;
#pragma unroll
      for (int i = 0; i < VC; ++i) v[i] = p.w[(size_t)(ch + i) * taps + j];
      return v;
    };
    fv w[TAPS ? TAPS : 1], h[TAPS ? TAPS : 1];
    if constexpr (TAPS > 0) {
#pragma unroll
      for (int j = 0; j < TAPS; ++j) w[j] = weight(j);
    }
    auto emit = [&](int e, const fv& acc) {
      tv y;
#pragma unroll
      for (int i = 0; i < VC; ++i) {
        y[i] = (T)(acc[i] * nls_lin::lin_sigmoid(acc[i]));
        ss[e] = fmaf((float)y[i], (float)y[i], ss[e]);
      }
      *reinterpret_cast<tv*>((T*)p.y + (size_t)(r0 + e) * p.ldy + ch) = y;
    };
    if constexpr (TAPS > 0 && TG > 1) {      // rows inside a run, their inputs too: all loads in flight together
      const int rn = p.tok_seq[r0];
      const int* run = p.runs + 4 * rn;
      if (r0 - (TAPS - 1) >= run[0] && r0 + TG <= run[0] + run[1] && run[2] >= 0) {
        fv x[TG + TAPS - 1];
#pragma unroll
        for (int e = 0; e < TG + TAPS - 1; ++e) x[e] = row(r0 - (TAPS - 1) + e);
#pragma unroll
        for (int e = 0; e < TG; ++e) {
          fv acc = w[TAPS - 1] * x[e + TAPS - 1];
#pragma unroll
          for (int j = 0; j + 1 < TAPS; ++j) acc += w[j] * x[e + j];
          emit(e, acc);
        }
        continue;
      }
    }
    int seen = -1;                           // run that h belongs to: its inputs at t - (taps - 1) .. t - 1
#pragma unroll
    for (int e = 0; e < TG; ++e) {
      const int t = r0 + e;
      if (t >= r1) break;
      const int rn = p.tok_seq[t];
      const int* run = p.runs + 4 * rn;
      const int t0 = run[0], n = run[1], slot = run[2], pos0 = run[3];
      if (slot < 0 || t < t0 || t >= t0 + n) continue;
      float* st = p.state + (size_t)slot * p.sstride + ch;
      auto kept = [&](int j) -> fv& { return *reinterpret_cast<fv*>(st + (size_t)j * nch); };
      auto input = [&](int u) {              // input of row u of this run, or of the tokens ahead of it
        return u >= t0 ? row(u) : pos0 > 0 ? kept(u - t0 + taps - 1) : (fv)(0.f);
      };
      const fv x = row(t);
      fv acc;
      if constexpr (TAPS > 0) {
        if (rn != seen) {
#pragma unroll
          for (int j = 0; j + 1 < TAPS; ++j) h[j] = input(t - (TAPS - 1) + j);
          seen = rn;
        }
        acc = w[TAPS - 1] * x;
#pragma unroll
        for (int j = 0; j + 1 < TAPS; ++j) acc += w[j] * h[j];
#pragma unroll
        for (int j = 0; j + 2 < TAPS; ++j) h[j] = h[j + 1];
        if (TAPS > 1) h[TAPS > 1 ? TAPS - 2 : 0] = x;
        if (n == 1)
#pragma unroll
          for (int j = 0; j + 1 < TAPS; ++j) kept(j) = h[j];
      } else {
        acc = weight(taps - 1) * x;
        for (int j = 0; j + 1 < taps; ++j) acc += weight(j) * input(t - (taps - 1) + j);
        if (n == 1)
          for (int j = 0; j + 1 < taps; ++j) kept(j) = j + 2 < taps ? (pos0 > 0 ? kept(j + 1) : (fv)(0.f)) : x;
      }
      emit(e, acc);
    }
  }
  if (!qk) return;
#pragma unroll
  for (int e = 0; e < TG; ++e) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) ss[e] += __shfl_xor(ss[e], o, 64);
    if (lane == 0 && r0 + e < r1)
      p.fac[(size_t)(r0 + e) * p.ldf + unit] = (unit < p.G ? 1.f / sqrtf((float)p.D) : 1.f) / sqrtf(ss[e] + 1e-6f);
  }
}

// the last taps - 1 inputs of every run of several tokens
template <typename T>
__global__ __launch_bounds__(256) void conv_tail_kernel(CV p) {
  const int* run = p.runs + 4 * blockIdx.y;
  const int t0 = run[0], n = run[1], slot = run[2], pos0 = run[3], keep = p.taps - 1;
  const int nch = 2 * p.G * p.D + p.H * p.V, ch = blockIdx.x * 256 + threadIdx.x;
  if (slot < 0 || n < 2 || ch >= nch) return;
  float* st = p.state + (size_t)slot * p.sstride + ch;
  for (int i = 0; i < keep; ++i) {           // (upwards: what is read lies behind what was written)
    const int t = n - keep + i;
    st[(size_t)i * nch] = t >= 0 ? (float)((const T*)p.z)[(size_t)(t0 + t) * p.ldz + ch]
                                 : pos0 > 0 ? st[(size_t)(i + n) * nch] : 0.f;
  }
}

template <typename T, int TAPS, int VC>
int conv_v(const CV& p, hipStream_t st) {
  const int units = 2 * p.G + p.H;
  if (p.T <= 512) hipLaunchKernelGGL((conv_kernel<T, TAPS, 1, VC>), dim3(p.T, (units + 3) / 4), dim3(256), 0, st, p);
  else hipLaunchKernelGGL((conv_kernel<T, TAPS, 8, VC>), dim3((p.T + 7) / 8, (units + 3) / 4), dim3(256), 0, st, p);
  return (int)hipGetLastError();
}

template <typename T, int TAPS>
int conv_t(const CV& p, hipStream_t st) {
  const bool pair = !((p.D | p.V | p.ldz | p.ldy | p.sstride) & 1) && !((uintptr_t)p.state & 7) &&
                    !(((uintptr_t)p.z | (uintptr_t)p.y) % (2 * sizeof(T)));
  return pair ? conv_v<T, TAPS, 2>(p, st) : conv_v<T, TAPS, 1>(p, st);
}

template <typename T>
int conv(const CV& p, int nruns, hipStream_t st) {
  const int rc = p.taps == 2 ? conv_t<T, 2>(p, st) : p.taps == 3 ? conv_t<T, 3>(p, st) : p.taps == 4 ? conv_t<T, 4>(p, st)
                                                                                                      : conv_t<T, 0>(p, st);
  if (rc || p.taps == 1 || nruns == p.T) return rc;
  hipLaunchKernelGGL(conv_tail_kernel<T>, dim3((2 * p.G * p.D + p.H * p.V + 255) / 256, nruns), dim3(256), 0, st, p);
  return (int)hipGetLastError();
}

// ---- one token per run. A workgroup per (head, run): a thread owns 4 value columns of the key rows g, g + GR, .., in registers
// (RPT of them; 0: more than fit, read again for the update). Decays: a, or (null) sigmoid(a2 low + a2b)^rate per channel, and the
// output's gate: gate, or (null) sigmoid(g2 lowg).
struct DS {
  const void *q, *k, *v;
  const float *fac, *beta;
  const float* a;
  const void *low, *a2;
  const float *a2b, *rate;         // [H * D]
  const void *gate, *lowg, *g2;
  const float* norm;               // [H * V]
  void* out;
  float* state;
  const int* runs;
  long ld, ldf, ldb, lda, ldz, ldg, ldout, sstride;
  int H, G, D, V, ra, rg;
  float eps;
};

template <typename T>
DEVI float low_dot(const T* x, const T* w, int n) {
  typedef T t8 __attribute__((ext_vector_type(8)));
  float z = 0.f;
  int i = 0;
  if ((n & 7) == 0)                          // (16-byte aligned rows)
#pragma unroll 4
    for (; i < n; i += 8) {
      const t8 a = *reinterpret_cast<const t8*>(x + i), b = *reinterpret_cast<const t8*>(w + i);
#pragma unroll
      for (int e = 0; e < 8; ++e) z = fmaf((float)a[e], (float)b[e], z);
    }
  for (; i < n; ++i) z = fmaf((float)x[i], (float)w[i], z);
  return z;
}

template <typename T, int RPT>
__global__ __launch_bounds__(256) void delta_step_kernel(DS p) {
  __shared__ __attribute__((aligned(16))) float qs[256], ks[256], ws[256], us[1024], red[1024];
  __shared__ float part[4];
  const int* run = p.runs + 4 * blockIdx.y;
  const int t = run[0], n = run[1], slot = run[2], pos0 = run[3];
  if (slot < 0 || n != 1) return;
  const int D = p.D, V = p.V, head = blockIdx.x, tid = threadIdx.x, hq = head / (p.H / p.G);
  const size_t hb = (size_t)head * D, hv = (size_t)head * V;
  const int C4 = V >> 2, GR = 256 / C4, c = (tid % C4) * 4, g = tid / C4;
  float* st = p.state + (size_t)slot * p.sstride + hb * V;
  const bool mine = g < GR;
  const f32x4 zero = f32x4{0.f, 0.f, 0.f, 0.f};
  f32x4 s[RPT ? RPT : 1];
  if constexpr (RPT > 0) {
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
      const int d = g + GR * i;
      s[i] = zero;
      if (mine && d < D && pos0 > 0) s[i] = *reinterpret_cast<const f32x4*>(st + (size_t)d * V + c);
    }
  }
  if (tid < D) {
    const T *qr = (const T*)p.q + (size_t)t * p.ld + (size_t)hq * D, *kr = (const T*)p.k + (size_t)t * p.ld + (size_t)hq * D;
    qs[tid] = (float)qr[tid] * p.fac[(size_t)t * p.ldf + hq];
    ks[tid] = (float)kr[tid] * p.fac[(size_t)t * p.ldf + p.G + hq];
    ws[tid] = p.a ? p.a[(size_t)t * p.lda + hb + tid]
                  : nls_lin::lin_sigpow(low_dot((const T*)p.low + (size_t)t * p.ldz, (const T*)p.a2 + (hb + tid) * p.ra, p.ra) +
                                            p.a2b[hb + tid], p.rate[hb + tid]);
  }
  __syncthreads();
  // S <- diag(a) S; the state's answer to k
  if (mine) {
    f32x4 y = zero;
    if constexpr (RPT > 0) {
#pragma unroll
      for (int i = 0; i < RPT; ++i) {
        const int d = min(g + GR * i, D - 1);
        s[i] *= ws[d];
        y += s[i] * ks[d];                   // (rows past D hold zeros)
      }
    } else if (pos0 > 0) {
      for (int d = g; d < D; d += GR) y += *reinterpret_cast<const f32x4*>(st + (size_t)d * V + c) * (ws[d] * ks[d]);
    }
    *reinterpret_cast<f32x4*>(red + g * V + c) = y;
  }
  __syncthreads();
  const float beta = p.beta[(size_t)t * p.ldb + head];
#pragma unroll
  for (int x = 0; x < 4; ++x) {
    const int e = tid + 256 * x;
    if (e < V) {
      float y = 0.f;
      for (int i = 0; i < GR; ++i) y += red[i * V + e];
      us[e] = beta * ((float)((const T*)p.v)[(size_t)t * p.ld + hv + e] - y);
    }
  }
  __syncthreads();
  if (mine) {
    const f32x4 u = *reinterpret_cast<const f32x4*>(us + c);
    f32x4 o = zero;
    if constexpr (RPT > 0) {
#pragma unroll
      for (int i = 0; i < RPT; ++i) {
        const int d = g + GR * i;
        if (d < D) {
          s[i] += u * ks[d];
          o += s[i] * qs[d];
          *reinterpret_cast<f32x4*>(st + (size_t)d * V + c) = s[i];
        }
      }
    } else {
      for (int d = g; d < D; d += GR) {
        float* sp = st + (size_t)d * V + c;
        const f32x4 x = (pos0 > 0 ? *reinterpret_cast<const f32x4*>(sp) * ws[d] : zero) + u * ks[d];
        o += x * qs[d];
        *reinterpret_cast<f32x4*>(sp) = x;
      }
    }
    *reinterpret_cast<f32x4*>(red + g * V + c) = o;
  }
  __syncthreads();
  float o[4], ss = 0.f;
#pragma unroll
  for (int x = 0; x < 4; ++x) {
    const int e = tid + 256 * x;
    o[x] = 0.f;
    if (e < V) {
      for (int i = 0; i < GR; ++i) o[x] += red[i * V + e];
      ss += o[x] * o[x];
    }
  }
#pragma unroll
  for (int x = 32; x > 0; x >>= 1) ss += __shfl_xor(ss, x, 64);
  if ((tid & 63) == 0) part[tid >> 6] = ss;
  __syncthreads();
  const float inv = 1.f / sqrtf((part[0] + part[1] + part[2] + part[3]) / (float)V + p.eps);
#pragma unroll
  for (int x = 0; x < 4; ++x) {
    const int e = tid + 256 * x;
    if (e < V) {
      const float gt = p.gate ? (float)((const T*)p.gate)[(size_t)t * p.ldg + hv + e]
                              : nls_lin::lin_sigmoid(low_dot((const T*)p.lowg + (size_t)t * p.ldz,
                                                             (const T*)p.g2 + (hv + e) * p.rg, p.rg));
      ((T*)p.out)[(size_t)t * p.ldout + hv + e] = (T)(o[x] * inv * p.norm[hv + e] * gt);
    }
  }
}

template <typename T>
int delta_step(const DS& p, int nruns, hipStream_t st) {
  const int GR = 256 / (p.V / 4), rpt = (p.D + GR - 1) / GR;
#define NLS_DS(N) \
  if (rpt <= N || N == 0) { \
    hipLaunchKernelGGL((delta_step_kernel<T, N>), dim3(p.H, nruns), dim3(256), 0, st, p); \
    return (int)hipGetLastError(); \
  }
  NLS_DS(4) NLS_DS(8) NLS_DS(16) NLS_DS(32) NLS_DS(0)
#undef NLS_DS
  return -1;
}

}  // namespace nls_gla

extern "C" {
using namespace nls_gla;

// z, y: [rows][q: G D | k: G D | v: H V], activation type; state [slots][sstride], [taps - 1][channels] of a slot
int nls_delta_conv(const void* z, long ldz, const float* w, void* y, long ldy, float* fac, long ldf, float* state, long sstride,
                   const int* runs, const int* tok_seq, int T, int nruns, int H, int G, int D, int V, int taps, int f32,
                   void* stream) {
  if (T < 1 || nruns < 1 || H < 1 || G < 1 || D < 1 || V < 1 || taps < 1 || (taps > 1 && !state) || ldf < 2L * G ||
      ldz < 2L * G * D + (long)H * V || ldy < 2L * G * D + (long)H * V)
    return -1;
  const CV p{z, y, w, fac, state, runs, tok_seq, ldz, ldy, ldf, sstride, T, H, G, D, V, taps};
  return f32 ? conv<float>(p, nruns, (hipStream_t)stream) : conv<__bf16>(p, nruns, (hipStream_t)stream);
}

// as nls_gla_scan, with the factors and beta of the delta rule; nseg > 1: rec [nruns][nseg][H][D][V], recm [nruns][nseg][H][D][D]
int nls_delta_scan(const void* q, const void* k, const void* v, long ld, const float* fac, long ldf, const float* beta, long ldb,
                   const float* a, long lda, float* o, long ldo, const float* norm, const void* gate, long ldg, void* out, long ldout,
                   float eps, float* state, long sstride, const int* runs, int nruns, int H, int G, int D, int V, int nseg, float* rec,
                   float* recm, int nt, int f32, void* stream) {
  const bool fused = norm && gate && out;
  if (nruns < 1 || H < 1 || G < 1 || H % G || D < 1 || V < 1 || nseg < 1 || nseg > 64 || (nseg > 1 && (!rec || !recm)) ||
      (!fused && !o) || !fac || !beta || ldf < 2L * G)
    return -1;
  GA p = gla_args(q, k, v, ld, a, lda, 1.f, o, ldo, norm, gate, ldg, out, ldout, eps, state, sstride, runs, H, D, V, nseg, rec, nullptr,
                  f32);
  p.fac = fac, p.beta = beta, p.recm = recm, p.ldf = ldf, p.ldb = ldb, p.G = G;
  return f32 ? delta_scan_f32(p, nruns, nt, (hipStream_t)stream) : delta_scan_bf16(p, nruns, nt, (hipStream_t)stream);
}

// every run has one token (or none); V a multiple of 4, at most 1024; D at most 256. low, lowg: rows of stride ldz, 16-byte aligned;
// a2 [H * D][ra], g2 [H * V][rg]
int nls_delta_step(const void* q, const void* k, const void* v, long ld, const float* fac, long ldf, const float* beta, long ldb,
                   const float* a, long lda, const void* low, const void* a2, const float* a2b, const float* rate, int ra,
                   const void* gate, long ldg, const void* lowg, const void* g2, int rg, long ldz, float* state, long sstride,
                   const int* runs, int nruns, const float* norm, void* out, long ldout, int H, int G, int D, int V, float eps,
                   int f32, void* stream) {
  if (nruns < 1 || H < 1 || G < 1 || H % G || D < 1 || D > 256 || V < 4 || V > 1024 || (V & 3) || (sstride & 3) || !fac || !beta ||
      !norm || !out || (!a && (!low || !a2 || !a2b || !rate || ra < 1)) || (!gate && (!lowg || !g2 || rg < 1)) ||
      (((uintptr_t)state | (uintptr_t)low | (uintptr_t)a2 | (uintptr_t)lowg | (uintptr_t)g2) & 15) || (ldz & 7))
    return -1;
  const DS p{q, k, v, fac, beta, a, low, a2, a2b, rate, gate, lowg, g2, norm, out, state, runs, ld, ldf, ldb, lda, ldz, ldg, ldout,
             sstride, H, G, D, V, ra, rg, eps};
  return f32 ? delta_step<float>(p, nruns, (hipStream_t)stream) : delta_step<__bf16>(p, nruns, (hipStream_t)stream);
}

}  // extern "C"
