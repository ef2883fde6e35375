// "wkv" time mixing (gfx950): the token shift, the recurrence over runs of tokens, and the entry points of its single-token step
// (scan.h).
//
// The scan is sequential in the tokens of a run, so a position's result does not depend on how its sequence was cut
// into steps. Parallelism is (run, head, value columns) x lanes: a lane holds DP / PARTS key rows of CPL value columns in
// registers, PARTS neighbouring lanes cover the keys and close the sum with in-row lane exchanges (DPP). Few runs take
// many key parts (short per-token chains on all CUs). Tokens are staged in LDS in chunks of CH as f32, the next chunk's
// loads in flight while the current one runs.
#include "scan.h"

namespace nls_wkv {
using namespace nls_scan;

// ---- token shift: m_s[t] = h[t] + (h[t - 1] - h[t]) * mu_s for NS mixes; h = the f32 residual row. The row before
// a run's first is the slot's previous token (zeros at position 0).
constexpr int NS = 5;
struct Mix {
  const float* x;
  const float* mu;      // [NS][D]
  const float* prev;    // [slots][prev stride]
  void* out;            // [NS][rows cap][ldo]
  const int* runs;      // [nruns][4]
  const int* tok_seq;   // row -> run
  long ldx, ldp, ldo, mstride;
  int D, f32;
};

template <typename T>
__global__ __launch_bounds__(256) void shift_mix_kernel(Mix p) {
  const int t = blockIdx.x;
  const int* run = p.runs + 4 * p.tok_seq[t];
  const int t0 = run[0], n = run[1], slot = run[2], pos0 = run[3];
  if (slot < 0 || t < t0 || t >= t0 + n) return;
  const float* h = p.x + (size_t)t * p.ldx;
  const float* q = t > t0 ? h - p.ldx : (pos0 > 0 ? p.prev + (size_t)slot * p.ldp : nullptr);
  T* o = reinterpret_cast<T*>(p.out) + (size_t)t * p.ldo;
  for (int i = blockIdx.y * 256 + threadIdx.x; i < p.D; i += gridDim.y * 256) {
    const float a = h[i], d = (q ? q[i] : 0.f) - a;
#pragma unroll
    for (int s = 0; s < NS; ++s) o[s * p.mstride + i] = (T)(a + d * p.mu[s * p.D + i]);
  }
}

// DP: key channels padded to a multiple of 32 (zeros past D)
template <typename T, int DP, int PARTS, int CPL>
__global__ __launch_bounds__(256) void wkv_scan_kernel(Scan p) {
  constexpr int WC = 256 / PARTS * CPL;          // value columns per workgroup
  constexpr int CH = DP <= 64 ? 32 : (DP <= 128 ? 16 : 8);   // tokens per staged chunk
  constexpr int R = DP / PARTS;                  // state rows per lane
  constexpr int LR = DP + 4;                     // LDS row stride
  constexpr int NV = (CH * DP + 255) / 256;      // staged values per thread and operand
  __shared__ __attribute__((aligned(16))) float rs[CH][LR], ks[CH][LR], ws[CH][LR];
  __shared__ __attribute__((aligned(16))) float vs[CH][WC], ruk[CH];
  const int* run = p.runs + 4 * blockIdx.y;
  const int t0 = run[0], n = run[1], slot = run[2], pos0 = run[3];
  if (slot < 0 || n < 1) return;
  const int D = p.D;
  const int ncb = (D + WC - 1) / WC;
  const int head = blockIdx.x / ncb, c0 = (blockIdx.x % ncb) * WC;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int part = lane & (PARTS - 1), col = (wave * (64 / PARTS) + lane / PARTS) * CPL;
  const int j = c0 + col;
  const size_t hb = (size_t)head * D;
  const T* rp = (const T*)p.r + hb;
  const T* kp = (const T*)p.k + hb;
  const T* vp = (const T*)p.v + hb;
  const float* wp = p.w + hb;
  float* st = p.state + (size_t)slot * p.sstride + hb * D;

  float S[CPL][R];
#pragma unroll
  for (int i = 0; i < R; ++i)
#pragma unroll
    for (int c = 0; c < CPL; ++c) {
      const int row = part * R + i;
      S[c][i] = (pos0 > 0 && row < D && j + c < D) ? st[(size_t)row * D + j + c] : 0.f;
    }
  float ur[DP / 16];                             // u of the bonus sums' columns
#pragma unroll
  for (int q = 0; q < DP / 16; ++q) {
    const int i = (threadIdx.x & 15) + 16 * q;
    ur[q] = i < D ? p.u[hb + i] : 0.f;
  }
  float fr[NV], fk[NV], fw[NV], fv[(CH * WC + 255) / 256];
  auto fetch = [&](int base) __attribute__((always_inline)) {
#pragma unroll
    for (int q = 0; q < NV; ++q) {
      const int e = threadIdx.x + q * 256, tt = e / DP, i = e % DP;
      const bool in = tt < CH && base + tt < n && i < D;
      const size_t row = (size_t)(t0 + min(base + tt, n - 1));
      fr[q] = in ? ld1(rp + row * p.ld + i) : 0.f;
      fk[q] = in ? ld1(kp + row * p.ld + i) : 0.f;
      fw[q] = in ? wp[row * p.ldw + i] : 0.f;
    }
#pragma unroll
    for (int q = 0; q < (CH * WC + 255) / 256; ++q) {
      const int e = threadIdx.x + q * 256, tt = e / WC, i = c0 + (e & (WC - 1));
      const bool in = tt < CH && base + tt < n && i < D;
      fv[q] = in ? ld1(vp + (size_t)(t0 + min(base + tt, n - 1)) * p.ld + i) : 0.f;
    }
  };
  fetch(0);
  for (int base = 0; base < n; base += CH) {
    __syncthreads();
#pragma unroll
    for (int q = 0; q < NV; ++q) {
      const int e = threadIdx.x + q * 256, tt = e / DP, i = e % DP;
      if (tt < CH) {
        rs[tt][i] = fr[q];
        ks[tt][i] = fk[q];
        ws[tt][i] = fw[q];
      }
    }
#pragma unroll
    for (int q = 0; q < (CH * WC + 255) / 256; ++q) {
      const int e = threadIdx.x + q * 256;
      if (e < CH * WC) vs[e / WC][e & (WC - 1)] = fv[q];
    }
    __syncthreads();
    if (base + CH < n) fetch(base + CH);
    // sum_i r u k of every staged token: 16 lanes each
#pragma unroll
    for (int t8 = 0; t8 < CH; t8 += 16) {
      const int tt = t8 + (threadIdx.x >> 4), l = threadIdx.x & 15;
      float a = 0.f;
      if (tt < CH)
#pragma unroll
        for (int q = 0; q < DP / 16; ++q) a += rs[tt][l + 16 * q] * ur[q] * ks[tt][l + 16 * q];
#pragma unroll
      for (int s = 8; s > 0; s >>= 1) a += __shfl_xor(a, s, 64);
      if (tt < CH && l == 0) ruk[tt] = a;
    }
    __syncthreads();
    // 8 tokens at a time, the next token's operands on their way while one is summed; lane part q keeps token q's output
    const int m = min(CH, n - base);
    f32x4 r4[2][R / 4], k4[2][R / 4], w4[2][R / 4];
    float v1[2][CPL];
    auto get = [&](int tt, int b) __attribute__((always_inline)) {
#pragma unroll
      for (int q = 0; q < R / 4; ++q) {
        r4[b][q] = *reinterpret_cast<const f32x4*>(&rs[tt][part * R + 4 * q]);
        k4[b][q] = *reinterpret_cast<const f32x4*>(&ks[tt][part * R + 4 * q]);
        w4[b][q] = *reinterpret_cast<const f32x4*>(&ws[tt][part * R + 4 * q]);
      }
#pragma unroll
      for (int c = 0; c < CPL; ++c) v1[b][c] = vs[tt][col + c];
    };
    auto token = [&](int b, float (&o)[CPL]) __attribute__((always_inline)) {
#pragma unroll
      for (int c = 0; c < CPL; ++c) {
        float o0 = 0.f, o1 = 0.f;
#pragma unroll
        for (int i4 = 0; i4 < R / 4; ++i4)
#pragma unroll
          for (int e = 0; e < 4; e += 2) {
            const int i = 4 * i4 + e;
            o0 = fmaf(r4[b][i4][e], S[c][i], o0);
            o1 = fmaf(r4[b][i4][e + 1], S[c][i + 1], o1);
            S[c][i] = fmaf(w4[b][i4][e], S[c][i], k4[b][i4][e] * v1[b][c]);
            S[c][i + 1] = fmaf(w4[b][i4][e + 1], S[c][i + 1], k4[b][i4][e + 1] * v1[b][c]);
          }
        o[c] = sum_parts<PARTS>(o0 + o1);
      }
    };
    get(0, 0);
    for (int t8 = 0; t8 < m; t8 += 8) {
      float mine[CPL], o[CPL];
#pragma unroll
      for (int c = 0; c < CPL; ++c) mine[c] = 0.f;
      const int last = m - 1 - t8, tt = t8 + (part & 7);
      const float rk = ruk[tt];
      if (last >= 7) {
#pragma unroll
        for (int q = 0; q < 8; ++q) {
          get(min(t8 + q + 1, CH - 1), (q & 1) ^ 1);
          token(q & 1, o);
#pragma unroll
          for (int c = 0; c < CPL; ++c) mine[c] = part == q ? o[c] : mine[c];
        }
      } else {
#pragma unroll
        for (int q = 0; q < 8; ++q) {
          get(min(t8 + q + 1, CH - 1), (q & 1) ^ 1);
          if (q > last) continue;              // (uniform)
          token(q & 1, o);
#pragma unroll
          for (int c = 0; c < CPL; ++c) mine[c] = part == q ? o[c] : mine[c];
        }
      }
      if (part < 8 && part <= last)
#pragma unroll
        for (int c = 0; c < CPL; ++c)
          if (j + c < D) p.o[(size_t)(t0 + base + tt) * p.ldo + hb + j + c] = fmaf(rk, vs[tt][col + c], mine[c]);
    }
  }
#pragma unroll
  for (int i = 0; i < R; ++i)
#pragma unroll
    for (int c = 0; c < CPL; ++c) {
      const int row = part * R + i;
      if (row < D && j + c < D) st[(size_t)row * D + j + c] = S[c][i];
    }
  // the run's last row is the next step's previous token (this layer's shift_mix, which reads it, came before)
  const int G = gridDim.x;
  for (int i = blockIdx.x * 256 + threadIdx.x; i < p.width; i += G * 256)
    p.prev[(size_t)slot * p.ldp + i] = p.x[(size_t)(t0 + n - 1) * p.ldx + i];
}

template <typename T, int DP>
int scan_d(const Scan& p, int nruns, hipStream_t st) {
  auto grid = [&](int wc) { return dim3(p.H * ((p.V + wc - 1) / wc), nruns); };
  if (DP < 64 || p.H * nruns * ((p.V + 31) / 32) >= 256)
    hipLaunchKernelGGL((wkv_scan_kernel<T, DP, 8, 1>), grid(32), dim3(256), 0, st, p);
  else
    hipLaunchKernelGGL((wkv_scan_kernel<T, DP, DP < 64 ? 8 : 16, 1>), grid(16), dim3(256), 0, st, p);
  return (int)hipGetLastError();
}

template <typename T>
int scan_t(const Scan& p, int nruns, hipStream_t st) {
  if (p.D <= 32) return scan_d<T, 32>(p, nruns, st);
  if (p.D <= 64) return scan_d<T, 64>(p, nruns, st);
  if (p.D <= 128) return scan_d<T, 128>(p, nruns, st);
  if (p.D <= 256) return scan_d<T, 256>(p, nruns, st);
  return -1;
}

Scan args(const void* r, const void* k, const void* v, long ld, const float* w, long ldw, const float* u, float* o, long ldo,
          float* state, long sstride, const float* x, long ldx, float* prev, long ldp, int width, const int* runs, int H, int D) {
  return Scan{r, k, v, w, u, o, state, x, prev, runs, ld, ldw, ldo, sstride, ldx, ldp, H, D, D, width, 1.f, nullptr, nullptr, nullptr, 0,
              0.f};
}

}  // namespace nls_wkv

extern "C" {
using namespace nls_wkv;

int nls_shift_mix(const float* x, long ldx, const float* mu, const float* prev, long ldp, void* out, long ldo,
                  long mstride, const int* runs, const int* tok_seq, int D, int T, int f32, void* stream) {
  if (T < 1 || D < 1) return -1;
  Mix p{x, mu, prev, out, runs, tok_seq, ldx, ldp, ldo, mstride, D, f32};
  const dim3 grid(T, T >= 256 ? 1 : min((D + 255) / 256, 16));
  if (f32) hipLaunchKernelGGL(shift_mix_kernel<float>, grid, dim3(256), 0, (hipStream_t)stream, p);
  else hipLaunchKernelGGL(shift_mix_kernel<__bf16>, grid, dim3(256), 0, (hipStream_t)stream, p);
  return (int)hipGetLastError();
}

int nls_wkv_scan(const void* r, const void* k, const void* v, long ld, const float* w, long ldw, const float* u,
                 float* o, long ldo, float* state, long sstride, const float* x, long ldx, float* prev, long ldp,
                 int width, const int* runs, int nruns, int H, int D, int f32, void* stream) {
  if (nruns < 1 || H < 1 || D < 1) return -1;
  const Scan p = args(r, k, v, ld, w, ldw, u, o, ldo, state, sstride, x, ldx, prev, ldp, width, runs, H, D);
  return f32 ? scan_t<float>(p, nruns, (hipStream_t)stream) : scan_t<__bf16>(p, nruns, (hipStream_t)stream);
}

// every run has one token (or none); D a multiple of 4
int nls_wkv_step(const void* r, const void* k, const void* v, long ld, const float* w, long ldw, const float* u,
                 float* state, long sstride, const float* x, long ldx, float* prev, long ldp, int width, const int* runs,
                 int nruns, const float* norm, const void* gate, long ldg, void* out, long ldout, int H, int D, float eps,
                 int f32, void* stream) {
  const Scan p = args(r, k, v, ld, w, ldw, u, nullptr, 0, state, sstride, x, ldx, prev, ldp, width, runs, H, D);
  return f32 ? step_rows<float, WKV>(p, nruns, norm, gate, ldg, out, ldout, eps, (hipStream_t)stream)
             : step_rows<__bf16, WKV>(p, nruns, norm, gate, ldg, out, ldout, eps, (hipStream_t)stream);
}

// per-head norm of D columns, norm weight and gate of a recurrence's output rows
int nls_scan_out(const float* o, long ldo, const float* norm, const void* gate, long ldg, void* out, long ld, int H,
                 int D, int T, float eps, int f32, void* stream) {
  return f32 ? out_rows<float>(o, ldo, norm, gate, ldg, out, ld, H, D, T, eps, (hipStream_t)stream)
             : out_rows<__bf16>(o, ldo, norm, gate, ldg, out, ld, H, D, T, eps, (hipStream_t)stream);
}

}  // extern "C"
