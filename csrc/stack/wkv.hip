// "wkv" time mixing (gfx950): the token shift and the entry points of its recurrence (scan.h).
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

template <typename T, int DP>
int scan_d(const Scan& p, int nruns, hipStream_t st) {
  auto grid = [&](int wc) { return dim3(p.H * ((p.V + wc - 1) / wc), nruns); };
  if (DP < 64 || p.H * nruns * ((p.V + 31) / 32) >= 256)
    hipLaunchKernelGGL((scan_kernel<T, WKV, DP, 8, 1>), grid(32), dim3(256), 0, st, p);
  else
    hipLaunchKernelGGL((scan_kernel<T, WKV, DP, DP < 64 ? 8 : 16, 1>), grid(16), dim3(256), 0, st, p);
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
  return Scan{r, k, v, w, u, o, state, x, prev, runs, nullptr, nullptr, ld, ldw, ldo, sstride, ldx, ldp, H, D, D, width, 1, 0, 1.f};
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
