// Causal attention over paged rows for any head widths, one workgroup per (token, query head), f32 arithmetic throughout:
// 32-bit models, and head widths that the MFMA kernels do not take.
#pragma once
#include "../kernels/common.h"

namespace nls_plain {

constexpr int NC = 4;         // output columns per thread: values of up to 256 * NC columns
constexpr int MAXK = 2048;    // key columns

struct PA {
  const void *q, *k, *v;
  void* out;
  const int* bt;              // block tables
  const int* tok_seq;
  const int* ctx_len;         // keys of each token (0: padded row)
  const float* gate;          // [T][ldg], a factor per token and head (null: none)
  long ldq, qhs;              // row and head strides of the queries
  long ldkv, khs;             // row and key-head strides of the cache
  long ldo, ohs;
  long ldg;
  int bts, bs, gs;            // gs: query heads per key head
  int Dk, Dv;                 // columns (Dk a multiple of 4)
  float scale;
  int window, keep, sink;     // window > 0: the newest `window` keys and the first `keep`; sink: one more in the denominator
};

template <typename T> DEVI f32x4 ld4(const T* p) {
  typedef T t4 __attribute__((ext_vector_type(4)));
  const t4 a = *reinterpret_cast<const t4*>(p);
  return f32x4{(float)a[0], (float)a[1], (float)a[2], (float)a[3]};
}

template <typename T>
__global__ __launch_bounds__(256) void attn_plain_kernel(PA p) {
  __shared__ __attribute__((aligned(16))) float q[MAXK], sc[64];
  const int t = blockIdx.x, h = blockIdx.y;
  const int ctx = p.ctx_len[t];
  const int* bt = p.bt + (size_t)p.tok_seq[t] * p.bts;
  const T* kc = reinterpret_cast<const T*>(p.k) + (size_t)(h / p.gs) * p.khs;
  const T* vc = reinterpret_cast<const T*>(p.v) + (size_t)(h / p.gs) * p.khs;
  const T* qr = reinterpret_cast<const T*>(p.q) + (size_t)t * p.ldq + (size_t)h * p.qhs;
  for (int i = threadIdx.x; i < p.Dk; i += 256) q[i] = (float)qr[i];
  __syncthreads();
  const int key = threadIdx.x >> 2, part = threadIdx.x & 3;
  float m = p.sink ? 0.f : -INFINITY, l = p.sink ? 1.f : 0.f, acc[NC] = {0.f, 0.f, 0.f, 0.f};
  const int low = p.window > 0 ? ctx - p.window : 0;                  // first key of the window
  for (int k0 = 0; k0 < ctx; k0 += 64) {
    if (k0 >= p.keep && k0 + 64 <= low) k0 = low & ~63;               // (none of the tiles between is seen)
    const int k = k0 + key;
    const bool see = k < ctx && (k >= low || k < p.keep);
    float s = 0.f;
    if (k < ctx) {
      const T* c = kc + ((size_t)bt[k / p.bs] * p.bs + k % p.bs) * p.ldkv;
      for (int d = part * 4; d < p.Dk; d += 16) {
        const f32x4 a = ld4(c + d), b = *reinterpret_cast<const f32x4*>(q + d);
#pragma unroll
        for (int e = 0; e < 4; ++e) s = fmaf(a[e], b[e], s);
      }
    }
    s += __shfl_xor(s, 1, 64);
    s += __shfl_xor(s, 2, 64);
    if (part == 0) sc[key] = see ? s * p.scale : -INFINITY;
    __syncthreads();
    float mn = m;
    for (int i = 0; i < 64; ++i) mn = fmaxf(mn, sc[i]);
    const float alpha = m == -INFINITY ? 0.f : expf(m - mn), base = mn == -INFINITY ? 0.f : mn;
    l *= alpha;
#pragma unroll
    for (int i = 0; i < NC; ++i) acc[i] *= alpha;
    m = mn;
    const int n = min(64, ctx - k0);
    for (int i = 0; i < n; ++i) {
      const float e = expf(sc[i] - base);
      l += e;
      const int kk = k0 + i;
      const T* c = vc + ((size_t)bt[kk / p.bs] * p.bs + kk % p.bs) * p.ldkv;
#pragma unroll
      for (int q4 = 0; q4 < NC; ++q4) {
        const int col = threadIdx.x + 256 * q4;
        if (col < p.Dv) acc[q4] = fmaf(e, (float)c[col], acc[q4]);
      }
    }
    __syncthreads();
  }
  const float inv = (l > 0.f ? 1.f / l : 0.f) * (p.gate ? p.gate[(size_t)t * p.ldg + h] : 1.f);
  T* y = reinterpret_cast<T*>(p.out) + (size_t)t * p.ldo + (size_t)h * p.ohs;
#pragma unroll
  for (int q4 = 0; q4 < NC; ++q4) {
    const int col = threadIdx.x + 256 * q4;
    if (col < p.Dv) y[col] = (T)(acc[q4] * inv);
  }
}

template <typename T>
int launch(const PA& p, int T_, int H, hipStream_t st) {
  if (T_ < 1 || H < 1 || H > 65535 || p.gs < 1 || p.Dk > MAXK || (p.Dk & 3) || (p.ldkv & 3) || (p.khs & 3) || p.Dv > 256 * NC ||
      p.bs < 1)
    return -1;
  hipLaunchKernelGGL(attn_plain_kernel<T>, dim3(T_, H), dim3(256), 0, st, p);
  return (int)hipGetLastError();
}

}  // namespace nls_plain
