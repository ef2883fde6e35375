// Attention whose heads' softmax weights are mixed, over paged rows, for any head count and widths: one workgroup per token,
// f32 arithmetic throughout (32-bit models, shapes that the MFMA kernels do not take). See talk_attn.hip.
#pragma once
#include "../kernels/common.h"

namespace nls_talk {

struct TalkArgs {
  const void *q, *k, *v;      // q [T][ldq], heads Dp apart; k, v: paged [slots][G][Dp]
  void* out;                  // [T][ldo], heads Dp apart
  const void* gate;           // [T][ldg] of the activation type, a factor per column, heads V apart (null: none)
  const void* talk;           // plain: f32 [H][H]; MFMA kernels: bf16 [32 kk][32 kk], kk = ceil(H / 32), zero past H
  const int *bt, *tok_seq, *ctx_len;
  long ldq, ldo, ldg;
  int bts, bs, H, G, Dp, V;   // V: columns of a value head
  float scale;
  int window;                 // > 0: a token at position i sees j <= i if i - j < window
};

namespace plain {

constexpr int KT = 32, NC = 8;

template <typename T>
__global__ __launch_bounds__(256) void talk_plain_kernel(TalkArgs p) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int t = blockIdx.x, H = p.H, Dp = p.Dp, gs = H / p.G, tid = threadIdx.x;
  float *q = sm, *sc = q + H * Dp, *mx = sc + H * (KT + 1), *ms = mx + H * (KT + 1), *ls = ms + H;
  const int ctx = p.ctx_len[t];
  if (ctx <= 0) return;
  const int* bt = p.bt + (size_t)p.tok_seq[t] * p.bts;
  const long ldkv = (long)p.G * Dp;
  const T *qr = (const T*)p.q + (size_t)t * p.ldq, *kc = (const T*)p.k, *vc = (const T*)p.v;
  const float* talk = (const float*)p.talk;
  for (int i = tid; i < H * Dp; i += 256) q[i] = (float)qr[i];
  for (int h = tid; h < H; h += 256) {
    ms[h] = -INFINITY;
    ls[h] = 0.f;
  }
  __syncthreads();
  const int low = p.window > 0 ? max(0, ctx - p.window) : 0;
  auto row = [&](int k) { return (size_t)((long)bt[k / p.bs] * p.bs + k % p.bs) * ldkv; };
  auto scores = [&](int k0) {           // sc[h][key]: scaled scores of keys k0 .. k0 + KT - 1 (-inf: not seen)
    for (int e = tid; e < H * KT; e += 256) {
      const int h = e / KT, k = k0 + e % KT;
      float s = -INFINITY;
      if (k < ctx) {
        const T* c = kc + row(k) + (size_t)(h / gs) * Dp;
        const float* a = q + h * Dp;
        s = 0.f;
        for (int d = 0; d < Dp; ++d) s = fmaf(a[d], (float)c[d], s);
        s *= p.scale;
      }
      sc[h * (KT + 1) + e % KT] = s;
    }
    __syncthreads();
  };
  for (int k0 = low; k0 < ctx; k0 += KT) {
    scores(k0);
    for (int h = tid; h < H; h += 256) {
      const float* s = sc + h * (KT + 1);
      float m = ms[h], l = ls[h], mn = m;
      for (int i = 0; i < KT; ++i) mn = fmaxf(mn, s[i]);
      l *= m == -INFINITY ? 0.f : expf(m - mn);
      for (int i = 0; i < KT; ++i) l += expf(s[i] - mn);
      ms[h] = mn;
      ls[h] = l;
    }
    __syncthreads();
  }
  float acc[NC];
#pragma unroll
  for (int i = 0; i < NC; ++i) acc[i] = 0.f;
  const int HV = H * p.V, o0 = blockIdx.y * 256 * NC;
  for (int k0 = low; k0 < ctx; k0 += KT) {
    scores(k0);
    for (int e = tid; e < H * KT; e += 256) {
      const int h = e / KT, i = h * (KT + 1) + e % KT;
      sc[i] = expf(sc[i] - ms[h]) / ls[h];
    }
    __syncthreads();
    for (int e = tid; e < H * KT; e += 256) {
      const int h = e / KT, i = e % KT;
      float w = 0.f;
      for (int g = 0; g < H; ++g) w = fmaf(talk[(size_t)h * H + g], sc[g * (KT + 1) + i], w);
      mx[h * (KT + 1) + i] = w;
    }
    __syncthreads();
    const int n = min(KT, ctx - k0);
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      const int o = o0 + tid + 256 * c;
      if (o >= HV) continue;
      const int h = o / p.V, d = o - h * p.V;
      const float* w = mx + h * (KT + 1);
      for (int i = 0; i < n; ++i) acc[c] = fmaf(w[i], (float)vc[row(k0 + i) + (size_t)(h / gs) * Dp + d], acc[c]);
    }
    __syncthreads();
  }
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int o = o0 + tid + 256 * c;
    if (o >= HV) continue;
    const int h = o / p.V, d = o - h * p.V;
    const float g = p.gate ? (float)((const T*)p.gate)[(size_t)t * p.ldg + o] : 1.f;
    ((T*)p.out)[(size_t)t * p.ldo + (size_t)h * Dp + d] = (T)(acc[c] * g);
  }
}

template <typename T>
int launch(const TalkArgs& p, int n, hipStream_t st) {
  const size_t lds = sizeof(float) * ((size_t)p.H * p.Dp + 2 * (size_t)p.H * (KT + 1) + 2 * (size_t)p.H);
  if (lds > 160 * 1024) return -1;
  static bool attr = false;
  if (!attr) {
    if (hipFuncSetAttribute((const void*)talk_plain_kernel<T>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024) != hipSuccess)
      return -1;
    attr = true;
  }
  hipLaunchKernelGGL(talk_plain_kernel<T>, dim3(n, (p.H * p.V + 256 * NC - 1) / (256 * NC)), dim3(256), lds, st, p);
  return (int)hipGetLastError();
}

}  // namespace plain
}  // namespace nls_talk
