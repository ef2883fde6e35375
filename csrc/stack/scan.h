// Gated linear recurrences with a per-channel decay (gfx950): what "wkv" time mixing (wkv.hip) and gated linear attention
// (gla.hip) share: the step of single tokens and the per-head output norm.
//
// Per head, with keys i and values j (state S [D][V], f32):
//   wkv: o_t[j] = sum_i r_t[i] (S[i][j] + u[i] k_t[i] v_t[j]);   S[i][j] = w_t[i] S[i][j] + k_t[i] v_t[j]
//   gla: S[i][j] = w_t[i] S[i][j] + k_t[i] v_t[j];               o_t[j] = rs sum_i r_t[i] S[i][j]
// A step of single tokens (decode) streams each head's state once with 16-byte accesses and ends with the head's norm and
// gate, or (norm null) with the plain outputs (step_kernel).
//
// A run = (first row, tokens, state slot, first position): consecutive rows of one sequence. A run at position 0
// starts from a zero state, any other from its slot; slot < 0 or 0 tokens: nothing to do (padded decode rows).
#pragma once
#include "lin.h"

namespace nls_scan {

enum Kind : int { WKV = 0, GLA = 1 };

template <typename T> DEVI float ld1(const T* p) { return (float)*p; }

template <int C>
DEVI float dpp_add(float v) {
  const int x = __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), C, 0xf, 0xf, true);
  return v + __builtin_bit_cast(float, x);
}
// sum over aligned groups of 8 or 16 lanes: quad swaps, half-row mirror, row mirror
template <int PARTS>
DEVI float sum_parts(float v) {
  v = dpp_add<0x141>(dpp_add<0x4E>(dpp_add<0xB1>(v)));
  return PARTS == 16 ? dpp_add<0x140>(v) : v;
}

struct Scan {
  const void *r, *k, *v;   // activation type, [rows][ld]: [H * D], [H * D], [H * V]
  const float* w;          // decays in [0, 1], f32 [rows][ldw]
  const float* u;          // wkv: [H * D]
  float* o;                // f32 [rows][ldo]: [H * V]
  float* state;            // [slots][sstride]: [H][D][V]
  const float* x;          // wkv: residual rows; the run's last becomes the slot's previous token (prev null: no such row)
  float* prev;
  const int* runs;
  long ld, ldw, ldo, sstride, ldx, ldp;
  int H, D, V, width;
  float rs;                // gla: factor of the output
  // gla step with the decays' last projection: w = sigmoid(a2 low + b)^ia (w above null)
  const void *low, *a2;    // [rows][ld], [H * D][rank]
  const float* a2b;
  int rank;
  float ia;
};

// ---- one token per run: the state of (run, head) is read and written once, 4 value columns per thread; then
// out = (o / rms(o)) * norm * gate, or (norm null) p.o. V is a multiple of 4, at most 1024; D at most 256.
template <typename T, int KIND>
__global__ __launch_bounds__(256) void step_kernel(Scan p, const float* __restrict__ norm, const T* __restrict__ gate,
                                                   long ldg, T* __restrict__ out, long ldout, float eps) {
  __shared__ __attribute__((aligned(16))) float rs[256], ks[256], ws[256], vs[1024], red[1024];
  __shared__ float part[8];
  const int* run = p.runs + 4 * blockIdx.y;
  const int t = run[0], n = run[1], slot = run[2], pos0 = run[3];
  if (slot < 0 || n != 1) return;
  const int D = p.D, V = p.V, head = blockIdx.x, tid = threadIdx.x;
  const size_t hb = (size_t)head * D, hv = (size_t)head * V;
  const int C4 = V >> 2, G = 256 / C4, c = (tid % C4) * 4, g = tid / C4;
  float* st = p.state + (size_t)slot * p.sstride + hb * V;
  float ruk = 0.f;
  if (tid < D) {
    const float r = ld1((const T*)p.r + (size_t)t * p.ld + hb + tid), k = ld1((const T*)p.k + (size_t)t * p.ld + hb + tid);
    rs[tid] = KIND == GLA ? r * p.rs : r;
    ks[tid] = k;
    if (KIND == WKV || p.w) {
      ws[tid] = p.w[(size_t)t * p.ldw + hb + tid];
    } else {
      const T *lo = (const T*)p.low + (size_t)t * p.ld, *a2 = (const T*)p.a2 + (hb + tid) * p.rank;
      float z = p.a2b[hb + tid];
      int i = 0;
      if ((p.rank & 7) == 0)                     // (16-byte aligned rows)
        for (; i < p.rank; i += 8) {
          typedef T t8 __attribute__((ext_vector_type(8)));
          const t8 x = *reinterpret_cast<const t8*>(lo + i), y = *reinterpret_cast<const t8*>(a2 + i);
#pragma unroll
          for (int e = 0; e < 8; ++e) z = fmaf((float)x[e], (float)y[e], z);
        }
      for (; i < p.rank; ++i) z = fmaf((float)lo[i], (float)a2[i], z);
      ws[tid] = nls_lin::lin_sigpow(z, p.ia);
    }
    if (KIND == WKV) ruk = r * p.u[hb + tid] * k;
  }
  for (int i = tid; i < V; i += 256) vs[i] = ld1((const T*)p.v + (size_t)t * p.ld + hv + i);
  if (KIND == WKV) {
#pragma unroll
    for (int q = 32; q > 0; q >>= 1) ruk += __shfl_xor(ruk, q, 64);
    if ((tid & 63) == 0) part[tid >> 6] = ruk;
  }
  __syncthreads();
  if (KIND == WKV) ruk = part[0] + part[1] + part[2] + part[3];
  if (g < G) {
    const f32x4 v = *reinterpret_cast<const f32x4*>(vs + c);
    f32x4 o = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int i = g; i < D; i += G) {
      float* sp = st + (size_t)i * V + c;
      const f32x4 s = pos0 > 0 ? *reinterpret_cast<const f32x4*>(sp) : f32x4{0.f, 0.f, 0.f, 0.f};
      const f32x4 s1 = s * ws[i] + v * ks[i];
      o += (KIND == WKV ? s : s1) * rs[i];
      *reinterpret_cast<f32x4*>(sp) = s1;
    }
    *reinterpret_cast<f32x4*>(red + g * V + c) = o;
  }
  __syncthreads();
  float o[4], ss = 0.f;
#pragma unroll
  for (int q = 0; q < 4; ++q) {
    const int e = tid + 256 * q;
    o[q] = 0.f;
    if (e < V) {
      for (int i = 0; i < G; ++i) o[q] += red[i * V + e];
      if (KIND == WKV) o[q] += ruk * vs[e];
      ss += o[q] * o[q];
      if (KIND == GLA && !norm) p.o[(size_t)t * p.ldo + hv + e] = o[q];
    }
  }
  if (KIND == GLA && !norm) return;
#pragma unroll
  for (int q = 32; q > 0; q >>= 1) ss += __shfl_xor(ss, q, 64);
  if ((tid & 63) == 0) part[4 + (tid >> 6)] = ss;
  __syncthreads();
  ss = part[4] + part[5] + part[6] + part[7];
  const float inv = 1.f / sqrtf(ss / (float)V + eps);
#pragma unroll
  for (int q = 0; q < 4; ++q) {
    const int e = tid + 256 * q;
    if (e < V)
      out[(size_t)t * ldout + hv + e] = (T)(o[q] * inv * norm[hv + e] * (float)gate[(size_t)t * ldg + hv + e]);
  }
  if (KIND != WKV || !p.prev) return;
  for (int i = blockIdx.x * 256 + tid; i < p.width; i += gridDim.x * 256)
    p.prev[(size_t)slot * p.ldp + i] = p.x[(size_t)t * p.ldx + i];
}

// ---- out = (o / rms(o) per head of D columns) * norm * gate
template <typename T>
__global__ __launch_bounds__(256) void out_kernel(const float* __restrict__ o, long ldo,
                                                      const float* __restrict__ norm, const T* __restrict__ gate,
                                                      long ldg, T* __restrict__ out, long ld, int H, int D, float eps) {
  const int t = blockIdx.x, lane = threadIdx.x & 63;
  for (int h = blockIdx.y * 4 + (threadIdx.x >> 6); h < H; h += gridDim.y * 4) {
    const float* p = o + (size_t)t * ldo + (size_t)h * D;
    float s = 0.f;
    for (int i = lane; i < D; i += 64) s += p[i] * p[i];
#pragma unroll
    for (int q = 32; q > 0; q >>= 1) s += __shfl_xor(s, q, 64);
    const float inv = 1.f / sqrtf(s / (float)D + eps);
    for (int i = lane; i < D; i += 64) {
      const int c = h * D + i;
      out[(size_t)t * ld + c] = (T)(p[i] * inv * norm[c] * (float)gate[(size_t)t * ldg + c]);
    }
  }
}

template <typename T>
int out_rows(const float* o, long ldo, const float* norm, const void* gate, long ldg, void* out, long ld, int H, int D, int T_,
             float eps, hipStream_t st) {
  if (T_ < 1 || H < 1 || D < 1) return -1;
  const dim3 grid(T_, T_ >= 256 ? 1 : min((H + 3) / 4, 64));
  hipLaunchKernelGGL(out_kernel<T>, grid, dim3(256), 0, st, o, ldo, norm, (const T*)gate, ldg, (T*)out, ld, H, D, eps);
  return (int)hipGetLastError();
}

template <typename T, int KIND>
int step_rows(const Scan& p, int nruns, const float* norm, const void* gate, long ldg, void* out, long ldout, float eps,
              hipStream_t st) {
  if (nruns < 1 || p.H < 1 || p.D < 1 || p.D > 256 || p.V < 4 || p.V > 1024 || (p.V & 3) || (p.sstride & 3)) return -1;
  hipLaunchKernelGGL((step_kernel<T, KIND>), dim3(p.H, nruns), dim3(256), 0, st, p, norm, (const T*)gate, ldg, (T*)out, ldout,
                     eps);
  return (int)hipGetLastError();
}

}  // namespace nls_scan
