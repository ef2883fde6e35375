// Gated linear recurrence with a per-channel decay ("wkv" time mixing), gfx950.
//
// Per head, with keys i and values j (state S [dim][dim], f32):
//   o_t[j] = sum_i r_t[i] (S[i][j] + u[i] k_t[i] v_t[j]);   S[i][j] = w_t[i] S[i][j] + k_t[i] v_t[j]
//
// The scan is sequential in the tokens of a run, so a position's result does not depend on how its sequence was cut
// into steps. Parallelism is (run, head, value columns) x lanes: a lane holds DP / PARTS key rows of CPL value columns in
// registers, PARTS neighbouring lanes cover the keys and close the sum with in-row lane exchanges (DPP). Few runs take
// many key parts (short per-token chains on all CUs). Tokens are staged in LDS in chunks of CH as f32, the next chunk's
// loads in flight while the current one runs.
// A step of single tokens (decode) streams each head's state once with 16-byte accesses and ends with the head's norm and
// gate (wkv_step_kernel).
//
// A run = (first row, tokens, state slot, first position): consecutive rows of one sequence. A run at position 0
// starts from a zero state, any other from its slot; slot < 0 or 0 tokens: nothing to do (padded decode rows).
#include "../kernels/common.h"

namespace nls_wkv {

template <typename T> DEVI float ld1(const T* p) { return (float)*p; }

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
  const void *r, *k, *v;   // activation type, [rows][ld]
  const float* w;          // decays in (0, 1), f32 [rows][ldw]
  const float* u;          // [H * D]
  float* o;                // f32 [rows][ldo]
  float* state;            // [slots][sstride]: [H][D][D]
  const float* x;          // residual rows: the run's last becomes the slot's previous token
  float* prev;
  const int* runs;
  long ld, ldw, ldo, sstride, ldx, ldp;
  int H, D, width;
};

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

// ---- one token per run: the state of (run, head) is read and written once, 4 value columns per thread; then
// out = (o / rms(o)) * norm * gate. D is a multiple of 4.
template <typename T>
__global__ __launch_bounds__(256) void wkv_step_kernel(Scan p, const float* __restrict__ norm, const T* __restrict__ gate,
                                                       long ldg, T* __restrict__ out, long ldout, float eps) {
  __shared__ __attribute__((aligned(16))) float rs[256], ks[256], ws[256], vs[256], red[1024 + 256];
  __shared__ float part[8];
  const int* run = p.runs + 4 * blockIdx.y;
  const int t = run[0], n = run[1], slot = run[2], pos0 = run[3];
  if (slot < 0 || n != 1) return;
  const int D = p.D, head = blockIdx.x, tid = threadIdx.x;
  const size_t hb = (size_t)head * D;
  const int C4 = D >> 2, G = 256 / C4, c = (tid % C4) * 4, g = tid / C4;
  float* st = p.state + (size_t)slot * p.sstride + hb * D;
  float ruk = 0.f;
  if (tid < D) {
    const float r = ld1((const T*)p.r + (size_t)t * p.ld + hb + tid), k = ld1((const T*)p.k + (size_t)t * p.ld + hb + tid);
    rs[tid] = r;
    ks[tid] = k;
    ws[tid] = p.w[(size_t)t * p.ldw + hb + tid];
    vs[tid] = ld1((const T*)p.v + (size_t)t * p.ld + hb + tid);
    ruk = r * p.u[hb + tid] * k;
  }
#pragma unroll
  for (int q = 32; q > 0; q >>= 1) ruk += __shfl_xor(ruk, q, 64);
  if ((tid & 63) == 0) part[tid >> 6] = ruk;
  __syncthreads();
  ruk = part[0] + part[1] + part[2] + part[3];
  if (g < G) {
    const f32x4 v = *reinterpret_cast<const f32x4*>(vs + c);
    f32x4 o = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int i = g; i < D; i += G) {
      float* sp = st + (size_t)i * D + c;
      const f32x4 s = pos0 > 0 ? *reinterpret_cast<const f32x4*>(sp) : f32x4{0.f, 0.f, 0.f, 0.f};
      o += s * rs[i];
      *reinterpret_cast<f32x4*>(sp) = s * ws[i] + v * ks[i];
    }
    *reinterpret_cast<f32x4*>(red + g * D + c) = o;
  }
  __syncthreads();
  float o = 0.f, ss = 0.f;
  if (tid < D) {
    for (int i = 0; i < G; ++i) o += red[i * D + tid];
    o += ruk * vs[tid];
    ss = o * o;
  }
#pragma unroll
  for (int q = 32; q > 0; q >>= 1) ss += __shfl_xor(ss, q, 64);
  if ((tid & 63) == 0) part[4 + (tid >> 6)] = ss;
  __syncthreads();
  ss = part[4] + part[5] + part[6] + part[7];
  if (tid < D) {
    const float inv = 1.f / sqrtf(ss / (float)D + eps);
    out[(size_t)t * ldout + hb + tid] = (T)(o * inv * norm[hb + tid] * (float)gate[(size_t)t * ldg + hb + tid]);
  }
  for (int i = blockIdx.x * 256 + tid; i < p.width; i += gridDim.x * 256)
    p.prev[(size_t)slot * p.ldp + i] = p.x[(size_t)t * p.ldx + i];
}

// ---- out = (o / rms(o) per head) * norm * gate
template <typename T>
__global__ __launch_bounds__(256) void wkv_out_kernel(const float* __restrict__ o, long ldo,
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

template <typename T, int DP>
int scan_d(const Scan& p, int nruns, hipStream_t st) {
  auto grid = [&](int wc) { return dim3(p.H * ((p.D + wc - 1) / wc), nruns); };
  if (DP < 64 || p.H * nruns * ((p.D + 31) / 32) >= 256)
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
  Scan p{r, k, v, w, u, o, state, x, prev, runs, ld, ldw, ldo, sstride, ldx, ldp, H, D, width};
  return f32 ? scan_t<float>(p, nruns, (hipStream_t)stream) : scan_t<__bf16>(p, nruns, (hipStream_t)stream);
}

// every run has one token (or none); D a multiple of 4
int nls_wkv_step(const void* r, const void* k, const void* v, long ld, const float* w, long ldw, const float* u,
                 float* state, long sstride, const float* x, long ldx, float* prev, long ldp, int width, const int* runs,
                 int nruns, const float* norm, const void* gate, long ldg, void* out, long ldout, int H, int D, float eps,
                 int f32, void* stream) {
  if (nruns < 1 || H < 1 || D < 4 || D > 256 || (D & 3) || (sstride & 3)) return -1;
  Scan p{r, k, v, w, u, nullptr, state, x, prev, runs, ld, ldw, 0, sstride, ldx, ldp, H, D, width};
  const dim3 grid(H, nruns);
  if (f32)
    hipLaunchKernelGGL(wkv_step_kernel<float>, grid, dim3(256), 0, (hipStream_t)stream, p, norm, (const float*)gate, ldg,
                       (float*)out, ldout, eps);
  else
    hipLaunchKernelGGL(wkv_step_kernel<__bf16>, grid, dim3(256), 0, (hipStream_t)stream, p, norm, (const __bf16*)gate, ldg,
                       (__bf16*)out, ldout, eps);
  return (int)hipGetLastError();
}

int nls_wkv_out(const float* o, long ldo, const float* norm, const void* gate, long ldg, void* out, long ld, int H,
                int D, int T, float eps, int f32, void* stream) {
  if (T < 1 || H < 1 || D < 1) return -1;
  const int gy = T >= 256 ? 1 : min((H + 3) / 4, 64);
  const dim3 grid(T, gy);
  if (f32)
    hipLaunchKernelGGL(wkv_out_kernel<float>, grid, dim3(256), 0, (hipStream_t)stream, o, ldo, norm,
                       (const float*)gate, ldg, (float*)out, ld, H, D, eps);
  else
    hipLaunchKernelGGL(wkv_out_kernel<__bf16>, grid, dim3(256), 0, (hipStream_t)stream, o, ldo, norm,
                       (const __bf16*)gate, ldg, (__bf16*)out, ld, H, D, eps);
  return (int)hipGetLastError();
}

}  // extern "C"
