// Gated linear recurrences with a per-channel decay (gfx950): the scan over runs of tokens, the step of single tokens and the
// per-head output norm, shared by "wkv" time mixing (wkv.hip) and gated linear attention (gla.hip).
//
// Per head, with keys i and values j (state S [D][V], f32):
//   wkv: o_t[j] = sum_i r_t[i] (S[i][j] + u[i] k_t[i] v_t[j]);   S[i][j] = w_t[i] S[i][j] + k_t[i] v_t[j]
//   gla: S[i][j] = w_t[i] S[i][j] + k_t[i] v_t[j];               o_t[j] = rs sum_i r_t[i] S[i][j]
//
// The scan is sequential in the tokens of a run (or of a segment of it, below), so that a position's result does not depend
// on how its sequence was cut into steps. Parallelism is (run, head, value columns) x lanes: a lane holds DP / PARTS key rows
// of CPL value columns in registers, PARTS neighbouring lanes cover the keys and close the sum with in-row lane exchanges
// (DPP). Few runs take many key parts (short per-token chains on all CUs). Tokens are staged in LDS in chunks of CH as f32,
// the next chunk's loads in flight while the current one runs.
// Segments (gla): a long run is cut into `nseg` segments that run in parallel, in two launches. The first runs segment 0 in
// full and, from a zero state, the end state and the product of decays of every further segment but the last; the second
// starts each of those and the last from end states chained over the segments before it. Only products with decays in
// [0, 1] appear, so nothing over- or underflows that would not in the plain recurrence.
// A step of single tokens (decode) streams each head's state once with 16-byte accesses and ends with the head's norm and
// gate (step_kernel).
//
// A run = (first row, tokens, state slot, first position): consecutive rows of one sequence. A run at position 0
// starts from a zero state, any other from its slot; slot < 0 or 0 tokens: nothing to do (padded decode rows).
#pragma once
#include "../kernels/common.h"

namespace nls_scan {

enum Kind : int { WKV = 0, GLA = 1 };
constexpr int MINSEG = 64;     // fewest tokens of a segment

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
  float* seg_s;            // segments: end states [run][nseg - 1][H][D][V] and decay products [run][nseg - 1][H][D]
  float* seg_w;
  long ld, ldw, ldo, sstride, ldx, ldp;
  int H, D, V, width;
  int nseg, pass;          // pass 0: the only or first launch, 1: the second
  float rs;                // gla: factor of the output
};

// DP: key channels padded to a multiple of 32 (zeros past D)
template <typename T, int KIND, int DP, int PARTS, int CPL>
__global__ __launch_bounds__(256) void scan_kernel(Scan p) {
  constexpr int WC = 256 / PARTS * CPL;          // value columns per workgroup
  constexpr int CH = DP <= 64 ? 32 : (DP <= 128 ? 16 : 8);   // tokens per staged chunk
  constexpr int R = DP / PARTS;                  // state rows per lane
  constexpr int LR = DP + 4;                     // LDS row stride
  constexpr int NV = (CH * DP + 255) / 256;      // staged values per thread and operand
  __shared__ __attribute__((aligned(16))) float rs[CH][LR], ks[CH][LR], ws[CH][LR];
  __shared__ __attribute__((aligned(16))) float vs[CH][WC], ruk[KIND == WKV ? CH : 1];
  const int* run = p.runs + 4 * blockIdx.y;
  int t0 = run[0], n = run[1];
  const int slot = run[2], pos0 = run[3];
  if (slot < 0 || n < 1) return;
  const int D = p.D, V = p.V;
  // the segment of this workgroup: rows t0 .. t0 + n - 1
  const int z = KIND == GLA ? (int)blockIdx.z + p.pass : 0;
  bool last = true;
  if (KIND == GLA && p.nseg > 1) {
    const int sl = max(MINSEG, ((n + p.nseg - 1) / p.nseg + 31) & ~31);
    if (z * sl >= n) return;
    last = (z + 1) * sl >= n;
    if (p.pass == 0 && z > 0 && last) return;
    t0 += z * sl;
    n = min(sl, n - z * sl);
  }
  const bool local = KIND == GLA && p.pass == 0 && z > 0;       // end state from zero, no outputs
  const int ncb = (V + WC - 1) / WC;
  const int head = blockIdx.x / ncb, c0 = (blockIdx.x % ncb) * WC;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int part = lane & (PARTS - 1), col = (wave * (64 / PARTS) + lane / PARTS) * CPL;
  const int j = c0 + col;
  const size_t hb = (size_t)head * D, hv = (size_t)head * V;
  const T* rp = (const T*)p.r + hb;
  const T* kp = (const T*)p.k + hb;
  const T* vp = (const T*)p.v + hv;
  const float* wp = p.w + hb;
  float* st = p.state + (size_t)slot * p.sstride + hb * V;
  const size_t sst = (size_t)p.H * D * V, swt = (size_t)p.H * D;                        // segment records
  float* sgs = p.seg_s + (size_t)blockIdx.y * (p.nseg - 1) * sst + hb * V;
  float* sgw = p.seg_w + (size_t)blockIdx.y * (p.nseg - 1) * swt + hb;

  float S[CPL][R], pw[KIND == GLA ? R : 1];
#pragma unroll
  for (int i = 0; i < R; ++i)
#pragma unroll
    for (int c = 0; c < CPL; ++c) {
      const int row = part * R + i;
      const bool in = row < D && j + c < V;
      if (KIND == GLA && z > 0) {
        float s = 0.f;
        if (!local && in) {
          s = sgs[(size_t)row * V + j + c];
          for (int q = 1; q < z; ++q) s = fmaf(sgw[q * swt + row], s, sgs[q * sst + (size_t)row * V + j + c]);
        }
        S[c][i] = s;
      } else {
        S[c][i] = pos0 > 0 && in ? st[(size_t)row * V + j + c] : 0.f;
      }
    }
#pragma unroll
  for (int i = 0; i < (KIND == GLA ? R : 1); ++i) pw[i] = 1.f;
  float ur[KIND == WKV ? DP / 16 : 1];           // u of the bonus sums' columns
  if constexpr (KIND == WKV)
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
      const bool in = tt < CH && base + tt < n && i < V;
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
    // wkv: sum_i r u k of every staged token, 16 lanes each
#pragma unroll
    for (int t8 = 0; KIND == WKV && t8 < CH; t8 += 16) {
      const int tt = t8 + (threadIdx.x >> 4), l = threadIdx.x & 15;
      float a = 0.f;
      if (tt < CH)
#pragma unroll
        for (int q = 0; q < DP / 16; ++q) a += rs[tt][l + 16 * q] * ur[q] * ks[tt][l + 16 * q];
#pragma unroll
      for (int s = 8; s > 0; s >>= 1) a += __shfl_xor(a, s, 64);
      if (tt < CH && l == 0) ruk[tt] = a;
    }
    if (KIND == WKV) __syncthreads();
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
      if constexpr (KIND == GLA) {
#pragma unroll
        for (int c = 0; c < CPL; ++c) {
          float o0 = 0.f, o1 = 0.f;
#pragma unroll
          for (int i4 = 0; i4 < R / 4; ++i4)
#pragma unroll
            for (int e = 0; e < 4; e += 2) {
              const int i = 4 * i4 + e;
              S[c][i] = fmaf(w4[b][i4][e], S[c][i], k4[b][i4][e] * v1[b][c]);
              S[c][i + 1] = fmaf(w4[b][i4][e + 1], S[c][i + 1], k4[b][i4][e + 1] * v1[b][c]);
              o0 = fmaf(r4[b][i4][e], S[c][i], o0);
              o1 = fmaf(r4[b][i4][e + 1], S[c][i + 1], o1);
            }
          o[c] = sum_parts<PARTS>(o0 + o1);
        }
        return;
      }
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
    if (local) {
      // state and decay products only
      for (int tt = 0; tt < m; ++tt) {
        get(tt, 0);
#pragma unroll
        for (int i = 0; i < R; ++i) {
          if constexpr (KIND == GLA) pw[i] *= w4[0][i >> 2][i & 3];
#pragma unroll
          for (int c = 0; c < CPL; ++c) S[c][i] = fmaf(w4[0][i >> 2][i & 3], S[c][i], k4[0][i >> 2][i & 3] * v1[0][c]);
        }
      }
      continue;
    }
    get(0, 0);
    for (int t8 = 0; t8 < m; t8 += 8) {
      float mine[CPL], o[CPL];
#pragma unroll
      for (int c = 0; c < CPL; ++c) mine[c] = 0.f;
      const int last = m - 1 - t8, tt = t8 + (part & 7);
      const float rk = KIND == WKV ? ruk[tt] : 0.f;
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
          if (j + c < V)
            p.o[(size_t)(t0 + base + tt) * p.ldo + hv + j + c] =
                KIND == WKV ? fmaf(rk, vs[tt][col + c], mine[c]) : p.rs * mine[c];
    }
  }
  float* dst = last ? st : sgs + z * sst;
#pragma unroll
  for (int i = 0; i < R; ++i)
#pragma unroll
    for (int c = 0; c < CPL; ++c) {
      const int row = part * R + i;
      // (the second launch leaves the records of its segments as they are: others read them)
      if (row < D && j + c < V && (last || p.pass == 0)) dst[(size_t)row * V + j + c] = S[c][i];
    }
  if constexpr (KIND == GLA) {
    if (local && j == 0)
#pragma unroll
      for (int i = 0; i < R; ++i)
        if (part * R + i < D) sgw[z * swt + part * R + i] = pw[i];
  }
  if (KIND != WKV || !p.prev) return;
  // the run's last row is the next step's previous token (this layer's shift_mix, which reads it, came before)
  const int G = gridDim.x;
  for (int i = blockIdx.x * 256 + threadIdx.x; i < p.width; i += G * 256)
    p.prev[(size_t)slot * p.ldp + i] = p.x[(size_t)(t0 + n - 1) * p.ldx + i];
}

// ---- one token per run: the state of (run, head) is read and written once, 4 value columns per thread; then
// out = (o / rms(o)) * norm * gate. V is a multiple of 4, at most 1024; D at most 256.
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
    ws[tid] = p.w[(size_t)t * p.ldw + hb + tid];
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
    }
  }
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
