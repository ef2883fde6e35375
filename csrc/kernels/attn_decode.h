// Decode attention over a paged bf16 / fp8 K/V cache on MFMA (gfx950), shared by the GGUF families (attention.hip) and the
// config-driven stacks (csrc/stack/attn.hip).
#pragma once
#include "common.h"

namespace nls_attn {

constexpr float LOG2E = 1.4426950408889634f;

// Keys per flash-decoding split. chunk > 0: fixed; chunk < 0: balanced over n_split with at least
// -chunk keys; chunk == 0: balanced with at least 64 keys below 1K of context, 128 at 1K-2K and 256 above
// (batch-1 A/B, profiles/attn_split_policy_b1.txt: 64-key splits win on short contexts, where the split's
// dependent K/V fetch chain dominates; 128-256-key splits at 1K-4K, where the merge of many partials does).
// With up to 64 splits at batch 1 (models/llama.py _SPLIT_CAP), 8K-32K contexts get 32-64 splits of
// 256-512 keys: 512 workgroups keep enough K/V in flight to stream the cache at HBM rate.
__device__ __forceinline__ int split_chunk(int chunk, int ctx, int n_split, int bs, int short_min = 64) {
  if (chunk > 0) return chunk;
  const int mn = chunk ? -chunk : (ctx >= 2048 ? 256 : (ctx >= 1024 ? 128 : short_min));
  return max(mn, ((ctx + n_split - 1) / n_split + bs - 1) / bs * bs);
}

// ---------------------------------------------------------------------------------------------------
// Decode attention on MFMA (large grids: batch x kv heads >= 1K workgroups). The VALU kernel of attention.hip
// spends ~170 vector instructions per 4 keys of a wave (dot products, cross-lane sums, the online
// softmax and 32 FMAs of P.V per lane): at batch 512 it runs at ~3.5 TB/s of K/V, bound by issue, not
// HBM (tools/attn_layout_probe.py: time linear in the context at every length). Here the G query heads
// of a kv head are the 16 COLUMNS of the MFMA tiles (G <= 16, the rest zero), so per 32 keys a wave
// issues 16 v_mfma_f32_16x16x32_bf16 and softmaxes 8 values per lane:
//   S^T = K Q^T   A = K rows straight from HBM into registers (lane (g, r): key r, dims 8g..8g+7 of
//                 each 32-dim k-step), B = Q^T (lane column r = head r, loaded once)
//   O^T += V^T P^T  A = V^T through LDS: the 32-key V tile is stored row-major with a 16-byte chunk XOR
//                 swizzle and read back transposed by ds_read_b64_tr_b16;
//                 B = P^T straight from the S^T accumulators (lane (g, r) holds keys 4g..4g+3 of each
//                 16-key n-tile for head r: the MFMA's k order is free, so V^T's transposed reads take
//                 rows {4g..4g+3} and {16+4g..16+4g+3} to match)
// The O^T accumulators keep head r in lane column r -- exactly where the softmax state of head r lives,
// so the rescale needs no cross-lane traffic. One wave per workgroup; the next 32 keys' K/V loads are
// in flight while the current ones are computed. Splits and the fused combine as the VALU kernel.
typedef short s16x4 __attribute__((ext_vector_type(4)));

// Merge of the na (<= 64) flash-decoding partials of (token t, kv head kh), run by the last split to
// finish, with every thread busy and no per-split round trip in series: one wave per head reduces the
// splits' (m, l) across its lanes into per-split weights f_s = 2^(m_s - M) / L (LDS), then each thread
// sums f_s * O_s for 4 dims of a head over a share of the splits (16-byte loads, all independent) and
// the shares are added through LDS. smem: >= 16 * 64 + 64 * WAVES * 4 floats.
template <int WAVES, int D, typename OUT>
DEVI void merge_splits(const float* __restrict__ part_o, const float* __restrict__ part_ml, int t, int h0, int G,
                       int Hq, int n_split, int na, OUT* __restrict__ out, long ldo, const float* __restrict__ gate, long ldg,
                       float* smem) {
  constexpr int NT = 64 * WAVES;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  float* f = smem;                                   // [16 heads][64 splits]
  f32x4* red = reinterpret_cast<f32x4*>(smem + 16 * 64);   // [NT] partial sums
  for (int h = wave; h < G; h += WAVES) {
    const size_t pb = ((size_t)t * Hq + h0 + h) * n_split;
    const float ms = lane < na ? part_ml[2 * (pb + lane)] : -INFINITY;
    const float ls = lane < na ? part_ml[2 * (pb + lane) + 1] : 0.f;
    float M = ms;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) M = fmaxf(M, __shfl_xor(M, o, 64));
    const float w = ms == -INFINITY ? 0.f : exp2f(ms - M);
    float L = w * ls;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) L += __shfl_xor(L, o, 64);
    f[h * 64 + lane] = L > 0.f ? w / L : 0.f;
  }
  __syncthreads();
  const int items = G * (D / 4);                     // (head, 4 dims)
  const int parts = items >= NT ? 1 : NT / items;    // split shares per item
  for (int i0 = 0; i0 < items; i0 += NT) {
    const int it = i0 + threadIdx.x % min(items, NT), pt = threadIdx.x / min(items, NT);
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    if (it < items && pt < parts) {
      const int h = it / (D / 4), d4 = it % (D / 4);
      const size_t pb = ((size_t)t * Hq + h0 + h) * n_split;
      const float* fw = f + h * 64;
#pragma unroll 4
      for (int s2 = pt; s2 < na; s2 += parts)
        acc += fw[s2] * *reinterpret_cast<const f32x4*>(part_o + (pb + s2) * D + 4 * d4);
    }
    red[threadIdx.x] = acc;
    __syncthreads();
    if (pt == 0 && it < items) {
      for (int p2 = 1; p2 < parts; ++p2) acc += red[threadIdx.x + p2 * min(items, NT)];
      const int h = it / (D / 4), d4 = it % (D / 4);
      typedef OUT o4 __attribute__((ext_vector_type(4)));
      if (gate) acc *= gate[(size_t)t * ldg + h0 + h];
      *reinterpret_cast<o4*>(out + (size_t)t * ldo + (size_t)(h0 + h) * D + 4 * d4) =
          o4{(OUT)acc[0], (OUT)acc[1], (OUT)acc[2], (OUT)acc[3]};
    }
    __syncthreads();
  }
}


// D: head dimension, 128 (Llama / Mistral / Qwen2), 64 (Granite-3.0), 32 or 256 (at most 2 waves): V rows of 2D bytes (D / 8
// 16-byte chunks, XOR swizzled within the row), D / 8 lanes per V row on the loads.
// Groups of more than 16 query heads take ceil(G / 16) workgroups (blockIdx.y = kv head * blocks + block of 16 heads).
// gate (optional): [rows][ldg], one factor per token and query head on the output.
// AttnMask: sink: the softmax's denominator holds one more, a score of 0 without a value (the state that the first wave of the
// first split starts from). WIN: keys j < keep or j >= ctx - window only. The kernel then walks an index over the visible
// keys (those of the kept ones' last group of 32 that are not kept are masked): the first `keep`, rounded up to a group, then
// `gap` positions further on; splits and groups start at multiples of 32, so no group spans the gap.
struct AttnMask {
  int window = 0, keep = 0, sink = 0;
};

template <typename KV, int WAVES, int D, typename OUT = act_t, bool WIN = false>
__global__ __launch_bounds__(64 * WAVES) void attn_decode_mfma_kernel(
    const __bf16* __restrict__ q, long ldq, const KV* __restrict__ kc, const KV* __restrict__ vc,
    const int* __restrict__ block_tables, int bt_stride, const int* __restrict__ tok_seq,
    const int* __restrict__ ctx_len, int Hkv, int Gq, int bs, float scale, int chunk, int n_split,
    OUT* __restrict__ out, long ldo, float* __restrict__ part_o, float* __restrict__ part_ml,
    int* __restrict__ cnt, const float* __restrict__ gate, long ldg, AttnMask mask) {
  static_assert(D == 32 || D == 64 || D == 128 || (D == 256 && WAVES <= 2), "head dimension");
  constexpr int NKK = D / 32, NDT = D / 16, KG = 32;
  constexpr int NCH = D / 8, LPR = NCH, RPI = 64 / LPR, NVL = KG / RPI;   // V: chunks per row, lanes per row,
                                                                          // rows per load, loads per 32 keys
  typedef KVRaw<KV> R;
  // per wave: one 32-key V tile (8 KiB; a wave's LDS ops run in order, so the next group's V is written
  // after this group's transposed reads without a second buffer); the space is reused for the cross-wave
  // merge and the split merge at the end
  constexpr int VB = WAVES * KG * D * 2, MB = WAVES > 1 ? (2 * WAVES * 16 + WAVES * 16 * D) * 4 : 0,
                CB = (16 * 64 + 64 * WAVES * 4) * 4;
  constexpr int SMEM = VB > MB ? (VB > CB ? VB : CB) : (MB > CB ? MB : CB);
  __shared__ __attribute__((aligned(16))) uint8_t Vsm[SMEM];
  const int t = blockIdx.x, split = blockIdx.z;
  const int nhb = (Gq + 15) >> 4, kh = nhb == 1 ? (int)blockIdx.y : (int)blockIdx.y / nhb;
  const int hofs = nhb == 1 ? 0 : ((int)blockIdx.y - kh * nhb) * 16;
  const int G = min(Gq - hofs, 16), h0 = kh * Gq + hofs;       // this workgroup's query heads: h0 .. h0 + G - 1
  const int lane = threadIdx.x & 63, g = lane >> 4, r = lane & 15;
  const int wave = WAVES == 1 ? 0 : __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  uint8_t* Vs = Vsm + wave * KG * D * 2;
  const int Hq = Hkv * Gq;
  const int last_pos = ctx_len[t], kept = WIN ? (mask.keep + KG - 1) & ~(KG - 1) : 0;
  const int gap = WIN ? max(0, last_pos - mask.window - kept) : 0;
  const int ctx = last_pos - gap;
  // short contexts: at least one 32-key group per wave of the workgroup per split (>= 64 keys)
  chunk = split_chunk(chunk, ctx, n_split, bs, KG * WAVES > 64 ? KG * WAVES : 64);
  if (WIN) chunk = (chunk + KG - 1) & ~(KG - 1);
  const int start = split * chunk;
  if (n_split > 1 && start >= ctx && ctx > 0) return;       // inactive split: combine skips it
  const int end = min(ctx, start + chunk);
  // active splits: with ONE (short context) the split writes the output itself -- no partials, no ticket
  const int na = ctx > 0 ? min(n_split, (ctx + chunk - 1) / chunk) : n_split;
  const bool direct = n_split == 1 || (na == 1 && cnt);
  const int* bt = block_tables + (size_t)tok_seq[t] * bt_stride;
  const float sl2 = scale * LOG2E;

  bf16x8 qf[NKK];
#pragma unroll
  for (int kk = 0; kk < NKK; ++kk) {
    qf[kk] = bf16x8{};
    if (r < G) qf[kk] = *reinterpret_cast<const bf16x8*>(q + (size_t)t * ldq + (size_t)(h0 + r) * D + kk * 32 + 8 * g);
  }
  f32x4 o[NDT];
#pragma unroll
  for (int c = 0; c < NDT; ++c) o[c] = f32x4{0.f, 0.f, 0.f, 0.f};
  const bool sink = mask.sink && split == 0 && wave == 0;
  float m = sink ? 0.f : -INFINITY, l = sink ? 1.f : 0.f;

  // Block-table entries come from a register window (lane i holds entry b0 + 64 * win + i, refreshed once
  // per 64 blocks), broadcast per 32-key group as wave-uniform values: the K/V loads of a group no
  // longer wait on a dependent block-table fetch (the chain that bound long contexts at small batch).
  // A group [base, base + 32) touches blocks base / bs .. (base + 31) / bs: at most NGB of them.
  constexpr int NGB = 4;                       // bs >= 16 (host-checked): <= 3 blocks per group
  const int b0 = start / bs;
  int btw = -1, btreg = 0;
  int gblk[NGB] = {0, 0, 0, 0};
  auto shift = [&](int base) { return WIN && base >= kept ? gap : 0; };  // position of a group's keys, less their index
  auto group_blocks = [&](int base0) __attribute__((always_inline)) {
    const int sh = shift(base0), base = base0 + sh, end_p = end + sh;
    const int bi0 = base / bs - b0;
    const int nbg = (min(base + KG, end_p) - 1) / bs - base / bs + 1;     // blocks this group touches
    const int win = bi0 >> 6;
    if (win != btw) {
      btw = win;
      const int e = b0 + win * 64 + lane;
      btreg = e * bs < (WIN ? last_pos : end) ? bt[e] : 0;        // (WIN: the window may reach across the gap)
    }
#pragma unroll
    for (int i = 0; i < NGB; ++i) {
      const int bi = bi0 + i;
      // (a block past the register window: one wave-uniform direct read)
      if (i < nbg) gblk[i] = (bi >> 6) == win ? __builtin_amdgcn_readlane(btreg, bi & 63) : bt[b0 + bi];
    }
  };
  auto kv_row = [&](int p, int base0) -> size_t {      // element offset of key p's row for this kv head
    const int base = base0 + shift(base0), pc = min(p, end - 1) - base0 + base;
    const int lb = pc / bs - base / bs;                // 0 .. NGB - 1
    const int blk = lb == 0 ? gblk[0] : (lb == 1 ? gblk[1] : (lb == 2 ? gblk[2] : gblk[3]));
    return ((size_t)((long)blk * bs + pc % bs) * Hkv + kh) * D;
  };
  // swizzled byte offset of 16-byte chunk ch of V row `row` (2D-byte rows): D = 128 conflict-free for the
  // transposed reads and the row writes; else the chunk ^ the row's low bits
  auto voff = [](int row, int ch) {
    if constexpr (D == 128) return row * 256 + 16 * (ch ^ (((row & 3) << 2) | ((row >> 2) & 3)));
    else return row * (2 * D) + 16 * (ch ^ (row & (NCH - 1)));
  };
  // K of 32 keys: [n-tile][k-step]; V of 32 keys: NVL rows per lane (row = RPI i + lane / LPR, chunk lane % LPR)
  typename R::raw kr[2][NKK], vr[NVL];
  auto load = [&](int base, typename R::raw (&K)[2][NKK], typename R::raw (&V)[NVL]) __attribute__((always_inline)) {
    group_blocks(base);
#pragma unroll
    for (int nt = 0; nt < 2; ++nt) {
      const size_t o0 = kv_row(base + 16 * nt + r, base);
#pragma unroll
      for (int kk = 0; kk < NKK; ++kk) K[nt][kk] = R::ld(kc + o0 + kk * 32 + 8 * g);
    }
#pragma unroll
    for (int i = 0; i < NVL; ++i) V[i] = R::ld(vc + kv_row(base + RPI * i + lane / LPR, base) + 8 * (lane % LPR));
  };
  auto store_v = [&](int buf, typename R::raw (&V)[NVL]) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < NVL; ++i)
      *reinterpret_cast<u32x4*>(Vs + voff(RPI * i + lane / LPR, lane % LPR)) = R::bf16(V[i]);
  };
  // wave w takes the 32-key groups w, w + WAVES, ... of the workgroup's range
  const int ngrp_all = end > start ? (end - start + KG - 1) / KG : 0;
  const int ngrp = ngrp_all > wave ? (ngrp_all - wave + WAVES - 1) / WAVES : 0;
  if (ngrp > 0) {
    load(start + wave * KG, kr, vr);
    store_v(0, vr);
  }
  for (int j = 0; j < ngrp; ++j) {
    const int base = start + (j * WAVES + wave) * KG;
    typename R::raw kn[2][NKK], vn[NVL];
    const bool more = j + 1 < ngrp;
    if (more) load(base + WAVES * KG, kn, vn);
    // ---- S^T = K Q^T: s[nt][i] = S[head r][key base + 16 nt + 4 g + i]
    f32x4 s[2];
#pragma unroll
    for (int nt = 0; nt < 2; ++nt) {
      s[nt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < NKK; ++kk)
        s[nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, R::bf16(kr[nt][kk])), qf[kk],
                                                        s[nt], 0, 0, 0);
    }
    // ---- online softmax of head r (base 2), keys past `end` masked
    float mx = -INFINITY;
#pragma unroll
    for (int nt = 0; nt < 2; ++nt)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int ki = base + 16 * nt + 4 * g + i, kp = ki + shift(base);
        const bool see = ki < end && (!WIN || kp < mask.keep || kp >= last_pos - mask.window);
        const float v = see ? s[nt][i] * sl2 : -INFINITY;
        s[nt][i] = v;
        mx = fmaxf(mx, v);
      }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float mn = fmaxf(m, mx);
    const float alpha = m == -INFINITY ? 0.f : exp2f(m - mn);
    float ps = 0.f;
    bf16x8 pb;
#pragma unroll
    for (int nt = 0; nt < 2; ++nt)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float pv = s[nt][i] == -INFINITY ? 0.f : exp2f(s[nt][i] - mn);
        ps += pv;
        pb[4 * nt + i] = (__bf16)pv;
      }
    ps += __shfl_xor(ps, 16, 64);
    ps += __shfl_xor(ps, 32, 64);
    l = l * alpha + ps;
    m = mn;
    // ---- O^T = O^T * alpha + V^T P^T over the 32 keys; V^T fragment of dim tile c: transposed reads of
    // rows {4g+q} and {16+4g+q}, columns 16c + 4p .. +3 (lane 4q + p of the group supplies the address)
    const uint8_t* vb = Vs;
    const int qq = r >> 2, pp = r & 3;
#pragma unroll
    for (int c = 0; c < NDT; ++c) {
      const int ch = 2 * c + (pp >> 1);
      const s16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
          (__attribute__((address_space(3))) s16x4*)(vb + voff(4 * g + qq, ch) + 8 * (pp & 1)));
      const s16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
          (__attribute__((address_space(3))) s16x4*)(vb + voff(16 + 4 * g + qq, ch) + 8 * (pp & 1)));
      typedef short s16x8 __attribute__((ext_vector_type(8)));
      const s16x8 a8 = __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7);
      o[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a8), pb, o[c] * alpha, 0, 0, 0);
    }
    if (more) {
      store_v((j + 1) & 1, vn);
#pragma unroll
      for (int nt = 0; nt < 2; ++nt)
#pragma unroll
        for (int kk = 0; kk < NKK; ++kk) kr[nt][kk] = kn[nt][kk];
    }
  }

  // ---- output. WAVES > 1: merge the waves' partial (m, l, O) of each head through LDS (the V tiles'
  // space), every thread finishing (head, dim) elements; WAVES == 1: lane (g, r) holds dims 16c + 4g + i of
  // head r in registers
  if constexpr (WAVES > 1) {
    float* mb = reinterpret_cast<float*>(Vsm);                      // [WAVES][16] m, [WAVES][16] l
    float* ob = mb + 2 * WAVES * 16;                                  // [WAVES][16 heads][D]
    __syncthreads();                                                  // every wave is done with its V tiles
    if (g == 0) {
      mb[wave * 16 + r] = m;
      mb[(WAVES + wave) * 16 + r] = l;
    }
#pragma unroll
    for (int c = 0; c < NDT; ++c)
      *reinterpret_cast<f32x4*>(ob + ((size_t)wave * 16 + r) * D + 16 * c + 4 * g) = o[c];
    __syncthreads();
    for (int e = threadIdx.x; e < G * D; e += 64 * WAVES) {
      const int h = e / D, d = e - h * D;
      float M = -INFINITY;
#pragma unroll
      for (int w = 0; w < WAVES; ++w) M = fmaxf(M, mb[w * 16 + h]);
      float L = 0.f, O = 0.f;
#pragma unroll
      for (int w = 0; w < WAVES; ++w) {
        const float mw = mb[w * 16 + h];
        const float f = mw == -INFINITY ? 0.f : exp2f(mw - M);
        L += mb[(WAVES + w) * 16 + h] * f;
        O += ob[((size_t)w * 16 + h) * D + d] * f;
      }
      const int qh2 = h0 + h;
      if (direct) {
        float v = L > 0.f ? O / L : 0.f;
        if (gate) v *= gate[(size_t)t * ldg + qh2];
        out[(size_t)t * ldo + (size_t)qh2 * D + d] = (OUT)v;
      } else {
        const size_t pi = ((size_t)t * Hq + qh2) * n_split + split;
        part_o[pi * D + d] = O;
        if (d == 0) {
          part_ml[2 * pi] = M;
          part_ml[2 * pi + 1] = L;
        }
      }
    }
    if (direct) return;
  } else {
    const int qh = h0 + r;
    if (direct) {
      if (r < G) {
        float inv = l > 0.f ? 1.f / l : 0.f;
        if (gate) inv *= gate[(size_t)t * ldg + qh];
#pragma unroll
        for (int c = 0; c < NDT; ++c) {
          typedef OUT o4 __attribute__((ext_vector_type(4)));
          *reinterpret_cast<o4*>(out + (size_t)t * ldo + (size_t)qh * D + 16 * c + 4 * g) =
              o4{(OUT)(o[c][0] * inv), (OUT)(o[c][1] * inv), (OUT)(o[c][2] * inv), (OUT)(o[c][3] * inv)};
        }
      }
      return;
    }
    if (r < G) {
      const size_t pi = ((size_t)t * Hq + qh) * n_split + split;
#pragma unroll
      for (int c = 0; c < NDT; ++c) *reinterpret_cast<f32x4*>(part_o + pi * D + 16 * c + 4 * g) = o[c];
      if (g == 0) {
        part_ml[2 * pi] = m;
        part_ml[2 * pi + 1] = l;
      }
    }
  }
  if (!cnt) return;
  // fused combine: the last active split of (token, kv head) to arrive merges them (as the VALU kernel)
  __shared__ int last;
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  __syncthreads();
  if (threadIdx.x == 0) {
    int* cp = cnt + (size_t)t * gridDim.y + blockIdx.y;
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "agent");
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    const int old = __hip_atomic_fetch_add(cp, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    last = old == na - 1;
    if (last) {
      __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "agent");
      __hip_atomic_store(cp, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
      asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    }
  }
  __syncthreads();
  if (!last) return;
  merge_splits<WAVES, D>(part_o, part_ml, t, h0, G, Hq, n_split, na, out, ldo, gate, ldg,
                         reinterpret_cast<float*>(Vsm));
}

}  // namespace nls_attn
