// Grouped-query attention of the config-driven stacks over paged keys and values, one row at a time (decoded tokens, short
// runs): the MFMA decode kernel of the GGUF families (kernels/attn_decode.h) with bf16 outputs and the output gate in its
// epilogue, or (32-bit models, other head widths) the plain kernel. Prompts: prefill_attn.hip.
#include "../kernels/attn_decode.h"
#include "attn_plain.h"

namespace nls_gqa {
using namespace nls_attn;

struct GA {
  const void *q, *k, *v;
  void* out;
  const float* gate;
  float *part_o, *part_ml;
  int* cnt;
  const int *bt, *tok_seq, *ctx_len;
  long ldq, ldo, ldg;
  int bts, bs, T, H, G, ns;
  float scale;
  AttnMask mask;
};

template <int W, int D, bool WIN>
int decode_w(const GA& a, hipStream_t st) {
  const int gq = a.H / a.G;
  hipLaunchKernelGGL((attn_decode_mfma_kernel<__bf16, W, D, __bf16, WIN>), dim3(a.T, a.G * ((gq + 15) / 16), a.ns), dim3(64 * W), 0,
                     st, (const __bf16*)a.q, a.ldq, (const __bf16*)a.k, (const __bf16*)a.v, a.bt, a.bts, a.tok_seq, a.ctx_len,
                     a.G, gq, a.bs, a.scale, 0, a.ns, (__bf16*)a.out, a.ldo, a.part_o, a.part_ml, a.cnt, a.gate, a.ldg, a.mask);
  return (int)hipGetLastError();
}

template <int W, int D>
int decode_t(const GA& a, hipStream_t st) {
  return a.mask.window > 0 ? decode_w<W, D, true>(a, st) : decode_w<W, D, false>(a, st);
}

// waves per workgroup: one once the grid fills the chip, eight on grids of at most a workgroup per CU
template <int D>
int decode_d(const GA& a, hipStream_t st) {
  const long n = (long)a.T * a.G * ((a.H / a.G + 15) / 16) * a.ns;
  if (n >= 1024) return decode_t<1, D>(a, st);
  if constexpr (D == 256) return decode_t<2, D>(a, st);
  else return n > 256 ? decode_t<4, D>(a, st) : decode_t<8, D>(a, st);
}

}  // namespace nls_gqa

extern "C" {

// q, out: [T][ld], heads Dp columns apart; k, v: paged [slots][G][Dp]; padding columns are zero. ns > 1: part_o [T][H][ns][Dp],
// part_ml [T][H][ns][2], cnt [T][workgroups per token] zeros (left zero). gate: optional. window > 0: a token at position i sees
// j <= i if i - j < window or j < keep. sink: one more in the denominator, a score of 0 without a value.
int nls_gqa_attn(const void* q, long ldq, const void* k, const void* v, const int* bt, int bts, int bs, const int* tok_seq,
                 const int* ctx_len, int T, int H, int G, int Dp, int ns, float scale, const float* gate, long ldg, void* out,
                 long ldo, float* part_o, float* part_ml, int* cnt, int window, int keep, int sink, int plain, int f32,
                 void* stream) {
  using namespace nls_gqa;
  if (T < 1 || G < 1 || H < 1 || H % G || Dp < 1 || bs < 1 || ns < 1 || ns > 64 || window < 0 || keep < 0 ||
      (ns > 1 && (!part_o || !part_ml || !cnt)))
    return -1;
  hipStream_t st = (hipStream_t)stream;
  if (plain || f32) {
    const nls_plain::PA a{q, k, v, out, bt, tok_seq, ctx_len, gate, ldq, Dp, (long)G * Dp, Dp, ldo, Dp, ldg, bts, bs, H / G, Dp, Dp,
                          scale, window, keep, sink};
    return f32 ? nls_plain::launch<float>(a, T, H, st) : nls_plain::launch<__bf16>(a, T, H, st);
  }
  if (bs < 16 || (ldq & 7) || (ldo & 3)) return -1;
  const GA a{q, k, v, out, gate, part_o, part_ml, cnt, bt, tok_seq, ctx_len, ldq, ldo, ldg, bts, bs, T, H, G, ns, scale,
             {window, keep, sink}};
  switch (Dp) {
    case 32: return decode_d<32>(a, st);
    case 64: return decode_d<64>(a, st);
    case 128: return decode_d<128>(a, st);
    case 256: return decode_d<256>(a, st);
  }
  return -1;
}

}  // extern "C"
