// From a fused projection row to the inputs of the gated delta rule (delta_scan.hip), in one launch:
// per token row
//   q, k [G heads], v [H heads]   short causal convolution over time, silu; q and k then made unit
//                                 vectors per head, x / sqrt(sum x^2 + 1e-6), q times qscale
//                                 -> fp32 rows, heads padded with zeros to DP / VP entries
//   la = -exp(A_log[h]) softplus(x_a + dt_bias[h]),  beta = sigmoid(x_b)     -> fp32 [rows, H]
// and, when an attention mixer reads the same projection row, that mixer's rotation and cache write
// (the units of qkv_prep.hip without a convolution).  The row is stored or still the fp32 split-K
// partials of the projection GEMM; the gate columns that later kernels read are then copied out.
// All arithmetic fp32; the convolution reads projected values rounded to the activation type.
//
// Units of a run (one wave each): G heads of q, G of k, H of v; with copies wanted (rows that
// arrive as partials) H heads of the gate; one unit for the numbers per head (decays, step sizes and
// the attention mixer's head gates).
#include "eia_prep.h"

struct DeltaPrepArgs {
  PrepRows rows;
  int q_off, k_off, v_off, g_off, b_off, a_off, H, G, D, Dv;
  const void* cw_q; const void* cw_k; const void* cw_v;
  void* state;                                // [slots, taps - 1, 2 G D + H Dv] projected values
  const float* expA; const float* dtb;        // [H]
  int taps; float qscale;
  const int* positions; const int* seq_slots; const int* cu; const int* work; int row_base;
  float* q; float* k; float* v; int DP, VP;   // [rows, G * DP], [rows, G * DP], [rows, H * VP]
  float* la; float* beta;                     // [rows, H]
  void* g_out; long ldg;                      // [rows, H * Dv] or null
  int hg_off, HG; void* hg_out;               // head gates of the attention mixer: [rows, HG] or null
};

EIA_DEV float dl_silu(float z) { return z / (1.0f + expf(-z)); }
EIA_DEV float dl_softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

template <typename T, int TAPS, int NE, int NR>
EIA_DEV void delta_prep_unit(const DeltaPrepArgs& a, const PrepRun& run, int unit) {
  const int lane = threadIdx.x & 63, n = run.n;
  const long row = run.row;
  const int nconv = 2 * a.G + a.H;
  if (unit >= nconv) {
    const int ng = a.g_out ? a.H : 0;
    if (unit < nconv + ng) {                           // gate columns of one head
      const int c0 = (unit - nconv) * a.Dv;
      for (int i = 0; i < n; ++i)
        for (int d = lane; d < a.Dv; d += 64)
          st_f32<T>((T*)a.g_out + (row + i) * a.ldg, c0 + d,
                    prep_load<T>(a.rows, row + i, a.g_off + c0 + d));
      return;
    }
    for (int i = 0; i < n; ++i) {                      // one number per head
      for (int h = lane; h < a.H; h += 64) {
        const float za = prep_load<T>(a.rows, row + i, a.a_off + h) + a.dtb[h];
        const float zb = prep_load<T>(a.rows, row + i, a.b_off + h);
        a.la[(row + i) * a.H + h] = -a.expA[h] * dl_softplus(za);
        a.beta[(row + i) * a.H + h] = 1.0f / (1.0f + expf(-zb));
      }
      if (a.hg_out)
        for (int h = lane; h < a.HG; h += 64)
          st_f32<T>((T*)a.hg_out + (row + i) * a.HG, h, prep_load<T>(a.rows, row + i, a.hg_off + h));
    }
    return;
  }
  const bool isq = unit < a.G, isk = !isq && unit < 2 * a.G;
  const int hh = isq ? unit : isk ? unit - a.G : unit - 2 * a.G;
  const int D = (isq || isk) ? a.D : a.Dv, P = (isq || isk) ? a.DP : a.VP;
  const int c0 = hh * D;
  const int col0 = (isq ? a.q_off : isk ? a.k_off : a.v_off) + c0;
  const int st0 = (isq ? 0 : isk ? a.G * a.D : 2 * a.G * a.D) + c0;
  const int ST = 2 * a.G * a.D + a.H * a.Dv;
  const T* cw = (const T*)(isq ? a.cw_q : isk ? a.cw_k : a.cw_v);
  int da[NE], db[NE];
  bool oka[NE], okb[NE];
  float ua[NE][NR], ub[NE][NR];
#pragma unroll
  for (int e = 0; e < NE; ++e) {
    da[e] = 2 * (lane + 64 * e);
    db[e] = da[e] + 1;
    oka[e] = da[e] < D;
    okb[e] = db[e] < D;
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      // (addresses clamped, no branches: the loads of a run are in flight together)
      ua[e][i] = prep_load<T>(a.rows, row + min(i, n - 1), col0 + (oka[e] ? da[e] : 0));
      ub[e][i] = prep_load<T>(a.rows, row + min(i, n - 1), col0 + (okb[e] ? db[e] : 0));
      if (!oka[e]) ua[e][i] = 0.f;
      if (!okb[e]) ub[e][i] = 0.f;
    }
  }
  const int slot = a.taps > 1 ? a.seq_slots[run.seq] : -1;
  prep_conv<T, TAPS, NE, NR>(a.rows, run, a.positions[row], cw, c0, col0,
                         slot >= 0 ? (T*)a.state + (long)slot * (a.taps - 1) * ST + st0 : nullptr,
                         ST, da, db, oka, okb, ua, ub, a.taps);
  float* dst = isq ? a.q + row * a.G * a.DP : isk ? a.k + row * a.G * a.DP : a.v + row * a.H * a.VP;
  const long ld = (long)((isq || isk) ? a.G : a.H) * P;
  dst += (long)hh * P;
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    if (i >= n) break;
    float ss = 0.f;
#pragma unroll
    for (int e = 0; e < NE; ++e) {
      ua[e][i] = dl_silu(ua[e][i]);                    // (channels past the head: silu(0) = 0)
      ub[e][i] = dl_silu(ub[e][i]);
      ss += ua[e][i] * ua[e][i] + ub[e][i] * ub[e][i];
    }
    float m = 1.f;
    if (isq || isk) m = (isq ? a.qscale : 1.f) / sqrtf(wave_sum(ss) + 1e-6f);
#pragma unroll
    for (int e = 0; e < NE; ++e)                       // (pad channels of the row: zeros)
      if (da[e] < P) {
        dst[i * ld + da[e]] = ua[e][i] * m;
        dst[i * ld + db[e]] = ub[e][i] * m;
      }
  }
}

// The attention mixer's units (w.H + 2 w.G; none when w.H is 0) come first.  TAPS: at least a.taps;
// NR: rows of a run (1 in decode steps).
template <typename T, int TAPS, int NE, int NR>
__global__ void __launch_bounds__(256)
delta_prep_kernel(const DeltaPrepArgs a, const QkvPrepArgs w, int units) {
  const int unit = blockIdx.y * 4 + (threadIdx.x >> 6), nw = w.H ? w.H + 2 * w.G : 0;
  if (unit >= units) return;
  const PrepRun run = prep_run(a.cu, a.work, a.row_base, blockIdx.x);
  if (run.n <= 0) return;
  if (unit < nw) qkv_prep_unit<T, 1, NE, NR>(w, run, unit);
  else delta_prep_unit<T, TAPS, NE, NR>(a, run, unit - nw);
}

// n_items: decode rows (work == nullptr) or prefill runs of QP_ROWS rows.  wH > 0: the attention
// mixer's heads (H wH, G wG, sizes wD / wDv, half-split or neighbouring rotation pairs) are prepared
// in the same launch.
EIA_API int eia_delta_prep(const void* x, long ld, const float* part, int sk, long pstride,
                           int q_off, int k_off, int v_off, int g_off, int b_off, int a_off, int H,
                           int G, int D, int Dv, const void* cw_q, const void* cw_k,
                           const void* cw_v, int taps, void* state, const float* expA,
                           const float* dtb, float qscale, const int* positions,
                           const int* seq_slots, const int* cu, const int* work, int row_base,
                           int n_items, float* q, float* k, float* v, int DP, int VP, float* la,
                           float* beta, void* g_out, long ldg, int hg_off, int HG, void* hg_out,
                           int wq_off, int wk_off, int wv_off, int wH, int wG, int wD, int wDv,
                           const float* inv_freq, int rot_dims, int half, float amp,
                           const int* slots, void* wq_out, long ldwq, void* kc, void* vc, int bs,
                           int is_bf16, hipStream_t st) {
  if (n_items < 0 || H < 1 || G < 1 || H % G || D < 1 || Dv < 1 || taps < 1 || taps > QP_TAPS ||
      (x == nullptr) == (part == nullptr) || (part && sk < 1) || !cw_q || !cw_k || !cw_v || !expA ||
      !dtb || !positions || (cu == nullptr) != (work == nullptr) || !q || !k || !v || !la || !beta ||
      DP < D || VP < Dv || DP % 2 || VP % 2 || (taps > 1 && (!state || !seq_slots)) || wH < 0 ||
      (hg_out && HG < 1) ||
      (wH && (wG < 1 || wH % wG || wD < 1 || wDv < 1 || bs < 1 || !slots || !wq_out || !kc || !vc ||
              rot_dims < 0 || rot_dims > wD || (rot_dims & 1) || (rot_dims && !inv_freq))))
    return EIA_BAD_SHAPE;
  if (DP > 256 || VP > 256 || wD > 256 || wDv > 256) return EIA_UNSUPPORTED;
  if (n_items == 0) return EIA_OK;
  DeltaPrepArgs a{{x, ld, part, sk, pstride, nullptr}, q_off, k_off, v_off, g_off, b_off, a_off, H, G,
                  D, Dv, cw_q, cw_k, cw_v, state, expA, dtb, taps, qscale, positions, seq_slots, cu, work,
                  row_base, q, k, v, DP, VP, la, beta, g_out, ldg, hg_off, HG, hg_out};
  QkvPrepArgs w{x, ld, part, sk, pstride, nullptr, wq_off, wk_off, wv_off, wH, wG, wD, wDv, nullptr,
                nullptr, nullptr, 1, nullptr, inv_freq, rot_dims, half, amp, 0, 0.f, nullptr, nullptr,
                0, positions, slots, nullptr, cu, work, row_base, wq_out, ldwq, kc, vc, bs};
  const int units = 2 * G + H + (g_out ? H : 0) + 1 + (wH ? wH + 2 * wG : 0);
  const dim3 grid(n_items, (units + 3) / 4);
  const bool wide = DP > 128 || VP > 128 || wD > 128 || wDv > 128;
#define DP_GO1(TT, N, NE, NR) \
  hipLaunchKernelGGL((delta_prep_kernel<TT, N, NE, NR>), grid, dim3(256), 0, st, a, w, units)
#define DP_GO(TT, N, NE)                                                       \
  do {                                                                        \
    if (work) DP_GO1(TT, N, NE, QP_ROWS); else DP_GO1(TT, N, NE, 1);          \
  } while (0)
#define DP_SIZES(TT)                                          \
  do {                                                        \
    if (taps <= 4) {                                          \
      if (wide) DP_GO(TT, 4, 2); else DP_GO(TT, 4, 1);        \
    } else {                                                  \
      if (wide) DP_GO(TT, 8, 2); else DP_GO(TT, 8, 1);        \
    }                                                         \
  } while (0)
  if (is_bf16) DP_SIZES(bf16_t); else DP_SIZES(float);
#undef DP_SIZES
#undef DP_GO
#undef DP_GO1
  EIA_LAUNCH_CHECK();
}
