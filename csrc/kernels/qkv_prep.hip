// From a fused projection row to attention inputs, in one launch: short causal convolution over
// time, rotation, per-head RMS norm without a weight, value mixing with an earlier layer's values,
// and the write of keys and values into the paged cache.
//
// Per token row (position p) and channel c of q, k or v (u: the projection, rounded to the
// activation type):
//   conv    y[p] = sum over lags d < taps of w[c, taps - 1 - d] u[p - d]   (no weights: y = u);
//           u is 0 ahead of token 0; tokens of earlier steps come from the sequence's state slot,
//           which carries its taps - 1 newest projected values
//   rotate  (q, k) the first rot_dims entries of every head turn by the position: pairs
//           (i, i + rot_dims/2) when half, else (2i, 2i + 1); angle p * inv_freq[i]; cos, sin * amp
//   norm    (q, k) every head divided by its root mean square, sqrt(mean + eps)
//   mix     (v) y <- (1 - lam) y + lam * v_first; or y is stored as v_first
// q -> q_out[t, H * D]; k -> key row of the token's cache slot; v -> value columns of the slot
// (page-transposed).  Slots < 0 write no cache rows.  All arithmetic fp32.
#include "eia_prep.h"

template <typename T, int TAPS, int NE>
__global__ void __launch_bounds__(256)
qkv_prep_kernel(const QkvPrepArgs a) {
  const int unit = blockIdx.y * (blockDim.x >> 6) + (threadIdx.x >> 6);
  if (unit >= a.H + 2 * a.G) return;
  const PrepRun run = prep_run(a.cu, a.work, a.row_base, blockIdx.x);
  if (run.n <= 0) return;
  qkv_prep_unit<T, TAPS, NE>(a, run, unit);
}

template <typename T, int NE>
static int qp_launch(const QkvPrepArgs& a, dim3 grid, hipStream_t st) {
  switch (a.taps) {
#define QP_CASE(N)                                                                              \
  case N:                                                                                       \
    hipLaunchKernelGGL((qkv_prep_kernel<T, N, NE>), grid, dim3(256), 0, st, a);                 \
    break;
    QP_CASE(1) QP_CASE(2) QP_CASE(3) QP_CASE(4) QP_CASE(5) QP_CASE(6) QP_CASE(7) QP_CASE(8)
#undef QP_CASE
    default: return EIA_UNSUPPORTED;
  }
  EIA_LAUNCH_CHECK();
}

// n_items: decode rows (work == nullptr) or prefill runs (pairs (sequence, first row of the run),
// runs of QP_ROWS rows, sequences relative to the pointers handed over).
EIA_API int eia_qkv_prep(const void* x, long ld, const float* part, int sk, long pstride,
                         const void* bias, int q_off, int k_off, int v_off, int H, int G, int D,
                         int Dv, const void* cw_q, const void* cw_k, const void* cw_v, int taps,
                         void* state, const float* inv_freq, int rot_dims, int half, float amp,
                         int norm, float eps, const float* lam, void* v_first, int v_mode,
                         const int* positions, const int* slots, const int* seq_slots,
                         const int* cu, const int* work, int row_base, int n_items, void* q_out,
                         long ldq, void* kc, void* vc, int bs, int is_bf16, hipStream_t st) {
  if (n_items < 0 || H < 1 || G < 1 || D < 1 || Dv < 1 || bs < 1 || taps < 1 || taps > QP_TAPS ||
      (x == nullptr) == (part == nullptr) || (part && sk < 1) || !positions || !slots || !q_out ||
      !kc || !vc || (cu == nullptr) != (work == nullptr) || rot_dims < 0 || rot_dims > D ||
      (rot_dims & 1) || (rot_dims && !inv_freq) || v_mode < 0 || v_mode > 2 ||
      (v_mode && !v_first) || (v_mode == 2 && !lam) ||
      (taps > 1 && (!cw_q || !cw_k || !cw_v || !state || !seq_slots)))
    return EIA_BAD_SHAPE;
  if (D > 256 || Dv > 256) return EIA_UNSUPPORTED;
  if (n_items == 0) return EIA_OK;
  QkvPrepArgs a{x, ld, part, sk, pstride, bias, q_off, k_off, v_off, H, G, D, Dv, cw_q, cw_k, cw_v,
                taps, state, inv_freq, rot_dims, half, amp, norm, eps, lam, v_first, v_mode,
                positions, slots, seq_slots, cu, work, row_base, q_out, ldq, kc, vc, bs};
  const dim3 grid(n_items, (H + 2 * G + 3) / 4);
  const bool wide = D > 128 || Dv > 128;
  if (is_bf16) return wide ? qp_launch<bf16_t, 2>(a, grid, st) : qp_launch<bf16_t, 1>(a, grid, st);
  return wide ? qp_launch<float, 2>(a, grid, st) : qp_launch<float, 1>(a, grid, st);
}
