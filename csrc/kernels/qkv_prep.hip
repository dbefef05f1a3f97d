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
//
// Work items are a run of up to QP_ROWS rows of one sequence (a decode row is a run of one); a
// wave owns one head (q, k or v) of a run, a lane one pair of its channels (two with heads above
// 128), so histories, rotation partners and the state slot's channels are all lane-local: the
// wave of a portion's first run reads the slot's old values of its channels and then stores the
// portion's last taps - 1 values there, with no other wave touching them.
#include "eia_common.h"

constexpr int QP_ROWS = 8;
constexpr int QP_TAPS = 8;          // largest number of taps

struct QkvPrepArgs {
  const void* x; long ld;                     // fused rows, or null and:
  const float* part; int sk; long pstride; const void* bias;
  int q_off, k_off, v_off, H, G, D, Dv;
  const void* cw_q; const void* cw_k; const void* cw_v; int taps;
  void* state;                                // [slots, taps - 1, (H + G) * D + G * Dv]
  const float* inv_freq; int rot_dims, half; float amp;
  int norm; float eps;
  const float* lam; void* v_first; int v_mode;   // 0: plain; 1: store; 2: mix
  const int* positions; const int* slots; const int* seq_slots;
  const int* cu; const int* work;             // prefill runs (cu relative to row_base); decode: null
  int row_base;
  void* q_out; long ldq; void* kc; void* vc; int bs;
};

template <typename T, int TAPS, int NE>
__global__ void __launch_bounds__(256)
qkv_prep_kernel(const QkvPrepArgs a) {
  constexpr int NH = TAPS > 1 ? TAPS - 1 : 1;
  const int lane = threadIdx.x & 63;
  const int unit = blockIdx.y * (blockDim.x >> 6) + (threadIdx.x >> 6);
  if (unit >= a.H + 2 * a.G) return;
  // the run: rows [row, row + n) of sequence seq, q0 rows into a portion of np rows
  int seq, q0 = 0, np = 1;
  long row;
  if (a.cu) {
    seq = a.work[2 * blockIdx.x];
    q0 = a.work[2 * blockIdx.x + 1];
    np = a.cu[seq + 1] - a.cu[seq];
    row = (long)a.row_base + a.cu[seq] + q0;
  } else {
    seq = blockIdx.x;
    row = (long)a.row_base + seq;
  }
  const int n = min(QP_ROWS, np - q0);
  if (n <= 0) return;
  const bool isq = unit < a.H, isk = !isq && unit < a.H + a.G;
  const int hh = isq ? unit : isk ? unit - a.H : unit - a.H - a.G;      // head within its kind
  const int D = (isq || isk) ? a.D : a.Dv;
  const int c0 = hh * D;                                                // first channel of its kind
  const int col0 = (isq ? a.q_off : isk ? a.k_off : a.v_off) + c0;      // ... in the fused row
  const int st0 = (isq ? 0 : isk ? a.H * a.D : (a.H + a.G) * a.D) + c0; // ... in the state row
  const int ST = (a.H + a.G) * a.D + a.G * a.Dv;
  const T* cw = (const T*)(isq ? a.cw_q : isk ? a.cw_k : a.cw_v);
  const T* X = (const T*)a.x;
  const T* B = (const T*)a.bias;
  const int rd = (isq || isk) ? a.rot_dims : 0, hd = rd >> 1;
  // lane slots: pair s of the head -> channels (da, db); rotated pairs first, then neighbours
  int da[NE], db[NE];
  bool oka[NE], okb[NE], rot[NE];
  float fr[NE];
#pragma unroll
  for (int e = 0; e < NE; ++e) {
    const int s = lane + 64 * e;
    rot[e] = s < hd;
    if (rot[e] && a.half) { da[e] = s; db[e] = s + hd; }
    else { da[e] = 2 * s; db[e] = 2 * s + 1; }        // (half: rd + 2 (s - hd) = 2 s)
    oka[e] = da[e] < D;
    okb[e] = db[e] < D;
    fr[e] = rot[e] ? a.inv_freq[s] : 0.f;
  }
  auto load = [&](long r, int d, bool ok) -> float {   // projected value, as the activation type
    if (!ok) return 0.f;
    if (X) return ld_f32<T>(X + r * a.ld, col0 + d);
    float v = B ? ld_f32<T>(B, col0 + d) : 0.f;
    const float* p = a.part + r * a.ld + col0 + d;
#pragma unroll 4
    for (int z = 0; z < a.sk; ++z) v += p[z * a.pstride];
    return (float)(T)v;
  };
  float ua[NE][QP_ROWS], ub[NE][QP_ROWS];
#pragma unroll
  for (int e = 0; e < NE; ++e)
#pragma unroll
    for (int i = 0; i < QP_ROWS; ++i) {
      ua[e][i] = i < n ? load(row + i, da[e], oka[e]) : 0.f;
      ub[e][i] = i < n ? load(row + i, db[e], okb[e]) : 0.f;
    }
  const int pos0 = a.positions[row];
  if constexpr (TAPS > 1) {
    const int slot = a.seq_slots[seq];
    T* S = (T*)a.state + (long)max(slot, 0) * (TAPS - 1) * ST + st0;
#pragma unroll
    for (int e = 0; e < NE; ++e) {
      float ha[NH], hb[NH], wa[TAPS], wb[TAPS];
#pragma unroll
      for (int j = 0; j < TAPS; ++j) {
        wa[j] = oka[e] ? ld_f32<T>(cw, (long)(c0 + da[e]) * TAPS + j) : 0.f;
        wb[j] = okb[e] ? ld_f32<T>(cw, (long)(c0 + db[e]) * TAPS + j) : 0.f;
      }
      // the TAPS - 1 values before the run: earlier rows of the portion, or the slot, or zeros
#pragma unroll
      for (int j = 0; j < NH; ++j) {
        const int back = TAPS - 1 - j;                 // tokens before the run's first row
        float va = 0.f, vb = 0.f;
        if (q0 > 0) {
          va = load(row - back, da[e], oka[e]);
          vb = load(row - back, db[e], okb[e]);
        } else if (pos0 >= back && slot >= 0) {
          if (oka[e]) va = ld_f32<T>(S, (long)j * ST + da[e]);
          if (okb[e]) vb = ld_f32<T>(S, (long)j * ST + db[e]);
        }
        ha[j] = va;
        hb[j] = vb;
      }
      if (q0 == 0 && slot >= 0) {                      // the slot after this portion
#pragma unroll
        for (int j = 0; j < NH; ++j) {
          const int idx = np - (TAPS - 1) + j;         // row of the portion; < 0: an older value
          float va = 0.f, vb = 0.f;
          if (idx >= 0) {
            va = load(row + idx, da[e], oka[e]);
            vb = load(row + idx, db[e], okb[e]);
          } else {
#pragma unroll
            for (int m = 0; m < NH; ++m)
              if (m == TAPS - 1 + idx) { va = ha[m]; vb = hb[m]; }
          }
          if (oka[e]) st_f32<T>(S, (long)j * ST + da[e], va);
          if (okb[e]) st_f32<T>(S, (long)j * ST + db[e], vb);
        }
      }
#pragma unroll
      for (int i = QP_ROWS - 1; i >= 0; --i) {         // last row first: earlier rows still hold u
        float ya = 0.f, yb = 0.f;
#pragma unroll
        for (int j = 0; j < TAPS; ++j) {
          const int r = i - (TAPS - 1) + j;
          ya += wa[j] * (r >= 0 ? ua[e][r >= 0 ? r : 0] : ha[r >= 0 ? 0 : TAPS - 1 + r]);
          yb += wb[j] * (r >= 0 ? ub[e][r >= 0 ? r : 0] : hb[r >= 0 ? 0 : TAPS - 1 + r]);
        }
        ua[e][i] = ya;
        ub[e][i] = yb;
      }
    }
  } else if (cw) {                                     // one tap: a factor per channel
#pragma unroll
    for (int e = 0; e < NE; ++e) {
      const float wa = oka[e] ? ld_f32<T>(cw, c0 + da[e]) : 0.f;
      const float wb = okb[e] ? ld_f32<T>(cw, c0 + db[e]) : 0.f;
#pragma unroll
      for (int i = 0; i < QP_ROWS; ++i) {
        ua[e][i] *= wa;
        ub[e][i] *= wb;
      }
    }
  }
  if (isq || isk) {
#pragma unroll
    for (int i = 0; i < QP_ROWS; ++i) {
      if (i >= n) break;
      const float pos = (float)(pos0 + i);
      float ss = 0.f;
#pragma unroll
      for (int e = 0; e < NE; ++e) {
        if (rot[e]) {
          float sn, cs;
          sincosf(pos * fr[e], &sn, &cs);
          sn *= a.amp;
          cs *= a.amp;
          const float u = ua[e][i], v = ub[e][i];
          ua[e][i] = u * cs - v * sn;
          ub[e][i] = v * cs + u * sn;
        }
        ss += ua[e][i] * ua[e][i] + ub[e][i] * ub[e][i];
      }
      const float inv = a.norm ? 1.0f / sqrtf(wave_sum(ss) / (float)D + a.eps) : 1.f;
      const long slot = isk ? (long)a.slots[row + i] : 0;
      if (slot < 0) continue;
      T* dst = isq ? (T*)a.q_out + (row + i) * a.ldq + c0
                   : (T*)a.kc + slot * ((long)a.G * a.D) + c0;
#pragma unroll
      for (int e = 0; e < NE; ++e) {
        if (oka[e]) st_f32<T>(dst, da[e], ua[e][i] * inv);
        if (okb[e]) st_f32<T>(dst, db[e], ub[e][i] * inv);
      }
    }
    return;
  }
  // values
  const long VW = (long)a.G * a.Dv;
  if (a.v_mode) {
    T* F = (T*)a.v_first;
    const float lam = a.v_mode == 2 ? a.lam[0] : 0.f;
#pragma unroll
    for (int e = 0; e < NE; ++e)
#pragma unroll
      for (int i = 0; i < QP_ROWS; ++i) {
        if (i >= n) break;
        T* f = F + (row + i) * VW + c0;
        if (a.v_mode == 1) {
          if (oka[e]) st_f32<T>(f, da[e], ua[e][i]);
          if (okb[e]) st_f32<T>(f, db[e], ub[e][i]);
        } else {
          if (oka[e]) ua[e][i] = (1.f - lam) * ua[e][i] + lam * ld_f32<T>(f, da[e]);
          if (okb[e]) ub[e][i] = (1.f - lam) * ub[e][i] + lam * ld_f32<T>(f, db[e]);
        }
      }
  }
  // eight consecutive tokens of one page: one 16-byte (bf16) or two (fp32) stores per column
  const long s0 = a.slots[row];
  bool run8 = n == QP_ROWS && s0 >= 0 && s0 % QP_ROWS == 0 && a.bs % QP_ROWS == 0;
  if (run8) {
#pragma unroll
    for (int i = 1; i < QP_ROWS; ++i) run8 = run8 && a.slots[row + i] == s0 + i;
  }
  T* V = (T*)a.vc;
#pragma unroll
  for (int e = 0; e < NE; ++e) {
    if (run8) {
      const long base = (s0 / a.bs) * VW * a.bs + s0 % a.bs;
      alignas(16) T ra[QP_ROWS], rb[QP_ROWS];
#pragma unroll
      for (int i = 0; i < QP_ROWS; ++i) { ra[i] = (T)ua[e][i]; rb[i] = (T)ub[e][i]; }
      constexpr int NV = QP_ROWS * sizeof(T) / 16;
      if (oka[e])
#pragma unroll
        for (int w = 0; w < NV; ++w)
          reinterpret_cast<uint4*>(V + base + (long)(c0 + da[e]) * a.bs)[w] =
              reinterpret_cast<const uint4*>(ra)[w];
      if (okb[e])
#pragma unroll
        for (int w = 0; w < NV; ++w)
          reinterpret_cast<uint4*>(V + base + (long)(c0 + db[e]) * a.bs)[w] =
              reinterpret_cast<const uint4*>(rb)[w];
      continue;
    }
#pragma unroll
    for (int i = 0; i < QP_ROWS; ++i) {
      if (i >= n) break;
      const long slot = a.slots[row + i];
      if (slot < 0) continue;
      const long base = (slot / a.bs) * VW * a.bs + slot % a.bs;
      if (oka[e]) st_f32<T>(V, base + (long)(c0 + da[e]) * a.bs, ua[e][i]);
      if (okb[e]) st_f32<T>(V, base + (long)(c0 + db[e]) * a.bs, ub[e][i]);
    }
  }
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
