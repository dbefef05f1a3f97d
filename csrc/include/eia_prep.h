// Device code of the launches that turn fused projection rows into mixer inputs (qkv_prep.hip,
// delta_scan.hip).  Work items are a run of up to QP_ROWS rows of one sequence (a decode row is a
// run of one); a wave owns one head of a run, a lane one pair of its channels (two with heads above
// 128), so convolution histories, rotation partners and the state slot's channels are all
// lane-local: the wave of a portion's first run reads the slot's old values of its channels and
// then stores the portion's last taps - 1 values there, with no other wave touching them.
#pragma once
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

// The run of a work item: rows [row, row + n) of sequence seq, q0 rows into a portion of np rows.
struct PrepRun { int seq, q0, np, n; long row; };
EIA_DEV PrepRun prep_run(const int* cu, const int* work, int row_base, int item) {
  PrepRun r{item, 0, 1, 1, (long)row_base + item};
  if (cu) {
    r.seq = work[2 * item];
    r.q0 = work[2 * item + 1];
    r.np = cu[r.seq + 1] - cu[r.seq];
    r.row = (long)row_base + cu[r.seq] + r.q0;
    r.n = min(QP_ROWS, r.np - r.q0);
  }
  return r;
}

// A fused projection row: stored (x, row stride ld) or fp32 split-K partials [sk, rows, ld] (+ bias).
struct PrepRows { const void* x; long ld; const float* part; int sk; long pstride; const void* bias; };
template <typename T>
EIA_DEV float prep_load(const PrepRows& p, long r, int col) {     // as the activation type
  if (p.x) return ld_f32<T>((const T*)p.x + r * p.ld, col);
  float v = p.bias ? ld_f32<T>((const T*)p.bias, col) : 0.f;
  const float* q = p.part + r * p.ld + col;
  for (int z0 = 0; z0 < p.sk; z0 += 4) {               // four partials in flight
    float u[4];
#pragma unroll
    for (int z = 0; z < 4; ++z) u[z] = q[min(z0 + z, p.sk - 1) * p.pstride];
#pragma unroll
    for (int z = 0; z < 4; ++z) v += z0 + z < p.sk ? u[z] : 0.f;
  }
  return (float)(T)v;
}

// Short causal convolution of a run's channels da[e], db[e] of one head (in place in ua, ub): the
// head's columns start at col0 in the fused row and at channel c0 of its weights cw [., taps],
// taps <= TAPS; S: the head's first channel in the sequence's history slot (rows of ST), null: no
// slot.
template <typename T, int TAPS, int NE, int NR>
EIA_DEV void prep_conv(const PrepRows& rows, const PrepRun& run, int pos0, const T* cw, int c0,
                       int col0, T* S, int ST, const int (&da)[NE], const int (&db)[NE],
                       const bool (&oka)[NE], const bool (&okb)[NE], float (&ua)[NE][NR],
                       float (&ub)[NE][NR], const int taps = TAPS) {
  constexpr int NH = TAPS > 1 ? TAPS - 1 : 1;
  const int j0 = TAPS - taps;                          // unused oldest taps
  auto load = [&](long r, int d, bool ok) -> float {            // (address clamped, no branch)
    const float v = prep_load<T>(rows, r, col0 + (ok ? d : 0));
    return ok ? v : 0.f;
  };
  if constexpr (TAPS > 1) {
#pragma unroll
    for (int e = 0; e < NE; ++e) {
      float ha[NH], hb[NH], wa[TAPS], wb[TAPS];
#pragma unroll
      for (int j = 0; j < TAPS; ++j) {
        const int jj = j >= j0 ? j - j0 : 0;
        wa[j] = ld_f32<T>(cw, (long)(c0 + (oka[e] ? da[e] : 0)) * taps + jj);
        wb[j] = ld_f32<T>(cw, (long)(c0 + (okb[e] ? db[e] : 0)) * taps + jj);
        if (j < j0 || !oka[e]) wa[j] = 0.f;
        if (j < j0 || !okb[e]) wb[j] = 0.f;
      }
      // the TAPS - 1 values before the run: earlier rows of the portion, or the slot, or zeros
#pragma unroll
      for (int j = 0; j < NH; ++j) {
        const int back = TAPS - 1 - j;                 // tokens before the run's first row
        float va = 0.f, vb = 0.f;
        if (j < j0) {
        } else if (run.q0 > 0) {
          va = load(run.row - back, da[e], oka[e]);
          vb = load(run.row - back, db[e], okb[e]);
        } else if (pos0 >= back && S) {
          va = ld_f32<T>(S, (long)(j - j0) * ST + (oka[e] ? da[e] : 0));
          vb = ld_f32<T>(S, (long)(j - j0) * ST + (okb[e] ? db[e] : 0));
        }
        ha[j] = va;
        hb[j] = vb;
      }
      if (run.q0 == 0 && S) {                          // the slot after this portion
#pragma unroll
        for (int j = 0; j < NH; ++j) {
          if (j < j0) continue;
          const int idx = run.np - (TAPS - 1) + j;     // row of the portion; < 0: an older value
          float va = 0.f, vb = 0.f;
          if (idx >= 0) {
            va = load(run.row + idx, da[e], oka[e]);
            vb = load(run.row + idx, db[e], okb[e]);
          } else {
#pragma unroll
            for (int m = 0; m < NH; ++m)
              if (m == TAPS - 1 + idx) { va = ha[m]; vb = hb[m]; }
          }
          if (oka[e]) st_f32<T>(S, (long)(j - j0) * ST + da[e], va);
          if (okb[e]) st_f32<T>(S, (long)(j - j0) * ST + db[e], vb);
        }
      }
#pragma unroll
      for (int i = NR - 1; i >= 0; --i) {         // last row first: earlier rows still hold u
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
  } else {                                    // one tap: a factor per channel
#pragma unroll
    for (int e = 0; e < NE; ++e) {
      const float wa = oka[e] ? ld_f32<T>(cw, c0 + da[e]) : 0.f;
      const float wb = okb[e] ? ld_f32<T>(cw, c0 + db[e]) : 0.f;
#pragma unroll
      for (int i = 0; i < NR; ++i) {
        ua[e][i] *= wa;
        ub[e][i] *= wb;
      }
    }
  }
}

// One unit (head of q, k or v) of a run of up to NR rows.
template <typename T, int TAPS, int NE, int NR = QP_ROWS>
EIA_DEV void qkv_prep_unit(const QkvPrepArgs& a, const PrepRun& run, int unit) {
  const int lane = threadIdx.x & 63;
  const int n = run.n;
  const long row = run.row;
  const bool isq = unit < a.H, isk = !isq && unit < a.H + a.G;
  const int hh = isq ? unit : isk ? unit - a.H : unit - a.H - a.G;      // head within its kind
  const int D = (isq || isk) ? a.D : a.Dv;
  const int c0 = hh * D;                                                // first channel of its kind
  const int col0 = (isq ? a.q_off : isk ? a.k_off : a.v_off) + c0;      // ... in the fused row
  const int st0 = (isq ? 0 : isk ? a.H * a.D : (a.H + a.G) * a.D) + c0; // ... in the state row
  const int ST = (a.H + a.G) * a.D + a.G * a.Dv;
  const T* cw = (const T*)(isq ? a.cw_q : isk ? a.cw_k : a.cw_v);
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
  const PrepRows rows{a.x, a.ld, a.part, a.sk, a.pstride, a.bias};
  auto load = [&](long r, int d, bool ok) -> float {            // (address clamped, no branch)
    const float v = prep_load<T>(rows, r, col0 + (ok ? d : 0));
    return ok ? v : 0.f;
  };
  float ua[NE][NR], ub[NE][NR];
#pragma unroll
  for (int e = 0; e < NE; ++e)
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      ua[e][i] = load(row + min(i, n - 1), da[e], oka[e]);      // (rows past the run: unused)
      ub[e][i] = load(row + min(i, n - 1), db[e], okb[e]);
    }
  const int pos0 = a.positions[row];
  if constexpr (TAPS > 1) {
    const int slot = a.seq_slots[run.seq];
    prep_conv<T, TAPS, NE, NR>(rows, run, pos0, cw, c0, col0,
                           slot >= 0 ? (T*)a.state + (long)slot * (TAPS - 1) * ST + st0 : nullptr,
                           ST, da, db, oka, okb, ua, ub);
  } else if (cw) {
    prep_conv<T, 1, NE, NR>(rows, run, pos0, cw, c0, col0, nullptr, 0, da, db, oka, okb, ua, ub);
  }
  if (isq || isk) {
#pragma unroll
    for (int i = 0; i < NR; ++i) {
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
      for (int i = 0; i < NR; ++i) {
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
  bool run8 = NR == QP_ROWS && n == QP_ROWS && s0 >= 0 && s0 % QP_ROWS == 0 && a.bs % QP_ROWS == 0;
  if (run8) {
#pragma unroll
    for (int i = 1; i < NR; ++i) run8 = run8 && a.slots[row + i] == s0 + i;
  }
  T* V = (T*)a.vc;
#pragma unroll
  for (int e = 0; e < NE; ++e) {
    if (run8) {
      const long base = (s0 / a.bs) * VW * a.bs + s0 % a.bs;
      alignas(16) T ra[NR], rb[NR];
#pragma unroll
      for (int i = 0; i < NR; ++i) { ra[i] = (T)ua[e][i]; rb[i] = (T)ub[e][i]; }
      constexpr int NV = NR * sizeof(T) / 16;
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
    for (int i = 0; i < NR; ++i) {
      if (i >= n) break;
      const long slot = a.slots[row + i];
      if (slot < 0) continue;
      const long base = (slot / a.bs) * VW * a.bs + slot % a.bs;
      if (oka[e]) st_f32<T>(V, base + (long)(c0 + da[e]) * a.bs, ua[e][i]);
      if (okb[e]) st_f32<T>(V, base + (long)(c0 + db[e]) * a.bs, ub[e][i]);
    }
  }
}
