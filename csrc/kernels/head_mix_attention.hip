// Softmax attention over a paged cache whose WEIGHTS are mixed across the heads before they meet
// the values (matrix-core form, bf16; the scalar form is window_attention.hip with talk_post):
//
//   s_g(i, j) = (q_g . k_j) * mult[g],  soft-capped when cap > 0
//   p_g       = softmax over the visible keys j <= i (i - j < window when window > 0)
//   out_h     = post * sum_j (sum_g T[h, g] p_g(j)) v_(h / (H / G))(j)
//
// The mixing needs every head's final normaliser, which an online softmax has only at the end --
// but it is linear, so it commutes with the sum over the keys: with A[g, r] = sum_j p_g(j) v_r(j),
// every head's weights applied to every kv head's values,
//
//   out_h = post * sum_g T[h, g] A[g, r(h)].
//
// One pass over the keys forms all A[g, r] (G value products per score instead of one) with the
// usual running (max, sum); a second small kernel merges key partitions, normalises and mixes.
// Scores, softmax weights, accumulators and the mixing are fp32; the weights enter the value
// product as a bf16 high part plus a bf16 remainder.
//
// Cache layout and operand tricks are those of window_attention.hip: token-major key rows
// [blocks, bs, G * D], values transposed inside a page [blocks, G * Dv, bs]; S^T (keys x columns)
// tiles whose rows are ordered so that a lane's accumulators are the B operand of the value
// product.
#include "eia_common.h"

struct HmArgs {
  const bf16_t* q; long ldq;        // [rows, H * D]
  const bf16_t* kc; const bf16_t* vc;
  const int* bt; int ldbt;
  const int* positions;
  const int* cu; const int* work;   // prefill items (sequence, first query); decode: null
  const int* lens;                  // decode: sequence lengths (0: padding row)
  const float* mult;                // [H]
  const float* talk;                // [H, H]
  bf16_t* out; long ldo;            // [rows, H * Dv]
  int H, G, D, Dv, bs, window;
  float cap, post;
  int nparts;
  float* acc;                       // [rows, nparts, H, G, Dv]: un-normalised A of every partition
  float* ml;                        // [rows, nparts, H, 2]: its running (max, sum)
};

typedef __attribute__((ext_vector_type(4))) unsigned int u32x4;
constexpr float HM_LOG2E = 1.4426950408889634f;
constexpr int HM_PAGES = 256;       // block -> page entries kept in LDS
constexpr int HM_QB = 32;           // queries per prefill work item

EIA_DEV float hm_softcap(float s, float cap, float icap2) {
  return cap - 2.f * cap * __builtin_amdgcn_rcpf(exp2f(s * icap2) + 1.f);
}
struct HmBlocks { int b0, n; };     // absolute 32-key blocks a row (or a 16-query tile) sees
EIA_DEV HmBlocks hm_blocks(int pos_first, int pos_last, int window) {
  const int b0 = (window > 0 ? max(0, pos_first - window + 1) : 0) >> 5;
  return HmBlocks{b0, (pos_last >> 5) - b0 + 1};
}
// key partitions a decode row really uses: about two blocks per wave of four
EIA_DEV int hm_parts(int nparts, int nblocks) { return min(nparts, max(1, (nblocks + 7) >> 3)); }

// ---------------------------------------------------------------------------------------------
// Prefill: a workgroup of four waves (four heads) owns a tile of 32 queries and NR kv heads'
// values (grid.z: the subset of kv heads); a wave owns one head and both 16-query halves, so
// every operand it reads feeds two (keys) or four (values: high part and remainder) products.
// The block's keys (NK distinct kv heads among the four heads) and values are staged in LDS,
// double buffered: the next block's global loads are in flight during this block's products.
// LDS rows are swizzled in 16-byte chunks so that the 16 lanes of an operand row group touch
// different banks.
template <int NK, int NR, int ND, int NDV>
struct HmStage {
  static constexpr int KC = ND * 4;                  // 16-byte chunks of a key row
  static constexpr int KCH = 32 * KC;                // chunks of one kv head's keys
  static constexpr int VCH = NDV * 16 * 4;           // chunks of one kv head's values
  static constexpr int TOT = NK * KCH + NR * VCH;    // chunks of one buffer
  static constexpr int PT = (TOT + 255) / 256;       // chunks per thread
};
// position of chunk j of a key row: 16 rows of one operand tile (rows 8 (c >> 2) + (c & 3) [+ 4])
// at the same chunk land in 16 different 16-byte columns of the banks
template <int ND> EIA_DEV int hm_kswz(int row, int j) {
  const int f = (row & 3) | ((row >> 3) << 2);
  return ND == 4 ? (j ^ f) : (j ^ (f >> 1));
}
EIA_DEV int hm_vswz(int row, int j) { return j ^ ((row >> 2) & 3); }

template <int NK, int NR, int ND, int NDV>
__global__ void __launch_bounds__(256, 2)
head_mix_prefill_kernel(const HmArgs a) {
  using S = HmStage<NK, NR, ND, NDV>;
  extern __shared__ u32x4 stage[];                   // [2][S::TOT]
  __shared__ int page_s[HM_PAGES];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int c = lane & 15, g = lane >> 4;
  const int H = a.H, G = a.G, D = a.D, Dv = a.Dv, bs = a.bs, rep = H / G;
  const int ndv = Dv >> 4;
  const long krow = (long)G * D, vpage = (long)G * Dv * bs;
  const int seq = a.work[2 * blockIdx.x], q0 = a.work[2 * blockIdx.x + 1];
  const int row0 = a.cu[seq] + q0, nq = min(HM_QB, a.cu[seq + 1] - row0);
  const int hw0 = blockIdx.y * 4, h = hw0 + wave;
  const bool on = h < H;
  const int hs = on ? h : H - 1;
  const int r0v = blockIdx.z * NR;
  const int* bt = a.bt + (long)seq * a.ldbt;
  const int pos_first = a.positions[row0], pos_last = a.positions[row0 + nq - 1];
  const HmBlocks kb = hm_blocks(pos_first, pos_last, a.window);
  for (int i = tid; i < min(kb.n, HM_PAGES); i += 256) page_s[i] = bt[((kb.b0 + i) << 5) / bs];
  const bf16x8 zero8 = {0, 0, 0, 0, 0, 0, 0, 0};
  bool row_ok[2];
  long row[2];
  int qpos[2];
  bf16x8 qf[2][ND];
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    row_ok[u] = 16 * u + c < nq;
    row[u] = row0 + (row_ok[u] ? 16 * u + c : 0);
    qpos[u] = a.positions[row[u]];
#pragma unroll
    for (int s = 0; s < ND; ++s) {
      const int d = 32 * s + 8 * g;
      const bf16x8 v = *reinterpret_cast<const bf16x8*>(a.q + row[u] * a.ldq + (long)hs * D +
                                                        (d < D ? d : 0));
      qf[u][s] = d < D ? v : zero8;
    }
  }
  const float mult = a.mult[hs], cap = a.cap, icap2 = cap > 0.f ? 2.f * HM_LOG2E / cap : 0.f;
  f32x4 acc[2][NR][NDV];
  float mrun[2], lrun[2];
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    mrun[u] = -1e30f;
    lrun[u] = 0.f;
#pragma unroll
    for (int r = 0; r < NR; ++r)
#pragma unroll
      for (int t = 0; t < NDV; ++t) acc[u][r][t] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  // this thread's chunks of a block: source offsets (elements from the block's first key / value
  // column) and LDS positions do not change from block to block
  // (KCH is a multiple of 256, so a thread's p-th chunk is a key chunk for all threads or none)
  int src[S::PT], dst[S::PT];
#pragma unroll
  for (int p = 0; p < S::PT; ++p) {
    const int x = tid + 256 * p;
    if (256 * p < NK * S::KCH) {
      const int k = x / S::KCH, y = x % S::KCH, r = y / S::KC, j = y % S::KC;
      const int kvh = min(hw0 + k * (4 / NK), H - 1) / rep;
      src[p] = r * G * D + kvh * D + (8 * j < D ? 8 * j : 0);
      dst[p] = k * S::KCH + r * S::KC + hm_kswz<ND>(r, j);
    } else {
      const int z = min(x, S::TOT - 1) - NK * S::KCH;
      const int rv = z / S::VCH, y = z % S::VCH, r = y >> 2, j = y & 3;
      src[p] = (min(r0v + rv, G - 1) * Dv + min(r, Dv - 1)) * bs + 8 * j;
      dst[p] = NK * S::KCH + rv * S::VCH + r * 4 + hm_vswz(r, j);
    }
  }
  u32x4 stg[S::PT];
  int off = (kb.b0 << 5) % bs;                       // the next block to fetch: place in its page
  auto fetch = [&](int b) {
    const long page = b < HM_PAGES ? page_s[b] : bt[((kb.b0 + b) << 5) / bs];
    const bf16_t* kp = a.kc + (page * bs + off) * krow;
    const bf16_t* vp = a.vc + page * vpage + off;
    off = off + 32 == bs ? 0 : off + 32;
#pragma unroll
    for (int p = 0; p < S::PT; ++p)
      stg[p] = *reinterpret_cast<const u32x4*>((256 * p < NK * S::KCH ? kp : vp) + src[p]);
  };
  auto put = [&](int buf) {
#pragma unroll
    for (int p = 0; p < S::PT; ++p)
      if (S::TOT % 256 == 0 || tid + 256 * p < S::TOT) stage[buf * S::TOT + dst[p]] = stg[p];
  };
  __syncthreads();                                   // page_s
  fetch(0);
  put(0);
  __syncthreads();
  const int kr0 = 8 * (c >> 2) + (c & 3);            // key of row c in tile 0 (tile 1: + 4)
  const int kslot = wave / (4 / NK);
  for (int b = 0; b < kb.n; ++b) {
    if (b + 1 < kb.n) fetch(b + 1);
    const u32x4* K = stage + (b & 1) * S::TOT + kslot * S::KCH;
    const u32x4* V = stage + (b & 1) * S::TOT + NK * S::KCH;
    const int key0 = (kb.b0 + b) << 5;
    f32x4 sc[2][2];
#pragma unroll
    for (int u = 0; u < 2; ++u) sc[u][0] = sc[u][1] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < ND; ++s) {                   // (past D: the query operand is zero)
      const bf16x8 k0 = *reinterpret_cast<const bf16x8*>(
          K + kr0 * S::KC + hm_kswz<ND>(kr0, 4 * s + g));
      const bf16x8 k1 = *reinterpret_cast<const bf16x8*>(
          K + (kr0 + 4) * S::KC + hm_kswz<ND>(kr0 + 4, 4 * s + g));
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        sc[u][0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k0, qf[u][s], sc[u][0], 0, 0, 0);
        sc[u][1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k1, qf[u][s], sc[u][1], 0, 0, 0);
      }
    }
    // a block that every query of the tile sees whole needs no mask
    const bool whole = nq == HM_QB && key0 + 31 <= pos_first &&
                       (a.window <= 0 || pos_last - key0 < a.window);
    bf16x8 ph[2], pl[2];
    float alpha[2];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      float v[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] = sc[u][e >> 2][e & 3] * mult;
      if (cap > 0.f) {
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = hm_softcap(v[e], cap, icap2);
      }
      if (!whole) {
        const int far = a.window > 0 ? a.window : 0x7fffffff;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const int back = qpos[u] - (key0 + 8 * g + e);
          v[e] = row_ok[u] && back >= 0 && back < far ? v[e] : -INFINITY;
        }
      }
      float mloc = -1e30f;
#pragma unroll
      for (int e = 0; e < 8; ++e) mloc = fmaxf(mloc, v[e]);
      mloc = fmaxf(mloc, __shfl_xor(mloc, 16, 64));
      mloc = fmaxf(mloc, __shfl_xor(mloc, 32, 64));
      const float mnew = fmaxf(mrun[u], mloc);
      alpha[u] = exp2f((mrun[u] - mnew) * HM_LOG2E);
      float psum = 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float p = exp2f((v[e] - mnew) * HM_LOG2E);
        const bf16_t hi = f2bf(p);
        ph[u][e] = hi;
        pl[u][e] = f2bf(p - bf2f(hi));
        psum += p;
      }
      psum += __shfl_xor(psum, 16, 64);
      psum += __shfl_xor(psum, 32, 64);
      lrun[u] = lrun[u] * alpha[u] + psum;
      mrun[u] = mnew;
    }
    if (__any(alpha[0] != 1.f || alpha[1] != 1.f)) {
#pragma unroll
      for (int u = 0; u < 2; ++u)
#pragma unroll
        for (int r = 0; r < NR; ++r)
#pragma unroll
          for (int t = 0; t < NDV; ++t) acc[u][r][t] *= alpha[u];
    }
#pragma unroll
    for (int r = 0; r < NR; ++r)
#pragma unroll
      for (int t = 0; t < NDV; ++t) {                // (tiles past Dv: staged repeats, not stored)
        const bf16x8 vf = *reinterpret_cast<const bf16x8*>(V + r * S::VCH + (16 * t + c) * 4 +
                                                           hm_vswz(16 * t + c, g));
#pragma unroll
        for (int u = 0; u < 2; ++u) {
          acc[u][r][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, ph[u], acc[u][r][t], 0, 0, 0);
          acc[u][r][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pl[u], acc[u][r][t], 0, 0, 0);
        }
      }
    if (b + 1 < kb.n) put((b + 1) & 1);              // (its last readers passed the barrier below)
    __syncthreads();
  }
  if (!on) return;
  // this lane holds, per kv head and tile t, value columns 16 t + 4 g + i of queries c, 16 + c
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    if (!row_ok[u]) continue;
    if (blockIdx.z == 0 && g == 0) {
      a.ml[(row[u] * H + h) * 2] = mrun[u];
      a.ml[(row[u] * H + h) * 2 + 1] = lrun[u];
    }
#pragma unroll
    for (int r = 0; r < NR; ++r) {
      if (r0v + r >= G) break;
      float* o = a.acc + ((row[u] * H + h) * G + r0v + r) * Dv + 4 * g;
#pragma unroll
      for (int t = 0; t < NDV; ++t)
        if (t < ndv) *reinterpret_cast<f32x4*>(o + 16 * t) = acc[u][r][t];
    }
  }
}

// ---------------------------------------------------------------------------------------------
// Decode: columns are HEADS.  A workgroup of four waves owns one row, up to 16 heads (all kv
// groups they belong to) and NR kv heads' values, and a partition of the row's 32-key blocks, of
// which each wave walks a quarter; every key and value is loaded once for all 16 heads.  The
// score of column c comes from the product with its own kv head's keys: for the other kv heads
// its query operand is zero.  The waves' (max, sum, A) are merged through LDS.
template <int NR, int ND, int NDV>
__global__ void __launch_bounds__(256, 1)
head_mix_decode_kernel(const HmArgs a) {
  constexpr int TC = 8;                              // value tiles merged per LDS round
  constexpr int KJ = 4;                              // kv heads' keys in flight together
  constexpr bool VLATE = NR * NDV >= 32;             // values requested behind the keys' products
  __shared__ f32x4 red[TC][4][64];
  __shared__ float ml_s[4][16][2];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int c = lane & 15, g = lane >> 4;
  const int H = a.H, G = a.G, D = a.D, Dv = a.Dv, bs = a.bs, rep = H / G;
  const int ndv = Dv >> 4;
  const long krow = (long)G * D, vpage = (long)G * Dv * bs;
  const int row = blockIdx.x, z = blockIdx.z;
  const int nsub = (G + NR - 1) / NR;
  const int h0 = (blockIdx.y / nsub) * 16, r0v = (blockIdx.y % nsub) * NR;
  if (a.lens && a.lens[row] <= 0) return;            // padding row: the merge writes zeros
  const int qpos = a.positions[row];
  const HmBlocks kb = hm_blocks(qpos, qpos, a.window);
  const int np = hm_parts(a.nparts, kb.n);
  if (z >= np) return;
  const int* bt = a.bt + (long)row * a.ldbt;
  const int h = h0 + c;
  const bool hok = h < H;
  const int grp = (hok ? h : h0) / rep;
  const int k_lo = h0 / rep, k_hi = (min(h0 + 16, H) - 1) / rep;
  const bf16x8 zero8 = {0, 0, 0, 0, 0, 0, 0, 0};
  bf16x8 qf[ND];
#pragma unroll
  for (int s = 0; s < ND; ++s) {
    const int d = 32 * s + 8 * g;
    const bf16x8 v = *reinterpret_cast<const bf16x8*>(a.q + (long)row * a.ldq + (long)(hok ? h : h0) * D +
                                                      (d < D ? d : 0));
    qf[s] = hok && d < D ? v : zero8;
  }
  const float mult = a.mult[hok ? h : h0], cap = a.cap;
  const float icap2 = cap > 0.f ? 2.f * HM_LOG2E / cap : 0.f;
  f32x4 acc[NR][NDV];
#pragma unroll
  for (int r = 0; r < NR; ++r)
#pragma unroll
    for (int t = 0; t < NDV; ++t) acc[r][t] = f32x4{0.f, 0.f, 0.f, 0.f};
  float mrun = -1e30f, lrun = 0.f;
  const int kr0 = 8 * (c >> 2) + (c & 3), dq = 8 * g;
  const int per = (kb.n + 4 * np - 1) / (4 * np);
  const int b_lo = (z * 4 + wave) * per, b_hi = min(kb.n, b_lo + per);
  for (int b = b_lo; b < b_hi; ++b) {
    const int key0 = (kb.b0 + b) << 5;
    const long page = bt[key0 / bs];
    const bf16_t* kp0 = a.kc + (page * bs + key0 % bs + kr0) * krow;
    const bf16_t* vp0 = a.vc + page * vpage + (long)c * bs + key0 % bs + dq;
    f32x4 s0 = {0.f, 0.f, 0.f, 0.f}, s1 = {0.f, 0.f, 0.f, 0.f};
    bf16x8 vf[NR][NDV];
    auto load_v = [&]() {
#pragma unroll
      for (int r = 0; r < NR; ++r) {
        const bf16_t* vp = vp0 + (long)min(r0v + r, G - 1) * Dv * bs;
#pragma unroll
        for (int t = 0; t < NDV; ++t)
          vf[r][t] = *reinterpret_cast<const bf16x8*>(vp + (long)(t < ndv ? t : 0) * 16 * bs);
      }
    };
    for (int k0 = k_lo; k0 <= k_hi; k0 += KJ) {      // a few kv heads' keys in flight together
      bf16x8 kf[KJ][2][ND];
#pragma unroll
      for (int j = 0; j < KJ; ++j) {
        const bf16_t* kp = kp0 + (long)min(k0 + j, k_hi) * D;
        if (k0 + j <= k_hi) {
#pragma unroll
          for (int s = 0; s < ND; ++s) {
            const int d = 32 * s + dq;
            kf[j][0][s] = *reinterpret_cast<const bf16x8*>(kp + (d < D ? d : 0));
            kf[j][1][s] = *reinterpret_cast<const bf16x8*>(kp + 4 * krow + (d < D ? d : 0));
          }
        }
      }
      if (!VLATE && k0 == k_lo) load_v();            // ... and the block's values behind them
#pragma unroll
      for (int j = 0; j < KJ; ++j) {
        if (k0 + j <= k_hi) {
          const bool mine = grp == k0 + j;
#pragma unroll
          for (int s = 0; s < ND; ++s) {
            const bf16x8 qm = mine ? qf[s] : zero8;
            // (d >= D: the query operand is zero and the key operand a finite repeat)
            s0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[j][0][s], qm, s0, 0, 0, 0);
            s1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[j][1][s], qm, s1, 0, 0, 0);
          }
        }
      }
    }
    if (VLATE) load_v();
    float v[8];
    bool vis[8];
    float mloc = -1e30f;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      v[e] = (e < 4 ? s0[e] : s1[e - 4]) * mult;
    }
    if (cap > 0.f) {
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] = hm_softcap(v[e], cap, icap2);
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const int key = key0 + 8 * g + e;
      vis[e] = key <= qpos && (a.window <= 0 || qpos - key < a.window);
      mloc = fmaxf(mloc, vis[e] ? v[e] : -1e30f);
    }
    mloc = fmaxf(mloc, __shfl_xor(mloc, 16, 64));
    mloc = fmaxf(mloc, __shfl_xor(mloc, 32, 64));
    const float mnew = fmaxf(mrun, mloc);
    const float alpha = exp2f((mrun - mnew) * HM_LOG2E);
    bf16x8 ph, pl;
    float psum = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const float p = vis[e] ? exp2f((v[e] - mnew) * HM_LOG2E) : 0.f;
      const bf16_t hi = f2bf(p);
      ph[e] = hi;
      pl[e] = f2bf(p - bf2f(hi));
      psum += p;
    }
    psum += __shfl_xor(psum, 16, 64);
    psum += __shfl_xor(psum, 32, 64);
    lrun = lrun * alpha + psum;
    mrun = mnew;
#pragma unroll
    for (int r = 0; r < NR; ++r)
#pragma unroll
      for (int t = 0; t < NDV; ++t) {
        f32x4 o = acc[r][t] * alpha;
        o = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[r][t], ph, o, 0, 0, 0);
        acc[r][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[r][t], pl, o, 0, 0, 0);
      }
  }
  // merge the four waves
  if (g == 0) {
    ml_s[wave][c][0] = mrun;
    ml_s[wave][c][1] = lrun;
  }
  __syncthreads();
  float m = ml_s[0][c][0];
#pragma unroll
  for (int w = 1; w < 4; ++w) m = fmaxf(m, ml_s[w][c][0]);
  float l = 0.f;
#pragma unroll
  for (int w = 0; w < 4; ++w) l += ml_s[w][c][1] * exp2f((ml_s[w][c][0] - m) * HM_LOG2E);
  const float f = exp2f((mrun - m) * HM_LOG2E);
  const long pr = ((long)row * a.nparts + z) * H + h;
  if (r0v == 0 && wave == 0 && g == 0 && hok) {
    a.ml[pr * 2] = m;
    a.ml[pr * 2 + 1] = l;
  }
#pragma unroll
  for (int x0 = 0; x0 < NR * NDV; x0 += TC) {
#pragma unroll
    for (int i = 0; i < TC; ++i)
      if (x0 + i < NR * NDV) red[i][wave][lane] = acc[(x0 + i) / NDV][(x0 + i) % NDV] * f;
    __syncthreads();
#pragma unroll
    for (int i0 = 0; i0 < TC; i0 += 4) {              // wave w sums tiles w, w + 4
      const int i = i0 + wave, x = x0 + i;
      const int r = r0v + x / NDV, t = x % NDV;
      if (x < NR * NDV && r < G && t < ndv && hok) {
        const f32x4 o = red[i][0][lane] + red[i][1][lane] + red[i][2][lane] + red[i][3][lane];
        *reinterpret_cast<f32x4*>(a.acc + (pr * G + r) * Dv + 16 * t + 4 * g) = o;
      }
    }
    __syncthreads();
  }
}

// ---------------------------------------------------------------------------------------------
// Merge of the key partitions, normalisation and head mixing: one workgroup per (row, kv head).
__global__ void __launch_bounds__(256)
head_mix_merge_kernel(const HmArgs a) {
  extern __shared__ float lds[];
  const int H = a.H, G = a.G, Dv = a.Dv, rep = H / G, NP = a.nparts;
  const long row = blockIdx.x;
  const int r = blockIdx.y, tid = threadIdx.x;
  bf16_t* out = a.out + row * a.ldo + (long)r * rep * Dv;
  if (a.lens && a.lens[row] <= 0) {
    for (int i = tid; i < rep * Dv; i += blockDim.x) out[i] = f2bf(0.f);
    return;
  }
  int np = 1;
  if (!a.cu) {
    const int pos = a.positions[row];
    np = hm_parts(NP, hm_blocks(pos, pos, a.window).n);
  }
  float* w_s = lds;                                   // [np, H] weight of a partition
  float* a_s = lds + NP * H;                          // [H, Dv] normalised A of this kv head
  for (int g = tid; g < H; g += blockDim.x) {
    float m = -1e30f, l = 0.f;
    for (int z = 0; z < np; ++z) m = fmaxf(m, a.ml[((row * NP + z) * H + g) * 2]);
    for (int z = 0; z < np; ++z) {
      const float w = exp2f((a.ml[((row * NP + z) * H + g) * 2] - m) * HM_LOG2E);
      l += w * a.ml[((row * NP + z) * H + g) * 2 + 1];
      w_s[z * H + g] = w;
    }
    const float inv = a.post / l;
    for (int z = 0; z < np; ++z) w_s[z * H + g] *= inv;
  }
  __syncthreads();
  const int v4 = Dv >> 2;
  for (int i = tid; i < H * v4; i += blockDim.x) {
    const int g = i / v4, d = (i - g * v4) * 4;
    f32x4 v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int z = 0; z < np; ++z)
      v += w_s[z * H + g] *
           *reinterpret_cast<const f32x4*>(a.acc + (((row * NP + z) * H + g) * G + r) * (long)Dv + d);
    *reinterpret_cast<f32x4*>(a_s + g * Dv + d) = v;
  }
  __syncthreads();
  for (int i = tid; i < rep * v4; i += blockDim.x) {
    const int j = i / v4, d = (i - j * v4) * 4;
    const float* T = a.talk + (long)(r * rep + j) * H;
    f32x4 v = {0.f, 0.f, 0.f, 0.f};
    for (int g = 0; g < H; ++g) v += T[g] * *reinterpret_cast<const f32x4*>(a_s + g * Dv + d);
    bf16x4 o;
#pragma unroll
    for (int e = 0; e < 4; ++e) o[e] = f2bf(v[e]);
    *reinterpret_cast<bf16x4*>(out + (long)j * Dv + d) = o;
  }
}

EIA_API int eia_head_mix_attn_ok(int H, int G, int D, int Dv, int bs) {
  return H >= 1 && H <= 64 && G >= 1 && H % G == 0 && D % 8 == 0 && D <= 128 && Dv % 16 == 0 &&
         Dv <= 128 && bs % 32 == 0;
}

// n_items: decode rows (cu == nullptr) or prefill work items; rows: rows of the part (prefill).
// acc fp32 [rows, nparts, H, G, Dv] and ml fp32 [rows, nparts, H, 2] are workspaces.
EIA_API int eia_head_mix_attn(const void* q, long ldq, const void* kc, const void* vc,
                              const int* bt, int ldbt, const int* positions, const int* cu,
                              const int* work, const int* lens, int n_items, int rows,
                              const float* mult, const float* talk, void* out, long ldo, int H,
                              int G, int D, int Dv, int bs, int window, float cap, float post,
                              int nparts, float* acc, float* ml, hipStream_t st) {
  if (n_items < 0 || rows < 0 || bs < 1 || !q || !kc || !vc || !bt || !positions || !mult ||
      !talk || !out || !acc || !ml || cap < 0.f || (cu == nullptr) != (work == nullptr) ||
      nparts < 1 || nparts > 64 || (cu && nparts != 1))
    return EIA_BAD_SHAPE;
  if (!eia_head_mix_attn_ok(H, G, D, Dv, bs)) return EIA_UNSUPPORTED;
  if (ldq % 8 || ldo % 4) return EIA_BAD_SHAPE;
  if (n_items == 0 || rows == 0) return EIA_OK;
  HmArgs a{(const bf16_t*)q, ldq, (const bf16_t*)kc, (const bf16_t*)vc, bt, ldbt, positions, cu,
           work, lens, mult, talk, (bf16_t*)out, ldo, H, G, D, Dv, bs, window, cap, post, nparts,
           acc, ml};
  const bool bk = D > 64, bv = Dv > 64;
#define HM_SIZES(L, NR)                                                                         \
  do {                                                                                          \
    if (bk && bv) L(NR, 4, 8);                                                                  \
    else if (bk) L(NR, 4, 4);                                                                   \
    else if (bv) L(NR, 2, 8);                                                                   \
    else L(NR, 2, 4);                                                                           \
  } while (0)
  if (cu) {
    // distinct kv heads among the four heads of a workgroup: 1, 2 or (any grouping) one per head
    const int rep = H / G, nk = rep % 4 == 0 ? 1 : rep % 2 == 0 ? 2 : 4;
#define HM_PRE1(NK, NR, ND_, NV_)                                                               \
  do {                                                                                          \
    constexpr int lds = 2 * HmStage<NK, NR, ND_, NV_>::TOT * 16;                                \
    if (lds > 48 * 1024)                                                                        \
      (void)hipFuncSetAttribute(                                                                \
          reinterpret_cast<const void*>(&head_mix_prefill_kernel<NK, NR, ND_, NV_>),            \
          hipFuncAttributeMaxDynamicSharedMemorySize, lds);                                     \
    hipLaunchKernelGGL((head_mix_prefill_kernel<NK, NR, ND_, NV_>),                             \
                       dim3(n_items, (H + 3) / 4, (G + NR - 1) / NR), dim3(256), lds, st, a);   \
  } while (0)
#define HM_PRE(NR, ND_, NV_)                                                                    \
  do {                                                                                          \
    if (nk == 1) HM_PRE1(1, NR, ND_, NV_);                                                      \
    else if (nk == 2) HM_PRE1(2, NR, ND_, NV_);                                                 \
    else HM_PRE1(4, NR, ND_, NV_);                                                              \
  } while (0)
    // (one kv head's values at a time where two do not fit the registers)
    if (G == 1 || (nk == 4 && bk && bv)) HM_SIZES(HM_PRE, 1); else HM_SIZES(HM_PRE, 2);
#undef HM_PRE1
#undef HM_PRE
  } else {
#define HM_DEC(NR, ND_, NV_)                                                                    \
  hipLaunchKernelGGL((head_mix_decode_kernel<NR, ND_, NV_>),                                    \
                     dim3(n_items, ((H + 15) / 16) * ((G + NR - 1) / NR), nparts), dim3(256), 0, \
                     st, a)
    if (G == 1) HM_SIZES(HM_DEC, 1);
    else if (G == 2) HM_SIZES(HM_DEC, 2);
    else HM_SIZES(HM_DEC, 4);
#undef HM_DEC
  }
#undef HM_SIZES
  const size_t lds = sizeof(float) * ((size_t)nparts * H + (size_t)H * Dv);
  hipLaunchKernelGGL(head_mix_merge_kernel, dim3(rows, G), dim3(256), lds, st, a);
  EIA_LAUNCH_CHECK();
}
