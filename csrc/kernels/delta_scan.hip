// Gated delta rule on per-sequence state slots: a matrix state S [dk, dv] per head whose answer to
// the key moves towards the value by the step size,
//
//   S <- a_t S_(t-1);   u_t = b_t (v_t - S^T k_t);   S_t = S + k_t u_t^T;   o_t = S_t^T q_t
//
// with one decay a_t = exp(la_t), la_t = -exp(A_log[h]) softplus(x_a + dt_bias[h]), and one step size
// b_t = sigmoid(x_b) per head and token.  q and k [G heads] and v [H heads] are projections that pass
// a short causal convolution over time and silu; q and k are made unit vectors per head,
// x / sqrt(sum x^2 + 1e-6), q is then scaled; head h reads q / k head h / (H / G).  Each head's o is
// divided by its root mean square, multiplied by a weight shared by the heads, by silu of its gate
// columns and by out_scale.
//
// q, k, v, la and b arrive as the fp32 rows that delta_prep.hip leaves.  Everything here is fp32, the
// matrix products included (v_mfma_f32_16x16x4_f32 in the chunk-parallel form).
//
// A sequence whose first row of the step is position 0 starts from zeros whatever its slot held, so
// slots are reused without clearing.  Batch layout: sequence s owns rows [cu[s], cu[s+1])
// (cu == nullptr: row s).
#include "eia_common.h"

EIA_DEV float dl_silu(float z) { return z / (1.0f + expf(-z)); }

// ---------------------------------------------------------------------------------------------
struct DeltaArgs {
  const float* q; const float* k; const float* v; const float* la; const float* beta;
  int H, G, D, Dv, DP, VP;
  const void* g; long ldg; const void* norm_w; float out_scale, eps;
  float* S; const int* slots; const int* cu; const int* positions; const int* seq_lens;
  void* y; long ldy;
};

// Token by token: one workgroup of 256 threads per (sequence, head).  Thread (rg, cg) owns rows
// rg, rg + RG, ... and columns 4 cg .. of S in registers (CGP = 2^LG column groups, RG = 256 / CGP row
// groups).  Per token one pass over the registers forms S^T k and S^T q of the state BEFORE the
// token; with them and k . q, u = b (v - a S^T k) and o = a S^T q + (k . q) u, so the update needs no
// second reduction (the four waves' partial sums of odd and even tokens alternate between two LDS
// buffers: one barrier per token).  Tokens are staged DS_TC at a time, (k, q) pairs zero past D.
// vec: 16-byte accesses to the state.
constexpr int DS_TC = 8;

template <typename T, int LG, int RPT>
__global__ void __launch_bounds__(256)
delta_scan_kernel(DeltaArgs a, int vec) {
  constexpr int CGP = 1 << LG, RG = 256 >> LG, CW = 4 * CGP, RW = RG * RPT;
  __shared__ __align__(16) float2 skq[DS_TC][RW];
  __shared__ __align__(16) float sv[DS_TC][CW], so[DS_TC][CW], sp[2][4][2][CW];
  __shared__ float dot[DS_TC], sa[DS_TC], sb[DS_TC];
  const int s = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int slot = a.slots[s];
  if (slot < 0 || (a.seq_lens && a.seq_lens[s] <= 0)) return;
  const int lo = a.cu ? a.cu[s] : s, hi = a.cu ? a.cu[s + 1] : s + 1;
  if (hi <= lo) return;
  const int H = a.H, G = a.G, D = a.D, Dv = a.Dv, DP = a.DP, VP = a.VP, kh = h / (H / G);
  const int cg = tid & (CGP - 1), rg = tid >> LG, c0 = 4 * cg;
  float* Sg = a.S + ((long)slot * H + h) * D * Dv;
  const bool fresh = a.positions[lo] == 0;
  f32x4 S[RPT];
#pragma unroll
  for (int ii = 0; ii < RPT; ++ii) {
    const int i = rg + RG * ii;
    S[ii] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (fresh || i >= D || c0 >= Dv) continue;
    if (vec) {
      S[ii] = *reinterpret_cast<const f32x4*>(Sg + (long)i * Dv + c0);
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (c0 + e < Dv) S[ii][e] = Sg[(long)i * Dv + c0 + e];
    }
  }
  const T* NW = static_cast<const T*>(a.norm_w);
  const T* GT = static_cast<const T*>(a.g);
  T* Y = static_cast<T*>(a.y);
  const int lane = tid & 63, wave = tid >> 6;
  for (int base = lo; base < hi; base += DS_TC) {
    const int nt = min(DS_TC, hi - base);
    __syncthreads();                                   // the previous tokens' LDS reads are done
    for (int idx = tid; idx < nt * RW; idx += 256) {
      const int t = idx / RW, d = idx % RW;
      const long r = ((long)(base + t) * G + kh) * DP + min(d, DP - 1);
      skq[t][d] = d < D ? make_float2(a.k[r], a.q[r]) : make_float2(0.f, 0.f);
    }
    for (int idx = tid; idx < nt * CW; idx += 256) {
      const int t = idx / CW, d = idx % CW;
      sv[t][d] = d < Dv ? a.v[((long)(base + t) * H + h) * VP + d] : 0.f;
    }
    if (tid < nt) {
      sa[tid] = expf(a.la[(long)(base + tid) * H + h]);
      sb[tid] = a.beta[(long)(base + tid) * H + h];
    }
    __syncthreads();
    for (int t = wave; t < nt; t += 4) {               // k . q
      float v = 0.f;
      for (int d = lane; d < RW; d += 64) v += skq[t][d].x * skq[t][d].y;
      v = wave_sum(v);
      if (lane == 0) dot[t] = v;
    }
    for (int t = 0; t < nt; ++t) {
      f32x4 ak = {0.f, 0.f, 0.f, 0.f}, aq = ak;
      float kr[RPT <= 16 ? RPT : 1];
#pragma unroll
      for (int ii = 0; ii < RPT; ++ii) {
        const float2 kq = skq[t][rg + RG * ii];
        if constexpr (RPT <= 16) kr[ii] = kq.x;
        ak += S[ii] * kq.x;
        aq += S[ii] * kq.y;
      }
#pragma unroll
      for (int o = CGP; o < 64; o <<= 1) {             // row groups inside the wave
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          ak[e] += __shfl_xor(ak[e], o, 64);
          aq[e] += __shfl_xor(aq[e], o, 64);
        }
      }
      if (lane < CGP) {
        *reinterpret_cast<f32x4*>(&sp[t & 1][wave][0][c0]) = ak;
        *reinterpret_cast<f32x4*>(&sp[t & 1][wave][1][c0]) = aq;
      }
      __syncthreads();
      f32x4 pk[4], pq[4];
#pragma unroll
      for (int z = 0; z < 4; ++z) {
        pk[z] = *reinterpret_cast<const f32x4*>(&sp[t & 1][z][0][c0]);
        pq[z] = *reinterpret_cast<const f32x4*>(&sp[t & 1][z][1][c0]);
      }
      const float at = sa[t];
      const f32x4 u = (*reinterpret_cast<const f32x4*>(&sv[t][c0]) -
                       (pk[0] + pk[1] + pk[2] + pk[3]) * at) * sb[t];
      if (rg == 0)
        *reinterpret_cast<f32x4*>(&so[t][c0]) = (pq[0] + pq[1] + pq[2] + pq[3]) * at + u * dot[t];
#pragma unroll
      for (int ii = 0; ii < RPT; ++ii)
        S[ii] = S[ii] * at + u * (RPT <= 16 ? kr[RPT <= 16 ? ii : 0] : skq[t][rg + RG * ii].x);
    }
    __syncthreads();
    for (int t = wave; t < nt; t += 4) {               // head RMS norm, weight, gate
      float ss = 0.f;
      for (int d = lane; d < Dv; d += 64) ss += so[t][d] * so[t][d];
      const float inv = a.out_scale / sqrtf(wave_sum(ss) / (float)Dv + a.eps);
      for (int d = lane; d < Dv; d += 64)
        st_f32<T>(Y + (long)(base + t) * a.ldy, (long)h * Dv + d,
                  so[t][d] * inv * ld_f32<T>(NW, d) *
                      dl_silu(ld_f32<T>(GT + (long)(base + t) * a.ldg, (long)h * Dv + d)));
    }
  }
#pragma unroll
  for (int ii = 0; ii < RPT; ++ii) {
    const int i = rg + RG * ii;
    if (i >= D || c0 >= Dv) continue;
    if (vec) {
      *reinterpret_cast<f32x4*>(Sg + (long)i * Dv + c0) = S[ii];
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (c0 + e < Dv) Sg[(long)i * Dv + c0 + e] = S[ii][e];
    }
  }
}

static bool delta_args_ok(const DeltaArgs& a, int nseq) {
  return nseq >= 0 && a.H >= 1 && a.G >= 1 && a.H % a.G == 0 && a.D >= 1 && a.Dv >= 1 &&
         a.DP >= a.D && a.VP >= a.Dv && a.q && a.k && a.v && a.la && a.beta && a.g && a.norm_w &&
         a.S && a.slots && a.positions && a.y;
}

template <typename T>
static int delta_step(const DeltaArgs& a, int nseq, hipStream_t st) {
  if (a.D > 256 || a.Dv > 256) return EIA_UNSUPPORTED;
  const int vec = a.Dv % 4 == 0 && reinterpret_cast<uintptr_t>(a.S) % 16 == 0;
  const dim3 grid(nseq, a.H);
#define DS_GO(LG, R) \
  hipLaunchKernelGGL((delta_scan_kernel<T, LG, R>), grid, dim3(256), 0, st, a, vec)
#define DS_ROWS(LG, R)                                                                \
  do {                                                                                \
    if (a.D <= 64) DS_GO(LG, R); else if (a.D <= 128) DS_GO(LG, 2 * R);               \
    else DS_GO(LG, 4 * R);                                                            \
  } while (0)
  if (a.Dv <= 64) DS_ROWS(4, 4); else if (a.Dv <= 128) DS_ROWS(5, 8); else DS_ROWS(6, 16);
#undef DS_ROWS
#undef DS_GO
  EIA_LAUNCH_CHECK();
}

// q, k [rows, G, DP], v [rows, H, VP] (fp32, zero past D / Dv), la, beta [rows, H]: the rows that
// eia_delta_prep leaves; g [rows, >= H * Dv], norm_w [Dv] and y [rows, >= H * Dv] are bf16 when
// is_bf16, else fp32; S fp32 [slots, H, D, Dv].
EIA_API int eia_delta_scan(const float* q, const float* k, const float* v, const float* la,
                           const float* beta, int H, int G, int D, int Dv, int DP, int VP,
                           const void* g, long ldg, const void* norm_w, float out_scale, float eps,
                           float* S, const int* slots, const int* cu, const int* positions,
                           const int* seq_lens, void* y, long ldy, int nseq, int is_bf16,
                           hipStream_t st) {
  DeltaArgs a{q, k, v, la, beta, H, G, D, Dv, DP, VP, g, ldg, norm_w, out_scale, eps, S, slots, cu,
              positions, seq_lens, y, ldy};
  if (!delta_args_ok(a, nseq)) return EIA_BAD_SHAPE;
  if (nseq == 0) return EIA_OK;
  return is_bf16 ? delta_step<bf16_t>(a, nseq, st) : delta_step<float>(a, nseq, st);
}

// ---------------------------------------------------------------------------------------------
// Chunk-parallel form for prompt portions (dk, dv <= 128).  A step's rows are cut into chunks of DC
// tokens (never across sequences).  With A_t the running sum of la inside a chunk and S the state
// before it, the chunk's updates solve a unit lower triangular system,
//
//   u_t + sum_(s<t) L_ts u_s = b_t v_t - b_t exp(A_t) S^T k_t,    L_ts = b_t exp(A_t - A_s) k_t . k_s
//
// whose right side is linear in S:  u = X - Y S  with (I + L) X = diag(b) V and
// (I + L) Y = diag(b exp(A)) K.
//   (1) X, Y of every chunk, in parallel (block forward substitution, 16-token blocks whose diagonal
//       inverses are formed first)
//   (2) a sequence's chunks in order, in parallel over heads and 16-column slices of the state:
//       u = X - Y S (replaces X), S <- exp(A_end) S + sum_t exp(A_end - A_t) k_t u_t^T
//   (3) outputs of every chunk, in parallel:
//       o_t = exp(A_t) S^T q_t + sum_(s<=t) exp(A_t - A_s) (q_t . k_s) u_s
// Every exponent is <= 0.  All products are fp32 matrix-core products (16x16x4): an accumulator's
// registers (row 4 (lane / 16) + i, column lane % 16) are, step i, the B operand of a product over
// its rows, so X, Y, u and S go from one product to the next in registers; an A operand's lane reads
// four consecutive k as one 16-byte access.
constexpr int DC = 64;                      // tokens per chunk
constexpr int DL = DC + 4;                  // LDS row pitch of the triangular blocks

struct DeltaChunkArgs {
  const int* chunks;                        // [nchunk, 4]: sequence, first row, tokens, unused
  const int* seq_first;                     // [nseq + 1]: first chunk of every sequence
  float* Y; float* X;                       // [rows, H, DP], [rows, H, VP]
  float* wsS;                               // [nchunk, H, DP, VP]: the state before each chunk
  float* cA; float* wsG;                    // [rows, H] running sums, [nchunk, H] their last
};

EIA_DEV f32x4 mm(f32x4 a, f32x4 b, f32x4 c) {          // four steps of a 16x16 product
#pragma unroll
  for (int i = 0; i < 4; ++i) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], b[i], c, 0, 0, 0);
  return c;
}

__global__ void __launch_bounds__(256)
delta_chunk_solve_kernel(DeltaArgs a, DeltaChunkArgs c) {
  __shared__ __align__(16) float Ls[DC][DL];           // -L
  __shared__ __align__(16) float Ts[4][16][20];        // inverses of the diagonal blocks
  __shared__ float sA[DC], sb[DC];
  const int ch = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int s = c.chunks[4 * ch], row0 = c.chunks[4 * ch + 1], n = c.chunks[4 * ch + 2];
  if (a.slots[s] < 0) return;
  const int H = a.H, G = a.G, DP = a.DP, VP = a.VP, kh = h / (H / G);
  const int g4 = lane >> 4, l16 = lane & 15;
  if (wave == 0) {                                     // running sums of the log decays
    float la = lane < n ? a.la[(long)(row0 + lane) * H + h] : 0.f;
#pragma unroll
    for (int o = 1; o < DC; o <<= 1) {
      const float up = __shfl_up(la, o, 64);
      if (lane >= o) la += up;
    }
    sA[lane] = la;
    sb[lane] = lane < n ? a.beta[(long)(row0 + lane) * H + h] : 0.f;
    if (lane < n) c.cA[(long)(row0 + lane) * H + h] = la;
    if (lane == n - 1) c.wsG[(long)ch * H + h] = la;
  }
  __syncthreads();
  const long ldk = (long)G * DP, ldv = (long)H * VP, ldx = (long)H * DP;
  const float* K = a.k + (long)kh * DP;
  const int nb = DP >> 4;
  {                                                    // rows 16 wave .. of -L
    const float* ka = K + (long)(row0 + min(16 * wave + l16, n - 1)) * ldk + 4 * g4;
    f32x4 kf[8];
#pragma unroll
    for (int b = 0; b < 8; ++b)
      if (b < nb) kf[b] = *reinterpret_cast<const f32x4*>(ka + 16 * b);
    for (int st = 0; st <= wave; ++st) {
      const float* kb = K + (long)(row0 + min(16 * st + l16, n - 1)) * ldk + 4 * g4;
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int b = 0; b < 8; ++b)
        if (b < nb) acc = mm(kf[b], *reinterpret_cast<const f32x4*>(kb + 16 * b), acc);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = 16 * wave + 4 * g4 + i, u = 16 * st + l16;
        Ls[t][u] = u < t ? -sb[t] * expf(sA[t] - sA[u]) * acc[i] : 0.f;
      }
    }
  }
  __syncthreads();
  {                                                    // column l16 of the wave's diagonal inverse
    float x[16];
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      float v = r == l16 ? 1.f : 0.f;
#pragma unroll
      for (int u = 0; u < r; ++u) v += Ls[16 * wave + r][16 * wave + u] * x[u];
      x[r] = v;
    }
    if (lane < 16) {
#pragma unroll
      for (int r = 0; r < 16; ++r) Ts[wave][r][l16] = x[r];
    }
  }
  __syncthreads();
  f32x4 lf[4][4], tf[4];                               // A operands: blocks of -L, inverses
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    tf[i] = *reinterpret_cast<const f32x4*>(&Ts[i][l16][4 * g4]);
#pragma unroll
    for (int k = 0; k < i; ++k) lf[i][k] = *reinterpret_cast<const f32x4*>(&Ls[16 * i + l16][16 * k + 4 * g4]);
  }
  float eb[4][4], bb[4][4];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int t = 16 * i + 4 * g4 + e;
      bb[i][e] = sb[t];
      eb[i][e] = sb[t] * expf(sA[t]);
    }
  const int nct = nb + (VP >> 4);
  for (int ct = wave; ct < nct; ct += 4) {             // 16 columns of Y, then of X
    const bool isy = ct < nb;
    const float* src = isy ? K + 16 * ct : a.v + (long)h * VP + 16 * (ct - nb);
    float* dst = isy ? c.Y + (long)h * DP + 16 * ct : c.X + (long)h * VP + 16 * (ct - nb);
    const long lds_ = isy ? ldk : ldv, ldd = isy ? ldx : ldv;
    f32x4 B[4], X[4];
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int t = 16 * i + 4 * g4 + e;
        B[i][e] = src[(long)(row0 + min(t, n - 1)) * lds_ + l16] * (isy ? eb[i][e] : bb[i][e]);
      }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      f32x4 r = B[i];
#pragma unroll
      for (int k = 0; k < i; ++k) r = mm(lf[i][k], X[k], r);
      X[i] = mm(tf[i], r, f32x4{0.f, 0.f, 0.f, 0.f});
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int t = 16 * i + 4 * g4 + e;
        if (t < n) dst[(long)(row0 + t) * ldd + l16] = X[i][e];
      }
    }
  }
}

// (2) one workgroup per (sequence, head, 16 state columns).  Wave w owns tokens 16 w .. of u and state
// row tiles w and w + 4; u and S pass between the waves through LDS.  The next chunk's operands are
// in flight while this one is worked on.
template <int NB>                                      // row tiles of the state (DP / 16 <= NB)
__global__ void __launch_bounds__(256)
delta_chunk_scan_kernel(DeltaArgs a, DeltaChunkArgs c) {
  constexpr int OWN = (NB + 3) / 4;
  __shared__ __align__(16) f32x4 Ss[NB][64];
  __shared__ __align__(16) f32x4 Us[4][64];
  const int s = blockIdx.x, h = blockIdx.y, cb = blockIdx.z;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g4 = lane >> 4, l16 = lane & 15;
  const int slot = a.slots[s];
  if (slot < 0) return;
  const int c0 = c.seq_first[s], c1 = c.seq_first[s + 1];
  if (c1 <= c0) return;
  const int H = a.H, G = a.G, D = a.D, Dv = a.Dv, DP = a.DP, VP = a.VP, kh = h / (H / G);
  const int nb = DP >> 4, col = 16 * cb + l16;
  const bool fresh = a.positions[c.chunks[4 * c0 + 1]] == 0;
  float* Sg = a.S + ((long)slot * H + h) * D * Dv;
  f32x4 S[OWN];
#pragma unroll
  for (int o = 0; o < OWN; ++o) {
    const int tl = wave + 4 * o;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int r = 16 * tl + 4 * g4 + i;
      S[o][i] = (!fresh && r < D && col < Dv) ? Sg[(long)r * Dv + col] : 0.f;
    }
    if (tl < nb) Ss[tl][lane] = S[o];
  }
  const long ldk = (long)G * DP, ldv = (long)H * VP, ldx = (long)H * DP;
  const float* K = a.k + (long)kh * DP;
  struct Op { f32x4 y[NB], x; float k[OWN][16]; float ca[4], ga; int row0, n; };
  auto load = [&](int ch, Op& p) {
    p.row0 = c.chunks[4 * ch + 1];
    p.n = c.chunks[4 * ch + 2];
    p.ga = c.wsG[(long)ch * H + h];
    const float* yp = c.Y + (long)(p.row0 + min(16 * wave + l16, p.n - 1)) * ldx + (long)h * DP + 4 * g4;
#pragma unroll
    for (int b = 0; b < NB; ++b)
      p.y[b] = *reinterpret_cast<const f32x4*>(yp + 16 * (b < nb ? b : 0));
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const long r = p.row0 + min(16 * wave + 4 * g4 + i, p.n - 1);
      p.x[i] = c.X[r * ldv + (long)h * VP + col];
      p.ca[i] = c.cA[r * H + h];
    }
#pragma unroll
    for (int o = 0; o < OWN; ++o) {
      const int d = 16 * (wave + 4 * o < nb ? wave + 4 * o : 0) + l16;
#pragma unroll
      for (int t = 0; t < 16; ++t)                     // token 16 (t / 4) + 4 g4 + t % 4
        p.k[o][t] = K[(long)(p.row0 + min(16 * (t >> 2) + 4 * g4 + (t & 3), p.n - 1)) * ldk + d];
    }
  };
  Op cur, nxt;
  load(c0, cur);
  __syncthreads();
  for (int ch = c0; ch < c1; ++ch) {
    load(ch + 1 < c1 ? ch + 1 : ch, nxt);
    // the state before the chunk, for the outputs
    float* w = c.wsS + ((long)ch * H + h) * DP * VP;
#pragma unroll
    for (int o = 0; o < OWN; ++o)
      if (wave + 4 * o < nb) {
#pragma unroll
        for (int i = 0; i < 4; ++i) w[(long)(16 * (wave + 4 * o) + 4 * g4 + i) * VP + col] = S[o][i];
      }
    f32x4 acc[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
    for (int b = 0; b < NB; ++b)
      if (b < nb) acc[b & 1] = mm(cur.y[b], Ss[b][lane], acc[b & 1]);
    f32x4 us;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = 16 * wave + 4 * g4 + i;
      const float u = cur.x[i] - acc[0][i] - acc[1][i];
      if (t < cur.n) c.X[(long)(cur.row0 + t) * ldv + (long)h * VP + col] = u;
      us[i] = t < cur.n ? u * expf(cur.ga - cur.ca[i]) : 0.f;
    }
    Us[wave][lane] = us;
    __syncthreads();
    const float eg = expf(cur.ga);
#pragma unroll
    for (int o = 0; o < OWN; ++o) {
      f32x4 v0 = S[o] * eg, v1 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int tt = 0; tt < 4; ++tt) {
        const f32x4 kv = {cur.k[o][4 * tt], cur.k[o][4 * tt + 1], cur.k[o][4 * tt + 2],
                          cur.k[o][4 * tt + 3]};
        if (tt & 1) v1 = mm(kv, Us[tt][lane], v1); else v0 = mm(kv, Us[tt][lane], v0);
      }
      S[o] = v0 + v1;
      if (wave + 4 * o < nb) Ss[wave + 4 * o][lane] = S[o];
    }
    __syncthreads();
    cur = nxt;
  }
#pragma unroll
  for (int o = 0; o < OWN; ++o)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int r = 16 * (wave + 4 * o) + 4 * g4 + i;
      if (r < D && col < Dv) Sg[(long)r * Dv + col] = S[o][i];
    }
}

// (3) one workgroup per (chunk, head); wave w owns queries 16 w ..
template <typename T, int NV>                          // value column tiles (VP / 16 <= NV)
__global__ void __launch_bounds__(256)
delta_chunk_out_kernel(DeltaArgs a, DeltaChunkArgs c) {
  __shared__ float sA[DC];
  const int ch = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int s = c.chunks[4 * ch], row0 = c.chunks[4 * ch + 1], n = c.chunks[4 * ch + 2];
  if (a.slots[s] < 0) return;
  const int H = a.H, G = a.G, Dv = a.Dv, DP = a.DP, VP = a.VP, kh = h / (H / G);
  const int g4 = lane >> 4, l16 = lane & 15, nb = DP >> 4, nv = VP >> 4;
  if (tid < DC) sA[tid] = c.cA[(long)(row0 + min(tid, n - 1)) * H + h];
  __syncthreads();
  if (16 * wave >= n) return;
  const long ldk = (long)G * DP, ldv = (long)H * VP;
  const int tq = 16 * wave + l16;                      // this lane's query
  const float* qp = a.q + (long)(row0 + min(tq, n - 1)) * ldk + (long)kh * DP + 4 * g4;
  f32x4 qf[8];
#pragma unroll
  for (int b = 0; b < 8; ++b)
    if (b < nb) qf[b] = *reinterpret_cast<const f32x4*>(qp + 16 * b);
  f32x4 o[NV];
#pragma unroll
  for (int t = 0; t < NV; ++t) o[t] = f32x4{0.f, 0.f, 0.f, 0.f};
  // weights of the chunk's own tokens: P^T = K Q^T, so that its registers are the A operand of P u
  for (int kt = 0; kt <= wave; ++kt) {
    const float* kp = a.k + (long)(row0 + min(16 * kt + l16, n - 1)) * ldk + (long)kh * DP + 4 * g4;
    f32x4 p = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int b = 0; b < 8; ++b)
      if (b < nb) p = mm(*reinterpret_cast<const f32x4*>(kp + 16 * b), qf[b], p);
    const float* up[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int tk = 16 * kt + 4 * g4 + i;
      p[i] = tk <= tq && tk < n ? p[i] * expf(sA[tq] - sA[tk]) : 0.f;
      up[i] = c.X + (long)(row0 + min(tk, n - 1)) * ldv + (long)h * VP + l16;
    }
#pragma unroll
    for (int t = 0; t < NV; ++t) {
      const int ct = t < nv ? t : 0;
      o[t] = mm(p, f32x4{up[0][16 * ct], up[1][16 * ct], up[2][16 * ct], up[3][16 * ct]}, o[t]);
    }
  }
  const float eA = expf(sA[tq]);
  const float* Sb = c.wsS + ((long)ch * H + h) * DP * VP + (long)4 * g4 * VP + l16;
#pragma unroll
  for (int b = 0; b < 8; ++b) {
    if (b >= nb) break;
    const f32x4 qa = qf[b] * eA;
    const float* sp = Sb + (long)16 * b * VP;
#pragma unroll
    for (int t = 0; t < NV; ++t) {
      const int ct = 16 * (t < nv ? t : 0);
      o[t] = mm(qa, f32x4{sp[ct], sp[VP + ct], sp[2 * VP + ct], sp[3 * VP + ct]}, o[t]);
    }
  }
  // head RMS norm (columns past Dv are zero), weight, gate
  const T* NW = static_cast<const T*>(a.norm_w);
  const T* GT = static_cast<const T*>(a.g);
  T* Yo = static_cast<T*>(a.y);
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    float ss = 0.f;
#pragma unroll
    for (int t = 0; t < NV; ++t) ss += t < nv ? o[t][i] * o[t][i] : 0.f;
    ss += __shfl_xor(ss, 1, 64);
    ss += __shfl_xor(ss, 2, 64);
    ss += __shfl_xor(ss, 4, 64);
    ss += __shfl_xor(ss, 8, 64);
    const int tr = 16 * wave + 4 * g4 + i;
    if (tr >= n) continue;
    const float inv = a.out_scale / sqrtf(ss / (float)Dv + a.eps);
    const long r = row0 + tr;
#pragma unroll
    for (int t = 0; t < NV; ++t) {
      const int d = 16 * t + l16;
      if (d < Dv)
        st_f32<T>(Yo + r * a.ldy, (long)h * Dv + d,
                  o[t][i] * inv * ld_f32<T>(NW, d) * dl_silu(ld_f32<T>(GT + r * a.ldg, (long)h * Dv + d)));
    }
  }
}

// As eia_delta_scan for sequences whose chunk list is given (chunks int32 [nchunk, 4]: sequence,
// first row, tokens (1 .. 64), 0; seq_first int32 [nseq + 1], indexed by sequence), with fp32
// workspaces Y [rows, H, DP], X [rows, H, VP], wsS [nchunk, H, DP, VP], cA [rows, H],
// wsG [nchunk, H]; DP and VP multiples of 16, at most 128.
EIA_API int eia_delta_scan_chunked(const float* q, const float* k, const float* v, const float* la,
                                   const float* beta, int H, int G, int D, int Dv, int DP, int VP,
                                   const void* g, long ldg, const void* norm_w, float out_scale,
                                   float eps, float* S, const int* slots, const int* positions,
                                   void* y, long ldy, int nseq, const int* chunks,
                                   const int* seq_first, int nchunk, float* Y, float* X, float* wsS,
                                   float* cA, float* wsG, int is_bf16, hipStream_t st) {
  DeltaArgs a{q, k, v, la, beta, H, G, D, Dv, DP, VP, g, ldg, norm_w, out_scale, eps, S, slots,
              nullptr, positions, nullptr, y, ldy};
  if (!delta_args_ok(a, nseq) || nchunk < 0 || !chunks || !seq_first || !Y || !X || !wsS || !cA ||
      !wsG || DP % 16 || VP % 16)
    return EIA_BAD_SHAPE;
  if (DP > 128 || VP > 128) return EIA_UNSUPPORTED;
  if (nseq == 0 || nchunk == 0) return EIA_OK;
  DeltaChunkArgs c{chunks, seq_first, Y, X, wsS, cA, wsG};
  const dim3 gc(nchunk, H), gs(nseq, H, VP / 16);
  hipLaunchKernelGGL(delta_chunk_solve_kernel, gc, dim3(256), 0, st, a, c);
  if (DP <= 64) hipLaunchKernelGGL((delta_chunk_scan_kernel<4>), gs, dim3(256), 0, st, a, c);
  else hipLaunchKernelGGL((delta_chunk_scan_kernel<8>), gs, dim3(256), 0, st, a, c);
#define DO_GO(TT, NV) \
  hipLaunchKernelGGL((delta_chunk_out_kernel<TT, NV>), gc, dim3(256), 0, st, a, c)
  if (is_bf16) { if (VP <= 64) DO_GO(bf16_t, 4); else DO_GO(bf16_t, 8); }
  else { if (VP <= 64) DO_GO(float, 4); else DO_GO(float, 8); }
#undef DO_GO
  EIA_LAUNCH_CHECK();
}
