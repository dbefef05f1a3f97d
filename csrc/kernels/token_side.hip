// End of a layer whose gated sublayers join an fp32 residual and whose per-layer token input
// follows, for prompt-sized batches (bf16): ONE launch per layer end, 16 token rows a workgroup.
//
//   x += y1 * sigmoid(g1) + y2 * sigmoid(g2)                      (y2 optional)
//   y  = W_proj (gelu_tanh(W_gate x) * table[ids, col0 .. col0 + N])
//   x += y / sqrt(mean(y^2) + eps) * w_side
//   h  = x / sqrt(mean(x^2) + eps) * w_next                       (h optional)
//
// The rows of a workgroup never leave it: the summed residual is kept as a bf16 tile in LDS for
// the first product (its fp32 form goes to memory and is read back behind the second one), the
// gated side values are a second LDS tile, and the output columns stay in the accumulators
// through both norms.  W_gate [NP, W] and W_proj [W, NP] (NP: N padded to a multiple of 128 with
// zero rows / columns) are read as matrix-core operands straight from L2, from copies packed in
// operand order -- [16-row tile][32-column step][lane r + 16 g][8]: row r of the tile, columns 8 g ..
// -- so that an operand is one contiguous KiB (row-major rows lie a power of two apart and would
// all meet in the same L2 channel).  Decode-sized batches
// (a workgroup per 16 rows would leave the chip empty) take the unfused launches.
#include "eia_common.h"

struct TokenSideArgs {
  float* x;
  const bf16_t* y1; long ld1; const bf16_t* g1; long lg1;
  const bf16_t* y2; long ld2; const bf16_t* g2; long lg2;
  const int* ids; const bf16_t* table; long ldt; int col0, vocab;
  const bf16_t* gate; const bf16_t* proj; const bf16_t* w_side; const bf16_t* w_next;
  bf16_t* h; long ldh;
  float eps;
  int rows, W, N, NP;
};

EIA_DEV float ts_sigmoid(float z) { return __builtin_amdgcn_rcpf(1.0f + __expf(-z)); }
EIA_DEV float ts_gelu_tanh(float z) {
  const float k0 = 0.7978845608028654f, k1 = 0.044715f;
  return 0.5f * z * (1.f + tanhf(k0 * (z + k1 * z * z * z)));
}
// sums v[i] over the 16 lanes of a column group; every lane gets its rows' totals
EIA_DEV f32x4 ts_sum16(f32x4 v) {
#pragma unroll
  for (int o = 8; o > 0; o >>= 1)
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] += __shfl_xor(v[i], o, 64);
  return v;
}

struct TsTrue { static constexpr bool value = true; };
struct TsFalse { static constexpr bool value = false; };

// NT: 16-column output tiles per wave (W <= 128 NT)
template <int NT>
__global__ void __launch_bounds__(512)
token_side_kernel(const TokenSideArgs a) {
  extern __shared__ char lds[];
  const int W = a.W, NP = a.NP;
  const int xp = W + 8, gp = NP + 8;                 // row pitches: 16 bytes past a bank round
  bf16_t* xs = reinterpret_cast<bf16_t*>(lds);       // [16][xp]
  bf16_t* gs = xs + 16 * xp;                         // [16][gp]
  __shared__ float red[2][8][16];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int c = lane & 15, g = lane >> 4;
  const long row0 = (long)blockIdx.x * 16;
  const int n = min(16, (int)(a.rows - row0));
  // (1) the gated residual sum, two rows a wave
#pragma unroll
  for (int q = 0; q < 2; ++q) {
    const int r = 2 * wave + q;
    bf16_t* xt = xs + r * xp;
    if (r >= n) {
      for (int k = 4 * lane; k < W; k += 256)
        *reinterpret_cast<bf16x4*>(xt + k) = bf16x4{f2bf(0.f), f2bf(0.f), f2bf(0.f), f2bf(0.f)};
      continue;
    }
    const long row = row0 + r;
    float* xr = a.x + row * W;
    const bf16_t* y1 = a.y1 + row * a.ld1;
    const bf16_t* g1 = a.g1 + row * a.lg1;
    const bf16_t* y2 = a.y2 ? a.y2 + row * a.ld2 : y1;
    const bf16_t* g2 = a.y2 ? a.g2 + row * a.lg2 : g1;
    const float two = a.y2 ? 1.f : 0.f;
    for (int k0 = 4 * lane; k0 < W; k0 += 1024) {      // four column steps' loads together
      f32x4 v[4];
      bf16x4 p[4][4];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int k = min(k0 + 256 * u, W - 4);
        v[u] = *reinterpret_cast<const f32x4*>(xr + k);
        p[u][0] = *reinterpret_cast<const bf16x4*>(y1 + k);
        p[u][1] = *reinterpret_cast<const bf16x4*>(g1 + k);
        p[u][2] = *reinterpret_cast<const bf16x4*>(y2 + k);
        p[u][3] = *reinterpret_cast<const bf16x4*>(g2 + k);
      }
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int k = k0 + 256 * u;
#pragma unroll
        for (int i = 0; i < 4; ++i)
          v[u][i] += bf2f(p[u][0][i]) * ts_sigmoid(bf2f(p[u][1][i])) +
                     two * bf2f(p[u][2][i]) * ts_sigmoid(bf2f(p[u][3][i]));
        if (k < W) {
          *reinterpret_cast<f32x4*>(xr + k) = v[u];
          *reinterpret_cast<bf16x4*>(xt + k) =
              bf16x4{f2bf(v[u][0]), f2bf(v[u][1]), f2bf(v[u][2]), f2bf(v[u][3])};
        }
      }
    }
  }
  __syncthreads();
  const bf16x8 zero8 = {0, 0, 0, 0, 0, 0, 0, 0};
  // (2) side values: tile (tokens 4 g + i) x (side channel 16 j + c)
  for (int j = wave; j < NP / 16; j += 8) {
    f32x4 u = {0.f, 0.f, 0.f, 0.f};
    const bf16_t* wr = a.gate + (long)j * 16 * W + 8 * lane;
    const bf16_t* xr = xs + c * xp + 8 * g;
    // eight steps' weights in flight ahead of the eight in use (a step past the row's end
    // repeats the last one against a zero operand)
    bf16x8 wv[8], wn[8];
    auto load = [&](int k0, bf16x8 (&d)[8]) {
#pragma unroll
      for (int q = 0; q < 8; ++q)
        d[q] = *reinterpret_cast<const bf16x8*>(wr + 16 * min(k0 + 32 * q, W - 32));
    };
    load(0, wn);
    for (int k0 = 0; k0 < W; k0 += 256) {
#pragma unroll
      for (int q = 0; q < 8; ++q) wv[q] = wn[q];
      load(k0 + 256, wn);
#pragma unroll
      for (int q = 0; q < 8; ++q) {
        const bf16x8 xv = *reinterpret_cast<const bf16x8*>(xr + min(k0 + 32 * q, W - 32));
        u = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k0 + 32 * q < W ? xv : zero8, wv[q], u, 0, 0, 0);
      }
    }
    const int col = 16 * j + c;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int r = 4 * g + i;
      float o = 0.f;
      if (r < n && col < a.N) {
        const int tok = min(max(a.ids[row0 + r], 0), a.vocab - 1);
        o = ts_gelu_tanh(u[i]) * bf2f(a.table[(long)tok * a.ldt + a.col0 + col]);
      }
      gs[r * gp + col] = f2bf(o);
    }
  }
  __syncthreads();
  // (3) y = G W_proj^T: this wave's column tiles wave, wave + 8, ...
  f32x4 y[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) y[t] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int tiles = W >> 4;
#pragma unroll 2
  for (int k = 0; k < NP; k += 32) {
    const bf16x8 ga = *reinterpret_cast<const bf16x8*>(gs + c * gp + k + 8 * g);
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const int tile = min(wave + 8 * t, tiles - 1); // (past the row's end: a repeat, not stored)
      y[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
          ga, *reinterpret_cast<const bf16x8*>(a.proj + (long)tile * 16 * NP + 16 * k + 8 * lane),
          y[t], 0, 0, 0);
    }
  }
  // (4) both norms.  Loads and stores run without a branch per tile (a row or tile past the end
  // repeats the last one's address and adds nothing to the sums), so they overlap.
  float live[4];                                     // rows of this lane that exist
  long xo[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    live[i] = 4 * g + i < n ? 1.f : 0.f;
    xo[i] = (row0 + min(4 * g + i, n - 1)) * W;
  }
  f32x4 ss = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int t = 0; t < NT; ++t) ss += y[t] * y[t] * (wave + 8 * t < tiles ? 1.f : 0.f);
  ss = ts_sum16(ss);
  if (c == 0) *reinterpret_cast<f32x4*>(&red[0][wave][4 * g]) = ss;
  // the summed residual (written in (1), other waves' rows included) of this lane's columns
  f32x4 xv[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const int col = 16 * min(wave + 8 * t, tiles - 1) + c;
#pragma unroll
    for (int i = 0; i < 4; ++i) xv[t][i] = a.x[xo[i] + col];
  }
  __syncthreads();
  f32x4 inv = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int w = 0; w < 8; ++w) inv += *reinterpret_cast<const f32x4*>(&red[0][w][4 * g]);
#pragma unroll
  for (int i = 0; i < 4; ++i) inv[i] = 1.0f / sqrtf(inv[i] / (float)W + a.eps);
  ss = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const bool on = wave + 8 * t < tiles;
    const float w = bf2f(a.w_side[16 * min(wave + 8 * t, tiles - 1) + c]);
    y[t] = xv[t] + y[t] * inv * w;
    ss += y[t] * y[t] * (on ? 1.f : 0.f);
  }
  auto store = [&](auto full) {
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      if (!decltype(full)::value && wave + 8 * t >= tiles) continue;
      const int col = 16 * (wave + 8 * t) + c;
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (decltype(full)::value || live[i] != 0.f) a.x[xo[i] + col] = y[t][i];
    }
  };
  const bool full = n == 16 && tiles == 8 * NT;      // (uniform)
  if (full) store(TsTrue{}); else store(TsFalse{});
  if (!a.h) return;
  ss = ts_sum16(ss);
  if (c == 0) *reinterpret_cast<f32x4*>(&red[1][wave][4 * g]) = ss;
  __syncthreads();
  inv = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int w = 0; w < 8; ++w) inv += *reinterpret_cast<const f32x4*>(&red[1][w][4 * g]);
#pragma unroll
  for (int i = 0; i < 4; ++i) inv[i] = 1.0f / sqrtf(inv[i] / (float)W + a.eps);
  // h through LDS (the residual tile is no longer read): rows leave as whole 8-byte units
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    if (wave + 8 * t >= tiles) break;                // (uniform)
    const int col = 16 * (wave + 8 * t) + c;
    const float w = bf2f(a.w_next[col]);
#pragma unroll
    for (int i = 0; i < 4; ++i) xs[(4 * g + i) * xp + col] = f2bf(y[t][i] * inv[i] * w);
  }
  __syncthreads();
#pragma unroll
  for (int q = 0; q < 2; ++q) {
    const int r = 2 * wave + q;
    if (r >= n) continue;
#pragma unroll 4
    for (int k = 4 * lane; k < W; k += 256)
      *reinterpret_cast<bf16x4*>(a.h + (row0 + r) * a.ldh + k) =
          *reinterpret_cast<const bf16x4*>(xs + r * xp + k);
  }
}

// Shapes of the fused form: W a multiple of 32 up to 2048, NP a multiple of 128 up to 512.
EIA_API int eia_token_side_ok(int W, int NP) {
  return W >= 32 && W % 32 == 0 && W <= 2048 && NP >= 128 && NP % 128 == 0 && NP <= 512;
}

EIA_API int eia_token_side(float* x, const void* y1, long ld1, const void* g1, long lg1,
                           const void* y2, long ld2, const void* g2, long lg2, const int* ids,
                           const void* table, long ldt, int col0, int vocab, const void* gate,
                           const void* proj, const void* w_side, const void* w_next, void* h,
                           long ldh, float eps, int rows, int W, int N, int NP, hipStream_t st) {
  if (rows < 0 || !x || !y1 || !g1 || (y2 && !g2) || !ids || !table || !gate || !proj || !w_side ||
      (h && !w_next) || N < 1 || N > NP || col0 < 0 || col0 + N > ldt || vocab < 1 || ld1 % 4 ||
      lg1 % 4 || ld2 % 4 || lg2 % 4)
    return EIA_BAD_SHAPE;
  if (!eia_token_side_ok(W, NP)) return EIA_UNSUPPORTED;
  if (ldh % 4 || reinterpret_cast<uintptr_t>(h) % 8) return EIA_BAD_SHAPE;
  const uintptr_t al = reinterpret_cast<uintptr_t>(y1) | reinterpret_cast<uintptr_t>(g1) |
                       reinterpret_cast<uintptr_t>(y2) | reinterpret_cast<uintptr_t>(g2);
  const uintptr_t al16 = reinterpret_cast<uintptr_t>(gate) | reinterpret_cast<uintptr_t>(proj);
  if (al % 8 || al16 % 16) return EIA_BAD_SHAPE;
  if (rows == 0) return EIA_OK;
  TokenSideArgs a{x, (const bf16_t*)y1, ld1, (const bf16_t*)g1, lg1, (const bf16_t*)y2, ld2,
                  (const bf16_t*)g2, lg2, ids, (const bf16_t*)table, ldt, col0, vocab,
                  (const bf16_t*)gate, (const bf16_t*)proj, (const bf16_t*)w_side,
                  (const bf16_t*)w_next, (bf16_t*)h, ldh, eps, rows, W, N, NP};
  const int lds = 16 * 2 * ((W + 8) + (NP + 8));
#define TS_LAUNCH(NT)                                                                           \
  do {                                                                                          \
    if (lds > 48 * 1024)                                                                        \
      (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&token_side_kernel<NT>),          \
                                hipFuncAttributeMaxDynamicSharedMemorySize, lds);               \
    hipLaunchKernelGGL(token_side_kernel<NT>, dim3((rows + 15) / 16), dim3(512), lds, st, a);   \
  } while (0)
  if (W <= 512) TS_LAUNCH(4);
  else if (W <= 1024) TS_LAUNCH(8);
  else TS_LAUNCH(16);
#undef TS_LAUNCH
  EIA_LAUNCH_CHECK();
}
