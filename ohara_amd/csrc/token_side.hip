// A layer's own embedding of the row's token, gated by the residual, with the residual updates on either side of it, in one launch:
//
//   x += norm(y);   z = gelu_tanh(Wg x) * e;   x += rms(Wp z) * side_w;   out = norm(x)
//
// with the roundings of the separate launches (x, z and Wp z to bf16, everything else fp32).  A workgroup of 16 waves owns R rows.
// Norms and updates: 16 / R waves per row, the row's residual stays in registers throughout.  First product: a wave takes a share of
// the columns of x for all outputs, the shares meet in LDS.  Second product: a wave takes every 16th strip of outputs.
#include "hybrid.h"

namespace {

struct SideArgs {
  float* x;
  const bf16_t* y;
  const float* norm_w;
  const uint4* wg;
  const uint4* wp;
  const bf16_t* table;
  const int64_t* ids;
  const float* side_w;
  const float* out_w;
  bf16_t* out;
  int d, dp, n, ldt, vocab, ldy, ldo, rows, R;  // dp: d rounded up to 8
  int center_y, center_out;
  float eps;
};

constexpr int SIDE_GS = 4;  // strips of 16 outputs of the first product worked on together

__host__ __device__ inline size_t side_tile_bytes(int R, int dp) { return (size_t)R * (dp + 8) * sizeof(bf16_t); }
__host__ __device__ inline size_t side_gate_bytes(int R, int n) { return (size_t)R * (((n + 31) & ~31) + 8) * sizeof(bf16_t); }

// four bf16 values in LDS (ld4 / st4 address device memory)
__device__ __forceinline__ void lds_put4(bf16_t* p, const float* v) {
  *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf(v[0], v[1]), pack_bf(v[2], v[3]));
}
__device__ __forceinline__ void lds_get4(const bf16_t* p, float* v) {
  const uint2 w = *reinterpret_cast<const uint2*>(p);
  v[0] = lo_bf(w.x); v[1] = hi_bf(w.x); v[2] = lo_bf(w.y); v[3] = hi_bf(w.y);
}

// NP: pieces of four columns per thread
template <int NP>
__global__ __launch_bounds__(1024) void token_side_kernel(SideArgs a) {
  constexpr bool EARLY = NP <= 2;  // registers for the weights of the later steps are there
  constexpr int GS = SIDE_GS, CH = 2;
  extern __shared__ __align__(16) unsigned char side_smem[];
  __shared__ float red[5][16];
  const int tid = threadIdx.x, lane = tid & 63, m = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int d = a.d, dp = a.dp, R = a.R, wpr = 16 / R, lda = dp + 8, np = (a.n + 31) & ~31, ldg = np + 8;
  bf16_t* At = reinterpret_cast<bf16_t*>(side_smem);                                  // [R][lda]: x, later Wp z
  bf16_t* Zt = reinterpret_cast<bf16_t*>(side_smem + side_tile_bytes(R, dp));         // [R][ldg]
  float* Ps = reinterpret_cast<float*>(side_smem + side_tile_bytes(R, dp) + side_gate_bytes(R, a.n));  // [16][GS][256]
  const int row0 = blockIdx.x * R, r = wave / wpr, sub = wave - r * wpr, row = row0 + r;
  const bool live = row < a.rows;
  const int KS = (dp + 31) >> 5, per = (KS + 15) / 16, j0 = wave * per, j1 = min(KS, j0 + per);
  const int strips = (a.n + 15) / 16;
  auto col = [&](int p) { return 4 * (sub * 64 + lane) + 256 * wpr * p; };

  float x[NP][4], y[NP][4], w[NP][4], sw[EARLY ? NP : 1][4], ow[EARLY ? NP : 1][4];
  float* xr = a.x + (size_t)row * d;
#pragma unroll
  for (int p = 0; p < NP; ++p) {
    const int i = col(p);
#pragma unroll
    for (int u = 0; u < 4; ++u) x[p][u] = y[p][u] = w[p][u] = 0.f;
    if (!live || i >= d) continue;
    ld4(xr + i, x[p]);
    ld4(a.y + (size_t)row * a.ldy + i, y[p]);
    ld4(a.norm_w + i, w[p]);
    if constexpr (EARLY) {
      ld4(a.side_w + i, sw[p]);
      ld4(a.out_w + i, ow[p]);
    }
  }
  // first product's weights and this thread's entry of the embedding: they wait for nothing
  uint4 wl[GS][CH];
  auto load_gate = [&](int s0, int j) {
#pragma unroll
    for (int s = 0; s < GS; ++s)
#pragma unroll
      for (int c = 0; c < CH; ++c) wl[s][c] = ldg16(a.wg + ((size_t)min(s0 + s, strips - 1) * KS + min(j + c, KS - 1)) * 64 + lane);
  };
  if constexpr (EARLY) load_gate(0, j0);
  const int zl = (tid >> 2) & 63, zr = zl & 15, zc = 16 * (tid >> 8) + 4 * (zl >> 4) + (tid & 3);  // row and output of the sums below
  const bf16_t* erow = a.table;
  if (zr < R && row0 + zr < a.rows) {
    int64_t id = a.ids[row0 + zr];
    if (id < 0 || id >= a.vocab) id = 0;  // the host validates ids; never read out of bounds
    erow += (size_t)id * a.ldt;
  }
  auto row_sum = [&](float v, int slot) {
    v = wave_sum(v);
    if (lane == 0) red[slot][wave] = v;
    __syncthreads();
    float t = red[slot][r * wpr];
    for (int k = 1; k < wpr; ++k) t += red[slot][r * wpr + k];
    return t;
  };
  auto total = [&](float (&v)[NP][4]) {
    float t = 0.f;
#pragma unroll
    for (int p = 0; p < NP; ++p) t += ((v[p][0] + v[p][1]) + v[p][2]) + v[p][3];  // zeros past the row's end
    return t;
  };
  auto squares = [&](float (&v)[NP][4]) {
    float t = 0.f;
#pragma unroll
    for (int p = 0; p < NP; ++p) t += ((v[p][0] * v[p][0] + v[p][1] * v[p][1]) + v[p][2] * v[p][2]) + v[p][3] * v[p][3];
    return t;
  };
  auto take_off = [&](float (&v)[NP][4], float mean) {
#pragma unroll
    for (int p = 0; p < NP; ++p)
#pragma unroll
      for (int u = 0; u < 4; ++u) v[p][u] = col(p) < d ? v[p][u] - mean : 0.f;
  };

  // ---- x += norm(y) ----
  if (a.center_y) take_off(y, row_sum(total(y), 0) / (float)d);
  const float iy = 1.0f / sqrtf(row_sum(squares(y), 1) / (float)d + a.eps);
#pragma unroll
  for (int p = 0; p < NP; ++p) {
    const int i = col(p);
#pragma unroll
    for (int u = 0; u < 4; ++u) x[p][u] += y[p][u] * iy * w[p][u];
    if (i < dp) lds_put4(At + r * lda + i, x[p]);  // columns d .. dp-1: zeros
  }
  for (int i = tid; i < R * (np - a.n); i += 1024) Zt[(i / (np - a.n)) * ldg + a.n + i % (np - a.n)] = 0;
  __syncthreads();

  // ---- z = gelu(Wg x) * e ----
  const uint4 zero = make_uint4(0, 0, 0, 0);
  for (int s0 = 0; s0 < strips; s0 += GS) {
    const float e = zr < R && 16 * s0 + zc < a.n ? bf2f(erow[16 * s0 + zc]) : 0.f;
    f32x4 acc[GS];
#pragma unroll
    for (int s = 0; s < GS; ++s) acc[s] = (f32x4){0.f, 0.f, 0.f, 0.f};
    for (int j = j0; j < j1; j += CH) {
      uint4 xv[CH];
      if (!(EARLY && s0 == 0 && j == j0)) load_gate(s0, j);
#pragma unroll
      for (int c = 0; c < CH; ++c) {
        const int k0 = 32 * (j + c) + 8 * g;
        const bool in = m < R && j + c < j1 && k0 < dp;
        const uint4 v = lds16(At + (in ? m * lda + k0 : 0));
        xv[c] = in ? v : zero;
      }
#pragma unroll
      for (int c = 0; c < CH; ++c)
#pragma unroll
        for (int s = 0; s < GS; ++s)
          acc[s] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, wl[s][c]), __builtin_bit_cast(bf16x8, xv[c]),
                                                           acc[s], 0, 0, 0);
    }
#pragma unroll
    for (int s = 0; s < GS; ++s) *reinterpret_cast<f32x4*>(Ps + (wave * GS + s) * 256 + 4 * lane) = acc[s];
    __syncthreads();
    float t = Ps[tid];
#pragma unroll
    for (int k = 1; k < 16; ++k) t += Ps[k * GS * 256 + tid];
    if (zr < R && 16 * s0 + zc < a.n) Zt[zr * ldg + 16 * s0 + zc] = f2bf(gelu_tanh(t) * e);
    __syncthreads();
  }

  // ---- Wp z, over the tile of x ----
  const int K2 = np >> 5, N2 = (dp + 15) / 16;
  for (int s0 = wave; s0 < N2; s0 += 16 * GS) {
    f32x4 acc[GS];
#pragma unroll
    for (int s = 0; s < GS; ++s) acc[s] = (f32x4){0.f, 0.f, 0.f, 0.f};
    for (int j = 0; j < K2; j += 2) {
      uint4 pl[GS][2], zv[2];
#pragma unroll
      for (int s = 0; s < GS; ++s)
#pragma unroll
        for (int c = 0; c < 2; ++c) pl[s][c] = ldg16(a.wp + ((size_t)min(s0 + 16 * s, N2 - 1) * K2 + min(j + c, K2 - 1)) * 64 + lane);
#pragma unroll
      for (int c = 0; c < 2; ++c) {
        const bool in = m < R && j + c < K2;
        const uint4 v = lds16(Zt + (in ? m * ldg + 32 * (j + c) + 8 * g : 0));
        zv[c] = in ? v : zero;
      }
#pragma unroll
      for (int c = 0; c < 2; ++c)
#pragma unroll
        for (int s = 0; s < GS; ++s)
          acc[s] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, pl[s][c]), __builtin_bit_cast(bf16x8, zv[c]),
                                                           acc[s], 0, 0, 0);
    }
#pragma unroll
    for (int s = 0; s < GS; ++s) {
      const int c = 16 * (s0 + 16 * s) + 4 * g;
      const float v[4] = {acc[s][0], acc[s][1], acc[s][2], acc[s][3]};
      if (m < R && c < dp) lds_put4(At + m * lda + c, v);
    }
  }
  __syncthreads();

  // ---- x += rms(Wp z) * side_w;  out = norm(x) ----
#pragma unroll
  for (int p = 0; p < NP; ++p) {
    const int i = col(p);
#pragma unroll
    for (int u = 0; u < 4; ++u) y[p][u] = 0.f;
    if (i >= d) continue;
    lds_get4(At + r * lda + i, y[p]);
    if constexpr (EARLY) {
#pragma unroll
      for (int u = 0; u < 4; ++u) w[p][u] = sw[p][u];
    } else {
      ld4(a.side_w + i, w[p]);
    }
  }
  const float is = 1.0f / sqrtf(row_sum(squares(y), 2) / (float)d + a.eps);
#pragma unroll
  for (int p = 0; p < NP; ++p) {
    const int i = col(p);
#pragma unroll
    for (int u = 0; u < 4; ++u) x[p][u] += y[p][u] * is * w[p][u];
    if (live && i < d) {
      st4(xr + i, x[p]);
      if constexpr (EARLY) {
#pragma unroll
        for (int u = 0; u < 4; ++u) w[p][u] = ow[p][u];
      } else {
        ld4(a.out_w + i, w[p]);
      }
    }
  }
  if (a.center_out) take_off(x, row_sum(total(x), 3) / (float)d);
  const float io = 1.0f / sqrtf(row_sum(squares(x), 4) / (float)d + a.eps);
  if (!live) return;
  bf16_t* o = a.out + (size_t)row * a.ldo;
  for (int i = d + sub * 64 + lane; i < a.ldo; i += 64 * wpr) o[i] = 0;
#pragma unroll
  for (int p = 0; p < NP; ++p) {
    const int i = col(p);
    if (i >= d) continue;
    float v[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) v[u] = x[p][u] * io * w[p][u];
    st4(o + i, v);
  }
}

template <int NP>
int launch_side(const SideArgs& a, hipStream_t st) {
  const size_t smem = side_tile_bytes(a.R, a.dp) + side_gate_bytes(a.R, a.n) + (size_t)16 * SIDE_GS * 256 * sizeof(float);
  (void)hipFuncSetAttribute((const void*)token_side_kernel<NP>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
  hipLaunchKernelGGL((token_side_kernel<NP>), dim3((unsigned)((a.rows + a.R - 1) / a.R)), dim3(1024), smem, st, a);
  return ohara_launch_status();
}

}  // namespace

extern "C" int ohara_token_side_bf16(float* x, int d, const uint16_t* y, int ldy, const float* norm_w, int center_y,
                                     const uint16_t* gate, const uint16_t* proj, int n, const uint16_t* table, int ldt,
                                     const int64_t* ids, int vocab, const float* side_w, float eps, const float* out_w, int center_out,
                                     int rows, int rows_per_group, uint16_t* out, int ldo, void* stream) {
  if (!x || !y || !norm_w || !gate || !proj || !table || !ids || !side_w || !out_w || !out) return OHARA_EINVAL;
  if (d < 1 || n < 1 || rows < 1 || vocab < 1 || ldy < d || ldt < n || ldo < d) return OHARA_EINVAL;
  if ((d & 3) || (ldy & 3) || (ldo & 3)) return OHARA_EINVAL;  // 8- and 16-byte accesses
  const int R = rows_per_group, dp = (d + 7) & ~7;
  if (R != 1 && R != 2 && R != 4 && R != 8 && R != 16) return OHARA_EINVAL;
  if (n > 256 || (int64_t)R * d > 16384) return OHARA_ESIZE;
  const SideArgs a{x, y, norm_w, reinterpret_cast<const uint4*>(gate), reinterpret_cast<const uint4*>(proj), table, ids, side_w, out_w,
                   out, d, dp, n, ldt, vocab, ldy, ldo, rows, R, center_y != 0, center_out != 0, eps};
  const int pieces = (d * R + 4095) / 4096;  // of a thread
  hipStream_t st = (hipStream_t)stream;
  return pieces <= 1 ? launch_side<1>(a, st) : (pieces <= 2 ? launch_side<2>(a, st) : launch_side<4>(a, st));
}
