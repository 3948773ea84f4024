// Retention: linear attention with one fixed decay g per head.  Per head, S (dim x vdim, fp32) from zero:
//   S <- g S + k v^T;   o = S^T q;   out = o / rms(o) * silu(gate).
//
// retention_step_kernel: one token per sequence, a workgroup per (sequence, head).
//
// Prompts: chunks of C = 128 tokens, n of them in the last chunk.  With S0 the state before a chunk,
//   o_i = g^(i+1) S0^T q_i + sum_{j <= i} g^(i-j) (q_i . k_j) v_j,     S1 = g^n S0 + sum_j g^(n-1-j) k_j v_j^T
//   retention_local_kernel   the sum in S1 of every chunk, all chunks in parallel
//   retention_scan_kernel    S0 of every chunk (in place of those sums) and the state after the last: a thread per four elements
//   retention_out_kernel     o, norm and gate of every chunk, all chunks in parallel
// The powers come from a table, so any decay from 0 to 1 is exact to fp32 and no exponent is positive.
#include "mfma_frag.h"

namespace {

constexpr int C = OHARA_RETENTION_CHUNK;
constexpr int KB = 64;  // tokens staged at a time

template <typename T>
struct RetentionArgs {
  OharaRetention r;
  const T* p;
  float* state;
  float* ws;
  T* out;
  int ldp, ldo;
  int chunk0, nchunks;  // chunks of this segment
  OharaSeq seq;
};

__host__ __device__ __forceinline__ int up(int v, int m) { return (v + m - 1) / m * m; }

// A chunk's state in the workspace: dim rounded up to 32, vdim to 16, padding zero, in the order of B fragments: tile
// (d / 32, v / 16) of 64 lanes x 8 floats.
__host__ __device__ __forceinline__ size_t state_floats(int D, int V) { return (size_t)up(D, 32) * up(V, 16); }

// ---- one token -------------------------------------------------------------------------------
template <typename T, int NT, int ROWS>  // threads; state rows a thread holds at most
__global__ __launch_bounds__(NT) void retention_step_kernel(RetentionArgs<T> a) {
  constexpr int NW = NT / 64;
  __shared__ __align__(16) float qs[256], ks[256], part[NT * 4];
  __shared__ float red[NW];
  const OharaRetention& r = a.r;
  const int H = r.heads, D = r.dim, V = r.vdim;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int b = blockIdx.x / H, h = blockIdx.x - b * H;
  const int pos = seq_start(a.seq, b);
  if (seq_tokens(a.seq, b) < 1 || pos < 0) return;
  // this thread's slice of the state: four columns, rows grp, grp + ngrp, ...
  const int c4 = V / 4, ngrp = NT / c4, grp = tid / c4, col = 4 * (tid - grp * c4);
  float* S = a.state + ((size_t)seq_slot(a.seq, b) * H + h) * D * V + col;
  float4 st[ROWS];
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
    const int d = grp + i * ngrp;
    st[i] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (grp < ngrp && d < D && pos > 0) st[i] = *reinterpret_cast<const float4*>(S + (size_t)d * V);
  }
  const T* p = a.p + (size_t)b * a.ldp;
  float v[4] = {0.f, 0.f, 0.f, 0.f}, gate = 0.f;
  if (grp < ngrp) ld4(p + r.off_v + h * V + col, v);
  if (tid < V) gate = ldv(p + r.off_g + h * V + tid);
  for (int i = tid; i < D; i += NT) {
    qs[i] = ldv(p + r.off_q + h * D + i);
    ks[i] = ldv(p + r.off_k + h * D + i) * r.k_scale;
  }
  const float decay = r.powers[(size_t)h * (C + 1) + 1];
  __syncthreads();
  float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
    const int d = grp + i * ngrp;
    if (grp < ngrp && d < D) {
      const float k = ks[d], q = qs[d];
      float4 s = st[i];
      s.x = decay * s.x + k * v[0]; s.y = decay * s.y + k * v[1]; s.z = decay * s.z + k * v[2]; s.w = decay * s.w + k * v[3];
      *reinterpret_cast<float4*>(S + (size_t)d * V) = s;
      o.x += s.x * q; o.y += s.y * q; o.z += s.z * q; o.w += s.w * q;
    }
  }
  if (grp < ngrp) *reinterpret_cast<float4*>(part + (size_t)grp * V + col) = o;
  __syncthreads();
  float y = 0.f;
  if (tid < V)
    for (int i = 0; i < ngrp; ++i) y += part[i * V + tid];
  const float ss = wave_sum(y * y);
  if (lane == 0) red[wave] = ss;
  __syncthreads();
  if (tid < V) {
    float tot = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) tot += red[w];  // V <= 256: the first four waves
    const float inv = r.out_scale / sqrtf(tot / (float)r.vdim_used + r.eps);
    stv(a.out + (size_t)b * a.ldo + h * V + tid, y * inv * silu_x(gate));
  }
}

// ---- prompts -----------------------------------------------------------------------------------
// Eight columns c .. c+7 of the four tokens t .. t+3 (t0: the block's first token; tokens from n on give zero), to LDS by column.
template <typename T, bool WIDE>
__device__ __forceinline__ void stage4x8(const T* rows, int ldp, int t, int n, bool in, const float* scale, T* dst, int ld, int plane) {
  Raw8<T> raw[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    if (in && t + i < n) raw[i].load(rows + (size_t)(t + i) * ldp);
    else raw[i].zero();
  }
  float x[4][8];
#pragma unroll
  for (int i = 0; i < 4; ++i) raw[i].get(x[i]);
#pragma unroll
  for (int c = 0; c < 8; ++c) {
    float y[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) y[i] = WIDE ? x[i][c] * scale[i] : x[i][c];
    if constexpr (WIDE) WideLds<T>::put4(dst + (size_t)c * ld, plane, y);
    else if constexpr (sizeof(T) == 2) *reinterpret_cast<uint2*>(dst + (size_t)c * ld) = make_uint2(pack_bf(y[0], y[1]), pack_bf(y[2], y[3]));
    else *reinterpret_cast<float4*>(dst + (size_t)c * ld) = make_float4(y[0], y[1], y[2], y[3]);
  }
}

template <typename T> constexpr int ld_tokens() { return KB + 16 / (int)sizeof(T); }  // a staged column of KB tokens, 16 bytes apart mod 128

__device__ __forceinline__ void ld_row8(const float* p, float* o) {  // eight floats from LDS
  const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
  o[0] = a.x; o[1] = a.y; o[2] = a.z; o[3] = a.w; o[4] = b.x; o[5] = b.y; o[6] = b.z; o[7] = b.w;
}

constexpr int VS = 64;  // value columns of a workgroup of retention_local_kernel

// sum_j g^(n-1-j) k_scale k_j v_j^T of a chunk, for VS of the value columns: a wave takes every fourth 16-row tile of the key channels.
template <typename T, int MT>  // 16-row tiles of a wave at most
__global__ __launch_bounds__(256) void retention_local_kernel(RetentionArgs<T> a, int nvs) {
  extern __shared__ __align__(16) unsigned char smem[];
  constexpr int LD = ld_tokens<T>();
  const OharaRetention& r = a.r;
  const int H = r.heads, D = r.dim, V = r.vdim;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, m = lane & 15, g = lane >> 4;
  const int ci = blockIdx.x / nvs, v0 = (blockIdx.x % nvs) * VS, h = blockIdx.y, b = blockIdx.z;
  const int len = seq_tokens(a.seq, b), s0 = (a.chunk0 + ci) * C;
  if (s0 >= len) return;
  const int n = min(C, len - s0);
  const int Dp = up(D, 32), Vp = up(V, 16), nc = min(VS, Vp - v0);
  T* Kt = reinterpret_cast<T*>(smem);  // [Dp][LD]
  T* Vt = Kt + (size_t)Dp * LD;        // planes of [VS][LD]
  const int plane = VS * LD;
  const T* rows = a.p + ((size_t)b * a.seq.seq_len + s0) * a.ldp;
  const float* pw = r.powers + (size_t)h * (C + 1);
  f32x4 acc[MT][4];
#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = (f32x4){0.f, 0.f, 0.f, 0.f};
  for (int t0 = 0; t0 < n; t0 += KB) {
    if (t0) __syncthreads();
    for (int i = tid; i < (Dp / 8) * (KB / 4); i += 256) {
      const int c = 8 * (i % (Dp / 8)), t = 4 * (i / (Dp / 8));
      stage4x8<T, false>(rows + r.off_k + h * D + c, a.ldp, t0 + t, n, c < D, nullptr, Kt + (size_t)c * LD + t, LD, 0);
    }
    for (int i = tid; i < (nc / 8) * (KB / 4); i += 256) {
      const int c = 8 * (i % (nc / 8)), t = 4 * (i / (nc / 8));
      float sc[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) sc[u] = pw[max(n - 1 - (t0 + t + u), 0)] * r.k_scale;
      stage4x8<T, true>(rows + r.off_v + h * V + v0 + c, a.ldp, t0 + t, n, v0 + c < V, sc, Vt + (size_t)c * LD + t, LD, plane);
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < KB; k += 32) {
      if (t0 + k >= n) break;
      Wide<T> vf[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) WideLds<T>::get(vf[j], Vt + (size_t)min(16 * j + m, nc - 1) * LD + k + 8 * g, plane);
#pragma unroll
      for (int i = 0; i < MT; ++i) {
        const int tile = wave + 4 * i;
        if (16 * tile >= Dp) break;
        Frag<T> kf;
        frag_load(kf, Kt + (size_t)(16 * tile + m) * LD + k + 8 * g);
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = mma(kf, vf[j], acc[i][j]);
      }
    }
  }
  float* w = a.ws + (((size_t)b * H + h) * a.nchunks + ci) * state_floats(D, V);
#pragma unroll
  for (int i = 0; i < MT; ++i) {
    const int tile = wave + 4 * i;
    if (16 * tile >= Dp) break;
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (16 * j < nc) {
        // rows 16 tile + 4 g .. + 3 are entries 4 (g & 1) .. of lane (m, 2 (tile & 1) + g / 2)
        float* o = w + ((size_t)((tile >> 1) * (Vp / 16) + v0 / 16 + j) * 64 + (2 * (tile & 1) + (g >> 1)) * 16 + m) * 8 + 4 * (g & 1);
        *reinterpret_cast<f32x4*>(o) = acc[i][j];
      }
  }
}

// The states before the chunks, in place of what the chunks add, and the state after the last one.
template <typename T>
__global__ __launch_bounds__(256) void retention_scan_kernel(RetentionArgs<T> a) {
  const OharaRetention& r = a.r;
  const int H = r.heads, D = r.dim, V = r.vdim, Vp = up(V, 16);
  const int h = blockIdx.y, b = blockIdx.z;
  const int len = seq_tokens(a.seq, b);
  const int nch = min(a.nchunks, (len + C - 1) / C - a.chunk0);
  const size_t sf = state_floats(D, V), e = 4 * ((size_t)blockIdx.x * 256 + threadIdx.x);
  if (nch < 1 || e >= sf) return;
  const int tile = (int)(e >> 9), lane = (int)(e >> 3) & 63;
  const int d = 32 * (tile / (Vp / 16)) + 8 * (lane >> 4) + (int)(e & 7), v = 16 * (tile % (Vp / 16)) + (lane & 15);
  float* S = a.state + ((size_t)seq_slot(a.seq, b) * H + h) * D * V + (size_t)d * V + v;
  const bool in = d < D && v < V;  // d is a multiple of 4: all four rows or none
  float* w = a.ws + ((size_t)b * H + h) * a.nchunks * sf + e;
  const float* pw = r.powers + (size_t)h * (C + 1);
  const float full = pw[C], last = pw[min(C, len - (a.chunk0 + nch - 1) * C)];
  f32x4 s = (f32x4){0.f, 0.f, 0.f, 0.f};
  if (in && !(a.chunk0 == 0 && seq_start(a.seq, b) == 0)) {
#pragma unroll
    for (int u = 0; u < 4; ++u) s[u] = S[(size_t)u * V];
  }
  constexpr int F = 8;  // chunks in flight
  for (int c0 = 0; c0 < nch; c0 += F) {
    f32x4 x[F];
#pragma unroll
    for (int i = 0; i < F; ++i) x[i] = *reinterpret_cast<const f32x4*>(w + (size_t)min(c0 + i, nch - 1) * sf);
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int i = 0; i < F; ++i) {
      if (c0 + i >= nch) break;
      *reinterpret_cast<f32x4*>(w + (size_t)(c0 + i) * sf) = s;
      const float dec = c0 + i == nch - 1 ? last : full;
#pragma unroll
      for (int u = 0; u < 4; ++u) s[u] = dec * s[u] + x[i][u];
    }
  }
  if (in) {
#pragma unroll
    for (int u = 0; u < 4; ++u) S[(size_t)u * V] = s[u];
  }
}

// A wave owns every fourth 16-column tile of the values for all C queries, so each element of the state is fetched (and split) once;
// the decayed scores of C queries x KB keys go through LDS.
template <typename T, int NT>  // 16-column tiles of a wave at most
__global__ __launch_bounds__(256, 1) void retention_out_kernel(RetentionArgs<T> a) {
  extern __shared__ __align__(16) unsigned char smem[];
  constexpr int LD = ld_tokens<T>(), QT = C / 16;
  __shared__ float pw[C + 1], red[4][C];
  const OharaRetention& r = a.r;
  const int H = r.heads, D = r.dim, V = r.vdim;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, m = lane & 15, g = lane >> 4;
  const int ci = blockIdx.x, h = blockIdx.y, b = blockIdx.z;
  const int len = seq_tokens(a.seq, b), s0 = (a.chunk0 + ci) * C;
  if (s0 >= len) return;
  const int n = min(C, len - s0);
  const int Dp = up(D, 32), Vp = up(V, 16), vt = Vp / 16;
  T* A = reinterpret_cast<T*>(smem);                  // decayed scores, planes of [C][LD]
  constexpr int plane = C * LD;
  T* Vt = A + (size_t)WideLds<T>::PLANES * plane;     // [Vp][LD]
  const T* rows = a.p + ((size_t)b * a.seq.seq_len + s0) * a.ldp;
  const T* qrows = rows + r.off_q + h * D;
  const T* krows = rows + r.off_k + h * D;
  for (int i = tid; i <= C; i += 256) pw[i] = r.powers[(size_t)h * (C + 1) + i];
  f32x4 acc[NT][QT];
#pragma unroll
  for (int i = 0; i < NT; ++i)
#pragma unroll
    for (int q = 0; q < QT; ++q) acc[i][q] = (f32x4){0.f, 0.f, 0.f, 0.f};
  // Row t, columns d .. d+7, loaded whatever t and d: rows past the chunk give scores nobody reads, columns past the head are zeroed.
  auto load_row = [&](Frag<T>& f, const T* base, int t, int d) {
    frag_load(f, base + (size_t)min(t, n - 1) * a.ldp + (d < D ? d : 0));
    if (d >= D) frag_zero(f);
  };
  __syncthreads();
  // the state's part
  if (!(a.chunk0 + ci == 0 && seq_start(a.seq, b) == 0)) {
    const float* w = a.ws + (((size_t)b * H + h) * a.nchunks + ci) * state_floats(D, V);
    for (int ds = 0; ds < Dp / 32; ++ds) {
      Frag<T> qf[QT];
#pragma unroll
      for (int q = 0; q < QT; ++q) load_row(qf[q], qrows, 16 * q + m, 32 * ds + 8 * g);
#pragma unroll
      for (int i = 0; i < NT; ++i) {
        const int tile = wave + 4 * i;
        if (tile >= vt) break;
        float sv[8];
        const float* sp = w + ((size_t)(ds * vt + tile) * 64 + lane) * 8;
        ld4(sp, sv);
        ld4(sp + 4, sv + 4);
        Wide<T> sw;
        wide_from(sw, sv);
#pragma unroll
        for (int q = 0; q < QT; ++q) acc[i][q] = mma(qf[q], sw, acc[i][q]);
      }
    }
#pragma unroll
    for (int q = 0; q < QT; ++q) {
      float dec[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) dec[u] = pw[16 * q + 4 * g + u + 1];
#pragma unroll
      for (int i = 0; i < NT; ++i)
#pragma unroll
        for (int u = 0; u < 4; ++u) acc[i][q][u] *= dec[u];
    }
  }
  // the chunk's own part, KB keys at a time
  for (int t0 = 0; t0 < n; t0 += KB) {
    if (t0) __syncthreads();  // everyone is done with the previous block
    for (int i = tid; i < (Vp / 8) * (KB / 4); i += 256) {
      const int c = 8 * (i % (Vp / 8)), t = 4 * (i / (Vp / 8));
      stage4x8<T, false>(rows + r.off_v + h * V + c, a.ldp, t0 + t, n, c < V, nullptr, Vt + (size_t)c * LD + t, LD, 0);
    }
    // scores transposed, S^T = K Q^T, so a lane's four are neighbouring keys of one query; a wave takes query tiles wave and wave + 4
    f32x4 sc[2][KB / 16];
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int j = 0; j < KB / 16; ++j) sc[i][j] = (f32x4){0.f, 0.f, 0.f, 0.f};
    for (int ds = 0; ds < Dp / 32; ++ds) {
      Frag<T> kf[KB / 16], qf[2];
#pragma unroll
      for (int i = 0; i < 2; ++i) load_row(qf[i], qrows, 16 * (wave + 4 * i) + m, 32 * ds + 8 * g);
#pragma unroll
      for (int j = 0; j < KB / 16; ++j) load_row(kf[j], krows, t0 + 16 * j + m, 32 * ds + 8 * g);
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < KB / 16; ++j) sc[i][j] = mma(kf[j], qf[i], sc[i][j]);
    }
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int q = 16 * (wave + 4 * i) + m;
#pragma unroll
      for (int j = 0; j < KB / 16; ++j) {
        float y[4];
#pragma unroll
        for (int u = 0; u < 4; ++u) {
          const int back = q - (t0 + 16 * j + 4 * g + u);
          y[u] = back >= 0 ? sc[i][j][u] * r.k_scale * pw[max(back, 0)] : 0.f;
        }
        WideLds<T>::put4(A + (size_t)q * LD + 16 * j + 4 * g, plane, y);
      }
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < KB; k += 32) {
      if (t0 + k >= n) break;
      Frag<T> vf[NT];
#pragma unroll
      for (int i = 0; i < NT; ++i) frag_load(vf[i], Vt + (size_t)(16 * min(wave + 4 * i, vt - 1) + m) * LD + k + 8 * g);
#pragma unroll
      for (int q = 0; q < QT; ++q) {
        if (16 * q + 15 < t0 + k) continue;  // all keys lie after the queries
        Wide<T> w;
        WideLds<T>::get(w, A + (size_t)(16 * q + m) * LD + k + 8 * g, plane);
#pragma unroll
        for (int i = 0; i < NT; ++i) acc[i][q] = mma(w, vf[i], acc[i][q]);
      }
    }
  }
  // norm over the head's columns, gate
#pragma unroll
  for (int q = 0; q < QT; ++q)
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < NT; ++i)
        if (wave + 4 * i < vt) ss += acc[i][q][u] * acc[i][q][u];
      ss = lanes_sum<8, 1>(ss);
      if (m == 0) red[wave][16 * q + 4 * g + u] = ss;
    }
  // half of the rows at a time through LDS, so that gates and outputs move eight columns per thread
  const int ldy = Vp + 4, v8 = V / 8;
  float* Y = reinterpret_cast<float*>(smem);  // [C / 2][ldy]
#pragma unroll
  for (int half = 0; half < 2; ++half) {
    __syncthreads();
#pragma unroll
    for (int q = 0; q < QT / 2; ++q)
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int t = 16 * q + 4 * g + u, tt = t + half * (C / 2);
        const float tot = ((red[0][tt] + red[1][tt]) + red[2][tt]) + red[3][tt];
        const float inv = r.out_scale / sqrtf(tot / (float)r.vdim_used + r.eps);
#pragma unroll
        for (int i = 0; i < NT; ++i)
          if (wave + 4 * i < vt) Y[t * ldy + 16 * (wave + 4 * i) + m] = acc[i][half * (QT / 2) + q][u] * inv;
      }
    __syncthreads();
    const int left = min(C / 2, n - half * (C / 2));
    for (int i = tid; i < left * v8; i += 256) {
      const int t = i / v8, c = 8 * (i - t * v8), tt = t + half * (C / 2);
      Raw8<T> gr;
      gr.load(rows + (size_t)tt * a.ldp + r.off_g + h * V + c);
      float z[8], y[8];
      gr.get(z);
      ld_row8(Y + t * ldy + c, y);
#pragma unroll
      for (int u = 0; u < 8; ++u) y[u] *= silu_x(z[u]);
      T* op = a.out + ((size_t)b * a.seq.seq_len + s0 + tt) * a.ldo + h * V + c;
      st4(op, y);
      st4(op + 4, y + 4);
    }
  }
}

template <typename T>
int retention_ok(const OharaRetention* r, const T* p, int ldp, const float* state, const T* out, int ldo, const OharaSeq* seq) {
  if (!r || !p || !state || !out || !seq_ok(seq) || !r->powers) return OHARA_EINVAL;
  if (r->heads < 1 || r->dim < 8 || r->vdim < 8 || ((r->dim | r->vdim) & 7)) return OHARA_EINVAL;
  if (r->vdim_used < 1 || r->vdim_used > r->vdim) return OHARA_EINVAL;
  if (r->dim > 256 || r->vdim > 256 || r->heads > 65535 || seq->batch > 65535) return OHARA_ESIZE;
  const int nk = r->heads * r->dim, nv = r->heads * r->vdim;
  if ((ldp & 7) || ((r->off_q | r->off_k | r->off_v | r->off_g) & 7) || (ldo & 3) || ldo < nv) return OHARA_EINVAL;
  for (int o : {r->off_q, r->off_k})
    if (o < 0 || o + nk > ldp) return OHARA_EINVAL;
  for (int o : {r->off_v, r->off_g})
    if (o < 0 || o + nv > ldp) return OHARA_EINVAL;
  return OHARA_OK;
}

template <typename T>
int retention_step(const OharaRetention* r, const T* p, int ldp, float* state, T* out, int ldo, const OharaSeq* seq, hipStream_t st) {
  const int rc = retention_ok<T>(r, p, ldp, state, out, ldo, seq);
  if (rc) return rc;
  if (seq->seq_len != 1) return OHARA_EINVAL;
  if ((int64_t)seq->batch * r->heads > INT32_MAX) return OHARA_ESIZE;
  RetentionArgs<T> a{};
  a.r = *r; a.p = p; a.ldp = ldp; a.state = state; a.out = out; a.ldo = ldo; a.seq = *seq;
  const dim3 grid((unsigned)(seq->batch * r->heads));
  const int c4 = r->vdim / 4;
  if (r->dim * r->vdim < 4096 && (256 / c4) * 16 >= r->dim)
    hipLaunchKernelGGL((retention_step_kernel<T, 256, 16>), grid, dim3(256), 0, st, a);
  else if ((1024 / c4) * 4 >= r->dim)
    hipLaunchKernelGGL((retention_step_kernel<T, 1024, 4>), grid, dim3(1024), 0, st, a);
  else
    hipLaunchKernelGGL((retention_step_kernel<T, 1024, 16>), grid, dim3(1024), 0, st, a);
  return ohara_launch_status();
}

template <typename K, typename... Args>
void launch_lds(K kernel, dim3 grid, size_t smem, hipStream_t st, Args... args) {
  if (smem > 64 * 1024) (void)hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
  hipLaunchKernelGGL(kernel, grid, dim3(256), smem, st, args...);
}

template <typename T>
int retention_prefill(const OharaRetention* r, const T* p, int ldp, float* state, void* ws, int64_t ws_bytes, T* out, int ldo,
                      const OharaSeq* seq, hipStream_t st) {
  const int rc = retention_ok<T>(r, p, ldp, state, out, ldo, seq);
  if (rc) return rc;
  if (!ws) return OHARA_EINVAL;
  RetentionArgs<T> a{};
  a.r = *r; a.p = p; a.ldp = ldp; a.state = state; a.ws = reinterpret_cast<float*>(ws); a.out = out; a.ldo = ldo; a.seq = *seq;
  const int D = r->dim, V = r->vdim, Dp = up(D, 32), Vp = up(V, 16), nvs = (V + VS - 1) / VS;
  const int64_t per_chunk = (int64_t)state_floats(D, V) * sizeof(float) * r->heads * seq->batch;
  const int all = (seq->seq_len + C - 1) / C;
  const int fit = (int)(ws_bytes / per_chunk < all ? ws_bytes / per_chunk : all);
  if (fit < 1) return OHARA_EINVAL;
  constexpr int LD = ld_tokens<T>(), PL = WideLds<T>::PLANES;
  const size_t local_lds = ((size_t)Dp + PL * VS) * LD * sizeof(T);
  size_t out_lds = ((size_t)PL * C + Vp) * LD * sizeof(T);
  if (out_lds < (size_t)(C / 2) * (Vp + 4) * sizeof(float)) out_lds = (size_t)(C / 2) * (Vp + 4) * sizeof(float);
  const dim3 block(256);
  for (int c0 = 0; c0 < all; c0 += fit) {
    a.chunk0 = c0;
    a.nchunks = all - c0 < fit ? all - c0 : fit;
    const unsigned H = (unsigned)r->heads, B = (unsigned)seq->batch;
    const dim3 lg((unsigned)(a.nchunks * nvs), H, B), og((unsigned)a.nchunks, H, B);
    if (Dp <= 64) launch_lds(retention_local_kernel<T, 1>, lg, local_lds, st, a, nvs);
    else if (Dp <= 128) launch_lds(retention_local_kernel<T, 2>, lg, local_lds, st, a, nvs);
    else launch_lds(retention_local_kernel<T, 4>, lg, local_lds, st, a, nvs);
    hipLaunchKernelGGL((retention_scan_kernel<T>), dim3((unsigned)((state_floats(D, V) + 1023) / 1024), H, B), block, 0, st, a);
    if (Vp <= 64) launch_lds(retention_out_kernel<T, 1>, og, out_lds, st, a);
    else if (Vp <= 128) launch_lds(retention_out_kernel<T, 2>, og, out_lds, st, a);
    else launch_lds(retention_out_kernel<T, 4>, og, out_lds, st, a);
  }
  return ohara_launch_status();
}

}  // namespace

extern "C" {

int ohara_retention_step_bf16(const OharaRetention* r, const uint16_t* p, int ldp, float* state, uint16_t* out, int ldo,
                              const OharaSeq* seq, void* stream) {
  return retention_step<bf16_t>(r, p, ldp, state, out, ldo, seq, (hipStream_t)stream);
}
int ohara_retention_step_f32(const OharaRetention* r, const float* p, int ldp, float* state, float* out, int ldo,
                             const OharaSeq* seq, void* stream) {
  return retention_step<float>(r, p, ldp, state, out, ldo, seq, (hipStream_t)stream);
}

int64_t ohara_retention_workspace_bytes(int heads, int dim, int vdim, int batch, int tokens) {
  if (heads < 1 || dim < 8 || dim > 256 || vdim < 8 || vdim > 256 || batch < 1 || tokens < 1) return OHARA_EINVAL;
  return (int64_t)state_floats(dim, vdim) * (int64_t)sizeof(float) * heads * batch * ((tokens + C - 1) / C);
}

int ohara_retention_prefill_bf16(const OharaRetention* r, const uint16_t* p, int ldp, float* state, void* workspace,
                                 int64_t workspace_bytes, uint16_t* out, int ldo, const OharaSeq* seq, void* stream) {
  return retention_prefill<bf16_t>(r, p, ldp, state, workspace, workspace_bytes, out, ldo, seq, (hipStream_t)stream);
}
int ohara_retention_prefill_f32(const OharaRetention* r, const float* p, int ldp, float* state, void* workspace,
                                int64_t workspace_bytes, float* out, int ldo, const OharaSeq* seq, void* stream) {
  return retention_prefill<float>(r, p, ldp, state, workspace, workspace_bytes, out, ldo, seq, (hipStream_t)stream);
}

}  // extern "C"
