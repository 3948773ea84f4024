// Gated delta rule with one decay per head and key channel or one per head, with its short convolutions, unit norms, step
// sizes and gated output norm.  Per value head, S (dim x vdim, fp32) from zero:
//   S <- diag(exp(lg)) S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q.
//
// delta_step_kernel: one token per sequence, everything in one launch, a workgroup per (sequence, value head).  The
// state's slice is requested before anything else, so its latency runs under the convolutions and the
// low-rank products.  o = S_new^T q is formed as (diag(exp(lg)) S)^T q + (q . k) u, so both products with
// the state share one pass over it.
//
// Prompts: tokens in chunks of C = 32.  With G the running sum of lg inside a chunk (inclusive) and S0 the state before it,
//   A_ij = beta_i sum_d k_id k_jd exp(G_id - G_jd)  (j < i)          B_ij = sum_d q_id k_jd exp(G_id - G_jd)  (j <= i)
//   (I + A) u = beta (v - (k exp(G)) S0)  =>  u = U - W S0,  (I + A) U = beta v,  (I + A) W = beta k exp(G)
//   o = (q exp(G)) S0 + B u               S1 = diag(exp(G_C)) S0 + (k exp(G_C - G))^T u
// chunk_solve_kernel forms U, W, B and the scaled q, k of every chunk on its own (all chunks in parallel); every
// exponent there is a sum of logarithms of decays of tokens between j and i, never positive, however strong the decay.
// chunk_walk_kernel carries the state over the chunks: a workgroup per (sequence, head, 16 value
// columns), all products on fp32 MFMA with the state in accumulators.
#include "hybrid.h"

namespace {

constexpr int C = 32;        // tokens per chunk
constexpr float UNIT_EPS = 1e-6f;

template <typename T>
struct DeltaArgs {
  OharaDelta d;
  const T* p;
  const T* za;
  const T* zg;
  float* state;
  T* ring;
  float* ws;
  float* o;
  T* out;
  int ldp, ldza, ldzg, ldo;
  int chunk0, nchunks;  // chunks of this segment
  OharaSeq seq;
};

__device__ __forceinline__ float out_gate(const OharaDelta& d, float z) {
  return d.flags & OHARA_DELTA_SILU_GATE ? silu_x(z) : sigmoid_x(z);
}

__host__ __device__ __forceinline__ int up(int v, int m) { return (v + m - 1) / m * m; }

// ---- one token -------------------------------------------------------------------------------
template <typename T, int NT, int STEP_ROWS>  // threads; state rows a thread holds at most
__global__ __launch_bounds__(NT) void delta_step_kernel(DeltaArgs<T> a) {
  constexpr int NW = NT / 64;
  __shared__ __align__(16) float qs[256], ks[256], gs[256], vs[256], us[256], gate[256];
  __shared__ __align__(16) float rk[NT * 4], rq[NT * 4];
  __shared__ float red[NW];
  const OharaDelta& dd = a.d;
  const int H = dd.heads, D = dd.dim, V = dd.vdim;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int b = blockIdx.x / H, h = blockIdx.x - b * H;
  const int rep = H / dd.kv_heads, kvh = h / rep;
  T* orow = a.out + (size_t)b * a.ldo;
  if (h == 0)
    for (int i = H * V + tid; i < a.ldo; i += NT) stv(orow + i, 0.f);
  const int pos = seq_start(a.seq, b);
  if (seq_tokens(a.seq, b) < 1 || pos < 0) return;
  const int slot = seq_slot(a.seq, b);

  // this thread's slice of the state: four columns, rows grp, grp + ngrp, ...
  const int Vp = up(V, 4), c4 = Vp / 4, ngrp = NT / c4;
  const int grp = tid / c4, col = 4 * (tid - grp * c4);
  float* S = a.state + ((size_t)slot * H + h) * D * Vp + col;
  float4 st[STEP_ROWS];
#pragma unroll
  for (int i = 0; i < STEP_ROWS; ++i) {
    const int r = grp + i * ngrp;
    st[i] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (grp < ngrp && r < D && pos > 0) st[i] = *reinterpret_cast<const float4*>(S + (size_t)r * Vp);
  }

  // short convolutions of this head's q, k, v channels
  const T* p = a.p + (size_t)b * a.ldp;
  const int nqk = dd.kv_heads * D, channels = 2 * nqk + H * V, taps = dd.taps;
  T* ring = a.ring + (size_t)slot * taps * channels;
  for (int i = tid; i < 2 * D + V; i += NT) {
    const int ch = i < D ? kvh * D + i : (i < 2 * D ? nqk + kvh * D + (i - D) : 2 * nqk + h * V + (i - 2 * D));
    const float cur = ldv(p + ch);
    float c = dd.conv_w[(size_t)(taps - 1) * channels + ch] * cur;
    for (int lag = 1; lag < taps; ++lag)
      if (pos >= lag) c += dd.conv_w[(size_t)(taps - 1 - lag) * channels + ch] * ldv(ring + (size_t)((pos - lag) % taps) * channels + ch);
    // the slot written belongs to the token `taps` back, which no workgroup of this launch reads
    if (i >= 2 * D || h == kvh * rep) ring[(size_t)(pos % taps) * channels + ch] = p[ch];
    const float y = silu_x(c);
    if (i < D) qs[i] = y;
    else if (i < 2 * D) ks[i - D] = y;
    else vs[i - 2 * D] = y;
  }
  // decays and output gates: eight lanes per row of a2 / g2, two rows and 128 columns in flight
  const float na = dd.neg_a[h];
  if (!dd.a2) {
    const float g = expf(na * softplus_x(ldv(p + dd.off_a + h) + dd.dt_bias[h]));
    for (int i = tid; i < D; i += NT) gs[i] = g;
  }
  if (!dd.g2)
    for (int i = tid; i < V; i += NT) gate[i] = out_gate(dd, ldv(p + dd.off_g + h * V + i));
  if (dd.a2 || dd.g2) {
    const int l8 = tid & 7;
    constexpr int RP = NT / 8;  // rows per pass
    const int r_end = dd.g2 ? D + V : D;
    for (int r0 = dd.a2 ? 0 : D; r0 < r_end; r0 += 2 * RP) {
      float s[2] = {0.f, 0.f};
      const int nmax = max(dd.rank_a, dd.rank_g);
      for (int i0 = 0; i0 < nmax; i0 += 128) {
        Raw8<T> wv[2][2], xv[2][2];
#pragma unroll
        for (int u = 0; u < 2; ++u) {
          const int r = r0 + u * RP + (tid >> 3);
          const bool isa = r < D;
          const int n = isa ? dd.rank_a : dd.rank_g;
          const T* wrow = isa ? (const T*)dd.a2 + ((size_t)h * D + r) * n : (const T*)dd.g2 + ((size_t)h * V + (r - D)) * n;
          const T* xr = p + (isa ? dd.off_a : dd.off_g);
#pragma unroll
          for (int e = 0; e < 2; ++e) {
            const int i = i0 + 64 * e + 8 * l8;
            if (r < r_end && i < n) {
              wv[u][e].load(wrow + i);
              xv[u][e].load(xr + i);
            } else {
              wv[u][e].zero();
              xv[u][e].zero();
            }
          }
        }
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
          for (int e = 0; e < 2; ++e) {
            float wf[8], xf[8];
            wv[u][e].get(wf);
            xv[u][e].get(xf);
#pragma unroll
            for (int c = 0; c < 8; ++c) s[u] = __builtin_fmaf(wf[c], xf[c], s[u]);
          }
      }
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        const int r = r0 + u * RP + (tid >> 3);
        const float z = lanes_sum<4, 1>(s[u]);
        if (r < r_end && l8 == 0) {
          if (r < D) gs[r] = expf(na * softplus_x(z + dd.dt_bias[(size_t)h * D + r]));
          else gate[r - D] = out_gate(dd, z);
        }
      }
    }
  }
  __syncthreads();
  // every wave forms the sums over q and k for itself
  float sq = 0.f, sk = 0.f, qk = 0.f;
  for (int i = lane; i < D; i += 64) {
    const float q = qs[i], k = ks[i];
    sq += q * q;
    sk += k * k;
    qk += q * k;
  }
  const float iq = (1.0f / sqrtf(wave_sum(sq) + UNIT_EPS)) * (1.0f / sqrtf((float)D));
  const float ik = 1.0f / sqrtf(wave_sum(sk) + UNIT_EPS);
  qk = wave_sum(qk) * iq * ik;
  const float beta = sigmoid_x(ldv(p + dd.off_b + h));

  // decayed state against k and q
  float4 pk = make_float4(0.f, 0.f, 0.f, 0.f), pq = pk;
#pragma unroll
  for (int i = 0; i < STEP_ROWS; ++i) {
    const int r = grp + i * ngrp;
    if (r < D) {
      const float g = gs[r], kk = ks[r] * ik, qq = qs[r] * iq;
      st[i].x *= g; st[i].y *= g; st[i].z *= g; st[i].w *= g;
      pk.x += st[i].x * kk; pk.y += st[i].y * kk; pk.z += st[i].z * kk; pk.w += st[i].w * kk;
      pq.x += st[i].x * qq; pq.y += st[i].y * qq; pq.z += st[i].z * qq; pq.w += st[i].w * qq;
    }
  }
  if (grp < ngrp) {
    *reinterpret_cast<float4*>(rk + (size_t)grp * Vp + col) = pk;
    *reinterpret_cast<float4*>(rq + (size_t)grp * Vp + col) = pq;
  }
  __syncthreads();
  float o = 0.f;
  if (tid < V) {
    float sk_ = 0.f, sq_ = 0.f;
    for (int i = 0; i < ngrp; ++i) {
      sk_ += rk[i * Vp + tid];
      sq_ += rq[i * Vp + tid];
    }
    const float u = beta * (vs[tid] - sk_);
    us[tid] = u;
    o = sq_ + qk * u;
  } else if (tid < Vp) {
    us[tid] = 0.f;
  }
  const float so = wave_sum(o * o);
  if (lane == 0) red[wave] = so;
  __syncthreads();
  if (grp < ngrp) {
    const float4 u = *reinterpret_cast<const float4*>(us + col);
#pragma unroll
    for (int i = 0; i < STEP_ROWS; ++i) {
      const int r = grp + i * ngrp;
      if (r < D) {
        const float kk = ks[r] * ik;
        *reinterpret_cast<float4*>(S + (size_t)r * Vp) =
            make_float4(st[i].x + kk * u.x, st[i].y + kk * u.y, st[i].z + kk * u.z, st[i].w + kk * u.w);
      }
    }
  }
  if (tid < V) {
    float tot = 0.f;
#pragma unroll
    for (int w = 0; w < (NW < 4 ? NW : 4); ++w) tot += red[w];  // V <= 256: the first four waves
    const float inv = 1.0f / sqrtf(tot / (float)V + dd.eps);
    stv(orow + h * V + tid, o * inv * dd.norm_w[tid] * gate[tid]);
  }
}

// ---- prompts: workspace ------------------------------------------------------------------------
// Per (sequence, head, chunk): W [C][Dp], q exp(G) [C][Dp], k exp(G_C - G) [Dp][C], U [C][Vq], B [C][C] and exp(G_C) [Dp] as
// floats, Dp = dim rounded up to 32 / 64 / 128 / 256, Vq = vdim rounded up to 16, padding zero.  The matrices lie in the
// order the walk's waves read them: 16 x 16 tiles of 64 float4, one per lane.  W, q, k and B: tile (row / 16, column / 16),
// lane (row % 16, g = column % 16 / 4) holds columns 4 g .. 4 g + 3; U: tile (column / 16, token / 16), lane (column % 16, g)
// holds tokens 4 g .. 4 g + 3.
__host__ __device__ __forceinline__ int dim_padded(int d) { return d <= 32 ? 32 : (d <= 64 ? 64 : (d <= 128 ? 128 : 256)); }
__host__ __device__ __forceinline__ size_t chunk_floats(int D, int V) {
  const int Dp = dim_padded(D), Vq = up(V, 16);
  return (size_t)3 * C * Dp + (size_t)C * Vq + C * C + Dp;
}

// Convolution + silu of the 8 channels ch .. ch+7 at the four tokens t .. t+3 of this call (TAPS at compile time: the
// rows' loads are issued together); tokens from len on give zero.
template <typename T, int TAPS>
__device__ __forceinline__ void conv8x4(const DeltaArgs<T>& a, const T* prow, const T* ring, int channels, int pos0, int len,
                                        int t, int ch, float (&y)[4][8]) {
  constexpr int NR = 4 + TAPS - 1;
  Raw8<T> raw[NR];
#pragma unroll
  for (int j = 0; j < NR; ++j) {
    const int s = t - (TAPS - 1) + j;
    if (s >= 0 && s < len) raw[j].load(prow + (size_t)s * a.ldp + ch);
    else if (s < 0 && pos0 + s >= 0) raw[j].load(ring + (size_t)((pos0 + s) % TAPS) * channels + ch);
    else raw[j].zero();
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int c = 0; c < 8; ++c) y[i][c] = 0.f;
#pragma unroll
  for (int k = 0; k < TAPS; ++k) {
    float w[8];
    const float* wp = a.d.conv_w + (size_t)k * channels + ch;
    ld4(wp, w);
    ld4(wp + 4, w + 4);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      float x[8];
      raw[i + k].get(x);
#pragma unroll
      for (int c = 0; c < 8; ++c) y[i][c] = __builtin_fmaf(w[c], x[c], y[i][c]);
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int c = 0; c < 8; ++c) y[i][c] = t + i < len ? silu_x(y[i][c]) : 0.f;
}

// TAPS > 0: that many taps and head sizes that are multiples of 8 (16-byte loads); 0: any.
template <typename T, int TAPS>
__global__ __launch_bounds__(256, 2) void chunk_solve_kernel(DeltaArgs<T> a) {
  extern __shared__ __align__(16) float sm[];
  const OharaDelta& dd = a.d;
  const int H = dd.heads, D = dd.dim, V = dd.vdim;
  const int Dp = dim_padded(D), Vq = up(V, 16), LD = Dp + 4;
  float* Q = sm;               // [C][LD]
  float* K = Q + C * LD;
  float* G = K + C * LD;       // running sum of the decays' logarithms
  float* X = G + C * LD;       // v: [C][Vq]
  float* A = X + C * Vq;       // [C][C + 4]
  float* B = A + C * (C + 4);
  float* beta = B + C * (C + 4);  // [C]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int ci = blockIdx.x, h = blockIdx.y, b = blockIdx.z;
  const int len = seq_tokens(a.seq, b);
  const int s0 = (a.chunk0 + ci) * C;
  if (s0 >= len) return;
  const int n = min(C, len - s0);  // tokens of this chunk
  const int pos0 = seq_start(a.seq, b), slot = seq_slot(a.seq, b);
  const int rep = H / dd.kv_heads, kvh = h / rep;
  const int nqk = dd.kv_heads * D, channels = 2 * nqk + H * V, taps = dd.taps;
  const T* ring = a.ring + (size_t)slot * taps * channels;
  const T* prow = a.p + (size_t)b * a.seq.seq_len * a.ldp;  // row of the sequence's first token in this call
  const T* zrow = a.za + (size_t)b * a.seq.seq_len * a.ldza + (size_t)h * D;
  const float na = dd.neg_a[h];
  const bool per_head = !dd.a2;  // one decay for all channels
  if (tid < C) beta[tid] = tid < n ? sigmoid_x(ldv(prow + (size_t)(s0 + tid) * a.ldp + dd.off_b + h)) : 0.f;
  if constexpr (TAPS > 0) {
    const int d8 = D / 8, v8 = V / 8;
    for (int it = tid; it < (2 * d8 + v8) * (C / 4); it += 256) {
      const int t = 4 * (it / (2 * d8 + v8)), c8 = it % (2 * d8 + v8);
      const int ch = c8 < d8 ? kvh * D + 8 * c8
                             : (c8 < 2 * d8 ? nqk + kvh * D + 8 * (c8 - d8) : 2 * nqk + h * V + 8 * (c8 - 2 * d8));
      float y[4][8];
      conv8x4<T, TAPS>(a, prow, ring, channels, pos0, len, s0 + t, ch, y);
      float* dst = c8 < d8 ? Q + t * LD + 8 * c8 : (c8 < 2 * d8 ? K + t * LD + 8 * (c8 - d8) : X + t * Vq + 8 * (c8 - 2 * d8));
      const int ld = c8 < 2 * d8 ? LD : Vq;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        *reinterpret_cast<float4*>(dst + i * ld) = make_float4(y[i][0], y[i][1], y[i][2], y[i][3]);
        *reinterpret_cast<float4*>(dst + i * ld + 4) = make_float4(y[i][4], y[i][5], y[i][6], y[i][7]);
      }
    }
    // decays: 8 channels of two tokens per thread and round
    for (int it = tid; !per_head && it < d8 * (C / 2); it += 256) {
      const int t = it / d8, c = 8 * (it % d8);
      Raw8<T> z[2];
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        if (t + 16 * i < n) z[i].load(zrow + (size_t)(s0 + t + 16 * i) * a.ldza + c);
        else z[i].zero();
      }
      float bias[8];
      ld4(dd.dt_bias + (size_t)h * D + c, bias);
      ld4(dd.dt_bias + (size_t)h * D + c + 4, bias + 4);
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        float x[8];
        z[i].get(x);
#pragma unroll
        for (int u = 0; u < 8; ++u) x[u] = t + 16 * i < n ? na * softplus_x(x[u] + bias[u]) : 0.f;
        float* dst = G + (t + 16 * i) * LD + c;
        *reinterpret_cast<float4*>(dst) = make_float4(x[0], x[1], x[2], x[3]);
        *reinterpret_cast<float4*>(dst + 4) = make_float4(x[4], x[5], x[6], x[7]);
      }
    }
    for (int i = tid; i < C * (Dp - D); i += 256) {
      const int t = i / (Dp - D), c = D + i % (Dp - D);
      Q[t * LD + c] = K[t * LD + c] = G[t * LD + c] = 0.f;
    }
    for (int i = tid; i < C * (Vq - V); i += 256) X[(i / (Vq - V)) * Vq + V + i % (Vq - V)] = 0.f;
  } else {
    auto conv = [&](int s, int ch) {
      float c = 0.f;
      for (int lag = 0; lag < taps; ++lag) {
        float x;
        if (lag <= s) x = ldv(prow + (size_t)(s - lag) * a.ldp + ch);
        else if (pos0 + s >= lag) x = ldv(ring + (size_t)((pos0 + s - lag) % taps) * channels + ch);
        else break;
        c += dd.conv_w[(size_t)(taps - 1 - lag) * channels + ch] * x;
      }
      return silu_x(c);
    };
    for (int i = tid; i < C * Dp; i += 256) {
      const int t = i / Dp, c = i - t * Dp;
      const bool in = t < n && c < D;
      Q[t * LD + c] = in ? conv(s0 + t, kvh * D + c) : 0.f;
      K[t * LD + c] = in ? conv(s0 + t, nqk + kvh * D + c) : 0.f;
      G[t * LD + c] = in && !per_head ? na * softplus_x(ldv(zrow + (size_t)(s0 + t) * a.ldza + c) + dd.dt_bias[(size_t)h * D + c]) : 0.f;
    }
    for (int i = tid; i < C * Vq; i += 256) {
      const int t = i / Vq, c = i - t * Vq;
      X[i] = t < n && c < V ? conv(s0 + t, 2 * nqk + h * V + c) : 0.f;
    }
  }
  if (per_head) {
    if (tid < C) A[tid] = tid < n ? na * softplus_x(ldv(prow + (size_t)(s0 + tid) * a.ldp + dd.off_a + h) + dd.dt_bias[h]) : 0.f;
    __syncthreads();
    for (int i = tid; i < C * D; i += 256) G[i / D * LD + i % D] = A[i / D];
  }
  __syncthreads();
  // unit q and k, and the diagonal of B: eight lanes per token; running sums: a channel per thread
  {
    const int t = tid >> 3, l8 = tid & 7;
    float *q = Q + t * LD, *k = K + t * LD, sq = 0.f, sk = 0.f, qk = 0.f;
    for (int c = 4 * l8; c < Dp; c += 32) {
      const float4 x = *reinterpret_cast<const float4*>(q + c), y = *reinterpret_cast<const float4*>(k + c);
      sq += ((x.x * x.x + x.y * x.y) + x.z * x.z) + x.w * x.w;
      sk += ((y.x * y.x + y.y * y.y) + y.z * y.z) + y.w * y.w;
      qk += ((x.x * y.x + x.y * y.y) + x.z * y.z) + x.w * y.w;
    }
    const float iq = (1.0f / sqrtf(lanes_sum<4, 1>(sq) + UNIT_EPS)) * (1.0f / sqrtf((float)D));
    const float ik = 1.0f / sqrtf(lanes_sum<4, 1>(sk) + UNIT_EPS);
    qk = lanes_sum<4, 1>(qk) * iq * ik;
    for (int c = 4 * l8; c < Dp; c += 32) {
      float4* x = reinterpret_cast<float4*>(q + c);
      float4* y = reinterpret_cast<float4*>(k + c);
      *x = make_float4(x->x * iq, x->y * iq, x->z * iq, x->w * iq);
      *y = make_float4(y->x * ik, y->y * ik, y->z * ik, y->w * ik);
    }
    if (l8 == 0) B[t * (C + 4) + t] = qk;
  }
  for (int c = tid; c < Dp; c += 256) {
    float v[C];
#pragma unroll
    for (int t = 0; t < C; ++t) v[t] = G[t * LD + c];
#pragma unroll
    for (int t = 1; t < C; ++t) v[t] += v[t - 1];
#pragma unroll
    for (int t = 1; t < C; ++t) G[t * LD + c] = v[t];
  }
  // above the diagonal
  for (int i = tid; i < C * C; i += 256) {
    const int r = i / C, c = i % C;
    if (c > r) B[r * (C + 4) + c] = 0.f;
    if (c >= r) A[r * (C + 4) + c] = 0.f;
  }
  __syncthreads();
  // Below the diagonal inside the two 16 x 16 blocks: a pair (i, j) per thread (120 each), exponents as they are.
  if (tid < 240) {
    const int blk = tid >= 120, q = tid - 120 * blk;
    int i = (int)((1.0f + sqrtf(1.0f + 8.0f * (float)q)) * 0.5f);  // row of the q-th pair: i (i - 1) / 2 <= q
    while (i * (i - 1) / 2 > q) --i;
    while (i * (i + 1) / 2 <= q) ++i;
    const int j = q - i * (i - 1) / 2 + 16 * blk;
    i += 16 * blk;
    const float *ki = K + i * LD, *qi = Q + i * LD, *gi = G + i * LD, *kj = K + j * LD, *gj = G + j * LD;
    float sa = 0.f, sb = 0.f;
#pragma unroll 2
    for (int c = 0; c < D; c += 4) {  // columns past D are zero
      const float4 k1 = *reinterpret_cast<const float4*>(ki + c), q1 = *reinterpret_cast<const float4*>(qi + c);
      const float4 g1 = *reinterpret_cast<const float4*>(gi + c), k2 = *reinterpret_cast<const float4*>(kj + c);
      const float4 g2 = *reinterpret_cast<const float4*>(gj + c);
      const float e0 = k2.x * __expf(g1.x - g2.x), e1 = k2.y * __expf(g1.y - g2.y);
      const float e2 = k2.z * __expf(g1.z - g2.z), e3 = k2.w * __expf(g1.w - g2.w);
      sa += k1.x * e0; sa += k1.y * e1; sa += k1.z * e2; sa += k1.w * e3;
      sb += q1.x * e0; sb += q1.y * e1; sb += q1.z * e2; sb += q1.w * e3;
    }
    A[i * (C + 4) + j] = sa * beta[i];
    B[i * (C + 4) + j] = sb;
  }
  // The block of tokens 16 .. 31 against 0 .. 15 on MFMA, both sides scaled to the sum R at token 15:
  // exp(G_i - G_j) = exp(G_i - R) exp(R - G_j), neither exponent positive.  Waves 0, 1: A; 2, 3: B; each half of the
  // channels.  (A product's k-slot g of step j stands for channel 4 g + j of its 16.)
  {
    const int m = lane & 15, g = lane >> 4;
    const float* left = (wave < 2 ? K : Q) + (16 + m) * LD;
    const float *gl = G + (16 + m) * LD, *kr = K + m * LD, *gr = G + m * LD, *R = G + 15 * LD;
    f32x4 acc = (f32x4){0.f, 0.f, 0.f, 0.f};
    for (int c = (wave & 1) * (Dp / 2) + 4 * g; c < (wave & 1) * (Dp / 2) + Dp / 2; c += 16) {
      const float4 l = *reinterpret_cast<const float4*>(left + c), g1 = *reinterpret_cast<const float4*>(gl + c);
      const float4 r = *reinterpret_cast<const float4*>(kr + c), g2 = *reinterpret_cast<const float4*>(gr + c);
      const float4 ref = *reinterpret_cast<const float4*>(R + c);
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(l.x * __expf(g1.x - ref.x), r.x * __expf(ref.x - g2.x), acc, 0, 0, 0);
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(l.y * __expf(g1.y - ref.y), r.y * __expf(ref.y - g2.y), acc, 0, 0, 0);
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(l.z * __expf(g1.z - ref.z), r.z * __expf(ref.z - g2.z), acc, 0, 0, 0);
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(l.w * __expf(g1.w - ref.w), r.w * __expf(ref.w - g2.w), acc, 0, 0, 0);
    }
    float* dst = (wave < 2 ? A : B) + (16 + 4 * g) * (C + 4) + m;
    if (wave & 1) {
#pragma unroll
      for (int r = 0; r < 4; ++r) dst[r * (C + 4)] = acc[r];
    }
    __syncthreads();
    if (!(wave & 1)) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float v = dst[r * (C + 4)] + acc[r];
        dst[r * (C + 4)] = wave < 2 ? v * beta[16 + 4 * g + r] : v;
      }
    }
  }
  __syncthreads();
  float* w = a.ws + (((size_t)b * H + h) * a.nchunks + ci) * chunk_floats(D, V);
  float* wW = w;
  float* wQ = wW + C * Dp;
  float* wK = wQ + C * Dp;
  float* wU = wK + C * Dp;
  float* wB = wU + C * Vq;
  float* wG = wB + C * C;
  const int ct = Dp / 16;  // column tiles
  for (int i = tid; i < C * Dp / 4; i += 256) {
    const int t = 16 * (i / (64 * ct)) + (i & 15), c = 16 * (i / 64 % ct) + 4 * (i >> 4 & 3);
    const float4 q = *reinterpret_cast<const float4*>(Q + t * LD + c), g = *reinterpret_cast<const float4*>(G + t * LD + c);
    *reinterpret_cast<float4*>(wQ + 4 * i) = make_float4(q.x * __expf(g.x), q.y * __expf(g.y), q.z * __expf(g.z), q.w * __expf(g.w));
  }
  for (int i = tid; i < C * Dp / 4; i += 256) {
    const int c = 16 * (i >> 7) + (i & 15), t = 16 * (i >> 6 & 1) + 4 * (i >> 4 & 3);
    const float last = G[(C - 1) * LD + c];
    float v[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) v[u] = K[(t + u) * LD + c] * __expf(last - G[(t + u) * LD + c]);
    *reinterpret_cast<float4*>(wK + 4 * i) = make_float4(v[0], v[1], v[2], v[3]);
  }
  {
    const int t = 16 * (tid >> 7) + (tid & 15), c = 16 * (tid >> 6 & 1) + 4 * (tid >> 4 & 3);
    *reinterpret_cast<float4*>(wB + 4 * tid) = *reinterpret_cast<const float4*>(B + t * (C + 4) + c);
  }
  for (int c = tid; c < Dp; c += 256) wG[c] = __expf(G[(C - 1) * LD + c]);
  __syncthreads();  // q has been read: its place takes W
  // forward substitution, a column per thread: rows of A are read by all lanes at once, the next one ahead of its use
  for (int c = tid; c < Dp + Vq; c += 256) {
    float x[C];
    const bool isw = c < Dp;
    const int vc = c - Dp;
#pragma unroll
    for (int t = 0; t < C; ++t) x[t] = beta[t] * (isw ? K[t * LD + c] * __expf(G[t * LD + c]) : X[t * Vq + vc]);
    float4 row[2][C / 4];
    row[1][0] = *reinterpret_cast<const float4*>(A + (C + 4));
#pragma unroll
    for (int t = 1; t < C; ++t) {
      if (t + 1 < C) {
#pragma unroll
        for (int j = 0; j < (t + 4) / 4; ++j) row[(t + 1) & 1][j] = *reinterpret_cast<const float4*>(A + (t + 1) * (C + 4) + 4 * j);
      }
      float s = x[t];
#pragma unroll
      for (int j = 0; j < t; ++j) {
        const float4 r = row[t & 1][j / 4];
        s -= ((j & 3) == 0 ? r.x : ((j & 3) == 1 ? r.y : ((j & 3) == 2 ? r.z : r.w))) * x[j];
      }
      x[t] = s;
      __builtin_amdgcn_sched_barrier(0);  // row by row: hoisting the reads of all of A would spill
    }
    if (isw) {
#pragma unroll
      for (int t = 0; t < C; ++t) Q[t * LD + c] = x[t];
    } else {
#pragma unroll
      for (int t = 0; t < C; t += 4)
        *reinterpret_cast<float4*>(wU + 4 * ((2 * (vc >> 4) + (t >> 4)) * 64 + 16 * (t >> 2 & 3) + (vc & 15))) =
            make_float4(x[t], x[t + 1], x[t + 2], x[t + 3]);
    }
  }
  __syncthreads();
  for (int i = tid; i < C * Dp / 4; i += 256) {
    const int t = 16 * (i / (64 * ct)) + (i & 15), c = 16 * (i / 64 % ct) + 4 * (i >> 4 & 3);
    *reinterpret_cast<float4*>(wW + 4 * i) = *reinterpret_cast<const float4*>(Q + t * LD + c);
  }
}

// The state over the chunks.  v_mfma_f32_16x16x4_f32: A lane (row = lane & 15, k = lane >> 4), B lane (k = lane >> 4,
// column = lane & 15), result row 4 (lane >> 4) + r, column lane & 15.  A step of 16 k's takes four products whose k-slot g
// of product j stands for k = 4 g + j, so a lane fetches the four A elements it needs as one float4.
//
// Eight waves: (u or o) x (two 16-token row tiles) x (two halves of the key channels); the state's 16-channel tiles are
// spread over all of them.  The halves of u meet where u is read, those of o in LDS one barrier later.
template <typename T, int DPT>  // Dp / 16
__global__ __launch_bounds__(512) void chunk_walk_kernel(DeltaArgs<T> a) {
  constexpr int Dp = 16 * DPT, MT = (DPT + 7) / 8, HT = DPT / 2, LS = Dp + 4, LU = C + 4;
  // by value column, so the four rows a lane holds of a result and the four k's it needs of an operand are one float4
  __shared__ __align__(16) float Sl[16 * LS];
  __shared__ __align__(16) float Un[2][16 * LU];
  __shared__ __align__(16) float On[16 * LU];
  const OharaDelta& dd = a.d;
  const int H = dd.heads, D = dd.dim, V = dd.vdim, Vp = up(V, 4), Vq = up(V, 16);
  const int tid = threadIdx.x, lane = tid & 63, m = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  // Workgroups are handed to the eight XCDs in turn: the column slices of one (sequence, head) get ids eight apart, so the
  // chunk operands they all read are fetched into one L2.
  const int nv = Vq / 16, local = blockIdx.x >> 3, pair = (local / nv) * 8 + (blockIdx.x & 7);
  if (pair >= a.seq.batch * H) return;
  const int v0 = (local % nv) * 16, h = pair % H, b = pair / H;
  const int len = seq_tokens(a.seq, b);
  const int nch = min(a.nchunks, (len + C - 1) / C - a.chunk0);
  if (nch < 1) return;
  const int pos0 = seq_start(a.seq, b);
  float* S = a.state + ((size_t)seq_slot(a.seq, b) * H + h) * D * Vp;
  const bool fresh = a.chunk0 == 0 && pos0 == 0;
  auto put4 = [](float* p, f32x4 v) { *reinterpret_cast<f32x4*>(p) = v; };
  f32x4 acc[MT];
#pragma unroll
  for (int i = 0; i < MT; ++i) {
    const int tile = wave + 8 * i;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = 16 * tile + 4 * g + r;
      acc[i][r] = (!fresh && tile < DPT && d < D && v0 + m < V) ? S[(size_t)d * Vp + v0 + m] : 0.f;
    }
    if (tile < DPT) put4(Sl + m * LS + 16 * tile + 4 * g, acc[i]);
  }
  const size_t cf = chunk_floats(D, V);
  const float* w = a.ws + ((size_t)b * H + h) * a.nchunks * cf;
  const bool left = wave < 4;           // waves 0 - 3: u; 4 - 7: o
  const int half = (wave >> 1) & 1;     // of the key channels
  const int mrow = 16 * (wave & 1);     // this wave's token rows
  const int s_first = a.chunk0 * C + mrow + 4 * g;  // token of the lane's first result row, chunk 0
  float* ob = a.o + (size_t)b * a.seq.seq_len * H * V + (size_t)h * V + v0 + m;
  // Operands of a chunk: three sets (two where registers end), the next chunks' loads are in flight during this one's
  // products.  No branch around a
  // load (what a wave does not need is fetched from a valid address and ignored), so the compiler can count them.
  struct Operands {
    float4 a[HT], k[MT][2], g[MT], b;
    f32x4 u;
  } op[DPT > 8 ? 2 : 3];
  auto fetch = [&](int ci, Operands& f) {
    const float* x = w + (size_t)min(ci, nch - 1) * cf;
    const float4* ap = reinterpret_cast<const float4*>(x + (left ? 0 : C * Dp)) + ((wave & 1) * DPT + half * HT) * 64 + lane;
#pragma unroll
    for (int i = 0; i < HT; ++i) f.a[i] = ap[64 * i];
    const float* kp = x + 2 * C * Dp;
    const float* up_ = kp + C * Dp;
    const float* bp = up_ + C * Vq;
    const float* gp = bp + C * C;
    f.u = reinterpret_cast<const f32x4*>(up_)[(2 * (v0 >> 4) + (wave & 1)) * 64 + lane];
    f.b = reinterpret_cast<const float4*>(bp)[(2 * (wave & 1) + half) * 64 + lane];
#pragma unroll
    for (int i = 0; i < MT; ++i) {
      const int tile = DPT % 8 == 0 ? wave + 8 * i : min(wave + 8 * i, DPT - 1);
#pragma unroll
      for (int j = 0; j < 2; ++j) f.k[i][j] = reinterpret_cast<const float4*>(kp)[(2 * tile + j) * 64 + lane];
      f.g[i] = *reinterpret_cast<const float4*>(gp + 16 * tile + 4 * g);
    }
  };
  auto mul4 = [&](float4 av, float4 bv, f32x4 c) {
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(av.x, bv.x, c, 0, 0, 0);
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(av.y, bv.y, c, 0, 0, 0);
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(av.z, bv.z, c, 0, 0, 0);
    return __builtin_amdgcn_mfma_f32_16x16x4f32(av.w, bv.w, c, 0, 0, 0);
  };
  f32x4 o = (f32x4){0.f, 0.f, 0.f, 0.f};
  // the other half of the last chunk's o is in LDS: add and store (waves of the first half)
  auto store_o = [&](int ci) {
    if (!left && half == 0) {
      const f32x4 p = *reinterpret_cast<const f32x4*>(On + m * LU + mrow + 4 * g);
      const int s = s_first + ci * C;
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (s + r < len && v0 + m < V) ob[(size_t)(s + r) * H * V] = o[r] + p[r];
    }
  };
  auto chunk = [&](int ci, const Operands& f) {
    float4 sv[HT];
#pragma unroll
    for (int i = 0; i < HT; ++i) sv[i] = *reinterpret_cast<const float4*>(Sl + m * LS + half * (Dp / 2) + 16 * i + 4 * g);
    if (ci > 0) store_o(ci - 1);
    f32x4 x = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < HT; ++i) x = mul4(f.a[i], sv[i], x);
    if (left) {
      if (half) put4(Un[1] + m * LU + mrow + 4 * g, (f32x4){-x[0], -x[1], -x[2], -x[3]});
      else put4(Un[0] + m * LU + mrow + 4 * g, (f32x4){f.u[0] - x[0], f.u[1] - x[1], f.u[2] - x[2], f.u[3] - x[3]});
    }
    __syncthreads();  // u is complete; the state and the last o in LDS have been read
    float4 uv[2];
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const float4 p = *reinterpret_cast<const float4*>(Un[0] + m * LU + 16 * j + 4 * g);
      const float4 q = *reinterpret_cast<const float4*>(Un[1] + m * LU + 16 * j + 4 * g);
      uv[j] = make_float4(p.x + q.x, p.y + q.y, p.z + q.z, p.w + q.w);
    }
#pragma unroll
    for (int i = 0; i < MT; ++i) {
      const int tile = wave + 8 * i;
      if (DPT % 8 == 0 || tile < DPT) {
        acc[i][0] *= f.g[i].x; acc[i][1] *= f.g[i].y; acc[i][2] *= f.g[i].z; acc[i][3] *= f.g[i].w;
#pragma unroll
        for (int j = 0; j < 2; ++j) acc[i] = mul4(f.k[i][j], uv[j], acc[i]);
        put4(Sl + m * LS + 16 * tile + 4 * g, acc[i]);
      }
    }
    if (!left) {  // each half takes 16 of the chunk's tokens of B u
      o = mul4(f.b, half ? uv[1] : uv[0], x);
      if (half) put4(On + m * LU + mrow + 4 * g, o);
    }
    __syncthreads();  // the new state is in LDS; u has been read
  };
  fetch(0, op[0]);
  if constexpr (DPT > 8) {
    __syncthreads();
    for (int ci = 0; ci < nch; ci += 2) {
      fetch(ci + 1, op[1]);
      chunk(ci, op[0]);
      if (ci + 1 >= nch) break;
      fetch(ci + 2, op[0]);
      chunk(ci + 1, op[1]);
    }
  } else {
    fetch(1, op[1]);
    __syncthreads();
    for (int ci = 0; ci < nch; ci += 3) {
      fetch(ci + 2, op[2]);
      chunk(ci, op[0]);
      if (ci + 1 >= nch) break;
      fetch(ci + 3, op[0]);
      chunk(ci + 1, op[1]);
      if (ci + 2 >= nch) break;
      fetch(ci + 4, op[1]);
      chunk(ci + 2, op[2]);
    }
  }
  store_o(nch - 1);
#pragma unroll
  for (int i = 0; i < MT; ++i) {
    const int tile = wave + 8 * i;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = 16 * tile + 4 * g + r;
      if (tile < DPT && d < D && v0 + m < V) S[(size_t)d * Vp + v0 + m] = acc[i][r];
    }
  }
}

// out = o / rms(o) * norm_w * gate: a wave per (row, head)
template <typename T>
__global__ __launch_bounds__(256) void delta_out_kernel(DeltaArgs<T> a) {
  const OharaDelta& dd = a.d;
  const int H = dd.heads, V = dd.vdim;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int row = blockIdx.x, b = row / a.seq.seq_len, s = row - b * a.seq.seq_len;
  T* orow = a.out + (size_t)row * a.ldo;
  const T* zg = dd.g2 ? a.zg + (size_t)row * a.ldzg : a.p + (size_t)row * a.ldp + dd.off_g;
  for (int i = H * V + threadIdx.x; i < a.ldo; i += 256) stv(orow + i, 0.f);
  if (s >= seq_tokens(a.seq, b)) return;
  for (int h = blockIdx.y * 4 + wave; h < H; h += 4 * gridDim.y) {
    const float* o = a.o + ((size_t)row * H + h) * V;
    float v[4], z[4], ss = 0.f;
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int c = lane + 64 * u;
      v[u] = c < V ? o[c] : 0.f;
      z[u] = c < V ? ldv(zg + (size_t)h * V + c) : 0.f;
      ss += v[u] * v[u];
    }
    const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)V + dd.eps);
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int c = lane + 64 * u;
      if (c < V) stv(orow + h * V + c, v[u] * inv * dd.norm_w[c] * out_gate(dd, z[u]));
    }
  }
}

bool delta_ok(const OharaDelta* d, int ldp) {
  if (!d || !d->conv_w || !d->neg_a || !d->dt_bias || !d->norm_w) return false;
  if (d->heads < 1 || d->kv_heads < 1 || d->heads % d->kv_heads || d->dim < 1 || d->vdim < 1 || d->taps < 1) return false;
  const int channels = 2 * d->kv_heads * d->dim + d->heads * d->vdim;
  if (d->a2 && (d->rank_a < 8 || ((d->rank_a | d->off_a) & 7))) return false;
  if (d->g2 && (d->rank_g < 8 || ((d->rank_g | d->off_g) & 7))) return false;
  const int na = d->a2 ? d->rank_a : d->heads, ng = d->g2 ? d->rank_g : d->heads * d->vdim;
  return (ldp & 7) == 0 && ldp >= channels && d->off_a >= channels && d->off_a + na <= ldp && d->off_g >= channels &&
         d->off_g + ng <= ldp && d->off_b >= channels && d->off_b + d->heads <= ldp;
}

template <typename T>
int delta_step(const OharaDelta* d, const T* p, int ldp, float* state, T* ring, T* out, int ldo, const OharaSeq* seq,
               hipStream_t st) {
  if (!delta_ok(d, ldp) || !p || !state || !ring || !out || !seq_ok(seq) || seq->seq_len != 1) return OHARA_EINVAL;
  if (ldo < d->heads * d->vdim) return OHARA_EINVAL;
  if (d->dim > 256 || d->vdim > 256) return OHARA_ESIZE;
  if ((int64_t)seq->batch * d->heads > INT32_MAX) return OHARA_ESIZE;
  DeltaArgs<T> a{};
  a.d = *d; a.p = p; a.ldp = ldp; a.state = state; a.ring = ring; a.out = out; a.ldo = ldo; a.seq = *seq;
  const dim3 grid((unsigned)(seq->batch * d->heads));
  const int c4 = up(d->vdim, 4) / 4;
  // 1024 threads from 64 x 64 states on: the launch is a chain of round trips, and with more threads each round fetches
  // more of the low-rank weights and the state.
  if (d->dim * d->vdim < 4096 && (256 / c4) * 16 >= d->dim)
    hipLaunchKernelGGL((delta_step_kernel<T, 256, 16>), grid, dim3(256), 0, st, a);
  else if ((1024 / c4) * 4 >= d->dim)
    hipLaunchKernelGGL((delta_step_kernel<T, 1024, 4>), grid, dim3(1024), 0, st, a);
  else
    hipLaunchKernelGGL((delta_step_kernel<T, 1024, 16>), grid, dim3(1024), 0, st, a);
  return ohara_launch_status();
}

template <typename T>
int delta_prefill(const OharaDelta* d, const T* p, int ldp, const T* za, int ldza, const T* zg, int ldzg, float* state,
                  const T* ring, void* ws, int64_t ws_bytes, float* o, T* out, int ldo, const OharaSeq* seq, hipStream_t st) {
  if (!delta_ok(d, ldp) || !p || (d->a2 && !za) || (d->g2 && !zg) || !state || !ring || !ws || !o || !out || !seq_ok(seq)) return OHARA_EINVAL;
  if (ldo < d->heads * d->vdim || (d->a2 && ldza < d->heads * d->dim) || (d->g2 && ldzg < d->heads * d->vdim)) return OHARA_EINVAL;
  if (d->dim > 256 || d->vdim > 256 || d->heads > 65535 || seq->batch > 65535) return OHARA_ESIZE;
  DeltaArgs<T> a{};
  a.d = *d; a.p = p; a.ldp = ldp; a.za = za; a.ldza = ldza; a.zg = zg; a.ldzg = ldzg; a.state = state;
  a.ring = const_cast<T*>(ring); a.ws = reinterpret_cast<float*>(ws); a.o = o; a.out = out; a.ldo = ldo; a.seq = *seq;
  const int Dp = dim_padded(d->dim);
  const int64_t per_chunk = (int64_t)chunk_floats(d->dim, d->vdim) * sizeof(float) * d->heads * seq->batch;
  const int all = (seq->seq_len + C - 1) / C;
  int fit = (int)(ws_bytes / per_chunk < all ? ws_bytes / per_chunk : all);
  if (fit < 1) return OHARA_EINVAL;
  const size_t smem = ((size_t)3 * C * (Dp + 4) + (size_t)C * up(d->vdim, 16) + 2 * C * (C + 4) + C) * sizeof(float);
  const int fast = ((d->dim | d->vdim) & 7) == 0 && d->taps <= 4 ? d->taps : 0;
  auto solve = [&](auto kernel) {
    if (smem > 64 * 1024) (void)hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
    hipLaunchKernelGGL(kernel, dim3((unsigned)a.nchunks, (unsigned)d->heads, (unsigned)seq->batch), dim3(256), smem, st, a);
  };
  const dim3 wgrid((unsigned)((d->heads * seq->batch + 7) / 8 * 8 * ((d->vdim + 15) / 16)));
  for (int c0 = 0; c0 < all; c0 += fit) {
    a.chunk0 = c0;
    a.nchunks = all - c0 < fit ? all - c0 : fit;
    switch (fast) {
      case 1: solve(chunk_solve_kernel<T, 1>); break;
      case 2: solve(chunk_solve_kernel<T, 2>); break;
      case 3: solve(chunk_solve_kernel<T, 3>); break;
      case 4: solve(chunk_solve_kernel<T, 4>); break;
      default: solve(chunk_solve_kernel<T, 0>); break;
    }
    switch (Dp) {
      case 32: hipLaunchKernelGGL((chunk_walk_kernel<T, 2>), wgrid, dim3(512), 0, st, a); break;
      case 64: hipLaunchKernelGGL((chunk_walk_kernel<T, 4>), wgrid, dim3(512), 0, st, a); break;
      case 128: hipLaunchKernelGGL((chunk_walk_kernel<T, 8>), wgrid, dim3(512), 0, st, a); break;
      default: hipLaunchKernelGGL((chunk_walk_kernel<T, 16>), wgrid, dim3(512), 0, st, a); break;
    }
  }
  const int rows = seq->batch * seq->seq_len;
  hipLaunchKernelGGL((delta_out_kernel<T>), dim3((unsigned)rows, (unsigned)((d->heads + 3) / 4)), dim3(256), 0, st, a);
  return ohara_launch_status();
}

}  // namespace

extern "C" {

int ohara_delta_step_bf16(const OharaDelta* d, const uint16_t* p, int ldp, float* state, uint16_t* ring, uint16_t* out,
                          int ldo, const OharaSeq* seq, void* stream) {
  return delta_step<bf16_t>(d, p, ldp, state, ring, out, ldo, seq, (hipStream_t)stream);
}
int ohara_delta_step_f32(const OharaDelta* d, const float* p, int ldp, float* state, float* ring, float* out, int ldo,
                         const OharaSeq* seq, void* stream) {
  return delta_step<float>(d, p, ldp, state, ring, out, ldo, seq, (hipStream_t)stream);
}

int64_t ohara_delta_workspace_bytes(int heads, int dim, int vdim, int batch, int tokens) {
  if (heads < 1 || dim < 1 || dim > 256 || vdim < 1 || vdim > 256 || batch < 1 || tokens < 1) return OHARA_EINVAL;
  return (int64_t)chunk_floats(dim, vdim) * (int64_t)sizeof(float) * heads * batch * ((tokens + C - 1) / C);
}

int ohara_delta_prefill_bf16(const OharaDelta* d, const uint16_t* p, int ldp, const uint16_t* za, int ldza,
                             const uint16_t* zg, int ldzg, float* state, const uint16_t* ring, void* workspace,
                             int64_t workspace_bytes, float* o_tmp, uint16_t* out, int ldo, const OharaSeq* seq,
                             void* stream) {
  return delta_prefill<bf16_t>(d, p, ldp, za, ldza, zg, ldzg, state, ring, workspace, workspace_bytes, o_tmp, out, ldo, seq,
                               (hipStream_t)stream);
}
int ohara_delta_prefill_f32(const OharaDelta* d, const float* p, int ldp, const float* za, int ldza, const float* zg,
                            int ldzg, float* state, const float* ring, void* workspace, int64_t workspace_bytes,
                            float* o_tmp, float* out, int ldo, const OharaSeq* seq, void* stream) {
  return delta_prefill<float>(d, p, ldp, za, ldza, zg, ldzg, state, ring, workspace, workspace_bytes, o_tmp, out, ldo, seq,
                              (hipStream_t)stream);
}

}  // extern "C"
