// Linear attention over a matrix state with one scalar decay per head and
// token, in two forms:
//
//   fixed decay : S_t = a_h S_(t-1) + k_t v_t^T,                  o_t = S_t^T q_t
//   delta rule  : S <- g_t S, u_t = beta_t (v_t - S^T k_t), S <- S + k_t u_t^T,
//                 o_t = S^T q_t
//
// S [d, dv] fp32 per (slot, head); a sequence whose first token of the launch
// sits at position 0 starts from zeros instead of the slot's old content. On
// the way in, fixed-decay queries and keys may pass silu (values too), be
// rotated by position (pairs i, i + n, from a table of cos and sin) and the keys
// be scaled; delta-rule queries and keys become unit vectors and the queries
// are scaled. All of it fp32.
//
//   lr_scan  : token by token, any sizes: a workgroup keeps 32 (or 16) columns
//              of one head's state in registers, 16 rows of 4 columns a thread at
//              most. Decode steps, short portions and key widths above 256.
//   lr_prep / lr_chunk : portions, 32 tokens at a time on the fp32 matrix cores
//              (v_mfma_f32_16x16x4_f32). With G the running sum of the log decays
//              inside a chunk and S_0 the state before it,
//                S_t = e^(G_t) S_0 + sum_{s <= t} e^(G_t - G_s) k_s u_s^T
//              where u = v for a fixed decay, and for the delta rule
//                u_t = beta_t (v_t - e^(G_t) S_0^T k_t
//                              - sum_{s < t} e^(G_t - G_s) (k_t . k_s) u_s),
//              that is U = M diag(beta) (V - e^G K S_0) with M = (I + A)^-1, A_ts =
//              beta_t e^(G_t - G_s) (k_t . k_s) for s < t. lr_prep works out what
//              does not need the state, every chunk at once: the prepared q and k,
//              the masked P_ts = e^(G_t - G_s) (q_t . k_s), M diag(beta), e^(G_t)
//              and e^(G_L - G_s). lr_chunk then walks a sequence's chunks in
//              order. Each of its waves owns 16 columns of the state in
//              accumulators for the whole portion; an accumulator register is at
//              once the B operand of the products that read it (contraction over
//              rows {4 g + r}, g = lane group, one register r a step), so the
//              state and u never leave their registers.
#include "seq_common.h"

#define LR_L 32          // tokens per chunk
#define LR_COLS 64       // value columns per workgroup of lr_chunk
#define LR_PS (LR_L + 4) // LDS row of an LR_L x LR_L matrix

struct LrArgs {
  float* o;                 // [T, H, dv]
  const void *q, *k, *v;    // [T, G, d], [T, G, d], [T, H, dv]
  int64_t qs, qh, ks, kh, vs, vh;   // token and head strides
  float q_scale, k_scale;
  int silu;
  const float* cs;          // [T, n_rot] pairs of cos, sin, or null
  int n_rot;
  const float* pw;          // fixed decay: [H, pw_n] powers 0, 1, 2, ... of a_h
  int pw_n;
  const float *gates, *a_log, *dt_bias;   // delta rule: [T, 2 H], [H], [H]
  float* state;             // [slots, H, d, dv]
  const int64_t* slots;
  const int *cu, *positions;
  int B, H, G, d, dv;
  // scratch of the chunked path
  float *qp, *kp;           // [T, G, d] prepared
  float *P, *M;             // [tiles, H, L, L]
  float *e_in, *w_out;      // [tiles, H, L]
  hipStream_t stream;
};

DEVINL float lr_silu(float z) { return z / (1.0f + expf(-z)); }
// ln(1 + e^z)
DEVINL float lr_softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

// log decay and step size of one token and head
DEVINL void lr_gates(const LrArgs& a, int64_t t, int h, float* logg, float* beta) {
  const float* z = a.gates + t * 2 * a.H;
  *beta = 1.0f / (1.0f + expf(-z[h]));
  *logg = -expf(a.a_log[h]) * lr_softplus(z[a.H + h] + a.dt_bias[h]);
}

// ---- token by token ----------------------------------------------------------------

// grid (column slices of CN * N, H, B); RG = 256 / CN row groups, thread = (row
// group, column group of N). LDS: q [d] | k [d] | v [CN N] | partial sums [4][CN N]
// x 2 | 2
template <typename T, int CN, int N, bool DELTA>
__global__ __launch_bounds__(256) void lr_scan_kernel(LrArgs a) {
  constexpr int RG = 256 / CN, CW = CN * N, RMAX = 16;
  extern __shared__ float lds[];
  const int b = blockIdx.z, h = blockIdx.y, g = h / (a.H / a.G);
  const int c0 = blockIdx.x * CW;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int cg = tid % CN, rg = tid / CN;
  const int d = a.d, dv = a.dv;
  const int t0 = a.cu ? a.cu[b] : b, t1 = a.cu ? a.cu[b + 1] : b + 1;
  if (t0 >= t1) return;
  float* sq = lds;
  float* sk = sq + d;
  float* sv = sk + d;
  float* p1 = sv + CW;
  float* p2 = p1 + 4 * CW;
  float* red = p2 + 4 * CW;

  float* S = a.state + (a.slots[b] * a.H + h) * (int64_t)d * dv;
  const int col = c0 + cg * N;
  const bool cok = col < dv;   // N == 4 only where dv is a multiple of 4
  const bool fresh = a.positions[t0] == 0;
  float s[RMAX][N];
#pragma unroll
  for (int r = 0; r < RMAX; ++r) {
    const int i = rg + r * RG;
#pragma unroll
    for (int j = 0; j < N; ++j) s[r][j] = 0.f;
    if (!fresh && cok && i < d) {
      if (N == 4) {
        const float4 x = *reinterpret_cast<const float4*>(S + (int64_t)i * dv + col);
        s[r][0] = x.x; s[r][1 % N] = x.y; s[r][2 % N] = x.z; s[r][3 % N] = x.w;
      } else {
        s[r][0] = S[(int64_t)i * dv + col];
      }
    }
  }
  const float fixed = DELTA ? 0.f : a.pw[(int64_t)h * a.pw_n + 1];
  const T* qb = (const T*)a.q + g * a.qh;
  const T* kb = (const T*)a.k + g * a.kh;
  const T* vb = (const T*)a.v + h * a.vh;

  for (int t = t0; t < t1; ++t) {
    __syncthreads();   // the previous token's reads are done
    const T* qr = qb + t * a.qs;
    const T* kr = kb + t * a.ks;
    const int n = a.cs ? a.n_rot / 2 : 0;
    const float* cs = a.cs ? a.cs + (int64_t)t * a.n_rot : nullptr;
    for (int i = tid; i < d; i += 256) {
      float x = ldf(qr + i), y = ldf(kr + i);
      if (a.silu) {
        x = lr_silu(x);
        y = lr_silu(y);
      }
      if (i < 2 * n) {
        const int m = i < n ? i : i - n;
        const int ip = i < n ? i + n : i - n;
        float xp = ldf(qr + ip), yp = ldf(kr + ip);
        if (a.silu) {
          xp = lr_silu(xp);
          yp = lr_silu(yp);
        }
        const float c = cs[2 * m], sn = i < n ? -cs[2 * m + 1] : cs[2 * m + 1];
        x = fmaf(xp, sn, x * c);
        y = fmaf(yp, sn, y * c);
      }
      sq[i] = x * a.q_scale;
      sk[i] = y * a.k_scale;
    }
    for (int j = tid; j < CW; j += 256) {
      float x = c0 + j < dv ? ldf(vb + t * a.vs + c0 + j) : 0.f;
      sv[j] = a.silu ? lr_silu(x) : x;
    }
    float dec = fixed, beta = 1.f;
    if (DELTA) {
      float lg;
      lr_gates(a, t, h, &lg, &beta);
      dec = expf(lg);
    }
    __syncthreads();
    float rq = 1.f, rk = 1.f;
    if (DELTA) {
      // unit vectors: the norms are applied where q and k are used
      if (wave < 2) {
        const float* x = wave ? sk : sq;
        float ss = 0.f;
        for (int i = lane; i < d; i += 64) ss = fmaf(x[i], x[i], ss);
        ss = wave_reduce_sum(ss);
        // the query already carries its scale: undo it inside the root
        const float sc = wave ? a.k_scale : a.q_scale;
        if (lane == 0) red[wave] = 1.0f / sqrtf(ss / (sc * sc) + 1e-6f);
      }
      __syncthreads();
      rq = red[0];
      rk = red[1];
    }
    float u[N];
#pragma unroll
    for (int j = 0; j < N; ++j) u[j] = sv[cg * N + j];
    if (DELTA) {
      float acc[N];
#pragma unroll
      for (int j = 0; j < N; ++j) acc[j] = 0.f;
#pragma unroll
      for (int r = 0; r < RMAX; ++r) {
        const int i = rg + r * RG;
        if (i < d) {
          const float ki = sk[i] * rk;
#pragma unroll
          for (int j = 0; j < N; ++j) {
            s[r][j] *= dec;
            acc[j] = fmaf(s[r][j], ki, acc[j]);
          }
        }
      }
#pragma unroll
      for (int j = 0; j < N; ++j) {
        for (int off = CN; off < 64; off <<= 1) acc[j] += __shfl_xor(acc[j], off, 64);
        if (lane < CN) p1[wave * CW + cg * N + j] = acc[j];
      }
      __syncthreads();
#pragma unroll
      for (int j = 0; j < N; ++j) {
        const int c = cg * N + j;
        const float m = p1[c] + p1[CW + c] + p1[2 * CW + c] + p1[3 * CW + c];
        u[j] = beta * (u[j] - m);
      }
    }
    float acc[N];
#pragma unroll
    for (int j = 0; j < N; ++j) acc[j] = 0.f;
#pragma unroll
    for (int r = 0; r < RMAX; ++r) {
      const int i = rg + r * RG;
      if (i < d) {
        const float ki = sk[i] * rk, qi = sq[i] * rq;
#pragma unroll
        for (int j = 0; j < N; ++j) {
          s[r][j] = DELTA ? fmaf(ki, u[j], s[r][j]) : fmaf(dec, s[r][j], ki * u[j]);
          acc[j] = fmaf(s[r][j], qi, acc[j]);
        }
      }
    }
#pragma unroll
    for (int j = 0; j < N; ++j) {
      for (int off = CN; off < 64; off <<= 1) acc[j] += __shfl_xor(acc[j], off, 64);
      if (lane < CN) p2[wave * CW + cg * N + j] = acc[j];
    }
    __syncthreads();
    for (int c = tid; c < CW; c += 256)
      if (c0 + c < dv)
        a.o[((int64_t)t * a.H + h) * dv + c0 + c] =
            p2[c] + p2[CW + c] + p2[2 * CW + c] + p2[3 * CW + c];
  }
#pragma unroll
  for (int r = 0; r < RMAX; ++r) {
    const int i = rg + r * RG;
    if (cok && i < d) {
      if (N == 4)
        *reinterpret_cast<float4*>(S + (int64_t)i * dv + col) =
            make_float4(s[r][0], s[r][1 % N], s[r][2 % N], s[r][3 % N]);
      else
        S[(int64_t)i * dv + col] = s[r][0];
    }
  }
}

// ---- chunks ------------------------------------------------------------------------

// which (sequence, chunk) a tile is; false past the last one
DEVINL bool lr_tile(const int* __restrict__ cu, int B, int tile, int* b_out, int* chunk) {
  for (int b = 0; b < B; ++b) {
    const int nt = (cu[b + 1] - cu[b] + LR_L - 1) / LR_L;
    if (tile < nt) {
      *b_out = b;
      *chunk = tile;
      return true;
    }
    tile -= nt;
  }
  return false;
}

// one 16 x 16 block of X Y^T, X and Y rows of D floats in LDS `xs` apart; lane group
// g holds rows 4 g + r, column lane % 16
template <int D>
DEVINL f32x4v lr_block(const float* x, const float* y, int xs, int l15, int g) {
  f32x4v c = {0.f, 0.f, 0.f, 0.f}, c2 = {0.f, 0.f, 0.f, 0.f};
  const float* xr = x + l15 * xs + 4 * g;
  const float* yr = y + l15 * xs + 4 * g;
#pragma unroll
  for (int f = 0; f < D; f += 32) {
    const float4 a = *reinterpret_cast<const float4*>(xr + f);
    const float4 b = *reinterpret_cast<const float4*>(yr + f);
    const float4 a2 = *reinterpret_cast<const float4*>(xr + f + 16);
    const float4 b2 = *reinterpret_cast<const float4*>(yr + f + 16);
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x, b.x, c, 0, 0, 0);
    c2 = __builtin_amdgcn_mfma_f32_16x16x4f32(a2.x, b2.x, c2, 0, 0, 0);
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.y, b.y, c, 0, 0, 0);
    c2 = __builtin_amdgcn_mfma_f32_16x16x4f32(a2.y, b2.y, c2, 0, 0, 0);
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.z, b.z, c, 0, 0, 0);
    c2 = __builtin_amdgcn_mfma_f32_16x16x4f32(a2.z, b2.z, c2, 0, 0, 0);
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.w, b.w, c, 0, 0, 0);
    c2 = __builtin_amdgcn_mfma_f32_16x16x4f32(a2.w, b2.w, c2, 0, 0, 0);
  }
  return c + c2;
}

// rows [0, LR_L) of X (n of them real, d of D columns real) into LDS as floats
template <typename T, int D, bool VEC>
DEVINL void lr_stage(const T* __restrict__ x, int64_t stride, int n, int d, bool silu,
                     float mult, float* __restrict__ dst) {
  constexpr int KS = D + 4;
  if (VEC) {
    for (int p = threadIdx.x; p < LR_L * (D / 8); p += 256) {
      const int t = p / (D / 8), f = (p % (D / 8)) * 8;
      float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
      if (t < n && f < d) {
        const T* src = x + t * stride + f;
        if (sizeof(T) == 2) {
          const bf16x8 raw = load_bf16x8(src);
#pragma unroll
          for (int e = 0; e < 8; ++e) v[e] = bf16x8_get(raw, e);
        } else {
          const float4 a = *reinterpret_cast<const float4*>(src);
          const float4 b = *reinterpret_cast<const float4*>(src + 4);
          v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w;
          v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
        }
        if (silu)
#pragma unroll
          for (int e = 0; e < 8; ++e) v[e] = lr_silu(v[e]);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] *= mult;
      }
      float* o = dst + t * KS + f;
      *reinterpret_cast<float4*>(o) = make_float4(v[0], v[1], v[2], v[3]);
      *reinterpret_cast<float4*>(o + 4) = make_float4(v[4], v[5], v[6], v[7]);
    }
  } else {
    for (int p = threadIdx.x; p < LR_L * D; p += 256) {
      const int t = p / D, f = p % D;
      float v = 0.f;
      if (t < n && f < d) {
        v = ldf(x + t * stride + f);
        if (silu) v = lr_silu(v);
        v *= mult;
      }
      dst[t * KS + f] = v;
    }
  }
}

// grid (tiles, H). LDS: Q, K [L][D + 4] | A [L][LR_PS] (delta rule)
template <typename T, int D, bool VEC, bool DELTA>
__global__ __launch_bounds__(256) void lr_prep_kernel(LrArgs a) {
  constexpr int KS = D + 4;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float g_hi[LR_L], g_lo[LR_L], s_beta[LR_L];
  float* Q = lds;
  float* K = Q + LR_L * KS;
  float* A = K + LR_L * KS;
  int b, chunk;
  if (!lr_tile(a.cu, a.B, blockIdx.x, &b, &chunk)) return;
  const int h = blockIdx.y, rep = a.H / a.G, gq = h / rep;
  const int t0 = a.cu[b] + chunk * LR_L;
  const int n = min(LR_L, a.cu[b + 1] - t0);
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int l15 = lane & 15, g = lane >> 4;
  const int64_t th = (int64_t)blockIdx.x * a.H + h;

  lr_stage<T, D, VEC>((const T*)a.q + t0 * a.qs + gq * a.qh, a.qs, n, a.d, a.silu,
                      DELTA ? 1.f : a.q_scale, Q);
  lr_stage<T, D, VEC>((const T*)a.k + t0 * a.ks + gq * a.kh, a.ks, n, a.d, a.silu,
                      DELTA ? 1.f : a.k_scale, K);
  if (DELTA && wave == 0) {
    // lane = token: running sums of the log decays in float64, kept as two floats
    float lg = 0.f, be = 0.f;
    if (lane < n) lr_gates(a, t0 + lane, h, &lg, &be);
    double F = (double)lg;
#pragma unroll
    for (int off = 1; off < LR_L; off <<= 1) {
      const double x = __shfl_up(F, off, 64);
      if (lane >= off) F += x;
    }
    const double FL = __shfl(F, LR_L - 1, 64);
    if (lane < LR_L) {
      const float hi = (float)F;
      g_hi[lane] = hi;
      g_lo[lane] = (float)(F - (double)hi);
      s_beta[lane] = be;
      a.e_in[th * LR_L + lane] = expf(hi);
      a.w_out[th * LR_L + lane] = lane < n ? expf((float)(FL - F)) : 0.f;
    }
  }
  if (!DELTA && tid < LR_L) {
    const float* pw = a.pw + (int64_t)h * a.pw_n;
    g_hi[tid] = pw[tid];   // a power per distance
    a.e_in[th * LR_L + tid] = pw[tid + 1];
    a.w_out[th * LR_L + tid] = tid < n ? pw[n - 1 - tid] : 0.f;
  }
  __syncthreads();
  if (DELTA) {
    // unit rows, 16 lanes a row
    for (int r = tid >> 4; r < 2 * LR_L; r += 16) {
      float* x = (r < LR_L ? Q + r * KS : K + (r - LR_L) * KS);
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < D; i += 16) ss = fmaf(x[i + l15], x[i + l15], ss);
#pragma unroll
      for (int off = 8; off > 0; off >>= 1) ss += __shfl_xor(ss, off, 64);
      const float m = (r < LR_L ? a.q_scale : a.k_scale) / sqrtf(ss + 1e-6f);
#pragma unroll
      for (int i = 0; i < D; i += 16) x[i + l15] *= m;
    }
    __syncthreads();
  } else if (a.cs != nullptr) {
    const int half = a.n_rot / 2;
    for (int p = tid; p < n * half; p += 256) {
      const int t = p / half, i = p % half;
      const float2 c = *reinterpret_cast<const float2*>(
          a.cs + (int64_t)(t0 + t) * a.n_rot + 2 * i);
      float* x = Q + t * KS + i;
      float u = x[0], w = x[half];
      x[0] = fmaf(-w, c.y, u * c.x);
      x[half] = fmaf(u, c.y, w * c.x);
      x = K + t * KS + i;
      u = x[0];
      w = x[half];
      x[0] = fmaf(-w, c.y, u * c.x);
      x[half] = fmaf(u, c.y, w * c.x);
    }
    __syncthreads();
  }
  // the prepared rows, once per query/key head
  if (h % rep == 0) {
    const int d = a.d;
    if (VEC) {
      for (int p = tid; p < n * (d / 4); p += 256) {
        const int t = p / (d / 4), f = (p % (d / 4)) * 4;
        const int64_t o = ((int64_t)(t0 + t) * a.G + gq) * d + f;
        *reinterpret_cast<float4*>(a.qp + o) = *reinterpret_cast<const float4*>(Q + t * KS + f);
        *reinterpret_cast<float4*>(a.kp + o) = *reinterpret_cast<const float4*>(K + t * KS + f);
      }
    } else {
      for (int p = tid; p < n * d; p += 256) {
        const int t = p / d, f = p % d;
        const int64_t o = ((int64_t)(t0 + t) * a.G + gq) * d + f;
        a.qp[o] = Q[t * KS + f];
        a.kp[o] = K[t * KS + f];
      }
    }
  }
  // P (jobs 0 .. 3) and A (jobs 4 .. 7), a 16 x 16 block (tb, sb) a job
  float* P = a.P + th * LR_L * LR_L;
  for (int job = wave; job < (DELTA ? 8 : 4); job += 4) {
    const int tb = (job >> 1) & 1, sb = job & 1;
    const bool is_a = job >= 4;
    f32x4v c = {0.f, 0.f, 0.f, 0.f};
    if (sb <= tb)
      c = lr_block<D>((is_a ? K : Q) + 16 * tb * KS, K + 16 * sb * KS, KS, l15, g);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = 16 * tb + 4 * g + r, s = 16 * sb + l15;
      float w = 0.f;
      if (is_a ? s < t : s <= t)
        w = DELTA ? expf((g_hi[t] - g_hi[s]) + (g_lo[t] - g_lo[s])) : g_hi[t - s];
      if (is_a) A[t * LR_PS + s] = c[r] * w * s_beta[t];
      else P[t * LR_L + s] = c[r] * w;
    }
  }
  if (!DELTA) return;
  __syncthreads();
  // column c of (I + A)^-1 by forward substitution, lane = column
  if (tid < LR_L) {
    float x[LR_L];
#pragma unroll
    for (int t = 0; t < LR_L; ++t) {
      float v = t == tid ? 1.f : 0.f;
#pragma unroll
      for (int s = 0; s + 4 <= t; s += 4) {
        const float4 m = *reinterpret_cast<const float4*>(A + t * LR_PS + s);
        v = fmaf(-m.x, x[s], v);
        v = fmaf(-m.y, x[s + 1], v);
        v = fmaf(-m.z, x[s + 2], v);
        v = fmaf(-m.w, x[s + 3], v);
      }
#pragma unroll
      for (int s = t & ~3; s < t; ++s) v = fmaf(-A[t * LR_PS + s], x[s], v);
      x[t] = v;
    }
    const float be = s_beta[tid];
    float* M = a.M + th * LR_L * LR_L + tid;
#pragma unroll
    for (int t = 0; t < LR_L; ++t) M[t * LR_L] = x[t] * be;
  }
}

// 8 (bf16) or 4 (float) value elements in flight
template <typename T>
struct LrPiece;
template <>
struct LrPiece<bf16_t> {
  static constexpr int N = 8;
  int4 v;
  DEVINL void zero() { v = make_int4(0, 0, 0, 0); }
  DEVINL void fetch(const bf16_t* p) { v = *reinterpret_cast<const int4*>(p); }
  DEVINL float get(int e) const {
    bf16x8 r;
    r.raw = v;
    return bf16x8_get(r, e);
  }
};
template <>
struct LrPiece<float> {
  static constexpr int N = 4;
  float v[4];
  DEVINL void zero() { v[0] = v[1] = v[2] = v[3] = 0.f; }
  DEVINL void fetch(const float* p) {
    const float4 x = *reinterpret_cast<const float4*>(p);
    v[0] = x.x; v[1] = x.y; v[2] = x.z; v[3] = x.w;
  }
  DEVINL float get(int e) const { return v[e]; }
};

// grid (column slices of 64, H, B), 4 waves of 16 columns.
// LDS: Q, K [L][D + 4] | V [L][68] | P [L][LR_PS] | M [L][LR_PS] (delta rule)
template <typename T, int D, bool VEC, bool DELTA>
__global__ __launch_bounds__(256) void lr_chunk_kernel(LrArgs a) {
  constexpr int KS = D + 4, VS = LR_COLS + 4, NB = D / 16, TB = LR_L / 16;
  constexpr int QC = LR_L * D / (256 * 4);            // float4 pieces a thread: q, k
  constexpr int VN = LrPiece<T>::N;
  constexpr int VC = LR_L * LR_COLS / (256 * VN);     // value pieces a thread
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float e_in[LR_L], w_out[LR_L];
  float* Q = lds;
  float* K = Q + LR_L * KS;
  float* V = K + LR_L * KS;
  float* P = V + LR_L * VS;
  float* M = P + LR_L * LR_PS;
  const int b = blockIdx.z, h = blockIdx.y, c0 = blockIdx.x * LR_COLS;
  const int t0 = a.cu[b], t1 = a.cu[b + 1];
  if (t0 >= t1) return;
  int tile = 0;
  for (int i = 0; i < b; ++i) tile += (a.cu[i + 1] - a.cu[i] + LR_L - 1) / LR_L;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int l15 = lane & 15, g = lane >> 4;
  const int d = a.d, dv = a.dv, gq = h / (a.H / a.G);
  const int jc = wave * 16 + l15, j = c0 + jc;
  const bool jok = j < dv;
  const bool busy = c0 + wave * 16 < dv;   // a wave with columns of its own

  float* S = a.state + (a.slots[b] * a.H + h) * (int64_t)d * dv;
  const bool fresh = a.positions[t0] == 0;
  f32x4v st[NB];
#pragma unroll
  for (int nb = 0; nb < NB; ++nb)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 16 * nb + 4 * g + r;
      st[nb][r] = (!fresh && jok && i < d) ? S[(int64_t)i * dv + j] : 0.f;
    }

  const float* qp = a.qp + (int64_t)gq * d;
  const float* kp = a.kp + (int64_t)gq * d;
  const int64_t qs = (int64_t)a.G * d;
  const T* vp = (const T*)a.v + h * a.vh;
  float4 qr[QC], kr[QC], pr, mr;
  LrPiece<T> vr[VC];
  float er = 0.f;
  auto fetch = [&](int tc, int tl) {
    const int n = min(LR_L, t1 - tc);
    const int64_t th = (int64_t)tl * a.H + h;
#pragma unroll
    for (int c = 0; c < QC; ++c) {
      const int p = c * 256 + tid, t = p / (D / 4), f = (p % (D / 4)) * 4;
      qr[c] = kr[c] = make_float4(0.f, 0.f, 0.f, 0.f);
      if (t < n) {
        const int64_t o = (int64_t)(tc + t) * qs + f;
        if (VEC) {
          if (f < d) {
            qr[c] = *reinterpret_cast<const float4*>(qp + o);
            kr[c] = *reinterpret_cast<const float4*>(kp + o);
          }
        } else {
          if (f < d) { qr[c].x = qp[o]; kr[c].x = kp[o]; }
          if (f + 1 < d) { qr[c].y = qp[o + 1]; kr[c].y = kp[o + 1]; }
          if (f + 2 < d) { qr[c].z = qp[o + 2]; kr[c].z = kp[o + 2]; }
          if (f + 3 < d) { qr[c].w = qp[o + 3]; kr[c].w = kp[o + 3]; }
        }
      }
    }
    if (VEC) {
#pragma unroll
      for (int c = 0; c < VC; ++c) {
        const int p = c * 256 + tid, t = p / (LR_COLS / VN);
        const int f = c0 + (p % (LR_COLS / VN)) * VN;
        if (t < n && f < dv) vr[c].fetch(vp + (int64_t)(tc + t) * a.vs + f);
        else vr[c].zero();
      }
    }
    pr = *reinterpret_cast<const float4*>(a.P + th * LR_L * LR_L + tid * 4);
    if (DELTA) mr = *reinterpret_cast<const float4*>(a.M + th * LR_L * LR_L + tid * 4);
    if (tid < LR_L) er = a.e_in[th * LR_L + tid];
    else if (tid < 2 * LR_L) er = a.w_out[th * LR_L + tid - LR_L];
  };
  auto stash = [&](int tc) {
#pragma unroll
    for (int c = 0; c < QC; ++c) {
      const int p = c * 256 + tid, t = p / (D / 4), f = (p % (D / 4)) * 4;
      *reinterpret_cast<float4*>(Q + t * KS + f) = qr[c];
      *reinterpret_cast<float4*>(K + t * KS + f) = kr[c];
    }
    if (VEC) {
#pragma unroll
      for (int c = 0; c < VC; ++c) {
        const int p = c * 256 + tid, t = p / (LR_COLS / VN);
        const int f = (p % (LR_COLS / VN)) * VN;
#pragma unroll
        for (int e = 0; e < VN; e += 4) {
          float x[4];
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            x[i] = vr[c].get(e + i);
            if (!DELTA && a.silu) x[i] = lr_silu(x[i]);
          }
          *reinterpret_cast<float4*>(V + t * VS + f + e) =
              make_float4(x[0], x[1], x[2], x[3]);
        }
      }
    } else {
      const int n = min(LR_L, t1 - tc);
      for (int p = tid; p < LR_L * LR_COLS; p += 256) {
        const int t = p / LR_COLS, f = p % LR_COLS;
        float x = 0.f;
        if (t < n && c0 + f < dv) x = ldf(vp + (int64_t)(tc + t) * a.vs + c0 + f);
        V[t * VS + f] = (!DELTA && a.silu) ? lr_silu(x) : x;
      }
    }
    const int pt = tid / (LR_L / 4), pf = (tid % (LR_L / 4)) * 4;
    *reinterpret_cast<float4*>(P + pt * LR_PS + pf) = pr;
    if (DELTA) *reinterpret_cast<float4*>(M + pt * LR_PS + pf) = mr;
    if (tid < LR_L) e_in[tid] = er;
    else if (tid < 2 * LR_L) w_out[tid - LR_L] = er;
  };

  fetch(t0, tile);
  for (int tc = t0; tc < t1; tc += LR_L, ++tile) {
    const int n = min(LR_L, t1 - tc);
    __syncthreads();   // the previous chunk's reads are done
    stash(tc);
    __syncthreads();
    if (tc + LR_L < t1) fetch(tc + LR_L, tile + 1);
    if (!busy) continue;   // its barriers are the loop's own two

    // ---- q . S_0 (and k . S_0) -------------------------------------------------------
    f32x4v O[TB], R[TB];
#pragma unroll
    for (int tb = 0; tb < TB; ++tb)
#pragma unroll
      for (int r = 0; r < 4; ++r) O[tb][r] = R[tb][r] = 0.f;
#pragma unroll
    for (int nb = 0; nb < NB; ++nb)
#pragma unroll
      for (int tb = 0; tb < TB; ++tb) {
        const float4 x = *reinterpret_cast<const float4*>(
            Q + (16 * tb + l15) * KS + 16 * nb + 4 * g);
        O[tb] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.x, st[nb][0], O[tb], 0, 0, 0);
        O[tb] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.y, st[nb][1], O[tb], 0, 0, 0);
        O[tb] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.z, st[nb][2], O[tb], 0, 0, 0);
        O[tb] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.w, st[nb][3], O[tb], 0, 0, 0);
        if (DELTA) {
          const float4 y = *reinterpret_cast<const float4*>(
              K + (16 * tb + l15) * KS + 16 * nb + 4 * g);
          R[tb] = __builtin_amdgcn_mfma_f32_16x16x4f32(y.x, st[nb][0], R[tb], 0, 0, 0);
          R[tb] = __builtin_amdgcn_mfma_f32_16x16x4f32(y.y, st[nb][1], R[tb], 0, 0, 0);
          R[tb] = __builtin_amdgcn_mfma_f32_16x16x4f32(y.z, st[nb][2], R[tb], 0, 0, 0);
          R[tb] = __builtin_amdgcn_mfma_f32_16x16x4f32(y.w, st[nb][3], R[tb], 0, 0, 0);
        }
      }
    // ---- u -------------------------------------------------------------------------------
    f32x4v U[TB];
#pragma unroll
    for (int tb = 0; tb < TB; ++tb)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = 16 * tb + 4 * g + r;
        const float v = V[t * VS + jc], e = e_in[t];
        O[tb][r] *= e;
        if (DELTA) R[tb][r] = fmaf(-e, R[tb][r], v);
        else U[tb][r] = v;
      }
    if (DELTA) {
#pragma unroll
      for (int tb = 0; tb < TB; ++tb) {
        f32x4v c = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int sb = 0; sb <= tb; ++sb) {
          const float4 x = *reinterpret_cast<const float4*>(
              M + (16 * tb + l15) * LR_PS + 16 * sb + 4 * g);
          c = __builtin_amdgcn_mfma_f32_16x16x4f32(x.x, R[sb][0], c, 0, 0, 0);
          c = __builtin_amdgcn_mfma_f32_16x16x4f32(x.y, R[sb][1], c, 0, 0, 0);
          c = __builtin_amdgcn_mfma_f32_16x16x4f32(x.z, R[sb][2], c, 0, 0, 0);
          c = __builtin_amdgcn_mfma_f32_16x16x4f32(x.w, R[sb][3], c, 0, 0, 0);
        }
        U[tb] = c;
      }
    }
    // ---- o += P u --------------------------------------------------------------------------
#pragma unroll
    for (int tb = 0; tb < TB; ++tb) {
#pragma unroll
      for (int sb = 0; sb <= tb; ++sb) {
        const float4 x = *reinterpret_cast<const float4*>(
            P + (16 * tb + l15) * LR_PS + 16 * sb + 4 * g);
        O[tb] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.x, U[sb][0], O[tb], 0, 0, 0);
        O[tb] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.y, U[sb][1], O[tb], 0, 0, 0);
        O[tb] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.z, U[sb][2], O[tb], 0, 0, 0);
        O[tb] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.w, U[sb][3], O[tb], 0, 0, 0);
      }
      if (jok) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int t = 16 * tb + 4 * g + r;
          if (t < n) a.o[((int64_t)(tc + t) * a.H + h) * dv + j] = O[tb][r];
        }
      }
    }
    // ---- the state after the chunk -----------------------------------------------------------
    const float dec = e_in[n - 1];
#pragma unroll
    for (int nb = 0; nb < NB; ++nb)
#pragma unroll
      for (int r = 0; r < 4; ++r) st[nb][r] *= dec;
#pragma unroll
    for (int tb = 0; tb < TB; ++tb)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = 16 * tb + 4 * g + r;
        const float u = U[tb][r] * w_out[t];
        const float* kr_ = K + t * KS + l15;
#pragma unroll
        for (int nb = 0; nb < NB; ++nb)
          st[nb] = __builtin_amdgcn_mfma_f32_16x16x4f32(kr_[16 * nb], u, st[nb], 0, 0, 0);
      }
  }
  if (jok) {
#pragma unroll
    for (int nb = 0; nb < NB; ++nb)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 16 * nb + 4 * g + r;
        if (i < d) S[(int64_t)i * dv + j] = st[nb][r];
      }
  }
}

// ---- launches -----------------------------------------------------------------------

template <typename F>
static void lr_raise_lds(F fn, size_t shm) {
  // gfx950 has 160 KB of LDS per CU; more than 64 KB per workgroup is opt-in
  if (shm > 64 * 1024)
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(fn),
                              hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024);
}

template <typename T, int D, bool VEC, bool DELTA>
static void launch_lr_chunk(const LrArgs& a, int tiles) {
  const size_t tile = sizeof(float) * 2 * LR_L * (D + 4);
  const size_t mat = sizeof(float) * LR_L * LR_PS;
  const size_t shm_p = tile + (DELTA ? mat : 0);
  const size_t shm_c = tile + sizeof(float) * LR_L * (LR_COLS + 4) + mat + (DELTA ? mat : 0);
  static bool raised = false;
  if (!raised) {
    lr_raise_lds(&lr_prep_kernel<T, D, VEC, DELTA>, shm_p);
    lr_raise_lds(&lr_chunk_kernel<T, D, VEC, DELTA>, shm_c);
    raised = true;
  }
  hipLaunchKernelGGL((lr_prep_kernel<T, D, VEC, DELTA>), dim3(tiles, a.H), dim3(256),
                     shm_p, a.stream, a);
  hipLaunchKernelGGL((lr_chunk_kernel<T, D, VEC, DELTA>),
                     dim3((a.dv + LR_COLS - 1) / LR_COLS, a.H, a.B), dim3(256), shm_c,
                     a.stream, a);
}

template <typename T, bool VEC, bool DELTA>
static void launch_lr_chunk_d(const LrArgs& a, int tiles) {
  if (a.d <= 64) launch_lr_chunk<T, 64, VEC, DELTA>(a, tiles);
  else if (a.d <= 128) launch_lr_chunk<T, 128, VEC, DELTA>(a, tiles);
  else launch_lr_chunk<T, 256, VEC, DELTA>(a, tiles);
}

template <typename T, int CN, int N, bool DELTA>
static void launch_lr_scan(const LrArgs& a) {
  constexpr int CW = CN * N;
  const size_t shm = sizeof(float) * (2 * (size_t)a.d + CW + 8 * CW + 2);
  hipLaunchKernelGGL((lr_scan_kernel<T, CN, N, DELTA>),
                     dim3((a.dv + CW - 1) / CW, a.H, a.B), dim3(256), shm, a.stream, a);
}

template <typename T, bool DELTA>
static void launch_lr(const LrArgs& a, int tiles, int vec) {
  if (tiles > 0) {
    if (vec) launch_lr_chunk_d<T, true, DELTA>(a, tiles);
    else launch_lr_chunk_d<T, false, DELTA>(a, tiles);
    return;
  }
  const bool n4 = a.dv % 4 == 0;
  if (a.d <= 512) {   // 32 row groups of at most 16 rows
    if (n4) launch_lr_scan<T, 8, 4, DELTA>(a);
    else launch_lr_scan<T, 8, 1, DELTA>(a);
  } else {            // 64 row groups
    if (n4) launch_lr_scan<T, 4, 4, DELTA>(a);
    else launch_lr_scan<T, 4, 1, DELTA>(a);
  }
}

extern "C" int linear_recurrence_chunk() { return LR_L; }

// strides: token and head strides of q, k, v. tiles > 0: chunks (d <= 256, cu and
// scratch given, tiles an upper bound of the chunks; vec: rows of q, k and v start
// 16-byte aligned, d and dv multiples of 8); 0: token by token (d <= 1024)
extern "C" void launch_linear_recurrence(
    float* o, const void* q, const void* k, const void* v, const int64_t* strides,
    float q_scale, float k_scale, int silu, const float* cs, int n_rot,
    const float* pw, int pw_n, const float* gates, const float* a_log,
    const float* dt_bias, float* state, const int64_t* slots, const int* cu,
    const int* positions, int B, int H, int G, int d, int dv, float* qp, float* kp,
    float* P, float* M, float* e_in, float* w_out, int tiles, int vec, int kind,
    hipStream_t stream) {
  if (B == 0) return;
  const LrArgs a{o, q, k, v, strides[0], strides[1], strides[2], strides[3], strides[4],
                 strides[5], q_scale, k_scale, silu, cs, n_rot, pw, pw_n, gates, a_log,
                 dt_bias, state, slots, cu, positions, B, H, G, d, dv, qp, kp, P, M,
                 e_in, w_out, stream};
  const bool delta = gates != nullptr;
  if (kind == 0) {
    if (delta) launch_lr<bf16_t, true>(a, tiles, vec);
    else launch_lr<bf16_t, false>(a, tiles, vec);
  } else {
    if (delta) launch_lr<float, true>(a, tiles, vec);
    else launch_lr<float, false>(a, tiles, vec);
  }
}
