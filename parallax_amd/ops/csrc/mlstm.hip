// Matrix LSTM: per head a matrix memory S [d, dv], a normaliser n [d] and a
// running maximum m, with scalar exponential gates per token,
//
//     i = cap tanh((z_i + b_i) / cap),   f = logsigmoid(cap tanh((z_f + b_f) / cap)),
//     m' = max(f + m, i),  a = exp(f + m - m'),  b = exp(i - m'),
//     S <- a S + b k v^T,  n <- a n + b k,
//     o = S^T q / (max(|n . q|, exp(-m')) + 1e-6),   q scaled by d^-1/2,
//
// then o / rms(o) * w * sigmoid(g) per head. State, gates and normalisation
// are fp32. A state row per (slot, head) is [S, row-major d x dv | n | m],
// `sw` floats apart; a sequence whose first token of the launch sits at
// position 0 starts from zeros instead of the slot's old content.
//
//   mlstm_step  : decode, one token per sequence: a workgroup per (head,
//                 sequence) streams the head's state through once (load,
//                 decay, add, multiply with q, store) and finishes the head's
//                 output in the same launch.
//   mlstm_scan  : any portion, token by token: a thread owns 16 rows of one
//                 state column in registers (G lanes share a column), as in
//                 gated linear attention; the normaliser is one more column
//                 whose values are 1.
//   mlstm_chunk : bf16 portions, 64 tokens at a time on the matrix cores. With
//                 F the running sum of f inside the chunk, G_s = i_s - F_s and
//                 M_t = max(m_0, max_{s <= t} G_s) the recurrence unrolls to
//                   S_t  = exp(m_0 - M_t) S_0 + sum_{s <= t} exp(G_s - M_t) k_s v_s^T,
//                   m_t  = F_t + M_t,
//                 every exponent <= 0 and F cancelled out of the weights. F, G
//                 and M are formed in float64 and kept as two floats each, so a
//                 difference of two large sums keeps fp32 accuracy. q, k and v
//                 are bf16 numbers, so q . k is exact on the bf16 matrix cores;
//                 fp32 factors (weights, state) are split into three bf16
//                 numbers that add up to them exactly, as in the row attention.
//   mlstm_out   : the head norm, weight and output gate of the two prompt
//                 kernels' results; the last token's maximum goes to the state.
#include "seq_common.h"

#define ML_EPS 1e-6f

DEVINL float ml_cap(float z, float cap) { return cap * tanhf(z / cap); }
DEVINL float ml_logsig(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }
DEVINL float ml_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }

template <typename T>
DEVINL void ml_load4(const T* p, float* v);
template <>
DEVINL void ml_load4<float>(const float* p, float* v) {
  const float4 a = *reinterpret_cast<const float4*>(p);
  v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w;
}

template <>
DEVINL void ml_load4<bf16_t>(const bf16_t* p, float* v) {
  const uint2 raw = *reinterpret_cast<const uint2*>(p);
  v[0] = bf16_bits_to_f32((uint16_t)(raw.x & 0xffff));
  v[1] = bf16_bits_to_f32((uint16_t)(raw.x >> 16));
  v[2] = bf16_bits_to_f32((uint16_t)(raw.y & 0xffff));
  v[3] = bf16_bits_to_f32((uint16_t)(raw.y >> 16));
}
template <typename T>
DEVINL void ml_store4(T* p, const float* v);
template <>
DEVINL void ml_store4<float>(float* p, const float* v) {
  *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
}
template <>
DEVINL void ml_store4<bf16_t>(bf16_t* p, const float* v) {
  uint2 raw;
  raw.x = (uint32_t)f32_to_bf16_bits(v[0]) | ((uint32_t)f32_to_bf16_bits(v[1]) << 16);
  raw.y = (uint32_t)f32_to_bf16_bits(v[2]) | ((uint32_t)f32_to_bf16_bits(v[3]) << 16);
  *reinterpret_cast<uint2*>(p) = raw;
}

// ---- decode ----------------------------------------------------------------------

// grid (H, B); N = 4 (dv a multiple of 4) or 1 columns per thread.
// LDS: q [d] | k [d] | v [dv] | o [dv] | partial sums [256 * N] | 8
template <typename T, int N>
__global__ __launch_bounds__(256) void mlstm_step_kernel(
    T* __restrict__ out, const T* __restrict__ q, int64_t q_stride,
    const T* __restrict__ k, int64_t k_stride, const T* __restrict__ v,
    int64_t v_stride, const T* __restrict__ g, int64_t g_stride,
    const float* __restrict__ gates, const float* __restrict__ gate_bias,
    const T* __restrict__ norm_w, float cap, float eps, float* __restrict__ state,
    int64_t sw, const int64_t* __restrict__ slots,
    const int* __restrict__ positions, int H, int d, int dv, float q_scale) {
  extern __shared__ float lds[];
  const int h = blockIdx.x;
  const int64_t t = blockIdx.y;
  const int tid = threadIdx.x;
  const int dvp = (dv + 3) & ~3, dp = (d + 3) & ~3;
  float* sq = lds;
  float* sk = sq + dp;
  float* sv = sk + dp;
  float* so = sv + dvp;
  float* part = so + dvp;
  float* red = part + 256 * N;

  for (int i = tid; i < d; i += 256) {
    sq[i] = ldf(q + t * q_stride + h * d + i) * q_scale;
    sk[i] = ldf(k + t * k_stride + h * d + i);
  }
  for (int j = tid; j < dv; j += 256) sv[j] = ldf(v + t * v_stride + h * dv + j);
  float* S = state + (slots[t] * H + h) * sw;
  float* nv = S + (int64_t)d * dv;
  const bool fresh = positions[t] == 0;
  const float gi = ml_cap(gates[t * 2 * H + h] + gate_bias[h], cap);
  const float gf = ml_logsig(ml_cap(gates[t * 2 * H + H + h] + gate_bias[H + h], cap));
  const float m0 = fresh ? 0.f : nv[d];
  const float m1 = fmaxf(gf + m0, gi);
  const float a = fresh ? 0.f : expf(gf + m0 - m1);
  const float b = expf(gi - m1);
  __syncthreads();   // q, k, v are staged; every thread has read m

  float nq = 0.f;
  for (int i = tid; i < d; i += 256) {
    float x = b * sk[i];
    if (!fresh) x = fmaf(a, nv[i], x);
    nv[i] = x;
    nq = fmaf(x, sq[i], nq);
  }
  if (tid == 0) nv[d] = m1;
  nq = block256_sum(nq, red);
  const float den = 1.0f / (fmaxf(fabsf(nq), expf(-m1)) + ML_EPS);

  const int ncg = dv / N;            // column groups
  for (int c0 = 0; c0 < ncg; c0 += 256) {
    const int cn = min(256, ncg - c0);
    const int rg_n = 256 / cn;       // row groups
    const int cg = tid % cn, rg = tid / cn;
    float acc[N];
#pragma unroll
    for (int j = 0; j < N; ++j) acc[j] = 0.f;
    if (rg < rg_n) {
      const int col = (c0 + cg) * N;
      float vv[N];
#pragma unroll
      for (int j = 0; j < N; ++j) vv[j] = sv[col + j];
      float* p = S + col;
#pragma unroll 8
      for (int i = rg; i < d; i += rg_n) {
        float s[N];
        const float bk = b * sk[i], qi = sq[i];
        if (!fresh) {
          if (N == 4) ml_load4<float>(p + (int64_t)i * dv, s);
          else s[0] = p[(int64_t)i * dv];
        }
#pragma unroll
        for (int j = 0; j < N; ++j) {
          s[j] = fresh ? bk * vv[j] : fmaf(a, s[j], bk * vv[j]);
          acc[j] = fmaf(s[j], qi, acc[j]);
        }
        if (N == 4)
          *reinterpret_cast<float4*>(p + (int64_t)i * dv) =
              make_float4(s[0], s[1 % N], s[2 % N], s[3 % N]);
        else
          p[(int64_t)i * dv] = s[0];
      }
    }
#pragma unroll
    for (int j = 0; j < N; ++j) part[tid * N + j] = acc[j];
    __syncthreads();
    for (int c = tid; c < cn * N; c += 256) {
      float o = 0.f;
      for (int r = 0; r < rg_n; ++r) o += part[(r * cn + c / N) * N + c % N];
      so[c0 * N + c] = o * den;
    }
    __syncthreads();
  }
  float ss = 0.f;
  for (int j = tid; j < dv; j += 256) ss = fmaf(so[j], so[j], ss);
  const float r = 1.0f / sqrtf(block256_sum(ss, red) / (float)dv + eps);
  for (int j = tid; j < dv; j += 256)
    stf(out + (t * H + h) * (int64_t)dv + j,
        so[j] * r * ldf(norm_w + h * dv + j) *
            ml_sigmoid(ldf(g + t * g_stride + h * dv + j)));
}

// ---- token-serial portions -------------------------------------------------------

#define ML_ROWS 16   // state rows per lane
#define ML_TC_MAX 16 // tokens staged per pass

// o [T, H, dv], nq and mm [T, H]: unnormalised sums, n . q, running maximum
template <typename T>
__global__ __launch_bounds__(256) void mlstm_scan_kernel(
    float* __restrict__ o, float* __restrict__ nq_out, float* __restrict__ mm,
    const T* __restrict__ q, int64_t q_stride, const T* __restrict__ k,
    int64_t k_stride, const T* __restrict__ v, int64_t v_stride,
    const float* __restrict__ gates, const float* __restrict__ gate_bias,
    float cap, float* __restrict__ state, int64_t sw,
    const int64_t* __restrict__ slots, const int* __restrict__ cu,
    const int* __restrict__ positions, int H, int d, int dv, int G, int TC,
    float q_scale) {
  extern __shared__ float lds[];
  __shared__ float s_i[ML_TC_MAX], s_f[ML_TC_MAX], s_a[ML_TC_MAX],
      s_b[ML_TC_MAX], s_m[ML_TC_MAX];
  const int b = blockIdx.z, h = blockIdx.y;
  const int C = 64 / G;  // columns per wave
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int g = lane / C;
  const int jb = wave * C + lane % C;  // column within the block
  const int j = blockIdx.x * 4 * C + jb;
  const bool is_n = j == dv;           // the normaliser: one column of ones
  const bool jvalid = j <= dv;
  const int t0 = cu ? cu[b] : b;
  const int t1 = cu ? cu[b + 1] : b + 1;
  if (t0 >= t1) return;
  const int dkp = G * ML_ROWS;
  float* sq = lds;
  float* sk = sq + TC * dkp;
  float* sv = sk + TC * dkp;  // [TC][4 * C]

  float* S = state + (slots[b] * H + h) * sw;
  float* col = is_n ? S + (int64_t)d * dv : S + j;
  const int64_t cstep = is_n ? 1 : dv;
  const bool fresh = positions[t0] == 0;
  // m is written back by mlstm_out, when every workgroup has read it
  float m = fresh ? 0.f : S[(int64_t)d * dv + d];
  float s[ML_ROWS];
#pragma unroll
  for (int r = 0; r < ML_ROWS; ++r) {
    const int i = g * ML_ROWS + r;
    s[r] = (!fresh && jvalid && i < d) ? col[i * cstep] : 0.f;
  }
  const float bi = gate_bias[h], bf = gate_bias[H + h];

  for (int tc = t0; tc < t1; tc += TC) {
    const int n = min(TC, t1 - tc);
    __syncthreads();
    for (int idx = threadIdx.x; idx < n * dkp; idx += 256) {
      const int tt = idx / dkp, i = idx % dkp;
      float qf = 0.f, kf = 0.f;
      if (i < d) {
        const int64_t tok = tc + tt;
        qf = ldf(q + tok * q_stride + h * d + i) * q_scale;
        kf = ldf(k + tok * k_stride + h * d + i);
      }
      sq[idx] = qf;
      sk[idx] = kf;
    }
    for (int idx = threadIdx.x; idx < n * 4 * C; idx += 256) {
      const int tt = idx / (4 * C), jj = idx % (4 * C);
      const int cj = blockIdx.x * 4 * C + jj;
      sv[idx] = cj < dv ? ldf(v + (int64_t)(tc + tt) * v_stride + h * dv + cj)
                        : (cj == dv ? 1.f : 0.f);
    }
    if (threadIdx.x < n) {
      const float* gr = gates + (int64_t)(tc + threadIdx.x) * 2 * H;
      s_i[threadIdx.x] = ml_cap(gr[h] + bi, cap);
      s_f[threadIdx.x] = ml_logsig(ml_cap(gr[H + h] + bf, cap));
    }
    __syncthreads();
    // every thread walks the chain of maxima (add and max only), thread tt
    // keeps token tt's factors
    for (int tt = 0; tt < n; ++tt) {
      const float fm = s_f[tt] + m;
      const float m1 = fmaxf(fm, s_i[tt]);
      if (threadIdx.x == tt) {
        s_a[tt] = expf(fm - m1);
        s_b[tt] = expf(s_i[tt] - m1);
        s_m[tt] = m1;
      }
      m = m1;
    }
    __syncthreads();
    for (int tt = 0; tt < n; ++tt) {
      const float a = s_a[tt], bv = s_b[tt] * sv[tt * 4 * C + jb];
      const float* aq = sq + tt * dkp + g * ML_ROWS;
      const float* ak = sk + tt * dkp + g * ML_ROWS;
      float acc = 0.f;
#pragma unroll
      for (int r = 0; r < ML_ROWS; ++r) {
        s[r] = fmaf(a, s[r], ak[r] * bv);
        acc = fmaf(s[r], aq[r], acc);
      }
      for (int off = C; off < 64; off <<= 1) acc += __shfl_xor(acc, off, 64);
      if (g == 0 && jvalid) {
        const int64_t th = (int64_t)(tc + tt) * H + h;
        if (is_n) {
          nq_out[th] = acc;
          mm[th] = s_m[tt];
        } else {
          o[th * dv + j] = acc;
        }
      }
    }
  }
  if (jvalid) {
#pragma unroll
    for (int r = 0; r < ML_ROWS; ++r) {
      const int i = g * ML_ROWS + r;
      if (i < d) col[i * cstep] = s[r];
    }
  }
}

// ---- portions in chunks on the matrix cores --------------------------------------

typedef float f32x16v __attribute__((ext_vector_type(16)));

#define MC_L 64        // tokens per chunk
#define MC_COLS 64     // value columns per workgroup
#define MC_KPAD 8      // bf16 elements of padding per [token][feature] row
#define MC_TS 68       // bf16 elements per [feature][token] row: 64 + 4 (136 bytes)

// x = hi + mid + lo exactly, each a bf16 number
DEVINL void ml_split3(float x, short& hi, short& mid, short& lo) {
  const uint32_t b0 = __float_as_uint(x) & 0xffff0000u;
  const float r1 = x - __uint_as_float(b0);
  const uint32_t b1 = __float_as_uint(r1) & 0xffff0000u;
  const float r2 = r1 - __uint_as_float(b1);
  hi = (short)(b0 >> 16);
  mid = (short)(b1 >> 16);
  lo = (short)(__float_as_uint(r2) >> 16);
}

// 8 elements of an LDS row for the operand slots of lane half h at step s:
// elements 16 s + 4 h + (0 .. 3) and 16 s + 8 + 4 h + (0 .. 3), the rows an
// accumulator's registers 8 s .. 8 s + 7 hold
DEVINL bf16x8v mc_slots(const bf16_t* row, int s, int half) {
  const int2 v0 = *reinterpret_cast<const int2*>(row + 16 * s + 4 * half);
  const int2 v1 = *reinterpret_cast<const int2*>(row + 16 * s + 8 + 4 * half);
  const int4 p = make_int4(v0.x, v0.y, v1.x, v1.y);
  return *reinterpret_cast<const bf16x8v*>(&p);
}

DEVINL double ml_shfl_up(double x, int off) {
  return __shfl_up(x, off, 64);
}

// Per sequence and head: grid (column slices of 64, H, B), 4 waves = 2 token
// halves x 2 column halves of 32. A wave keeps its 32 columns of the whole
// state in accumulators (lane = column, registers = key features), as the B
// operand of q . S and the accumulator of the update alike; the two waves of a
// column half hold the same numbers. D: padded key width (64 | 128).
template <int D>
__global__ __launch_bounds__(256, 2) void mlstm_chunk_kernel(
    float* __restrict__ o, float* __restrict__ nq_out, float* __restrict__ mm,
    const bf16_t* __restrict__ q, int64_t q_stride, const bf16_t* __restrict__ k,
    int64_t k_stride, const bf16_t* __restrict__ v, int64_t v_stride,
    const float* __restrict__ gates, const float* __restrict__ gate_bias,
    float cap, float* __restrict__ state, int64_t sw,
    const int64_t* __restrict__ slots, const int* __restrict__ cu,
    const int* __restrict__ positions, int H, int d, int dv, float q_scale) {
  constexpr int KS = D + MC_KPAD;
  constexpr int NB = D / 32;                 // state blocks of 32 features
  constexpr int QC = MC_L * D / (256 * 8);   // 16-byte pieces per thread: q, k
  constexpr int VC = MC_L * MC_COLS / (256 * 8);
  __shared__ __attribute__((aligned(16))) bf16_t Qs[MC_L * KS];
  __shared__ __attribute__((aligned(16))) bf16_t Ks[MC_L * KS];
  __shared__ __attribute__((aligned(16))) bf16_t Kt[D * MC_TS];
  __shared__ __attribute__((aligned(16))) bf16_t Vt[MC_COLS * MC_TS];
  __shared__ float sn[D];                    // normaliser
  __shared__ float nqp[4 * MC_L];            // partial n . q
  __shared__ float g_hi[MC_L], g_lo[MC_L], m_hi[MC_L], m_lo[MC_L];
  __shared__ float e_in[MC_L];               // exp(m_0 - M_t)
  __shared__ float w_out[MC_L];              // exp(G_s - M_L)
  __shared__ float m_tok[MC_L];
  __shared__ float s_end[2];                 // exp(m_0 - M_L), m_L

  const int b = blockIdx.z, h = blockIdx.y, c0 = blockIdx.x * MC_COLS;
  const int t0 = cu[b], t1 = cu[b + 1];
  if (t0 >= t1) return;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int half = lane >> 5, l31 = lane & 31;
  const int tt0 = (wave & 1) * 32;           // this wave's tokens of the chunk
  const int jc = (wave >> 1) * 32 + l31;     // its column within the slice
  const int j = c0 + jc;
  const bool jok = j < dv;
  const bool owner = blockIdx.x == 0;        // this slice keeps the normaliser

  float* S = state + (slots[b] * H + h) * sw;
  const bool fresh = positions[t0] == 0;
  float m0 = fresh ? 0.f : S[(int64_t)d * dv + d];
  f32x16v st[NB];
#pragma unroll
  for (int nb = 0; nb < NB; ++nb)
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int i = 32 * nb + 8 * (r >> 2) + 4 * half + (r & 3);
      st[nb][r] = (!fresh && jok && i < d) ? S[(int64_t)i * dv + j] : 0.f;
    }
  if (owner)
    for (int i = tid; i < D; i += 256)
      sn[i] = (!fresh && i < d) ? S[(int64_t)d * dv + i] : 0.f;
  const float bi = gate_bias[h], bf = gate_bias[H + h];

  int4 qr[QC], kr[QC], vr[VC];
  float zi = 0.f, zf = 0.f;
  auto fetch = [&](int tc) {
    const int n = min(MC_L, t1 - tc);
#pragma unroll
    for (int c = 0; c < QC; ++c) {
      const int p = c * 256 + tid;
      const int tt = p / (D / 8), f = (p % (D / 8)) * 8;
      const bool on = tt < n && f < d;
      qr[c] = on ? *reinterpret_cast<const int4*>(q + (int64_t)(tc + tt) * q_stride + h * d + f)
                 : make_int4(0, 0, 0, 0);
      kr[c] = on ? *reinterpret_cast<const int4*>(k + (int64_t)(tc + tt) * k_stride + h * d + f)
                 : make_int4(0, 0, 0, 0);
    }
#pragma unroll
    for (int c = 0; c < VC; ++c) {
      const int p = c * 256 + tid;
      const int tt = p / (MC_COLS / 8), f = c0 + (p % (MC_COLS / 8)) * 8;
      vr[c] = (tt < n && f < dv)
                  ? *reinterpret_cast<const int4*>(v + (int64_t)(tc + tt) * v_stride + h * dv + f)
                  : make_int4(0, 0, 0, 0);
    }
    if (wave == 0 && lane < n) {
      const float* gr = gates + (int64_t)(tc + lane) * 2 * H;
      zi = gr[h];
      zf = gr[H + h];
    }
  };
  auto stash = [&]() {
#pragma unroll
    for (int c = 0; c < QC; ++c) {
      const int p = c * 256 + tid;
      const int tt = p / (D / 8), f = (p % (D / 8)) * 8;
      *reinterpret_cast<int4*>(Qs + tt * KS + f) = qr[c];
      *reinterpret_cast<int4*>(Ks + tt * KS + f) = kr[c];
      const uint32_t w[4] = {(uint32_t)kr[c].x, (uint32_t)kr[c].y,
                             (uint32_t)kr[c].z, (uint32_t)kr[c].w};
#pragma unroll
      for (int e = 0; e < 8; ++e)
        Kt[(f + e) * MC_TS + tt] =
            (bf16_t)((e & 1) ? (w[e >> 1] >> 16) : (w[e >> 1] & 0xffffu));
    }
#pragma unroll
    for (int c = 0; c < VC; ++c) {
      const int p = c * 256 + tid;
      const int tt = p / (MC_COLS / 8), f = (p % (MC_COLS / 8)) * 8;
      const uint32_t w[4] = {(uint32_t)vr[c].x, (uint32_t)vr[c].y,
                             (uint32_t)vr[c].z, (uint32_t)vr[c].w};
#pragma unroll
      for (int e = 0; e < 8; ++e)
        Vt[(f + e) * MC_TS + tt] =
            (bf16_t)((e & 1) ? (w[e >> 1] >> 16) : (w[e >> 1] & 0xffffu));
    }
  };

  fetch(t0);
  for (int tc = t0; tc < t1; tc += MC_L) {
    const int n = min(MC_L, t1 - tc);
    __syncthreads();   // the previous chunk's reads are done
    stash();
    if (wave == 0) {
      // lane = token: F (running sum), G, M in float64
      const bool on = lane < n;
      const float gi = ml_cap(zi + bi, cap);
      const float gf = ml_logsig(ml_cap(zf + bf, cap));
      double F = on ? (double)gf : 0.0;
#pragma unroll
      for (int off = 1; off < 64; off <<= 1) {
        const double u = ml_shfl_up(F, off);
        if (lane >= off) F += u;
      }
      const double Gd = on ? (double)gi - F : -INFINITY;
      double M = fmax((double)m0, Gd);
#pragma unroll
      for (int off = 1; off < 64; off <<= 1) {
        const double u = ml_shfl_up(M, off);
        if (lane >= off) M = fmax(M, u);
      }
      const double ML = __shfl(M, 63, 64);
      const float gh = (float)Gd, mh = (float)M;
      g_hi[lane] = gh;
      g_lo[lane] = on ? (float)(Gd - (double)gh) : 0.f;
      m_hi[lane] = mh;
      m_lo[lane] = (float)(M - (double)mh);
      e_in[lane] = expf((float)((double)m0 - M));
      w_out[lane] = on ? expf((float)(Gd - ML)) : 0.f;
      m_tok[lane] = (float)(F + M);
      if (lane == 63) {
        s_end[0] = expf((float)((double)m0 - ML));
        s_end[1] = (float)(F + ML);
      }
    }
    __syncthreads();
    if (tc + MC_L < t1) fetch(tc + MC_L);

    // ---- q . S_0, then times exp(m_0 - M_t) ---------------------------------------
    f32x16v O;
#pragma unroll
    for (int r = 0; r < 16; ++r) O[r] = 0.f;
    const bf16_t* qrow = Qs + (tt0 + l31) * KS;
#pragma unroll
    for (int nb = 0; nb < NB; ++nb)
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        bf16x8v ph, pm, pl;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          short a, bb, c;
          ml_split3(st[nb][8 * s + e], a, bb, c);
          ph[e] = a;
          pm[e] = bb;
          pl[e] = c;
        }
        const bf16x8v a = mc_slots(qrow + 32 * nb, s, half);
        O = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, ph, O, 0, 0, 0);
        O = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, pm, O, 0, 0, 0);
        O = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, pl, O, 0, 0, 0);
      }
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int t = tt0 + 8 * (r >> 2) + 4 * half + (r & 3);
      O[r] *= e_in[t] * q_scale;
    }
    // ---- inside the chunk: scores (lane = token t, registers = tokens s), decay,
    //      then the product with the values --------------------------------------
    float rowsum = 0.f;
    const int tq = tt0 + l31;
    const float mh = m_hi[tq], ml = m_lo[tq];
#pragma unroll
    for (int sb = 0; sb < 2; ++sb) {
      if (32 * sb > tt0) break;        // those tokens come later
      f32x16v P;
#pragma unroll
      for (int r = 0; r < 16; ++r) P[r] = 0.f;
      const bf16_t* krow = Ks + (32 * sb + l31) * KS + 8 * half;
      const bf16_t* qr8 = qrow + 8 * half;
#pragma unroll
      for (int s = 0; s < D / 16; ++s) {
        const bf16x8v a = *reinterpret_cast<const bf16x8v*>(krow + 16 * s);
        const bf16x8v bq = *reinterpret_cast<const bf16x8v*>(qr8 + 16 * s);
        P = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, bq, P, 0, 0, 0);
      }
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int s = 32 * sb + 8 * (r >> 2) + 4 * half + (r & 3);
        const float w = s <= tq ? __expf((g_hi[s] - mh) + (g_lo[s] - ml)) : 0.f;
        P[r] *= w * q_scale;
        rowsum += P[r];
      }
      const bf16_t* vrow = Vt + jc * MC_TS + 32 * sb;
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        bf16x8v ph, pm, pl;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          short a, bb, c;
          ml_split3(P[8 * s + e], a, bb, c);
          ph[e] = a;
          pm[e] = bb;
          pl[e] = c;
        }
        const bf16x8v bv = mc_slots(vrow, s, half);
        O = __builtin_amdgcn_mfma_f32_32x32x16_bf16(ph, bv, O, 0, 0, 0);
        O = __builtin_amdgcn_mfma_f32_32x32x16_bf16(pm, bv, O, 0, 0, 0);
        O = __builtin_amdgcn_mfma_f32_32x32x16_bf16(pl, bv, O, 0, 0, 0);
      }
    }
    if (jok) {
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int t = tt0 + 8 * (r >> 2) + 4 * half + (r & 3);
        if (t < n) o[((int64_t)(tc + t) * H + h) * dv + j] = O[r];
      }
    }
    if (owner) {
      // n . q: the rows' sums (one wave per token half) plus n_0 . q
      rowsum += __shfl_xor(rowsum, 32, 64);
      {
        const int t = tid & 63, qd = tid >> 6;   // a quarter of the features each
        float s = 0.f;
        for (int i = qd * (D / 4); i < (qd + 1) * (D / 4); i += 8) {
          const bf16x8 raw = load_bf16x8(Qs + t * KS + i);
#pragma unroll
          for (int e = 0; e < 8; ++e) s = fmaf(bf16x8_get(raw, e), sn[i + e], s);
        }
        nqp[qd * MC_L + t] = s;
      }
      __syncthreads();   // uniform: `owner` is the same for the whole workgroup
      if (wave < 2 && half == 0 && tq < n) {
        const float s = nqp[tq] + nqp[MC_L + tq] + nqp[2 * MC_L + tq] + nqp[3 * MC_L + tq];
        const int64_t th = (int64_t)(tc + tq) * H + h;
        nq_out[th] = rowsum + s * q_scale * e_in[tq];
        mm[th] = m_tok[tq];
      }
      const float dec = s_end[0];
      for (int i = tid; i < D; i += 256) {
        float s = dec * sn[i];
        for (int t = 0; t < MC_L; t += 4) {
          const uint2 raw = *reinterpret_cast<const uint2*>(Kt + i * MC_TS + t);
          s = fmaf(w_out[t], bf16_bits_to_f32((uint16_t)(raw.x & 0xffff)), s);
          s = fmaf(w_out[t + 1], bf16_bits_to_f32((uint16_t)(raw.x >> 16)), s);
          s = fmaf(w_out[t + 2], bf16_bits_to_f32((uint16_t)(raw.y & 0xffff)), s);
          s = fmaf(w_out[t + 3], bf16_bits_to_f32((uint16_t)(raw.y >> 16)), s);
        }
        sn[i] = s;   // read again after the next chunk's first barrier
      }
    }
    // ---- the state at the end of the chunk -----------------------------------------
    {
      const float dec = s_end[0];
#pragma unroll
      for (int nb = 0; nb < NB; ++nb)
#pragma unroll
        for (int r = 0; r < 16; ++r) st[nb][r] *= dec;
      const bf16_t* vrow = Vt + jc * MC_TS;
#pragma unroll
      for (int s = 0; s < MC_L / 16; ++s) {
        const int2 w0 = *reinterpret_cast<const int2*>(vrow + 16 * s + 8 * half);
        const int2 w1 = *reinterpret_cast<const int2*>(vrow + 16 * s + 8 * half + 4);
        const int4 wp = make_int4(w0.x, w0.y, w1.x, w1.y);
        const bf16x8v raw = *reinterpret_cast<const bf16x8v*>(&wp);
        bf16x8v ph, pm, pl;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          short a, bb, c;
          ml_split3(bf16_bits_to_f32((uint16_t)raw[e]) * w_out[16 * s + 8 * half + e],
                    a, bb, c);
          ph[e] = a;
          pm[e] = bb;
          pl[e] = c;
        }
#pragma unroll
        for (int nb = 0; nb < NB; ++nb) {
          const bf16_t* kt = Kt + (32 * nb + l31) * MC_TS + 16 * s + 8 * half;
          const int2 v0 = *reinterpret_cast<const int2*>(kt);
          const int2 v1 = *reinterpret_cast<const int2*>(kt + 4);
          const int4 pk = make_int4(v0.x, v0.y, v1.x, v1.y);
          const bf16x8v a = *reinterpret_cast<const bf16x8v*>(&pk);
          st[nb] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, ph, st[nb], 0, 0, 0);
          st[nb] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, pm, st[nb], 0, 0, 0);
          st[nb] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, pl, st[nb], 0, 0, 0);
        }
      }
      m0 = s_end[1];
    }
  }
  // the two waves of a column half hold the same state: the first one stores it
  if ((wave & 1) == 0 && jok) {
#pragma unroll
    for (int nb = 0; nb < NB; ++nb)
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int i = 32 * nb + 8 * (r >> 2) + 4 * half + (r & 3);
        if (i < d) S[(int64_t)i * dv + j] = st[nb][r];
      }
  }
  if (owner) {
    __syncthreads();
    for (int i = tid; i < d; i += 256) S[(int64_t)d * dv + i] = sn[i];
  }
}

// ---- head norm and output gate ---------------------------------------------------

// lpr lanes per (token, head), 64 / lpr of those per wave. VEC: 4 consecutive
// values per lane (dv a multiple of 4, at most 256; rows aligned), lpr a power of
// two with 4 lpr >= dv; else lpr = 64 and a lane strides over the row.
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void mlstm_out_kernel(
    T* __restrict__ out, const float* __restrict__ o,
    const float* __restrict__ nq, const float* __restrict__ mm,
    const T* __restrict__ g, int64_t g_stride, const T* __restrict__ w,
    float eps, float* __restrict__ state, int64_t sw,
    const int64_t* __restrict__ slots, const int* __restrict__ cu, int B,
    int64_t rows, int H, int d, int dv, int lpr) {
  const int lane = threadIdx.x & 63;
  const int sub = lane % lpr;
  const int64_t row = ((int64_t)blockIdx.x * 4 + (threadIdx.x >> 6)) * (64 / lpr) + lane / lpr;
  const bool on = row < rows;     // all lanes stay for the reductions
  const int64_t r_ = on ? row : rows - 1;
  const int64_t t = r_ / H;
  const int h = (int)(r_ % H);
  const float m = mm[r_];
  const float den = 1.0f / (fmaxf(fabsf(nq[r_]), expf(-m)) + ML_EPS);
  const float* x = o + r_ * dv;
  const T* gr = g + t * g_stride + h * dv;
  T* dst = out + r_ * dv;
  float v[4] = {0.f, 0.f, 0.f, 0.f};
  float ss = 0.f;
  if (VEC) {
    const int i = sub * 4;
    if (i < dv) ml_load4<float>(x + i, v);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      v[j] *= den;
      ss = fmaf(v[j], v[j], ss);
    }
  } else {
    for (int i = sub; i < dv; i += 64) {
      const float z = x[i] * den;
      ss = fmaf(z, z, ss);
    }
  }
  for (int off = lpr >> 1; off > 0; off >>= 1) ss += __shfl_xor(ss, off, 64);
  if (!on) return;
  const float r = 1.0f / sqrtf(ss / (float)dv + eps);
  if (VEC) {
    const int i = sub * 4;
    if (i < dv) {
      float gv[4], wv[4];
      ml_load4<T>(gr + i, gv);
      ml_load4<T>(w + h * dv + i, wv);
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = v[j] * r * wv[j] * ml_sigmoid(gv[j]);
      ml_store4<T>(dst + i, v);
    }
  } else {
    for (int i = sub; i < dv; i += 64)
      stf(dst + i, x[i] * (den * r) * ldf(w + h * dv + i) * ml_sigmoid(ldf(gr + i)));
  }
  // a sequence's last token leaves its maximum in the state
  for (int b = sub; b < B; b += lpr) {
    const int e0 = cu ? cu[b] : b, e1 = cu ? cu[b + 1] : b + 1;
    if (e1 > e0 && e1 - 1 == t)
      state[(slots[b] * H + h) * sw + (int64_t)d * dv + d] = m;
  }
}

template <typename T>
static void launch_mlstm_t(void* out, float* o, float* nq, float* mm,
                           const void* q, int64_t q_stride, const void* k,
                           int64_t k_stride, const void* v, int64_t v_stride,
                           const void* g, int64_t g_stride, const float* gates,
                           const float* gate_bias, const void* norm_w, float cap,
                           float eps, float* state, int64_t sw,
                           const int64_t* slots, const int* cu,
                           const int* positions, int T_, int B, int H, int d,
                           int dv, float q_scale, int path, hipStream_t stream) {
  if (path == 0) {
    const int N = dv % 4 == 0 ? 4 : 1;
    const size_t shm = sizeof(float) * (2 * ((d + 3) & ~3) + 2 * ((dv + 3) & ~3) +
                                        256 * N + 8);
#define MS_CALL(NN)                                                            \
  hipLaunchKernelGGL((mlstm_step_kernel<T, NN>), dim3(H, B), dim3(256), shm,   \
                     stream, (T*)out, (const T*)q, q_stride, (const T*)k,      \
                     k_stride, (const T*)v, v_stride, (const T*)g, g_stride,   \
                     gates, gate_bias, (const T*)norm_w, cap, eps, state, sw,  \
                     slots, positions, H, d, dv, q_scale)
    if (N == 4) MS_CALL(4);
    else MS_CALL(1);
#undef MS_CALL
    return;
  }
  if (path == 2 && sizeof(T) == 2) {
    const dim3 grid((dv + MC_COLS - 1) / MC_COLS, H, B);
#define MC_CALL(DD)                                                           \
  hipLaunchKernelGGL((mlstm_chunk_kernel<DD>), grid, dim3(256), 0, stream, o, \
                     nq, mm, (const bf16_t*)q, q_stride, (const bf16_t*)k,    \
                     k_stride, (const bf16_t*)v, v_stride, gates, gate_bias,  \
                     cap, state, sw, slots, cu, positions, H, d, dv, q_scale)
    if (d <= 64) MC_CALL(64);
    else MC_CALL(128);
#undef MC_CALL
  } else {
    int G = 1;
    while (G * ML_ROWS < d) G <<= 1;  // host checked d <= 64 * ML_ROWS
    const int C = 64 / G;
    const dim3 grid((dv + 1 + 4 * C - 1) / (4 * C), H, B);
    const size_t per_token = sizeof(float) * (size_t)(2 * G * ML_ROWS + 4 * C);
    int TC = (int)((48 << 10) / per_token);
    TC = TC < 1 ? 1 : (TC > ML_TC_MAX ? ML_TC_MAX : TC);
    hipLaunchKernelGGL((mlstm_scan_kernel<T>), grid, dim3(256), per_token * TC,
                       stream, o, nq, mm, (const T*)q, q_stride, (const T*)k,
                       k_stride, (const T*)v, v_stride, gates, gate_bias, cap,
                       state, sw, slots, cu, positions, H, d, dv, G, TC, q_scale);
  }
  const int64_t rows = (int64_t)T_ * H;
  const int esz = sizeof(T);
  const bool vec = dv % 4 == 0 && dv <= 256 && g_stride % 4 == 0 &&
                   ((uintptr_t)g % (4 * esz)) == 0 &&
                   ((uintptr_t)norm_w % (4 * esz)) == 0;
  int lpr = 64;
  if (vec)
    while (lpr > 1 && lpr * 2 >= dv) lpr >>= 1;   // the smallest with 4 lpr >= dv
  const int64_t per_block = 4 * (64 / lpr);
#define MO_CALL(V)                                                             \
  hipLaunchKernelGGL((mlstm_out_kernel<T, V>),                                 \
                     dim3((rows + per_block - 1) / per_block), dim3(256), 0,   \
                     stream, (T*)out, o, nq, mm, (const T*)g, g_stride,        \
                     (const T*)norm_w, eps, state, sw, slots, cu, B, rows, H,  \
                     d, dv, lpr)
  if (vec) MO_CALL(true);
  else MO_CALL(false);
#undef MO_CALL
}

// path 0: one token per sequence (cu null); 1: token-serial; 2: chunks (bf16,
// d <= 128, widths in multiples of 8, 16-byte aligned rows, cu given)
extern "C" void launch_mlstm(void* out, float* o, float* nq, float* mm,
                             const void* q, int64_t q_stride, const void* k,
                             int64_t k_stride, const void* v, int64_t v_stride,
                             const void* g, int64_t g_stride, const float* gates,
                             const float* gate_bias, const void* norm_w,
                             float cap, float eps, float* state, int64_t sw,
                             const int64_t* slots, const int* cu,
                             const int* positions, int T_, int B, int H, int d,
                             int dv, float q_scale, int path, int kind,
                             hipStream_t stream) {
  if (T_ == 0 || B == 0) return;
#define ML_ARGS                                                               \
  out, o, nq, mm, q, q_stride, k, k_stride, v, v_stride, g, g_stride, gates,  \
      gate_bias, norm_w, cap, eps, state, sw, slots, cu, positions, T_, B, H, \
      d, dv, q_scale, path, stream
  if (kind == 0) launch_mlstm_t<bf16_t>(ML_ARGS);
  else launch_mlstm_t<float>(ML_ARGS);
#undef ML_ARGS
}
