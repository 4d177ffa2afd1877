// Projections to a few columns whose consumers want fp32 (gates of a
// recurrence, router logits), and the router built on them.
//
//   linear_f32    : out [T, N] fp32 = x [T, K] bf16 . w [N, K]^T bf16.
//   route_softmax : rows 0 .. E of w are experts: z = x w^T + bias, the `top`
//                   largest (lower index first among equals), weights = softmax
//                   over those; rows E .. N are handed out as fp32 outputs. With
//                   groups > 1 the experts form equal runs of neighbours and only
//                   those of the `keep` runs with the largest single logit count.
//
// One workgroup takes 16 tokens and up to 16 NT columns. Its NW waves share out
// the contraction (wave w takes every NW-th block of 32) on the bf16 matrix
// cores with fp32 accumulators and add up through LDS, so a decode step of a
// few tokens still has NW x NT independent load streams in flight. For the
// router the 16 rows of logits never leave LDS: a wave picks the experts of
// 16 / NW tokens, one expert per round (a lane owns experts lane, lane + 64,
// ...).
#include "seq_common.h"

#define SL_TOK 16

// 8 consecutive elements of a row at column k, zeros beyond K
template <bool VEC>
DEVINL bf16x8v sl_load8(const bf16_t* row, int k, int K) {
  bf16x8v r = {};
  if (VEC) {
    if (k < K) r = *reinterpret_cast<const bf16x8v*>(row + k);
  } else {
#pragma unroll
    for (int e = 0; e < 8; ++e)
      if (k + e < K) r[e] = (short)row[k + e];
  }
  return r;
}

// LDS: [NW][16][NT * 16 + 1] partial sums; afterwards plane 0 holds the sums
template <int NT, int NW, bool VEC, bool ROUTE>
__global__ __launch_bounds__(NW * 64) void small_linear_kernel(
    float* __restrict__ out, const bf16_t* __restrict__ x, int64_t x_stride,
    const bf16_t* __restrict__ w, int T_, int N, int K,
    int64_t* __restrict__ ids, float* __restrict__ wts,
    const float* __restrict__ bias, int E, int top, int groups, int keep) {
  constexpr int NP = NT * 16 + 1;
  extern __shared__ float red[];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int l15 = lane & 15, l4 = lane >> 4;
  const int t0 = blockIdx.x * SL_TOK, n0 = blockIdx.y * NT * 16;

  const bool tok_ok = t0 + l15 < T_;
  const bf16_t* xr = x + (int64_t)min(t0 + l15, T_ - 1) * x_stride;
  f32x4v acc[NT] = {};
#pragma unroll 4
  for (int k0 = wave * 32; k0 < K; k0 += NW * 32) {
    const int k = k0 + l4 * 8;
    bf16x8v a = sl_load8<VEC>(xr, k, K);
    if (!tok_ok) a = bf16x8v{};
    bf16x8v b[NT];
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const int n = n0 + i * 16 + l15;
      b[i] = bf16x8v{};
      if (n < N) b[i] = sl_load8<VEC>(w + (int64_t)n * K, k, K);
    }
#pragma unroll
    for (int i = 0; i < NT; ++i)
      acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b[i], acc[i], 0, 0, 0);
  }
  // element (lane, reg): token (lane >> 4) * 4 + reg, column lane & 15
#pragma unroll
  for (int i = 0; i < NT; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r)
      red[(wave * SL_TOK + l4 * 4 + r) * NP + i * 16 + l15] = acc[i][r];
  __syncthreads();
  for (int idx = threadIdx.x; idx < SL_TOK * NT * 16; idx += NW * 64) {
    const int m = idx / (NT * 16), n = idx % (NT * 16);
    float v = red[m * NP + n];
#pragma unroll
    for (int wv = 1; wv < NW; ++wv) v += red[(wv * SL_TOK + m) * NP + n];
    const int t = t0 + m, col = n0 + n;
    if (ROUTE) {
      if (col < E && bias != nullptr) v += bias[col];
      red[m * NP + n] = v;   // read and written by this thread only
      if (t < T_ && col >= E && col < N) out[(int64_t)t * (N - E) + col - E] = v;
    } else if (t < T_ && col < N) {
      out[(int64_t)t * N + col] = v;
    }
  }
  if (!ROUTE) return;
  __syncthreads();
  constexpr int EC = (NT * 16 + 63) / 64;
  for (int mm = 0; mm < SL_TOK / NW; ++mm) {
    const int m = wave * (SL_TOK / NW) + mm, t = t0 + m;
    if (t >= T_) break;
    float v[EC];
#pragma unroll
    for (int c = 0; c < EC; ++c) {
      const int e = lane + 64 * c;
      v[c] = e < E ? red[m * NP + e] : -INFINITY;
    }
    if (groups > 1) {
      // lane = group (at most 64): its largest logit, then its rank among the
      // groups (lower index first among equals)
      const int gs = E / groups;
      float best = -INFINITY;
      if (lane < groups)
        for (int i = 0; i < gs; ++i) best = fmaxf(best, red[m * NP + lane * gs + i]);
      int rank = 0;
      for (int o = 0; o < groups; ++o) {
        const float ob = __shfl(best, o, 64);
        rank += ob > best || (ob == best && o < lane);
      }
      const unsigned long long in = __ballot(lane < groups && rank < keep);
#pragma unroll
      for (int c = 0; c < EC; ++c) {
        const int e = lane + 64 * c;
        if (e < E && !((in >> (e / gs)) & 1)) v[c] = -INFINITY;
      }
    }
    float mine = -INFINITY;  // lane r keeps the r-th choice's logit
    int mine_id = 0;
    for (int r = 0; r < top; ++r) {
      float bv = v[0];
      int be = lane;
#pragma unroll
      for (int c = 1; c < EC; ++c)
        if (v[c] > bv) {
          bv = v[c];
          be = lane + 64 * c;
        }
#pragma unroll
      for (int off = 32; off > 0; off >>= 1) {
        const float ov = __shfl_xor(bv, off, 64);
        const int oe = __shfl_xor(be, off, 64);
        if (ov > bv || (ov == bv && oe < be)) {
          bv = ov;
          be = oe;
        }
      }
#pragma unroll
      for (int c = 0; c < EC; ++c)
        if (be == lane + 64 * c) v[c] = -INFINITY;
      if (lane == r) {
        mine = bv;
        mine_id = be;
      }
    }
    const float mx = __shfl(mine, 0, 64);   // the first choice is the largest
    const float p = lane < top ? expf(mine - mx) : 0.f;
    const float sum = wave_reduce_sum(p);
    if (lane < top) {
      ids[(int64_t)t * top + lane] = min(mine_id, E - 1);  // NaN logits: still an expert
      wts[(int64_t)t * top + lane] = p / sum;
    }
  }
}

template <int NT>
static void launch_sl(float* out, const bf16_t* x, int64_t x_stride,
                      const bf16_t* w, int T_, int N, int K, int64_t* ids,
                      float* wts, const float* bias, int E, int top, int groups,
                      int keep, bool vec, hipStream_t stream) {
  const dim3 grid((T_ + SL_TOK - 1) / SL_TOK, (N + NT * 16 - 1) / (NT * 16));
  constexpr int NW = NT <= 4 ? 8 : 4;   // partial sums within 64 KB of LDS
  const size_t shm = sizeof(float) * NW * SL_TOK * (NT * 16 + 1);
#define SL_CALL(V, R)                                                         \
  hipLaunchKernelGGL((small_linear_kernel<NT, NW, V, R>), grid, dim3(NW * 64), \
                     shm, stream, out, x, x_stride, w, T_, N, K, ids, wts, bias, E, \
                     top, groups, keep)
  if (ids != nullptr) {
    if (vec) SL_CALL(true, true);
    else SL_CALL(false, true);
  } else {
    if (vec) SL_CALL(true, false);
    else SL_CALL(false, false);
  }
#undef SL_CALL
}

// ids null: plain projection. A router's N (at most 240) is one workgroup's.
extern "C" void launch_small_linear(float* out, const void* x, int64_t x_stride,
                                    const void* w, int T_, int N, int K,
                                    int64_t* ids, float* wts, const float* bias,
                                    int E, int top, int groups, int keep,
                                    hipStream_t stream) {
  if (T_ == 0 || N == 0) return;
  const bf16_t* xp = (const bf16_t*)x;
  const bf16_t* wp = (const bf16_t*)w;
  const bool vec = K % 8 == 0 && x_stride % 8 == 0 && ((uintptr_t)x % 16) == 0 &&
                   ((uintptr_t)w % 16) == 0;
#define SL_ARGS out, xp, x_stride, wp, T_, N, K, ids, wts, bias, E, top, groups, keep, vec, stream
  if (N <= 16) launch_sl<1>(SL_ARGS);
  else if (N <= 32) launch_sl<2>(SL_ARGS);
  else if (N <= 64 || ids == nullptr) launch_sl<4>(SL_ARGS);
  else if (N <= 128) launch_sl<8>(SL_ARGS);
  else launch_sl<15>(SL_ARGS);  // 240 columns: 61 KB of LDS
#undef SL_ARGS
}
