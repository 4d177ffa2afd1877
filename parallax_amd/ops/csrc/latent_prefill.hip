// Sliding-window attention over a latent cache for prompt portions, with keys
// and values expanded once per portion instead of absorbing every query into
// the latent space.
//
// A cache row is [latent c (rank) | rotated key part (dr)], shared by all heads.
// With r rows of context a portion needs 2 r rank H (dn + dv) operations to expand
// them to per-head keys W_uk c and values W_uv c (one library GEMM) and then
// dn + dr + dv per (query, key, head) instead of the 2 rank + dr of the absorbed
// form, several times less for the usual sizes.
//
//   latent_gather    : the context rows of every sequence of the batch (the keys
//                      its portion can see) out of the paged cache into two dense
//                      matrices, latents and rotated parts.
//   latent_expanded_attention : a workgroup takes 128 consecutive tokens of one
//                      sequence and one head, 32 queries per wave; 32 keys per
//                      step are staged in LDS for the four waves. Products as in
//                      the row attention on the bf16 matrix cores:
//                          S^T (32 keys x 32 queries) = K . Q^T,
//                          O^T (dv x 32 queries)     += V^T . P^T,
//                      the weights already laid out as the second product's
//                      operand. Unrotated queries and keys are bf16 numbers (one
//                      instruction per 16 features, exact products, fp32 sums);
//                      rotated queries are fp32 and enter as three bf16 parts
//                      that add up to them, and so do the softmax weights. A sink
//                      starts the running maximum with the denominator 1.
#include "seq_common.h"

typedef float f32x16v __attribute__((ext_vector_type(16)));

#define LP_Q 128     // queries per workgroup
#define LP_K 32      // keys per step
#define LP_VS 36     // bf16 elements per transposed value row: 32 keys + 4

// plan: [0, B] row offsets of the sequences' contexts, [B + 1, 2 B] the position
// of each context's first row
__global__ __launch_bounds__(128) void latent_gather_kernel(
    bf16_t* __restrict__ lat, bf16_t* __restrict__ rot,
    const bf16_t* __restrict__ cache, const int* __restrict__ block_tables,
    int bt_stride, const int* __restrict__ plan, int B, int block_size, int rank,
    int dr) {
  const int row = blockIdx.x;
  int b = 0;
  while (b + 1 < B && row >= plan[b + 1]) ++b;
  const int j = plan[B + 1 + b] + row - plan[b];
  const int E = rank + dr;
  const bf16_t* src =
      cache + ((int64_t)block_tables[(int64_t)b * bt_stride + j / block_size] * block_size +
               j % block_size) * E;
  for (int i = threadIdx.x * 8; i < E; i += 128 * 8) {
    const int4 v = *reinterpret_cast<const int4*>(src + i);
    if (i < rank) *reinterpret_cast<int4*>(lat + (int64_t)row * rank + i) = v;
    else *reinterpret_cast<int4*>(rot + (int64_t)row * dr + i - rank) = v;
  }
}

extern "C" void launch_latent_gather(void* lat, void* rot, const void* cache,
                                     const int* block_tables, int bt_stride,
                                     const int* plan, int B, int rows,
                                     int block_size, int rank, int dr,
                                     hipStream_t stream) {
  if (rows == 0) return;
  hipLaunchKernelGGL(latent_gather_kernel, dim3(rows), dim3(128), 0, stream,
                     (bf16_t*)lat, (bf16_t*)rot, (const bf16_t*)cache,
                     block_tables, bt_stride, plan, B, block_size, rank, dr);
}

// x = hi + mid + lo exactly, each a bf16 number
DEVINL void lp_split3(float x, short& hi, short& mid, short& lo) {
  const uint32_t b0 = __float_as_uint(x) & 0xffff0000u;
  const float r1 = x - __uint_as_float(b0);
  const uint32_t b1 = __float_as_uint(r1) & 0xffff0000u;
  const float r2 = r1 - __uint_as_float(b1);
  hi = (short)(b0 >> 16);
  mid = (short)(b1 >> 16);
  lo = (short)(__float_as_uint(r2) >> 16);
}

// grid (H, tiles): heads fastest, so that with 8 | H a head's tiles run on one
// XCD and share its L2. DN, DR: padded unrotated and rotated widths, DVB: 32-wide
// blocks of the padded value width.
template <int DN, int DR, int DVB>
__global__ __launch_bounds__(256, 2) void latent_expanded_attention_kernel(
    bf16_t* __restrict__ out, const bf16_t* __restrict__ q, int64_t q_stride,
    const float* __restrict__ q_rot, const bf16_t* __restrict__ kv,
    int64_t kv_stride, const bf16_t* __restrict__ k_rot,
    const int* __restrict__ plan, const int* __restrict__ cu, int B,
    const int* __restrict__ positions, int H, int dn, int dr, int dv, int window,
    float scale, const float* __restrict__ sink) {
  constexpr int KS = DN + DR + 8;
  constexpr int DV = DVB * 32;
  __shared__ __attribute__((aligned(16))) bf16_t Ks[LP_K * KS];
  __shared__ __attribute__((aligned(16))) bf16_t Vt[DV * LP_VS];

  const int h = blockIdx.x;
  int tile = gridDim.y - 1 - blockIdx.y, b = 0;   // the longest runs first
  for (; b < B; ++b) {
    const int nt = (cu[b + 1] - cu[b] + LP_Q - 1) / LP_Q;
    if (tile < nt) break;
    tile -= nt;
  }
  if (b == B) return;
  const int t0 = cu[b] + tile * LP_Q;
  const int nq = min(LP_Q, cu[b + 1] - t0);
  const int p0 = positions[t0], p_last = p0 + nq - 1;
  const int klo = max(0, p0 - window + 1);
  const int nk = p_last - klo + 1;
  const int row0 = plan[b] + klo - plan[B + 1 + b];   // the first key's row

  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int half = lane >> 5, col = lane & 31;
  const int nqw = min(32, nq - wave * 32);            // this wave's queries (<= 0: none)
  const int pw0 = p0 + wave * 32, pw_last = pw0 + nqw - 1;
  const bool qvalid = col < nqw;
  const int pq = pw0 + col;
  const int64_t tq = t0 + min(wave * 32 + col, nq - 1);

  bf16x8v qn[DN / 16], rh[DR / 16], rm[DR / 16], rl[DR / 16];
  {
    const bf16_t* src = q + tq * q_stride + (int64_t)h * (dn + dr);
#pragma unroll
    for (int s = 0; s < DN / 16; ++s) {
      const int f = 16 * s + 8 * half;
      qn[s] = bf16x8v{};
      if (qvalid && f < dn) qn[s] = *reinterpret_cast<const bf16x8v*>(src + f);
    }
    const float* rsrc = q_rot + (tq * H + h) * (int64_t)dr;
#pragma unroll
    for (int s = 0; s < DR / 16; ++s)
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int f = 16 * s + 8 * half + e;
        short a, m, l;
        lp_split3((qvalid && f < dr) ? rsrc[f] : 0.f, a, m, l);
        rh[s][e] = a;
        rm[s][e] = m;
        rl[s][e] = l;
      }
  }

  f32x16v acc[DVB];
#pragma unroll
  for (int k = 0; k < DVB; ++k)
#pragma unroll
    for (int i = 0; i < 16; ++i) acc[k][i] = 0.f;
  float mx = sink ? sink[h] : -INFINITY, l = sink ? 1.f : 0.f;

  // staging role: 8 threads per key row, 8 elements each at a time
  const int srow = threadIdx.x >> 3, ssub = threadIdx.x & 7;
  constexpr int KC = DN / 64, VC = (DV + 63) / 64;
  int4 kraw[KC], vraw[VC], rraw;
  auto fetch = [&](int u0) {
    const int u = u0 + srow;
    const bool on = u < nk;
    const int64_t row = row0 + (on ? u : 0);
    const bf16_t* kr = kv + row * kv_stride + (int64_t)h * dn;
    const bf16_t* vr = kv + row * kv_stride + (int64_t)H * dn + (int64_t)h * dv;
#pragma unroll
    for (int c = 0; c < KC; ++c) {
      const int f = ssub * 8 + 64 * c;
      kraw[c] = (on && f < dn) ? *reinterpret_cast<const int4*>(kr + f)
                               : make_int4(0, 0, 0, 0);
    }
    rraw = (on && ssub * 8 < dr)
               ? *reinterpret_cast<const int4*>(k_rot + row * dr + ssub * 8)
               : make_int4(0, 0, 0, 0);
#pragma unroll
    for (int c = 0; c < VC; ++c) {
      const int f = ssub * 8 + 64 * c;
      vraw[c] = (on && f < dv) ? *reinterpret_cast<const int4*>(vr + f)
                               : make_int4(0, 0, 0, 0);
    }
  };
  auto stash = [&]() {
#pragma unroll
    for (int c = 0; c < KC; ++c)
      *reinterpret_cast<int4*>(Ks + srow * KS + ssub * 8 + 64 * c) = kraw[c];
    if (ssub * 8 < DR)
      *reinterpret_cast<int4*>(Ks + srow * KS + DN + ssub * 8) = rraw;
#pragma unroll
    for (int c = 0; c < VC; ++c) {
      const int f = ssub * 8 + 64 * c;
      if (f < DV) {
        const uint32_t w[4] = {(uint32_t)vraw[c].x, (uint32_t)vraw[c].y,
                               (uint32_t)vraw[c].z, (uint32_t)vraw[c].w};
#pragma unroll
        for (int e = 0; e < 8; ++e)
          Vt[(f + e) * LP_VS + srow] =
              (bf16_t)((e & 1) ? (w[e >> 1] >> 16) : (w[e >> 1] & 0xffffu));
      }
    }
  };

  fetch(0);
  for (int u0 = 0; u0 < nk; u0 += LP_K) {
    __syncthreads();  // the previous step's reads are done
    stash();
    __syncthreads();
    if (u0 + LP_K < nk) fetch(u0 + LP_K);
    const int jt0 = klo + u0;
    // keys that none of this wave's queries sees
    if (nqw <= 0 || jt0 > pw_last || jt0 + LP_K - 1 <= pw0 - window) continue;

    f32x16v S;
#pragma unroll
    for (int i = 0; i < 16; ++i) S[i] = 0.f;
    const bf16_t* krow = Ks + col * KS + 8 * half;
#pragma unroll
    for (int s = 0; s < DN / 16; ++s) {
      const bf16x8v a = *reinterpret_cast<const bf16x8v*>(krow + 16 * s);
      S = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, qn[s], S, 0, 0, 0);
    }
#pragma unroll
    for (int s = 0; s < DR / 16; ++s) {
      const bf16x8v a = *reinterpret_cast<const bf16x8v*>(krow + DN + 16 * s);
      S = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, rh[s], S, 0, 0, 0);
      S = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, rm[s], S, 0, 0, 0);
      S = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, rl[s], S, 0, 0, 0);
    }
    // mask, running maximum, weights (lane = query, registers = 16 of the keys)
    const bool interior = nqw == 32 && u0 + LP_K <= nk && jt0 + LP_K - 1 <= pw0 &&
                          pw_last - jt0 < window;
    float tmax = -INFINITY;
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int u = u0 + 8 * i + 4 * half + j;
        const int jt = klo + u;
        const bool vis = interior ||
                         (qvalid && u < nk && jt <= pq && pq - jt < window);
        const float sc = vis ? S[4 * i + j] * scale : -INFINITY;
        S[4 * i + j] = sc;
        tmax = fmaxf(tmax, sc);
      }
    tmax = fmaxf(tmax, __shfl_xor(tmax, 32, 64));
    const float m_new = fmaxf(mx, tmax);
    float corr = 1.f, psum = 0.f;
    if (m_new == -INFINITY) {
#pragma unroll
      for (int i = 0; i < 16; ++i) S[i] = 0.f;
    } else {
      corr = __expf(mx - m_new);
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const float p = __expf(S[i] - m_new);
        S[i] = p;
        psum += p;
      }
    }
    psum += __shfl_xor(psum, 32, 64);
    l = l * corr + psum;
    mx = m_new;
#pragma unroll
    for (int k = 0; k < DVB; ++k)
#pragma unroll
      for (int i = 0; i < 16; ++i) acc[k][i] *= corr;
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      bf16x8v ph, pm, pl;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        short a, m, lw;
        lp_split3(S[8 * s + e], a, m, lw);
        ph[e] = a;
        pm[e] = m;
        pl[e] = lw;
      }
#pragma unroll
      for (int k = 0; k < DVB; ++k) {
        const bf16_t* vrow = Vt + (32 * k + col) * LP_VS + 16 * s + 4 * half;
        const int2 v0 = *reinterpret_cast<const int2*>(vrow);
        const int2 v1 = *reinterpret_cast<const int2*>(vrow + 8);
        const int4 packed = make_int4(v0.x, v0.y, v1.x, v1.y);
        const bf16x8v a = *reinterpret_cast<const bf16x8v*>(&packed);
        acc[k] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, ph, acc[k], 0, 0, 0);
        acc[k] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, pm, acc[k], 0, 0, 0);
        acc[k] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, pl, acc[k], 0, 0, 0);
      }
    }
  }
  if (!qvalid) return;
  const float inv = l > 0.f ? 1.0f / l : 0.f;
  bf16_t* dst = out + (tq * H + h) * (int64_t)dv;
#pragma unroll
  for (int k = 0; k < DVB; ++k)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int f = 32 * k + 8 * i + 4 * half;
      if (f < dv) {
        uint2 w;
        w.x = (uint32_t)f32_to_bf16_bits(acc[k][4 * i] * inv) |
              ((uint32_t)f32_to_bf16_bits(acc[k][4 * i + 1] * inv) << 16);
        w.y = (uint32_t)f32_to_bf16_bits(acc[k][4 * i + 2] * inv) |
              ((uint32_t)f32_to_bf16_bits(acc[k][4 * i + 3] * inv) << 16);
        *reinterpret_cast<uint2*>(dst + f) = w;
      }
    }
}

// what the kernel tiles: widths in multiples of 8 within the template sizes
extern "C" int latent_expanded_supported(int dn, int dr, int dv) {
  return dn % 8 == 0 && dr % 8 == 0 && dv % 8 == 0 && dn >= 8 && dr >= 8 &&
         dn <= 128 && dr <= 64 && dv <= 128;
}

// tiles: an upper bound on the number of 128-token tiles (T / 128 + B)
extern "C" void launch_latent_expanded_attention(
    void* out, const void* q, int64_t q_stride, const float* q_rot,
    const void* kv, int64_t kv_stride, const void* k_rot, const int* plan,
    const int* cu, int B, const int* positions, int tiles, int H, int dn, int dr,
    int dv, int window, float scale, const float* sink, hipStream_t stream) {
  if (tiles == 0) return;
#define LP_CALL(N, R, V)                                                       \
  hipLaunchKernelGGL((latent_expanded_attention_kernel<N, R, V>),              \
                     dim3(H, tiles), dim3(256), 0, stream, (bf16_t*)out,       \
                     (const bf16_t*)q, q_stride, q_rot, (const bf16_t*)kv,     \
                     kv_stride, (const bf16_t*)k_rot, plan, cu, B, positions,  \
                     H, dn, dr, dv, window, scale, sink)
#define LP_V(N, R)                  \
  {                                 \
    if (dv <= 64) LP_CALL(N, R, 2); \
    else LP_CALL(N, R, 4);          \
  }
#define LP_R(N)              \
  {                          \
    if (dr <= 32) LP_V(N, 32) \
    else LP_V(N, 64)         \
  }
  if (dn <= 64) LP_R(64)
  else LP_R(128)
#undef LP_R
#undef LP_V
#undef LP_CALL
}
