// Gated linear attention: per head a [dk, dv] fp32 state with a decay per key
// channel,
//
//     S_t = diag(alpha_t) S_(t-1) + k_t v_t^T ,   o_t = S_t^T q_t ,
//     alpha = sigmoid(z + z_bias)^(1/tau)   (computed as exp(logsigmoid / tau)).
//
// The recurrence runs token by token inside the kernel, so a prompt cut into
// portions, or decoded one token at a time, goes through the very same
// operations in the same order. Parallelism comes from the state's columns:
// o_t[j] only needs column j of S, so a thread owns (part of) one column in
// registers for the whole portion. G lanes share a column when dk > 16 (each
// holds 16 rows; their partial dot products meet through wave shuffles).
// q, k, the decay and v of 16 tokens at a time are staged in LDS by the whole
// block, which also turns z into alpha once per (token, channel) and not once
// per column.
//
// The state lives in fp32 slots [slot, H, dk, dv]; a sequence whose first
// token of this launch sits at position 0 starts from zeros instead of the
// slot's old content. A decode step is the same kernel with one token per
// sequence.
#include "seq_common.h"

#define GLA_TC_MAX 16  // tokens staged per pass (fewer when dk is large)
#define GLA_ROWS 16  // state rows per lane

template <typename T>
__global__ __launch_bounds__(256) void gla_recurrence_kernel(
    float* __restrict__ o, const T* __restrict__ q, const T* __restrict__ k,
    const T* __restrict__ v, const T* __restrict__ z, int64_t q_stride,
    int64_t k_stride, int64_t v_stride, int64_t z_stride,
    const T* __restrict__ z_bias, float* __restrict__ state,
    const int64_t* __restrict__ slots, const int* __restrict__ cu,
    const int* __restrict__ positions, int H, int dk, int dv, int G, int TC,
    float inv_tau, float q_scale) {
  extern __shared__ float lds[];
  const int b = blockIdx.z, h = blockIdx.y;
  const int C = 64 / G;  // columns per wave
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int g = lane / C;
  const int jb = wave * C + lane % C;  // column within the block
  const int j = blockIdx.x * 4 * C + jb;
  const bool jvalid = j < dv;
  const int t0 = cu ? cu[b] : b;
  const int t1 = cu ? cu[b + 1] : b + 1;
  if (t0 >= t1) return;
  const int dkp = G * GLA_ROWS;  // padded rows (pad: q = k = alpha = 0)
  float* sq = lds;
  float* sk = sq + TC * dkp;
  float* sa = sk + TC * dkp;
  float* sv = sa + TC * dkp;  // [TC][4 * C]

  const int64_t slot = slots[b];
  float* S = state + ((slot * H + h) * (int64_t)dk) * dv;
  const bool fresh = positions[t0] == 0;
  float s[GLA_ROWS];
#pragma unroll
  for (int r = 0; r < GLA_ROWS; ++r) {
    const int i = g * GLA_ROWS + r;
    s[r] = (!fresh && jvalid && i < dk) ? S[(int64_t)i * dv + j] : 0.f;
  }

  for (int tc = t0; tc < t1; tc += TC) {
    const int n = min(TC, t1 - tc);
    __syncthreads();
    for (int idx = threadIdx.x; idx < n * dkp; idx += 256) {
      const int tt = idx / dkp, i = idx % dkp;
      float qf = 0.f, kf = 0.f, af = 0.f;
      if (i < dk) {
        const int64_t tok = tc + tt;
        const int c = h * dk + i;
        qf = ldf(q + tok * q_stride + c) * q_scale;
        kf = ldf(k + tok * k_stride + c);
        const float zf = ldf(z + tok * z_stride + c) + ldf(z_bias + c);
        const float logsig = fminf(zf, 0.f) - log1pf(expf(-fabsf(zf)));
        af = expf(logsig * inv_tau);
      }
      sq[idx] = qf;
      sk[idx] = kf;
      sa[idx] = af;
    }
    for (int idx = threadIdx.x; idx < n * 4 * C; idx += 256) {
      const int tt = idx / (4 * C), jj = idx % (4 * C);
      const int col = blockIdx.x * 4 * C + jj;
      sv[idx] = col < dv
                    ? ldf(v + (int64_t)(tc + tt) * v_stride + h * dv + col)
                    : 0.f;
    }
    __syncthreads();
    for (int tt = 0; tt < n; ++tt) {
      const float vj = sv[tt * 4 * C + jb];
      const float* aq = sq + tt * dkp + g * GLA_ROWS;
      const float* ak = sk + tt * dkp + g * GLA_ROWS;
      const float* aa = sa + tt * dkp + g * GLA_ROWS;
      float acc = 0.f;
#pragma unroll
      for (int r = 0; r < GLA_ROWS; ++r) {
        s[r] = aa[r] * s[r] + ak[r] * vj;
        acc = fmaf(s[r], aq[r], acc);
      }
      for (int off = C; off < 64; off <<= 1) acc += __shfl_xor(acc, off, 64);
      if (g == 0 && jvalid) o[((int64_t)(tc + tt) * H + h) * dv + j] = acc;
    }
  }
  if (jvalid) {
#pragma unroll
    for (int r = 0; r < GLA_ROWS; ++r) {
      const int i = g * GLA_ROWS + r;
      if (i < dk) S[(int64_t)i * dv + j] = s[r];
    }
  }
}

template <typename T>
DEVINL void gn4_load(const T* p, float* v);
template <>
DEVINL void gn4_load<float>(const float* p, float* v) {
  const float4 a = *reinterpret_cast<const float4*>(p);
  v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w;
}
template <>
DEVINL void gn4_load<bf16_t>(const bf16_t* p, float* v) {
  const uint2 raw = *reinterpret_cast<const uint2*>(p);
  v[0] = bf16_bits_to_f32((uint16_t)(raw.x & 0xffff));
  v[1] = bf16_bits_to_f32((uint16_t)(raw.x >> 16));
  v[2] = bf16_bits_to_f32((uint16_t)(raw.y & 0xffff));
  v[3] = bf16_bits_to_f32((uint16_t)(raw.y >> 16));
}
template <typename T>
DEVINL void gn4_store(T* p, const float* v);
template <>
DEVINL void gn4_store<float>(float* p, const float* v) {
  *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
}
template <>
DEVINL void gn4_store<bf16_t>(bf16_t* p, const float* v) {
  uint2 raw;
  raw.x = (uint32_t)f32_to_bf16_bits(v[0]) | ((uint32_t)f32_to_bf16_bits(v[1]) << 16);
  raw.y = (uint32_t)f32_to_bf16_bits(v[2]) | ((uint32_t)f32_to_bf16_bits(v[3]) << 16);
  *reinterpret_cast<uint2*>(p) = raw;
}

// silu(z) or sigmoid(z)
DEVINL float gn_act(float z, bool sigmoid) {
  const float s = 1.0f / (1.0f + expf(-z));
  return sigmoid ? s : z * s;
}

// out[t, h*dv + j] = o[t,h,j] / rms(o[t,h,:]) * w[j] * act(gate[t, h*dv + j]), w
// null = no weight. lpr lanes per (token, head): VEC: 4 values per lane (dv a
// multiple of 4, at most 256, rows aligned), lpr a power of two with 4 lpr >= dv;
// else a wave per row.
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void gated_rmsnorm_kernel(
    T* __restrict__ out, const float* __restrict__ o, const T* __restrict__ gate,
    int64_t gate_stride, const T* __restrict__ w, float eps, int64_t rows, int H,
    int dv, int lpr, int sigmoid) {
  const int lane = threadIdx.x & 63, sub = lane % lpr;
  const int64_t row =
      ((int64_t)blockIdx.x * 4 + (threadIdx.x >> 6)) * (64 / lpr) + lane / lpr;
  const bool on = row < rows;   // all lanes stay for the reductions
  const int64_t r_ = on ? row : rows - 1;
  const int64_t t = r_ / H;
  const int h = (int)(r_ % H);
  const float* x = o + r_ * dv;
  const T* gr = gate + t * gate_stride + h * dv;
  T* dst = out + r_ * dv;
  float v[4] = {0.f, 0.f, 0.f, 0.f};
  float sq = 0.f;
  if (VEC) {
    if (sub * 4 < dv) gn4_load<float>(x + sub * 4, v);
#pragma unroll
    for (int j = 0; j < 4; ++j) sq = fmaf(v[j], v[j], sq);
  } else {
    for (int i = sub; i < dv; i += 64) sq = fmaf(x[i], x[i], sq);
  }
  for (int off = lpr >> 1; off > 0; off >>= 1) sq += __shfl_xor(sq, off, 64);
  if (!on) return;
  const float r = 1.0f / sqrtf(sq / (float)dv + eps);
  if (VEC) {
    const int i = sub * 4;
    if (i < dv) {
      float gv[4], wv[4] = {1.f, 1.f, 1.f, 1.f};
      gn4_load<T>(gr + i, gv);
      if (w) gn4_load<T>(w + i, wv);
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = v[j] * r * wv[j] * gn_act(gv[j], sigmoid);
      gn4_store<T>(dst + i, v);
    }
  } else {
    for (int i = sub; i < dv; i += 64)
      stf(dst + i, x[i] * r * (w ? ldf(w + i) : 1.f) * gn_act(ldf(gr + i), sigmoid));
  }
}

// the same with ONE norm over a token's whole row of n = H dv values and a weight
// that wide; a workgroup per token, the row in registers up to n = 4096 (VEC)
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void gated_rmsnorm_row_kernel(
    T* __restrict__ out, const float* __restrict__ o, const T* __restrict__ gate,
    int64_t gate_stride, const T* __restrict__ w, float eps, int n, int sigmoid) {
  __shared__ float scratch[8];
  const int64_t t = blockIdx.x;
  const float* x = o + t * (int64_t)n;
  const T* gr = gate + t * gate_stride;
  T* dst = out + t * (int64_t)n;
  float sq = 0.f;
  if (VEC) {
    float v[4][4];
#pragma unroll
    for (int c = 0; c < 4; ++c) {
      const int i = (c * 256 + threadIdx.x) * 4;
      if (i < n) {
        gn4_load<float>(x + i, v[c]);
#pragma unroll
        for (int j = 0; j < 4; ++j) sq = fmaf(v[c][j], v[c][j], sq);
      }
    }
    sq = block256_sum(sq, scratch);
    const float r = 1.0f / sqrtf(sq / (float)n + eps);
#pragma unroll
    for (int c = 0; c < 4; ++c) {
      const int i = (c * 256 + threadIdx.x) * 4;
      if (i < n) {
        float gv[4], wv[4] = {1.f, 1.f, 1.f, 1.f};
        gn4_load<T>(gr + i, gv);
        if (w) gn4_load<T>(w + i, wv);
#pragma unroll
        for (int j = 0; j < 4; ++j) v[c][j] = v[c][j] * r * wv[j] * gn_act(gv[j], sigmoid);
        gn4_store<T>(dst + i, v[c]);
      }
    }
  } else {
    for (int i = threadIdx.x; i < n; i += 256) sq = fmaf(x[i], x[i], sq);
    sq = block256_sum(sq, scratch);
    const float r = 1.0f / sqrtf(sq / (float)n + eps);
    for (int i = threadIdx.x; i < n; i += 256)
      stf(dst + i, x[i] * r * (w ? ldf(w + i) : 1.f) * gn_act(ldf(gr + i), sigmoid));
  }
}

template <typename T>
static void launch_gla_t(float* o, const void* q, const void* k, const void* v,
                         const void* z, int64_t q_stride, int64_t k_stride,
                         int64_t v_stride, int64_t z_stride, const void* z_bias,
                         float* state, const int64_t* slots, const int* cu,
                         const int* positions, int B, int H, int dk, int dv,
                         float inv_tau, float q_scale, hipStream_t stream) {
  int G = 1;
  while (G * GLA_ROWS < dk) G <<= 1;  // host checked dk <= 64 * GLA_ROWS
  const int C = 64 / G;
  const dim3 grid((dv + 4 * C - 1) / (4 * C), H, B);
  const size_t per_token = sizeof(float) * (size_t)(3 * G * GLA_ROWS + 4 * C);
  int TC = (int)((48 << 10) / per_token);
  TC = TC < 1 ? 1 : (TC > GLA_TC_MAX ? GLA_TC_MAX : TC);
  const size_t shm = per_token * TC;
  hipLaunchKernelGGL((gla_recurrence_kernel<T>), grid, dim3(256), shm, stream,
                     o, (const T*)q, (const T*)k, (const T*)v, (const T*)z,
                     q_stride, k_stride, v_stride, z_stride, (const T*)z_bias,
                     state, slots, cu, positions, H, dk, dv, G, TC,
                     inv_tau, q_scale);
}

extern "C" void launch_gla_recurrence(
    float* o, const void* q, const void* k, const void* v, const void* z,
    int64_t q_stride, int64_t k_stride, int64_t v_stride, int64_t z_stride,
    const void* z_bias, float* state, const int64_t* slots, const int* cu,
    const int* positions, int B, int H, int dk, int dv, float inv_tau,
    float q_scale, int kind, hipStream_t stream) {
  if (B == 0) return;
  if (kind == 0)
    launch_gla_t<bf16_t>(o, q, k, v, z, q_stride, k_stride, v_stride, z_stride,
                         z_bias, state, slots, cu, positions, B, H, dk, dv,
                         inv_tau, q_scale, stream);
  else
    launch_gla_t<float>(o, q, k, v, z, q_stride, k_stride, v_stride, z_stride,
                        z_bias, state, slots, cu, positions, B, H, dk, dv,
                        inv_tau, q_scale, stream);
}

template <typename T>
static void launch_gated_rmsnorm_t(T* out, const float* o, const T* gate,
                                   int64_t gate_stride, const T* w, float eps, int T_,
                                   int H, int dv, int whole, int sigmoid,
                                   hipStream_t stream) {
  const int n = whole ? H * dv : dv;
  const bool vec = n % 4 == 0 && n <= (whole ? 4096 : 256) && gate_stride % 4 == 0 &&
                   ((uintptr_t)gate % (4 * sizeof(T))) == 0 &&
                   ((uintptr_t)w % (4 * sizeof(T))) == 0;
  if (whole) {
    if (vec)
      hipLaunchKernelGGL((gated_rmsnorm_row_kernel<T, true>), dim3(T_), dim3(256), 0,
                         stream, out, o, gate, gate_stride, w, eps, n, sigmoid);
    else
      hipLaunchKernelGGL((gated_rmsnorm_row_kernel<T, false>), dim3(T_), dim3(256), 0,
                         stream, out, o, gate, gate_stride, w, eps, n, sigmoid);
    return;
  }
  int lpr = 64;
  if (vec)
    while (lpr > 1 && lpr * 2 >= dv) lpr >>= 1;   // the smallest with 4 lpr >= dv
  const int64_t rows = (int64_t)T_ * H, per_block = 4 * (64 / lpr);
  const dim3 grid((rows + per_block - 1) / per_block);
  if (vec)
    hipLaunchKernelGGL((gated_rmsnorm_kernel<T, true>), grid, dim3(256), 0, stream, out,
                       o, gate, gate_stride, w, eps, rows, H, dv, lpr, sigmoid);
  else
    hipLaunchKernelGGL((gated_rmsnorm_kernel<T, false>), grid, dim3(256), 0, stream, out,
                       o, gate, gate_stride, w, eps, rows, H, dv, lpr, sigmoid);
}

extern "C" void launch_gated_rmsnorm(void* out, const float* o, const void* gate,
                                     int64_t gate_stride, const void* w,
                                     float eps, int T_, int H, int dv, int whole,
                                     int sigmoid, int kind, hipStream_t stream) {
  if (T_ == 0 || H == 0) return;
  if (kind == 0)
    launch_gated_rmsnorm_t<bf16_t>((bf16_t*)out, o, (const bf16_t*)gate, gate_stride,
                                   (const bf16_t*)w, eps, T_, H, dv, whole, sigmoid,
                                   stream);
  else
    launch_gated_rmsnorm_t<float>((float*)out, o, (const float*)gate, gate_stride,
                                  (const float*)w, eps, T_, H, dv, whole, sigmoid,
                                  stream);
}
