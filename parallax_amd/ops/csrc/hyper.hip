// Hyper-connected residual streams (several fp32 copies of the residual that
// every sublayer reads as one weighted sum and writes back to with a matrix),
// and the elementwise ends of such a stack.
//
//   embed_streams  : out[t] = the token's embedding row, once per stream, fp32.
//   hyper_rmsnorm  : writes one sublayer's result z back and reads the next
//                    sublayer's input:
//                      z   = y + y_bias + sigmoid(gate2[t]) * y2
//                      x_t <- sum_s mix[s, t] x_s + write[t] z
//                      u   = sum_s read[s] x_s,  h = u / rms(u) * w.
//                    One 256-thread workgroup per token; a token's streams are
//                    loaded once, combined in registers and stored once; up to
//                    width 4096 u stays in registers for the norm (16-byte
//                    accesses), wider or odd rows form it again from the
//                    thread's own elements.
//   biased_glu     : act([gate | up] + bias) over a strided view.
//   softcap_logits : cap * tanh(x * scale / cap) in fp32.
#include "seq_common.h"

#include <algorithm>

#define HY_CH 4  // 256 threads x 4 elements x HY_CH = width 4096 in registers

template <typename T>
DEVINL void hy_load4(const T* p, float* v);
template <>
DEVINL void hy_load4<bf16_t>(const bf16_t* p, float* v) {
  const uint2 raw = *reinterpret_cast<const uint2*>(p);
  v[0] = bf16_bits_to_f32((uint16_t)(raw.x & 0xffff));
  v[1] = bf16_bits_to_f32((uint16_t)(raw.x >> 16));
  v[2] = bf16_bits_to_f32((uint16_t)(raw.y & 0xffff));
  v[3] = bf16_bits_to_f32((uint16_t)(raw.y >> 16));
}
template <>
DEVINL void hy_load4<float>(const float* p, float* v) {
  const float4 a = *reinterpret_cast<const float4*>(p);
  v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w;
}
template <typename T>
DEVINL void hy_store4(T* p, const float* v);
template <>
DEVINL void hy_store4<bf16_t>(bf16_t* p, const float* v) {
  uint2 raw;
  raw.x = (uint32_t)f32_to_bf16_bits(v[0]) | ((uint32_t)f32_to_bf16_bits(v[1]) << 16);
  raw.y = (uint32_t)f32_to_bf16_bits(v[2]) | ((uint32_t)f32_to_bf16_bits(v[3]) << 16);
  *reinterpret_cast<uint2*>(p) = raw;
}
template <>
DEVINL void hy_store4<float>(float* p, const float* v) {
  *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
}

// ---- embed_streams -----------------------------------------------------------

template <typename T>
__global__ __launch_bounds__(256) void embed_streams_kernel(
    float* __restrict__ out, const int64_t* __restrict__ ids,
    const T* __restrict__ table, int64_t vocab, int W, int S) {
  const int64_t t = blockIdx.x;
  int64_t id = ids[t];
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);  // never read off the table
  const T* e = table + id * (int64_t)W;
  float* o = out + t * (int64_t)W * S;
  for (int i = threadIdx.x; i < W; i += 256) {
    const float v = ldf(e + i);
    for (int s = 0; s < S; ++s) o[(int64_t)s * W + i] = v;
  }
}

// ---- hyper_rmsnorm -----------------------------------------------------------

template <typename T>
struct HyArgs {
  float* x;
  const T* y;          // or y32
  const float* y32;
  int64_t y_stride;
  const T* y_bias;     // [W] or null
  const T* y2;         // [T, W] or null
  int64_t y2_stride;
  const float* gate2;  // [T], row stride gate2_stride
  int64_t gate2_stride;
  const float* mix;    // [S, S] (from, to), or null: no update
  const float* wr;     // [S]
  const float* rd;     // [S] or null: no read
  const T* w;          // [W]
  float eps;
  T* out;
  int W;
  int S;
};

// N elements (4 or 1) of every stream at column i: update, store, return u
template <typename T, int S, int N>
DEVINL void hy_columns(const HyArgs<T>& a, float* xr, int64_t row, float sg,
                       int i, float* u) {
  constexpr int MS = S > 0 ? S : 16;
  const int ns = S > 0 ? S : a.S;
  float v[MS][N];
#pragma unroll
  for (int s = 0; s < MS; ++s)
    if (s < ns) {
      if (N == 4) hy_load4<float>(xr + (int64_t)s * a.W + i, v[s]);
      else v[s][0] = xr[(int64_t)s * a.W + i];
    }
  if (a.mix != nullptr) {
    float z[N];
    if (a.y32 != nullptr) {
      if (N == 4) hy_load4<float>(a.y32 + row * a.y_stride + i, z);
      else z[0] = a.y32[row * a.y_stride + i];
    } else {
      if (N == 4) hy_load4<T>(a.y + row * a.y_stride + i, z);
      else z[0] = ldf(a.y + row * a.y_stride + i);
    }
    if (a.y_bias != nullptr) {
#pragma unroll
      for (int j = 0; j < N; ++j) z[j] += ldf(a.y_bias + i + j);
    }
    if (a.y2 != nullptr) {
      float b[N];
      if (N == 4) hy_load4<T>(a.y2 + row * a.y2_stride + i, b);
      else b[0] = ldf(a.y2 + row * a.y2_stride + i);
#pragma unroll
      for (int j = 0; j < N; ++j) z[j] = fmaf(sg, b[j], z[j]);
    }
    float nv[MS][N];
#pragma unroll
    for (int t = 0; t < MS; ++t)
      if (t < ns) {
        const float w = a.wr[t];
#pragma unroll
        for (int j = 0; j < N; ++j) nv[t][j] = w * z[j];
#pragma unroll
        for (int s = 0; s < MS; ++s)
          if (s < ns) {
            const float m = a.mix[s * ns + t];
#pragma unroll
            for (int j = 0; j < N; ++j) nv[t][j] = fmaf(m, v[s][j], nv[t][j]);
          }
      }
#pragma unroll
    for (int s = 0; s < MS; ++s)
      if (s < ns) {
        if (N == 4) hy_store4<float>(xr + (int64_t)s * a.W + i, nv[s]);
        else xr[(int64_t)s * a.W + i] = nv[s][0];
#pragma unroll
        for (int j = 0; j < N; ++j) v[s][j] = nv[s][j];
      }
  }
#pragma unroll
  for (int j = 0; j < N; ++j) u[j] = 0.f;
  if (a.rd != nullptr) {
#pragma unroll
    for (int s = 0; s < MS; ++s)
      if (s < ns) {
        const float r = a.rd[s];
#pragma unroll
        for (int j = 0; j < N; ++j) u[j] = fmaf(r, v[s][j], u[j]);
      }
  }
}

template <typename T, int S, bool VEC>
__global__ __launch_bounds__(256) void hyper_rmsnorm_kernel(HyArgs<T> a) {
  __shared__ float red[8];
  const int64_t row = blockIdx.x;
  const int W = a.W;
  const int ns = S > 0 ? S : a.S;
  float* xr = a.x + row * (int64_t)W * ns;
  float sg = 0.f;
  if (a.mix != nullptr && a.y2 != nullptr)
    sg = 1.0f / (1.0f + expf(-a.gate2[row * a.gate2_stride]));
  float ss = 0.f;
  if (VEC) {
    float u[HY_CH][4];
#pragma unroll
    for (int c = 0; c < HY_CH; ++c) {
      const int i = (c * 256 + threadIdx.x) * 4;
      if (i < W) {
        hy_columns<T, S, 4>(a, xr, row, sg, i, u[c]);
#pragma unroll
        for (int j = 0; j < 4; ++j) ss = fmaf(u[c][j], u[c][j], ss);
      }
    }
    if (a.rd == nullptr) return;
    const float r = 1.0f / sqrtf(block256_sum(ss, red) / (float)W + a.eps);
    T* o = a.out + row * (int64_t)W;
#pragma unroll
    for (int c = 0; c < HY_CH; ++c) {
      const int i = (c * 256 + threadIdx.x) * 4;
      if (i < W) {
        float wv[4], h[4];
        hy_load4<T>(a.w + i, wv);
#pragma unroll
        for (int j = 0; j < 4; ++j) h[j] = u[c][j] * r * wv[j];
        hy_store4<T>(o + i, h);
      }
    }
  } else {
    for (int i = threadIdx.x; i < W; i += 256) {
      float u;
      hy_columns<T, S, 1>(a, xr, row, sg, i, &u);
      ss = fmaf(u, u, ss);
    }
    if (a.rd == nullptr) return;
    const float r = 1.0f / sqrtf(block256_sum(ss, red) / (float)W + a.eps);
    T* o = a.out + row * (int64_t)W;
    for (int i = threadIdx.x; i < W; i += 256) {
      float u = 0.f;   // the thread's own elements again
      for (int s = 0; s < ns; ++s) u = fmaf(a.rd[s], xr[(int64_t)s * W + i], u);
      stf(o + i, u * r * ldf(a.w + i));
    }
  }
}

template <typename T>
static void launch_hyper_t(const HyArgs<T>& a, int rows, bool vec,
                           hipStream_t stream) {
#define HY_CALL(SS, V)                                                         \
  hipLaunchKernelGGL((hyper_rmsnorm_kernel<T, SS, V>), dim3(rows), dim3(256), 0, \
                     stream, a)
#define HY_S(SS)                     \
  {                                  \
    if (vec) HY_CALL(SS, true);      \
    else HY_CALL(SS, false);         \
  }
  switch (a.S) {
    case 1: HY_S(1); break;
    case 2: HY_S(2); break;
    case 3: HY_S(3); break;
    case 4: HY_S(4); break;
    default: HY_S(0); break;
  }
#undef HY_S
#undef HY_CALL
}

extern "C" void launch_hyper_rmsnorm(
    float* x, const void* y, int y_is_f32, int64_t y_stride, const void* y_bias,
    const void* y2, int64_t y2_stride, const float* gate2, int64_t gate2_stride,
    const float* mix, const float* wr, const float* rd, const void* w, float eps,
    void* out, int rows, int W, int S, int kind, hipStream_t stream) {
  if (rows == 0) return;
  const int esz = kind == 0 ? 2 : 4;
  const int ysz = y_is_f32 ? 4 : esz;
  const bool vec =
      W % 4 == 0 && W <= 1024 * HY_CH &&
      (y == nullptr || (y_stride % 4 == 0 && ((uintptr_t)y % (4 * ysz)) == 0)) &&
      (y2 == nullptr || (y2_stride % 4 == 0 && ((uintptr_t)y2 % (4 * esz)) == 0)) &&
      (w == nullptr || ((uintptr_t)w % (4 * esz)) == 0);
#define HY_ARGS(TT)                                                            \
  HyArgs<TT> {                                                                 \
    x, y_is_f32 ? nullptr : (const TT*)y, y_is_f32 ? (const float*)y : nullptr, \
        y_stride, (const TT*)y_bias, (const TT*)y2, y2_stride, gate2,          \
        gate2_stride, mix, wr, rd, (const TT*)w, eps, (TT*)out, W, S           \
  }
  if (kind == 0) launch_hyper_t<bf16_t>(HY_ARGS(bf16_t), rows, vec, stream);
  else launch_hyper_t<float>(HY_ARGS(float), rows, vec, stream);
#undef HY_ARGS
}

extern "C" void launch_embed_streams(float* out, const int64_t* ids,
                                     const void* table, int64_t vocab, int W,
                                     int S, int T_, int kind,
                                     hipStream_t stream) {
  if (T_ == 0) return;
  if (kind == 0)
    hipLaunchKernelGGL((embed_streams_kernel<bf16_t>), dim3(T_), dim3(256), 0,
                       stream, out, ids, (const bf16_t*)table, vocab, W, S);
  else
    hipLaunchKernelGGL((embed_streams_kernel<float>), dim3(T_), dim3(256), 0,
                       stream, out, ids, (const float*)table, vocab, W, S);
}

// ---- biased_glu ------------------------------------------------------------------

DEVINL float hy_gelu_tanh(float z) {
  return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}
DEVINL float hy_silu(float z) { return z / (1.0f + expf(-z)); }

// x [rows, 2 I] (row stride free), bias [2 I] or null -> out [rows, I]
template <typename T, bool GELU, bool VEC>
__global__ __launch_bounds__(256) void biased_glu_kernel(
    T* __restrict__ out, const T* __restrict__ x, int64_t x_stride,
    const T* __restrict__ bias, int I, int64_t n) {
  const int64_t stride = (int64_t)gridDim.x * 256;
  constexpr int N = VEC ? 4 : 1;
  const int In = I / N;
  for (int64_t k = (int64_t)blockIdx.x * 256 + threadIdx.x; k < n; k += stride) {
    const int64_t row = k / In;
    const int c = (int)(k % In) * N;
    const T* p = x + row * x_stride + c;
    float g[N], u[N], o[N];
    if (VEC) {
      hy_load4<T>(p, g);
      hy_load4<T>(p + I, u);
    } else {
      g[0] = ldf(p);
      u[0] = ldf(p + I);
    }
#pragma unroll
    for (int j = 0; j < N; ++j) {
      if (bias != nullptr) {
        g[j] += ldf(bias + c + j);
        u[j] += ldf(bias + I + c + j);
      }
      o[j] = (GELU ? hy_gelu_tanh(g[j]) : hy_silu(g[j])) * u[j];
    }
    if (VEC) hy_store4<T>(out + row * (int64_t)I + c, o);
    else stf(out + row * (int64_t)I + c, o[0]);
  }
}

extern "C" void launch_biased_glu(void* out, const void* x, int64_t x_stride,
                                  const void* bias, int I, int rows, int gelu,
                                  int kind, hipStream_t stream) {
  if (rows == 0 || I == 0) return;
  const int esz = kind == 0 ? 2 : 4;
  const bool vec = I % 4 == 0 && x_stride % 4 == 0 && ((uintptr_t)x % (4 * esz)) == 0;
  const int64_t n = (int64_t)rows * (vec ? I / 4 : I);
  const int blocks = (int)std::min<int64_t>((n + 255) / 256, 256 * 16);
#define BG_CALL(TT, G, V)                                                     \
  hipLaunchKernelGGL((biased_glu_kernel<TT, G, V>), dim3(blocks), dim3(256), 0, \
                     stream, (TT*)out, (const TT*)x, x_stride,                \
                     (const TT*)bias, I, n)
#define BG_T(TT)                          \
  {                                       \
    if (gelu) {                           \
      if (vec) BG_CALL(TT, true, true);   \
      else BG_CALL(TT, true, false);      \
    } else {                              \
      if (vec) BG_CALL(TT, false, true);  \
      else BG_CALL(TT, false, false);     \
    }                                     \
  }
  if (kind == 0) BG_T(bf16_t)
  else BG_T(float)
#undef BG_T
#undef BG_CALL
}

// ---- softcap_logits --------------------------------------------------------------

template <typename T, bool VEC>
__global__ __launch_bounds__(256) void softcap_logits_kernel(
    float* __restrict__ out, const T* __restrict__ x, float scale, float cap,
    int64_t n) {
  const int64_t stride = (int64_t)gridDim.x * 256;
  constexpr int N = VEC ? 4 : 1;
  for (int64_t k = (int64_t)blockIdx.x * 256 + threadIdx.x; k < n; k += stride) {
    float v[N];
    if (VEC) hy_load4<T>(x + k * 4, v);
    else v[0] = ldf(x + k);
#pragma unroll
    for (int j = 0; j < N; ++j) {
      v[j] *= scale;
      if (cap > 0.f) v[j] = cap * tanhf(v[j] / cap);
    }
    if (VEC) hy_store4<float>(out + k * 4, v);
    else out[k] = v[0];
  }
}

extern "C" void launch_softcap_logits(float* out, const void* x, float scale,
                                      float cap, int64_t n, int kind,
                                      hipStream_t stream) {
  if (n == 0) return;
  const bool vec = n % 4 == 0;
  const int64_t m = vec ? n / 4 : n;
  const int blocks = (int)std::min<int64_t>((m + 255) / 256, 256 * 16);
#define SC_CALL(TT, V)                                                         \
  hipLaunchKernelGGL((softcap_logits_kernel<TT, V>), dim3(blocks), dim3(256), 0, \
                     stream, out, (const TT*)x, scale, cap, m)
  if (kind == 0) {
    if (vec) SC_CALL(bf16_t, true);
    else SC_CALL(bf16_t, false);
  } else {
    if (vec) SC_CALL(float, true);
    else SC_CALL(float, false);
  }
#undef SC_CALL
}
