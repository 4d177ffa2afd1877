// Causal depthwise convolution over time with silu, and the table of a rotation
// by position.
//
//   short_conv       : out[t, c] = silu(sum_i w[c, i] x[t - taps + 1 + i, c]) over
//                      packed sequences; inputs before a portion come from the
//                      slot's state [C, taps - 1] (zeros when the portion begins
//                      at position 0). A thread takes 4 channels (or 1) of 8
//                      consecutive tokens, the window in registers for up to 4
//                      taps. A second launch then moves the last taps - 1
//                      inputs into the state, when every window has read it.
//   short_conv_step  : one token per sequence: a thread per channel reads its
//                      window, writes the output and shifts the state.
//   rope_table       : (cos, sin) of pos * freq[i], angles in fp32.
#include "seq_common.h"

#define SC_RUN 8   // tokens per thread

DEVINL float sc_silu(float z) { return z / (1.0f + expf(-z)); }

template <typename T, int N>
DEVINL void sc_load(const T* p, float* v) {
  if (N == 4 && sizeof(T) == 2) {
    const uint2 raw = *reinterpret_cast<const uint2*>(p);
    v[0] = bf16_bits_to_f32((uint16_t)(raw.x & 0xffff));
    v[1 % N] = bf16_bits_to_f32((uint16_t)(raw.x >> 16));
    v[2 % N] = bf16_bits_to_f32((uint16_t)(raw.y & 0xffff));
    v[3 % N] = bf16_bits_to_f32((uint16_t)(raw.y >> 16));
  } else if (N == 4) {
    const float4 a = *reinterpret_cast<const float4*>(p);
    v[0] = a.x; v[1 % N] = a.y; v[2 % N] = a.z; v[3 % N] = a.w;
  } else {
    v[0] = ldf(p);
  }
}

template <typename T, int N>
DEVINL void sc_store(T* p, const float* v) {
  if (N == 4 && sizeof(T) == 2) {
    uint2 raw;
    raw.x = (uint32_t)f32_to_bf16_bits(v[0]) | ((uint32_t)f32_to_bf16_bits(v[1 % N]) << 16);
    raw.y = (uint32_t)f32_to_bf16_bits(v[2 % N]) | ((uint32_t)f32_to_bf16_bits(v[3 % N]) << 16);
    *reinterpret_cast<uint2*>(p) = raw;
  } else if (N == 4) {
    *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1 % N], v[2 % N], v[3 % N]);
  } else {
    stf(p, v[0]);
  }
}

// the input of channel c at token t of the portion t0 ..: from x, or, before the
// portion, from the state (sc = the channel's taps - 1 past inputs) or zero
template <typename T>
DEVINL float sc_in(const T* __restrict__ x, int64_t stride, const T* __restrict__ st,
                   int t, int t0, int n, int c, bool fresh) {
  if (t >= t0) return ldf(x + (int64_t)t * stride + c);
  return fresh ? 0.f : ldf(st + (int64_t)c * n + (n + t - t0));
}

// grid (token runs, channel blocks of 256 N); TAPS 0: any number, read one by one
template <typename T, int N, int TAPS>
__global__ __launch_bounds__(256) void short_conv_kernel(
    T* __restrict__ out, const T* __restrict__ x, int64_t stride,
    const T* __restrict__ w, const T* __restrict__ state,
    const int64_t* __restrict__ slots, const int* __restrict__ cu,
    const int* __restrict__ positions, int B, int C, int taps) {
  int run = blockIdx.x, b = 0;
  for (; b < B; ++b) {
    const int nr = (cu[b + 1] - cu[b] + SC_RUN - 1) / SC_RUN;
    if (run < nr) break;
    run -= nr;
  }
  if (b == B) return;
  const int c = (blockIdx.y * 256 + threadIdx.x) * N;
  if (c >= C) return;
  const int t0 = cu[b], t1 = cu[b + 1];
  const int ta = t0 + run * SC_RUN, tb = min(ta + SC_RUN, t1);
  const int n = taps - 1;
  const bool fresh = positions[t0] == 0;
  const T* st = state + slots[b] * (int64_t)C * n;
  if (TAPS > 0) {
    constexpr int TN = TAPS > 0 ? TAPS : 1;
    float wv[TN][N], win[SC_RUN + TN - 1][N];
#pragma unroll
    for (int i = 0; i < TN; ++i)
#pragma unroll
      for (int j = 0; j < N; ++j) wv[i][j] = ldf(w + (int64_t)(c + j) * TN + i);
#pragma unroll
    for (int r = 0; r < SC_RUN + TN - 1; ++r) {
      const int t = ta - (TN - 1) + r;
      if (t >= tb) {
#pragma unroll
        for (int j = 0; j < N; ++j) win[r][j] = 0.f;
      } else if (t >= t0) {
        sc_load<T, N>(x + (int64_t)t * stride + c, win[r]);
      } else {
#pragma unroll
        for (int j = 0; j < N; ++j)
          win[r][j] = sc_in<T>(x, stride, st, t, t0, n, c + j, fresh);
      }
    }
#pragma unroll
    for (int r = 0; r < SC_RUN; ++r) {
      if (ta + r < tb) {
        float y[N];
#pragma unroll
        for (int j = 0; j < N; ++j) {
          float s = 0.f;
#pragma unroll
          for (int i = 0; i < TN; ++i) s = fmaf(wv[i][j], win[r + i][j], s);
          y[j] = sc_silu(s);
        }
        sc_store<T, N>(out + (int64_t)(ta + r) * C + c, y);
      }
    }
  } else {
    for (int t = ta; t < tb; ++t)
      for (int j = 0; j < N; ++j) {
        float s = 0.f;
        for (int i = 0; i < taps; ++i)
          s = fmaf(ldf(w + (int64_t)(c + j) * taps + i),
                   sc_in<T>(x, stride, st, t - n + i, t0, n, c + j, fresh), s);
        stf(out + (int64_t)t * C + c + j, sc_silu(s));
      }
  }
}

// the last taps - 1 inputs of every portion, oldest first; grid (channel blocks, B)
template <typename T>
__global__ __launch_bounds__(256) void short_conv_state_kernel(
    const T* __restrict__ x, int64_t stride, T* __restrict__ state,
    const int64_t* __restrict__ slots, const int* __restrict__ cu,
    const int* __restrict__ positions, int C, int n) {
  const int b = blockIdx.y, c = blockIdx.x * 256 + threadIdx.x;
  const int t0 = cu[b], t1 = cu[b + 1];
  if (t0 >= t1 || c >= C) return;
  const bool fresh = positions[t0] == 0;
  T* st = state + slots[b] * (int64_t)C * n + (int64_t)c * n;
  // entry i becomes the input at t1 - n + i; entries still taken from the state lie
  // further on in it, so walking upwards reads them before they are replaced
  for (int i = 0; i < n; ++i) {
    const int t = t1 - n + i;
    if (t >= t0) st[i] = x[(int64_t)t * stride + c];
    else if (fresh) stf(st + i, 0.f);
    else st[i] = st[n + t - t0];
  }
}

// one token per sequence; grid (channel blocks, B)
template <typename T>
__global__ __launch_bounds__(256) void short_conv_step_kernel(
    T* __restrict__ out, const T* __restrict__ x, int64_t stride,
    const T* __restrict__ w, T* __restrict__ state, const int64_t* __restrict__ slots,
    const int* __restrict__ positions, int C, int taps) {
  const int b = blockIdx.y, c = blockIdx.x * 256 + threadIdx.x;
  if (c >= C) return;
  const int n = taps - 1;
  const bool fresh = positions[b] == 0;
  T* st = state + slots[b] * (int64_t)C * n + (int64_t)c * n;
  const T* wr = w + (int64_t)c * taps;
  const T cur = x[(int64_t)b * stride + c];
  float s = 0.f;
  for (int i = 0; i < n; ++i) {
    const float past = fresh ? 0.f : ldf(st + i);
    s = fmaf(ldf(wr + i), past, s);
    if (i > 0) stf(st + i - 1, past);
  }
  if (n > 0) st[n - 1] = cur;
  s = fmaf(ldf(wr + n), ldf(&cur), s);
  stf(out + (int64_t)b * C + c, sc_silu(s));
}

template <typename T>
static void launch_sc(void* out, const void* x, int64_t stride, const void* w,
                      void* state, const int64_t* slots, const int* cu,
                      const int* positions, int T_, int B, int C, int taps,
                      hipStream_t stream) {
  const T* xp = (const T*)x;
  if (cu == nullptr) {
    hipLaunchKernelGGL((short_conv_step_kernel<T>), dim3((C + 255) / 256, B), dim3(256), 0,
                       stream, (T*)out, xp, stride, (const T*)w, (T*)state, slots,
                       positions, C, taps);
    return;
  }
  const bool vec = C % 4 == 0 && stride % 4 == 0 && ((uintptr_t)x % (4 * sizeof(T))) == 0;
  const int runs = (T_ + SC_RUN - 1) / SC_RUN + B;   // an upper bound
#define SC_CALL(N, TP)                                                               \
  hipLaunchKernelGGL((short_conv_kernel<T, N, TP>), dim3(runs, (C / N + 255) / 256),  \
                     dim3(256), 0, stream, (T*)out, xp, stride, (const T*)w,          \
                     (const T*)state, slots, cu, positions, B, C, taps)
#define SC_TAPS(N)                                                                   \
  if (taps == 2) SC_CALL(N, 2);                                                      \
  else if (taps == 3) SC_CALL(N, 3);                                                 \
  else if (taps == 4) SC_CALL(N, 4);                                                 \
  else SC_CALL(N, 0)
  if (vec) {
    SC_TAPS(4);
  } else {
    SC_TAPS(1);
  }
#undef SC_TAPS
#undef SC_CALL
  if (taps > 1)
    hipLaunchKernelGGL((short_conv_state_kernel<T>), dim3((C + 255) / 256, B), dim3(256), 0,
                       stream, xp, stride, (T*)state, slots, cu, positions, C, taps - 1);
}

extern "C" void launch_short_conv(void* out, const void* x, int64_t stride,
                                  const void* w, void* state, const int64_t* slots,
                                  const int* cu, const int* positions, int T_, int B,
                                  int C, int taps, int kind, hipStream_t stream) {
  if (T_ == 0 || B == 0 || C == 0) return;
  if (kind == 0)
    launch_sc<bf16_t>(out, x, stride, w, state, slots, cu, positions, T_, B, C, taps, stream);
  else
    launch_sc<float>(out, x, stride, w, state, slots, cu, positions, T_, B, C, taps, stream);
}

// ---- rotation table ---------------------------------------------------------------

__global__ __launch_bounds__(256) void rope_table_kernel(float* __restrict__ out,
                                                         const int* __restrict__ positions,
                                                         const float* __restrict__ freq,
                                                         int n, int64_t total) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= total) return;
  float sn, cs;
  sincosf((float)positions[i / n] * freq[i % n], &sn, &cs);
  *reinterpret_cast<float2*>(out + 2 * i) = make_float2(cs, sn);
}

extern "C" void launch_rope_table(float* out, const int* positions, const float* freq,
                                  int n, int T_, hipStream_t stream) {
  const int64_t total = (int64_t)T_ * n;
  if (total == 0) return;
  hipLaunchKernelGGL(rope_table_kernel, dim3((total + 255) / 256), dim3(256), 0, stream,
                     out, positions, freq, n, total);
}
