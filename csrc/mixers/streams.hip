// A residual of several streams per token (gfx950): X [T, n, W] fp32.  A sublayer reads u = sum_s in[s] x_s
// through an RMS norm; its output y goes back into all streams at once,
//     x_t <- sum_s mix[s, t] x_s + out[t] ((y + bias) * scale),
// and the next sublayer's u and norm are taken in the same pass.  One workgroup per token; a thread owns
// whole columns (all n streams of them), so the mix needs no exchange and X is read and written once; u
// waits in LDS for the row's mean square.  Sublayer outputs and weights are bf16 or fp32 (template T);
// the streams, their coefficients, sums and norms are fp32.
#include <algorithm>

#include "mix_common.h"

namespace mxs {

constexpr int kMaxStreams = 32;      // coefficients held in LDS by the form for any stream count
constexpr int kStreamRow = 12 * 1024;  // widest row whose u waits in LDS (48 KB)

template <typename T> __device__ __forceinline__ void load4(const T* p, float* o, bool vec);
template <> __device__ __forceinline__ void load4<float>(const float* p, float* o, bool vec) {
  if (vec) {
    const float4 a = *reinterpret_cast<const float4*>(p);
    o[0] = a.x; o[1] = a.y; o[2] = a.z; o[3] = a.w;
  } else {
    for (int e = 0; e < 4; ++e) o[e] = p[e];
  }
}
template <> __device__ __forceinline__ void load4<bf16_t>(const bf16_t* p, float* o, bool vec) {
  if (vec) {
    const uint2 a = *reinterpret_cast<const uint2*>(p);
    o[0] = bf2f_lo(a.x); o[1] = bf2f_hi(a.x); o[2] = bf2f_lo(a.y); o[3] = bf2f_hi(a.y);
  } else {
    for (int e = 0; e < 4; ++e) o[e] = bf2f(p[e]);
  }
}
__device__ __forceinline__ void store4(float* p, const float* v) { *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]); }
__device__ __forceinline__ void store4(bf16_t* p, const float* v) {
  uint2 a;
  a.x = pack2(v[0], v[1]); a.y = pack2(v[2], v[3]);
  *reinterpret_cast<uint2*>(p) = a;
}

// NS: streams, known at compile time.  START: the streams begin as the embedding row instead of being read.
// Rows are whole 4-element pieces (W % 4 == 0); vec: the sublayer's rows and the weights are aligned to them.
template <typename T, int NS, bool START>
__global__ void __launch_bounds__(256) streams_kernel(float* __restrict__ X, const T* __restrict__ y, long y_stride,
                                                      const int64_t* __restrict__ ids, long vocab,
                                                      const T* __restrict__ bias, const T* __restrict__ scale,
                                                      const float* __restrict__ coeffs, const T* __restrict__ norm_w,
                                                      T* __restrict__ h, int W, float eps, float w_offset, int in_lds, int vec) {
  __shared__ float scratch[16];
  extern __shared__ float urow[];  // [W] when in_lds
  const long t = blockIdx.x;
  float mix[NS][NS], wo[NS], wi[NS];
  if constexpr (START) {
#pragma unroll
    for (int s = 0; s < NS; ++s) wi[s] = coeffs[s];
  } else {
#pragma unroll
    for (int s = 0; s < NS; ++s) {
#pragma unroll
      for (int d = 0; d < NS; ++d) mix[s][d] = coeffs[s * NS + d];
      wo[s] = coeffs[NS * NS + s];
      wi[s] = coeffs[NS * NS + NS + s];
    }
  }
  const T* yr;
  if constexpr (START) {
    long id = ids[t];
    id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);  // padding rows carry any id
    yr = y + id * static_cast<long>(W);
  } else {
    yr = y + t * y_stride;
  }
  float* xr = X + t * static_cast<long>(NS) * W;
  auto read_u = [&](int c, float* u) {  // the new streams' combination, from memory (own writes)
#pragma unroll
    for (int e = 0; e < 4; ++e) u[e] = 0.f;
#pragma unroll
    for (int s = 0; s < NS; ++s) {
      float v[4];
      load4<float>(xr + static_cast<long>(s) * W + c, v, true);
#pragma unroll
      for (int e = 0; e < 4; ++e) u[e] += wi[s] * v[e];
    }
  };
  float ss = 0.f;
  for (int c = threadIdx.x * 4; c < W; c += 1024) {
    float d[4], u[4] = {0.f, 0.f, 0.f, 0.f};
    load4<T>(yr + c, d, vec);
    if constexpr (START) {
#pragma unroll
      for (int s = 0; s < NS; ++s) {
        store4(xr + static_cast<long>(s) * W + c, d);
#pragma unroll
        for (int e = 0; e < 4; ++e) u[e] += wi[s] * d[e];
      }
    } else {
      float x[NS][4];
#pragma unroll
      for (int s = 0; s < NS; ++s) load4<float>(xr + static_cast<long>(s) * W + c, x[s], true);
      if (bias) {
        float b[4];
        load4<T>(bias + c, b, vec);
#pragma unroll
        for (int e = 0; e < 4; ++e) d[e] += b[e];
      }
      if (scale) {
        float b[4];
        load4<T>(scale + c, b, vec);
#pragma unroll
        for (int e = 0; e < 4; ++e) d[e] *= b[e];
      }
#pragma unroll
      for (int q = 0; q < NS; ++q) {
        float v[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          float a = wo[q] * d[e];
#pragma unroll
          for (int s = 0; s < NS; ++s) a += mix[s][q] * x[s][e];
          v[e] = a;
          u[e] += wi[q] * a;
        }
        store4(xr + static_cast<long>(q) * W + c, v);
      }
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) ss += u[e] * u[e];
    if (in_lds) store4(urow + c, u);
  }
  const float r = rsqrtf(block_sum(ss, scratch) / static_cast<float>(W) + eps);
  for (int c = threadIdx.x * 4; c < W; c += 1024) {
    float u[4], w[4];
    if (in_lds) load4<float>(urow + c, u, true);
    else read_u(c, u);
    load4<T>(norm_w + c, w, vec);
#pragma unroll
    for (int e = 0; e < 4; ++e) u[e] = u[e] * r * (w_offset + w[e]);
    T* hp = h + t * W + c;
    if (vec) {
      store4(hp, u);
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) stf(hp + e, u[e]);
    }
  }
}

// Any stream count up to kMaxStreams and any width: one column per thread step, its old values in LDS.
template <typename T>
__global__ void __launch_bounds__(256) streams_any_kernel(float* __restrict__ X, int n, const T* __restrict__ y, long y_stride,
                                                          const int64_t* __restrict__ ids, long vocab,
                                                          const T* __restrict__ bias, const T* __restrict__ scale,
                                                          const float* __restrict__ coeffs, const T* __restrict__ norm_w,
                                                          T* __restrict__ h, int W, float eps, float w_offset) {
  __shared__ float scratch[16];
  __shared__ float cf[kMaxStreams * kMaxStreams + 2 * kMaxStreams];
  extern __shared__ float xs[];  // [n][256]
  const bool start = ids != nullptr;
  const int nc = start ? n : n * n + 2 * n;
  for (int i = threadIdx.x; i < nc; i += blockDim.x) cf[i] = coeffs[i];
  __syncthreads();
  const float* wi = start ? cf : cf + n * n + n;
  const long t = blockIdx.x;
  const T* yr;
  if (start) {
    long id = ids[t];
    id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
    yr = y + id * static_cast<long>(W);
  } else {
    yr = y + t * y_stride;
  }
  float* xr = X + t * static_cast<long>(n) * W;
  float* my = xs + threadIdx.x;
  float ss = 0.f;
  for (int c = threadIdx.x; c < W; c += blockDim.x) {
    float d = ldf(yr + c), u = 0.f;
    if (start) {
      for (int s = 0; s < n; ++s) {
        xr[static_cast<long>(s) * W + c] = d;
        u += wi[s] * d;
      }
    } else {
      if (bias) d += ldf(bias + c);
      if (scale) d *= ldf(scale + c);
      for (int s = 0; s < n; ++s) my[s * 256] = xr[static_cast<long>(s) * W + c];
      for (int q = 0; q < n; ++q) {
        float a = cf[n * n + q] * d;
        for (int s = 0; s < n; ++s) a += cf[s * n + q] * my[s * 256];
        xr[static_cast<long>(q) * W + c] = a;
        u += wi[q] * a;
      }
    }
    ss += u * u;
  }
  const float r = rsqrtf(block_sum(ss, scratch) / static_cast<float>(W) + eps);
  for (int c = threadIdx.x; c < W; c += blockDim.x) {
    float u = 0.f;
    for (int s = 0; s < n; ++s) u += wi[s] * xr[static_cast<long>(s) * W + c];
    stf(h + t * W + c, u * r * (w_offset + ldf(norm_w + c)));
  }
}

template <typename T>
static bool launch_streams_t(float* X, int n, const T* y, long y_stride, const int64_t* ids, long vocab, const T* bias,
                             const T* scale, const float* coeffs, const T* norm_w, T* h, int rows, int W, float eps,
                             float w_offset, hipStream_t st) {
  if (n < 1 || n > kMaxStreams) return false;
  if (n <= 4 && W % 4 == 0 && reinterpret_cast<uintptr_t>(X) % 16 == 0) {
    const size_t al = 4 * sizeof(T);
    auto ok = [&](const void* p) { return reinterpret_cast<uintptr_t>(p) % al == 0; };
    const int vec = ok(y) && ok(bias) && ok(scale) && ok(norm_w) && ok(h) && (ids != nullptr || (y_stride * sizeof(T)) % al == 0);
    const int in_lds = W <= kStreamRow;
    const size_t shm = in_lds ? static_cast<size_t>(W) * sizeof(float) : 0;
#define MIX_ST(NS)                                                                                                       \
  do {                                                                                                                   \
    if (ids) hipLaunchKernelGGL((streams_kernel<T, NS, true>), dim3(rows), dim3(256), shm, st, X, y, y_stride, ids, vocab, \
                                bias, scale, coeffs, norm_w, h, W, eps, w_offset, in_lds, vec);                          \
    else hipLaunchKernelGGL((streams_kernel<T, NS, false>), dim3(rows), dim3(256), shm, st, X, y, y_stride, ids, vocab,    \
                            bias, scale, coeffs, norm_w, h, W, eps, w_offset, in_lds, vec);                              \
  } while (0)
    if (n == 1) MIX_ST(1);
    else if (n == 2) MIX_ST(2);
    else if (n == 3) MIX_ST(3);
    else MIX_ST(4);
#undef MIX_ST
  } else {
    hipLaunchKernelGGL(streams_any_kernel<T>, dim3(rows), dim3(256), static_cast<size_t>(n) * 256 * sizeof(float), st, X, n, y,
                       y_stride, ids, vocab, bias, scale, coeffs, norm_w, h, W, eps, w_offset);
  }
  MXS_CHECK_LAUNCH();
  return true;
}

// ids != nullptr: y is the embedding table and the streams start as its rows; coeffs = in [n].
// Otherwise coeffs = mix [n, n] | out [n] | in [n].
bool launch_streams(float* X, int n, const void* y, long y_stride, const int64_t* ids, long vocab, const void* bias,
                    const void* scale, const float* coeffs, const void* norm_w, void* h, int rows, int W, float eps,
                    float w_offset, bool bf, hipStream_t st) {
  if (rows == 0) return true;
  if (bf)
    return launch_streams_t<bf16_t>(X, n, (const bf16_t*)y, y_stride, ids, vocab, (const bf16_t*)bias, (const bf16_t*)scale,
                                    coeffs, (const bf16_t*)norm_w, (bf16_t*)h, rows, W, eps, w_offset, st);
  return launch_streams_t<float>(X, n, (const float*)y, y_stride, ids, vocab, (const float*)bias, (const float*)scale, coeffs,
                                 (const float*)norm_w, (float*)h, rows, W, eps, w_offset, st);
}

// ---- activations of feed-forwards: silu, gelu in its exact and its tanh form, with or without a gate
__device__ __forceinline__ float act_f(float z, int kind) {
  if (kind == 0) return silu_f(z);
  if (kind == 1) return 0.5f * z * (1.f + erff(z * 0.70710678118654752f));
  return 0.5f * z * (1.f + tanhf(0.79788456080286536f * (z + 0.044715f * z * z * z)));
}

// out [R, F] = act(x[:, :F]) (* x[:, F:] when gated); 16-byte pieces where rows allow them
template <typename T>
__global__ void __launch_bounds__(256) act_kernel(T* __restrict__ out, const T* __restrict__ x, long x_stride, int F, long n,
                                                  int kind, int gated, int vec) {
  constexpr int EL = El<T>::N;
  const long step = static_cast<long>(gridDim.x) * blockDim.x;
  const long i0 = blockIdx.x * static_cast<long>(blockDim.x) + threadIdx.x;
  if (vec) {
    const int per = F / EL;
    for (long i = i0; i < n / EL; i += step) {
      const long r = i / per;
      const int c = static_cast<int>(i - r * per) * EL;
      float a[EL], g[EL];
      load16(x + r * x_stride + c, a);
      if (gated) load16(x + r * x_stride + F + c, g);
#pragma unroll
      for (int e = 0; e < EL; ++e) a[e] = gated ? act_f(a[e], kind) * g[e] : act_f(a[e], kind);
      store16(out + r * F + c, a);
    }
    return;
  }
  for (long i = i0; i < n; i += step) {
    const long r = i / F;
    const int c = static_cast<int>(i - r * F);
    const T* xr = x + r * x_stride;
    const float a = act_f(ldf(xr + c), kind);
    stf(out + i, gated ? a * ldf(xr + F + c) : a);
  }
}

void launch_act(void* out, const void* x, long x_stride, int rows, int F, int kind, bool gated, bool bf, hipStream_t st) {
  const long n = static_cast<long>(rows) * F;
  if (n == 0) return;
  const int el = bf ? 8 : 4;
  const int vec = F % el == 0 && x_stride % el == 0 && reinterpret_cast<uintptr_t>(x) % 16 == 0 &&
                  reinterpret_cast<uintptr_t>(out) % 16 == 0;
  const long units = vec ? n / el : n;
  const int blocks = static_cast<int>(std::min<long>((units + 255) / 256, 8192));
  if (bf)
    hipLaunchKernelGGL(act_kernel<bf16_t>, dim3(blocks), dim3(256), 0, st, (bf16_t*)out, (const bf16_t*)x, x_stride, F, n, kind,
                       gated ? 1 : 0, vec);
  else
    hipLaunchKernelGGL(act_kernel<float>, dim3(blocks), dim3(256), 0, st, (float*)out, (const float*)x, x_stride, F, n, kind,
                       gated ? 1 : 0, vec);
  MXS_CHECK_LAUNCH();
}

}  // namespace mxs
