// Shared device helpers for the gfx950 kernels: storage types, conversions, wave reductions.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

#define SA_WAVE 64

// dtype codes of the C interface
enum { SA_F32 = 0, SA_BF16 = 1 };

// error codes of the C interface (0 = ok, >0 = hipError_t of the launch)
enum { SA_ERR_ARG = -1, SA_ERR_UNSUPPORTED = -2 };

struct bf16_t {
  uint16_t v;
};

__device__ __forceinline__ float bf16_bits_to_float(uint32_t bits16) {
  return __uint_as_float(bits16 << 16);
}

// round to nearest even; NaN stays NaN
__device__ __forceinline__ uint16_t float_to_bf16_bits(float f) {
  uint32_t u = __float_as_uint(f);
  if ((u & 0x7fffffffu) > 0x7f800000u) return (uint16_t)((u >> 16) | 0x0040u);
  u += 0x7fffu + ((u >> 16) & 1u);
  return (uint16_t)(u >> 16);
}

__device__ __forceinline__ float to_float(float x) { return x; }
__device__ __forceinline__ float to_float(bf16_t x) { return bf16_bits_to_float(x.v); }

template <typename T>
__device__ __forceinline__ T from_float(float x);
template <>
__device__ __forceinline__ float from_float<float>(float x) {
  return x;
}
template <>
__device__ __forceinline__ bf16_t from_float<bf16_t>(float x) {
  bf16_t r;
  r.v = float_to_bf16_bits(x);
  return r;
}

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int o = SA_WAVE / 2; o > 0; o >>= 1) v += __shfl_xor(v, o, SA_WAVE);
  return v;
}

__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
  for (int o = SA_WAVE / 2; o > 0; o >>= 1) v = fmaxf(v, __shfl_xor(v, o, SA_WAVE));
  return v;
}

// sum over a block of up to 1024 threads; `scratch` holds at least 16 floats of LDS
__device__ __forceinline__ float block_sum(float v, float* scratch) {
  const int lane = threadIdx.x & (SA_WAVE - 1);
  const int wave = threadIdx.x / SA_WAVE;
  const int nwaves = (blockDim.x + SA_WAVE - 1) / SA_WAVE;
  v = wave_sum(v);
  __syncthreads();
  if (lane == 0) scratch[wave] = v;
  __syncthreads();
  float t = 0.f;
  for (int i = 0; i < nwaves; ++i) t += scratch[i];
  return t;
}

// Gated feed-forwards multiply an activated "gate" branch with a second, linear branch:
//   silu           g sigmoid(g) * u
//   gelu_tanh      0.5 g (1 + tanh(sqrt(2/pi) (g + 0.044715 g^3))) * u
//   clamped_swish  g' sigmoid(1.702 g') * (u' + 1), g' = min(g, limit), u' = clamp(u, -limit, limit)
enum { SA_GATE_SILU = 0, SA_GATE_GELU_TANH = 1, SA_GATE_CLAMPED_SWISH = 2, SA_GATE_KINDS = 3 };

__device__ __forceinline__ float gate_mul(float g, float u, int kind, float limit) {
  if (kind == SA_GATE_GELU_TANH)
    return (0.5f * g * (1.f + tanhf(0.7978845608028654f * (g + 0.044715f * g * g * g)))) * u;
  if (kind == SA_GATE_CLAMPED_SWISH) {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    return (g / (1.f + expf(-1.702f * g))) * (u + 1.f);
  }
  return (g / (1.f + expf(-g))) * u;
}

// e^x in a few instructions (a result below the normal range may come out as 0, one above it as infinity): 2^t with
// t = x log2(e) rounded, corrected by what the rounding of t lost, r = x log2(e) - t, as 2^t (1 + r ln 2); within two
// units in the last place.
__device__ __forceinline__ float short_exp(float x) {
  const float L2E = 1.44269502162933349609375f, L2E_LO = 1.925963033500011e-8f;
  const float t = x * L2E;
  float r = fmaf(x, L2E, -t);
  r = fmaf(x, L2E_LO, r);
  const float e = __builtin_amdgcn_exp2f(t);
  return fmaf(e, r * 0.693147182464599609375f, e);
}

// sigmoid(z) and z sigmoid(z) with that exponential and the hardware's reciprocal: within a few units in the last place
// (the exponent is kept below the overflow: beyond 80 the results are e^z and z e^z, which is nothing, either way)
__device__ __forceinline__ float short_sigmoid(float z) {
  return __builtin_amdgcn_rcpf(1.f + short_exp(fminf(-z, 80.f)));
}
__device__ __forceinline__ float short_silu(float z) { return z * short_sigmoid(z); }

// the first key that a query at position p sees: of its own run of `chunk` positions (counted from position 0) where
// chunk > 0, of the last `window` keys where window > 0, else the first of all
__device__ __forceinline__ int first_seen_key(int p, int window, int chunk) {
  if (chunk > 0) return p - p % chunk;
  return window > 0 ? max(0, p - window + 1) : 0;
}

// sin and cos of an angle of up to 4e6 rad (a position times a frequency of at most 1), to about
// 1e-6: the library's sincosf spends over a thousand cycles on arguments this large.  The multiple
// of 2 pi is taken off in three steps whose constants have few enough bits for the first two
// remainders to be exact (6.28125 = 201/32; 2029/2^20; the rest: with k < 2^20 the first remainder
// is a multiple of 2^-5 below 2^11, the second a multiple of 2^-20 below 4), the last remainder
// goes to the hardware's sine and cosine, which take their argument in turns.  Callers keep their
// angles within the bound (the rotary part refuses longer contexts when it is loaded).
__device__ __forceinline__ void sincos_reduced(float x, float* sn, float* cs) {
  const float k = rintf(x * 0.15915494309189535f);
  float r = fmaf(-k, 6.28125f, x);
  r = fmaf(-k, 1.93500518798828125e-3f, r);
  r = fmaf(-k, 3.0199159776e-7f, r);
  const float t = r * 0.15915494309189535f;
  *sn = __builtin_amdgcn_sinf(t);
  *cs = __builtin_amdgcn_cosf(t);
}

#define SA_LAUNCH_CHECK()                      \
  do {                                         \
    hipError_t e__ = hipGetLastError();        \
    if (e__ != hipSuccess) return (int)e__;    \
  } while (0)

// compute units of the current device (asked once per device; 256 if the runtime will not say)
static inline int compute_units() {
  static int cached[64] = {};
  int dev = 0;
  if (hipGetDevice(&dev) != hipSuccess || dev < 0 || dev >= 64) return 256;
  if (!cached[dev]) {
    int n = 0;
    if (hipDeviceGetAttribute(&n, hipDeviceAttributeMultiprocessorCount, dev) != hipSuccess || n <= 0) n = 256;
    cached[dev] = n;
  }
  return cached[dev];
}
