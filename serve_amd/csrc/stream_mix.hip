// A residual stream of S copies X_1 .. X_S (fp32 [T, S, d]) that sublayers read as a weighted sum and write back to
// through a matrix (hyper-connections).  One kernel does what lies between two sublayers:
//
//   X_t <- sum_s M[s, t] X_s + b_t (y + bias)         all streams at once from the old ones (M indexed [from, to])
//   u    = sum_t a_t X_t                              the copies as the next sublayer reads them
//   h    = u / sqrt(mean(u^2) + eps) * w              its norm
//
// y (null: no update, the streams stay as they are) is what the sublayer left, in one of three forms: [T, d]; fp32
// [parts, T, d] partial sums of a product, added in order; or the rows of a token's experts (fp32 [T parts, d]) with
// their weights (fp32 [T, parts]), where a row whose id is `experts` or above is the sublayer's own input (an
// identity expert: its row of `yk` holds nothing).  With `rows`, output row r takes source row rows[r] and X is left
// as it is (the sum in front of the output head).  All arithmetic is fp32; the template types are storage.
#include "common.h"

#define SM_MAX_STREAMS 16
#define SM_MAX_WIDTH 16000          // (a row of floats in LDS)

struct StreamOutput {
  const void* y;              // see above; storage type TD
  long long row_stride, part_stride;
  int parts;
  const float* wts;           // [T, parts] or null (1)
  const int* ids;             // [T, parts] or null; ids >= experts: the row is `own` (storage type TA)
  int experts;
  const void* own;
  const float* bias;          // [d] or null
};

template <typename T>
__device__ __forceinline__ float4 sm_load4(const T* p);
template <>
__device__ __forceinline__ float4 sm_load4<float>(const float* p) { return *reinterpret_cast<const float4*>(p); }
template <>
__device__ __forceinline__ float4 sm_load4<bf16_t>(const bf16_t* p) {
  const uint2 u = *reinterpret_cast<const uint2*>(p);
  return make_float4(bf16_bits_to_float(u.x & 0xffffu), bf16_bits_to_float(u.x >> 16), bf16_bits_to_float(u.y & 0xffffu),
                     bf16_bits_to_float(u.y >> 16));
}
__device__ __forceinline__ void sm_store4(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }
__device__ __forceinline__ void sm_store4(bf16_t* p, float4 v) {
  uint2 u;
  u.x = (uint32_t)float_to_bf16_bits(v.x) | ((uint32_t)float_to_bf16_bits(v.y) << 16);
  u.y = (uint32_t)float_to_bf16_bits(v.z) | ((uint32_t)float_to_bf16_bits(v.w) << 16);
  *reinterpret_cast<uint2*>(p) = u;
}
__device__ __forceinline__ void sm_fma(float4& a, float c, const float4& v) {
  a.x = fmaf(c, v.x, a.x);
  a.y = fmaf(c, v.y, a.y);
  a.z = fmaf(c, v.z, a.z);
  a.w = fmaf(c, v.w, a.w);
}

// d % 4 == 0, S streams, up to PMAX parts (loads of a thread's group are issued together, parts beyond the count are
// read from a clamped place and dropped).  One workgroup a row; u waits in LDS (d floats) for the row's sum of squares.
template <int S, typename TA, typename TD, int PMAX>
__global__ __launch_bounds__(1024) void stream_mix_vec_kernel(float* x, StreamOutput out, const float* __restrict__ mix,
                                                              const float* __restrict__ to, const float* __restrict__ from,
                                                              const float* __restrict__ w, TA* __restrict__ h,
                                                              const int* __restrict__ rows, float eps, int d) {
  extern __shared__ __attribute__((aligned(16))) float sm_u[];
  __shared__ float scratch[16];
  const int r = blockIdx.x;
  const size_t t = rows ? rows[r] : r;
  float* xr = x + t * (size_t)S * d;
  const TD* yr = reinterpret_cast<const TD*>(out.y);
  float m[S][S], b[S], a[S], pw[PMAX];
  bool own[PMAX];
#pragma unroll
  for (int s = 0; s < S; ++s) a[s] = from[s];
  if (yr) {
    yr += t * out.row_stride;
#pragma unroll
    for (int s = 0; s < S; ++s) {
      b[s] = to[s];
#pragma unroll
      for (int q = 0; q < S; ++q) m[s][q] = mix[s * S + q];
    }
#pragma unroll
    for (int p = 0; p < PMAX; ++p) {
      pw[p] = p < out.parts ? (out.wts ? out.wts[t * out.parts + p] : 1.f) : 0.f;
      own[p] = out.ids && p < out.parts && out.ids[t * out.parts + p] >= out.experts;
    }
  }
  const int groups = d >> 2;
  float ss = 0.f;
  for (int g = threadIdx.x; g < groups; g += blockDim.x) {
    const int i = g * 4;
    float4 v[S];
#pragma unroll
    for (int s = 0; s < S; ++s) v[s] = *reinterpret_cast<const float4*>(xr + (size_t)s * d + i);
    if (yr) {
      float4 y = make_float4(0.f, 0.f, 0.f, 0.f), part[PMAX];
      if (out.ids) {
        const float4 mine = sm_load4<TA>(reinterpret_cast<const TA*>(out.own) + t * d + i);
#pragma unroll
        for (int p = 0; p < PMAX; ++p) {
          part[p] = mine;
          if (!own[p]) part[p] = sm_load4<TD>(yr + (size_t)min(p, out.parts - 1) * out.part_stride + i);
        }
        // (a part beyond the count may have been read from an identity expert's row, which holds nothing)
#pragma unroll
        for (int p = 0; p < PMAX; ++p)
          if (p < out.parts) sm_fma(y, pw[p], part[p]);
      } else {
#pragma unroll
        for (int p = 0; p < PMAX; ++p) part[p] = sm_load4<TD>(yr + (size_t)min(p, out.parts - 1) * out.part_stride + i);
#pragma unroll
        for (int p = 0; p < PMAX; ++p)
          if (p < out.parts) sm_fma(y, pw[p], part[p]);
      }
      if (out.bias) {
        const float4 bv = *reinterpret_cast<const float4*>(out.bias + i);
        y.x += bv.x; y.y += bv.y; y.z += bv.z; y.w += bv.w;
      }
      float4 nv[S];
#pragma unroll
      for (int q = 0; q < S; ++q) {
        nv[q] = make_float4(b[q] * y.x, b[q] * y.y, b[q] * y.z, b[q] * y.w);
#pragma unroll
        for (int s = 0; s < S; ++s) sm_fma(nv[q], m[s][q], v[s]);
      }
#pragma unroll
      for (int q = 0; q < S; ++q) {
        v[q] = nv[q];
        if (!rows) *reinterpret_cast<float4*>(xr + (size_t)q * d + i) = nv[q];
      }
    }
    float4 u = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
    for (int s = 0; s < S; ++s) sm_fma(u, a[s], v[s]);
    ss += u.x * u.x + u.y * u.y + u.z * u.z + u.w * u.w;
    *reinterpret_cast<float4*>(sm_u + i) = u;
  }
  ss = block_sum(ss, scratch);
  const float rs = 1.0f / sqrtf(ss / (float)d + eps);
  TA* hr = h + (size_t)r * d;
  for (int g = threadIdx.x; g < groups; g += blockDim.x) {
    const int i = g * 4;
    const float4 u = *reinterpret_cast<const float4*>(sm_u + i), wv = *reinterpret_cast<const float4*>(w + i);
    sm_store4(hr + i, make_float4((u.x * rs) * wv.x, (u.y * rs) * wv.y, (u.z * rs) * wv.z, (u.w * rs) * wv.w));
  }
}

// Any d, any number of streams up to SM_MAX_STREAMS, any number of parts: an element a thread at a time.
template <typename TA, typename TD>
__global__ __launch_bounds__(256) void stream_mix_kernel(float* x, int S, StreamOutput out, const float* __restrict__ mix,
                                                         const float* __restrict__ to, const float* __restrict__ from,
                                                         const float* __restrict__ w, TA* __restrict__ h,
                                                         const int* __restrict__ rows, float eps, int d) {
  extern __shared__ __attribute__((aligned(16))) float sm_u[];
  __shared__ float scratch[16];
  const int r = blockIdx.x;
  const size_t t = rows ? rows[r] : r;
  float* xr = x + t * (size_t)S * d;
  const TD* yr = reinterpret_cast<const TD*>(out.y);
  if (yr) yr += t * out.row_stride;
  float ss = 0.f;
  for (int i = threadIdx.x; i < d; i += blockDim.x) {
    float v[SM_MAX_STREAMS];
#pragma unroll
    for (int s = 0; s < SM_MAX_STREAMS; ++s) v[s] = s < S ? xr[(size_t)s * d + i] : 0.f;
    float u = 0.f;
    if (yr) {
      float y = 0.f;
      for (int p = 0; p < out.parts; ++p) {
        const bool own = out.ids && out.ids[t * out.parts + p] >= out.experts;
        const float part = own ? to_float(reinterpret_cast<const TA*>(out.own)[t * d + i]) : to_float(yr[(size_t)p * out.part_stride + i]);
        y = fmaf(out.wts ? out.wts[t * out.parts + p] : 1.f, part, y);
      }
      if (out.bias) y += out.bias[i];
      for (int q = 0; q < S; ++q) {
        float nv = to[q] * y;
#pragma unroll
        for (int s = 0; s < SM_MAX_STREAMS; ++s)
          if (s < S) nv = fmaf(mix[s * S + q], v[s], nv);
        if (!rows) xr[(size_t)q * d + i] = nv;
        u = fmaf(from[q], nv, u);
      }
    } else {
#pragma unroll
      for (int s = 0; s < SM_MAX_STREAMS; ++s)
        if (s < S) u = fmaf(from[s], v[s], u);
    }
    ss += u * u;
    sm_u[i] = u;
  }
  ss = block_sum(ss, scratch);
  const float rs = 1.0f / sqrtf(ss / (float)d + eps);
  for (int i = threadIdx.x; i < d; i += blockDim.x) h[(size_t)r * d + i] = from_float<TA>((sm_u[i] * rs) * w[i]);
}

template <typename TA, typename TD>
static int launch_stream_mix(float* x, int S, const StreamOutput& out, const float* mix, const float* to, const float* from,
                             const float* w, void* h, const int* rows, float eps, int R, int d, hipStream_t stream) {
  const size_t lds = (((size_t)d + 3) & ~(size_t)3) * sizeof(float);
  const uintptr_t at = (uintptr_t)x | (uintptr_t)out.y | (uintptr_t)out.own | (uintptr_t)out.bias | (uintptr_t)w | (uintptr_t)h;
  const bool vec = (d & 3) == 0 && !(at & 15) && S >= 2 && S <= 4 && out.parts <= 8 && !(out.row_stride & 3) && !(out.part_stride & 3);
  if (!vec) {
    hipLaunchKernelGGL((stream_mix_kernel<TA, TD>), dim3(R), dim3(d >= 256 ? 256 : 64), lds, stream, x, S, out, mix, to, from,
                       w, (TA*)h, rows, eps, d);
    SA_LAUNCH_CHECK();
    return 0;
  }
  // few rows: a group of four values a thread, so that a row is one trip to memory and not a chain of them
  const int groups = d >> 2;
  const int full = groups >= 1024 ? 1024 : (groups + 63) / 64 * 64;
  const dim3 grid(R), block(R <= 256 || full < 256 ? full : 256);
#define GO(S_, P_)                                                                                                      \
  hipLaunchKernelGGL((stream_mix_vec_kernel<S_, TA, TD, P_>), grid, block, lds, stream, x, out, mix, to, from, w, (TA*)h, \
                     rows, eps, d)
#define GO_S(S_)                    \
  do {                              \
    if (out.parts <= 1) GO(S_, 1);  \
    else if (out.parts <= 4) GO(S_, 4); \
    else GO(S_, 8);                 \
  } while (0)
  if (S == 2) GO_S(2);
  else if (S == 3) GO_S(3);
  else GO_S(4);
#undef GO_S
#undef GO
  SA_LAUNCH_CHECK();
  return 0;
}

// x fp32 [T, S, d]; R rows of h [R, d] (R = T without `rows`).  y_dtype: storage of y.
extern "C" int sa_stream_mix(float* x, int S, const void* y, int y_dtype, long long row_stride, long long part_stride,
                             int parts, const float* wts, const int* ids, int experts, const void* own, const float* bias,
                             const float* mix, const float* to, const float* from, const float* w, void* h, int act_dtype,
                             const int* rows, float eps, int R, int d, hipStream_t stream) {
  if (R <= 0) return 0;
  if (!x || !from || !w || !h || d <= 0 || d > SM_MAX_WIDTH || S <= 0 || S > SM_MAX_STREAMS || parts < 1) return SA_ERR_ARG;
  if (y && (!mix || !to)) return SA_ERR_ARG;
  if (ids && (!y || !own || !wts || y_dtype != SA_F32)) return SA_ERR_ARG;
  const StreamOutput out = {y, row_stride, part_stride, parts, wts, ids, experts, own, bias};
  if (act_dtype == SA_F32 && (!y || y_dtype == SA_F32))
    return launch_stream_mix<float, float>(x, S, out, mix, to, from, w, h, rows, eps, R, d, stream);
  if (act_dtype == SA_BF16 && (!y || y_dtype == SA_F32))
    return launch_stream_mix<bf16_t, float>(x, S, out, mix, to, from, w, h, rows, eps, R, d, stream);
  if (act_dtype == SA_BF16 && y_dtype == SA_BF16)
    return launch_stream_mix<bf16_t, bf16_t>(x, S, out, mix, to, from, w, h, rows, eps, R, d, stream);
  return SA_ERR_UNSUPPORTED;
}
