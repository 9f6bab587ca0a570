// A recurrence whose gates read the current token alone, element by element over W channels:
//
//   S_t = (1 - z_t) S_(t-1) + z_t c_t,     y_t = S_t silu(g_t)
//   z = sigmoid(zeta + b_z),  c = u + 1/2 where u = upsilon + b_u >= 0, else sigmoid(u)
//
// rows fp32 [T, 3 W] = [zeta | upsilon | g], or [parts, T, 3 W] partial sums of a product that are added in order;
// bias fp32 [2 W] = [b_z | b_u]; a request's state is W floats of its row.  fp32 throughout.
//
// Two ways over a step's tokens.  Segments of at most GA_SHORT tokens (decoding): a thread a channel and segment.  Longer
// ones: the step's tokens are cut into tiles of GA_TILE wherever they lie, a thread a channel and tile (which passes over
// the short segments in it).  A first kernel runs every tile
// for what its last, still open segment adds to a state (`add`) and how much it shrinks one (`shrink`), or, where that
// segment began inside the tile, for the state itself; a second starts each tile from the state that these make of
// the tiles before it, and writes the outputs and, at the segments' ends, the requests' states.
#include <type_traits>

#include "common.h"

#define GA_TILE 32
#define GA_SHORT 16
#define GA_AHEAD 4          // tokens whose loads are in flight together ...
#define GA_RUN 16           // ... and in runs of at least so many
#define GA_CHAIN 32         // tiles whose rows are read together on the way to a tile's first state

// PMAX: upper bound of `parts`; the parts are loaded together, one beyond `parts` from a clamped address and dropped
template <int PMAX>
__device__ __forceinline__ float sum_parts(const float* __restrict__ p, int parts, size_t part_stride) {
  float a[PMAX];
#pragma unroll
  for (int q = 0; q < PMAX; ++q) a[q] = p[(size_t)min(q, parts - 1) * part_stride];
  float v = a[0];
#pragma unroll
  for (int q = 1; q < PMAX; ++q) v += q < parts ? a[q] : 0.f;
  return v;
}

__device__ __forceinline__ float gate_of(float zeta) { return short_sigmoid(zeta); }
__device__ __forceinline__ float candidate_of(float u) { return u >= 0.f ? u + 0.5f : short_sigmoid(u); }

// grid (ceil(W / blockDim), B)
template <typename TA, int PMAX>
__global__ __launch_bounds__(256) void gated_average_segment_kernel(
    const float* __restrict__ rows, int parts, size_t part_stride, const float* __restrict__ bias,
    float* __restrict__ state, long long state_stride, const int* __restrict__ cu_q, const int* __restrict__ state_slots,
    TA* __restrict__ y, int W) {
  const int c = blockIdx.x * blockDim.x + threadIdx.x;
  if (c >= W) return;
  const int seg = blockIdx.y;
  const int t0 = cu_q[seg], t1 = cu_q[seg + 1];
  if (t1 - t0 > GA_SHORT) return;
  const int slot = state_slots[seg];
  float* st = slot >= 0 ? state + (size_t)slot * state_stride + c : nullptr;
  const float bz = bias[c], bu = bias[W + c];
  float S = st ? *st : 0.f;
  for (int t = t0; t < t1; ++t) {
    const float* r = rows + (size_t)t * 3 * W + c;
    const float zeta = sum_parts<PMAX>(r, parts, part_stride), u = sum_parts<PMAX>(r + W, parts, part_stride);
    const float g = sum_parts<PMAX>(r + 2 * W, parts, part_stride);
    const float z = gate_of(zeta + bz);
    S = fmaf(z, candidate_of(u + bu), (1.f - z) * S);
    y[(size_t)t * W + c] = from_float<TA>(S * short_silu(g));
  }
  if (st) *st = S;
}

// A tile's last segment where it goes on in the next tile: scratch row `tile` = [shrink | add | start] (W each).  The
// segment began in this tile: shrink 0, add its state at the tile's end, start the state it began from (the tile's own
// second pass reads it there: by then the request's row may already hold what the segment leaves).
// grid (ceil(W / 256), tiles)
template <int PMAX>
__global__ __launch_bounds__(256) void gated_average_tile_state_kernel(
    const float* __restrict__ rows, int parts, size_t part_stride, const float* __restrict__ bias,
    const float* __restrict__ state, long long state_stride, const int* __restrict__ cu_q,
    const int* __restrict__ seg_of_token, const int* __restrict__ state_slots, float* __restrict__ scratch, int T, int W) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= W) return;
  const int tile = blockIdx.y;
  const int last = min((tile + 1) * GA_TILE, T) - 1;
  const int seg = seg_of_token[last];
  if (cu_q[seg + 1] <= last + 1) return;                    // the tile's last segment ends with it
  const int begin = cu_q[seg];
  if (cu_q[seg + 1] - begin <= GA_SHORT) return;            // (the other kernel's)
  const bool inside = begin >= tile * GA_TILE;
  const int slot = state_slots[seg];
  const float bz = bias[c], bu = bias[W + c];
  const float start = inside && slot >= 0 ? state[(size_t)slot * state_stride + c] : 0.f;
  float S = start, shrink = inside ? 0.f : 1.f;
  auto run = [&](int a, auto ahead) __attribute__((always_inline)) {
    constexpr int N = decltype(ahead)::value;
    float zr[N], ur[N];
#pragma unroll
    for (int i = 0; i < N; ++i) {
      const float* r = rows + (size_t)min(a + i, last) * 3 * W + c;
      zr[i] = sum_parts<PMAX>(r, parts, part_stride);
      ur[i] = sum_parts<PMAX>(r + W, parts, part_stride);
    }
#pragma unroll
    for (int i = 0; i < N; ++i) {
      if (a + i > last) break;
      const float z = gate_of(zr[i] + bz), keep = 1.f - z;
      S = fmaf(z, candidate_of(ur[i] + bu), keep * S);
      shrink *= keep;
    }
  };
  int a = max(begin, tile * GA_TILE);
  if (PMAX == 1)
    for (; a + GA_RUN <= last + 1; a += GA_RUN) run(a, std::integral_constant<int, GA_RUN>{});
  for (; a <= last; a += GA_AHEAD) run(a, std::integral_constant<int, GA_AHEAD>{});
  float* out = scratch + (size_t)tile * 3 * W + c;
  out[0] = shrink;
  out[W] = S;
  out[2 * W] = start;
}

// grid (ceil(W / 256), tiles)
template <typename TA, int PMAX>
__global__ __launch_bounds__(256) void gated_average_tile_kernel(
    const float* __restrict__ rows, int parts, size_t part_stride, const float* __restrict__ bias,
    float* __restrict__ state, long long state_stride, const int* __restrict__ cu_q, const int* __restrict__ seg_of_token,
    const int* __restrict__ state_slots, const float* __restrict__ scratch, TA* __restrict__ y, int T, int W) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= W) return;
  const int tile = blockIdx.y;
  const int first = tile * GA_TILE, last = min(first + GA_TILE, T) - 1;
  const float bz = bias[c], bu = bias[W + c];
  int seg = seg_of_token[first];
  if (seg_of_token[last] - seg == last - first && cu_q[seg] == first && cu_q[seg_of_token[last] + 1] == last + 1 && last > first)
    return;                                                  // single tokens throughout
  float S = 0.f;
  if (cu_q[seg] < first && cu_q[seg + 1] - cu_q[seg] > GA_SHORT) {
    // the tile begins inside a segment: the chain through the tiles before it, from the one in which the segment began
    int p = cu_q[seg] / GA_TILE;
    S = scratch[(size_t)p * 3 * W + W + c];
    for (++p; p < tile; p += GA_CHAIN) {
      float shrink[GA_CHAIN], add[GA_CHAIN];
#pragma unroll
      for (int i = 0; i < GA_CHAIN; ++i) {
        const float* r = scratch + (size_t)min(p + i, tile - 1) * 3 * W + c;
        shrink[i] = r[0];
        add[i] = r[W];
      }
#pragma unroll
      for (int i = 0; i < GA_CHAIN; ++i)
        if (p + i < tile) S = fmaf(shrink[i], S, add[i]);
    }
  }
  for (int t = first; t <= last;) {
    // the run of one segment's tokens inside the tile
    const int begin = cu_q[seg], end = cu_q[seg + 1];
    const int stop = min(end, last + 1);
    if (end - begin <= GA_SHORT) {
      t = stop;
      if (t <= last) seg = seg_of_token[t];
      continue;
    }
    const int slot = state_slots[seg];
    if (t == begin) {
      if (end > last + 1) S = scratch[(size_t)tile * 3 * W + 2 * W + c];
      else S = slot >= 0 ? state[(size_t)slot * state_stride + c] : 0.f;
    }
    auto run = [&](auto ahead) __attribute__((always_inline)) {
      constexpr int N = decltype(ahead)::value;
      float zr[N], ur[N], gr[N];
#pragma unroll
      for (int i = 0; i < N; ++i) {
        const float* r = rows + (size_t)min(t + i, stop - 1) * 3 * W + c;
        zr[i] = sum_parts<PMAX>(r, parts, part_stride);
        ur[i] = sum_parts<PMAX>(r + W, parts, part_stride);
        gr[i] = sum_parts<PMAX>(r + 2 * W, parts, part_stride);
      }
#pragma unroll
      for (int i = 0; i < N; ++i) {
        if (t + i >= stop) break;
        const float z = gate_of(zr[i] + bz);
        S = fmaf(z, candidate_of(ur[i] + bu), (1.f - z) * S);
        y[(size_t)(t + i) * W + c] = from_float<TA>(S * short_silu(gr[i]));
      }
    };
    if (PMAX == 1)
      for (; t + GA_RUN <= stop; t += GA_RUN) run(std::integral_constant<int, GA_RUN>{});
    for (; t < stop; t += GA_AHEAD) run(std::integral_constant<int, GA_AHEAD>{});
    t = stop;
    if (stop == end && slot >= 0) state[(size_t)slot * state_stride + c] = S;
    if (t <= last) seg = seg_of_token[t];
  }
}

template <typename TA, int PMAX>
static int launch_gated_average(const float* rows, int parts, const float* bias, float* state, long long state_stride,
                                const int* cu_q, const int* seg_of_token, const int* state_slots, void* y, float* scratch,
                                int T, int B, int W, int short_segments, int long_segments, hipStream_t stream) {
  const size_t part_stride = (size_t)T * 3 * W;
  if (short_segments) {
    // few segments: small workgroups, so that more of them share the channels
    const int threads = (long long)B * W >= 256LL * 4 * 256 ? 256 : 64;
    hipLaunchKernelGGL((gated_average_segment_kernel<TA, PMAX>), dim3((W + threads - 1) / threads, B), dim3(threads), 0,
                       stream, rows, parts, part_stride, bias, state, state_stride, cu_q, state_slots, (TA*)y, W);
    SA_LAUNCH_CHECK();
  }
  if (!long_segments) return 0;
  const int tiles = (T + GA_TILE - 1) / GA_TILE;
  if (tiles > 65535 || (tiles > 1 && !scratch)) return SA_ERR_ARG;
  dim3 grid((W + 255) / 256, tiles), block(256);
  if (tiles > 1) {
    hipLaunchKernelGGL((gated_average_tile_state_kernel<PMAX>), grid, block, 0, stream, rows, parts, part_stride, bias,
                       state, state_stride, cu_q, seg_of_token, state_slots, scratch, T, W);
    SA_LAUNCH_CHECK();
  }
  hipLaunchKernelGGL((gated_average_tile_kernel<TA, PMAX>), grid, block, 0, stream, rows, parts, part_stride, bias, state,
                     state_stride, cu_q, seg_of_token, state_slots, scratch, (TA*)y, T, W);
  SA_LAUNCH_CHECK();
  return 0;
}

// short_segments / long_segments: whether the step may have segments of at most, of more than GA_SHORT tokens; the latter
// go by tiles, with `scratch` fp32 [ceil(T / GA_TILE), 3 W] where there is more than one
extern "C" int sa_gated_average(const float* rows, int parts, const float* bias, float* state, long long state_stride,
                                const int* cu_q, const int* seg_of_token, const int* state_slots, void* y, int dtype,
                                float* scratch, int T, int B, int W, int short_segments, int long_segments,
                                hipStream_t stream) {
  if (T <= 0 || B <= 0) return 0;
  if (!rows || parts < 1 || parts > 8 || !bias || !state || !cu_q || !seg_of_token || !state_slots || !y || W <= 0 ||
      state_stride < W || B > 65535 || (!short_segments && !long_segments))
    return SA_ERR_ARG;
#define GO(TA, PM)                                                                                                   \
  launch_gated_average<TA, PM>(rows, parts, bias, state, state_stride, cu_q, seg_of_token, state_slots, y, scratch, T, B, \
                               W, short_segments, long_segments, stream)
  if (dtype == SA_F32) return parts == 1 ? GO(float, 1) : (parts <= 4 ? GO(float, 4) : GO(float, 8));
  if (dtype == SA_BF16) return parts == 1 ? GO(bf16_t, 1) : (parts <= 4 ? GO(bf16_t, 4) : GO(bf16_t, 8));
#undef GO
  return SA_ERR_UNSUPPORTED;
}
