// Around the attention of a mixer whose queries, keys and values pass a short causal convolution over time, and whose
// heads may be several maps over the same values:
//
//   conv_rope_kv_write   rows z [T, q: H M D | k: G M D | v: G Dv] (one product), per channel c
//                          u_t = z_t + bias,   y_t = sum_j w[c, j] u_(t - taps + 1 + j)    (zeros before the sequence)
//                        then the first `rot` dims of every map of every query and key head turned by the position
//                        (pairs (2i, 2i + 1) or (i, i + rot / 2)), and keys and values to the token's cache slot.
//   differential_heads   o = a_1 - lambda a_2 per head, over its root mean square, times a constant and sigmoid(gate)
//
// A head's M maps share the values, so the cache holds ONE key/value head per group whose key is the maps' keys side by
// side, [k_1 | .. | k_M | 0] (Dp places, as many as the values' Dp), and every (head, map) is a query head of its own
// with zeros outside its map: q_1 = [q_1 | 0], q_2 = [0 | q_2].  Its scores are the map's own, the values are stored
// and read once for all maps, and the paged attention kernels run unchanged.
//
// State: a request's row holds the last taps - 1 rows of z (fp32, oldest first, without the bias, [taps - 1, C] from
// `off` on).  Steps in which every segment is one token update it here; after any other step `conv_state_update` does.
// All arithmetic is fp32; the template types are storage.
#include "common.h"

#define CA_MAX_TAPS 16
#define CA_RUN 4                  // consecutive tokens a thread of the prompt kernel takes (4 or 8; 8 was slower by 1 us of 11)
#define CA_THREADS 64             // (with 256: slower by 1 to 2 us of 11)

struct ConvRows {
  const float* bias;          // [C] or null
  const float* w;             // [C, taps]
  float* state;
  long long ss, off;
  const int* positions;
  const int* seg_of_token;
  const int* cu_q;
  const int* state_slots;
  int taps, C;
};

template <typename TA>
__device__ __forceinline__ void ca_sincos(float a, float* sn, float* cs) {
  if (sizeof(TA) == 2) sincos_reduced(a, sn, cs);      // 16-bit storage keeps 8 bits of the result
  else sincosf(a, sn, cs);
}

// ---------------------------------------------------------------------------------------------
// The general form: any sizes.  A thread an element of the padded queries and keys (the first element of a pair makes
// both), then an element of the values.
// ---------------------------------------------------------------------------------------------
template <typename TA>
__device__ __forceinline__ float conv_at(const TA* __restrict__ z, long long zs, const ConvRows& in, int t, int c, int pos,
                                         int li, int slot) {
  const float b = in.bias ? in.bias[c] : 0.f;
  float acc = 0.f;
  for (int j = 0; j < in.taps; ++j) {
    const int back = in.taps - 1 - j;
    float u = 0.f;
    if (li >= back) u = to_float(z[(size_t)(t - back) * zs + c]) + b;
    else if (pos >= back && slot >= 0) u = in.state[(size_t)slot * in.ss + in.off + (size_t)(j + li) * in.C + c] + b;
    acc = fmaf(in.w[(size_t)c * in.taps + j], u, acc);
  }
  return acc;
}

template <typename TA>
__global__ __launch_bounds__(256) void conv_rope_kv_write_kernel(
    const TA* __restrict__ z, long long zs, ConvRows in, TA* __restrict__ q_out, const int* __restrict__ slot,
    TA* __restrict__ k_pages, TA* __restrict__ v_pages, const float* __restrict__ freq, int rot, int adjacent, int T, int H,
    int G, int M, int D, int Dv, int Dp, int page_size, long long qk_blocks) {
  const TA zero = from_float<TA>(0.f);
  const int units = H * M + (slot ? G : 0);
  const bool is_qk = (long long)blockIdx.x < qk_blocks;
  const long long idx = ((long long)blockIdx.x - (is_qk ? 0 : qk_blocks)) * blockDim.x + threadIdx.x;
  if (is_qk) {
    if (idx >= (long long)T * units * Dp) return;
    const int i = (int)(idx % Dp);
    const long long tu = idx / Dp;
    const int u = (int)(tu % units), t = (int)(tu / units);
    const bool is_q = u < H * M;
    TA* dst;
    int first, col;                     // the places first .. first + len - 1 of dst are the channels from col on
    int len;
    if (is_q) {
      dst = q_out + ((size_t)t * H * M + u) * Dp;
      first = (u % M) * D;
      len = D;
      col = u * D;
    } else {
      const int s = slot[t];
      if (s < 0) return;
      const int g = u - H * M, page = s / page_size, off = s - page * page_size;
      dst = k_pages + (((size_t)page * G + g) * page_size + off) * Dp;
      first = 0;
      len = M * D;
      col = H * M * D + g * M * D;
    }
    if (i < first || i >= first + len) {
      dst[i] = zero;
      return;
    }
    const int e = (i - first) % D;      // the dim inside its map
    const int c = col + i - first;
    const int seg = in.seg_of_token[t], li = t - in.cu_q[seg], pos = in.positions[t], st = in.state_slots[seg];
    if (e >= rot) {
      dst[i] = from_float<TA>(conv_at(z, zs, in, t, c, pos, li, st));
      return;
    }
    const int half = rot >> 1;
    if (adjacent ? (e & 1) != 0 : e >= half) return;                  // (its partner writes both)
    const int step = adjacent ? 1 : half;
    float sn, cs;
    ca_sincos<TA>((float)pos * freq[adjacent ? e >> 1 : e], &sn, &cs);
    const float p0 = conv_at(z, zs, in, t, c, pos, li, st), p1 = conv_at(z, zs, in, t, c + step, pos, li, st);
    dst[i] = from_float<TA>(p0 * cs - p1 * sn);
    dst[i + step] = from_float<TA>(p1 * cs + p0 * sn);
    return;
  }
  if (!slot || idx >= (long long)T * G * Dp) return;
  const int t = (int)(idx % T);                                       // neighbouring lanes on neighbouring tokens
  const int gi = (int)(idx / T);
  const int g = gi / Dp, i = gi - g * Dp;
  const int s = slot[t];
  if (s < 0) return;
  const int page = s / page_size, off = s - page * page_size;
  TA out = zero;
  if (i < Dv) {
    const int seg = in.seg_of_token[t];
    out = from_float<TA>(conv_at(z, zs, in, t, (H + G) * M * D + g * Dv + i, in.positions[t], t - in.cu_q[seg], in.state_slots[seg]));
  }
  v_pages[(((size_t)page * G + g) * Dp + i) * page_size + off] = out;
}

// ---------------------------------------------------------------------------------------------
// bf16, pairs (2i, 2i + 1), up to 4 taps, D, Dv, Dp and the row stride multiples of 8, aligned arrays: a thread takes eight
// channels of TT consecutive tokens, so that a row of z is loaded once per TT tokens and thread (and taps - 1 rows in front
// of them).  TT 1: steps of single tokens, which also leave their rows in the state (`update`: every segment is one token).
// Zeros of the padding are written by the threads that hold the row's data.  Rows of z and the state's (copies of earlier rows of z) are kept as
// the bf16 bits they are.
// ---------------------------------------------------------------------------------------------
__device__ __forceinline__ void ca_unpack8(const uint4& v, float* f) {
  const uint32_t w[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
  for (int k = 0; k < 4; ++k) {
    f[2 * k] = bf16_bits_to_float(w[k] & 0xffffu);
    f[2 * k + 1] = bf16_bits_to_float(w[k] >> 16);
  }
}
typedef __bf16 ca_bf16x2_t __attribute__((ext_vector_type(2)));
typedef float ca_float2_t __attribute__((ext_vector_type(2)));
// two floats to two bf16 (round to nearest even) in one v_cvt_pk_bf16_f32
__device__ __forceinline__ uint32_t ca_pack2(float a, float b) {
  const ca_float2_t f = {a, b};
  return __builtin_bit_cast(uint32_t, __builtin_convertvector(f, ca_bf16x2_t));
}
__device__ __forceinline__ uint4 ca_pack8(const float* f) {
  return make_uint4(ca_pack2(f[0], f[1]), ca_pack2(f[2], f[3]), ca_pack2(f[4], f[5]), ca_pack2(f[6], f[7]));
}

__device__ __forceinline__ void ca_load8(const float* __restrict__ p, float* f) {
  const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
  f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w;
  f[4] = b.x; f[5] = b.y; f[6] = b.z; f[7] = b.w;
}

template <int TAPS, int TT>
__global__ __launch_bounds__(CA_THREADS) void conv_rope_kv_write_vec_kernel(
    const bf16_t* __restrict__ z, long long zs, ConvRows in, bf16_t* __restrict__ q_out, const int* __restrict__ slot,
    bf16_t* __restrict__ k_pages, bf16_t* __restrict__ v_pages, const float* __restrict__ freq, int rot, int T, int H, int G,
    int M, int D, int Dv, int Dp, int page_size, int update) {
  // data vectors of eight places: a (head, map) has D / 8, a group's keys M D / 8, its values Dv / 8
  const int nq = D >> 3, nk = M * nq, nv = Dv >> 3, row = Dp >> 3;
  const int qv = H * M * nq, kv = slot ? G * nk : 0, vv_ = slot ? G * nv : 0;
  const int item = blockIdx.x * blockDim.x + threadIdx.x;
  if (item >= qv + kv + vv_) return;
  const int t0 = blockIdx.y * TT;
  const int nt = min(TT, T - t0);
  const bool is_q = item < qv, is_k = !is_q && item < qv + kv;
  const int rel = is_q ? item : (is_k ? item - qv : item - qv - kv);
  const int per = is_q ? nq : (is_k ? nk : nv);
  const int u = rel / per, mine = rel - u * per;                     // (head, map) or group; which of its vectors
  const int first = is_q ? (u % M) * nq : 0;                         // the row's vector at which the data begin
  const int i0 = (first + mine) * 8;
  const int e0 = (is_k ? i0 % D : mine * 8);                         // the first dim inside its map
  const int c = (is_q ? u * D : (is_k ? H * M * D + u * M * D : (H + G) * M * D + u * Dv)) + mine * 8;      // first channel
  const uint4 none = make_uint4(0u, 0u, 0u, 0u);
  // the rest of a row is zeros: its vectors are dealt to the threads that hold the row's data
  if (row > per) {
    for (int n = 0; n < nt; ++n) {
      const int t = t0 + n;
      const int s = is_q ? 0 : slot[t];
      if (s < 0) continue;
      const int page = s / page_size, off = s - page * page_size;
      for (int j = mine; j < row - per; j += per) {
        const int at = (j < first ? j : j + per) * 8;
        if (is_q) {
          *reinterpret_cast<uint4*>(q_out + ((size_t)t * H * M + u) * Dp + at) = none;
        } else if (is_k) {
          *reinterpret_cast<uint4*>(k_pages + (((size_t)page * G + u) * page_size + off) * Dp + at) = none;
        } else {
          bf16_t* vp = v_pages + (((size_t)page * G + u) * Dp + at) * page_size + off;
#pragma unroll
          for (int k = 0; k < 8; ++k) vp[(size_t)k * page_size].v = 0;
        }
      }
    }
  }
  float w[8][TAPS], b[8];
#pragma unroll
  for (int k = 0; k < 2 * TAPS; ++k) {          // (c is a multiple of 8: 8 TAPS floats from an aligned place)
    const float4 v = *reinterpret_cast<const float4*>(in.w + (size_t)c * TAPS + 4 * k);
    const float f[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
    for (int j = 0; j < 4; ++j) w[(4 * k + j) / TAPS][(4 * k + j) % TAPS] = f[j];
  }
#pragma unroll
  for (int k = 0; k < 8; ++k) b[k] = 0.f;
  if (in.bias) ca_load8(in.bias + c, b);
  const bool turned = !(is_q || is_k) ? false : e0 < rot;
  float fr[4] = {0.f, 0.f, 0.f, 0.f};
  if (turned) {
#pragma unroll
    for (int k = 0; k < 4; ++k)
      if (e0 + 2 * k < rot) fr[k] = freq[(e0 >> 1) + k];
  }
  // row `back` rows in front of token t of a segment: from z, or from the request's state; `live`: it is of the sequence
  auto row_at = [&](int t, int li, int pos, int st, int back, bool& live) -> uint4 {
    live = pos >= back;
    if (li >= back) return *reinterpret_cast<const uint4*>(z + (size_t)(t - back) * zs + c);
    if (!live || st < 0) {
      live = false;
      return none;
    }
    const float* p = in.state + (size_t)st * in.ss + in.off + (size_t)(TAPS - 1 - back + li) * in.C + c;
    float f[8];
    ca_load8(p, f);
    return ca_pack8(f);
  };
  auto store = [&](int t, int pos, float* o) {
    if (turned) {
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        if (e0 + 2 * k < rot) {
          float sn, cs;
          sincos_reduced((float)pos * fr[k], &sn, &cs);
          const float p0 = o[2 * k], p1 = o[2 * k + 1];
          o[2 * k] = p0 * cs - p1 * sn;
          o[2 * k + 1] = p1 * cs + p0 * sn;
        }
      }
    }
    if (is_q) {
      *reinterpret_cast<uint4*>(q_out + ((size_t)t * H * M + u) * Dp + i0) = ca_pack8(o);
      return;
    }
    const int s = slot[t];
    if (s < 0) return;
    const int page = s / page_size, off = s - page * page_size;
    if (is_k) {
      *reinterpret_cast<uint4*>(k_pages + (((size_t)page * G + u) * page_size + off) * Dp + i0) = ca_pack8(o);
    } else {
      bf16_t* vp = v_pages + (((size_t)page * G + u) * Dp + i0) * page_size + off;
#pragma unroll
      for (int k = 0; k < 8; ++k) vp[(size_t)k * page_size] = from_float<bf16_t>(o[k]);
    }
  };
  const int seg = in.seg_of_token[t0];
  if (TT > 1 && nt == TT && in.seg_of_token[t0 + TT - 1] == seg) {
    // a run inside one segment: its rows and the taps - 1 in front of it are loaded at one go
    const int li0 = t0 - in.cu_q[seg], pos0 = in.positions[t0], st = in.state_slots[seg];
    uint4 raw[TT + TAPS - 1];
    bool live[TT + TAPS - 1];
#pragma unroll
    for (int r = 0; r < TAPS - 1; ++r) raw[r] = row_at(t0, li0, pos0, st, TAPS - 1 - r, live[r]);
#pragma unroll
    for (int n = 0; n < TT; ++n) {
      raw[TAPS - 1 + n] = *reinterpret_cast<const uint4*>(z + (size_t)(t0 + n) * zs + c);
      live[TAPS - 1 + n] = true;
    }
    // values whose tokens lie side by side in one page leave as one vector a channel
    bool side_by_side = false;
    int s0 = -1;
    if (!is_q && !is_k) {
      s0 = slot[t0];
      side_by_side = s0 >= 0 && (s0 & (TT - 1)) == 0 && (page_size & (TT - 1)) == 0;
#pragma unroll
      for (int n = 1; n < TT; ++n) side_by_side = side_by_side && slot[t0 + n] == s0 + n;
    }
    uint32_t vv[8][TT / 2 > 0 ? TT / 2 : 1];
#pragma unroll
    for (int n = 0; n < TT; ++n) {
      float o[8];
#pragma unroll
      for (int k = 0; k < 8; ++k) o[k] = 0.f;
#pragma unroll
      for (int j = 0; j < TAPS; ++j) {
        float f[8];
        ca_unpack8(raw[n + j], f);
        const float on = live[n + j] ? 1.f : 0.f;
#pragma unroll
        for (int k = 0; k < 8; ++k) o[k] = fmaf(w[k][j], on * (f[k] + b[k]), o[k]);
      }
      if (side_by_side) {
#pragma unroll
        for (int k = 0; k < 8; ++k) {
          const uint32_t bits = float_to_bf16_bits(o[k]);
          if (n & 1) vv[k][n >> 1] |= bits << 16;
          else vv[k][n >> 1] = bits;
        }
      } else {
        store(t0 + n, pos0 + n, o);
      }
    }
    if (side_by_side) {
      const int page = s0 / page_size, off = s0 - page * page_size;
      bf16_t* vp = v_pages + (((size_t)page * G + u) * Dp + i0) * page_size + off;
#pragma unroll
      for (int k = 0; k < 8; ++k) {
        if constexpr (TT == 8) *reinterpret_cast<uint4*>(vp + (size_t)k * page_size) = make_uint4(vv[k][0], vv[k][1], vv[k][2], vv[k][3]);
        else if constexpr (TT == 4) *reinterpret_cast<uint2*>(vp + (size_t)k * page_size) = make_uint2(vv[k][0], vv[k][1]);
      }
    }
    return;
  }
  for (int n = 0; n < nt; ++n) {
    const int t = t0 + n;
    const int sg = in.seg_of_token[t], li = t - in.cu_q[sg], pos = in.positions[t], st = in.state_slots[sg];
    uint4 raw[TAPS];
    bool live[TAPS];
#pragma unroll
    for (int j = 0; j < TAPS; ++j) raw[j] = row_at(t, li, pos, st, TAPS - 1 - j, live[j]);
    float o[8];
#pragma unroll
    for (int k = 0; k < 8; ++k) o[k] = 0.f;
#pragma unroll
    for (int j = 0; j < TAPS; ++j) {
      float f[8];
      ca_unpack8(raw[j], f);
      const float on = live[j] ? 1.f : 0.f;
#pragma unroll
      for (int k = 0; k < 8; ++k) o[k] = fmaf(w[k][j], on * (f[k] + b[k]), o[k]);
    }
    store(t, pos, o);
    if (TT == 1 && update && st >= 0 && TAPS > 1) {
      // the token's own row and the newest of the rows before it (this thread alone reads and writes these channels)
      float* p = in.state + (size_t)st * in.ss + in.off + c;
#pragma unroll
      for (int j = 1; j < TAPS; ++j) {
        float f[8];
        ca_unpack8(raw[j], f);
        float4* dst = reinterpret_cast<float4*>(p + (size_t)(j - 1) * in.C);
        dst[0] = make_float4(f[0], f[1], f[2], f[3]);
        dst[1] = make_float4(f[4], f[5], f[6], f[7]);
      }
    }
  }
}

// whether the kernel for eight channels a thread takes these sizes
static bool conv_vec_fits(int act_dtype, long long zs, const ConvRows& in, int rot, int adjacent, int D, int Dv, int Dp,
                          uintptr_t at) {
  if (in.taps > 1) at |= (uintptr_t)(in.state + in.off);
  at |= (uintptr_t)in.bias | (uintptr_t)in.w;
  return act_dtype == SA_BF16 && in.taps <= 4 && (adjacent || rot == 0) && !((D | Dv | Dp) & 7) && !(zs & 7) && !(in.ss & 3) &&
         !(at & 15);
}

// single_tokens: every segment of the step is one token.  *updated: 1 if the state has been updated (or there is none to
// keep), 0 if the caller still has to.
extern "C" int sa_conv_rope_kv_write(const void* z, long long zs, int act_dtype, const float* bias, const float* w, int taps,
                                     float* state, long long state_stride, long long conv_off, const int* positions,
                                     const int* seg_of_token, const int* cu_q, const int* state_slots, void* q_out,
                                     const int* slot, void* k_pages, void* v_pages, const float* freq, int rot, int adjacent,
                                     int T, int H, int G, int M, int D, int Dv, int Dp, int page_size, int single_tokens,
                                     int* updated, hipStream_t stream) {
  *updated = 0;
  if (T <= 0) return 0;
  if (!z || !w || !q_out || !positions || !seg_of_token || !cu_q || !state_slots || H <= 0 || G <= 0 || M <= 0 || D <= 0 ||
      Dv <= 0 || Dp < M * D || Dp < Dv || page_size <= 0 || taps < 1 || taps > CA_MAX_TAPS || (taps > 1 && !state))
    return SA_ERR_ARG;
  if (rot < 0 || rot % 2 || rot > D || (rot > 0 && !freq) || (slot && (!k_pages || !v_pages))) return SA_ERR_ARG;
  const int C = H * M * D + (slot ? G * (M * D + Dv) : 0);
  if (zs < C) return SA_ERR_ARG;
  const ConvRows in = {bias, w, state, state_stride, conv_off, positions, seg_of_token, cu_q, state_slots, taps, C};
  const uintptr_t at = (uintptr_t)z | (uintptr_t)q_out | (slot ? (uintptr_t)k_pages | (uintptr_t)v_pages : 0);
  if (conv_vec_fits(act_dtype, zs, in, rot, adjacent, D, Dv, Dp, at)) {
    const int items = (H * M * D + (slot ? G * (M * D + Dv) : 0)) >> 3;
    const int tt = single_tokens || T < 512 ? 1 : CA_RUN;
    const long long gy = ((long long)T + tt - 1) / tt;
    if (gy > 65535) return SA_ERR_ARG;
    dim3 grid((items + CA_THREADS - 1) / CA_THREADS, (unsigned)gy), block(CA_THREADS);
#define GO(TAPS_, TT_)                                                                                                     \
  hipLaunchKernelGGL((conv_rope_kv_write_vec_kernel<TAPS_, TT_>), grid, block, 0, stream, (const bf16_t*)z, zs, in,          \
                     (bf16_t*)q_out, slot, (bf16_t*)k_pages, (bf16_t*)v_pages, freq, rot, T, H, G, M, D, Dv, Dp, page_size, \
                     single_tokens)
#define GO_TT(TAPS_)           \
  do {                         \
    if (tt == 1) GO(TAPS_, 1); \
    else GO(TAPS_, CA_RUN);    \
  } while (0)
    if (taps == 1) GO_TT(1);
    else if (taps == 2) GO_TT(2);
    else if (taps == 3) GO_TT(3);
    else GO_TT(4);
#undef GO_TT
#undef GO
    SA_LAUNCH_CHECK();
    *updated = single_tokens || taps == 1;
    return 0;
  }
  *updated = taps == 1;
  const int threads = 256;
  const long long qk_blocks = ((long long)T * (H * M + (slot ? G : 0)) * Dp + threads - 1) / threads;
  const long long v_blocks = slot ? ((long long)T * G * Dp + threads - 1) / threads : 0;
  if (qk_blocks + v_blocks > 0x7fffffffLL) return SA_ERR_ARG;
  dim3 grid((unsigned)(qk_blocks + v_blocks)), block(threads);
  if (act_dtype == SA_F32)
    hipLaunchKernelGGL(conv_rope_kv_write_kernel<float>, grid, block, 0, stream, (const float*)z, zs, in, (float*)q_out, slot,
                       (float*)k_pages, (float*)v_pages, freq, rot, adjacent, T, H, G, M, D, Dv, Dp, page_size, qk_blocks);
  else if (act_dtype == SA_BF16)
    hipLaunchKernelGGL(conv_rope_kv_write_kernel<bf16_t>, grid, block, 0, stream, (const bf16_t*)z, zs, in, (bf16_t*)q_out,
                       slot, (bf16_t*)k_pages, (bf16_t*)v_pages, freq, rot, adjacent, T, H, G, M, D, Dv, Dp, page_size, qk_blocks);
  else return SA_ERR_UNSUPPORTED;
  SA_LAUNCH_CHECK();
  return 0;
}

// ---------------------------------------------------------------------------------------------
// a [T, 2 H, Dp] (head h's two maps at 2 h and 2 h + 1, Dv values and padding each) ->
// out[t, h, :] = N(a_1 - lambda a_2) * scale * sigmoid(gate[t, h, :]),  N(y) = y / sqrt(mean(y^2) + eps) over Dv
// gate: rows of g_stride elements, the logits from column g_col on [H Dv] (null: no gate).  A wave takes 64 / LG heads, LG
// lanes a head; a lane takes VEC neighbouring values at a time.
// ---------------------------------------------------------------------------------------------
#define DH_KEEP(vec) ((vec) == 8 ? 2 : 10)

template <typename TA, int VEC>
__device__ __forceinline__ void dh_load(const TA* p, float* f) {
  if (VEC == 8 && sizeof(TA) == 2) {
    ca_unpack8(*reinterpret_cast<const uint4*>(p), f);
  } else {
#pragma unroll
    for (int k = 0; k < VEC; ++k) f[k] = to_float(p[k]);
  }
}

template <typename TA, int VEC>
__global__ __launch_bounds__(256) void differential_heads_kernel(const TA* __restrict__ a, const TA* __restrict__ gate,
                                                                 long long g_stride, int g_col, TA* __restrict__ out,
                                                                 float lambda, float scale, float eps, long long total, int H,
                                                                 int Dv, int Dp, int lg) {
  const long long unit = ((long long)blockIdx.x * 256 + threadIdx.x) / lg;
  const int lane = threadIdx.x & (lg - 1);
  const bool on = unit < total;
  const long long th = on ? unit : 0;
  const long long t = th / H;
  const int h = (int)(th - t * H);
  const TA* a1 = a + (size_t)(2 * th) * Dp;
  const TA* a2 = a1 + Dp;
  constexpr int KEEP = DH_KEEP(VEC);      // rounds of values kept between the sum and the scaling
  float o[KEEP][VEC];
  float ss = 0.f;
#pragma unroll
  for (int n = 0; n < KEEP; ++n) {
    const int i = (lane + n * lg) * VEC;
#pragma unroll
    for (int k = 0; k < VEC; ++k) o[n][k] = 0.f;
    if (i < Dv) {
      float p[VEC], q[VEC];
      dh_load<TA, VEC>(a1 + i, p);
      dh_load<TA, VEC>(a2 + i, q);
#pragma unroll
      for (int k = 0; k < VEC; ++k) {
        o[n][k] = p[k] - lambda * q[k];
        ss = fmaf(o[n][k], o[n][k], ss);
      }
    }
  }
  for (int s = lg >> 1; s > 0; s >>= 1) ss += __shfl_xor(ss, s, SA_WAVE);
  if (!on) return;
  const float rs = (1.0f / sqrtf(ss / (float)Dv + eps)) * scale;
#pragma unroll
  for (int n = 0; n < KEEP; ++n) {
    const int i = (lane + n * lg) * VEC;
    if (i >= Dv) continue;
    float g[VEC];
    if (gate) {
      dh_load<TA, VEC>(gate + (size_t)t * g_stride + g_col + (size_t)h * Dv + i, g);
#pragma unroll
      for (int k = 0; k < VEC; ++k) g[k] = 1.0f / (1.0f + expf(-g[k]));
    } else {
#pragma unroll
      for (int k = 0; k < VEC; ++k) g[k] = 1.f;
    }
    TA* dst = out + (size_t)th * Dv + i;
    float r[VEC];
#pragma unroll
    for (int k = 0; k < VEC; ++k) r[k] = (o[n][k] * rs) * g[k];
    if (VEC == 8 && sizeof(TA) == 2) {
      *reinterpret_cast<uint4*>(dst) = ca_pack8(r);
    } else {
#pragma unroll
      for (int k = 0; k < VEC; ++k) dst[k] = from_float<TA>(r[k]);
    }
  }
}

extern "C" int sa_differential_heads(const void* a, const void* gate, long long g_stride, int g_col, void* out, int dtype,
                                     float lambda, float scale, float eps, int T, int H, int Dv, int Dp, hipStream_t stream) {
  if (T <= 0) return 0;
  if (!a || !out || H <= 0 || Dv <= 0 || Dp < Dv || g_col < 0) return SA_ERR_ARG;
  const uintptr_t at = (uintptr_t)a | (uintptr_t)out | (uintptr_t)gate;
  const bool vec = dtype == SA_BF16 && !((Dv | Dp | g_col) & 7) && !(g_stride & 7) && !(at & 15);
  const int per = vec ? 8 : 1;
  int lg = 1;
  while (lg < SA_WAVE && lg * per < Dv) lg <<= 1;
  if (Dv > DH_KEEP(per) * lg * per) return SA_ERR_ARG;
  const long long total = (long long)T * H;
  const long long blocks = (total * lg + 255) / 256;
  if (blocks > 0x7fffffffLL) return SA_ERR_ARG;
  dim3 grid((unsigned)blocks), block(256);
  if (vec)
    hipLaunchKernelGGL((differential_heads_kernel<bf16_t, 8>), grid, block, 0, stream, (const bf16_t*)a, (const bf16_t*)gate,
                       g_stride, g_col, (bf16_t*)out, lambda, scale, eps, total, H, Dv, Dp, lg);
  else if (dtype == SA_BF16)
    hipLaunchKernelGGL((differential_heads_kernel<bf16_t, 1>), grid, block, 0, stream, (const bf16_t*)a, (const bf16_t*)gate,
                       g_stride, g_col, (bf16_t*)out, lambda, scale, eps, total, H, Dv, Dp, lg);
  else if (dtype == SA_F32)
    hipLaunchKernelGGL((differential_heads_kernel<float, 1>), grid, block, 0, stream, (const float*)a, (const float*)gate,
                       g_stride, g_col, (float*)out, lambda, scale, eps, total, H, Dv, Dp, lg);
  else return SA_ERR_UNSUPPORTED;
  SA_LAUNCH_CHECK();
  return 0;
}
