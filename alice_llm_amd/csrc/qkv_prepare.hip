// From the rows of a fused q | k | v (| ...) projection to the attention kernels' operands, for mixers whose
// projections have biases, whose rotation pairs neighbouring dimensions, covers a part of the head, or also
// turns the values: bias add, rotation, q out, k and v into their places of the paged cache (row-major pages).
//
// The rows come in float32 (the projection's sums, nothing rounded on the way) or in the activation dtype; the
// outputs are in the activation dtype TO.  Pairing: interleaved (2i, 2i + 1) or halves (i, i + R/2) over the
// rotated width R <= d of q and k heads; the pair (u, v) at position p becomes (u cos a - v sin a,
// v cos a + u sin a), a = p * f_i, from tables [positions, R/2].  With value tables [positions, dv/2] every value
// head is turned the same way over all its dv dimensions by its own position (the attention kernel turns the
// head's output back by the query's position).
//
// With norm weights the q columns (all heads together) and the k columns (likewise) are each divided by their root
// mean square over the whole projection, eps inside the root, and multiplied by a weight of that length, after the
// bias and before the rotation; projection_rms_kernel finds the two factors of every token first, in 32-bit.  With a norm a
// head instead, every q head and every k head is divided by its own root mean square and multiplied by a weight of d numbers
// that the q heads share (and one that the k heads share): qkv_prepare_heads_kernel, a wave a head, the head in registers; it
// also writes pages in the matrix-core kernels' fragment order.
#include "common.h"
#include "alice_hip.h"
#include "kv_layout.h"

namespace {

// inv[t, part] = 1 / sqrt(mean over the part's columns of (row + bias)^2 + eps); part 0: the q columns [0, n_q),
// part 1: the k columns [n_q, n_q + n_k).
template <typename TI>
__global__ __launch_bounds__(256) void projection_rms_kernel(const TI* __restrict__ rows, int row_w, const float* __restrict__ bias,
                                                             float* __restrict__ inv, int n_q, int n_k, float eps) {
  __shared__ float red[17];
  const int t = blockIdx.x, part = blockIdx.y;
  const int c0 = part ? n_q : 0, n = part ? n_k : n_q;
  const TI* row = rows + (size_t)t * row_w;
  float ss = 0.f;
  for (int c = threadIdx.x; c < n; c += blockDim.x) {
    float x = load_f32(row, (size_t)c0 + c);
    if (bias) x += bias[c0 + c];
    ss = fmaf(x, x, ss);
  }
  ss = block_sum(ss, red);
  if (threadIdx.x == 0) inv[(size_t)t * 2 + part] = 1.f / sqrtf(ss / (float)n + eps);
}

template <typename TI, typename TO>
__global__ void qkv_prepare_kernel(const TI* __restrict__ rows, int row_w, const float* __restrict__ bias,
                                   const float* __restrict__ norm_w, const float* __restrict__ inv_rms,
                                   TO* __restrict__ q_out, TO* __restrict__ k_pool, TO* __restrict__ v_pool,
                                   const float* __restrict__ cos_t, const float* __restrict__ sin_t, int R, int interleaved,
                                   const float* __restrict__ vcos, const float* __restrict__ vsin,
                                   const int* __restrict__ positions, const int* __restrict__ seq_of_token,
                                   const int* __restrict__ block_table, int bt_stride, int nH, int nKV, int d, int dv,
                                   int page_size, int n_pages) {
  const int t = blockIdx.x, h = blockIdx.y;
  const int pos = positions[t];
  const TI* row = rows + (size_t)t * row_w;
  const int tp = pos % page_size;
  int page = -1;
  if (k_pool) {
    page = block_table[(size_t)seq_of_token[t] * bt_stride + pos / page_size];
    if (page < 0 || page >= n_pages) page = -1;
  }
  if (h < nH + nKV) {
    const bool is_q = h < nH;
    if (!is_q && page < 0) return;
    const size_t col0 = (size_t)h * d;                         // k heads follow the q heads
    TO* dst = is_q ? q_out + ((size_t)t * nH + h) * d
                   : k_pool + (((size_t)page * nKV + (h - nH)) * page_size + tp) * d;
    const int half = R >> 1;
    const float inv = norm_w ? inv_rms[(size_t)t * 2 + (is_q ? 0 : 1)] : 1.f;
    for (int i = threadIdx.x; i < half; i += blockDim.x) {
      const int e0 = interleaved ? 2 * i : i, e1 = interleaved ? 2 * i + 1 : i + half;
      float x0 = load_f32(row, col0 + e0), x1 = load_f32(row, col0 + e1);
      if (bias) { x0 += bias[col0 + e0]; x1 += bias[col0 + e1]; }
      if (norm_w) { x0 = x0 * inv * norm_w[col0 + e0]; x1 = x1 * inv * norm_w[col0 + e1]; }
      float y0, y1;
      rotate_pair(x0, x1, cos_t[(size_t)pos * half + i], sin_t[(size_t)pos * half + i], y0, y1);
      store_f32(dst, e0, y0);
      store_f32(dst, e1, y1);
    }
    for (int e = R + threadIdx.x; e < d; e += blockDim.x) {
      float x = load_f32(row, col0 + e);
      if (bias) x += bias[col0 + e];
      if (norm_w) x = x * inv * norm_w[col0 + e];
      store_f32(dst, e, x);
    }
  } else if (page >= 0) {
    const int hv = h - nH - nKV;
    const size_t col0 = (size_t)(nH + nKV) * d + (size_t)hv * dv;
    TO* dst = v_pool + (((size_t)page * nKV + hv) * page_size + tp) * dv;
    if (vcos) {
      const int half = dv >> 1;
      for (int i = threadIdx.x; i < half; i += blockDim.x) {
        const int e0 = interleaved ? 2 * i : i, e1 = interleaved ? 2 * i + 1 : i + half;
        float x0 = load_f32(row, col0 + e0), x1 = load_f32(row, col0 + e1);
        if (bias) { x0 += bias[col0 + e0]; x1 += bias[col0 + e1]; }
        float y0, y1;
        rotate_pair(x0, x1, vcos[(size_t)pos * half + i], vsin[(size_t)pos * half + i], y0, y1);
        store_f32(dst, e0, y0);
        store_f32(dst, e1, y1);
      }
    } else {
      for (int e = threadIdx.x; e < dv; e += blockDim.x) {
        float x = load_f32(row, col0 + e);
        if (bias) x += bias[col0 + e];
        store_f32(dst, e, x);
      }
    }
  }
}

// A wave takes one head of R consecutive tokens, four heads a block; a lane holds up to NP pairs of the head (d <= 128 NP): the
// rotation's pairs first, then the unrotated dimensions two by two (of an odd number the last alone).  VEC: all pairs are
// neighbours and go to and from memory as one.  norm_w: [2, d], the q heads' weight and the k heads'.
// Values in the fragment layout: eight positions of one dimension are neighbours in memory (see kv_layout.h), so where a step
// brings all eight, the wave of the first of them writes for all.
struct HeadsArgs {
  int row_w, R, interleaved, bt_stride, T, nH, nKV, d, dv, page_size, n_pages, n_heads, layout;
  float eps;
  const float *bias, *norm_w, *cos_t, *sin_t;
  const int *positions, *seq_of_token, *block_table;
};

template <typename TI> __device__ __forceinline__ void load_pair(const TI* p, size_t i, float& x, float& y);
template <> __device__ __forceinline__ void load_pair<float>(const float* p, size_t i, float& x, float& y) {
  const float2 v = *reinterpret_cast<const float2*>(p + i);
  x = v.x;
  y = v.y;
}
template <> __device__ __forceinline__ void load_pair<bf16_t>(const bf16_t* p, size_t i, float& x, float& y) {
  const uint32_t v = *reinterpret_cast<const uint32_t*>(p + i);
  x = bf16_bits_to_f32(v & 0xffffu);
  y = bf16_bits_to_f32(v >> 16);
}
__device__ __forceinline__ void store_pair(float* p, size_t i, float x, float y) { *reinterpret_cast<float2*>(p + i) = float2{x, y}; }
__device__ __forceinline__ void store_pair(bf16_t* p, size_t i, float x, float y) { *reinterpret_cast<uint32_t*>(p + i) = pack_bf16x2(x, y); }

template <typename TI>
__device__ __forceinline__ float value_of(const TI* rows, const HeadsArgs& a, int t, size_t col) {
  const float x = load_f32(rows, (size_t)t * a.row_w + col);
  return a.bias ? x + a.bias[col] : x;
}

template <typename T> __device__ __forceinline__ void load4(const T* p, size_t i, float (&x)[4]);
template <> __device__ __forceinline__ void load4<float>(const float* p, size_t i, float (&x)[4]) {
  const float4 v = *reinterpret_cast<const float4*>(p + i);
  x[0] = v.x; x[1] = v.y; x[2] = v.z; x[3] = v.w;
}
template <> __device__ __forceinline__ void load4<bf16_t>(const bf16_t* p, size_t i, float (&x)[4]) {
  const uint2 v = *reinterpret_cast<const uint2*>(p + i);
  x[0] = bf16_bits_to_f32(v.x & 0xffffu); x[1] = bf16_bits_to_f32(v.x >> 16);
  x[2] = bf16_bits_to_f32(v.y & 0xffffu); x[3] = bf16_bits_to_f32(v.y >> 16);
}

// One token's value heads [h0, h1) by one wave.  V4: four neighbouring columns a lane (rows, bias and head size allow it).
template <typename TI, typename TO, bool V4>
__device__ __forceinline__ void put_values(const TI* rows, TO* v_pool, const HeadsArgs& a, int t, int h0, int h1, int pos, int page, int lane) {
  const size_t c0 = (size_t)(a.nH + a.nKV) * a.d;              // the first value column
  TO* dst = v_pool + (size_t)page * a.nKV * a.page_size * a.dv;
  const int tp = pos % a.page_size, begin = h0 * a.dv, end = h1 * a.dv;
  if (a.layout == 0) {
    for (int c = begin + lane; c < end; c += 64)
      store_f32(dst, ((size_t)(c / a.dv) * a.page_size + tp) * a.dv + c % a.dv, value_of(rows, a, t, c0 + c));
    return;
  }
  if constexpr (sizeof(TO) == 2) {
    const int back = (pos & 31) - (pos & 12), lead = t - back, last = lead + 19;       // the unit's first token and its last, if here
    bool whole = lead >= 0 && last < a.T;
    if (whole) {
      const int s = a.seq_of_token[t];
      whole = a.seq_of_token[lead] == s && a.seq_of_token[last] == s && a.positions[lead] == pos - back && a.positions[last] == pos - back + 19;
    }
    const size_t head = (size_t)a.page_size * a.dv;
    if (!whole) {
      for (int c = begin + lane; c < end; c += 64)
        store_f32(dst, (c / a.dv) * head + v_offset(1, tp, c % a.dv, a.dv), value_of(rows, a, t, c0 + c));
      return;
    }
    if (back) return;
    constexpr int N = V4 ? 4 : 1;
    for (int c = begin + lane * N; c < end; c += 64 * N) {
      float x[8][N];
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const int tj = t + (j & 3) + 16 * (j >> 2);
        if constexpr (V4) load4<TI>(rows + (size_t)tj * a.row_w, c0 + c, x[j]);
        else x[j][0] = load_f32(rows, (size_t)tj * a.row_w + c0 + c);
      }
#pragma unroll
      for (int i = 0; i < N; ++i) {
        const float bias = a.bias ? a.bias[c0 + c + i] : 0.f;
        float y[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) y[j] = x[j][i] + bias;
        *reinterpret_cast<uint4*>(dst + (c / a.dv) * head + v_offset(1, tp, (c + i) % a.dv, a.dv)) =
            uint4{pack_bf16x2(y[0], y[1]), pack_bf16x2(y[2], y[3]), pack_bf16x2(y[4], y[5]), pack_bf16x2(y[6], y[7])};
      }
    }
  }
}

template <typename TI, typename TO, int NP, int NR, bool VEC>
__global__ __launch_bounds__(256) void qkv_prepare_heads_kernel(const TI* __restrict__ rows, TO* __restrict__ q_out, TO* __restrict__ k_pool,
                                                                TO* __restrict__ v_pool, HeadsArgs a) {
  const int t0 = blockIdx.x * NR, h = blockIdx.y * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (h >= a.n_heads) return;
  const int d = a.d;
  int pos[NR], page[NR];
#pragma unroll
  for (int r = 0; r < NR; ++r) {
    const int t = min(t0 + r, a.T - 1);
    pos[r] = a.positions[t];
    page[r] = -1;
    if (k_pool && h >= a.nH) {
      page[r] = a.block_table[(size_t)a.seq_of_token[t] * a.bt_stride + pos[r] / a.page_size];
      if (page[r] < 0 || page[r] >= a.n_pages || t0 + r >= a.T) page[r] = -1;
    }
  }
  if (h >= a.nH + a.nKV) {
#pragma unroll
    for (int r = 0; r < NR; ++r)
      if (page[r] >= 0) put_values<TI, TO, false>(rows, v_pool, a, t0 + r, h - a.nH - a.nKV, h - a.nH - a.nKV + 1, pos[r], page[r], lane);
    return;
  }
  const bool is_q = h < a.nH;
  const size_t col0 = (size_t)h * d;
  const float* w = a.norm_w + (is_q ? 0 : d);
  const int half = a.R >> 1, n_pairs = half + (d - a.R + 1) / 2;
  int e0[NP], e1[NP];
  bool on0[NP], on1[NP];
  float w0[NP], w1[NP], x0[NR][NP], x1[NR][NP], cs[NR][NP], sn[NR][NP];
#pragma unroll
  for (int k = 0; k < NP; ++k) {                                // every load before the first use
    const int i = lane + 64 * k;
    const bool turned = i < half;
    e0[k] = VEC ? 2 * i : turned ? (a.interleaved ? 2 * i : i) : a.R + 2 * (i - half);
    e1[k] = VEC ? 2 * i + 1 : turned ? (a.interleaved ? 2 * i + 1 : i + half) : e0[k] + 1;
    on0[k] = i < n_pairs;
    on1[k] = on0[k] && e1[k] < d;
    w0[k] = w1[k] = 0.f;
    if constexpr (VEC) {
      if (on0[k]) load_pair<float>(w, e0[k], w0[k], w1[k]);
    } else {
      if (on0[k]) w0[k] = w[e0[k]];
      if (on1[k]) w1[k] = w[e1[k]];
    }
#pragma unroll
    for (int r = 0; r < NR; ++r) {
      const TI* row = rows + (size_t)min(t0 + r, a.T - 1) * a.row_w;
      x0[r][k] = x1[r][k] = 0.f;
      if constexpr (VEC) {
        if (on0[k]) load_pair<TI>(row, col0 + e0[k], x0[r][k], x1[r][k]);
      } else {
        if (on0[k]) x0[r][k] = load_f32(row, col0 + e0[k]);
        if (on1[k]) x1[r][k] = load_f32(row, col0 + e1[k]);
      }
      cs[r][k] = turned ? a.cos_t[(size_t)pos[r] * half + i] : 1.f;
      sn[r][k] = turned ? a.sin_t[(size_t)pos[r] * half + i] : 0.f;
    }
  }
  float ss[NR];
#pragma unroll
  for (int r = 0; r < NR; ++r) {
    ss[r] = 0.f;
#pragma unroll
    for (int k = 0; k < NP; ++k) {
      if (a.bias && on0[k]) x0[r][k] += a.bias[col0 + e0[k]];
      if (a.bias && on1[k]) x1[r][k] += a.bias[col0 + e1[k]];
      ss[r] = fmaf(x0[r][k], x0[r][k], fmaf(x1[r][k], x1[r][k], ss[r]));
    }
  }
#pragma unroll
  for (int r = 0; r < NR; ++r) ss[r] = wave_sum(ss[r]);
#pragma unroll
  for (int r = 0; r < NR; ++r) {
    const int t = t0 + r;
    if (is_q ? t >= a.T : page[r] < 0) continue;
    const float inv = 1.f / sqrtf(ss[r] / (float)d + a.eps);
    TO* dst = is_q ? q_out + ((size_t)t * a.nH + h) * d : k_pool + ((size_t)page[r] * a.nKV + (h - a.nH)) * a.page_size * d;
    const int tp = pos[r] % a.page_size;
    auto at = [&](int e) -> size_t { return is_q ? (size_t)e : k_offset(a.layout, tp, e, d); };
#pragma unroll
    for (int k = 0; k < NP; ++k) {
      float y0, y1;
      rotate_pair(x0[r][k] * inv * w0[k], x1[r][k] * inv * w1[k], cs[r][k], sn[r][k], y0, y1);
      if constexpr (VEC) {
        if (on0[k]) store_pair(dst, at(e0[k]), y0, y1);         // (an even element and the next one are neighbours in both layouts)
      } else {
        if (on0[k]) store_f32(dst, at(e0[k]), y0);
        if (on1[k]) store_f32(dst, at(e1[k]), y1);
      }
    }
  }
}

template <typename T> __device__ __forceinline__ void load8(const T* p, float (&x)[8]);
template <> __device__ __forceinline__ void load8<float>(const float* p, float (&x)[8]) {
  const float4 u = *reinterpret_cast<const float4*>(p), v = *reinterpret_cast<const float4*>(p + 4);
  x[0] = u.x; x[1] = u.y; x[2] = u.z; x[3] = u.w; x[4] = v.x; x[5] = v.y; x[6] = v.z; x[7] = v.w;
}
template <> __device__ __forceinline__ void load8<bf16_t>(const bf16_t* p, float (&x)[8]) {
  const uint4 u = *reinterpret_cast<const uint4*>(p);
  const uint32_t w[4] = {u.x, u.y, u.z, u.w};
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    x[2 * i] = bf16_bits_to_f32(w[i] & 0xffffu);
    x[2 * i + 1] = bf16_bits_to_f32(w[i] >> 16);
  }
}
__device__ __forceinline__ void store8(float* p, const float (&y)[8]) {
  *reinterpret_cast<float4*>(p) = float4{y[0], y[1], y[2], y[3]};
  *reinterpret_cast<float4*>(p + 4) = float4{y[4], y[5], y[6], y[7]};
}
__device__ __forceinline__ void store8(bf16_t* p, const float (&y)[8]) {
  *reinterpret_cast<uint4*>(p) = uint4{pack_bf16x2(y[0], y[1]), pack_bf16x2(y[2], y[3]), pack_bf16x2(y[4], y[5]), pack_bf16x2(y[6], y[7])};
}

// The same for heads of d = 8 LPH numbers turned in neighbouring pairs (the turned part a multiple of 8): eight numbers a
// lane, LPH lanes a head, so that a wave takes neighbouring heads of a token and the work around a head (its place, the sum
// over its lanes, the root) is one instruction for all of them.  The blocks beyond the first qk_blocks take the values.
template <typename TI, typename TO, int LPH>
__global__ __launch_bounds__(256) void qkv_prepare_wide_kernel(const TI* __restrict__ rows, TO* __restrict__ q_out, TO* __restrict__ k_pool,
                                                               TO* __restrict__ v_pool, HeadsArgs a, int qk_blocks, int heads_a_wave) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  constexpr int d = 8 * LPH;
  if ((int)blockIdx.x >= qk_blocks) {
    const int per = a.nKV / heads_a_wave, item = (blockIdx.x - qk_blocks) * 4 + wave, t = item / per, hv = item % per * heads_a_wave;
    if (t >= a.T) return;
    const int pos = a.positions[t], page = a.block_table[(size_t)a.seq_of_token[t] * a.bt_stride + pos / a.page_size];
    if (page >= 0 && page < a.n_pages) put_values<TI, TO, true>(rows, v_pool, a, t, hv, hv + heads_a_wave, pos, page, lane);
    return;
  }
  const int n_qk = a.nH + a.nKV, item = blockIdx.x * (256 / LPH) + threadIdx.x / LPH;
  const bool on = item < a.T * n_qk;
  const int t = on ? item / n_qk : a.T - 1, h = on ? item % n_qk : 0, e = (threadIdx.x % LPH) * 8;
  const bool is_q = h < a.nH;
  float x[8], w[8], c[4], sn[4];
  load8<TI>(rows + (size_t)t * a.row_w + (size_t)h * d + e, x);
  load8<float>(a.norm_w + (is_q ? 0 : d) + e, w);
  const int pos = a.positions[t], half = a.R >> 1;
  int page = 0;
  if (!is_q) page = a.block_table[(size_t)a.seq_of_token[t] * a.bt_stride + pos / a.page_size];
  const bool turned = e < a.R;
  const float4 c4 = turned ? *reinterpret_cast<const float4*>(a.cos_t + (size_t)pos * half + (e >> 1)) : float4{1.f, 1.f, 1.f, 1.f};
  const float4 s4 = turned ? *reinterpret_cast<const float4*>(a.sin_t + (size_t)pos * half + (e >> 1)) : float4{0.f, 0.f, 0.f, 0.f};
  c[0] = c4.x; c[1] = c4.y; c[2] = c4.z; c[3] = c4.w;
  sn[0] = s4.x; sn[1] = s4.y; sn[2] = s4.z; sn[3] = s4.w;
  if (a.bias) {
    float b[8];
    load8<float>(a.bias + (size_t)h * d + e, b);
#pragma unroll
    for (int i = 0; i < 8; ++i) x[i] += b[i];
  }
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < 8; ++i) ss = fmaf(x[i], x[i], ss);
#pragma unroll
  for (int o = 1; o < LPH; o <<= 1) ss += __shfl_xor(ss, o, 64);
  const float inv = 1.f / sqrtf(ss / (float)d + a.eps);
  float y[8];
#pragma unroll
  for (int i = 0; i < 4; ++i) rotate_pair(x[2 * i] * inv * w[2 * i], x[2 * i + 1] * inv * w[2 * i + 1], c[i], sn[i], y[2 * i], y[2 * i + 1]);
  if (!on) return;
  if (is_q) store8(q_out + ((size_t)t * a.nH + h) * d + e, y);
  else if (page >= 0 && page < a.n_pages)
    store8(k_pool + ((size_t)page * a.nKV + (h - a.nH)) * a.page_size * d + k_offset(a.layout, pos % a.page_size, e, d), y);
}

template <typename TI, typename TO>
void launch_heads(const void* rows, void* q_out, void* k_pool, void* v_pool, const HeadsArgs& a, hipStream_t stream) {
  const bool vec = a.interleaved && a.d % 2 == 0 && a.row_w % 2 == 0 &&
                   (((uintptr_t)rows | (uintptr_t)q_out | (uintptr_t)k_pool | (uintptr_t)a.norm_w) & 7) == 0;
  const uintptr_t all = (uintptr_t)rows | (uintptr_t)q_out | (uintptr_t)k_pool | (uintptr_t)a.norm_w | (uintptr_t)a.cos_t | (uintptr_t)a.sin_t | (uintptr_t)a.bias;
  if (a.interleaved && (a.d == 64 || a.d == 128 || a.d == 256) && a.R % 8 == 0 && a.row_w % 8 == 0 && a.dv % 4 == 0 && (all & 15) == 0 &&
      (long)a.T * (a.nH + a.nKV) < (1L << 30)) {
    const int heads_a_wave = a.T >= 1024 && a.nKV > 0 ? a.nKV : 1;    // (few tokens: more waves)
    const int qk_blocks = ceil_div(a.T * (a.nH + a.nKV), 256 * 8 / a.d), blocks = qk_blocks + ceil_div(a.T * (a.nKV / heads_a_wave), 4);
#define GO(LPH) qkv_prepare_wide_kernel<TI, TO, LPH><<<blocks, 256, 0, stream>>>((const TI*)rows, (TO*)q_out, (TO*)k_pool, (TO*)v_pool, a, qk_blocks, heads_a_wave)
    if (a.d == 64) GO(8);
    else if (a.d == 128) GO(16);
    else GO(32);
#undef GO
    return;
  }
  const int nr = a.T >= 1024 ? 4 : 1;                           // many tokens: more loads of a wave in flight
  const dim3 g(ceil_div(a.T, nr), ceil_div(a.n_heads, 4));
#define GO(NP, NR, VEC) qkv_prepare_heads_kernel<TI, TO, NP, NR, VEC><<<g, 256, 0, stream>>>((const TI*)rows, (TO*)q_out, (TO*)k_pool, (TO*)v_pool, a)
#define BY_VEC(NP, NR)          \
  do {                          \
    if (vec) GO(NP, NR, true);  \
    else GO(NP, NR, false);     \
  } while (0)
  if (a.d <= 128) { if (nr == 4) BY_VEC(1, 4); else BY_VEC(1, 1); }
  else { if (nr == 4) BY_VEC(2, 4); else BY_VEC(2, 1); }
#undef BY_VEC
#undef GO
}

// x[t, c] += (a ? a[t, c] : 0) + (v ? v[c] : 0)
__global__ void add_rows_kernel(float* __restrict__ x, const float* __restrict__ a, const float* __restrict__ v, long n, int W) {
  const long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= n) return;
  float s = x[i];
  if (a) s += a[i];
  if (v) s += v[i % W];
  x[i] = s;
}

}  // namespace

extern "C" int alice_qkv_prepare(const void* rows, int rows_dtype, int row_width, const float* bias, void* q_out, void* k_pool,
                                 void* v_pool, int out_dtype, const float* cos_t, const float* sin_t, int rotary_dim,
                                 int interleaved, const float* vcos, const float* vsin, const int* positions,
                                 const int* seq_of_token, const int* block_table, int bt_stride, int T, int nH, int nKV,
                                 int d, int dv, int page_size, int n_pages, const float* norm_w, int norm_heads, float norm_eps,
                                 float* inv_rms, int kv_layout, hipStream_t stream) {
  ALICE_CHECK(dtype_ok(rows_dtype) && dtype_ok(out_dtype), "qkv_prepare: unknown dtype");
  ALICE_CHECK(norm_w == nullptr || (norm_eps > 0.f && (norm_heads || inv_rms != nullptr)), "qkv_prepare: the norm needs a positive eps, and over the whole projection its workspace");
  ALICE_CHECK(norm_w == nullptr || !norm_heads || (d <= 256 && vcos == nullptr), "qkv_prepare: the norm a head takes heads of up to 256 and values as they are");
  ALICE_CHECK(kv_layout == 0 || (kv_layout == 1 && norm_w && norm_heads && out_dtype == DT_BF16 && d % 32 == 0 && dv % 32 == 0 && (k_pool == nullptr || page_size == 64) &&
                                 (((uintptr_t)k_pool | (uintptr_t)v_pool) & 15) == 0),
              "qkv_prepare: pages in fragment order come with the norm a head, bfloat16, pages of 64 and head sizes that are multiples of 32");
  ALICE_CHECK(rows_dtype == DT_F32 || rows_dtype == out_dtype, "qkv_prepare: rows are float32 or in the outputs' dtype");
  ALICE_CHECK(T >= 0 && nH >= 1 && nKV >= 0 && d >= 1 && dv >= 1, "qkv_prepare: bad sizes T=%d nH=%d nKV=%d d=%d dv=%d", T, nH, nKV, d, dv);
  ALICE_CHECK(rotary_dim >= 0 && rotary_dim <= d && rotary_dim % 2 == 0, "qkv_prepare: rotated width %d must be even and at most %d", rotary_dim, d);
  ALICE_CHECK((cos_t == nullptr) == (sin_t == nullptr) && (rotary_dim == 0 || cos_t != nullptr), "qkv_prepare: a rotated width needs both tables");
  ALICE_CHECK((vcos == nullptr) == (vsin == nullptr) && (vcos == nullptr || dv % 2 == 0), "qkv_prepare: turning the values needs both tables and an even size");
  ALICE_CHECK((k_pool == nullptr) == (v_pool == nullptr), "qkv_prepare: key and value pools must come together");
  ALICE_CHECK(k_pool == nullptr || (block_table && seq_of_token && page_size > 0 && n_pages > 0 && nKV >= 1 && bt_stride > 0),
              "qkv_prepare: a cache write needs the block table, the token-to-sequence map and the page geometry");
  ALICE_CHECK(row_width >= (nH + (k_pool ? nKV : 0)) * d + (k_pool ? nKV * dv : 0), "qkv_prepare: rows of %d elements are too short for the heads", row_width);
  ALICE_CHECK(nH + 2 * nKV <= 65535, "qkv_prepare: too many heads for one launch");
  if (T == 0) return 0;
  dim3 grid(T, nH + (k_pool ? 2 * nKV : 0));
  if (norm_w && norm_heads) {
    const HeadsArgs ha{row_width, rotary_dim, interleaved, bt_stride, T, nH, k_pool ? nKV : 0, d, dv, page_size > 0 ? page_size : 1, n_pages,
                       nH + (k_pool ? 2 * nKV : 0), kv_layout, norm_eps, bias, norm_w, cos_t, sin_t, positions, seq_of_token, block_table};
    if (rows_dtype == DT_F32 && out_dtype == DT_F32) launch_heads<float, float>(rows, q_out, k_pool, v_pool, ha, stream);
    else if (rows_dtype == DT_F32) launch_heads<float, bf16_t>(rows, q_out, k_pool, v_pool, ha, stream);
    else launch_heads<bf16_t, bf16_t>(rows, q_out, k_pool, v_pool, ha, stream);
    ALICE_LAUNCH_CHECK();
    return 0;
  }
  const int threads = 64;
  if (norm_w) {
    dim3 g0(T, k_pool ? 2 : 1);
    if (rows_dtype == DT_F32) projection_rms_kernel<float><<<g0, 256, 0, stream>>>((const float*)rows, row_width, bias, inv_rms, nH * d, k_pool ? nKV * d : 0, norm_eps);
    else projection_rms_kernel<bf16_t><<<g0, 256, 0, stream>>>((const bf16_t*)rows, row_width, bias, inv_rms, nH * d, k_pool ? nKV * d : 0, norm_eps);
    ALICE_LAUNCH_CHECK();
  }
#define GO(TI, TO)                                                                                                          \
  qkv_prepare_kernel<TI, TO><<<grid, threads, 0, stream>>>((const TI*)rows, row_width, bias, norm_w, inv_rms, (TO*)q_out, (TO*)k_pool, (TO*)v_pool, \
      cos_t, sin_t, rotary_dim, interleaved, vcos, vsin, positions, seq_of_token, block_table, bt_stride, nH, nKV, d, dv, page_size, n_pages)
  if (rows_dtype == DT_F32 && out_dtype == DT_F32) GO(float, float);
  else if (rows_dtype == DT_F32) GO(float, bf16_t);
  else GO(bf16_t, bf16_t);
#undef GO
  ALICE_LAUNCH_CHECK();
  return 0;
}

extern "C" int alice_add_rows(float* x, const float* a, const float* v, int T, int W, hipStream_t stream) {
  ALICE_CHECK(x && T >= 0 && W >= 1, "add_rows: bad arguments");
  const long n = (long)T * W;
  if (n == 0 || (!a && !v)) return 0;
  add_rows_kernel<<<ceil_div(n, 256), 256, 0, stream>>>(x, a, v, n, W);
  ALICE_LAUNCH_CHECK();
  return 0;
}
