// Linear attention with a constant decay a head ("lightning"): per sequence and head a matrix state S [d, dv] in 32-bit
// floats, carried from token to token in the cache's state rows:
//   S_t = g S_(t-1) + k_t v_t^T,    o_t = S_t^T q_t,     g the head's decay.
// q, k and v are rows of projections in the activation dtype, either already passed through silu (`act` 0) or passed
// through it here on the way in (`act` 1).  Everything else is 32-bit on both paths: the powers of the decays come from
// a table made on the host in 64-bit ([H, CHUNK + 1]: g^0 .. g^CHUNK), sums and the state are float32, and so is the
// read-out, which the norm behind it wants whole.
//
// lightning_walk_kernel: single tokens and short pieces.  A block per (sequence, head, 16 VEC columns); a thread holds
// VEC neighbouring columns of every 16th row of the state in registers, read once and written once a step.
//
// Longer pieces go a chunk of 64 tokens at a time.  With S the state ahead of a chunk, and j, r places in it,
//   o_j = g^(j+1) S^T q_j + sum_(r <= j) g^(j-r) (k_r . q_j) v_r,      S' = g^n S + sum_r g^(n-1-r) k_r v_r^T.
// lightning_states_kernel walks a sequence's chunks for 16 value columns of a head with the state in the matrix
// instruction's accumulators, and leaves the state ahead of every chunk in the workspace (the end state goes to the
// cache); lightning_outputs_kernel then takes all chunks side by side: the chunk's q k^T, weighted and masked, and the
// two products with the state and the values.  All products are on the 32-bit matrix instruction
// (v_mfma_f32_16x16x4_f32).  Which rows and which state row belong to a sequence is read on the device (cu_seqlens,
// slots), so a launch depends on sizes only.
#include "common.h"
#include "alice_hip.h"

namespace {

typedef float f32x4_t __attribute__((ext_vector_type(4)));

constexpr int CHUNK = ALICE_LIGHTNING_CHUNK;
constexpr int NT = 256;              // threads a block
constexpr int PS = CHUNK + 2;        // row length of the weighted products in LDS

__device__ __forceinline__ float silu_f(float z) { return z / (1.f + expf(-z)); }

struct LightningArgs {
  const void* rows; int row_w, q_col, k_col, v_col, act, vec4;
  const float* powers;                 // [H, CHUNK + 1]
  float* out;                          // [T, H dv]
  float* states;                       // [chunks, H, d, dv]: the state ahead of every chunk
  const int* cu_seqlens; const int* slots;
  float* S;                            // [slots, H, d, dv]
  int n_seqs, H, d, dv;
};

template <typename TX>
__device__ __forceinline__ float in1(const LightningArgs& a, size_t i) {
  const float x = load_f32(reinterpret_cast<const TX*>(a.rows), i);
  return a.act ? silu_f(x) : x;
}

// Four neighbouring elements k .. k + 3 of a head's part of a row (n elements from p on), as they are stored: they are
// converted where they are used, so that a thread's loads are all on their way before it waits for the first.  Loads are
// unconditional: an element beyond the part repeats one within it.  V4: rows and parts are whole groups of four.
template <typename TX, bool V4> struct Raw4;
template <> struct Raw4<float, true> {
  float4 v;
  __device__ __forceinline__ void load(const float* p, int k, int n) { v = *reinterpret_cast<const float4*>(p + min(k, n - 4)); }
  __device__ __forceinline__ float4 f32() const { return v; }
};
template <> struct Raw4<bf16_t, true> {
  uint2 v;
  __device__ __forceinline__ void load(const bf16_t* p, int k, int n) { v = *reinterpret_cast<const uint2*>(p + min(k, n - 4)); }
  __device__ __forceinline__ float4 f32() const {
    return float4{bf16_bits_to_f32(v.x & 0xffffu), bf16_bits_to_f32(v.x >> 16), bf16_bits_to_f32(v.y & 0xffffu), bf16_bits_to_f32(v.y >> 16)};
  }
};
template <typename TX> struct Raw4<TX, false> {
  TX v[4];
  __device__ __forceinline__ void load(const TX* p, int k, int n) {
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = p[min(k + i, n - 1)];
  }
  __device__ __forceinline__ float4 f32() const { return float4{load_f32(v, 0), load_f32(v, 1), load_f32(v, 2), load_f32(v, 3)}; }
};
__device__ __forceinline__ float4 activated(const LightningArgs& a, float4 x) {
  return a.act ? float4{silu_f(x.x), silu_f(x.y), silu_f(x.z), silu_f(x.w)} : x;
}
// Zeros at the elements k .. that are beyond n.
__device__ __forceinline__ float4 within(float4 x, int k, int n) {
  return float4{k < n ? x.x : 0.f, k + 1 < n ? x.y : 0.f, k + 2 < n ? x.z : 0.f, k + 3 < n ? x.w : 0.f};
}

// ------------------------------------------------------------------------------------------ single tokens, short pieces

template <typename TX, int VEC, int RI>
__global__ __launch_bounds__(NT) void lightning_walk_kernel(LightningArgs a) {
  constexpr int CB = 16 * VEC;
  __shared__ float sq[2][16 * RI], sk[2][16 * RI];
  __shared__ float red[2][4][CB];
  const int s = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int cg = tid & 15, rg = tid >> 4;                  // rows rg, rg + 16, ...; columns j0 .. j0 + VEC - 1
  const int c0 = blockIdx.z * CB, j0 = c0 + cg * VEC;
  const int t0 = a.cu_seqlens[s], t1 = a.cu_seqlens[s + 1];
  if (t1 <= t0) return;
  const int H = a.H, d = a.d, dv = a.dv;
  float* Sh = a.S + ((size_t)a.slots[s] * H + h) * d * dv;
  const float decay = a.powers[(size_t)h * (CHUNK + 1) + 1];
  const bool on = j0 < dv;                                 // VEC > 1: dv is a multiple of VEC
  float st[RI][VEC];
#pragma unroll
  for (int i = 0; i < RI; ++i) {
    const int r = rg + 16 * i;
    const bool ok = on && r < d;
    if (VEC == 4) {
      const float4 x = ok ? *reinterpret_cast<const float4*>(Sh + (size_t)r * dv + j0) : float4{0.f, 0.f, 0.f, 0.f};
      st[i][0] = x.x; st[i][1 % VEC] = x.y; st[i][2 % VEC] = x.z; st[i][3 % VEC] = x.w;
    } else {
#pragma unroll
      for (int c = 0; c < VEC; ++c) st[i][c] = ok ? Sh[(size_t)r * dv + j0 + c] : 0.f;
    }
  }
  for (int t = t0; t < t1; ++t) {
    const int buf = (t - t0) & 1;
    const size_t row = (size_t)t * a.row_w;
    for (int r = tid; r < 16 * RI; r += NT) {
      sq[buf][r] = r < d ? in1<TX>(a, row + a.q_col + h * d + r) : 0.f;
      sk[buf][r] = r < d ? in1<TX>(a, row + a.k_col + h * d + r) : 0.f;
    }
    float v[VEC], acc[VEC];
#pragma unroll
    for (int c = 0; c < VEC; ++c) {
      v[c] = on ? in1<TX>(a, row + a.v_col + h * dv + j0 + c) : 0.f;
      acc[c] = 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < RI; ++i) {
      const float k = sk[buf][rg + 16 * i], q = sq[buf][rg + 16 * i];
#pragma unroll
      for (int c = 0; c < VEC; ++c) {
        st[i][c] = fmaf(decay, st[i][c], k * v[c]);
        acc[c] = fmaf(st[i][c], q, acc[c]);
      }
    }
#pragma unroll
    for (int c = 0; c < VEC; ++c) {
      acc[c] += __shfl_xor(acc[c], 16, 64);
      acc[c] += __shfl_xor(acc[c], 32, 64);
      if (lane < 16) red[buf][wave][cg * VEC + c] = acc[c];
    }
    __syncthreads();
    if (tid < CB && c0 + tid < dv)
      a.out[(size_t)t * H * dv + h * dv + c0 + tid] = (red[buf][0][tid] + red[buf][1][tid]) + (red[buf][2][tid] + red[buf][3][tid]);
  }
#pragma unroll
  for (int i = 0; i < RI; ++i) {
    const int r = rg + 16 * i;
    if (!on || r >= d) continue;
    if (VEC == 4) *reinterpret_cast<float4*>(Sh + (size_t)r * dv + j0) = float4{st[i][0], st[i][1 % VEC], st[i][2 % VEC], st[i][3 % VEC]};
    else {
#pragma unroll
      for (int c = 0; c < VEC; ++c) Sh[(size_t)r * dv + j0 + c] = st[i][c];
    }
  }
}

// ------------------------------------------------------------------------------------------ chunks: the states

// A block: one sequence, one head, 16 value columns, all chunks in order.  Wave w holds the state's row tiles
// w TW .. w TW + TW - 1 (DP = 64 TW rows) as accumulators.
template <typename TX, int TW, bool V4>
__global__ __launch_bounds__(NT) void lightning_states_kernel(LightningArgs a) {
  constexpr int DP = 64 * TW, KS = DP + 16;                // 16 mod 32 banks: two rows of 16 neighbours meet in no bank
  constexpr int NK = CHUNK * DP / 4 / NT;                  // groups of four a thread fetches of the keys
  extern __shared__ __align__(16) float lds[];
  float* Ks = lds;                                         // [CHUNK][KS], each token's key times its decay to the chunk's end
  float* Vs = Ks + CHUNK * KS;                             // [CHUNK][16]
  const int s = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * 16, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int t0 = a.cu_seqlens[s], t1 = a.cu_seqlens[s + 1];
  if (t1 <= t0) return;
  const int H = a.H, d = a.d, dv = a.dv;
  size_t chunk = 0;                                        // this sequence's first chunk in the workspace
  for (int i = 0; i < s; ++i) chunk += (a.cu_seqlens[i + 1] - a.cu_seqlens[i] + CHUNK - 1) / CHUNK;
  const float* pw = a.powers + (size_t)h * (CHUNK + 1);
  float* Sh = a.S + ((size_t)a.slots[s] * H + h) * d * dv;
  const int col = v0 + (lane & 15), r0 = wave * TW * 16 + (lane >> 4) * 4;
  const bool col_ok = col < dv;
  f32x4_t acc[TW];
#pragma unroll
  for (int i = 0; i < TW; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int r = r0 + i * 16 + e;
      acc[i][e] = (col_ok && r < d) ? Sh[(size_t)r * dv + col] : 0.f;
    }
  const TX* rows = reinterpret_cast<const TX*>(a.rows);
  Raw4<TX, V4> pk[NK], pv;                                 // (a token beyond the chunk's last repeats it, with a weight of zero)
  auto fetch = [&](int c0) {
    const int last = min(CHUNK, t1 - c0) - 1;
#pragma unroll
    for (int u = 0; u < NK; ++u) {
      const int i = tid + u * NT, j = min(i / (DP / 4), last), k = (i % (DP / 4)) * 4;
      pk[u].load(rows + (size_t)(c0 + j) * a.row_w + a.k_col + h * d, k, d);
    }
    pv.load(rows + (size_t)(c0 + min(tid / 4, last)) * a.row_w + a.v_col + h * dv, v0 + (tid % 4) * 4, dv);
  };
  // the decays to the chunk's end of the tokens whose keys this thread stages: fixed but for the last, shorter chunk
  float pwk[NK];
  auto weights = [&](int len) {
#pragma unroll
    for (int u = 0; u < NK; ++u) {
      const int j = (tid + u * NT) / (DP / 4);
      pwk[u] = j < len ? pw[len - 1 - j] : 0.f;
    }
  };
  fetch(t0);
  weights(min(CHUNK, t1 - t0));
  for (int c0 = t0; c0 < t1; c0 += CHUNK, ++chunk) {
    const int len = min(CHUNK, t1 - c0);
    if (len < CHUNK && c0 != t0) weights(len);
#pragma unroll
    for (int u = 0; u < NK; ++u) {
      const int i = tid + u * NT, j = i / (DP / 4), k = (i % (DP / 4)) * 4;
      const float4 x = activated(a, pk[u].f32());
      *reinterpret_cast<float4*>(Ks + j * KS + k) = float4{x.x * pwk[u], x.y * pwk[u], x.z * pwk[u], x.w * pwk[u]};
    }
    *reinterpret_cast<float4*>(Vs + (tid / 4) * 16 + (tid % 4) * 4) = activated(a, pv.f32());
    const float keep = pw[len];
    if (c0 + CHUNK < t1) fetch(c0 + CHUNK);                // on its way during the products (the barriers wait for LDS only)
    float* dst = a.states + (chunk * H + h) * d * dv;
#pragma unroll
    for (int i = 0; i < TW; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int r = r0 + i * 16 + e;
        if (col_ok && r < d) dst[(size_t)r * dv + col] = acc[i][e];
      }
    lds_barrier();
    f32x4_t c1[TW], c2[TW];
#pragma unroll
    for (int i = 0; i < TW; ++i) c1[i] = c2[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    const float* ka = Ks + (lane >> 4) * KS + wave * TW * 16 + (lane & 15);
    const float* vb = Vs + (lane >> 4) * 16 + (lane & 15);
#pragma unroll 4
    for (int kk = 0; kk < CHUNK; kk += 8) {
      const float b0 = vb[kk * 16], b1 = vb[(kk + 4) * 16];
#pragma unroll
      for (int i = 0; i < TW; ++i) {
        c1[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(ka[kk * KS + i * 16], b0, c1[i], 0, 0, 0);
        c2[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(ka[(kk + 4) * KS + i * 16], b1, c2[i], 0, 0, 0);
      }
    }
#pragma unroll
    for (int i = 0; i < TW; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) acc[i][e] = fmaf(keep, acc[i][e], c1[i][e] + c2[i][e]);
    lds_barrier();                                         // the buffers have been read
  }
#pragma unroll
  for (int i = 0; i < TW; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int r = r0 + i * 16 + e;
      if (col_ok && r < d) Sh[(size_t)r * dv + col] = acc[i][e];
    }
}

// ------------------------------------------------------------------------------------------ chunks: the read-outs

// A block: one chunk of one head, all its value columns.  TW as above; a wave takes CT column tiles of 16 at a time
// against the chunk's four row tiles: the state's and the values' elements come straight from memory (each is used by
// one wave only), q and the weighted q k^T from LDS.
template <typename TX, int TW, int CT, bool V4>
__global__ __launch_bounds__(NT) void lightning_outputs_kernel(LightningArgs a) {
  constexpr int DP = 64 * TW, QS = DP + 18;                // 18 mod 32 banks: 16 rows x 2 neighbours meet in no bank
  constexpr int NK = CHUNK * DP / 4 / NT;
  extern __shared__ __align__(16) float lds[];
  float* Qs = lds;                                         // [CHUNK][QS]
  float* Ks = Qs + CHUNK * QS;                             // [CHUNK][QS], then the weighted products [CHUNK][PS]
  const int h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int H = a.H, d = a.d, dv = a.dv;
  int at = blockIdx.x, c0 = -1, len = 0;
  for (int s = 0; s < a.n_seqs; ++s) {                     // the chunks are dealt to the sequences in order
    const int b = a.cu_seqlens[s], n = a.cu_seqlens[s + 1] - b, nc = (n + CHUNK - 1) / CHUNK;
    if (at < nc) {
      c0 = b + at * CHUNK;
      len = min(CHUNK, n - at * CHUNK);
      break;
    }
    at -= nc;
  }
  if (c0 < 0) return;
  const float* pw = a.powers + (size_t)h * (CHUNK + 1);
  const TX* rows = reinterpret_cast<const TX*>(a.rows);
  {
    // a token beyond the chunk's last repeats it: its row and column of the products are never used
    Raw4<TX, V4> rq[NK], rk[NK];
#pragma unroll
    for (int u = 0; u < NK; ++u) {
      const int i = tid + u * NT, j = min(i / (DP / 4), len - 1), k = (i % (DP / 4)) * 4;
      const TX* row = rows + (size_t)(c0 + j) * a.row_w;
      rq[u].load(row + a.q_col + h * d, k, d);
      rk[u].load(row + a.k_col + h * d, k, d);
    }
#pragma unroll
    for (int u = 0; u < NK; ++u) {
      const int i = tid + u * NT, j = i / (DP / 4), k = (i % (DP / 4)) * 4;
      const float4 q = within(activated(a, rq[u].f32()), k, d), x = within(activated(a, rk[u].f32()), k, d);
      float2* qd = reinterpret_cast<float2*>(Qs + j * QS + k);
      float2* kd = reinterpret_cast<float2*>(Ks + j * QS + k);
      qd[0] = float2{q.x, q.y}; qd[1] = float2{q.z, q.w};
      kd[0] = float2{x.x, x.y}; kd[1] = float2{x.z, x.w};
    }
  }
  __syncthreads();
  // q k^T on and below the diagonal: ten tiles of 16 x 16, up to three a wave
  f32x4_t p[3];
#pragma unroll
  for (int n = 0; n < 3; ++n) {
    p[n] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    const int tile = wave + 4 * n;
    if (tile < 10) {
      const int ti = tile < 1 ? 0 : tile < 3 ? 1 : tile < 6 ? 2 : 3, tj = tile - ti * (ti + 1) / 2;
      const float* qa = Qs + (ti * 16 + (lane & 15)) * QS + (lane >> 4);
      const float* kb = Ks + (tj * 16 + (lane & 15)) * QS + (lane >> 4);
      f32x4_t c1 = {0.f, 0.f, 0.f, 0.f}, c2 = c1, c3 = c1;
#pragma unroll 2
      for (int kk = 0; kk < DP; kk += 16) {                // four chains of products that do not wait for each other
        p[n] = __builtin_amdgcn_mfma_f32_16x16x4f32(qa[kk], kb[kk], p[n], 0, 0, 0);
        c1 = __builtin_amdgcn_mfma_f32_16x16x4f32(qa[kk + 4], kb[kk + 4], c1, 0, 0, 0);
        c2 = __builtin_amdgcn_mfma_f32_16x16x4f32(qa[kk + 8], kb[kk + 8], c2, 0, 0, 0);
        c3 = __builtin_amdgcn_mfma_f32_16x16x4f32(qa[kk + 12], kb[kk + 12], c3, 0, 0, 0);
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) p[n][e] += (c1[e] + c2[e]) + c3[e];
    }
  }
  __syncthreads();                                         // the keys have been read: their place takes the weighted products
#pragma unroll
  for (int n = 0; n < 3; ++n) {
    const int tile = wave + 4 * n;
    if (tile < 10) {
      const int ti = tile < 1 ? 0 : tile < 3 ? 1 : tile < 6 ? 2 : 3, tj = tile - ti * (ti + 1) / 2;
      const int r = tj * 16 + (lane & 15);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int j = ti * 16 + (lane >> 4) * 4 + e;
        Ks[j * PS + r] = r <= j ? p[n][e] * pw[j - r] : 0.f;
      }
    }
  }
  __syncthreads();
  const float* S0 = a.states + ((size_t)blockIdx.x * H + h) * d * dv;
  for (int ct0 = wave * CT; ct0 * 16 < dv; ct0 += 4 * CT) {
    f32x4_t acc[CT][4];
    int col[CT];
    bool ok[CT];
#pragma unroll
    for (int c = 0; c < CT; ++c) {
      col[c] = (ct0 + c) * 16 + (lane & 15);
      ok[c] = col[c] < dv;
#pragma unroll
      for (int i = 0; i < 4; ++i) acc[c][i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    }
    // four products' elements of the state, then of the values, are fetched while the four before them are multiplied (an
    // element beyond the head's sizes or the chunk's tokens repeats one within: it meets a zero or is not stored)
    float b[4][CT], bs[4][CT];
    TX bv[4][CT];
    auto fetch_state = [&](int kk) {
#pragma unroll
      for (int n = 0; n < 4; ++n) {
        const float* p = S0 + (size_t)min(kk + n * 4 + (lane >> 4), d - 1) * dv;
#pragma unroll
        for (int c = 0; c < CT; ++c) bs[n][c] = p[min(col[c], dv - 1)];
      }
    };
    auto fetch_values = [&](int kk) {
#pragma unroll
      for (int n = 0; n < 4; ++n) {
        const TX* p = rows + (size_t)(c0 + min(kk + n * 4 + (lane >> 4), len - 1)) * a.row_w + a.v_col + h * dv;
#pragma unroll
        for (int c = 0; c < CT; ++c) bv[n][c] = p[min(col[c], dv - 1)];
      }
    };
    const float* qa = Qs + (lane & 15) * QS + (lane >> 4);
    fetch_state(0);
    for (int kk = 0; kk < DP; kk += 16) {
#pragma unroll
      for (int n = 0; n < 4; ++n)
#pragma unroll
        for (int c = 0; c < CT; ++c) b[n][c] = bs[n][c];
      if (kk + 16 < DP) fetch_state(kk + 16); else fetch_values(0);
#pragma unroll
      for (int n = 0; n < 4; ++n)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float q = qa[i * 16 * QS + kk + n * 4];
#pragma unroll
          for (int c = 0; c < CT; ++c) acc[c][i] = __builtin_amdgcn_mfma_f32_16x16x4f32(q, b[n][c], acc[c][i], 0, 0, 0);
        }
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float w = pw[i * 16 + (lane >> 4) * 4 + e + 1];
#pragma unroll
        for (int c = 0; c < CT; ++c) acc[c][i][e] *= w;
      }
    const float* pa = Ks + (lane & 15) * PS + (lane >> 4);
#pragma unroll
    for (int g = 0; g < 4; ++g) {
#pragma unroll
      for (int n = 0; n < 4; ++n)
#pragma unroll
        for (int c = 0; c < CT; ++c) {
          b[n][c] = load_f32(&bv[n][c], 0);
          if (a.act) b[n][c] = silu_f(b[n][c]);
        }
      if (g < 3) fetch_values(g * 16 + 16);
#pragma unroll
      for (int n = 0; n < 4; ++n) {
        const int kk = g * 16 + n * 4;
#pragma unroll
        for (int i = g; i < 4; ++i) {
          const float q = pa[i * 16 * PS + kk];
#pragma unroll
          for (int c = 0; c < CT; ++c) acc[c][i] = __builtin_amdgcn_mfma_f32_16x16x4f32(q, b[n][c], acc[c][i], 0, 0, 0);
        }
      }
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int j = i * 16 + (lane >> 4) * 4 + e;
#pragma unroll
        for (int c = 0; c < CT; ++c)
          if (ok[c] && j < len) a.out[(size_t)(c0 + j) * H * dv + h * dv + col[c]] = acc[c][i][e];
      }
  }
}

template <typename K>
bool raise_lds(K kernel, size_t bytes, bool* raised) {
  if (bytes <= 48 * 1024 || *raised) return true;
  if (hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024) != hipSuccess) return false;
  *raised = true;                      // once a process and instance
  return true;
}

template <typename TX, int TW, bool V4>
int launch_chunks(const LightningArgs& a, long chunks, hipStream_t stream) {
  constexpr int DP = 64 * TW;
  constexpr size_t lds_s = (size_t)(CHUNK * (DP + 16) + CHUNK * 16) * sizeof(float), lds_o = (size_t)2 * CHUNK * (DP + 18) * sizeof(float);
  static bool rs = false, r1 = false, r2 = false;
  ALICE_CHECK(raise_lds(lightning_states_kernel<TX, TW, V4>, lds_s, &rs), "lightning: %zu bytes of LDS were refused", lds_s);
  lightning_states_kernel<TX, TW, V4><<<dim3(a.n_seqs, a.H, ceil_div(a.dv, 16)), NT, lds_s, stream>>>(a);
  ALICE_LAUNCH_CHECK();
  const dim3 grid((unsigned)chunks, a.H);
  if (a.dv <= 64) {
    ALICE_CHECK(raise_lds(lightning_outputs_kernel<TX, TW, 1, V4>, lds_o, &r1), "lightning: %zu bytes of LDS were refused", lds_o);
    lightning_outputs_kernel<TX, TW, 1, V4><<<grid, NT, lds_o, stream>>>(a);
  } else {
    ALICE_CHECK(raise_lds(lightning_outputs_kernel<TX, TW, 2, V4>, lds_o, &r2), "lightning: %zu bytes of LDS were refused", lds_o);
    lightning_outputs_kernel<TX, TW, 2, V4><<<grid, NT, lds_o, stream>>>(a);
  }
  ALICE_LAUNCH_CHECK();
  return 0;
}

template <typename TX>
int launch(const LightningArgs& a, int chunked, long chunks, hipStream_t stream) {
  if (chunked) {
#define GO(TW) (a.vec4 ? launch_chunks<TX, TW, true>(a, chunks, stream) : launch_chunks<TX, TW, false>(a, chunks, stream))
    if (a.d <= 64) return GO(1);
    if (a.d <= 128) return GO(2);
    return GO(4);
#undef GO
  }
  const int vec = a.dv % 4 == 0 ? 4 : 1;
  const dim3 grid(a.n_seqs, a.H, ceil_div(a.dv, 16 * vec));
#define GO(VEC, RI) lightning_walk_kernel<TX, VEC, RI><<<grid, NT, 0, stream>>>(a)
  if (vec == 4) { if (a.d <= 64) GO(4, 4); else if (a.d <= 128) GO(4, 8); else GO(4, 16); }
  else { if (a.d <= 64) GO(1, 4); else if (a.d <= 128) GO(1, 8); else GO(1, 16); }
#undef GO
  ALICE_LAUNCH_CHECK();
  return 0;
}

}  // namespace

// Chunks that a step of T tokens in n_seqs sequences has at most.
extern "C" long alice_lightning_chunks(int T, int n_seqs) { return (long)T / CHUNK + n_seqs; }

extern "C" int alice_lightning(const void* rows, int rows_dtype, int row_w, int q_col, int k_col, int v_col, int act,
                               const float* powers, float* out, float* states, const int* cu_seqlens, const int* slots, float* S,
                               int T, int n_seqs, int n_slots, int H, int d, int dv, int chunked, hipStream_t stream) {
  ALICE_CHECK(rows && powers && out && cu_seqlens && slots && S && dtype_ok(rows_dtype), "lightning: a pointer is missing or the dtype is unknown");
  ALICE_CHECK(T >= 0 && n_seqs >= 0 && n_slots >= 1 && H >= 1 && H <= 65535 && d >= 1 && dv >= 1, "lightning: bad sizes H=%d d=%d dv=%d", H, d, dv);
  ALICE_CHECK(d <= ALICE_LIGHTNING_MAX_KEY_DIM, "lightning: key size %d is beyond %d, the range of this kernel", d, ALICE_LIGHTNING_MAX_KEY_DIM);
  ALICE_CHECK(q_col >= 0 && k_col >= 0 && v_col >= 0 && q_col + H * d <= row_w && k_col + H * d <= row_w && v_col + H * dv <= row_w,
              "lightning: rows of %d elements are too short for the heads", row_w);
  ALICE_CHECK(ceil_div(dv, 16) <= 65535, "lightning: too many value columns for one launch");
  ALICE_CHECK(!chunked || states, "lightning: the chunks need a workspace");
  if (T == 0 || n_seqs == 0) return 0;
  const int unit = rows_dtype == DT_F32 ? 16 : 8;
  const int vec4 = row_w % 4 == 0 && q_col % 4 == 0 && k_col % 4 == 0 && v_col % 4 == 0 && d % 4 == 0 && dv % 4 == 0 && (uintptr_t)rows % unit == 0;
  LightningArgs a{rows, row_w, q_col, k_col, v_col, act, vec4, powers, out, states, cu_seqlens, slots, S, n_seqs, H, d, dv};
  const long chunks = alice_lightning_chunks(T, n_seqs);
  DISPATCH_DTYPE(rows_dtype, TX, return launch<TX>(a, chunked, chunks, stream));
}
