// A mixture of experts' router and the weighting of the experts' middle activations.
//
// route_kernel: a wave per token.  From the router's logits z [T, E] (32-bit sums of the projection) plus a bias
// it picks the `top` largest (of equal logits the lower index), takes the softmax over the picked logits only, and
// writes a dense row of weights [E]: the picked experts' weights, zero elsewhere.  All in 32-bit.
//
// route_scored_kernel: a router whose scores are a softmax over all its outputs, or a sigmoid of each.  The last outputs may
// be identity experts (they give the token's own input back and have no matrices).  A correction is added to the scores
// for the choice only; the outputs form equal groups of neighbours, and only experts of the groups with the largest choice
// in them (or the largest sum of their two largest choices) can be chosen; the chosen experts' scores, divided by their
// sum and times a constant, are the weights.  A wave per token, all in 32-bit.
//
// scale_columns_kernel: y[t, e F + j] = x[t, e F + j] * w[t, e] for rows made of E parts of F columns: the experts'
// middle activations side by side, each multiplied by its expert's weight of that token (a zero for an expert that
// the token does not use), so that one down projection over all parts gives the weighted sum of the experts.
//
// The grouped products (bfloat16, weights in the matrix cores' fragment layout): the (token, expert) pairs of a step are
// put in the order of their experts and tokens, every expert's run padded to whole tiles of 64 or 128 rows (a block an
// expert: route_count_kernel counts, route_place_kernel places and labels; which row is whose is device data, so a launch
// depends on sizes only).  A block of expert_tile_kernel takes one tile of rows, all of one expert, and 128 of that expert's
// middle columns (gate and up, then act(gate) * up * routing weight, rounded once) or 256 outputs of its slice of the
// side-by-side down matrices: the rows, gathered from the tokens', are staged in LDS two k-tiles at a time and shared by the
// four waves, each of which streams its own weight tiles, a stage ahead.  expert_combine_kernel adds a token's rows.  Only
// the experts that tokens chose are read, and each row meets only its own expert.
//
// Steps of few tokens read every chosen expert's matrices once and do little else (expert_few_*): a block of the first
// kernel takes one expert and 16 of its middle columns, and ends at once if no token of the step chose it; its four waves
// share the inner dimension and meet in LDS.  A block of the second takes 16 outputs and every splits-th of the chosen
// experts, adds each one's products to its sums a token, and leaves partial sums for the residual add.  In both the tokens that
// chose the expert stand side by side as the products' columns, 16 to a set.  The shared expert is one more expert with sizes of its own, chosen by every token,
// and the identity experts' share is added by the first split.  Which experts are chosen is read on the device.
#include "linear_mfma.h"

namespace {

constexpr int MAX_EXPERTS = 1024;

__global__ __launch_bounds__(64) void route_kernel(const float* __restrict__ z, const float* __restrict__ bias, float* __restrict__ w,
                                                   int E, int top) {
  __shared__ float zs[MAX_EXPERTS];
  __shared__ float ws[MAX_EXPERTS];
  const int t = blockIdx.x, lane = threadIdx.x;
  for (int e = lane; e < E; e += 64) {
    zs[e] = z[(size_t)t * E + e] + (bias ? bias[e] : 0.f);
    ws[e] = 0.f;
  }
  __syncthreads();
  float first = 0.f, sum = 0.f;
  for (int n = 0; n < top; ++n) {
    float best = -INFINITY;
    int at = E;
    for (int e = lane; e < E; e += 64)
      if (ws[e] == 0.f && (zs[e] > best || (zs[e] == best && e < at))) { best = zs[e]; at = e; }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ob = __shfl_xor(best, o, 64);
      const int oa = __shfl_xor(at, o, 64);
      if (ob > best || (ob == best && oa < at)) { best = ob; at = oa; }
    }
    if (at >= E) break;                                // (only if every logit is NaN)
    if (n == 0) first = best;
    const float p = expf(best - first);                // the first pick is the largest: exponents are never positive
    sum += p;
    __syncthreads();
    if (lane == 0) ws[at] = p;
    __syncthreads();
  }
  const float inv = sum > 0.f ? 1.f / sum : 0.f;
  for (int e = lane; e < E; e += 64) w[(size_t)t * E + e] = ws[e] * inv;
}

// The largest of the wave's (value, index) pairs, of equal values the lower index; every lane gets it.
__device__ __forceinline__ void wave_argmax(float& best, int& at) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) {
    const float ob = __shfl_xor(best, o, 64);
    const int oa = __shfl_xor(at, o, 64);
    if (ob > best || (ob == best && oa < at)) { best = ob; at = oa; }
  }
}

__global__ __launch_bounds__(64) void route_scored_kernel(const float* __restrict__ z, int z_w, const float* __restrict__ correction,
                                                          float* __restrict__ w, float* __restrict__ side, int E, int n, int top,
                                                          int groups, int keep, int shared_mode, int sigmoid, int group_best,
                                                          float weight_scale) {
  __shared__ float score[MAX_EXPERTS], choice[MAX_EXPERTS], wt[MAX_EXPERTS], best_of[MAX_EXPERTS];
  const int t = blockIdx.x, lane = threadIdx.x;
  const float* zt = z + (size_t)t * z_w;
  float sum = 1.f;
  if (sigmoid) {
    for (int e = lane; e < n; e += 64) score[e] = 1.f / (1.f + expf(-zt[e]));
  } else {
    float m = -INFINITY;
    for (int e = lane; e < n; e += 64) m = fmaxf(m, zt[e]);
    m = wave_max(m);
    sum = 0.f;
    for (int e = lane; e < n; e += 64) {
      const float x = expf(zt[e] - m);
      score[e] = x;
      sum += x;
    }
    sum = wave_sum(sum);
  }
  for (int e = lane; e < n; e += 64) {                 // (a lane reads the scores that it wrote itself)
    const float x = score[e] / sum;
    score[e] = x;
    choice[e] = x + (correction ? correction[e] : 0.f);
    wt[e] = 0.f;
  }
  __syncthreads();
  if (keep < groups) {
    const int gs = n / groups;
    for (int g = lane; g < groups; g += 64) {
      float b = -INFINITY, second = -INFINITY;
      for (int e = g * gs; e < (g + 1) * gs; ++e) {
        const float x = choice[e];
        second = fmaxf(second, fminf(b, x));
        b = fmaxf(b, x);
      }
      best_of[g] = group_best == 2 && gs > 1 ? b + second : b;
    }
    __syncthreads();
    for (int k = 0; k < keep; ++k) {                   // the kept groups are marked by +infinity
      float b = -INFINITY;
      int at = groups;
      for (int g = lane; g < groups; g += 64)
        if (best_of[g] < INFINITY && (at == groups || best_of[g] > b)) { b = best_of[g]; at = g; }
      wave_argmax(b, at);
      __syncthreads();
      if (lane == 0 && at < groups) best_of[at] = INFINITY;
      __syncthreads();
    }
    for (int e = lane; e < n; e += 64)
      if (best_of[e / gs] < INFINITY) choice[e] = -INFINITY;
    __syncthreads();
  }
  float total = 0.f;
  for (int k = 0; k < top; ++k) {
    float b = -INFINITY;
    int at = n;
    for (int e = lane; e < n; e += 64)
      if (choice[e] > b) { b = choice[e]; at = e; }
    wave_argmax(b, at);
    if (at >= n) break;                                // (only if the scores are not numbers)
    total += score[at];
    __syncthreads();
    if (lane == 0) {
      wt[at] = score[at];
      choice[at] = -INFINITY;
    }
    __syncthreads();
  }
  const float inv = weight_scale / (total + 1e-20f);
  float id = 0.f;
  for (int e = lane; e < n; e += 64) {
    const float x = wt[e] * inv;
    if (e < E) w[(size_t)t * E + e] = x;
    else id += x;
  }
  id = wave_sum(id);
  if (lane == 0) {
    side[2 * (size_t)t] = id;
    side[2 * (size_t)t + 1] = shared_mode == 1 ? 1.f / (1.f + expf(-zt[n])) : (shared_mode == 2 ? 1.f : 0.f);
  }
}

template <typename TI, typename TO>
__global__ void scale_columns_kernel(const TI* __restrict__ x, const float* __restrict__ w, TO* __restrict__ y, long n, int E, int F) {
  for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (long)gridDim.x * blockDim.x) {
    const long t = i / ((long)E * F);
    const int e = (int)((i / F) % E);
    store_f32(y, (size_t)i, load_f32(x, (size_t)i) * w[t * E + e]);
  }
}

// ------------------------------------------------------------------------------------------ grouped products

// count[e]: the tokens that use expert e.  w: [T, E] routing weights (zero: not chosen).
__global__ __launch_bounds__(1024) void route_count_kernel(const float* __restrict__ w, int T, int E, int* __restrict__ count) {
  __shared__ int part[16];
  const int e = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  int n = 0;
  for (int t = threadIdx.x; t < T; t += 1024) n += w[(size_t)t * E + e] > 0.f;
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) n += __shfl_xor(n, o, 64);
  if (lane == 0) part[wave] = n;
  __syncthreads();
  if (threadIdx.x == 0) {
    int total = 0;
    for (int i = 0; i < 16; ++i) total += part[i];
    count[e] = total;
  }
}

// A block an expert: its tokens in order into its run of rows.  row_token / row_weight [R] (padding: -1, 0); tile_expert
// [R / tile] (-1: no rows); token_rows [T, top]: where each token's rows went, in the order of the experts (-1: fewer).
__global__ __launch_bounds__(1024) void route_place_kernel(const float* __restrict__ w, const int* __restrict__ count, int T, int E, int top,
                                                           int R, int tile, int* __restrict__ row_token, float* __restrict__ row_weight,
                                                           int* __restrict__ tile_expert, int* __restrict__ token_rows) {
  __shared__ int part[17];
  const int e = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  auto padded = [&](int i) { return (count[i] + tile - 1) / tile * tile; };
  int before = 0;
  for (int i = tid; i < e; i += 1024) before += padded(i);
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) before += __shfl_xor(before, o, 64);
  if (lane == 0) part[wave] = before;
  __syncthreads();
  int off = 0;
  for (int i = 0; i < 16; ++i) off += part[i];
  const int mine = count[e], run = padded(e);
  for (int i = tid; i < run / tile; i += 1024) tile_expert[off / tile + i] = e;
  if (e == E - 1)
    for (int i = (off + run) / tile + tid; i < R / tile; i += 1024) tile_expert[i] = -1;
  for (int i = mine + tid; i < run; i += 1024) {
    row_token[off + i] = -1;
    row_weight[off + i] = 0.f;
  }
  int base = off;
  for (int t0 = 0; t0 < T; t0 += 1024) {
    const int t = t0 + tid;
    const float x = t < T ? w[(size_t)t * E + e] : 0.f;
    const unsigned long long m = __ballot(x > 0.f);
    __syncthreads();                                   // the last round's counts have been read
    if (lane == 0) part[wave] = __popcll(m);
    __syncthreads();
    int at = base, all = 0;
    for (int i = 0; i < 16; ++i) {
      const int n = part[i];
      at += i < wave ? n : 0;
      all += n;
    }
    base += all;
    if (t < T) {
      int slot = 0;                                    // how many of the token's experts come before this one
      if (x > 0.f || e == E - 1)
        for (int i = 0; i < e; ++i) slot += w[(size_t)t * E + i] > 0.f;
      if (x > 0.f) {
        const int r = at + __popcll(m & ((1ull << lane) - 1ull));
        row_token[r] = t;
        row_weight[r] = x;
        if (slot < top) token_rows[(size_t)t * top + slot] = r;
        ++slot;
      }
      if (e == E - 1)
        for (; slot < top; ++slot) token_rows[(size_t)t * top + slot] = -1;
    }
  }
}

struct GroupArgs {
  const bf16_t* x;                     // DOWN false: the tokens' rows [T, K]; true: the middle rows [R, K]
  const bf16_t* wf;                    // fragment layout of [all gates; all ups] ([2 E F, W]) or of the down matrices ([W, E F])
  const int* row_token; const float* row_weight; const int* tile_expert;
  bf16_t* mid;                         // [R, F]
  float* out;                          // [R, W]
  int K, W, F, E, gx, gy;
  float epi;
};

// One tile of 16 TM rows against 4 weight tiles of 16 a wave (gate, up, gate, up; or four of the down matrices).
template <bool DOWN, int TM>
__global__ __launch_bounds__(256, 2) void expert_tile_kernel(GroupArgs a) {
  constexpr int WN = 4, KC = 2, XJ = TM / 4;
  __shared__ __align__(16) u32x4 xs[2][KC][TM][64];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, g = lane >> 4, c = lane & 15;
  // blocks that share weight tiles (neighbouring row tiles of one expert) run on the same XCD
  const int id = blockIdx.x, per = (a.gx * a.gy + 7) >> 3, item = (id & 7) * per + (id >> 3);
  if ((id >> 3) >= per || item >= a.gx * a.gy) return;
  const int bx = item / a.gy, by = item % a.gy, e = a.tile_expert[by], r0 = by * 16 * TM;
  if (e < 0) return;
  const int KT = (a.K + 31) / 32;                          // (DOWN: F is a multiple of 32, an expert's k-tiles are its own)
  const bf16_t* wsrc[WN];
  int col[WN];                                             // the first column of the wave's tile i; the matrix's width or more: none
#pragma unroll
  for (int i = 0; i < WN; ++i) {
    if (DOWN) {
      const int n = (bx * 4 + wave) * WN + i, n_tiles = (a.W + 15) / 16;
      col[i] = n * 16;
      wsrc[i] = a.wf + ((size_t)min(n, n_tiles - 1) * ((size_t)a.E * a.F / 32) + (size_t)e * a.F / 32) * 512 + lane * 8;
    } else {
      const int p = (bx * 4 + wave) * (WN / 2) + (i >> 1), f = min(p, a.F / 16 - 1);
      col[i] = p * 16;
      wsrc[i] = a.wf + (((i & 1) ? (size_t)a.E * a.F / 16 : 0) + (size_t)e * a.F / 16 + f) * KT * 512 + lane * 8;
    }
  }
  const bf16_t* xsrc[XJ];
#pragma unroll
  for (int j = 0; j < XJ; ++j) {
    const int r = r0 + (XJ * wave + j) * 16 + c;
    xsrc[j] = a.x + (size_t)(DOWN ? r : max(a.row_token[r], 0)) * a.K;       // (a padded row reads token 0's; its weight is 0)
  }
  f32x4 acc[WN][TM];
#pragma unroll
  for (int i = 0; i < WN; ++i)
#pragma unroll
    for (int j = 0; j < TM; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  const bf16_t* zero = reinterpret_cast<const bf16_t*>(g_zero_tile) + lane * 8;
  u32x4 xr[KC][XJ], wk[KC][WN];
  auto stage_load = [&](int s) {                           // beyond the last k-tile the weights are zeros
#pragma unroll
    for (int kc = 0; kc < KC; ++kc)
#pragma unroll
      for (int j = 0; j < XJ; ++j) xr[kc][j] = *reinterpret_cast<const u32x4*>(xsrc[j] + min((s * KC + kc) * 32 + g * 8, a.K - 8));
  };
  auto stage_store = [&](int buf) {
#pragma unroll
    for (int kc = 0; kc < KC; ++kc)
#pragma unroll
      for (int j = 0; j < XJ; ++j) xs[buf][kc][XJ * wave + j][lane] = xr[kc][j];
  };
  const int S = (KT + KC - 1) / KC;
  stage_load(0);
  stage_store(0);
#pragma unroll
  for (int kc = 0; kc < KC; ++kc)
#pragma unroll
    for (int i = 0; i < WN; ++i) wk[kc][i] = *reinterpret_cast<const u32x4*>(kc < KT ? wsrc[i] + (size_t)kc * 512 : zero);
  auto stage_mfma = [&](int s, bool more) {
#pragma unroll
    for (int kc = 0; kc < KC; ++kc) {
      u32x4 xf[TM];
#pragma unroll
      for (int j = 0; j < TM; ++j) xf[j] = xs[s & 1][kc][j][lane];
      const int next = (s + 1) * KC + kc;
#pragma unroll
      for (int i = 0; i < WN; ++i) {
#pragma unroll
        for (int j = 0; j < TM; ++j) acc[i][j] = mfma16(wk[kc][i], xf[j], acc[i][j]);
        if (more) {                                        // this tile's registers are free: the same tile of the next stage
          __builtin_amdgcn_sched_barrier(0);
          wk[kc][i] = *reinterpret_cast<const u32x4*>(next < KT ? wsrc[i] + (size_t)next * 512 : zero);
          __builtin_amdgcn_sched_barrier(0);
        }
      }
    }
  };
  for (int s = 0; s + 1 < S; ++s) {
    stage_load(s + 1);
    __builtin_amdgcn_sched_barrier(0);
    __syncthreads();
    stage_mfma(s, true);
    stage_store((s + 1) & 1);
  }
  __syncthreads();
  stage_mfma(S - 1, false);
#pragma unroll
  for (int j = 0; j < TM; ++j) {
    const int r = r0 + j * 16 + c;
    if (DOWN) {
#pragma unroll
      for (int i = 0; i < WN; ++i)
        if (col[i] < a.W) store4(a.out, (size_t)r * a.W, col[i] + g * 4, a.W, acc[i][j]);
    } else {
      const float wr = a.row_weight[r];
#pragma unroll
      for (int p = 0; p < WN / 2; ++p) {
        if (col[2 * p] >= a.F) continue;
        f32x4 o;
#pragma unroll
        for (int i = 0; i < 4; ++i) o[i] = wr == 0.f ? 0.f : gated_act(acc[2 * p][j][i], acc[2 * p + 1][j][i], a.epi, false) * wr;
        store4(a.mid, (size_t)r * a.F, col[2 * p] + g * 4, a.F, o);
      }
    }
  }
}

// Rows of a tile: 128 where the experts' runs are long enough on average, else 64.
int group_tile(int T, int E, int top) { return (long)T * top >= 96L * E ? 128 : 64; }

template <int TM>
int launch_group(GroupArgs a, const void* gate_up, const void* down, const void* x, int R, hipStream_t stream) {
  const int W = a.W, F = a.F;
  a.gy = R / (16 * TM);
  a.x = (const bf16_t*)x;
  a.wf = (const bf16_t*)gate_up;
  a.K = W;
  a.gx = ceil_div(F, 128);
  expert_tile_kernel<false, TM><<<8 * ceil_div((long)a.gx * a.gy, 8), 256, 0, stream>>>(a);
  ALICE_LAUNCH_CHECK();
  a.x = a.mid;
  a.wf = (const bf16_t*)down;
  a.K = F;
  a.gx = ceil_div(W, 256);
  expert_tile_kernel<true, TM><<<8 * ceil_div((long)a.gx * a.gy, 8), 256, 0, stream>>>(a);
  ALICE_LAUNCH_CHECK();
  return 0;
}

// ------------------------------------------------------------------------------------------ few tokens

struct FewArgs {
  const bf16_t* x;                     // [T, W]
  const float* w;                      // [T, E], zero: not chosen
  const float* side;                   // [T, 2] or null: (identity weight, the shared expert's gate)
  const bf16_t* gate_up;               // fragment layout of [2 E F, W]
  const bf16_t* down;                  // fragment layout of [W, E F]
  const bf16_t* shared_gate_up;        // fragment layout of [2 Fs, W], or null
  const bf16_t* shared_down;           // fragment layout of [W, Fs]
  bf16_t* mid;                         // [T, E F + Fs]
  float* out;                          // [splits, T, W]
  int T, W, F, E, Fs, splits;
  float epi, shared_epi;
};

// The weight with which token t uses expert e (e == E: the shared one).
__device__ __forceinline__ float few_weight(const FewArgs& a, int t, int e) {
  if (t >= a.T) return 0.f;
  return e < a.E ? a.w[(size_t)t * a.E + e] : a.side[2 * (size_t)t + 1];
}

// RS: tokens a step in sets of 16.  The tokens that use the expert stand side by side as the products' columns, whichever
// they are, so most blocks need one set.
template <int RS>
__global__ __launch_bounds__(256) void expert_few_gate_up_kernel(FewArgs a) {
  __shared__ f32x4 part[4][2][64];
  const int e = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, g = lane >> 4, c = lane & 15;
  const bool shared = e == a.E;
  const int F = shared ? a.Fs : a.F, f0 = blockIdx.x * 16;
  if (f0 >= F) return;
  const float wt = few_weight(a, lane, e);                // lane = token (at most 64)
  const unsigned long long used = __ballot(wt != 0.f);
  if (used == 0ull) return;
  const int n_used = __popcll(used), sets = RS == 1 ? 1 : (n_used + 15) >> 4;
  const unsigned long long below = (1ull << lane) - 1ull;
  // lane i: the i-th token that uses the expert, then the others
  const int token_at = __builtin_amdgcn_ds_permute((wt != 0.f ? __popcll(used & below) : n_used + __popcll(~used & below)) * 4, lane);
  const int KT = (a.W + 31) / 32;
  const bf16_t* base = shared ? a.shared_gate_up : a.gate_up;
  const int first = shared ? f0 : e * F + f0, half = shared ? F : a.E * F;
  const bf16_t* wg = base + (size_t)(first / 16) * KT * 512 + lane * 8;
  const bf16_t* wu = base + (size_t)((half + first) / 16) * KT * 512 + lane * 8;
  int token[RS];
  f32x4 ag[RS], au[RS];
#pragma unroll
  for (int s = 0; s < RS; ++s) {
    token[s] = __shfl(token_at, s * 16 + c, 64);
    ag[s] = au[s] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  // A burst of N k-tiles: the first set's rows (from the L2) and the weight tiles are all on their way before the first product.
  auto burst = [&](auto count, int kt0) {
    constexpr int N = decltype(count)::value;
    u32x4 vg[N], vu[N], b[N];
    auto rows = [&](int s) {
      const bf16_t* xr = a.x + (size_t)min(token[s], a.T - 1) * a.W;
#pragma unroll
      for (int u = 0; u < N; ++u) b[u] = u32x4{0u, 0u, 0u, 0u};
      if (s * 16 + c < n_used) {                           // (no row is read for a column without a token)
#pragma unroll
        for (int u = 0; u < N; ++u)                        // a row's last, partial k-tile: the weights are zero there
          b[u] = *reinterpret_cast<const u32x4*>(xr + min((kt0 + 4 * u) * 32 + g * 8, a.W - 8));
      }
    };
    rows(0);
#pragma unroll
    for (int u = 0; u < N; ++u) {
      vg[u] = *reinterpret_cast<const u32x4*>(wg + (size_t)(kt0 + 4 * u) * 512);
      vu[u] = *reinterpret_cast<const u32x4*>(wu + (size_t)(kt0 + 4 * u) * 512);
    }
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int s = 0; s < RS; ++s) {
      if (s >= sets) break;                                // (the same for the whole block)
      if (s > 0) rows(s);
#pragma unroll
      for (int u = 0; u < N; ++u) {
        ag[s] = mfma16(vg[u], b[u], ag[s]);
        au[s] = mfma16(vu[u], b[u], au[s]);
      }
    }
  };
  constexpr int U = 8;                                    // weight tiles in flight: 2 U loads of 1 KB a wave
  int kt = wave;
  for (; kt + 4 * (U - 1) < KT; kt += 4 * U) burst(std::integral_constant<int, U>{}, kt);
  if (kt + 4 * 3 < KT) { burst(std::integral_constant<int, 4>{}, kt); kt += 16; }
  if (kt + 4 < KT) { burst(std::integral_constant<int, 2>{}, kt); kt += 8; }
  if (kt < KT) burst(std::integral_constant<int, 1>{}, kt);
#pragma unroll
  for (int s = 0; s < RS; ++s) {
    if (s >= sets) break;
    if (s > 0) __syncthreads();                           // the last set's parts have been read
    part[wave][0][lane] = ag[s];
    part[wave][1][lane] = au[s];
    __syncthreads();
    if (wave != s % 4) continue;
    const float wr = __shfl(wt, token[s], 64);
    f32x4 gs = part[0][0][lane], us = part[0][1][lane];
#pragma unroll
    for (int n = 1; n < 4; ++n) {
      gs += part[n][0][lane];
      us += part[n][1][lane];
    }
    f32x4 o;
#pragma unroll
    for (int i = 0; i < 4; ++i) o[i] = gated_act(gs[i], us[i], shared ? a.shared_epi : a.epi, false) * wr;
    if (wr != 0.f) store4(a.mid, (size_t)token[s] * (a.E * a.F + a.Fs), e * a.F + f0 + g * 4, e * a.F + F, o);
  }
}

// 16 outputs of every splits-th chosen expert: again the expert's tokens side by side; a wave adds each expert's products to
// its own sums a token in LDS, and the four waves' sums meet at the end.
template <int RS>
__global__ __launch_bounds__(256) void expert_few_down_kernel(FewArgs a) {
  __shared__ unsigned short list[MAX_EXPERTS + 1];
  __shared__ unsigned long long users[MAX_EXPERTS + 1];
  __shared__ int n_list;
  __shared__ f32x4 sums[4][16 * RS][4];                   // [wave][token][four of the 16 outputs]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g = lane >> 4, c = lane & 15;
  const int n0 = blockIdx.x * 16, z = blockIdx.y, n_exp = a.E + (a.Fs > 0 ? 1 : 0), row = a.E * a.F + a.Fs;
  if (wave == 0) {                                        // the chosen experts in their order
    int n = 0;
    for (int e0 = 0; e0 < n_exp; e0 += 64) {
      const int e = e0 + lane;
      const float* col = e < a.E ? a.w + e : a.side + 1;
      const int stride = e < a.E ? a.E : 2;
      unsigned long long who = 0ull;                      // bit t: token t uses the expert
      if (e < n_exp)
        for (int t0 = 0; t0 < a.T; t0 += 8) {             // eight loads on their way at a time
          float v[8];
#pragma unroll
          for (int j = 0; j < 8; ++j) v[j] = col[(size_t)min(t0 + j, a.T - 1) * stride];
#pragma unroll
          for (int j = 0; j < 8; ++j)
            if (t0 + j < a.T && v[j] != 0.f) who |= 1ull << (t0 + j);
        }
      const unsigned long long m = __ballot(who != 0ull);
      if (who) {
        const int at = n + __popcll(m & ((1ull << lane) - 1ull));
        list[at] = (unsigned short)e;
        users[at] = who;
      }
      n += __popcll(m);
    }
    if (lane == 0) n_list = n;
  }
#pragma unroll
  for (int s = 0; s < RS; ++s) sums[wave][s * 16 + (lane >> 2)][lane & 3] = f32x4{0.f, 0.f, 0.f, 0.f};
  __syncthreads();
  const int KT = (a.E * a.F + 31) / 32, KTS = (a.Fs + 31) / 32;
  const unsigned long long below = (1ull << lane) - 1ull;
  for (int i = z; i < n_list; i += a.splits) {
    const int e = list[i];
    const unsigned long long who = users[i];
    const bool shared = e == a.E, mine = (who >> lane) & 1ull;
    const int n_used = __popcll(who), sets = RS == 1 ? 1 : (n_used + 15) >> 4;
    const int kts = (shared ? a.Fs : a.F) / 32;           // F and Fs are multiples of 32: an expert's k-tiles are its own
    const bf16_t* wd = (shared ? a.shared_down + (size_t)(n0 / 16) * KTS * 512 : a.down + ((size_t)(n0 / 16) * KT + e * a.F / 32) * 512) + lane * 8;
    const int token_at = __builtin_amdgcn_ds_permute((mine ? __popcll(who & below) : n_used + __popcll(~who & below)) * 4, lane);
    int token[RS];
    f32x4 acc[RS];
#pragma unroll
    for (int s = 0; s < RS; ++s) {
      token[s] = __shfl(token_at, s * 16 + c, 64);
      acc[s] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    auto burst = [&](auto count, int kt0) {               // as above
      constexpr int N = decltype(count)::value;
      u32x4 v[N], b[N];
      auto rows = [&](int s) {
        const bf16_t* mr = a.mid + (size_t)min(token[s], a.T - 1) * row + e * a.F + g * 8;
#pragma unroll
        for (int u = 0; u < N; ++u) b[u] = u32x4{0u, 0u, 0u, 0u};
        if (s * 16 + c < n_used) {
#pragma unroll
          for (int u = 0; u < N; ++u) b[u] = *reinterpret_cast<const u32x4*>(mr + (kt0 + 4 * u) * 32);
        }
      };
      rows(0);
#pragma unroll
      for (int u = 0; u < N; ++u) v[u] = *reinterpret_cast<const u32x4*>(wd + (size_t)(kt0 + 4 * u) * 512);
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int s = 0; s < RS; ++s) {
        if (s >= sets) break;                              // (the same for the whole block)
        if (s > 0) rows(s);
#pragma unroll
        for (int u = 0; u < N; ++u) acc[s] = mfma16(v[u], b[u], acc[s]);
      }
    };
    constexpr int U = 8;
    int kt = wave;
    for (; kt + 4 * (U - 1) < kts; kt += 4 * U) burst(std::integral_constant<int, U>{}, kt);
    if (kt + 4 * 3 < kts) { burst(std::integral_constant<int, 4>{}, kt); kt += 16; }
    if (kt + 4 < kts) { burst(std::integral_constant<int, 2>{}, kt); kt += 8; }
    if (kt < kts) burst(std::integral_constant<int, 1>{}, kt);
#pragma unroll
    for (int s = 0; s < RS; ++s)
      if (s * 16 + c < n_used) sums[wave][token[s]][g] += acc[s];      // (n_used <= T <= 16 RS: no set is left out)
  }
  __syncthreads();
  for (int j = tid; j < a.T * 4; j += 256) {
    const int t = j >> 2, q = j & 3, n = n0 + q * 4;
    f32x4 o = (sums[0][t][q] + sums[1][t][q]) + (sums[2][t][q] + sums[3][t][q]);
    if (z == 0 && a.side) {
      const float id = a.side[2 * (size_t)t];
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (n + i < a.W) o[i] = fmaf(id, bf16_to_f32(a.x[(size_t)t * a.W + n + i]), o[i]);
    }
    store4(a.out + (size_t)z * a.T * a.W, (size_t)t * a.W, n, a.W, o);
  }
}

// y[t, c] = the sum of the token's rows of `rows` [R, W], or of the n_base partial rows base[s][t]; with `side` also
// side[t][0] x[t, c] (the identity experts give the input back) + side[t][1] * (the sum of the shared expert's partial rows).
template <typename TX, int V>
__global__ void expert_combine_kernel(const float* __restrict__ rows, const int* __restrict__ token_rows, int top,
                                      const float* __restrict__ base, int n_base, const TX* __restrict__ x, const float* __restrict__ side,
                                      const float* __restrict__ shared, int n_shared, float* __restrict__ y, int T, int W) {
  const int t = blockIdx.x, c = (blockIdx.y * blockDim.x + threadIdx.x) * V;       // V neighbouring columns a thread (W a multiple of V)
  if (c >= W) return;
  const size_t at = (size_t)t * W + c, all = (size_t)T * W;
  float s[V], u[V];
#pragma unroll
  for (int i = 0; i < V; ++i) s[i] = u[i] = 0.f;
  auto add = [&](float (&d)[V], const float* p) {
    if constexpr (V == 4) {
      const float4 v = *reinterpret_cast<const float4*>(p);
      d[0] += v.x; d[1] += v.y; d[2] += v.z; d[3] += v.w;
    } else {
      d[0] += p[0];
    }
  };
  if (rows) {
    for (int j = 0; j < top; ++j) {
      const int r = token_rows[(size_t)t * top + j];
      if (r >= 0) add(s, rows + (size_t)r * W + c);
    }
  }
  for (int i = 0; i < n_base; ++i) add(s, base + i * all + at);
  if (side) {
    const float id = side[2 * (size_t)t], sg = side[2 * (size_t)t + 1];
    for (int i = 0; i < n_shared; ++i) add(u, shared + i * all + at);
#pragma unroll
    for (int i = 0; i < V; ++i) s[i] = fmaf(sg, u[i], fmaf(id, load_f32(x, at + i), s[i]));
  }
  if constexpr (V == 4) *reinterpret_cast<float4*>(y + at) = float4{s[0], s[1], s[2], s[3]};
  else y[at] = s[0];
}

// Four columns a thread where rows are whole 16-byte units.
template <typename TX>
void launch_combine(const float* rows, const int* token_rows, int top, const float* base, int n_base, const TX* x, const float* side,
                    const float* shared, int n_shared, float* y, int T, int W, hipStream_t stream) {
  if (W % 4 == 0 && (((uintptr_t)rows | (uintptr_t)base | (uintptr_t)shared | (uintptr_t)y) & 15) == 0)
    expert_combine_kernel<TX, 4><<<dim3(T, ceil_div(W, 1024)), 256, 0, stream>>>(rows, token_rows, top, base, n_base, x, side, shared, n_shared, y, T, W);
  else
    expert_combine_kernel<TX, 1><<<dim3(T, ceil_div(W, 256)), 256, 0, stream>>>(rows, token_rows, top, base, n_base, x, side, shared, n_shared, y, T, W);
}

}  // namespace

// Rows that the grouped products of a step of T tokens need: every pair and every expert's padding, in whole tiles.
extern "C" long alice_expert_rows(int T, int E, int top) {
  const int tile = group_tile(T, E, top);
  return ((long)T * top + (long)E * (tile - 1) + tile - 1) / tile * tile;
}

// The routed feed-forward by grouped products, see the top of the file.  x: [T, W] bfloat16; weights: [T, E] float32 of
// alice_route_topk; gate_up, down: fragment layouts of [2 E F, W] and [W, E F]; y: [T, W] float32.  Workspaces for
// side, shared: null, or what alice_expert_combine adds (the identity experts' weight and the shared expert's gate a token,
// the shared expert's partial rows).  R = alice_expert_rows(T, E, top): ints [2 R + R / 64 + T top + E] (row_token, tile_expert, token_rows, the experts' counts; the row
// weights share the ints' buffer as floats), mid [R, F] bfloat16, rows [R, W] float32.
extern "C" int alice_expert_products(const void* x, const float* weights, const void* gate_up, const void* down, float* y, int* ints,
                                     void* mid, float* rows, int T, int W, int F, int E, int top, float epi, const float* side,
                                     const float* shared, int n_shared, hipStream_t stream) {
  ALICE_CHECK(n_shared == 0 || (side && shared), "expert_products: a shared expert needs its rows and its gate");
  ALICE_CHECK(x && weights && gate_up && down && y && ints && mid && rows, "expert_products: a pointer is missing");
  ALICE_CHECK(T >= 1 && E >= 1 && E <= MAX_EXPERTS && top >= 1 && top <= E, "expert_products: 1 <= top <= experts <= %d", MAX_EXPERTS);
  ALICE_CHECK(W >= 8 && W % 8 == 0 && F >= 32 && F % 32 == 0, "expert_products: the width must be a multiple of 8 and the experts' a multiple of 32");
  const long R = alice_expert_rows(T, E, top);
  const int tile = group_tile(T, E, top);
  ALICE_CHECK(R < (1L << 30) && (long)T * E < (1L << 40) && R / tile * (long)ceil_div(F > W ? F : W, 128) < (1L << 28), "expert_products: too many rows for one launch");
  int* row_token = ints;
  float* row_weight = reinterpret_cast<float*>(ints + R);
  int* tile_expert = ints + 2 * R;
  int* token_rows = tile_expert + R / tile;
  int* count = token_rows + (long)T * top;
  route_count_kernel<<<E, 1024, 0, stream>>>(weights, T, E, count);
  ALICE_LAUNCH_CHECK();
  route_place_kernel<<<E, 1024, 0, stream>>>(weights, count, T, E, top, (int)R, tile, row_token, row_weight, tile_expert, token_rows);
  ALICE_LAUNCH_CHECK();
  GroupArgs a{};
  a.row_token = row_token;
  a.row_weight = row_weight;
  a.tile_expert = tile_expert;
  a.mid = (bf16_t*)mid;
  a.out = rows;
  a.W = W;
  a.F = F;
  a.E = E;
  a.epi = epi;
  if (const int rc = tile == 128 ? launch_group<8>(a, gate_up, down, x, (int)R, stream) : launch_group<4>(a, gate_up, down, x, (int)R, stream)) return rc;
  launch_combine<bf16_t>(rows, token_rows, top, nullptr, 0, (const bf16_t*)x, side, shared, n_shared, y, T, W, stream);
  ALICE_LAUNCH_CHECK();
  return 0;
}

// How many partial sums alice_expert_few leaves: enough blocks for the chip.
extern "C" int alice_expert_few_splits(int W) {
  const int s = 512 / ceil_div(W, 16);
  return s < 1 ? 1 : (s > 8 ? 8 : s);
}

// The routed feed-forward for at most 64 tokens, see expert_few_*_kernel.  x: [T, W] bfloat16; w: [T, E]; gate_up, down,
// shared_gate_up, shared_down: fragment layouts (the latter two null and shared_width 0 without a shared expert); side
// [T, 2] or null; mid: [T, E F + shared_width] bfloat16; out: [alice_expert_few_splits(W), T, W] float32 partial sums.
extern "C" int alice_expert_few(const void* x, const float* w, const float* side, const void* gate_up, const void* down,
                                const void* shared_gate_up, const void* shared_down, void* mid, float* out, int T, int W, int F, int E,
                                int shared_width, float epi, float shared_epi, hipStream_t stream) {
  ALICE_CHECK(x && w && gate_up && down && mid && out, "expert_few: a pointer is missing");
  ALICE_CHECK(T >= 1 && T <= 64 && E >= 1 && E <= MAX_EXPERTS, "expert_few: %d tokens (1..64) or %d experts (1..%d)", T, E, MAX_EXPERTS);
  ALICE_CHECK(W >= 8 && W % 8 == 0 && F >= 32 && F % 32 == 0 && shared_width >= 0 && shared_width % 32 == 0,
              "expert_few: the width must be a multiple of 8 and the experts' of 32");
  ALICE_CHECK(shared_width == 0 || (side && shared_gate_up && shared_down), "expert_few: a shared expert needs its matrices and its gate");
  FewArgs a{(const bf16_t*)x, w, side, (const bf16_t*)gate_up, (const bf16_t*)down, (const bf16_t*)shared_gate_up, (const bf16_t*)shared_down,
            (bf16_t*)mid, out, T, W, F, E, shared_width, alice_expert_few_splits(W), epi, shared_epi};
  const dim3 g1(ceil_div(F > shared_width ? F : shared_width, 16), E + (shared_width > 0 ? 1 : 0)), g2(ceil_div(W, 16), a.splits);
#define GO(RS)                                                      \
  do {                                                              \
    expert_few_gate_up_kernel<RS><<<g1, 256, 0, stream>>>(a);       \
    ALICE_LAUNCH_CHECK();                                           \
    expert_few_down_kernel<RS><<<g2, 256, 0, stream>>>(a);          \
  } while (0)
  if (T <= 16) GO(1);
  else if (T <= 32) GO(2);
  else GO(4);
#undef GO
  ALICE_LAUNCH_CHECK();
  return 0;
}

extern "C" int alice_route_topk(const float* z, const float* bias, float* w, int T, int E, int top, hipStream_t stream) {
  ALICE_CHECK(z && w, "route_topk: a pointer is missing");
  ALICE_CHECK(T >= 0 && E >= 1 && E <= MAX_EXPERTS && top >= 1 && top <= E, "route_topk: 1 <= top <= experts <= %d", MAX_EXPERTS);
  if (T == 0) return 0;
  route_kernel<<<T, 64, 0, stream>>>(z, bias, w, E, top);
  ALICE_LAUNCH_CHECK();
  return 0;
}

extern "C" int alice_route_scored(const float* z, int z_w, const float* correction, float* w, float* side, int T, int experts,
                                  int identity, int top, int groups, int keep, int shared_mode, int sigmoid, int group_best,
                                  float weight_scale, hipStream_t stream) {
  ALICE_CHECK(z && w && side, "route_scored: a pointer is missing");
  const int n = experts + identity;
  ALICE_CHECK(T >= 0 && experts >= 1 && identity >= 0 && n <= MAX_EXPERTS && top >= 1 && top <= n, "route_scored: 1 <= top <= outputs <= %d", MAX_EXPERTS);
  ALICE_CHECK(groups >= 1 && n % groups == 0 && keep >= 1 && keep <= groups && (long)keep * (n / groups) >= top,
              "route_scored: %d groups must divide %d outputs, and the kept ones hold at least `top` of them", groups, n);
  ALICE_CHECK(shared_mode >= 0 && shared_mode <= 2 && (group_best == 1 || group_best == 2), "route_scored: unknown shared_mode %d or group_best %d", shared_mode, group_best);
  ALICE_CHECK(z_w >= n + (shared_mode == 1 ? 1 : 0), "route_scored: rows of %d logits are too short", z_w);
  if (T == 0) return 0;
  route_scored_kernel<<<T, 64, 0, stream>>>(z, z_w, correction, w, side, experts, n, top, groups, keep, shared_mode, sigmoid, group_best, weight_scale);
  ALICE_LAUNCH_CHECK();
  return 0;
}

extern "C" int alice_expert_combine(const float* base, int n_base, const void* x, int x_dtype, const float* side, const float* shared,
                                    int n_shared, float* y, int T, int W, hipStream_t stream) {
  ALICE_CHECK(base && n_base >= 1 && x && side && y && dtype_ok(x_dtype), "expert_combine: a pointer is missing or the dtype is unknown");
  ALICE_CHECK(T >= 0 && W >= 1 && n_shared >= 0 && (n_shared == 0 || shared), "expert_combine: bad sizes");
  if (T == 0) return 0;
  DISPATCH_DTYPE(x_dtype, TX, (launch_combine<TX>(nullptr, nullptr, 0, base, n_base, (const TX*)x, side, shared, n_shared, y, T, W, stream)));
  ALICE_LAUNCH_CHECK();
  return 0;
}

extern "C" int alice_scale_columns(const void* x, int x_dtype, const float* w, void* y, int y_dtype, int T, int E, int F,
                                   hipStream_t stream) {
  ALICE_CHECK(x && w && y && dtype_ok(x_dtype) && dtype_ok(y_dtype), "scale_columns: a pointer is missing or a dtype is unknown");
  ALICE_CHECK(T >= 0 && E >= 1 && F >= 1, "scale_columns: bad sizes");
  const long n = (long)T * E * F;
  if (n == 0) return 0;
  const int blocks = (int)((n + 255) / 256 < (1L << 20) ? (n + 255) / 256 : (1L << 20));      // beyond that a thread takes several elements
#define GO(TI, TO) scale_columns_kernel<TI, TO><<<blocks, 256, 0, stream>>>((const TI*)x, w, (TO*)y, n, E, F)
  if (x_dtype == DT_F32 && y_dtype == DT_F32) GO(float, float);
  else if (x_dtype == DT_F32) GO(float, bf16_t);
  else if (y_dtype == DT_F32) GO(bf16_t, float);
  else GO(bf16_t, bf16_t);
#undef GO
  ALICE_LAUNCH_CHECK();
  return 0;
}
