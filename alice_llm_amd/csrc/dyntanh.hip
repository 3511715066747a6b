// The residual add with norms that act element by element (dynamic tanh: tanh(a v) * w + b, no mean and no variance):
//   b   = the sum of `n_partials` slices of `branch`
//   b   = w_post ? tanh(a_post b) * w_post + b_post : b
//   x   = resid + b, written back to resid                       (only when branch is given)
//   out = w_pre ? tanh(a_pre x) * w_pre + b_pre : x              (only when out is given)
// all in 32-bit.  Nothing is summed over a row, so any thread may take any element: a thread takes V neighbouring
// columns (whose weights it reads once) of R rows, with every row's loads issued before the first use; there is no barrier
// and no block-wide sum, and rows of any width spread over as many blocks as the chip wants.
#include "common.h"
#include "alice_hip.h"

namespace {

struct DynTanhArgs {
  float* resid;
  const float* branch;
  int n_partials;
  size_t partial_stride;
  const float *w_post, *b_post, *w_pre, *b_pre;
  float a_post, a_pre;
  void* out;
  const int* rows;
  int T, H, out_layout;
};

template <int V> __device__ __forceinline__ void load_v(float (&d)[V], const float* p) {
  if constexpr (V == 4) {
    const float4 v = *reinterpret_cast<const float4*>(p);
    d[0] = v.x; d[1] = v.y; d[2] = v.z; d[3] = v.w;
  } else {
    d[0] = p[0];
  }
}

template <typename TO, bool FULL, int V, int R>
__global__ __launch_bounds__(256) void add_dyntanh_kernel(DynTanhArgs a) {
  const int c = (blockIdx.y * blockDim.x + threadIdx.x) * V, r0 = blockIdx.x * R;
  if (c >= a.H) return;
  float x[R][V], b[R][V], wp[V], bp[V], wq[V], bq[V];
  size_t at[R];
#pragma unroll
  for (int j = 0; j < R; ++j) {
    const int r = min(r0 + j, a.T - 1);
    at[j] = (size_t)(a.rows ? a.rows[r] : r) * a.H + c;
    load_v<V>(x[j], a.resid + at[j]);
  }
  if (a.branch) {
#pragma unroll
    for (int j = 0; j < R; ++j) load_v<V>(b[j], a.branch + at[j]);
  }
  if (a.w_post) {
    load_v<V>(wp, a.w_post + c);
    load_v<V>(bp, a.b_post + c);
  }
  if (a.w_pre) {
    load_v<V>(wq, a.w_pre + c);
    load_v<V>(bq, a.b_pre + c);
  }
  if (a.branch) {
    constexpr int CH = R == 1 ? 4 : 1;                       // partial sums in flight, added in their order
    for (int p0 = 1; p0 < a.n_partials; p0 += CH) {
      float t[CH][R][V];
#pragma unroll
      for (int p = 0; p < CH; ++p)
#pragma unroll
        for (int j = 0; j < R; ++j) load_v<V>(t[p][j], a.branch + (size_t)min(p0 + p, a.n_partials - 1) * a.partial_stride + at[j]);
#pragma unroll
      for (int p = 0; p < CH; ++p) {
        if (p0 + p >= a.n_partials) break;
#pragma unroll
        for (int j = 0; j < R; ++j)
#pragma unroll
          for (int i = 0; i < V; ++i) b[j][i] += t[p][j][i];
      }
    }
#pragma unroll
    for (int j = 0; j < R; ++j) {
#pragma unroll
      for (int i = 0; i < V; ++i) {
        float v = b[j][i];
        if (a.w_post) v = fmaf(FULL ? tanh_full(a.a_post * v) : tanh_fast(a.a_post * v), wp[i], bp[i]);
        x[j][i] += v;
      }
      if (r0 + j >= a.T) continue;
      if constexpr (V == 4) *reinterpret_cast<float4*>(a.resid + at[j]) = float4{x[j][0], x[j][1], x[j][2], x[j][3]};
      else a.resid[at[j]] = x[j][0];
    }
  }
  if (!a.out) return;
#pragma unroll
  for (int j = 0; j < R; ++j) {
    const int r = r0 + j;
    if (r >= a.T) break;
    float y[V];
#pragma unroll
    for (int i = 0; i < V; ++i)
      y[i] = a.w_pre ? fmaf(FULL ? tanh_full(a.a_pre * x[j][i]) : tanh_fast(a.a_pre * x[j][i]), wq[i], bq[i]) : x[j][i];
    const size_t o = out_index(a.out_layout, r, c, a.H);      // four consecutive elements are neighbours in both layouts
    if constexpr (V == 1) store_f32((TO*)a.out, o, y[0]);
    else if constexpr (sizeof(TO) == 4) *reinterpret_cast<float4*>((float*)a.out + o) = float4{y[0], y[1], y[2], y[3]};
    else *reinterpret_cast<uint2*>((bf16_t*)a.out + o) = uint2{pack_bf16x2(y[0], y[1]), pack_bf16x2(y[2], y[3])};
  }
}

template <typename TO, bool FULL>
void launch(const DynTanhArgs& a, bool vec, hipStream_t stream) {
  const int cols = vec ? a.H / 4 : a.H;
  const int threads = cols >= 256 ? 256 : ceil_div(cols, 64) * 64;
  // many rows: a thread's weights serve four of them; few rows: as many blocks as there are
  const int R = vec && a.T >= 1024 ? 4 : 1;
  const dim3 grid(ceil_div(a.T, R), ceil_div(cols, threads));
  if (R == 4) add_dyntanh_kernel<TO, FULL, 4, 4><<<grid, threads, 0, stream>>>(a);
  else if (vec) add_dyntanh_kernel<TO, FULL, 4, 1><<<grid, threads, 0, stream>>>(a);
  else add_dyntanh_kernel<TO, FULL, 1, 1><<<grid, threads, 0, stream>>>(a);
}

}  // namespace

extern "C" int alice_add_dyntanh(float* resid, const float* branch, int n_partials, long partial_stride, const float* w_post,
                                 const float* b_post, float a_post, const float* w_pre, const float* b_pre, float a_pre, void* out,
                                 int out_dtype, const int* rows, int T, int H, int full_precision, int out_layout,
                                 hipStream_t stream) {
  ALICE_CHECK(T >= 0 && H > 0, "add_dyntanh: bad sizes T=%d H=%d", T, H);
  ALICE_CHECK(resid && (branch || out), "add_dyntanh: the residual stream is missing, or there is nothing to do");
  ALICE_CHECK((w_post == nullptr) == (b_post == nullptr) && (w_pre == nullptr) == (b_pre == nullptr), "add_dyntanh: a norm has a weight and a bias");
  ALICE_CHECK((!w_post || branch) && (!w_pre || out), "add_dyntanh: a norm without its operand");
  ALICE_CHECK(dtype_ok(out_dtype), "add_dyntanh: unknown dtype");
  ALICE_CHECK(!(rows && branch), "add_dyntanh: a row gather cannot be combined with a residual add");
  ALICE_CHECK(n_partials >= 1 && n_partials <= 64, "add_dyntanh: n_partials %d out of range", n_partials);
  ALICE_CHECK(out_layout == 0 || (out_layout == 1 && out && out_dtype == DT_BF16 && H % 32 == 0),
              "add_dyntanh: output in fragment order needs bfloat16 and a width that is a multiple of 32");
  ALICE_CHECK(H <= (1 << 23), "add_dyntanh: rows of %d elements are too wide for one launch", H);
  if (T == 0) return 0;
  const DynTanhArgs a{resid, branch, n_partials, (size_t)partial_stride, w_post, b_post, w_pre, b_pre, a_post, a_pre, out, rows, T, H, out_layout};
  const bool vec = H % 4 == 0 && partial_stride % 4 == 0 &&
                   (((uintptr_t)resid | (uintptr_t)branch | (uintptr_t)out | (uintptr_t)w_post | (uintptr_t)b_post | (uintptr_t)w_pre | (uintptr_t)b_pre) & 15) == 0;
  DISPATCH_DTYPE(out_dtype, TO, {
    if (full_precision) launch<TO, true>(a, vec, stream); else launch<TO, false>(a, vec, stream);
  });
  ALICE_LAUNCH_CHECK();
  return 0;
}
