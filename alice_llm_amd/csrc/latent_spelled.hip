// Latent attention of long prompts with every head's keys and values spelled out for the length of a step: with many
// queries a key it costs less to make a head's key [Uk_h c | kr] (d + r numbers) and value Uv_h c (dv) once than to let
// every query meet the whole latent row (R + r for the score, R for the sum).  The cache keeps its latent rows; a step's
// keys and values live in a workspace laid out like a cache in fragment order (pages of 64 positions, heads of W numbers,
// W the matrix-core attention's head size that holds both, zeros beyond), so that kernel runs on them as they are.
//
//   latent_gather_kernel   the latents c of every position of the step's sequences, page by page, as contiguous rows for
//                          the product with [Uk; Uv] (zeros behind a sequence's last position), and the workspace's page table
//   latent_expand_kernel   from that product's rows and the cached rotated parts, a page of keys and a page of values a head
//   latent_heads_kernel    rows of heads moved between strides: a query's plain and rotated part (turned here) into heads of
//                          W numbers with zeros behind, and the attention's outputs back without the padding
#include "common.h"
#include "alice_hip.h"
#include "kv_layout.h"

namespace {

typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
constexpr int PAGE = 64;              // positions of a workspace page

// The sequence and page within it of workspace page v (the pages are dealt to the sequences in order), or -1.
__device__ __forceinline__ int page_owner(int v, const int* __restrict__ context_lens, int n_seqs, int& p) {
  for (int s = 0; s < n_seqs; ++s) {
    const int n = (context_lens[s] + PAGE - 1) / PAGE;
    if (v < n) {
      p = v;
      return s;
    }
    v -= n;
  }
  return -1;
}

__device__ __forceinline__ const bf16_t* cached_row(const bf16_t* __restrict__ pool, const int* __restrict__ bt, int page_size, int D, int pos) {
  return pool + ((size_t)bt[pos / page_size] * page_size + pos % page_size) * D;
}

__global__ __launch_bounds__(256) void latent_gather_kernel(const bf16_t* __restrict__ pool, const int* __restrict__ context_lens, int n_seqs,
                                                            const int* __restrict__ block_table, int bt_stride, int page_size, int R, int D,
                                                            bf16_t* __restrict__ rows, int* __restrict__ table, int table_stride) {
  int p = 0;
  const int v = blockIdx.x, s = page_owner(v, context_lens, n_seqs, p);
  if (s < 0) return;
  if (threadIdx.x == 0 && blockIdx.y == 0) table[(size_t)s * table_stride + p] = v;
  const int len = context_lens[s], per = R / 8;
  const int* bt = block_table + (size_t)s * bt_stride;
  for (int i = blockIdx.y * 256 + threadIdx.x; i < PAGE * per; i += 256 * gridDim.y) {
    const int t = i / per, e = (i % per) * 8, pos = p * PAGE + t;
    u32x4 x = {0u, 0u, 0u, 0u};
    if (pos < len) x = *reinterpret_cast<const u32x4*>(cached_row(pool, bt, page_size, D, pos) + e);
    *reinterpret_cast<u32x4*>(rows + ((size_t)v * PAGE + t) * R + e) = x;
  }
}

template <int W>
__global__ __launch_bounds__(256) void latent_expand_kernel(const bf16_t* __restrict__ kv, const bf16_t* __restrict__ pool,
                                                            const int* __restrict__ context_lens, int n_seqs, const int* __restrict__ block_table,
                                                            int bt_stride, int page_size, int R, int r, int H, int d, int dv,
                                                            bf16_t* __restrict__ k_out, bf16_t* __restrict__ v_out) {
  constexpr int VROW = W + 8;
  __shared__ __align__(16) bf16_t vs[PAGE][VROW];
  int p = 0;
  const int v = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, s = page_owner(v, context_lens, n_seqs, p);
  if (s < 0) return;
  const int len = context_lens[s], row_w = H * (d + dv);
  const int* bt = block_table + (size_t)s * bt_stride;
  const bf16_t* rows = kv + (size_t)v * PAGE * row_w;
  bf16_t* kp = k_out + ((size_t)v * H + h) * PAGE * W;
  bf16_t* vp = v_out + ((size_t)v * H + h) * PAGE * W;
  for (int i = tid; i < PAGE * dv / 8; i += 256) {
    const int t = i / (dv / 8), e = (i % (dv / 8)) * 8;
    *reinterpret_cast<u32x4*>(&vs[t][e]) = *reinterpret_cast<const u32x4*>(rows + (size_t)t * row_w + H * d + h * dv + e);
  }
#pragma unroll
  for (int i = tid; i < PAGE * W / 8; i += 256) {          // neighbouring threads: neighbouring positions (a tile's lanes)
    const int t = i % PAGE, e = (i / PAGE) * 8, pos = p * PAGE + t;
    u32x4 x = {0u, 0u, 0u, 0u};
    if (e < d) x = *reinterpret_cast<const u32x4*>(rows + (size_t)t * row_w + h * d + e);
    else if (e < d + r && pos < len) x = *reinterpret_cast<const u32x4*>(cached_row(pool, bt, page_size, R + r, pos) + R + e - d);
    *reinterpret_cast<u32x4*>(kp + k_offset(1, t, e, W)) = x;
  }
  __syncthreads();
#pragma unroll
  for (int i = tid; i < PAGE * W / 8; i += 256) {          // a lane's eight values: two runs of four positions of one dimension
    const int lane = i & 63, e = ((i >> 6) % (W / 16)) * 16 + (lane & 15), b = (i >> 6) / (W / 16), t0 = b * 32 + (lane >> 4) * 4;
    uint32_t w[4] = {0u, 0u, 0u, 0u};
    if (e < dv) {
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int t = t0 + 16 * (j >> 1) + 2 * (j & 1);
        w[j] = (uint32_t)vs[t][e].bits | ((uint32_t)vs[t + 1][e].bits << 16);
      }
    }
    *reinterpret_cast<u32x4*>(vp + (size_t)i * 8) = u32x4{w[0], w[1], w[2], w[3]};
  }
}

// y[t, h, 0:n] = x[t, h, 0:n]; y[t, h, n:n+r] = x[t, h, n:n+r] turned in pairs (2i, 2i + 1) by the token's position; zeros up
// to y_head.  Eight elements a thread.
__global__ __launch_bounds__(256) void latent_heads_kernel(const bf16_t* __restrict__ x, int x_head, bf16_t* __restrict__ y, int y_head,
                                                           int H, int n, int r, const float* __restrict__ cos_t,
                                                           const float* __restrict__ sin_t, const int* __restrict__ positions) {
  const int t = blockIdx.x, i = blockIdx.y * 256 + threadIdx.x, per = y_head / 8;
  if (i >= H * per) return;
  const int h = i / per, e = (i % per) * 8;
  const bf16_t* src = x + ((size_t)t * H + h) * x_head + e;
  u32x4 v = {0u, 0u, 0u, 0u};
  if (e < n + r) v = *reinterpret_cast<const u32x4*>(src);
  if (e >= n && e < n + r) {
    const size_t at = (size_t)positions[t] * (r >> 1) + ((e - n) >> 1);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      float y0, y1;
      rotate_pair(bf16_bits_to_f32(v[j] & 0xffffu), bf16_bits_to_f32(v[j] >> 16), cos_t[at + j], sin_t[at + j], y0, y1);
      v[j] = pack_bf16x2(y0, y1);
    }
  }
  *reinterpret_cast<u32x4*>(y + ((size_t)t * H + h) * y_head + e) = v;
}

bool aligned16(const void* p) { return ((uintptr_t)p & 15) == 0; }

}  // namespace

// The head size of the workspace (64, 128 or 256) for these sizes, 0 where they are not covered.
extern "C" int alice_latent_spelled_head(int kv_rank, int rot_dim, int d, int dv) {
  const int k = d + rot_dim, m = k > dv ? k : dv;
  if (kv_rank % 8 || rot_dim % 8 || d % 8 || dv % 8 || d < 8 || dv < 8 || kv_rank < 8 || m > 256) return 0;
  return m <= 64 ? 64 : (m <= 128 ? 128 : 256);
}

// pool: bfloat16 [pages, 1, page_size, kv_rank + rot_dim]; n_pages: the sum over the sequences of ceil(context / 64); rows:
// bfloat16 [n_pages 64, kv_rank]; table: int32 [n_seqs, table_stride], the workspace's page table.
extern "C" int alice_latent_gather(const void* pool, const int* context_lens, int n_seqs, const int* block_table, int bt_stride,
                                   int page_size, int kv_rank, int rot_dim, void* rows, int* table, int table_stride, int n_pages,
                                   hipStream_t stream) {
  ALICE_CHECK(pool && context_lens && block_table && rows && table, "latent_gather: a pointer is missing");
  ALICE_CHECK(n_seqs >= 1 && bt_stride >= 1 && page_size >= 1 && table_stride >= 1 && n_pages >= 0 && kv_rank >= 8 && kv_rank % 8 == 0 &&
              rot_dim >= 0 && rot_dim % 8 == 0, "latent_gather: bad sizes");
  ALICE_CHECK(aligned16(pool) && aligned16(rows), "latent_gather: operands are not aligned");
  if (n_pages == 0) return 0;
  latent_gather_kernel<<<dim3(n_pages, 8), 256, 0, stream>>>((const bf16_t*)pool, context_lens, n_seqs, block_table, bt_stride, page_size, kv_rank,
                                                    kv_rank + rot_dim, (bf16_t*)rows, table, table_stride);
  ALICE_LAUNCH_CHECK();
  return 0;
}

// kv: bfloat16 [n_pages 64, H d + H dv], the product of alice_latent_gather's rows with [Uk; Uv]; k_out, v_out: bfloat16
// [n_pages, H, 64, alice_latent_spelled_head(...)] in fragment order.
extern "C" int alice_latent_expand(const void* kv, const void* pool, const int* context_lens, int n_seqs, const int* block_table,
                                   int bt_stride, int page_size, int kv_rank, int rot_dim, int H, int d, int dv, void* k_out, void* v_out,
                                   int n_pages, hipStream_t stream) {
  ALICE_CHECK(kv && pool && context_lens && block_table && k_out && v_out, "latent_expand: a pointer is missing");
  const int W = alice_latent_spelled_head(kv_rank, rot_dim, d, dv);
  ALICE_CHECK(W != 0, "latent_expand: sizes d=%d rot_dim=%d dv=%d kv_rank=%d are not covered", d, rot_dim, dv, kv_rank);
  ALICE_CHECK(n_seqs >= 1 && bt_stride >= 1 && page_size >= 1 && n_pages >= 0 && H >= 1 && H <= 65535, "latent_expand: bad sizes");
  ALICE_CHECK(aligned16(kv) && aligned16(pool) && aligned16(k_out) && aligned16(v_out), "latent_expand: operands are not aligned");
  if (n_pages == 0) return 0;
#define GO(W) latent_expand_kernel<W><<<dim3(n_pages, H), 256, 0, stream>>>((const bf16_t*)kv, (const bf16_t*)pool, context_lens, n_seqs, \
      block_table, bt_stride, page_size, kv_rank, rot_dim, H, d, dv, (bf16_t*)k_out, (bf16_t*)v_out)
  if (W == 64) GO(64);
  else if (W == 128) GO(128);
  else GO(256);
#undef GO
  ALICE_LAUNCH_CHECK();
  return 0;
}

// x: bfloat16 [T, H, x_head]; y: bfloat16 [T, H, y_head], see latent_heads_kernel.
extern "C" int alice_latent_heads(const void* x, int x_head, void* y, int y_head, int T, int H, int n, int rot_dim, const float* cos_t,
                                  const float* sin_t, const int* positions, hipStream_t stream) {
  ALICE_CHECK(x && y && T >= 0 && H >= 1, "latent_heads: bad sizes or a missing pointer");
  ALICE_CHECK(n >= 8 && n % 8 == 0 && rot_dim >= 0 && rot_dim % 8 == 0 && x_head % 8 == 0 && y_head % 8 == 0 && x_head >= n + rot_dim &&
              y_head >= n + rot_dim, "latent_heads: parts of %d and %d numbers do not fit heads of %d and %d (multiples of 8)", n, rot_dim, x_head, y_head);
  ALICE_CHECK(rot_dim == 0 || (cos_t && sin_t && positions), "latent_heads: a rotated part needs both tables and the positions");
  ALICE_CHECK(aligned16(x) && aligned16(y), "latent_heads: operands are not aligned");
  ALICE_CHECK(ceil_div((long)H * y_head / 8, 256) <= 65535, "latent_heads: too many heads for one launch");
  if (T == 0) return 0;
  latent_heads_kernel<<<dim3(T, ceil_div((long)H * y_head / 8, 256)), 256, 0, stream>>>((const bf16_t*)x, x_head, (bf16_t*)y, y_head, H, n, rot_dim,
                                                                                    cos_t, sin_t, positions);
  ALICE_LAUNCH_CHECK();
  return 0;
}
