// Attention over a paged low-rank latent (gfx950). A token's cache row [latent c (R) | rotated key part (rp)]
// serves all heads; per head the unrotated key is W_uk c, the value W_uv c. ops/latent_attention.py has the
// equations of the two ways to evaluate it.
//
//  * rotation_table: cos / sin of p base^(-2 i / dims) per token, once per step for all layers;
//  * latent_append: norms of the query latent and of c, rotation of the key part, cache write;
//  * generic form (fp32, any size): one workgroup per (token, head);
//  * token form (decode, short continuations; bf16): latent_absorb forms W_uk^T q per head,
//    latent_token runs one workgroup per (token, 32 heads, key split) with 64-key tiles of the cache in LDS,
//    read by rows for the scores and transposed for the weighted sum of latents -- each cache byte crosses
//    HBM once for all heads --, latent_merge adds the splits and latent_expand applies W_uv (one token: the merge
//    is its prologue);
//  * tile form (prompts; bf16): keys and values of the window are expanded by a library product, then one
//    workgroup per (256 queries, head) in the flash manner (8 waves of 32 queries, 64-key tiles loaded straight
//    to a double-buffered LDS ring). The rotated key part is read from the gathered cache rows, queries are
//    rotated on the way into their registers.
// Only visible keys are enumerated (window: i sees 0 <= i - j < window). Scores, softmax and sums are fp32.
#include "sxe_common.h"
#include "sxe_mfma.h"
#include "sxe_tile.h"
#include <torch/library.h>
#include <type_traits>

namespace sxe {
namespace lt {
using namespace mf;

constexpr int kThreads = 256;

__global__ __launch_bounds__(kThreads) void rotation_table_kernel(const int64_t* __restrict pos, int T, int half, double lbase,
                                                                  float* __restrict out) {
  const int i = blockIdx.x * kThreads + threadIdx.x;
  if (i >= T * half) return;
  const int t = i / half, d = i - t * half;
  const double a = (double)pos[t] * exp2(-lbase * (double)d / (double)half);
  double s, c;
  sincos(a, &s, &c);
  out[2 * i] = (float)c;
  out[2 * i + 1] = (float)s;
}

// ---------------------------------------------------------------------------------------------- append
struct AppendArgs {
  const void* proj;  // [T, ld]: query latent | latent | key part
  int64_t ld;
  const void *qw, *kw;
  const float* rot;  // [T, rot_dim / 2, 2]
  const int64_t* slots;
  void *cq, *cache;  // [T, q_rank]; [blocks * bs, row]
  int q_rank, rank, R, rot_dim, row;
  int64_t nslots;
  float eps;
};

template <DT T, int V>
__device__ __forceinline__ void ldv(const typename dt_traits<T>::storage* p, float (&v)[V]) {
  if constexpr (V == 8) load8<T>(p, v);
  else v[0] = to_f32<T>(*p);
}
template <DT T, int V>
__device__ __forceinline__ void stv(typename dt_traits<T>::storage* p, const float (&v)[V]) {
  if constexpr (V == 8) store8<T>(p, v);
  else *p = from_f32<T>(v[0]);
}

template <DT T, int V>
__global__ __launch_bounds__(kThreads) void latent_append_kernel(AppendArgs a) {
  using S = typename dt_traits<T>::storage;
  __shared__ float red[2][kThreads / 64];
  const int64_t t = blockIdx.x;
  const S* row = static_cast<const S*>(a.proj) + t * a.ld;
  const int n = a.q_rank + a.rank;
  float sq = 0.f, sk = 0.f, v[V], w[V];
  for (int c = threadIdx.x * V; c < n; c += kThreads * V) {
    ldv<T, V>(row + c, v);
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < V; ++i) s += v[i] * v[i];
    if (c < a.q_rank) sq += s;
    else sk += s;
  }
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  if ((threadIdx.x & 63) == 0) {
    red[0][threadIdx.x >> 6] = sq;
    red[1][threadIdx.x >> 6] = sk;
  }
  __syncthreads();
  sq = red[0][0] + red[0][1] + red[0][2] + red[0][3];
  sk = red[1][0] + red[1][1] + red[1][2] + red[1][3];
  const float rq = 1.f / sqrtf(sq / (float)a.q_rank + a.eps), rk = 1.f / sqrtf(sk / (float)a.rank + a.eps);
  const int64_t slot = a.slots[t];
  const bool keep = slot >= 0 && slot < a.nslots;
  S* dst = static_cast<S*>(a.cache) + (keep ? slot : 0) * a.row;
  for (int c = threadIdx.x * V; c < n; c += kThreads * V) {
    ldv<T, V>(row + c, v);
    const bool q = c < a.q_rank;
    ldv<T, V>(q ? static_cast<const S*>(a.qw) + c : static_cast<const S*>(a.kw) + c - a.q_rank, w);
#pragma unroll
    for (int i = 0; i < V; ++i) v[i] = v[i] * (q ? rq : rk) * w[i];
    if (q) stv<T, V>(static_cast<S*>(a.cq) + t * a.q_rank + c, v);
    else if (keep) stv<T, V>(dst + c - a.q_rank, v);
  }
  const int half = a.rot_dim / 2;
  if (keep)
    for (int i = threadIdx.x; i < half; i += kThreads) {
      const float x = to_f32<T>(row[n + i]), y = to_f32<T>(row[n + half + i]);
      const float c = a.rot[(t * half + i) * 2], s = a.rot[(t * half + i) * 2 + 1];
      dst[a.R + i] = from_f32<T>(x * c - y * s);
      dst[a.R + half + i] = from_f32<T>(y * c + x * s);
    }
}

// --------------------------------------------------------------------------------------- generic form
struct Args {
  const void* q;  // [T, H * (dim + rot_dim)]
  const float* rot;
  const int* rows;  // [n, 2]: sequence, row of q
  const int *table, *q_start, *q_len, *kv_len;  // table [S, max blocks]
  const void* cache;
  int64_t nblocks;
  int maxb, bs, H, dim, rot_dim, rank, R, row, vdim, window;
  float scale;
};

// visible keys [lo, hi) of query row t of sequence s
__device__ __forceinline__ void key_range(const Args& a, int s, int t, int& lo, int& hi) {
  const int pos = a.kv_len[s] - a.q_len[s] + (t - a.q_start[s]);
  hi = min(pos + 1, a.maxb * a.bs);
  lo = a.window > 0 ? max(0, pos + 1 - a.window) : 0;
}
__device__ __forceinline__ int64_t cache_at(const Args& a, int s, int j) {
  const int b = j / a.bs;
  int64_t blk = a.table[(int64_t)s * a.maxb + b];
  if (blk < 0 || blk >= a.nblocks) blk = 0;
  return (blk * a.bs + (j - b * a.bs)) * a.row;
}

// grid (n, H); uk [H, rank, dim], uv [H, vdim, rank]
template <DT T>
__global__ __launch_bounds__(kThreads) void latent_generic_kernel(Args a, const typename dt_traits<T>::storage* __restrict uk,
                                                                  const typename dt_traits<T>::storage* __restrict uv,
                                                                  typename dt_traits<T>::storage* __restrict out) {
  using S = typename dt_traits<T>::storage;
  extern __shared__ float sm[];
  __shared__ float red[2][kThreads / 64];
  float* qa = sm;                // [rank + rot_dim]
  float* ol = qa + a.rank + a.rot_dim;  // [rank]
  float* p = ol + a.rank;        // [kThreads]
  const int s = a.rows[2 * blockIdx.x], t = a.rows[2 * blockIdx.x + 1], h = blockIdx.y, half = a.rot_dim / 2;
  const S* q = static_cast<const S*>(a.q) + ((int64_t)t * a.H + h) * (a.dim + a.rot_dim);
  for (int r = threadIdx.x; r < a.rank; r += kThreads) {
    float x = 0.f;
    for (int d = 0; d < a.dim; ++d) x += to_f32<T>(q[d]) * to_f32<T>(uk[((int64_t)h * a.rank + r) * a.dim + d]);
    qa[r] = x * a.scale;
    ol[r] = 0.f;
  }
  for (int i = threadIdx.x; i < half; i += kThreads) {
    const float x = to_f32<T>(q[a.dim + i]), y = to_f32<T>(q[a.dim + half + i]);
    const float c = a.rot[((int64_t)t * half + i) * 2], sn = a.rot[((int64_t)t * half + i) * 2 + 1];
    qa[a.rank + i] = (x * c - y * sn) * a.scale;
    qa[a.rank + half + i] = (y * c + x * sn) * a.scale;
  }
  __syncthreads();
  int lo, hi;
  key_range(a, s, t, lo, hi);
  const S* cache = static_cast<const S*>(a.cache);
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  float M = -INFINITY, L = 0.f;
  for (int j0 = lo; j0 < hi; j0 += kThreads) {
    const int j = j0 + threadIdx.x;
    float x = -INFINITY;
    if (j < hi) {
      const S* c = cache + cache_at(a, s, j);
      x = 0.f;
      for (int r = 0; r < a.rank; ++r) x += qa[r] * to_f32<T>(c[r]);
      for (int r = 0; r < a.rot_dim; ++r) x += qa[a.rank + r] * to_f32<T>(c[a.R + r]);
    }
    float m = wave_max(x);
    if (lane == 0) red[0][wave] = m;
    __syncthreads();
    m = fmaxf(fmaxf(red[0][0], red[0][1]), fmaxf(red[0][2], red[0][3]));
    const float Mn = fmaxf(M, m), f = M == -INFINITY ? 0.f : expf(M - Mn), e = j < hi ? expf(x - Mn) : 0.f;
    p[threadIdx.x] = e;
    float l = wave_sum(e);
    if (lane == 0) red[1][wave] = l;
    __syncthreads();
    L = L * f + red[1][0] + red[1][1] + red[1][2] + red[1][3];
    M = Mn;
    const int nj = min(kThreads, hi - j0);
    for (int r = threadIdx.x; r < a.rank; r += kThreads) {
      float o = ol[r] * f;
      for (int i = 0; i < nj; ++i) o += p[i] * to_f32<T>(cache[cache_at(a, s, j0 + i) + r]);
      ol[r] = o;
    }
    __syncthreads();
  }
  const float inv = L > 0.f ? 1.f / L : 0.f;
  for (int v = threadIdx.x; v < a.vdim; v += kThreads) {
    float o = 0.f;
    for (int r = 0; r < a.rank; ++r) o += ol[r] * to_f32<T>(uv[((int64_t)h * a.vdim + v) * a.rank + r]);
    out[((int64_t)t * a.H + h) * a.vdim + v] = from_f32<T>(o * inv);
  }
}

// ----------------------------------------------------------------------- per-head products (token form)
__device__ __forceinline__ f32x4 mfma16(bf16x8 a, bf16x8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}

// y = x W^T for 16 rows x and 16 rows of W (both K contiguous, K % 8 == 0): the workgroup's 4 waves split K;
// thread i gets element (row i / 16, column i % 16). xrow / wrow: the lane's row (l16), always readable.
__device__ __forceinline__ float head_product(const unsigned short* xrow, const unsigned short* wrow, int K, float (*part)[16][17]) {
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, l16 = lane & 15, g = lane >> 4;
  constexpr int U = 4;
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
  for (int k0 = w * 32; k0 < K; k0 += U * 128) {
    u32x4 a[U], b[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = k0 + u * 128 + 8 * g;
      a[u] = b[u] = u32x4{0u, 0u, 0u, 0u};
      if (k < K) {
        a[u] = *reinterpret_cast<const u32x4*>(xrow + k);
        b[u] = *reinterpret_cast<const u32x4*>(wrow + k);
      }
    }
#pragma unroll
    for (int u = 0; u < U; ++u) acc = mfma16(__builtin_bit_cast(bf16x8, a[u]), __builtin_bit_cast(bf16x8, b[u]), acc);
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) part[w][4 * g + i][l16] = acc[i];
  __syncthreads();
  const int r = threadIdx.x >> 4, c = threadIdx.x & 15;
  return part[0][r][c] + part[1][r][c] + part[2][r][c] + part[3][r][c];
}

// grid (R / 64 + 1, H, ceil(n / 16)) -> qa [n, H, row] bf16: W_uk^T q | rotated q, zero-padded; uk [H, rank, dim].
// A wave takes 16 columns and the whole (short) inner dimension.
__global__ __launch_bounds__(kThreads) void latent_absorb_kernel(Args a, int n, const unsigned short* __restrict uk,
                                                                 unsigned short* __restrict qa) {
  const int h = blockIdx.y, i0 = blockIdx.z * 16, half = a.rot_dim / 2, l16 = threadIdx.x & 15, g = (threadIdx.x & 63) >> 4;
  const unsigned short* q = static_cast<const unsigned short*>(a.q);
  if ((int)blockIdx.x * 64 < a.R) {
    const int c = blockIdx.x * 64 + (threadIdx.x >> 6) * 16 + l16;
    const int64_t row = a.rows[2 * min(i0 + l16, n - 1) + 1];
    const unsigned short* xr = q + (row * a.H + h) * (a.dim + a.rot_dim);
    const unsigned short* wr = uk + ((int64_t)h * a.rank + min(c, a.rank - 1)) * a.dim;
    constexpr int U = 4;
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < a.dim; k0 += U * 32) {
      u32x4 x[U], w[U];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int k = k0 + u * 32 + 8 * g;
        x[u] = w[u] = u32x4{0u, 0u, 0u, 0u};
        if (k < a.dim) {
          x[u] = *reinterpret_cast<const u32x4*>(xr + k);
          w[u] = *reinterpret_cast<const u32x4*>(wr + k);
        }
      }
#pragma unroll
      for (int u = 0; u < U; ++u) acc = mfma16(__builtin_bit_cast(bf16x8, x[u]), __builtin_bit_cast(bf16x8, w[u]), acc);
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = i0 + 4 * g + e;
      if (i < n) qa[((int64_t)i * a.H + h) * a.row + c] = c < a.rank ? f32_to_bf16(acc[e]) : 0;
    }
    return;
  }
  const int rp = a.row - a.R;
  for (int x = threadIdx.x; x < 16 * rp; x += kThreads) {
    const int i = i0 + x / rp, d = x % rp;
    if (i >= n) continue;
    const int64_t row = a.rows[2 * i + 1];
    float v = 0.f;
    if (d < a.rot_dim) {
      const unsigned short* qr = q + (row * a.H + h) * (a.dim + a.rot_dim) + a.dim;
      const int j = d < half ? d : d - half;
      const float u = bf16_to_f32(qr[j]), y = bf16_to_f32(qr[half + j]);
      const float co = a.rot[(row * half + j) * 2], si = a.rot[(row * half + j) * 2 + 1];
      v = d < half ? u * co - y * si : y * co + u * si;
    }
    qa[((int64_t)i * a.H + h) * a.row + a.R + d] = f32_to_bf16(v);
  }
}

// weights of a (token, head)'s splits, 2^(M_s - M) / sum, by one wave; ml: its (max, sum) of split 0
__device__ __forceinline__ void split_weights(const float* ml, int64_t stride, int splits, float* wts) {
  const int lane = threadIdx.x & 63;
  float M = -INFINITY, L = 0.f;
  for (int s = lane; s < splits; s += 64) M = fmaxf(M, ml[s * stride]);
  M = wave_max(M);
  for (int s = lane; s < splits; s += 64) {
    const float m = ml[s * stride], f = m == -INFINITY ? 0.f : exp2f(m - M);
    wts[s] = f;
    if (f > 0.f) L += f * ml[s * stride + 1];
  }
  L = wave_sum(L);
  const float inv = L > 0.f ? 1.f / L : 0.f;
  for (int s = lane; s < splits; s += 64) wts[s] *= inv;  // the lane's own entries
}

// 4 merged components: a split without keys has not written its part
__device__ __forceinline__ f32x4 merged4(const float* p, int64_t stride, int splits, const float* wts) {
  f32x4 v = {0.f, 0.f, 0.f, 0.f};
  constexpr int U = 8;
  for (int s0 = 0; s0 < splits; s0 += U) {
    f32x4 t[U];
#pragma unroll
    for (int u = 0; u < U; ++u) t[u] = *reinterpret_cast<const f32x4*>(p + min(s0 + u, splits - 1) * stride);
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const float f = s0 + u < splits ? wts[min(s0 + u, splits - 1)] : 0.f;
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] += f > 0.f ? f * t[u][e] : 0.f;
    }
  }
  return v;
}

constexpr int kMaxSplits = 256;

// grid (H, n): ol [n, H, R] bf16
__global__ __launch_bounds__(128) void latent_merge_kernel(Args a, int n, int splits, const float* __restrict po,
                                                           const float* __restrict pml, unsigned short* __restrict ol) {
  __shared__ float wts[kMaxSplits];
  const int64_t th = (int64_t)blockIdx.y * a.H + blockIdx.x, ss = (int64_t)n * a.H;
  if (threadIdx.x < 64) split_weights(pml + th * 2, ss * 2, splits, wts);
  __syncthreads();
  for (int c = threadIdx.x * 4; c < a.R; c += 512) {
    const f32x4 v = merged4(po + th * a.R + c, ss * a.R, splits, wts);
    *reinterpret_cast<u16x4*>(ol + th * a.R + c) = u16x4{f32_to_bf16(v[0]), f32_to_bf16(v[1]), f32_to_bf16(v[2]), f32_to_bf16(v[3])};
  }
}

// grid (ceil(vdim / 16), H, ceil(n / 16)): out[row, h, :] = W_uv ol; uv [H, vdim, rank]. MERGE: n == 1, the merged
// latent is formed here.
template <bool MERGE>
__global__ __launch_bounds__(kThreads) void latent_expand_kernel(Args a, int n, int splits, const float* __restrict po,
                                                                 const float* __restrict pml, const unsigned short* __restrict ol,
                                                                 const unsigned short* __restrict uv, unsigned short* __restrict out) {
  __shared__ float part[4][16][17], wts[MERGE ? kMaxSplits : 1];
  __shared__ __attribute__((aligned(16))) unsigned short x[MERGE ? 512 : 8];
  const int c0 = blockIdx.x * 16, h = blockIdx.y, i0 = blockIdx.z * 16, l16 = threadIdx.x & 15;
  const unsigned short* xr = x;
  if constexpr (MERGE) {
    if (threadIdx.x < 64) split_weights(pml + h * 2, (int64_t)a.H * 2, splits, wts);
    __syncthreads();
    if (threadIdx.x * 4 < a.R) {
      const int c = threadIdx.x * 4;
      const f32x4 v = merged4(po + (int64_t)h * a.R + c, (int64_t)a.H * a.R, splits, wts);
      *reinterpret_cast<u16x4*>(x + c) = u16x4{f32_to_bf16(v[0]), f32_to_bf16(v[1]), f32_to_bf16(v[2]), f32_to_bf16(v[3])};
    }
    __syncthreads();
  } else {
    xr = ol + ((int64_t)min(i0 + l16, n - 1) * a.H + h) * a.R;
  }
  const float v = head_product(xr, uv + ((int64_t)h * a.vdim + min(c0 + l16, a.vdim - 1)) * a.rank, a.rank, part);
  const int i = i0 + (threadIdx.x >> 4), c = c0 + l16;
  if (i < n && c < a.vdim) out[((int64_t)a.rows[2 * i + 1] * a.H + h) * a.vdim + c] = f32_to_bf16(v);
}

// ------------------------------------------------------------------------------------------ token form
constexpr int kKeys = 64;       // keys of a tile of the tile form
constexpr int kTok = 64, kTokWaves = 8;  // ... of the token form
constexpr int kSRow = kTok + 4;  // fp32 score row of a head

constexpr int kTabMax = 1024;   // most block-table entries of a split (kept in LDS)

// barrier without waiting for the loads in flight
__device__ __forceinline__ void lds_barrier() {
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
}
// PN 256-byte panels hold the latent (R = 128 PN), a 128-byte one the rotated part. grid (n, ceil(H / 32), splits).
// Tiles arrive by direct-to-LDS loads, one ahead. 8 waves: scores of (16 keys, 16 heads) each; then the 32-column
// tiles w, w + 8, .. of the latent sum, all heads.
template <int PN>
__global__ __launch_bounds__(64 * kTokWaves, 1) void latent_token_kernel(Args a, int n, const unsigned short* __restrict qa,
                                                                         float* __restrict po, float* __restrict pml) {
  char* smem = tl::lds;
  constexpr int PANEL = kTok * 256, SLOT = PN * PANEL + kTok * 128, NS = 4 * PN + 2, ROW = 128 * PN + 64;
  constexpr int CT = 4 * PN, NT = (CT + kTokWaves - 1) / kTokWaves;
  float* ls = reinterpret_cast<float*>(smem + 2 * SLOT);          // [32 heads][kSRow]
  int* tab = reinterpret_cast<int*>(smem + 2 * SLOT + 32 * kSRow * 4);  // [kTabMax]
  const int i = blockIdx.x, g = blockIdx.y, sp = blockIdx.z;
  const int s = a.rows[2 * i], t = a.rows[2 * i + 1];
  const int lane = threadIdx.x & 63, w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int l16 = lane & 15, q16 = lane >> 4, l32 = lane & 31, hh = lane >> 5;
  int lo, hi;
  key_range(a, s, t, lo, hi);
  {  // this split's keys, whole tiles
    const int tiles = (hi - lo + kTok - 1) / kTok, per = (tiles + gridDim.z - 1) / gridDim.z;
    lo = min(hi, lo + sp * per * kTok);
    hi = min(hi, lo + per * kTok);
  }
  const int ntiles = (hi - lo + kTok - 1) / kTok, b0 = lo / a.bs;
  const unsigned short* cache = static_cast<const unsigned short*>(a.cache);
  const int* row = a.table + (int64_t)s * a.maxb + b0;
  auto at = [&](int j, auto entry) {  // cache row of key j; past the end: the last one (masked)
    j = min(j, hi - 1);
    const int b = j / a.bs;
    int64_t blk = entry(min(b - b0, kTabMax - 1));
    if (blk < 0 || blk >= a.nblocks) blk = 0;
    return cache + (blk * a.bs + (j - b * a.bs)) * ROW;
  };
  const int r0 = 4 * w + (lane >> 4), r2 = 8 * w + (lane >> 3);  // rows this lane loads: r0, r0 + 32 (one swizzle); r2
  const int c0 = ((lane & 15) ^ tl::swz<128>(r0)) * 8, c2 = ((lane & 7) ^ tl::swz<64>(r2)) * 8;
  auto issue = [&](int j0, char* slot, auto entry) {
    const unsigned short *p0 = at(j0 + r0, entry), *p1 = at(j0 + 32 + r0, entry), *p2 = at(j0 + r2, entry);
#pragma unroll
    for (int p = 0; p < PN; ++p) {
      tl::glds16(p0 + p * 128 + c0, slot + p * PANEL + w * 1024);
      tl::glds16(p1 + p * 128 + c0, slot + p * PANEL + (w + 8) * 1024);
    }
    tl::glds16(p2 + PN * 128 + c2, slot + PN * PANEL + w * 1024);
  };
  // the first tile takes its blocks from memory; the table is in LDS for the others
  if (ntiles > 0) issue(lo, smem, [&](int x) { return row[x]; });
  if (ntiles > 1)
    for (int x = threadIdx.x; x < min((hi - 1) / a.bs - b0 + 1, kTabMax); x += 64 * kTokWaves) tab[x] = row[x];
  bf16x8 qf[NS];  // B fragments of 16 heads
  {
    const int h = 32 * g + 16 * (w >> 2) + l16;
    const unsigned short* qr = qa + ((int64_t)i * a.H + min(h, a.H - 1)) * ROW + q16 * 8;
#pragma unroll
    for (int k = 0; k < NS; ++k) qf[k] = *reinterpret_cast<const bf16x8*>(qr + k * 32);
  }
  // LDS read offsets: score rows (chunks q16 + 4 i of a panel: the swizzle's low bits move with i), value columns
  const int kr = 16 * (w & 3) + l16;
  int ko[4], kp[2];
#pragma unroll
  for (int k = 0; k < 4; ++k) ko[k] = tl::off<128>(kr, 4 * k + q16);
#pragma unroll
  for (int k = 0; k < 2; ++k) kp[k] = tl::off<64>(kr, 4 * k + q16);
  int vo[NT][2];
  {
    tl::LaneOffs<128> o;
    o.init(lane);
#pragma unroll
    for (int j = 0; j < NT; ++j)
#pragma unroll
      for (int x = 0; x < 4; ++x)
        if (((w + kTokWaves * j) & 3) == x) {
          vo[j][0] = o.tr[x][0] + ((w + kTokWaves * j) >> 2) * PANEL;
          vo[j][1] = o.tr[x][1] + ((w + kTokWaves * j) >> 2) * PANEL;
        }
  }
  f32x16 acc[NT];
#pragma unroll
  for (int j = 0; j < NT; ++j) acc[j] = zero16();
  float M = -INFINITY, L = 0.f;
  const float sc2 = a.scale * LOG2E;
  // one copy of the loop body: few tiles run per workgroup, so instructions fetched twice would cost more than
  // the slot's address arithmetic
#pragma unroll 1
  for (int tile = 0; tile < ntiles; ++tile) {
    const int j0 = lo + tile * kTok, cur = tile & 1;
    const char *lk = smem + cur * SLOT, *lr = lk + PN * PANEL;
    tl::wait_loads();
    lds_barrier();  // the tile has landed for every wave, and every wave is done with the one before
    if (tile + 1 < ntiles) issue(j0 + kTok, smem + (cur ^ 1) * SLOT, [&](int x) { return tab[x]; });
    f32x4 s0 = {0.f, 0.f, 0.f, 0.f}, s1 = s0;  // keys 16 (w & 3) + 4 q16 + e, head 16 (w >> 2) + l16
    bf16x8 kf[NS];
#pragma unroll
    for (int k = 0; k < 4 * PN; ++k) kf[k] = tl::row_at(lk + (k >> 2) * PANEL, ko[k & 3]);
#pragma unroll
    for (int k = 0; k < 2; ++k) kf[4 * PN + k] = tl::row_at(lr, kp[k]);
#pragma unroll
    for (int k = 0; k < NS; k += 2) {
      s0 = mfma16(kf[k], qf[k], s0);
      s1 = mfma16(kf[k + 1], qf[k + 1], s1);
    }
    const int kj = 16 * (w & 3) + 4 * q16;
#pragma unroll
    for (int e = 0; e < 4; ++e) s0[e] = j0 + kj + e < hi ? (s0[e] + s1[e]) * sc2 : -INFINITY;
    *reinterpret_cast<f32x4*>(ls + (16 * (w >> 2) + l16) * kSRow + kj) = s0;
    lds_barrier();
    // every wave forms all weights of the tile: lane = head l32, keys 8 x + 4 hh + e
    f32x4 p[8];
    float m = -INFINITY;
#pragma unroll
    for (int x = 0; x < 8; ++x) p[x] = *reinterpret_cast<const f32x4*>(ls + l32 * kSRow + 8 * x + 4 * hh);
    bf16x8 vf[4][NT];
#pragma unroll
    for (int x = 0; x < 4; ++x)
#pragma unroll
      for (int j = 0; j < NT; ++j)
        if (CT % kTokWaves == 0 || w + kTokWaves * j < CT) vf[x][j] = tl::tr_at(lk + 16 * x * 256, vo[j]);
#pragma unroll
    for (int x = 0; x < 8; ++x) m = fmaxf(m, fmaxf(fmaxf(p[x][0], p[x][1]), fmaxf(p[x][2], p[x][3])));
    m = fmaxf(m, xor32(m));
    const float Mn = fmaxf(M, m), f = fast_exp2(M - Mn);  // a tile has a visible key: Mn is finite
    float l = 0.f;
#pragma unroll
    for (int x = 0; x < 8; ++x)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        p[x][e] = fast_exp2(p[x][e] - Mn);
        l += p[x][e];
      }
    L = L * f + l + xor32(l);
    if (__any(Mn > M)) {
#pragma unroll
      for (int j = 0; j < NT; ++j)
#pragma unroll
        for (int e = 0; e < 16; ++e) acc[j][e] *= f;
    }
    M = Mn;
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      bf16x8 b;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        b[e] = (__bf16)p[2 * x][e];
        b[4 + e] = (__bf16)p[2 * x + 1][e];
      }
#pragma unroll
      for (int j = 0; j < NT; ++j)
        if (CT % kTokWaves == 0 || w + kTokWaves * j < CT) acc[j] = mfma(vf[x][j], b, acc[j]);
    }
  }
  const int h = 32 * g + l32;
  if (h < a.H) {
    const int64_t th = ((int64_t)sp * n + i) * a.H + h;
    if (w == 0 && hh == 0) {
      pml[th * 2] = M;
      pml[th * 2 + 1] = L;
    }
    if (ntiles > 0) {
#pragma unroll
      for (int j = 0; j < NT; ++j) {
        const int ct = w + kTokWaves * j;
        if (ct >= CT) break;
        float* o = po + th * a.R + ct * 32 + 4 * hh;
#pragma unroll
        for (int e = 0; e < 4; ++e)
          *reinterpret_cast<f32x4*>(o + 8 * e) = f32x4{acc[j][4 * e], acc[j][4 * e + 1], acc[j][4 * e + 2], acc[j][4 * e + 3]};
      }
    }
  }
}

// ------------------------------------------------------------------------------------------- tile form
constexpr int kQ = 256, kTileWaves = 8;

struct TileArgs {
  const unsigned short *q, *kv, *lat;  // [T, H (dim + rot)], [Nk, H (dim + vdim)], [Nk, row]
  const float* rot;
  const int *chunks, *first, *q_start, *q_len, *kv_len;
  unsigned short* out;  // [T, H vdim]
  int64_t ldkv;
  int H, dim, rot_dim, vdim, R, row, window, Nk;
  float scale;
};

// One 64-key tile of a wave's online softmax: S^T = K Q^T (a lane holds one query's scores), the weights are the
// B operand of O^T += V^T P^T as they are. MASK: some key of the tile is hidden from some query of the wave.
template <bool MASK, int DN, int VP>
__device__ __forceinline__ void latent_tile_step(const tl::LaneOffs<DN>& ok, const tl::LaneOffs<64>& orr, const tl::LaneOffs<VP>& ov,
                                                 const char* lk, const bf16x8 (&qn)[DN / 16], const bf16x8 (&qr)[4],
                                                 f32x16 (&acc)[VP / 32], float& M, float& L, float c, int j0, int pw, int lane,
                                                 int win) {
  const char *lr = lk + kKeys * 2 * DN, *lv = lr + kKeys * 128;
  const int l32 = lane & 31, hh = lane >> 5;
  // halves of the tile hidden from the whole wave: in front of every window, behind every query
  const bool skip0 = MASK && pw - (j0 + 31) >= win, skip1 = MASK && j0 + 32 > pw + 31;
  f32x16 s[2];
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    s[j] = zero16();
    if (j == 0 ? skip0 : skip1) continue;
#pragma unroll
    for (int k = 0; k < DN / 16; ++k) s[j] = mfma(tl::row_at(lk + 32 * j * 2 * DN, ok.row[k]), qn[k], s[j]);
#pragma unroll
    for (int k = 0; k < 4; ++k) s[j] = mfma(tl::row_at(lr + 32 * j * 128, orr.row[k]), qr[k], s[j]);
  }
  float mx = -INFINITY;
  int dd = pw + l32 - j0 - 4 * hh;  // distance to the lane's first key row
  if (MASK) asm volatile("" : "+v"(dd));
#pragma unroll
  for (int j = 0; j < 2; ++j)
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      if (MASK) s[j][i] = (unsigned)(dd - 32 * j - acc_row(i, 0)) < (unsigned)win ? s[j][i] : -INFINITY;
      mx = fmaxf(mx, s[j][i]);
    }
  mx = fmaxf(mx, xor32(mx)) * c;
  // the reference maximum moves only when a tile exceeds it by 2^8; the sums are rescaled only then
  const bool grow = mx > M + 8.f;
  const float Mn = grow ? mx : M, ref = Mn == -INFINITY ? 0.f : Mn, alpha = fast_exp2(M - ref);
  float ps = 0.f;
#pragma unroll
  for (int j = 0; j < 2; ++j)
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const float p = fast_exp2(__builtin_fmaf(s[j][i], c, -ref));
      s[j][i] = p;
      ps += p;
    }
  L = L * alpha + ps;
  M = Mn;
  if (__any(grow)) {
#pragma unroll
    for (int t = 0; t < VP / 32; ++t)
#pragma unroll
      for (int i = 0; i < 16; ++i) acc[t][i] *= alpha;
  }
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    if (j == 0 ? skip0 : skip1) continue;
#pragma unroll
    for (int x = 0; x < 2; ++x) {
      const bf16x8 p = acc_to_b(s[j], x);
#pragma unroll
      for (int t = 0; t < VP / 32; ++t) acc[t] = mfma(tl::tr_at(lv + (32 * j + 16 * x) * 2 * VP, ov.tr[t]), p, acc[t]);
    }
  }
}

// 8 rotated query components d0 .. d0 + 7 (zeros beyond rot_dim); qr: the head's rotated part, cs its table row
__device__ __forceinline__ bf16x8 rotated8(const unsigned short* qr, const float* cs, int d0, int rot_dim) {
  const int half = rot_dim / 2;
  bf16x8 r;
#pragma unroll
  for (int e = 0; e < 8; ++e) r[e] = (__bf16)0.f;
  if (d0 >= rot_dim) return r;
  if (half % 8 == 0) {
    const bool lo = d0 < half;
    const int j0 = lo ? d0 : d0 - half;
    float u[8], y[8], t[16];
    load8<DT::BF16>(qr + j0, u);
    load8<DT::BF16>(qr + half + j0, y);
#pragma unroll
    for (int e = 0; e < 4; ++e) *reinterpret_cast<f32x4*>(t + 4 * e) = *reinterpret_cast<const f32x4*>(cs + 2 * j0 + 4 * e);
#pragma unroll
    for (int e = 0; e < 8; ++e)
      r[e] = (__bf16)(lo ? u[e] * t[2 * e] - y[e] * t[2 * e + 1] : y[e] * t[2 * e] + u[e] * t[2 * e + 1]);
    return r;
  }
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    const int d = d0 + e;
    if (d < rot_dim) {
      const int j = d < half ? d : d - half;
      const float u = bf16_to_f32(qr[j]), y = bf16_to_f32(qr[half + j]), co = cs[2 * j], si = cs[2 * j + 1];
      r[e] = (__bf16)(d < half ? u * co - y * si : y * co + u * si);
    }
  }
  return r;
}

// DN, VP: dim and vdim padded to 64 / 128; the rotated part is padded to 64. grid (H, chunks of kQ rows): a head's
// chunks share an XCD when the heads are a multiple of its count
template <int DN, int VP>
__global__ __launch_bounds__(64 * kTileWaves, 1) void latent_tile_kernel(TileArgs a) {
  char* smem = tl::lds;
  constexpr int KB = kKeys * 2 * DN, RB = kKeys * 128, SLOT = KB + RB + kKeys * 2 * VP;
  const int c = gridDim.y - 1 - blockIdx.y, h = blockIdx.x;  // late chunks see more keys: first
  const int s = a.chunks[3 * c], row0 = a.chunks[3 * c + 1], n = a.chunks[3 * c + 2];
  const int pos0 = a.kv_len[s] - a.q_len[s] + (row0 - a.q_start[s]), plast = pos0 + n - 1;
  const int f0 = a.first[2 * s], fp = a.first[2 * s + 1];  // list row and position of the first listed key
  const int win = a.window > 0 ? a.window : 0x7fffffff;
  const int lo = max(fp, a.window > 0 ? pos0 + 1 - a.window : 0), ntiles = (plast - lo) / kKeys + 1;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, l32 = lane & 31, hh = lane >> 5;
  const unsigned short *kb = a.kv + h * a.dim, *vb = a.kv + a.H * a.dim + h * a.vdim, *rb = a.lat + a.R;
  auto issue = [&](int t, char* slot) {
    const int j0 = lo + t * kKeys;
    auto at = [&](int r) { return (int64_t)min(max(f0 + min(j0 + r, plast) - fp, 0), a.Nk - 1); };
    tl::load_tile<kKeys, DN, kTileWaves>(slot, a.dim / 8, [&](int r) { return kb + at(r) * a.ldkv; });
    tl::load_tile<kKeys, 64, kTileWaves>(slot + KB, a.rot_dim / 8, [&](int r) { return rb + at(r) * a.row; });
    tl::load_tile<kKeys, VP, kTileWaves>(slot + KB + RB, a.vdim / 8, [&](int r) { return vb + at(r) * a.ldkv; });
  };
  issue(0, smem);
  bf16x8 qn[DN / 16], qr[4];
  {
    const int64_t t = row0 + min(w * 32 + l32, n - 1);
    const unsigned short* q = a.q + (t * a.H + h) * (a.dim + a.rot_dim);
#pragma unroll
    for (int k = 0; k < DN / 16; ++k) {
      u32x4 z = {0u, 0u, 0u, 0u};
      if (16 * k + 8 * hh < a.dim) z = *reinterpret_cast<const u32x4*>(q + 16 * k + 8 * hh);
      qn[k] = __builtin_bit_cast(bf16x8, z);
    }
#pragma unroll
    for (int k = 0; k < 4; ++k) qr[k] = rotated8(q + a.dim, a.rot + t * a.rot_dim, 16 * k + 8 * hh, a.rot_dim);
  }
  const int pw = pos0 + w * 32;  // the wave's first position
  tl::LaneOffs<DN> ok;
  tl::LaneOffs<64> orr;
  tl::LaneOffs<VP> ov;
  ok.init(lane);
  orr.init(lane);
  ov.init(lane);
  f32x16 acc[VP / 32];
#pragma unroll
  for (int j = 0; j < VP / 32; ++j) acc[j] = zero16();
  float M = -INFINITY, L = 0.f;
  const float sc = a.scale * LOG2E;
  tl::wait_loads();
  __syncthreads();
  auto step = [&](int t, auto slot) {
    constexpr int CUR = decltype(slot)::value;
    if (t + 1 < ntiles) issue(t + 1, smem + (CUR ^ 1) * SLOT);
    const int j0 = lo + t * kKeys;
    const char* lk = smem + CUR * SLOT;
    if (w * 32 < n && j0 <= pw + 31 && pw - (j0 + kKeys - 1) < win) {
      if (j0 + kKeys - 1 <= pw && pw + 31 - j0 < win)
        latent_tile_step<false, DN, VP>(ok, orr, ov, lk, qn, qr, acc, M, L, sc, j0, pw, lane, win);
      else
        latent_tile_step<true, DN, VP>(ok, orr, ov, lk, qn, qr, acc, M, L, sc, j0, pw, lane, win);
    }
    tl::wait_loads();
    __syncthreads();
  };
  for (int t = 0; t < ntiles; t += 2) {
    step(t, std::integral_constant<int, 0>{});
    if (t + 1 < ntiles) step(t + 1, std::integral_constant<int, 1>{});
  }
  const int t = w * 32 + l32;
  L += xor32(L);
  if (t < n) {
    const float inv = L > 0.f ? 1.f / L : 0.f;
    unsigned short* o = a.out + ((int64_t)(row0 + t) * a.H + h) * a.vdim;
#pragma unroll
    for (int j = 0; j < VP / 32; ++j)
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        const int v = j * 32 + 8 * g + 4 * hh;
        if (v < a.vdim) {
          u16x4 r;
#pragma unroll
          for (int e = 0; e < 4; ++e) r[e] = f32_to_bf16(acc[j][4 * g + e] * inv);
          *reinterpret_cast<u16x4*>(o + v) = r;
        }
      }
  }
}

inline bool aligned(const void* p, size_t n) { return reinterpret_cast<uintptr_t>(p) % n == 0; }

// The fields of Args every form uses; q may be [T, H (dim + rot)] or None
void check_batch(const at::Tensor& rows, const at::Tensor& table, const at::Tensor& q_start, const at::Tensor& q_len,
                 const at::Tensor& kv_len, const at::Tensor& cache) {
  const int64_t S = q_start.numel();
  SXE_CHECK(rows.is_cuda() && rows.scalar_type() == at::kInt && rows.is_contiguous() && rows.dim() == 2 && rows.size(1) == 2,
            "latent_attention: rows int32 [n, 2]");
  SXE_CHECK(table.is_cuda() && table.scalar_type() == at::kInt && table.is_contiguous() && table.dim() == 2 && table.size(0) == S,
            "latent_attention: block table int32 [S, blocks]");
  for (const auto* t : {&q_start, &q_len, &kv_len})
    SXE_CHECK(t->is_cuda() && t->is_contiguous() && t->scalar_type() == at::kInt && t->numel() == S, "latent_attention: int32 [S]");
  SXE_CHECK(cache.is_cuda() && cache.dim() == 4 && cache.size(1) == 1 && cache.is_contiguous(),
            "latent_attention: cache [blocks, 1, bs, row] contiguous");
}

}  // namespace lt

at::Tensor rotation_table(const at::Tensor& positions, int64_t dims, double base) {
  SXE_CHECK_CUDA(positions);
  SXE_CHECK(positions.scalar_type() == at::kLong && positions.is_contiguous() && dims > 0 && dims % 2 == 0 && base > 0,
            "rotation_table: positions int64, even dims");
  const int64_t T = positions.numel(), half = dims / 2;
  auto out = at::empty({T, half, 2}, positions.options().dtype(at::kFloat));
  if (T == 0) return out;
  SXE_CHECK(T * half < (1ll << 31), "rotation_table: too large");
  c10::DeviceGuard g(positions.device());
  hipLaunchKernelGGL(lt::rotation_table_kernel, dim3((T * half + lt::kThreads - 1) / lt::kThreads), dim3(lt::kThreads), 0,
                     cur_stream(), positions.data_ptr<int64_t>(), (int)T, (int)half, std::log2(base), out.data_ptr<float>());
  SXE_LAUNCH_CHECK();
  return out;
}

at::Tensor latent_append(const at::Tensor& proj, const at::Tensor& qw, const at::Tensor& kw, at::Tensor cache,
                         const at::Tensor& slots, const at::Tensor& rot, int64_t q_rank, int64_t rank, int64_t R, int64_t rot_dim,
                         double eps) {
  SXE_CHECK_CUDA(proj);
  const int64_t T = proj.size(0);
  SXE_CHECK(proj.dim() == 2 && proj.stride(1) == 1 && proj.size(1) >= q_rank + rank + rot_dim, "latent_append: proj");
  SXE_CHECK(qw.is_contiguous() && qw.numel() == q_rank && kw.is_contiguous() && kw.numel() == rank && qw.is_cuda() && kw.is_cuda() &&
                qw.scalar_type() == proj.scalar_type() && kw.scalar_type() == proj.scalar_type(), "latent_append: norm weights");
  SXE_CHECK(cache.is_cuda() && cache.dim() == 4 && cache.size(1) == 1 && cache.is_contiguous() &&
                cache.scalar_type() == proj.scalar_type() && R >= rank && cache.size(3) >= R + rot_dim,
            "latent_append: cache [blocks, 1, bs, row]");
  SXE_CHECK(slots.is_cuda() && slots.scalar_type() == at::kLong && slots.is_contiguous() && slots.numel() == T, "latent_append: slots");
  SXE_CHECK(rot.is_cuda() && rot.scalar_type() == at::kFloat && rot.is_contiguous() && rot.numel() == T * rot_dim && rot_dim % 2 == 0,
            "latent_append: rotation table");
  auto cq = at::empty({T, q_rank}, proj.options());
  if (T == 0) return cq;
  c10::DeviceGuard g(proj.device());
  lt::AppendArgs a{proj.data_ptr(), proj.stride(0), qw.data_ptr(), kw.data_ptr(), rot.data_ptr<float>(), slots.data_ptr<int64_t>(),
                   cq.data_ptr(), cache.data_ptr(), (int)q_rank, (int)rank, (int)R, (int)rot_dim, (int)cache.size(3),
                   cache.size(0) * cache.size(2), (float)eps};
  const bool vec = q_rank % 8 == 0 && rank % 8 == 0 && proj.stride(0) % 8 == 0 && cache.size(3) % 8 == 0 &&
                   lt::aligned(a.proj, 16) && lt::aligned(a.qw, 16) && lt::aligned(a.kw, 16) && lt::aligned(a.cq, 16) &&
                   lt::aligned(a.cache, 16);
  SXE_DISPATCH_DT(dtype_of(proj), D, {
    if (vec) hipLaunchKernelGGL((lt::latent_append_kernel<D, 8>), dim3(T), dim3(lt::kThreads), 0, cur_stream(), a);
    else hipLaunchKernelGGL((lt::latent_append_kernel<D, 1>), dim3(T), dim3(lt::kThreads), 0, cur_stream(), a);
  });
  SXE_LAUNCH_CHECK();
  return cq;
}

// q [T, H (dim + rot)], uk [H, rank, dim], uv [H, vdim, rank], out [T, H vdim]; rows of `rows` are written
void latent_attention_generic(const at::Tensor& q, const at::Tensor& uk, const at::Tensor& uv, const at::Tensor& cache,
                              const at::Tensor& rot, const at::Tensor& rows, const at::Tensor& table, const at::Tensor& q_start,
                              const at::Tensor& q_len, const at::Tensor& kv_len, at::Tensor out, int64_t rot_dim, int64_t R,
                              double scale, int64_t window) {
  SXE_CHECK_CUDA(q);
  lt::check_batch(rows, table, q_start, q_len, kv_len, cache);
  const int64_t n = rows.size(0), H = uk.size(0), rank = uk.size(1), dim = uk.size(2), vdim = uv.size(1);
  SXE_CHECK(q.is_contiguous() && q.dim() == 2 && q.size(1) == H * (dim + rot_dim) && uk.is_contiguous() && uv.is_contiguous() &&
                uv.size(0) == H && uv.size(2) == rank && out.is_contiguous() && out.size(0) == q.size(0) && out.size(1) == H * vdim &&
                cache.size(3) >= R + rot_dim && R >= rank,
            "latent_attention: shapes");
  SXE_CHECK(rot.is_contiguous() && rot.scalar_type() == at::kFloat && rot.numel() == q.size(0) * rot_dim, "latent_attention: rotation");
  for (const auto* t : {&uk, &uv, &cache, (const at::Tensor*)&out})
    SXE_CHECK(t->is_cuda() && t->scalar_type() == q.scalar_type(), "latent_attention: one dtype");
  if (n == 0) return;
  c10::DeviceGuard g(q.device());
  lt::Args a{q.data_ptr(), rot.data_ptr<float>(), rows.data_ptr<int>(), table.data_ptr<int>(), q_start.data_ptr<int>(),
             q_len.data_ptr<int>(), kv_len.data_ptr<int>(), cache.data_ptr(), cache.size(0), (int)table.size(1), (int)cache.size(2),
             (int)H, (int)dim, (int)rot_dim, (int)rank, (int)R, (int)cache.size(3), (int)vdim, (int)window, (float)scale};
  const size_t lds = sizeof(float) * (2 * rank + rot_dim + lt::kThreads);
  SXE_CHECK(lds <= 150 * 1024 && H <= 65535, "latent_attention: latent of ", rank, " does not fit a workgroup");
  SXE_DISPATCH_DT(dtype_of(q), D, {
    using S = dt_traits<D>::storage;
    SXE_HIP_CHECK(hipFuncSetAttribute((const void*)lt::latent_generic_kernel<D>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    hipLaunchKernelGGL((lt::latent_generic_kernel<D>), dim3(n, H), dim3(lt::kThreads), lds, cur_stream(), a,
                       static_cast<const S*>(uk.data_ptr()), static_cast<const S*>(uv.data_ptr()), static_cast<S*>(out.data_ptr()));
  });
  SXE_LAUNCH_CHECK();
}

// The token form's launches; out [T, H vdim], bf16; cache rows of R = 128 i <= 512 latent and 64 rotated columns
void latent_attention_token(const at::Tensor& q, const at::Tensor& uk, const at::Tensor& uv, const at::Tensor& cache,
                            const at::Tensor& rot, const at::Tensor& rows, const at::Tensor& table, const at::Tensor& q_start,
                            const at::Tensor& q_len, const at::Tensor& kv_len, at::Tensor out, int64_t splits, int64_t rot_dim,
                            int64_t R, double scale, int64_t window) {
  SXE_CHECK_CUDA(q);
  lt::check_batch(rows, table, q_start, q_len, kv_len, cache);
  const int64_t n = rows.size(0), H = uk.size(0), rank = uk.size(1), dim = uk.size(2), vdim = uv.size(1), row = cache.size(3);
  SXE_CHECK(q.is_contiguous() && q.dim() == 2 && q.size(1) == H * (dim + rot_dim) && uk.is_contiguous() && uv.is_contiguous() &&
                uv.size(0) == H && uv.size(2) == rank && out.is_contiguous() && out.size(0) == q.size(0) && out.size(1) == H * vdim &&
                R >= rank && R % 128 == 0 && R <= 512 && row == R + 64 && rot_dim <= 64 && scale > 0 && dim % 8 == 0 && rank % 8 == 0 &&
                rot_dim % 2 == 0 && (dim + rot_dim) % 8 == 0,
            "latent_attention: shapes");
  SXE_CHECK(rot.is_contiguous() && rot.scalar_type() == at::kFloat && rot.numel() == q.size(0) * rot_dim, "latent_attention: rotation");
  for (const auto* t : {&q, &uk, &uv, &cache, (const at::Tensor*)&out})
    SXE_CHECK(t->is_cuda() && t->scalar_type() == at::kBFloat16, "latent_attention: token form takes bf16");
  SXE_CHECK(lt::aligned(cache.data_ptr(), 16) && splits >= 1 && splits <= lt::kMaxSplits && H <= 65535 && n <= 65535, "latent_attention: splits");
  if (n == 0) return;
  c10::DeviceGuard g(q.device());
  lt::Args a{q.data_ptr(), rot.data_ptr<float>(), rows.data_ptr<int>(), table.data_ptr<int>(), q_start.data_ptr<int>(),
             q_len.data_ptr<int>(), kv_len.data_ptr<int>(), cache.data_ptr(), cache.size(0), (int)table.size(1), (int)cache.size(2),
             (int)H, (int)dim, (int)rot_dim, (int)rank, (int)R, (int)row, (int)vdim, (int)window, (float)scale};
  {  // a split's block-table entries fit in LDS
    const int64_t bs = cache.size(2), most = window > 0 ? std::min<int64_t>(window, table.size(1) * bs) : table.size(1) * bs;
    const int64_t per = std::max<int64_t>(1, (lt::kTabMax - 2) * bs / lt::kTok - 1) * lt::kTok;
    splits = std::max(splits, (most + per - 1) / per);
    SXE_CHECK(splits <= lt::kMaxSplits, "latent_attention: ", most, " keys in blocks of ", bs, " are too many");
  }
  SXE_CHECK((n + 15) / 16 <= 65535 && lt::aligned(q.data_ptr(), 16) && lt::aligned(uk.data_ptr(), 16) && lt::aligned(uv.data_ptr(), 16),
            "latent_attention: 16-byte aligned operands");
  auto f32 = q.options().dtype(at::kFloat);
  auto qa = at::empty({n, H, row}, q.options()), po = at::empty({splits, n, H, R}, f32), pml = at::empty({splits, n, H, 2}, f32);
  auto u16 = [](const at::Tensor& t) { return static_cast<unsigned short*>(t.data_ptr()); };
  const unsigned nz = (unsigned)((n + 15) / 16);
  hipLaunchKernelGGL(lt::latent_absorb_kernel, dim3(R / 64 + 1, H, nz), dim3(lt::kThreads), 0, cur_stream(), a, (int)n,
                     (const unsigned short*)u16(uk), u16(qa));
  auto token = [&](auto kern, int PN) {
    const size_t lds = 2 * lt::kTok * (PN * 256 + 128) + 32 * lt::kSRow * sizeof(float) + lt::kTabMax * sizeof(int);
    SXE_HIP_CHECK(hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    hipLaunchKernelGGL(kern, dim3(n, (H + 31) / 32, splits), dim3(64 * lt::kTokWaves), lds, cur_stream(), a, (int)n,
                       (const unsigned short*)u16(qa), po.data_ptr<float>(), pml.data_ptr<float>());
  };
  if (R == 128) token(lt::latent_token_kernel<1>, 1);
  else if (R == 256) token(lt::latent_token_kernel<2>, 2);
  else if (R == 384) token(lt::latent_token_kernel<3>, 3);
  else token(lt::latent_token_kernel<4>, 4);
  const float *ppo = po.data_ptr<float>(), *pm = pml.data_ptr<float>();
  const dim3 eg((vdim + 15) / 16, H, nz);
  if (n == 1) {
    hipLaunchKernelGGL(lt::latent_expand_kernel<true>, eg, dim3(lt::kThreads), 0, cur_stream(), a, (int)n, (int)splits, ppo, pm,
                       (const unsigned short*)nullptr, (const unsigned short*)u16(uv), u16(out));
  } else {
    auto ol = at::empty({n, H, R}, q.options());
    hipLaunchKernelGGL(lt::latent_merge_kernel, dim3(H, n), dim3(128), 0, cur_stream(), a, (int)n, (int)splits, ppo, pm, u16(ol));
    hipLaunchKernelGGL(lt::latent_expand_kernel<false>, eg, dim3(lt::kThreads), 0, cur_stream(), a, (int)n, (int)splits, ppo, pm,
                       (const unsigned short*)u16(ol), (const unsigned short*)u16(uv), u16(out));
  }
  SXE_LAUNCH_CHECK();
}

// chunks int32 [n, 3]: (sequence, first row, rows <= kQ); kv [Nk, H (dim + vdim)]: all heads' keys, then all heads' values; lat [Nk, row]: the cache rows they come from
void latent_attention_tile(const at::Tensor& q, const at::Tensor& kv, const at::Tensor& lat, const at::Tensor& rot,
                           const at::Tensor& chunks, int64_t size, const at::Tensor& first, const at::Tensor& q_start,
                           const at::Tensor& q_len, const at::Tensor& kv_len, at::Tensor out, int64_t H, int64_t dim, int64_t rot_dim, int64_t vdim, int64_t R,
                           double scale, int64_t window) {
  SXE_CHECK_CUDA(q);
  const int64_t S = q_start.numel(), nc = chunks.size(0), Nk = kv.size(0);
  for (const auto* t : {&q, &kv, &lat, (const at::Tensor*)&out})
    SXE_CHECK(t->is_cuda() && t->scalar_type() == at::kBFloat16 && t->is_contiguous() && t->dim() == 2 && lt::aligned(t->data_ptr(), 16),
              "latent_attention: tile form takes bf16 rows");
  SXE_CHECK(dim <= 128 && vdim <= 128 && rot_dim <= 64 && dim % 8 == 0 && vdim % 8 == 0 && rot_dim % 8 == 0 &&
                q.size(1) == H * (dim + rot_dim) && kv.size(1) == H * (dim + vdim) && lat.size(0) == Nk && lat.size(1) >= R + rot_dim &&
                R % 8 == 0 && lat.size(1) % 8 == 0 && out.size(0) == q.size(0) && out.size(1) == H * vdim,
            "latent_attention: tile form shapes");
  SXE_CHECK(chunks.is_cuda() && chunks.scalar_type() == at::kInt && chunks.is_contiguous() && chunks.dim() == 2 && chunks.size(1) == 3 &&
                size == lt::kQ && first.is_cuda() && first.scalar_type() == at::kInt && first.is_contiguous() && first.numel() == 2 * S,
            "latent_attention: tables");
  for (const auto* t : {&q_start, &q_len, &kv_len})
    SXE_CHECK(t->is_cuda() && t->is_contiguous() && t->scalar_type() == at::kInt && t->numel() == S, "latent_attention: int32 [S]");
  SXE_CHECK(rot.is_contiguous() && rot.scalar_type() == at::kFloat && rot.numel() == q.size(0) * rot_dim, "latent_attention: rotation");
  if (nc == 0 || Nk == 0) return;
  SXE_CHECK(nc <= 65535, "latent_attention: chunks");
  c10::DeviceGuard g(q.device());
  auto u16 = [](const at::Tensor& t) { return static_cast<unsigned short*>(t.data_ptr()); };
  lt::TileArgs a{u16(q), u16(kv), u16(lat), rot.data_ptr<float>(), chunks.data_ptr<int>(), first.data_ptr<int>(), q_start.data_ptr<int>(),
                 q_len.data_ptr<int>(), kv_len.data_ptr<int>(), u16(out), kv.stride(0), (int)H, (int)dim, (int)rot_dim, (int)vdim, (int)R,
                 (int)lat.size(1), (int)window, (int)Nk, (float)scale};
  auto go = [&](auto kern, int DN, int VP) {
    const size_t lds = 2 * lt::kKeys * (2 * DN + 128 + 2 * VP);
    SXE_HIP_CHECK(hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    hipLaunchKernelGGL(kern, dim3(H, nc), dim3(64 * lt::kTileWaves), lds, cur_stream(), a);
  };
  if (dim <= 64 && vdim <= 64) go(lt::latent_tile_kernel<64, 64>, 64, 64);
  else if (dim <= 64) go(lt::latent_tile_kernel<64, 128>, 64, 128);
  else if (vdim <= 64) go(lt::latent_tile_kernel<128, 64>, 128, 64);
  else go(lt::latent_tile_kernel<128, 128>, 128, 128);
  SXE_LAUNCH_CHECK();
}

}  // namespace sxe

TORCH_LIBRARY_FRAGMENT(sxe, m) {
  m.def("rotation_table(Tensor positions, int dims, float base) -> Tensor");
  m.def("latent_append(Tensor proj, Tensor qw, Tensor kw, Tensor(a!) cache, Tensor slots, Tensor rot, int q_rank, int rank, int R, "
        "int rot_dim, float eps) -> Tensor");
  m.def("latent_attention_generic(Tensor q, Tensor uk, Tensor uv, Tensor cache, Tensor rot, Tensor rows, Tensor table, "
        "Tensor q_start, Tensor q_len, Tensor kv_len, Tensor(a!) out, int rot_dim, int R, float scale, int window) -> ()");
  m.def("latent_attention_token(Tensor q, Tensor uk, Tensor uv, Tensor cache, Tensor rot, Tensor rows, Tensor table, "
        "Tensor q_start, Tensor q_len, Tensor kv_len, Tensor(a!) out, int splits, int rot_dim, int R, float scale, int window) -> ()");
  m.def("latent_attention_tile(Tensor q, Tensor kv, Tensor lat, Tensor rot, Tensor chunks, int size, Tensor first, Tensor q_start, "
        "Tensor q_len, Tensor kv_len, Tensor(a!) out, int H, int dim, int rot_dim, int vdim, int R, float scale, int window) -> ()");
}
TORCH_LIBRARY_IMPL(sxe, CUDA, m) {
  m.impl("rotation_table", &sxe::rotation_table);
  m.impl("latent_append", &sxe::latent_append);
  m.impl("latent_attention_generic", &sxe::latent_attention_generic);
  m.impl("latent_attention_token", &sxe::latent_attention_token);
  m.impl("latent_attention_tile", &sxe::latent_attention_tile);
}
