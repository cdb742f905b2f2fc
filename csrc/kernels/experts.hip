// Routed experts without a host synchronisation (gfx950): routing, expert-sorted row lists, expert products.
//
//  * route_logits: h . router^T in fp32. bf16 operands go through the matrix cores (products of two bf16
//    numbers are exact in fp32 and the accumulation is fp32), anything else through a plain fp32 kernel.
//    One to four tokens: the norm that produces h is the kernel's prologue (sxe_sandwich.h).
//  * route_top: the k largest logits of a token (lowest index first among equals) and the softmax over them.
//  * lists: (token, choice) assignments sorted by expert: row -> token, row -> weight, (token, choice) -> row,
//    expert offsets and the experts that have rows. A row's place inside its expert depends on the order of
//    atomics, its result does not.
//  * expert_gemm: y[r] = weight[r] * act(x[token(r)] . W[e]^T) for rows sorted by expert.
//      skinny form (bf16, few rows per expert): one workgroup per (expert with rows, 16 columns) streams the
//      expert's weight rows once per 16 rows, K split over its waves;
//      generic form: any size and dtype, fp32 accumulation.
//    Many rows per expert: grouped_gemm.hip.
#include "sxe_common.h"
#include "sxe_mfma.h"
#include "sxe_sandwich.h"
#include <torch/library.h>

namespace sxe {
namespace ex {
using namespace mf;

enum : int { ACT_NONE = 0, ACT_RELU2 = 1, ACT_SILU = 2 };

__device__ __forceinline__ float apply_act(float x, int act) {
  if (act == ACT_RELU2) {
    x = fmaxf(x, 0.f);
    return x * x;
  }
  return act == ACT_SILU ? x / (1.f + expf(-x)) : x;
}

// ---------------------------------------------------------------------------------------------- routing
// grid (ceil(T / 32), ceil(E / 32)), NW waves share K; K % 16 == 0, 16-byte aligned rows
template <int NW>
__global__ __launch_bounds__(64 * NW) void route_logits_kernel(const unsigned short* __restrict x, int64_t ldx,
                                                               const unsigned short* __restrict w, int T, int E, int K,
                                                               float* __restrict z) {
  __shared__ float part[NW][32][33];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l32 = lane & 31, hh = lane >> 5;
  const int t0 = blockIdx.x * 32, e0 = blockIdx.y * 32;
  const unsigned short* xr = x + (int64_t)min(t0 + l32, T - 1) * ldx + 8 * hh;
  const unsigned short* wr = w + (int64_t)min(e0 + l32, E - 1) * K + 8 * hh;
  f32x16 acc = zero16();
  constexpr int U = 8;
  for (int k0 = wave * U * 16; k0 < K; k0 += NW * U * 16) {
    u32x4 a[U], b[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = k0 + u * 16;
      a[u] = b[u] = u32x4{0u, 0u, 0u, 0u};
      if (k < K) {
        a[u] = *reinterpret_cast<const u32x4*>(xr + k);
        b[u] = *reinterpret_cast<const u32x4*>(wr + k);
      }
    }
#pragma unroll
    for (int u = 0; u < U; ++u) acc = mfma(__builtin_bit_cast(bf16x8, a[u]), __builtin_bit_cast(bf16x8, b[u]), acc);
  }
#pragma unroll
  for (int i = 0; i < 16; ++i) part[wave][acc_row(i, hh)][l32] = acc[i];
  __syncthreads();
  for (int i = threadIdx.x; i < 1024; i += 64 * NW) {
    const int t = i >> 5, e = i & 31;
    if (t0 + t >= T || e0 + e >= E) continue;
    float s = 0.f;
#pragma unroll
    for (int q = 0; q < NW; ++q) s += part[q][t][e];
    z[(int64_t)(t0 + t) * E + e0 + e] = s;
  }
}

// one wave per (token, expert)
template <DT T>
__global__ __launch_bounds__(256) void route_logits_generic_kernel(const typename dt_traits<T>::storage* __restrict x, int64_t ldx,
                                                                   const typename dt_traits<T>::storage* __restrict w, int E, int K,
                                                                   float* __restrict z) {
  const int t = blockIdx.x, e = blockIdx.y * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (e >= E) return;
  float s = 0.f;
  for (int k = lane; k < K; k += 64) s += to_f32<T>(x[t * ldx + k]) * to_f32<T>(w[(int64_t)e * K + k]);
  s = wave_sum(s);
  if (lane == 0) z[(int64_t)t * E + e] = s;
}

// few tokens, bf16, K % 8 == 0, 16-byte aligned rows: 16 tokens x 16 experts per workgroup, 16 waves share K in
// super-steps of 256 whose loads are all in flight together. grid (ceil(E / 16), ceil(T / 16))
__global__ __launch_bounds__(1024) void route_logits_few_kernel(const unsigned short* __restrict x, int64_t ldx,
                                                                const unsigned short* __restrict w, int T, int E, int K,
                                                                float* __restrict z) {
  __shared__ float part[16][16][17];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l16 = lane & 15, g = lane >> 4;
  const int e0 = blockIdx.x * 16, t0 = blockIdx.y * 16;
  const unsigned short* xr = x + (int64_t)min(t0 + l16, T - 1) * ldx + 8 * g;
  const unsigned short* wr = w + (int64_t)min(e0 + l16, E - 1) * K + 8 * g;
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
  for (int k0 = wave * 256; k0 < K; k0 += 16 * 256) {
    u32x4 a[8], b[8];
#pragma unroll
    for (int u = 0; u < 8; ++u) {
      const int k = k0 + u * 32;
      a[u] = b[u] = u32x4{0u, 0u, 0u, 0u};
      if (k + 8 * g < K) {
        a[u] = *reinterpret_cast<const u32x4*>(xr + k);
        b[u] = *reinterpret_cast<const u32x4*>(wr + k);
      }
    }
#pragma unroll
    for (int u = 0; u < 8; ++u)
      acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a[u]), __builtin_bit_cast(bf16x8, b[u]), acc, 0, 0, 0);
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) part[wave][4 * g + i][l16] = acc[i];
  __syncthreads();
  const int t = threadIdx.x >> 4, e = threadIdx.x & 15;
  if (threadIdx.x < 256 && t0 + t < T && e0 + e < E) {
    float s = 0.f;
#pragma unroll
    for (int q = 0; q < 16; ++q) s += part[q][t][e];
    z[(int64_t)(t0 + t) * E + e0 + e] = s;
  }
}

// decode: h is built by every workgroup (norms around the residual sum) and written, with the sum, by the first;
// one wave per expert. grid (ceil(E / 8)); M <= 4 rows
__global__ __launch_bounds__(512) void route_sandwich_kernel(sw::Args a, const unsigned short* __restrict w, int M, int E, int K,
                                                             unsigned short* __restrict h, float* __restrict z) {
  extern __shared__ __attribute__((aligned(16))) unsigned short act[];  // [M][K]
  __shared__ float red[8][sw::kMaxM], rinv[sw::kMaxM];
  const int e = blockIdx.x * 8 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  const unsigned short* wr = w + (int64_t)min(e, E - 1) * K;
  constexpr int U = 8;  // router chunks in flight across the prologue
  u16x8 wv[U];
#pragma unroll
  for (int u = 0; u < U; ++u) {
    const int c = u * 512 + lane * 8;
    wv[u] = *reinterpret_cast<const u16x8*>(wr + (c < K ? c : 0));
  }
  sw::build<512, 2, true>(a, M, K, blockIdx.x == 0, act, rinv, red);
  if (blockIdx.x == 0)
    for (int i = threadIdx.x * 8; i < M * K; i += 512 * 8) *reinterpret_cast<u16x8*>(h + i) = *reinterpret_cast<u16x8*>(act + i);
  if (e >= E) return;
  float s[sw::kMaxM] = {0.f, 0.f, 0.f, 0.f};
  auto add = [&](const u16x8& wc, int c) {
#pragma unroll
    for (int m = 0; m < sw::kMaxM; ++m) {
      if (m >= M) break;
      float b[8];
      load8<DT::BF16>(act + m * K + c, b);
#pragma unroll
      for (int i = 0; i < 8; ++i) s[m] += bf16_to_f32(wc[i]) * b[i];
    }
  };
#pragma unroll
  for (int u = 0; u < U; ++u)
    if (u * 512 + lane * 8 < K) add(wv[u], u * 512 + lane * 8);
  for (int c = U * 512 + lane * 8; c < K; c += 512) add(*reinterpret_cast<const u16x8*>(wr + c), c);
#pragma unroll
  for (int m = 0; m < sw::kMaxM; ++m) {
    const float v = wave_sum(s[m]);
    if (lane == 0 && m < M) z[(int64_t)m * E + e] = v;
  }
}

constexpr int kMaxE = 1024;

// the k largest of a token's logits and their softmax weights, by one wave
__device__ __forceinline__ void route_top(const float* __restrict z, int t, int E, int k, int* idx, float* wt) {
  const int lane = threadIdx.x & 63;
  constexpr int N = kMaxE / 64;
  float v[N];
#pragma unroll
  for (int i = 0; i < N; ++i) v[i] = lane + 64 * i < E ? z[(int64_t)t * E + lane + 64 * i] : -INFINITY;
  float top = 0.f, sum = 0.f;
  for (int j = 0; j < k; ++j) {
    float b = -INFINITY;
    int bi = kMaxE;
#pragma unroll
    for (int i = 0; i < N; ++i)
      if (v[i] > b) {
        b = v[i];
        bi = lane + 64 * i;
      }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ob = __shfl_xor(b, o, 64);
      const int oi = __shfl_xor(bi, o, 64);
      if (ob > b || (ob == b && oi < bi)) {
        b = ob;
        bi = oi;
      }
    }
    bi = min(bi, E - 1);  // nothing comparable left (not-a-number logits): still a valid expert
#pragma unroll
    for (int i = 0; i < N; ++i)
      if (lane + 64 * i == bi) v[i] = -INFINITY;
    if (j == 0) top = b;
    const float e = expf(b - top);
    sum += e;
    if (lane == (j & 63)) {  // the lane that divides by the sum below
      idx[(int64_t)t * k + j] = bi;
      wt[(int64_t)t * k + j] = e;
    }
  }
  for (int j = lane; j < k; j += 64) wt[(int64_t)t * k + j] /= sum;
}

// one wave per token, 4 waves per workgroup
__global__ __launch_bounds__(256) void route_top_kernel(const float* __restrict z, int T, int E, int k, int* __restrict idx,
                                                        float* __restrict wt) {
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (t < T) route_top(z, t, E, k, idx, wt);
}

// ------------------------------------------------------------------------------------------------ lists
constexpr int kListThreads = 1024;

// R <= kListThreads: everything in one workgroup; z (logits of R / k tokens) or null: choose the experts first
__global__ __launch_bounds__(kListThreads) void moe_lists_small_kernel(const float* __restrict z, int* expert, float* wt, int R,
                                                                       int k, int E, int* __restrict token, float* __restrict ws,
                                                                       int* __restrict slots, int* __restrict offs,
                                                                       int* __restrict active) {
  __shared__ int cnt[kMaxE], off[kMaxE + 1];
  __shared__ int se[kListThreads];
  __shared__ float sw_[kListThreads];
  const int i = threadIdx.x;
  for (int e = i; e < E; e += kListThreads) cnt[e] = 0;
  if (z != nullptr)
    for (int t = i >> 6; t < R / k; t += kListThreads / 64) route_top(z, t, E, k, se, sw_);
  __syncthreads();
  int e = 0, rank = 0;
  float w = 0.f;
  if (i < R) {
    if (z != nullptr) {
      expert[i] = se[i];
      wt[i] = sw_[i];
    }
    e = z != nullptr ? se[i] : min(max(expert[i], 0), E - 1);
    w = z != nullptr ? sw_[i] : wt[i];
    rank = atomicAdd(&cnt[e], 1);
  }
  __syncthreads();
  if (i < 64) {  // one wave scans the counts, 64 at a time
    int base = 0, na = 0;
    for (int e0 = 0; e0 < E; e0 += 64) {
      const int c = e0 + i < E ? cnt[e0 + i] : 0;
      int s = c;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const int u = __shfl_up(s, o, 64);
        if (i >= o) s += u;
      }
      const unsigned long long m = __ballot(c > 0);
      if (e0 + i < E) {
        off[e0 + i] = base + s - c;
        if (c > 0) active[1 + na + __popcll(m & ((1ull << i) - 1))] = e0 + i;
      }
      base += __shfl(s, 63, 64);
      na += __popcll(m);
    }
    if (i == 0) {
      off[E] = base;
      active[0] = na;
    }
  }
  __syncthreads();
  for (int x = i; x <= E; x += kListThreads) offs[x] = off[x];
  if (i < R) {
    const int r = off[e] + rank;
    token[r] = i / k;
    ws[r] = w;
    slots[i] = r;
  }
}

// counts zeroed; slots receives the rank of an assignment inside its expert
__global__ __launch_bounds__(kListThreads) void moe_rank_kernel(const int* __restrict expert, int R, int E, int* __restrict counts,
                                                                int* __restrict slots) {
  __shared__ int cnt[kMaxE], base[kMaxE];
  const int i = blockIdx.x * kListThreads + threadIdx.x;
  for (int e = threadIdx.x; e < E; e += kListThreads) cnt[e] = 0;
  __syncthreads();
  int e = 0, rank = 0;
  if (i < R) {
    e = min(max(expert[i], 0), E - 1);
    rank = atomicAdd(&cnt[e], 1);
  }
  __syncthreads();
  for (int x = threadIdx.x; x < E; x += kListThreads) base[x] = cnt[x] ? atomicAdd(&counts[x], cnt[x]) : 0;
  __syncthreads();
  if (i < R) slots[i] = base[e] + rank;
}

__global__ __launch_bounds__(kListThreads) void moe_place_kernel(const int* __restrict expert, const float* __restrict wt, int R, int k,
                                                                 int E, const int* __restrict counts, int* __restrict token,
                                                                 float* __restrict ws, int* __restrict slots, int* __restrict offs,
                                                                 int* __restrict active) {
  __shared__ int off[kMaxE + 1];
  const int tid = threadIdx.x, i = blockIdx.x * kListThreads + tid;
  if (tid < 64) {
    int base = 0, na = 0;
    for (int e0 = 0; e0 < E; e0 += 64) {
      const int c = e0 + tid < E ? counts[e0 + tid] : 0;
      int s = c;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const int u = __shfl_up(s, o, 64);
        if (tid >= o) s += u;
      }
      const unsigned long long m = __ballot(c > 0);
      if (e0 + tid < E) {
        off[e0 + tid] = base + s - c;
        if (c > 0 && blockIdx.x == 0) active[1 + na + __popcll(m & ((1ull << tid) - 1))] = e0 + tid;
      }
      base += __shfl(s, 63, 64);
      na += __popcll(m);
    }
    if (tid == 0) {
      off[E] = base;
      if (blockIdx.x == 0) active[0] = na;
    }
  }
  __syncthreads();
  if (blockIdx.x == 0)
    for (int x = tid; x <= E; x += kListThreads) offs[x] = off[x];
  if (i < R) {
    const int e = min(max(expert[i], 0), E - 1), r = off[e] + slots[i];
    token[r] = i / k;
    ws[r] = wt[i];
    slots[i] = r;
  }
}

// ------------------------------------------------------------------------------------- expert products
struct GemmArgs {
  const void *x, *w;        // x [rows, ldx]; w [E, N, K]
  int64_t ldx;
  const int *offs, *active, *token;  // token: row -> row of x, or nullptr (row itself)
  const float* ws;          // row scale or nullptr
  void* y;                  // [R, N]
  int R, E, N, K, Tx, act;  // Tx: rows of x
};

__device__ __forceinline__ f32x4 mfma16(bf16x8 a, bf16x8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}

// the expert of a workgroup and its rows; false: nothing to do (uniform)
__device__ __forceinline__ bool expert_rows(const GemmArgs& a, int i, int& e, int& lo, int& hi) {
  if (i >= a.active[0]) return false;
  e = a.active[1 + i];
  lo = a.offs[e];
  hi = min(a.offs[e + 1], a.R);
  return lo >= 0 && lo < hi;
}

// grid (ceil(N / 16), experts that may have rows); NW waves split K in super-steps of 256; K % 8 == 0.
// MB blocks of 16 rows share a pass over the weights.
template <int NW, int MB>
__global__ __launch_bounds__(64 * NW) void expert_skinny_kernel(GemmArgs a) {
  __shared__ float part[NW][MB][16][17];
  int e, lo, hi;
  if (!expert_rows(a, blockIdx.y, e, lo, hi)) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l16 = lane & 15, g = lane >> 4, n0 = blockIdx.x * 16;
  const unsigned short* w = static_cast<const unsigned short*>(a.w) + ((int64_t)e * a.N + min(n0 + l16, a.N - 1)) * a.K + 8 * g;
  const unsigned short* x = static_cast<const unsigned short*>(a.x);
  constexpr int U = 8;
  for (int r0 = lo; r0 < hi; r0 += 16 * MB) {
    const unsigned short* xr[MB];
#pragma unroll
    for (int m = 0; m < MB; ++m) {
      const int r = min(r0 + 16 * m + l16, hi - 1);
      const int tr = a.token != nullptr ? min(max(a.token[r], 0), a.Tx - 1) : r;
      xr[m] = x + (int64_t)tr * a.ldx + 8 * g;
    }
    f32x4 acc[MB];
#pragma unroll
    for (int m = 0; m < MB; ++m) acc[m] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int k0 = wave * 256; k0 < a.K; k0 += NW * 256) {
      u32x4 wf[U], xf[MB][U];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int k = k0 + u * 32;
        wf[u] = u32x4{0u, 0u, 0u, 0u};
        if (k + 8 * g < a.K) wf[u] = *reinterpret_cast<const u32x4*>(w + k);
#pragma unroll
        for (int m = 0; m < MB; ++m) {
          xf[m][u] = u32x4{0u, 0u, 0u, 0u};
          if (k + 8 * g < a.K) xf[m][u] = *reinterpret_cast<const u32x4*>(xr[m] + k);
        }
      }
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int m = 0; m < MB; ++m)
          acc[m] = mfma16(__builtin_bit_cast(bf16x8, xf[m][u]), __builtin_bit_cast(bf16x8, wf[u]), acc[m]);
    }
    if (r0 != lo) __syncthreads();  // the previous pass's sums are read
#pragma unroll
    for (int m = 0; m < MB; ++m)
#pragma unroll
      for (int i = 0; i < 4; ++i) part[wave][m][4 * g + i][l16] = acc[m][i];
    __syncthreads();
    for (int i = threadIdx.x; i < MB * 256; i += 64 * NW) {
      const int m = i >> 8, rr = (i >> 4) & 15, c = i & 15, r = r0 + 16 * m + rr;
      if (r >= hi || n0 + c >= a.N) continue;
      float s = 0.f;
#pragma unroll
      for (int q = 0; q < NW; ++q) s += part[q][m][rr][c];
      s = apply_act(s, a.act);
      if (a.ws != nullptr) s *= a.ws[r];
      static_cast<unsigned short*>(a.y)[(int64_t)r * a.N + n0 + c] = f32_to_bf16(s);
    }
  }
}

// grid (ceil(N / 64), experts that may have rows, row tiles): 16 rows x 64 columns per pass
template <DT T>
__global__ __launch_bounds__(256) void expert_generic_kernel(GemmArgs a) {
  using S = typename dt_traits<T>::storage;
  __shared__ float sx[16][33], sw[64][33];
  int e, lo, hi;
  if (!expert_rows(a, blockIdx.y, e, lo, hi)) return;
  const int n0 = blockIdx.x * 64, c = threadIdx.x & 63, rq = threadIdx.x >> 6;  // thread: column c, rows rq + 4 i
  const S *x = static_cast<const S*>(a.x), *w = static_cast<const S*>(a.w) + (int64_t)e * a.N * a.K;
  for (int r0 = lo + blockIdx.z * 16; r0 < hi; r0 += gridDim.z * 16) {
    float acc[4] = {0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < a.K; k0 += 32) {
      for (int i = threadIdx.x; i < 16 * 32; i += 256) {
        const int r = r0 + (i >> 5), k = k0 + (i & 31);
        float v = 0.f;
        if (r < hi && k < a.K) {
          const int tr = a.token != nullptr ? min(max(a.token[r], 0), a.Tx - 1) : r;
          v = to_f32<T>(x[(int64_t)tr * a.ldx + k]);
        }
        sx[i >> 5][i & 31] = v;
      }
      for (int i = threadIdx.x; i < 64 * 32; i += 256) {
        const int n = n0 + (i >> 5), k = k0 + (i & 31);
        sw[i >> 5][i & 31] = n < a.N && k < a.K ? to_f32<T>(w[(int64_t)n * a.K + k]) : 0.f;
      }
      __syncthreads();
#pragma unroll
      for (int k = 0; k < 32; ++k) {
        const float wv = sw[c][k];
#pragma unroll
        for (int i = 0; i < 4; ++i) acc[i] += sx[rq + 4 * i][k] * wv;
      }
      __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int r = r0 + rq + 4 * i;
      if (r < hi && n0 + c < a.N) {
        float s = apply_act(acc[i], a.act);
        if (a.ws != nullptr) s *= a.ws[r];
        static_cast<S*>(a.y)[(int64_t)r * a.N + n0 + c] = from_f32<T>(s);
      }
    }
  }
}

inline bool aligned(const void* p, size_t n) { return reinterpret_cast<uintptr_t>(p) % n == 0; }

}  // namespace ex

namespace ex {

void route_logits(const at::Tensor& h, const at::Tensor& router, at::Tensor& z) {
  SXE_CHECK(h.dim() == 2 && h.stride(1) == 1 && router.dim() == 2 && router.is_contiguous() && router.is_cuda() &&
                router.size(1) == h.size(1) && router.scalar_type() == h.scalar_type(), "route: h [T, K], router [E, K]");
  const int64_t T = h.size(0), K = h.size(1), E = router.size(0);
  SXE_CHECK(E > 0 && E <= kMaxE && T < (1ll << 31), "route: up to ", kMaxE, " experts");
  const bool vec = h.scalar_type() == at::kBFloat16 && h.stride(0) % 8 == 0 && aligned(h.data_ptr(), 16) && aligned(router.data_ptr(), 16);
  auto u16 = [](const at::Tensor& t) { return static_cast<const unsigned short*>(t.data_ptr()); };
  if (vec && K % 8 == 0 && T <= 256) {
    hipLaunchKernelGGL(route_logits_few_kernel, dim3((E + 15) / 16, (T + 15) / 16), dim3(1024), 0, cur_stream(), u16(h), h.stride(0),
                       u16(router), (int)T, (int)E, (int)K, z.data_ptr<float>());
  } else if (vec && K % 16 == 0) {
    hipLaunchKernelGGL(route_logits_kernel<4>, dim3((T + 31) / 32, (E + 31) / 32), dim3(256), 0, cur_stream(), u16(h), h.stride(0),
                       u16(router), (int)T, (int)E, (int)K, z.data_ptr<float>());
  } else {
    SXE_DISPATCH_DT(dtype_of(h), D, {
      using S = dt_traits<D>::storage;
      hipLaunchKernelGGL((route_logits_generic_kernel<D>), dim3(T, (E + 3) / 4), dim3(256), 0, cur_stream(),
                         static_cast<const S*>(h.data_ptr()), h.stride(0), static_cast<const S*>(router.data_ptr()), (int)E, (int)K,
                         z.data_ptr<float>());
    });
  }
}

// logits [T, E] -> [expert int32 [T, k], weight fp32 [T, k], token int32 [R], weight fp32 [R], slots int32 [T, k],
// offsets int32 [E + 1], active int32 [1 + E] (count, then the experts that have rows)]
std::vector<at::Tensor> choose(const at::Tensor& z, int64_t k) {
  const int64_t T = z.size(0), E = z.size(1), R = T * k;
  SXE_CHECK(k > 0 && k <= E && R < (1ll << 31), "route: top ", k, " of ", E);
  auto io = z.options().dtype(at::kInt);
  auto idx = at::empty({T, k}, io), token = at::empty({R}, io), slots = at::empty({T, k}, io), offs = at::empty({E + 1}, io),
       active = at::empty({E + 1}, io);
  auto wt = at::empty({T, k}, z.options()), ws = at::empty({R}, z.options());
  if (R == 0) return {idx, wt, token, ws, slots, offs, active};
  const bool small = R <= kListThreads, one = small && T <= 16;  // one: a wave per token chooses in the same workgroup
  if (!one)
    hipLaunchKernelGGL(route_top_kernel, dim3((T + 3) / 4), dim3(256), 0, cur_stream(), z.data_ptr<float>(), (int)T, (int)E, (int)k,
                       idx.data_ptr<int>(), wt.data_ptr<float>());
  if (small) {
    hipLaunchKernelGGL(moe_lists_small_kernel, dim3(1), dim3(kListThreads), 0, cur_stream(), one ? z.data_ptr<float>() : nullptr,
                       idx.data_ptr<int>(), wt.data_ptr<float>(), (int)R, (int)k, (int)E, token.data_ptr<int>(), ws.data_ptr<float>(),
                       slots.data_ptr<int>(), offs.data_ptr<int>(), active.data_ptr<int>());
  } else {
    auto counts = at::empty({E}, io);
    counts.zero_();
    const dim3 grid((R + kListThreads - 1) / kListThreads);
    hipLaunchKernelGGL(moe_rank_kernel, grid, dim3(kListThreads), 0, cur_stream(), idx.data_ptr<int>(), (int)R, (int)E,
                       counts.data_ptr<int>(), slots.data_ptr<int>());
    hipLaunchKernelGGL(moe_place_kernel, grid, dim3(kListThreads), 0, cur_stream(), idx.data_ptr<int>(), wt.data_ptr<float>(), (int)R,
                       (int)k, (int)E, counts.data_ptr<int>(), token.data_ptr<int>(), ws.data_ptr<float>(), slots.data_ptr<int>(),
                       offs.data_ptr<int>(), active.data_ptr<int>());
  }
  return {idx, wt, token, ws, slots, offs, active};
}

}  // namespace ex

// h [T, K], router [E, K] -> the chosen experts, their weights and the expert-sorted lists (ex::choose)
std::vector<at::Tensor> route_topk(const at::Tensor& h, const at::Tensor& router, int64_t k) {
  SXE_CHECK_CUDA(h);
  c10::DeviceGuard g(h.device());
  auto z = at::empty({h.size(0), router.size(0)}, h.options().dtype(at::kFloat));
  if (h.size(0) > 0) ex::route_logits(h, router, z);
  auto out = ex::choose(z, k);
  SXE_LAUNCH_CHECK();
  return out;
}

// Decode: v = x + rms(y) wp [+ add], h = rms(v) wn, then route_topk(h). Returns [v fp32 [M, K], h bf16 [M, K], route_topk's].
std::vector<at::Tensor> route_sandwich(const at::Tensor& x, const at::Tensor& y, const at::Tensor& wp, const at::Tensor& wn,
                                       const c10::optional<at::Tensor>& slots, const c10::optional<at::Tensor>& add, double eps,
                                       const at::Tensor& router, int64_t k) {
  SXE_CHECK_CUDA(x);
  SXE_CHECK(x.scalar_type() == at::kFloat && x.dim() == 2 && x.is_contiguous(), "route_sandwich: x fp32 [M, K]");
  const int64_t M = x.size(0), K = x.size(1), E = router.size(0);
  SXE_CHECK(M >= 1 && M <= sw::kMaxM && K % 8 == 0 && M * K <= 2 * 8 * 512, "route_sandwich: up to 4 rows, M K <= 8192");
  const bool has_s = slots.has_value() && slots->defined(), has_a = add.has_value() && add->defined();
  SXE_CHECK(y.is_cuda() && y.scalar_type() == at::kBFloat16 && y.dim() == 2 && y.is_contiguous() && y.size(1) == K &&
                (has_s || y.size(0) == M), "route_sandwich: y bf16 [M, K]");
  for (const auto* p : {&wp, &wn})
    SXE_CHECK(p->is_cuda() && p->scalar_type() == at::kBFloat16 && p->is_contiguous() && p->numel() == K, "route_sandwich: norms");
  SXE_CHECK(router.is_cuda() && router.scalar_type() == at::kBFloat16 && router.is_contiguous() && router.dim() == 2 &&
                router.size(1) == K && E > 0 && E <= ex::kMaxE, "route_sandwich: router bf16 [E, K]");
  if (has_s)
    SXE_CHECK(slots->is_cuda() && slots->scalar_type() == at::kInt && slots->is_contiguous() && slots->dim() == 2 &&
                  slots->size(0) == M && slots->numel() <= y.size(0), "route_sandwich: slots int32 [M, k]");
  if (has_a)
    SXE_CHECK(add->is_cuda() && add->scalar_type() == at::kFloat && add->is_contiguous() && add->sizes() == x.sizes(),
              "route_sandwich: add like x");
  for (const void* q : {(const void*)x.data_ptr(), (const void*)y.data_ptr(), (const void*)wp.data_ptr(), (const void*)wn.data_ptr(),
                        (const void*)router.data_ptr(), has_a ? (const void*)add->data_ptr() : nullptr})
    SXE_CHECK(ex::aligned(q, 16), "route_sandwich: 16-byte aligned operands");
  c10::DeviceGuard g(x.device());
  auto v = at::empty_like(x), h = at::empty({M, K}, y.options()), z = at::empty({M, E}, x.options());
  auto u16 = [](const at::Tensor& t) { return static_cast<unsigned short*>(t.data_ptr()); };
  sw::Args a{u16(y), u16(wp), u16(wn), x.data_ptr<float>(), has_a ? add->data_ptr<float>() : nullptr,
             has_s ? slots->data_ptr<int>() : nullptr, has_s ? (int)slots->size(1) : 1, (float)eps, v.data_ptr<float>()};
  hipLaunchKernelGGL(ex::route_sandwich_kernel, dim3((E + 7) / 8), dim3(512), M * K * 2, cur_stream(), a, (const unsigned short*)u16(router),
                     (int)M, (int)E, (int)K, u16(h), z.data_ptr<float>());
  std::vector<at::Tensor> out{v, h};
  for (auto& t : ex::choose(z, k)) out.push_back(t);
  SXE_LAUNCH_CHECK();
  return out;
}

// x [Tx, K], w [E, N, K]; rows sorted by expert (offs, active of ex::choose); token int32 [R] or None (x has R rows);
// ws fp32 [R] or None -> [R, N]
at::Tensor expert_gemm(const at::Tensor& x, const at::Tensor& w, const at::Tensor& offs, const at::Tensor& active,
                       const c10::optional<at::Tensor>& token, const c10::optional<at::Tensor>& ws, int64_t R, int64_t act) {
  SXE_CHECK_CUDA(x);
  SXE_CHECK(x.dim() == 2 && x.stride(1) == 1 && w.dim() == 3 && w.is_contiguous() && w.is_cuda() && w.size(2) == x.size(1) &&
                w.scalar_type() == x.scalar_type(), "expert_gemm: x [T, K], w [E, N, K]");
  const int64_t E = w.size(0), N = w.size(1), K = w.size(2);
  const bool has_t = token.has_value() && token->defined(), has_w = ws.has_value() && ws->defined();
  for (const auto* t : {&offs, &active})
    SXE_CHECK(t->is_cuda() && t->is_contiguous() && t->scalar_type() == at::kInt && t->numel() == E + 1, "expert_gemm: lists int32 [E + 1]");
  if (has_t) {
    SXE_CHECK(token->is_cuda() && token->is_contiguous() && token->scalar_type() == at::kInt && token->numel() == R, "expert_gemm: token");
  } else {
    SXE_CHECK(x.size(0) == R, "expert_gemm: x [R, K]");
  }
  if (has_w)
    SXE_CHECK(ws->is_cuda() && ws->is_contiguous() && ws->scalar_type() == at::kFloat && ws->numel() == R, "expert_gemm: weights");
  SXE_CHECK(R < (1ll << 31) && act >= 0 && act <= 2, "expert_gemm: sizes");
  auto y = at::empty({R, N}, x.options());
  if (R == 0 || N == 0) return y;
  c10::DeviceGuard g(x.device());
  ex::GemmArgs a{x.data_ptr(), w.data_ptr(), x.stride(0), offs.data_ptr<int>(), active.data_ptr<int>(),
                 has_t ? token->data_ptr<int>() : nullptr, has_w ? ws->data_ptr<float>() : nullptr, y.data_ptr(), (int)R, (int)E,
                 (int)N, (int)K, (int)x.size(0), (int)act};
  const int64_t ne = std::min(E, R);
  if (x.scalar_type() == at::kBFloat16 && K % 8 == 0 && x.stride(0) % 8 == 0 && ex::aligned(x.data_ptr(), 16) &&
      ex::aligned(w.data_ptr(), 16)) {
    const dim3 grid((N + 15) / 16, ne);
    auto go = [&](auto kern, int nw) { hipLaunchKernelGGL(kern, grid, dim3(64 * nw), 0, cur_stream(), a); };
    const bool two = R > 8 * E;
    if (K >= 2048) two ? go(ex::expert_skinny_kernel<8, 2>, 8) : go(ex::expert_skinny_kernel<8, 1>, 8);
    else two ? go(ex::expert_skinny_kernel<4, 2>, 4) : go(ex::expert_skinny_kernel<4, 1>, 4);
  } else {
    const int64_t z = std::min<int64_t>(64, std::max<int64_t>(1, R / E / 16 + 1));
    SXE_DISPATCH_DT(dtype_of(x), D, hipLaunchKernelGGL((ex::expert_generic_kernel<D>), dim3((N + 63) / 64, ne, z), dim3(256), 0,
                                                       cur_stream(), a));
  }
  SXE_LAUNCH_CHECK();
  return y;
}

}  // namespace sxe

TORCH_LIBRARY_FRAGMENT(sxe, m) {
  m.def("route_topk(Tensor h, Tensor router, int k) -> Tensor[]");
  m.def("route_sandwich(Tensor x, Tensor y, Tensor wp, Tensor wn, Tensor? slots, Tensor? add, float eps, Tensor router, int k) -> "
        "Tensor[]");
  m.def("expert_gemm(Tensor x, Tensor w, Tensor offs, Tensor active, Tensor? token, Tensor? ws, int R, int act) -> Tensor");
}
TORCH_LIBRARY_IMPL(sxe, CUDA, m) {
  m.impl("route_topk", &sxe::route_topk);
  m.impl("route_sandwich", &sxe::route_sandwich);
  m.impl("expert_gemm", &sxe::expert_gemm);
}
