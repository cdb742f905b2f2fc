// Paged attention whose per-head weights are mixed across heads after the softmax (gfx950), with the
// score and mask variants such designs combine -- each one an optional argument:
//   * score_h(i, j) = scale q_h(i) . k_c(j) - r1_h ln(1 + r2_h (i - j))      (distance bias)
//   * i sees j <= i with i - j < window or j < keep_first                    (window with kept first keys)
//   * the softmax denominator also holds exp(sink_h)                         (sink: no key, no value)
//   * w_h(i, j) = sum_g talk[h, g] p_g(i, j), then head h applies w_h to the values of its own
//     key/value head c = h / (nq / nkv)                                      (talking heads)
//   * out *= sigmoid(gate) element by element                                (output gate)
// The mix couples all heads of a token BEFORE the value product and needs normalised weights, so a
// one-pass online softmax cannot carry it: every form below first finds the row's log-sum-exp, then
// forms the weights.
//
// Only visible keys are ever touched: position p has n0 = min(keep_first, lo) kept keys in front of
// its window [lo, p], lo = max(0, p + 1 - window), enumerated as one compact run of n0 + p + 1 - lo keys.
// Caches are [blocks, nkv, bs, D] views (k and v separately, block stride free).
#include "sxe_common.h"
#include <torch/library.h>
#include <climits>
#include <set>

namespace sxe {
namespace ma {

constexpr float kLog2e = 1.4426950408889634f;

struct Args {
  const void* q;  // [T, nq, Dk] dense
  const void *kc, *vc;
  int64_t k_block, v_block;  // elements between blocks
  const int* block_table;
  int max_blocks;
  const int *q_start, *q_len, *kv_len;
  int S, T, nq, nkv, dk, dv, Dk, Dv, bs;  // dk / dv real sizes, Dk / Dv row lengths of the caches
  int bs_shift;                           // log2(bs) (matrix-core forms)
  float scale;
  int window, keep_first;      // window 0: every key <= i
  const float *r1, *r2, *sink;  // [nq] or null (r1, r2 together)
  const float* talk;           // [nq, nq] or null
  const void* gate;            // [T, gate_ld] or null
  int64_t gate_ld;
  void* out;                   // [T, nq * dv]
};

struct Vis {
  int n0, lo, n;  // kept keys, window start, number of visible keys
};
__device__ __forceinline__ Vis visible(int pos, int window, int keep_first) {
  Vis v;
  v.lo = window > 0 ? max(0, pos + 1 - window) : 0;
  v.n0 = min(keep_first, v.lo);
  v.n = v.n0 + pos + 1 - v.lo;
  return v;
}
__device__ __forceinline__ int vis_key(const Vis& v, int c) { return c < v.n0 ? c : v.lo + c - v.n0; }

// ---- any type, any sizes: one workgroup per token, all heads -----------------------------------
constexpr int kGenThreads = 256, kGenKeys = 32;

template <DT T>
__global__ __launch_bounds__(kGenThreads) void mix_attn_generic_kernel(Args a, int max_q_len) {
  using S = typename dt_traits<T>::storage;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int seq = blockIdx.x / max_q_len, tok = blockIdx.x - seq * max_q_len;
  if (tok >= a.q_len[seq]) return;
  const int pos = a.kv_len[seq] - a.q_len[seq] + tok;
  const int64_t t = a.q_start[seq] + tok;
  const int G = a.nq / a.nkv, tid = threadIdx.x;
  float* ql = lds;                              // [nq * dk]
  float* ol = ql + a.nq * a.dk;                 // [nq * dv]
  float* pl = ol + a.nq * a.dv;                 // [nq][kGenKeys]
  float* wl = pl + a.nq * kGenKeys;             // [nq][kGenKeys]
  float* ml = wl + a.nq * kGenKeys;             // [nq]
  float* ll = ml + a.nq;                        // [nq]
  const S* q = static_cast<const S*>(a.q) + t * a.nq * a.Dk;
  for (int e = tid; e < a.nq * a.dk; e += kGenThreads) {
    const int h = e / a.dk;
    ql[e] = to_f32<T>(q[h * a.Dk + e - h * a.dk]);
  }
  for (int e = tid; e < a.nq * a.dv; e += kGenThreads) ol[e] = 0.f;
  for (int h = tid; h < a.nq; h += kGenThreads) {
    ml[h] = a.sink != nullptr ? a.sink[h] : -INFINITY;
    ll[h] = a.sink != nullptr ? 1.f : 0.f;
  }
  const Vis vis = visible(pos, a.window, a.keep_first);
  const int* bt = a.block_table + (int64_t)seq * a.max_blocks;
  for (int pass = 0; pass < 2; ++pass) {
    for (int c0 = 0; c0 < vis.n; c0 += kGenKeys) {
      const int nk = min(kGenKeys, vis.n - c0);
      __syncthreads();
      for (int e = tid; e < a.nq * kGenKeys; e += kGenThreads) {
        const int h = e / kGenKeys, kk = e - h * kGenKeys;
        float s = -INFINITY;
        if (kk < nk) {
          const int key = vis_key(vis, c0 + kk);
          const S* k = static_cast<const S*>(a.kc) + bt[key / a.bs] * a.k_block +
                       ((int64_t)(h / G) * a.bs + key % a.bs) * a.Dk;
          const float* qh = ql + h * a.dk;
          float d = 0.f;
          for (int i = 0; i < a.dk; ++i) d += qh[i] * to_f32<T>(k[i]);
          s = d * a.scale;
          if (a.r1 != nullptr) s -= a.r1[h] * logf(1.f + a.r2[h] * (float)(pos - key));
        }
        pl[e] = pass == 0 ? s : (kk < nk ? expf(s - ml[h]) / ll[h] : 0.f);
      }
      __syncthreads();
      if (pass == 0) {
        for (int h = tid; h < a.nq; h += kGenThreads) {
          float m = ml[h], l = ll[h];
          for (int kk = 0; kk < nk; ++kk) m = fmaxf(m, pl[h * kGenKeys + kk]);
          l *= ml[h] == -INFINITY ? 0.f : expf(ml[h] - m);
          for (int kk = 0; kk < nk; ++kk) l += expf(pl[h * kGenKeys + kk] - m);
          ml[h] = m;
          ll[h] = l;
        }
        continue;
      }
      const float* wt = pl;
      if (a.talk != nullptr) {
        for (int e = tid; e < a.nq * kGenKeys; e += kGenThreads) {
          const int h = e / kGenKeys, kk = e - h * kGenKeys;
          float w = 0.f;
          for (int g = 0; g < a.nq; ++g) w += a.talk[h * a.nq + g] * pl[g * kGenKeys + kk];
          wl[e] = w;
        }
        wt = wl;
        __syncthreads();
      }
      for (int e = tid; e < a.nq * a.dv; e += kGenThreads) {
        const int h = e / a.dv, d = e - h * a.dv;
        float o = ol[e];
        for (int kk = 0; kk < nk; ++kk) {
          const int key = vis_key(vis, c0 + kk);
          const S* v = static_cast<const S*>(a.vc) + bt[key / a.bs] * a.v_block +
                       ((int64_t)(h / G) * a.bs + key % a.bs) * a.Dv;
          o += wt[h * kGenKeys + kk] * to_f32<T>(v[d]);
        }
        ol[e] = o;
      }
    }
  }
  S* out = static_cast<S*>(a.out) + t * a.nq * a.dv;
  const S* gate = a.gate != nullptr ? static_cast<const S*>(a.gate) + t * a.gate_ld : nullptr;
  for (int e = tid; e < a.nq * a.dv; e += kGenThreads) {
    float o = ol[e];
    if (gate != nullptr) o /= 1.f + expf(-to_f32<T>(gate[e]));
    out[e] = from_f32<T>(o);
  }
}

// ---- matrix-core building blocks (bf16, head rows D = 64 / 128 / 256) ------------------------------
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef short i16x4 __attribute__((ext_vector_type(4)));
typedef short i16x8 __attribute__((ext_vector_type(8)));
typedef unsigned u32x4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ f32x4 mfma16(bf16x8 a, bf16x8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ bf16x8 frag(const unsigned short* p) {
  return __builtin_bit_cast(bf16x8, *reinterpret_cast<const u32x4*>(p));
}
__device__ __forceinline__ float ex2(float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ float lg2(float x) { return __builtin_amdgcn_logf(x); }

// swizzle of the 16-byte chunks of row `row` of a [rows][D bf16] LDS image (transposed reads conflict-free)
template <int D>
__device__ __forceinline__ int chunk_xor(int row) {
  constexpr int CH = D / 8;
  return (((row & 3) << 2) | ((row >> 2) & 3)) & (CH >= 16 ? 15 : CH - 1);
}
// lane group g's 4-row block of a 16-row tile in transposed reads (see paged_attn.hip)
__device__ __forceinline__ int kperm(int g) { return ((g & 1) << 3) | ((g & 2) << 1); }

// V^T operand of a 16x16x32 product: lane (g, i) holds column 16 dt + i of rows r0 + kperm(g) + 0..3 and
// of the same rows 16 further down
template <int D>
__device__ __forceinline__ bf16x8 v_frag(const char* img, int r0, int dt, int lane) {
  const int g = lane >> 4, i = lane & 15, p4 = i & 3;
  const int ra = r0 + kperm(g) + (i >> 2);  // r0 a multiple of 16: the row 16 further down has the same swizzle
  const int at = ra * 2 * D + ((16 * ((p4 >> 1) ^ chunk_xor<D>(ra)) + 8 * (p4 & 1)) ^ (32 * dt));
  const i16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
      (__attribute__((address_space(3))) i16x4*)(const_cast<char*>(img) + at));
  const i16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
      (__attribute__((address_space(3))) i16x4*)(const_cast<char*>(img) + at + 32 * D));
  return __builtin_bit_cast(bf16x8, __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7));
}

// a value the compiler cannot see through: what is computed from it stays inside the loop
__device__ __forceinline__ int opaque(int v) {
  asm volatile("" : "+v"(v));
  return v;
}
// two bf16 in a word. Weights p enter the head mix as p = hi + lo, lo = bf16(p - hi), which is p to ~2^-17.
__device__ __forceinline__ unsigned pack2(float a, float b) {
  typedef __bf16 bf16x2 __attribute__((ext_vector_type(2)));
  const bf16x2 v = {(__bf16)a, (__bf16)b};
  return __builtin_bit_cast(unsigned, v);
}

// LDS byte address of a pointer into shared memory (wave-uniform, for m0)
__device__ __forceinline__ unsigned lds_at(const char* p) {
  return __builtin_amdgcn_readfirstlane((unsigned)(uintptr_t)(const __attribute__((address_space(3))) char*)p);
}
// the same with a base per lane
__device__ __forceinline__ void dma16(unsigned lds, const void* src) {
  asm volatile("s_mov_b32 m0, %0\n\tglobal_load_lds_dwordx4 %1, off" ::"s"(lds), "v"(src) : "memory");
}
__device__ __forceinline__ const unsigned short* uniform_ptr(const unsigned short* p) {
  const uint64_t v = (uint64_t)p;
  const unsigned lo = __builtin_amdgcn_readfirstlane((unsigned)v), hi = __builtin_amdgcn_readfirstlane((unsigned)(v >> 32));
  return reinterpret_cast<const unsigned short*>(((uint64_t)hi << 32) | lo);
}
// 16 bytes per lane from base + off straight to LDS at lds + 16 lane. Inline asm: the compiler's wait-count
// pass would put a full wait before every later LDS read that might alias it.
__device__ __forceinline__ void dma16(unsigned lds, const void* base, unsigned off) {
  asm volatile("s_mov_b32 m0, %0\n\tglobal_load_lds_dwordx4 %1, %2" ::"s"(lds), "v"(off), "s"(base) : "memory");
}
// LDS traffic of this wave done, then the workgroup barrier; loads from memory stay in flight across it
__device__ __forceinline__ void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

// ---- token form: scores of one token through memory ------------------------------------------------
// Two launches for tokens that come alone (decode, short continuations, any head count): the first
// computes biased scores of one kv head's query heads over a split of the token's visible keys, writes
// them (log2 domain, fp32) and each split's (max, sum); the second turns the scores of ALL heads into
// weights, mixes them for one kv head's query heads and multiplies that head's values. A split's output
// is already normalised, so splits just add up.
struct TokArgs {
  float* scores;  // [rows, nq, nv]
  float* ml;      // [splits, rows, nq, 2]
  float* part;    // [splits, rows, nq, dv] (splits > 1)
  int nv, splits, keys_per_split;
  int nt, tok0, min_len, max_len;  // rows = S * nt: tokens tok0 .. + nt - 1 of sequences of min_len .. max_len new ones
};

template <int D>
struct TokGeo {
  static constexpr int NT = D >= 256 ? 2 : 4;
  static constexpr int KC = 16 * NT, KS = D / 32, DT = D / 16;
  static constexpr int VIMG = KC * 2 * D;
};
constexpr int kTokWaves = 4, kMaxHeads = 256;

struct TokRow {
  int seq, pos;
  int64_t t;
  bool ok;
};
__device__ __forceinline__ TokRow tok_row(const Args& a, const TokArgs& k, int row) {
  TokRow r;
  r.seq = row / k.nt;
  const int tok = k.tok0 + row - r.seq * k.nt, ql = a.q_len[r.seq];
  r.ok = tok < ql && ql >= k.min_len && ql <= k.max_len;
  r.pos = a.kv_len[r.seq] - ql + tok;
  r.t = a.q_start[r.seq] + tok;
  return r;
}

// the kv heads of one row on one XCD: they share its scores through that L2
__device__ __forceinline__ int tok_block() {
  const int n = gridDim.x, b = blockIdx.x;
  return n % 8 == 0 ? (b & 7) * (n / 8) + (b >> 3) : b;
}

template <int D>
__global__ __launch_bounds__(256) void mix_scores_kernel(Args a, TokArgs k) {
  using P = TokGeo<D>;
  constexpr int NT = P::NT, KC = P::KC, KS = P::KS;
  __shared__ float red[kTokWaves][16][2];
  const int blk = tok_block(), row = blk / a.nkv, c = blk - row * a.nkv, split = blockIdx.y;
  const TokRow r = tok_row(a, k, row);
  if (!r.ok) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, g = lane >> 4, i = lane & 15, G = a.nq / a.nkv;
  const Vis vis = visible(r.pos, a.window, a.keep_first);
  const int cb = split * k.keys_per_split, ce = min(vis.n, cb + k.keys_per_split);
  const int* bt = a.block_table + (int64_t)r.seq * a.max_blocks;
  const unsigned short* kc = static_cast<const unsigned short*>(a.kc);
  const int rows = gridDim.x / a.nkv;
  const float sc2 = a.scale * kLog2e;
  for (int h0 = 0; h0 < G; h0 += 16) {
    const bool hok = h0 + i < G;
    const int h = c * G + (hok ? h0 + i : 0);
    bf16x8 qb[KS];
    const unsigned short* qp = static_cast<const unsigned short*>(a.q) + (r.t * a.nq + h) * D + 8 * g;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) qb[ks] = frag(qp + 32 * ks);
    const float r1 = a.r1 != nullptr ? a.r1[h] : 0.f, r2 = a.r1 != nullptr ? a.r2[h] : 0.f;
    float m = -INFINITY, l = 0.f;
    float* srow = k.scores + ((int64_t)row * a.nq + h) * k.nv;
    for (int kb = cb + wave * KC; kb < ce; kb += kTokWaves * KC) {
      bf16x8 kr[NT][KS];
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        const int key = vis_key(vis, min(kb + 16 * t + i, ce - 1));
        const unsigned short* kp =
            kc + bt[key >> a.bs_shift] * a.k_block + ((c << a.bs_shift) + (key & (a.bs - 1))) * D + 8 * g;
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) kr[t][ks] = frag(kp + 32 * ks);
      }
      f32x4 s[NT];
      float mx = -INFINITY;
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        s[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) s[t] = mfma16(kr[t][ks], qb[ks], s[t]);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int ci = kb + 16 * t + 4 * g + e;
          const float d = (float)(r.pos - vis_key(vis, ci));
          s[t][e] = ci < ce ? s[t][e] * sc2 - r1 * lg2(1.f + r2 * d) : -INFINITY;
          mx = fmaxf(mx, s[t][e]);
        }
        const int ci = kb + 16 * t + 4 * g;  // < nv: nv is a multiple of 64 and ci of 4
        if (hok && ci < ce) *reinterpret_cast<f32x4*>(srow + ci) = s[t];
      }
      const float mn = fmaxf(m, mx);
      if (mn != -INFINITY) {
        l *= ex2(m - mn);
#pragma unroll
        for (int t = 0; t < NT; ++t)
#pragma unroll
          for (int e = 0; e < 4; ++e) l += ex2(s[t][e] - mn);
        m = mn;
      }
    }
#pragma unroll
    for (int o = 16; o < 64; o <<= 1) {
      const float m2 = __shfl_xor(m, o, 64), l2 = __shfl_xor(l, o, 64), mn = fmaxf(m, m2);
      l = mn == -INFINITY ? 0.f : l * ex2(m - mn) + l2 * ex2(m2 - mn);
      m = mn;
    }
    __syncthreads();
    if (g == 0) {
      red[wave][i][0] = m;
      red[wave][i][1] = l;
    }
    __syncthreads();
    if (threadIdx.x < 16 && h0 + (int)threadIdx.x < G) {
      float M = -INFINITY, L = 0.f;
#pragma unroll
      for (int w = 0; w < kTokWaves; ++w) M = fmaxf(M, red[w][threadIdx.x][0]);
      if (M != -INFINITY)
#pragma unroll
        for (int w = 0; w < kTokWaves; ++w) L += red[w][threadIdx.x][1] * ex2(red[w][threadIdx.x][0] - M);
      float* o = k.ml + (((int64_t)split * rows + row) * a.nq + c * G + h0 + threadIdx.x) * 2;
      o[0] = M;
      o[1] = L;
    }
  }
}

template <int D>
__global__ __launch_bounds__(256, 2) void mix_values_kernel(Args a, TokArgs k) {
  using P = TokGeo<D>;
  constexpr int NT = P::NT, KC = P::KC, DT = P::DT;
  extern __shared__ __attribute__((aligned(16))) char smem[];  // V images, then the wave-merge buffer
  __shared__ int64_t voff[kTokWaves][KC];
  __shared__ __attribute__((aligned(16))) float lse[kMaxHeads];
  __shared__ __attribute__((aligned(16))) unsigned short tl[16][kMaxHeads + 8];
  const int blk = tok_block(), row = blk / a.nkv, c = blk - row * a.nkv, split = blockIdx.y;
  const TokRow r = tok_row(a, k, row);
  if (!r.ok) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, g = lane >> 4, i = lane & 15, G = a.nq / a.nkv;
  const Vis vis = visible(r.pos, a.window, a.keep_first);
  const int cb = split * k.keys_per_split, ce = min(vis.n, cb + k.keys_per_split);
  const int* bt = a.block_table + (int64_t)r.seq * a.max_blocks;
  const int rows = gridDim.x / a.nkv, HP = (a.nq + 31) / 32 * 32;
  char* vimg = smem + wave * P::VIMG;
  float* mrg = reinterpret_cast<float*>(smem);  // [kTokWaves][16][D] after the key loop
  const unsigned short* vc = static_cast<const unsigned short*>(a.vc);
  const float* srow = k.scores + (int64_t)row * a.nq * k.nv;
  const int kb0 = cb + wave * KC;
  float raw[NT][8];
  // scores of heads 0 .. 31 for the chunk at kb (lane i <-> key kperm(i >> 2) + (i & 3), heads 8 g .. + 7)
  auto load_scores = [&](int kb) {
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const int ci = kb + 16 * t + kperm(i >> 2) + (i & 3);
        raw[t][j] = srow[(int64_t)min(8 * g + j, a.nq - 1) * k.nv + min(ci, k.nv - 1)];
      }
  };
  auto stage_v = [&](int kb) {
    if (lane < KC) {
      const int key = vis_key(vis, min(kb + lane, ce - 1));
      voff[wave][lane] = bt[key >> a.bs_shift] * a.v_block + ((c << a.bs_shift) + (key & (a.bs - 1))) * D;
    }
    __builtin_amdgcn_s_waitcnt(0xc07f);  // lgkmcnt(0)
    __builtin_amdgcn_wave_barrier();
    constexpr int CH = D / 8, RPK = 64 / CH;
    const unsigned dst = lds_at(vimg);
#pragma unroll
    for (int n = 0; n < KC / RPK; ++n) {
      const int rw = RPK * n + lane / CH, ch = (lane % CH) ^ chunk_xor<D>(rw);
      dma16(dst + n * 1024, vc + voff[wave][rw] + ch * 8);
    }
  };
  auto lse_of_rows = [&]() {  // log-sum-exp of every head's row, sink included
    const float2* ml = reinterpret_cast<const float2*>(k.ml);
    for (int h = threadIdx.x; h < a.nq; h += 256) {
      float M = a.sink != nullptr ? a.sink[h] * kLog2e : -INFINITY, L = a.sink != nullptr ? 1.f : 0.f;
      for (int s0 = 0; s0 < k.splits; s0 += 8) {
        float2 v[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) v[u] = ml[((int64_t)min(s0 + u, k.splits - 1) * rows + row) * a.nq + h];
        float mn = M;
#pragma unroll
        for (int u = 0; u < 8; ++u) mn = s0 + u < k.splits ? fmaxf(mn, v[u].x) : mn;
        L = M == -INFINITY ? 0.f : L * ex2(M - mn);
#pragma unroll
        for (int u = 0; u < 8; ++u) L += s0 + u < k.splits && v[u].x != -INFINITY ? v[u].y * ex2(v[u].x - mn) : 0.f;
        M = mn;
      }
      lse[h] = M + lg2(L);
    }
    for (int h = a.nq + threadIdx.x; h < HP; h += 256) lse[h] = INFINITY;  // heads past nq: weight 0
  };
  for (int h0 = 0; h0 < G; h0 += 16) {
    const bool some = kb0 < ce;
    if (h0 > 0) __syncthreads();  // the previous pass is done with `tl` and the merge buffer
    if (some) {
      load_scores(kb0);
      stage_v(kb0);
    }
    if (h0 == 0) lse_of_rows();
    for (int e = threadIdx.x; e < 16 * HP; e += 256) {
      const int n = e / HP, gg = e - n * HP;
      float v = 0.f;
      if (h0 + n < G && gg < a.nq)
        v = a.talk != nullptr ? a.talk[(int64_t)(c * G + h0 + n) * a.nq + gg] : (gg == c * G + h0 + n ? 1.f : 0.f);
      tl[n][gg] = f32_to_bf16(v);
    }
    __syncthreads();
    f32x4 o[DT];
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) o[dt] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int kb = kb0; kb < ce; kb += kTokWaves * KC) {
      const int kn = kb + kTokWaves * KC;
      // W^T = P^T T^T: rows = keys, columns = this group's heads
      f32x4 w[NT];
#pragma unroll
      for (int t = 0; t < NT; ++t) w[t] = f32x4{0.f, 0.f, 0.f, 0.f};
      for (int kk = 0; kk < HP; kk += 32) {
        const bf16x8 tb = *reinterpret_cast<const bf16x8*>(&tl[i][kk + 8 * g]);
        const f32x4 la = *reinterpret_cast<const f32x4*>(&lse[kk + 8 * g]), lb = *reinterpret_cast<const f32x4*>(&lse[kk + 8 * g + 4]);
#pragma unroll
        for (int t = 0; t < NT; ++t) {
          const int ci = kb + 16 * t + kperm(i >> 2) + (i & 3);
          u32x4 hi, lo;
          float p[8];
          if (kk > 0)
#pragma unroll
            for (int j = 0; j < 8; ++j)
              raw[t][j] = srow[(int64_t)min(kk + 8 * g + j, a.nq - 1) * k.nv + min(ci, k.nv - 1)];
#pragma unroll
          for (int j = 0; j < 8; ++j) p[j] = ci < ce ? ex2(raw[t][j] - (j < 4 ? la[j & 3] : lb[j & 3])) : 0.f;
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            hi[j] = pack2(p[2 * j], p[2 * j + 1]);
            lo[j] = pack2(p[2 * j] - __uint_as_float(hi[j] << 16), p[2 * j + 1] - __uint_as_float(hi[j] & 0xffff0000u));
          }
          w[t] = mfma16(__builtin_bit_cast(bf16x8, hi), tb, w[t]);
          w[t] = mfma16(__builtin_bit_cast(bf16x8, lo), tb, w[t]);
        }
      }
      if (kn < ce) {  // the next chunk's scores are in flight while this one's values are multiplied
        load_scores(kn);
        asm volatile("s_waitcnt vmcnt(%0)" ::"n"(8 * NT) : "memory");  // this wave's V image has landed
      } else {
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
      }
      __builtin_amdgcn_wave_barrier();
#pragma unroll
      for (int pp = 0; pp < NT / 2; ++pp) {
        const bf16x8 pb = __builtin_bit_cast(bf16x8, u32x4{pack2(w[2 * pp][0], w[2 * pp][1]), pack2(w[2 * pp][2], w[2 * pp][3]),
                                                           pack2(w[2 * pp + 1][0], w[2 * pp + 1][1]),
                                                           pack2(w[2 * pp + 1][2], w[2 * pp + 1][3])});
#pragma unroll
        for (int dt = 0; dt < DT; ++dt) o[dt] = mfma16(v_frag<D>(vimg, 32 * pp, dt, lane), pb, o[dt]);
      }
      __builtin_amdgcn_s_waitcnt(0xc07f);  // the V image is read before the next chunk overwrites it
      __builtin_amdgcn_wave_barrier();
      if (kn < ce) stage_v(kn);
    }
    __syncthreads();  // every wave is done with its V image (the merge buffer aliases it)
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) *reinterpret_cast<f32x4*>(mrg + (wave * 16 + i) * D + 16 * dt + 4 * g) = o[dt];
    __syncthreads();
    const int nh = min(16, G - h0);
    for (int e = threadIdx.x; e < nh * a.dv; e += 256) {
      const int n = e / a.dv, d = e - n * a.dv, h = c * G + h0 + n;
      float v = 0.f;
#pragma unroll
      for (int w = 0; w < kTokWaves; ++w) v += mrg[(w * 16 + n) * D + d];
      const int64_t col = (int64_t)h * a.dv + d;
      if (k.splits == 1) {
        if (a.gate != nullptr)
          v /= 1.f + __expf(-bf16_to_f32(static_cast<const unsigned short*>(a.gate)[r.t * a.gate_ld + col]));
        static_cast<unsigned short*>(a.out)[r.t * a.nq * a.dv + col] = f32_to_bf16(v);
      } else {
        k.part[((int64_t)split * rows + row) * a.nq * a.dv + col] = v;
      }
    }
  }
}

// out = (sum over splits) * sigmoid(gate)
__global__ __launch_bounds__(256) void mix_reduce_kernel(Args a, TokArgs k) {
  const int row = blockIdx.x, rows = gridDim.x;
  const TokRow r = tok_row(a, k, row);
  if (!r.ok) return;
  const int n = a.nq * a.dv;
  for (int col = blockIdx.y * 256 + threadIdx.x; col < n; col += gridDim.y * 256) {
    float v = 0.f;
    for (int s0 = 0; s0 < k.splits; s0 += 8) {  // eight loads in flight, then their sum
      float p[8];
#pragma unroll
      for (int u = 0; u < 8; ++u) p[u] = k.part[((int64_t)min(s0 + u, k.splits - 1) * rows + row) * n + col];
#pragma unroll
      for (int u = 0; u < 8; ++u) v += s0 + u < k.splits ? p[u] : 0.f;
    }
    if (a.gate != nullptr)
      v /= 1.f + __expf(-bf16_to_f32(static_cast<const unsigned short*>(a.gate)[r.t * a.gate_ld + col]));
    static_cast<unsigned short*>(a.out)[r.t * n + col] = f32_to_bf16(v);
  }
}

// ---- tile form: 16 consecutive tokens of a sequence, all heads -------------------------------------
// Prompts and long continuations. First launch: log-sum-exp of every (token, head) row, one wave per (16
// tokens, kv head). Second launch: one 8-wave workgroup per 16 tokens; wave w owns HPW query heads.
// Per 32-key tile: (a) every wave computes its heads' weights 2^(s - lse) (S^T = K Q^T, K fragments
// straight from the cache, shared by the heads of a kv head) and puts their bf16 head and remainder
// into LDS; (b) the waves mix: W = P T^T as matrix products over the head axis, 4 (token, 16-key)
// tiles a wave, W to LDS in the order of the value product's operand; (c) every wave multiplies its
// heads' W with its kv head's V (row image in LDS, transposed reads). The value product of a tile and the
// weights of the next one lie between the same two barriers, so two barriers a tile suffice.
// The distance bias takes 47 values per (head, tile) -- one logarithm per lane, handed round by
// ds_bpermute -- instead of one per score.
struct TileArgs {
  float* lse;            // [T, nq]
  unsigned short* talk;  // [2][64][8] bf16: lane l's operand of the mix, T[16 n + (l & 15)][8 (l >> 4) .. + 7]
  float* part;           // [splits, S * max_len, nq * dv] (splits > 1)
  int min_len, max_len, tiles, splits;  // sequences with q_len >= min_len; 16-token tiles per sequence
  int vec;               // gate and output rows allow 8-byte accesses
};
constexpr int kTileWaves = 8, kTileKeys = 32, kTileHeads = 32;

struct TileIdx {
  int seq, p0, ntok;  // sequence, first position, tokens in the tile
  int64_t t0;
  bool ok;
};
// wave-uniform values that the compiler would otherwise keep in vector registers
__device__ __forceinline__ int uni(int v) { return __builtin_amdgcn_readfirstlane(v); }
__device__ __forceinline__ float uni(float v) {
  return __builtin_bit_cast(float, __builtin_amdgcn_readfirstlane(__builtin_bit_cast(int, v)));
}
__device__ __forceinline__ TileIdx tile_idx(const Args& a, const TileArgs& k, int id) {
  TileIdx x;
  x.seq = uni(id / k.tiles);
  const int tok = (id - x.seq * k.tiles) * 16, ql = x.seq < a.S ? uni(a.q_len[x.seq]) : 0;
  x.ok = tok < ql && ql >= k.min_len;
  if (!x.ok) return x;
  x.p0 = uni(a.kv_len[x.seq]) - ql + tok;
  x.ntok = min(16, ql - tok);
  x.t0 = uni(a.q_start[x.seq]) + tok;
  return x;
}

// 32-key tiles of a token tile: [0, kt) cover the kept keys in front of the window, then [wt, end)
struct KeyTiles {
  int kt, wt, n;
};
__device__ __forceinline__ KeyTiles key_tiles(const Args& a, const TileIdx& x) {
  KeyTiles k;
  const int lo = a.window > 0 ? max(0, x.p0 + 1 - a.window) : 0;
  k.wt = lo / kTileKeys;
  k.kt = min(k.wt, (a.keep_first + kTileKeys - 1) / kTileKeys);
  k.n = k.kt + (x.p0 + x.ntok - 1) / kTileKeys + 1 - k.wt;
  return k;
}
__device__ __forceinline__ int key0(const KeyTiles& k, int n) { return (n < k.kt ? n : k.wt + n - k.kt) * kTileKeys; }

// whether some (token, key) pair of the tile is hidden
__device__ __forceinline__ bool needs_mask(const Args& a, const TileIdx& x, int k0) {
  const int k1 = k0 + kTileKeys - 1;
  if (k1 > x.p0) return true;
  return a.window > 0 && x.p0 + 15 - k0 >= a.window && k1 >= a.keep_first;
}
__device__ __forceinline__ bool sees(const Args& a, int pos, int key) {
  return key <= pos && (a.window <= 0 || pos - key < a.window || key < a.keep_first);
}

template <int D>
__global__ __launch_bounds__(256) void mix_lse_kernel(Args a, TileArgs k, int total) {
  constexpr int KS = D / 32, HB = 4;  // heads per round
  if (blockIdx.x == 0)  // the next launch's operand of the head mix (no mix: the identity)
    for (int e = threadIdx.x; e < 1024; e += 256) {
      const int h = 16 * (e >> 9) + ((e >> 3) & 15), gg = 8 * ((e >> 7) & 3) + (e & 7);
      float f = h == gg ? 1.f : 0.f;
      if (a.talk != nullptr) f = h < a.nq && gg < a.nq ? a.talk[h * a.nq + gg] : 0.f;
      k.talk[e] = f32_to_bf16(f);
    }
  const int unit = blockIdx.x * 4 + uni((int)threadIdx.x >> 6);
  if (unit >= total) return;
  const int c = uni(unit % a.nkv);
  const TileIdx x = tile_idx(a, k, unit / a.nkv);
  if (!x.ok) return;
  const int lane = threadIdx.x & 63, g = lane >> 4, i = lane & 15, G = uni(a.nq / a.nkv);
  const KeyTiles kt = key_tiles(a, x);
  const int* bt = a.block_table + (int64_t)x.seq * a.max_blocks;
  const unsigned short *kc = static_cast<const unsigned short*>(a.kc), *q = static_cast<const unsigned short*>(a.q);
  const int tok = min(i, x.ntok - 1);
  const float sc2 = a.scale * kLog2e;
  const int bidx = 4 * (4 * g - i + 15);
  for (int h0 = 0; h0 < G; h0 += HB) {
    bf16x8 qb[HB][KS];
    float m[HB], l[HB], r1[HB], r2[HB];
#pragma unroll
    for (int hh = 0; hh < HB; ++hh) {
      const int h = c * G + min(h0 + hh, G - 1);
      const unsigned short* qp = q + ((x.t0 + tok) * a.nq + h) * D + 8 * g;
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) qb[hh][ks] = frag(qp + 32 * ks);
      m[hh] = -INFINITY;
      l[hh] = 0.f;
      r1[hh] = a.r1 != nullptr ? uni(a.r1[h]) * (-1.f / sc2) : 0.f;  // bias in units of the raw product
      r2[hh] = a.r1 != nullptr ? uni(a.r2[h]) : 0.f;
    }
    bf16x8 kr[2][KS];
    int blocks = 0;  // block ids of 64 tiles, one a lane
    auto load_k = [&](int n) {
      if ((n & 63) == 0) blocks = bt[key0(kt, min(n + lane, kt.n - 1)) >> a.bs_shift];
      const unsigned short* base = kc + (int64_t)__builtin_amdgcn_readlane(blocks, n & 63) * a.k_block +
                                   ((c << a.bs_shift) + (key0(kt, n) & (a.bs - 1))) * D;
#pragma unroll
      for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) kr[t][ks] = frag(base + (unsigned)(i * D + 8 * g + 16 * t * D + 32 * ks));
    };
    load_k(0);
    for (int n = 0; n < kt.n; ++n) {
      const int k0 = key0(kt, n);
      const bool msk = needs_mask(a, x, k0);
      const float dl = (float)max(0, x.p0 - k0 + 15 - lane);  // the distance whose bias this lane computes
      f32x4 s[HB][2];
#pragma unroll
      for (int hh = 0; hh < HB; ++hh) {
        const int tb = __builtin_bit_cast(int, r1[hh] * lg2(1.f + r2[hh] * dl));
#pragma unroll
        for (int t = 0; t < 2; ++t) {
#pragma unroll
          for (int e = 0; e < 4; ++e)
            s[hh][t][e] = __builtin_bit_cast(float, __builtin_amdgcn_ds_bpermute(bidx + 4 * (16 * t + e), tb));
#pragma unroll
          for (int ks = 0; ks < KS; ++ks) s[hh][t] = mfma16(kr[t][ks], qb[hh][ks], s[hh][t]);
        }
      }
      if (n + 1 < kt.n) load_k(n + 1);
      if (msk) {
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const bool vis = sees(a, x.p0 + i, k0 + 16 * t + 4 * g + e);
#pragma unroll
            for (int hh = 0; hh < HB; ++hh) s[hh][t][e] = vis ? s[hh][t][e] : -INFINITY;
          }
      }
#pragma unroll
      for (int hh = 0; hh < HB; ++hh) {  // max and sum of raw products + bias (scale > 0: the order is the scores')
        float mx = m[hh];
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
          for (int e = 0; e < 4; ++e) mx = fmaxf(mx, s[hh][t][e]);
        const float mr = mx == -INFINITY ? 0.f : mx * sc2;
        float ls = l[hh] * ex2(m[hh] * sc2 - mr);
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
          for (int e = 0; e < 4; ++e) ls += ex2(s[hh][t][e] * sc2 - mr);
        l[hh] = ls;
        m[hh] = mx;
      }
    }
#pragma unroll
    for (int hh = 0; hh < HB; ++hh) {
      if (h0 + hh >= G) break;
      float M = m[hh] * sc2, L = l[hh];
#pragma unroll
      for (int o = 16; o < 64; o <<= 1) {
        const float m2 = __shfl_xor(M, o, 64), l2 = __shfl_xor(L, o, 64), mn = fmaxf(M, m2);
        L = mn == -INFINITY ? 0.f : L * ex2(M - mn) + l2 * ex2(m2 - mn);
        M = mn;
      }
      const int h = c * G + h0 + hh;
      if (a.sink != nullptr) {
        const float sk = a.sink[h] * kLog2e, mn = fmaxf(M, sk);
        L = L * ex2(M - mn) + ex2(sk - mn);
        M = mn;
      }
      if (g == 0 && i < x.ntok) k.lse[(x.t0 + i) * a.nq + h] = M + lg2(L);
    }
  }
}

// ONE_KV: every wave's HPW heads exist and belong to one kv head (nq / nkv a multiple of HPW)
template <int D, int HPW, bool ONE_KV>
__global__ __launch_bounds__(kTileWaves * 64, 2) void mix_tile_kernel(Args a, TileArgs k, int total) {
  constexpr int KS = D / 32, DT = D / 16, PB = 16 * kTileKeys * kTileHeads * 2, VIMG = kTileKeys * 2 * D;
  constexpr int NP = (HPW + 1) / 2;       // bf16 pairs of heads
  constexpr int NMIX = HPW == 4 ? 2 : 1;  // 16-head tiles of the mix
  extern __shared__ __attribute__((aligned(16))) char smem[];
  char *phi = smem, *plo = smem + PB, *wbuf = smem + 2 * PB;
  // consecutive tiles of a sequence share most of their window: keep them on one XCD's L2
  const int per = (total + 7) / 8, id = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
  if (id >= total) return;
  const TileIdx x = tile_idx(a, k, id);
  if (!x.ok) return;
  const int lane_ = threadIdx.x & 63, wave = uni((int)threadIdx.x >> 6), G = uni(a.nq / a.nkv);
  const int g = lane_ >> 4, i = lane_ & 15;
  char* vimg = smem + 3 * PB + wave * VIMG;
  const KeyTiles kt = key_tiles(a, x);
  const int* bt = a.block_table + (int64_t)x.seq * a.max_blocks;
  const unsigned short *kc = static_cast<const unsigned short*>(a.kc), *vc = static_cast<const unsigned short*>(a.vc);
  const int hw = wave * HPW;  // first head of this wave
  const int nh = min(HPW, a.nq - hw);
  const int tok = min(i, x.ntok - 1);
  const float sc2 = a.scale * kLog2e, nsc = -1.f / sc2;
  // heads past nq are never written by a wave: their weights stay zero
  for (int e = threadIdx.x; e < 2 * PB / 16; e += kTileWaves * 64) reinterpret_cast<u32x4*>(smem)[e] = u32x4{0u, 0u, 0u, 0u};
  bf16x8 qb[HPW][KS];
  float lse[HPW], r1[HPW], r2[HPW];
  int kvh[HPW];
  f32x4 o[HPW][DT];
#pragma unroll
  for (int hh = 0; hh < HPW; ++hh) {
    const int h = min(hw + hh, a.nq - 1);
    const unsigned short* qp = static_cast<const unsigned short*>(a.q) + ((x.t0 + tok) * a.nq + h) * D + 8 * g;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) qb[hh][ks] = frag(qp + 32 * ks);
    lse[hh] = k.lse[(x.t0 + tok) * a.nq + h];
    kvh[hh] = uni(h / G);
    r1[hh] = a.r1 != nullptr ? uni(a.r1[h]) * nsc : 0.f;  // bias in units of the raw product
    r2[hh] = a.r1 != nullptr ? uni(a.r2[h]) : 0.f;
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) o[hh][dt] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  bf16x8 kr[KS];

  // block ids of 64 tiles, one a lane (a load per tile would wait behind the image in flight)
  int blocks = 0;
  auto fetch_blocks = [&](int n) { blocks = bt[key0(kt, min(n + lane_, kt.n - 1)) >> a.bs_shift]; };
  auto row_of = [&](int n, int c) {  // element offset / D inside its block of the tile's first key, kv head c
    return (c << a.bs_shift) + (key0(kt, n) & (a.bs - 1));
  };
  // K fragments of half t (16 keys) of tile n, kv head c
  auto load_k = [&](int lane, int c, int n, int t) {
    const unsigned short* base =
        kc + (int64_t)__builtin_amdgcn_readlane(blocks, n & 63) * a.k_block + (row_of(n, c) + 16 * t) * D;
    const unsigned off = (lane & 15) * D + 8 * (lane >> 4);
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) kr[ks] = frag(base + off + 32 * ks);
  };
  // V rows of tile n, kv head c -> this wave's image
  auto stage_v = [&](int lane, int c, int n) {
    constexpr int CH = D / 8, RPK = 64 / CH;
    const unsigned short* base = vc + (int64_t)__builtin_amdgcn_readlane(blocks, n & 63) * a.v_block + row_of(n, c) * D;
    const unsigned dst = lds_at(vimg), off = (lane / CH) * 2 * D + 16 * ((lane % CH) ^ chunk_xor<D>(lane / CH));
#pragma unroll
    for (int j = 0; j < kTileKeys / RPK; ++j)  // the swizzles of lane / CH and of RPK j are disjoint bits
      dma16(dst + j * 1024, base + j * 512, off ^ (16 * chunk_xor<D>(RPK * j)));
  };
  // the weights of this wave's heads over one tile, to LDS; K of the tile's first half is in kr
  auto weights = [&](int n) {
    const int lane = opaque(lane_), g = lane >> 4, i = lane & 15;
    const int k0 = key0(kt, n);
    const bool msk = needs_mask(a, x, k0);
    __builtin_amdgcn_s_waitcnt(0x0f70);  // vmcnt(0): K of the first half
    stage_v(lane, kvh[0], n);
    const float dl = (float)max(0, x.p0 - k0 + 15 - lane);  // the distance whose bias this lane computes
    int tbl[HPW];
#pragma unroll
    for (int hh = 0; hh < HPW; ++hh) tbl[hh] = __builtin_bit_cast(int, r1[hh] * lg2(1.f + r2[hh] * dl));
    const int bx = 4 * (4 * g - i + 15);
    // row (token i, key 16 t + 4 g + (e ^ i & 3)), chunk of this wave's heads
    const int at0 = i * (kTileKeys * 2 * kTileHeads) + (4 * g + (i & 3)) * (2 * kTileHeads) +
                    16 * (((2 * hw) >> 4) ^ ((i >> 2) & 3)) + ((2 * hw) & 15);
#pragma unroll
    for (int t = 0; t < 2; ++t) {
      f32x4 sc[HPW];  // starts from the bias (in units of the raw product), then + q . k
#pragma unroll
      for (int hh = 0; hh < HPW; ++hh)
#pragma unroll
        for (int e = 0; e < 4; ++e)
          sc[hh][e] = __builtin_bit_cast(float, __builtin_amdgcn_ds_bpermute(bx + 4 * (16 * t + e), tbl[hh]));
#pragma unroll
      for (int hh = 0; hh < HPW; ++hh) {
        if constexpr (!ONE_KV)
          if (hh > 0 && kvh[hh] != kvh[hh - 1]) load_k(lane, kvh[hh], n, t);
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) sc[hh] = mfma16(kr[ks], qb[hh][ks], sc[hh]);
      }
      if (t == 0) {
        load_k(lane, kvh[0], n, 1);
      } else {  // the next tile's first half, in flight across mix and value product
        if (((n + 1) & 63) == 0) fetch_blocks(n + 1);
        load_k(lane, kvh[0], min(n + 1, kt.n - 1), 0);
      }
      if (msk) {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const bool vis = sees(a, x.p0 + i, k0 + 16 * t + 4 * g + e);
#pragma unroll
          for (int hh = 0; hh < HPW; ++hh) sc[hh][e] = vis ? sc[hh][e] : -INFINITY;
        }
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        unsigned ph[NP], pl[NP];
#pragma unroll
        for (int hp = 0; hp < NP; ++hp) {
          const float p0 = ex2(sc[2 * hp][e] * sc2 - lse[2 * hp]);
          float p1 = 0.f;
          if constexpr (HPW > 1) p1 = ex2(sc[2 * hp + 1][e] * sc2 - lse[2 * hp + 1]);
          if constexpr (!ONE_KV && HPW > 1) p1 = 2 * hp + 1 < nh ? p1 : 0.f;
          ph[hp] = pack2(p0, p1);
          pl[hp] = pack2(p0 - __uint_as_float(ph[hp] << 16), p1 - __uint_as_float(ph[hp] & 0xffff0000u));
          if constexpr (!ONE_KV)
            if (2 * hp >= nh) ph[hp] = pl[hp] = 0u;
        }
        char* at = phi + (at0 ^ (e * 2 * kTileHeads)) + t * (16 * 2 * kTileHeads);
        if constexpr (HPW == 4) {
          *reinterpret_cast<uint2*>(at) = uint2{ph[0], ph[1]};
          *reinterpret_cast<uint2*>(at + PB) = uint2{pl[0], pl[1]};
        } else if constexpr (HPW == 2) {
          *reinterpret_cast<unsigned*>(at) = ph[0];
          *reinterpret_cast<unsigned*>(at + PB) = pl[0];
        } else {
          *reinterpret_cast<unsigned short*>(at) = (unsigned short)ph[0];
          *reinterpret_cast<unsigned short*>(at + PB) = (unsigned short)pl[0];
        }
      }
    }
  };

  // a small batch splits the key tiles over workgroups: weights are normalised, so the splits' outputs add up
  const int nb = kt.n * blockIdx.y / k.splits, ne = kt.n * (blockIdx.y + 1) / k.splits;
  if (nh > 0 && nb < ne) {
    fetch_blocks(nb & ~63);
    load_k(lane_, kvh[0], nb, 0);
  }
  lds_barrier();  // the zeroed weights
  if (nh > 0 && nb < ne) weights(nb);
  for (int n = nb; n < ne; ++n) {
    bf16x8 tb[NMIX];  // read again for every tile: registers that the weights need
#pragma unroll
    for (int nn = 0; nn < NMIX; ++nn) tb[nn] = frag(k.talk + (nn * 64 + opaque(lane_)) * 8);
    lds_barrier();
    // ---- mix: this wave's tokens 2 wave, 2 wave + 1, both 16-key halves ------------------------------
    {
      const int lane = opaque(lane_), g = lane >> 4, i = lane & 15;
      // lane: head h = i (+ 16), keys 16 t + 4 g .. + 3 of token q -> chunk of the lane group that reads those rows of V
      const int ch = ((g & 1) << 1) | (g >> 1), wt0 = i * (16 * 2 * kTileKeys) + 16 * (ch ^ ((i >> 2) & 3));
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int q = 2 * wave + (u >> 1), t = u & 1;
        const int at = ((i * (2 * kTileHeads) + 16 * g) ^ ((q & 3) * (2 * kTileHeads) + 16 * ((q >> 2) & 3))) +
                       (q * kTileKeys + 16 * t) * (2 * kTileHeads);
        const bf16x8 hi = *reinterpret_cast<const bf16x8*>(phi + at), lo = *reinterpret_cast<const bf16x8*>(plo + at);
#pragma unroll
        for (int nn = 0; nn < NMIX; ++nn) {
          f32x4 w = {0.f, 0.f, 0.f, 0.f};
          w = mfma16(hi, tb[nn], w);
          w = mfma16(lo, tb[nn], w);
          const int wt = wt0 + nn * (16 * 16 * 2 * kTileKeys) + (q ^ (i & 3)) * (2 * kTileKeys) + 8 * t;
          *reinterpret_cast<uint2*>(wbuf + wt) = uint2{pack2(w[0], w[1]), pack2(w[2], w[3])};
        }
      }
    }
    // the V image: older than the K fragments in flight for the next tile
    asm volatile("s_waitcnt vmcnt(%0)" ::"n"(KS) : "memory");
    lds_barrier();
    // ---- O^T += V^T W^T, then the next tile's weights ------------------------------------------------
    if (nh > 0) {
      const int lane = opaque(lane_), g = lane >> 4, i = lane & 15;
      bf16x8 wf[HPW];
#pragma unroll
      for (int hh = 0; hh < HPW; ++hh) {
        const int h = hw + hh;  // < 32: eight waves of at most four heads
        wf[hh] = *reinterpret_cast<const bf16x8*>(wbuf + (h * 16 + (i ^ (h & 3))) * (2 * kTileKeys) + 16 * (g ^ ((h >> 2) & 3)));
      }
      if constexpr (ONE_KV) {
#pragma unroll
        for (int dt = 0; dt < DT; ++dt) {
          const bf16x8 vf = v_frag<D>(vimg, 0, dt, lane);
#pragma unroll
          for (int hh = 0; hh < HPW; ++hh) o[hh][dt] = mfma16(vf, wf[hh], o[hh][dt]);
        }
      } else {
#pragma unroll
        for (int hh = 0; hh < HPW; ++hh) {  // the wave's heads span several kv heads: stage each V in turn
          if (hh >= nh) break;
          if (hh > 0 && kvh[hh] != kvh[hh - 1]) {
            __builtin_amdgcn_s_waitcnt(0xc07f);  // the image has been read
            stage_v(lane, kvh[hh], n);
            asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
          }
#pragma unroll
          for (int dt = 0; dt < DT; ++dt) o[hh][dt] = mfma16(v_frag<D>(vimg, 0, dt, lane), wf[hh], o[hh][dt]);
        }
      }
      __builtin_amdgcn_s_waitcnt(0xc07f);  // V and W reads are done before the image is refilled
      if (n + 1 < ne) weights(n + 1);
    }
  }
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  if (i >= x.ntok) return;
  const int64_t t = x.t0 + i, cols = (int64_t)a.nq * a.dv;
  float* part = nullptr;
  if (k.splits > 1)
    part = k.part + ((int64_t)blockIdx.y * a.S * k.max_len + (int64_t)x.seq * k.max_len + (x.t0 + i - a.q_start[x.seq])) * cols;
  unsigned short* out = static_cast<unsigned short*>(a.out) + t * cols;
  const unsigned short* gate =
      a.gate != nullptr && part == nullptr ? static_cast<const unsigned short*>(a.gate) + t * a.gate_ld : nullptr;
#pragma unroll
  for (int hh = 0; hh < HPW; ++hh) {
    if (hh >= nh) break;
    const int64_t col0 = (int64_t)(hw + hh) * a.dv + 4 * g;
    u16x4 gv[DT];
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {  // a head's gate values are all in flight before the first is used
      const int d = 16 * dt + 4 * g;
      gv[dt] = u16x4{0, 0, 0, 0};
      if (gate == nullptr || d >= a.dv) continue;
      if (k.vec) {
        gv[dt] = *reinterpret_cast<const u16x4*>(gate + col0 + 16 * dt);
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (d + e < a.dv) gv[dt][e] = gate[col0 + 16 * dt + e];
      }
    }
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      const int d = 16 * dt + 4 * g;
      if (d >= a.dv) continue;
      f32x4 v = o[hh][dt];
      if (gate != nullptr)
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] *= __builtin_amdgcn_rcpf(1.f + __expf(-bf16_to_f32(gv[dt][e])));
      if (k.vec) {
        if (part != nullptr) *reinterpret_cast<f32x4*>(part + col0 + 16 * dt) = v;
        else *reinterpret_cast<uint2*>(out + col0 + 16 * dt) = uint2{pack2(v[0], v[1]), pack2(v[2], v[3])};
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          if (d + e >= a.dv) continue;
          if (part != nullptr) part[col0 + 16 * dt + e] = v[e];
          else out[col0 + 16 * dt + e] = f32_to_bf16(v[e]);
        }
      }
    }
  }
}

}  // namespace ma

namespace {

const float* head_vec(const c10::optional<at::Tensor>& t, int64_t n, const char* what) {
  if (!t.has_value() || !t->defined()) return nullptr;
  SXE_CHECK(t->scalar_type() == at::kFloat && t->is_contiguous() && t->numel() == n && t->is_cuda(), "mix_attention: ",
            what, " fp32 with ", n, " elements");
  return t->data_ptr<float>();
}

// dynamic LDS above 64 KiB must be opted into, once per kernel
template <typename F>
void allow_lds(F* kern, size_t bytes) {
  static std::set<const void*> done;
  const void* f = reinterpret_cast<const void*>(kern);
  if (done.insert(f).second)
    SXE_HIP_CHECK(hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes));
}

template <int D>
void launch_tokens_d(const ma::Args& a, const ma::TokArgs& k, int rows, bool keep_part) {
  const dim3 grid(rows * a.nkv, k.splits);
  constexpr int merge = ma::kTokWaves * 16 * D * 4, img = ma::kTokWaves * ma::TokGeo<D>::VIMG;
  constexpr size_t lds = img > merge ? img : merge;
  hipLaunchKernelGGL(ma::mix_scores_kernel<D>, grid, dim3(256), 0, cur_stream(), a, k);
  allow_lds(ma::mix_values_kernel<D>, lds);
  hipLaunchKernelGGL(ma::mix_values_kernel<D>, grid, dim3(256), lds, cur_stream(), a, k);
  if (k.splits > 1 && !keep_part) {
    const int cols = a.nq * a.dv;
    hipLaunchKernelGGL(ma::mix_reduce_kernel, dim3(rows, std::min(64, (cols + 255) / 256)), dim3(256), 0, cur_stream(), a, k);
  }
  SXE_LAUNCH_CHECK();
}

// keep_part: with several splits leave their outputs unsummed and return them [splits, rows, nq dv]
at::Tensor launch_tokens(const ma::Args& a, const at::Tensor& q, int nv, int splits, int tok0, int nt, int max_len,
                         bool keep_part = false) {
  ma::TokArgs k{};
  const int rows = a.S * nt;
  int kps = (nv + std::max(1, splits) - 1) / std::max(1, splits);
  kps = (kps + 63) / 64 * 64;
  k.nv = nv;
  k.keys_per_split = kps;
  k.splits = (nv + kps - 1) / kps;
  k.nt = nt;
  k.tok0 = tok0;
  k.max_len = max_len;
  const auto f32 = q.options().dtype(at::kFloat);
  auto scores = at::empty({(int64_t)rows * a.nq * nv}, f32), ml = at::empty({(int64_t)k.splits * rows * a.nq * 2}, f32);
  at::Tensor part;
  if (k.splits > 1) part = at::empty({k.splits, rows, (int64_t)a.nq * a.dv}, f32);
  k.scores = scores.data_ptr<float>();
  k.ml = ml.data_ptr<float>();
  k.part = k.splits > 1 ? part.data_ptr<float>() : nullptr;
  if (a.Dk == 64) launch_tokens_d<64>(a, k, rows, keep_part);
  else if (a.Dk == 128) launch_tokens_d<128>(a, k, rows, keep_part);
  else launch_tokens_d<256>(a, k, rows, keep_part);
  return part;
}

template <int D, int HPW>
void launch_tile_kernel(const ma::Args& a, const ma::TileArgs& k, int total) {
  constexpr size_t lds = 3 * 16 * ma::kTileKeys * ma::kTileHeads * 2 + ma::kTileWaves * ma::kTileKeys * 2 * D;
  auto go = [&](auto kern) {
    allow_lds(kern, lds);
    hipLaunchKernelGGL(kern, dim3((total + 7) / 8 * 8, k.splits), dim3(ma::kTileWaves * 64), lds, cur_stream(), a, k, total);
  };
  if (a.nq / a.nkv % HPW == 0) go(ma::mix_tile_kernel<D, HPW, true>);
  else go(ma::mix_tile_kernel<D, HPW, false>);
}

void launch_tiles(const ma::Args& a, const at::Tensor& q, int min_len, int max_q_len, int max_keys) {
  ma::TileArgs k{};
  auto lse = at::empty({(int64_t)a.T * a.nq}, q.options().dtype(at::kFloat)), talk = at::empty({1024}, q.options());
  k.lse = lse.data_ptr<float>();
  k.talk = static_cast<unsigned short*>(talk.data_ptr());
  k.min_len = min_len;
  k.max_len = max_q_len;
  k.tiles = (max_q_len + 15) / 16;
  const int total = a.S * k.tiles, units = total * a.nkv;
  k.vec = a.dv % 4 == 0 && a.gate_ld % 4 == 0 && reinterpret_cast<uintptr_t>(a.gate) % 8 == 0;
  // one workgroup per compute unit: fewer tiles than units split their keys (while a split keeps 8 tiles of 32)
  k.splits = std::max(1, std::min(std::min(4, kNumCUs / total), max_keys / (8 * ma::kTileKeys)));
  at::Tensor part;
  if (k.splits > 1) {
    part = at::empty({(int64_t)k.splits * a.S * max_q_len * a.nq * a.dv}, q.options().dtype(at::kFloat));
    k.part = part.data_ptr<float>();
  }
  if (a.Dk == 64) hipLaunchKernelGGL(ma::mix_lse_kernel<64>, dim3((units + 3) / 4), dim3(256), 0, cur_stream(), a, k, units);
  else hipLaunchKernelGGL(ma::mix_lse_kernel<128>, dim3((units + 3) / 4), dim3(256), 0, cur_stream(), a, k, units);
  const int hpw = a.nq <= 8 ? 1 : a.nq <= 16 ? 2 : 4;
#define SXE_MIX_TILE(D)                                     \
  do {                                                      \
    if (hpw == 1) launch_tile_kernel<D, 1>(a, k, total);     \
    else if (hpw == 2) launch_tile_kernel<D, 2>(a, k, total); \
    else launch_tile_kernel<D, 4>(a, k, total);              \
  } while (0)
  if (a.Dk == 64) SXE_MIX_TILE(64);
  else SXE_MIX_TILE(128);
#undef SXE_MIX_TILE
  if (k.splits > 1) {
    ma::TokArgs r{};
    r.part = k.part;
    r.splits = k.splits;
    r.nt = max_q_len;
    r.min_len = min_len;
    r.max_len = INT_MAX;
    const int rows = a.S * max_q_len;
    hipLaunchKernelGGL(ma::mix_reduce_kernel, dim3(rows, std::min(16, (a.nq * a.dv + 255) / 256)), dim3(256), 0, cur_stream(), a, r);
  }
  SXE_LAUNCH_CHECK();
}

}  // namespace

// q [T, nq, Dk], kc / vc [blocks, nkv, bs, Dk / Dv] -> out [T, nq * dv]; see the top of the file.
// min_q_len / max_q_len bound every q_len. form: 0 = by shape, 1 = any-size kernel (fp32 always), 2 = token
// form, 3 = tile form. splits: KV splits of the token form. part: see mix_attention_parts.
static at::Tensor mix_attention_impl(const at::Tensor& q, const at::Tensor& kc, const at::Tensor& vc, const at::Tensor& block_table,
                         const at::Tensor& q_start, const at::Tensor& q_len, const at::Tensor& kv_len,
                         int64_t min_q_len, int64_t max_q_len, int64_t max_kv_len, int64_t splits, int64_t dk, int64_t dv, double scale, int64_t window,
                         int64_t keep_first, const c10::optional<at::Tensor>& r1, const c10::optional<at::Tensor>& r2,
                         const c10::optional<at::Tensor>& sink, const c10::optional<at::Tensor>& talk,
                         const c10::optional<at::Tensor>& gate, int64_t form, at::Tensor* part) {
  SXE_CHECK_CUDA(q);
  SXE_CHECK(q.dim() == 3 && q.is_contiguous(), "mix_attention: q [T, nq, Dk] contiguous");
  const int64_t T = q.size(0), nq = q.size(1), nkv = kc.size(1), S = block_table.size(0);
  for (auto* c : {&kc, &vc})
    SXE_CHECK(c->dim() == 4 && c->size(1) == nkv && c->stride(3) == 1 && c->stride(2) == c->size(3) &&
                  c->stride(1) == c->size(2) * c->size(3) && c->scalar_type() == q.scalar_type() && c->is_cuda(),
              "mix_attention: caches [blocks, nkv, bs, D]");
  SXE_CHECK(kc.size(0) == vc.size(0) && kc.size(2) == vc.size(2) && kc.size(3) == q.size(2) && kc.size(3) >= dk &&
                vc.size(3) >= dv && nkv > 0 && nq % nkv == 0,
            "mix_attention: head layout");
  SXE_CHECK(block_table.scalar_type() == at::kInt && block_table.is_contiguous() && block_table.dim() == 2 &&
                block_table.is_cuda() && block_table.size(1) * kc.size(2) >= max_kv_len,
            "mix_attention: block_table int32 [S, max_blocks] covering max_kv_len");
  for (auto* t : {&q_start, &q_len, &kv_len})
    SXE_CHECK(t->scalar_type() == at::kInt && t->is_contiguous() && t->numel() == S && t->is_cuda(),
              "mix_attention: q_start/q_len/kv_len int32 [S]");
  auto out = at::empty({T, nq * dv}, q.options());
  if (T == 0 || S == 0 || max_q_len == 0) return out;
  ma::Args a{};
  a.q = q.data_ptr();
  a.kc = kc.data_ptr();
  a.vc = vc.data_ptr();
  a.k_block = kc.stride(0);
  a.v_block = vc.stride(0);
  a.block_table = block_table.data_ptr<int>();
  a.max_blocks = block_table.size(1);
  a.q_start = q_start.data_ptr<int>();
  a.q_len = q_len.data_ptr<int>();
  a.kv_len = kv_len.data_ptr<int>();
  a.S = S;
  a.T = T;
  a.nq = nq;
  a.nkv = nkv;
  a.dk = dk;
  a.dv = dv;
  a.Dk = kc.size(3);
  a.Dv = vc.size(3);
  a.bs = kc.size(2);
  while ((1 << a.bs_shift) < a.bs) ++a.bs_shift;
  a.scale = (float)scale;
  a.window = (int)std::max<int64_t>(0, window);
  a.keep_first = (int)std::max<int64_t>(0, keep_first);
  a.r1 = head_vec(r1, nq, "r1");
  a.r2 = head_vec(r2, nq, "r2");
  SXE_CHECK((a.r1 == nullptr) == (a.r2 == nullptr), "mix_attention: r1 and r2 together");
  a.sink = head_vec(sink, nq, "sink");
  a.talk = head_vec(talk, nq * nq, "talk");
  if (gate.has_value() && gate->defined()) {
    SXE_CHECK(gate->dim() == 2 && gate->stride(1) == 1 && gate->size(0) == T && gate->size(1) == nq * dv &&
                  gate->scalar_type() == q.scalar_type() && gate->is_cuda(),
              "mix_attention: gate [T, nq * dv] like q");
    a.gate = gate->data_ptr();
    a.gate_ld = gate->stride(0);
  }
  a.out = out.data_ptr();
  c10::DeviceGuard g(q.device());
  const int64_t D = kc.size(3);
  const bool mfma = q.scalar_type() == at::kBFloat16 && D == vc.size(3) && (D == 64 || D == 128 || D == 256) &&
                    nq <= ma::kMaxHeads && (1 << a.bs_shift) == a.bs && scale > 0 &&
                    kc.stride(0) % 8 == 0 && vc.stride(0) % 8 == 0 &&
                    reinterpret_cast<uintptr_t>(a.kc) % 16 == 0 && reinterpret_cast<uintptr_t>(a.vc) % 16 == 0;
  const bool tile_ok = mfma && nq <= ma::kTileHeads && D <= 128 && a.bs % ma::kTileKeys == 0;
  SXE_CHECK(form != 2 || mfma, "mix_attention: token form needs bf16 rows of 64, 128 or 256, a scale > 0 and a power-of-two block size");
  SXE_CHECK(form != 3 || tile_ok, "mix_attention: tile form needs bf16 rows of 64 or 128, <= 32 heads, blocks of 32 n");
  if (part != nullptr) {
    SXE_CHECK(mfma && max_q_len == 1 && T == S, "mix_attention_parts: one token per sequence on the matrix-core form");
    const int64_t keys = std::min<int64_t>(max_kv_len, a.window > 0 ? a.window + a.keep_first : max_kv_len);
    *part = launch_tokens(a, q, (int)((keys + 63) / 64 * 64), (int)splits, 0, 1, INT_MAX, true);
    return out;
  }
  if (mfma && form != 1) {
    constexpr int64_t kTileMin = 8;  // shorter runs of new tokens go token by token
    const int64_t tile_min = form == 2 || !tile_ok ? INT_MAX : form == 3 ? 1 : kTileMin;
    const int64_t keys = std::min<int64_t>(max_kv_len, a.window > 0 ? a.window + a.keep_first : max_kv_len);
    if (max_q_len >= tile_min) launch_tiles(a, q, (int)tile_min, (int)max_q_len, (int)keys);
    if (min_q_len < tile_min) {
      // the scores of one launch stay within 256 MiB: long runs of tokens take several
      const int64_t nv = (keys + 63) / 64 * 64;
      const int64_t run = std::min(max_q_len, tile_min - 1);
      const int64_t per = std::max<int64_t>(1, (int64_t(1) << 28) / (S * nq * nv * 4));
      for (int64_t t0 = 0; t0 < run; t0 += per)
        launch_tokens(a, q, (int)nv, (int)splits, (int)t0, (int)std::min(per, run - t0), (int)std::min<int64_t>(tile_min - 1, INT_MAX));
    }
    return out;
  }
  const size_t lds = sizeof(float) * (nq * (dk + dv) + 2 * nq * ma::kGenKeys + 2 * nq);
  SXE_CHECK(lds <= 160 * 1024, "mix_attention: heads x sizes exceed the LDS of one compute unit");
  SXE_DISPATCH_DT(dtype_of(q), D, {
    static bool attr = false;
    if (!attr) {
      SXE_HIP_CHECK(hipFuncSetAttribute(reinterpret_cast<const void*>(&ma::mix_attn_generic_kernel<D>),
                                        hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024));
      attr = true;
    }
    hipLaunchKernelGGL(ma::mix_attn_generic_kernel<D>, dim3(S * max_q_len), dim3(ma::kGenThreads), lds, cur_stream(), a,
                       (int)max_q_len);
  });
  SXE_LAUNCH_CHECK();
  return out;
}

at::Tensor mix_attention(const at::Tensor& q, const at::Tensor& kc, const at::Tensor& vc, const at::Tensor& block_table,
                         const at::Tensor& q_start, const at::Tensor& q_len, const at::Tensor& kv_len, int64_t min_q_len,
                         int64_t max_q_len, int64_t max_kv_len, int64_t splits, int64_t dk, int64_t dv, double scale,
                         int64_t window, int64_t keep_first, const c10::optional<at::Tensor>& r1,
                         const c10::optional<at::Tensor>& r2, const c10::optional<at::Tensor>& sink,
                         const c10::optional<at::Tensor>& talk, const c10::optional<at::Tensor>& gate, int64_t form) {
  return mix_attention_impl(q, kc, vc, block_table, q_start, q_len, kv_len, min_q_len, max_q_len, max_kv_len, splits, dk, dv,
                            scale, window, keep_first, r1, r2, sink, talk, gate, form, nullptr);
}

// Decode (one token per sequence, rows in token order): [out, part]. One split: out as mix_attention's and an
// empty part. Several: out unwritten and part fp32 [splits, T, nq dv], whose sum over the splits (times the
// sigmoid of the gate) is the output -- for a consumer that adds them itself (skinny_gemm_gatesum).
std::vector<at::Tensor> mix_attention_parts(const at::Tensor& q, const at::Tensor& kc, const at::Tensor& vc,
                                            const at::Tensor& block_table, const at::Tensor& q_start,
                                            const at::Tensor& q_len, const at::Tensor& kv_len, int64_t max_kv_len,
                                            int64_t splits, int64_t dk, int64_t dv, double scale, int64_t window,
                                            int64_t keep_first, const c10::optional<at::Tensor>& r1,
                                            const c10::optional<at::Tensor>& r2, const c10::optional<at::Tensor>& sink,
                                            const c10::optional<at::Tensor>& talk, const c10::optional<at::Tensor>& gate) {
  at::Tensor part;
  auto out = mix_attention_impl(q, kc, vc, block_table, q_start, q_len, kv_len, 1, 1, max_kv_len, splits, dk, dv, scale,
                                window, keep_first, r1, r2, sink, talk, gate, 0, &part);
  if (!part.defined()) part = at::empty({0}, q.options().dtype(at::kFloat));
  return {out, part};
}

}  // namespace sxe

TORCH_LIBRARY_FRAGMENT(sxe, m) {
  m.def("mix_attention(Tensor q, Tensor kc, Tensor vc, Tensor block_table, Tensor q_start, Tensor q_len, Tensor kv_len, "
        "int min_q_len, int max_q_len, int max_kv_len, int splits, int dk, int dv, float scale, int window, int keep_first, Tensor? r1, Tensor? r2, "
        "Tensor? sink, Tensor? talk, Tensor? gate, int form=0) -> Tensor");
  m.def("mix_attention_parts(Tensor q, Tensor kc, Tensor vc, Tensor block_table, Tensor q_start, Tensor q_len, "
        "Tensor kv_len, int max_kv_len, int splits, int dk, int dv, float scale, int window, int keep_first, Tensor? r1, "
        "Tensor? r2, Tensor? sink, Tensor? talk, Tensor? gate) -> Tensor[]");
}
TORCH_LIBRARY_IMPL(sxe, CUDA, m) {
  m.impl("mix_attention", &sxe::mix_attention);
  m.impl("mix_attention_parts", &sxe::mix_attention_parts);
}
