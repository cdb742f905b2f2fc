// Linear attention with a per-head decay and a state carried from token to token (gfx950):
//   S_t = decay S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t,   q, k, v = act(projection)
// The state [slots, heads, dim, vdim] is fp32 in every form; a sequence without earlier tokens starts from
// zero whatever its slot holds.
//
//  * step form (decode, short continuations, fp32, any size): one workgroup per (sequence, head, columns of
//    the state); the state's columns stay in registers while the workgroup walks the new tokens.
//  * chunk form (prompts, bf16): over chunks of tokens counted from the first new one, for in-chunk index i
//      1. chunk_state: D = sum_t decay^(n-1-t) k_t v_t^T of every (chunk, head), matrix products over tokens;
//      2. state_scan: element by element through a sequence's chunks, S_in(c+1) = decay^n S_in(c) + D(c); the
//         incoming state replaces D, the last one goes to the sequence's slot;
//      3. chunk_out: o_i = decay^(i+1) S_in^T q_i + sum_(j<=i) decay^(i-j) (q_i . k_j) v_j.
//    1. also leaves the activated keys and values in the projection, so 3. takes its tiles straight to LDS.
//    Everything with a decay or a state in it keeps ~2^-17: the decayed keys of 1. and the state of 3. enter
//    the matrix products as two bf16 numbers (head and remainder); the in-chunk weight of 3. is rounded once,
//    as the operand of the value product, like the other attention kernels' weights.
#include "sxe_common.h"
#include "sxe_mfma.h"
#include "sxe_tile.h"
#include <torch/library.h>
#include <type_traits>

namespace sxe {
namespace la {
using namespace mf;

constexpr int kThreads = 256;

struct Args {
  const void* proj;  // [T, ld]: q | k | v heads
  int64_t ld;
  float* state;      // [slots, H, dim, vdim]
  const float* decay;  // [2, H]: decay, log2(decay)
  const int *q_start, *q_len, *kv_len, *slots;
  void* out;         // [T, H * vdim]
  int H, dim, vdim, nslots, T;
  bool act;
};

__device__ __forceinline__ float silu(float x) { return x / (1.f + expf(-x)); }

// the activated projection as the compute dtype holds it
template <DT T>
__device__ __forceinline__ float fetch(const typename dt_traits<T>::storage* p, bool act) {
  const float v = to_f32<T>(*p);
  return act ? to_f32<T>(from_f32<T>(silu(v))) : v;
}

// ------------------------------------------------------------------------------------------ step form
constexpr int kLanes = 8;              // threads along a state row
constexpr int kRows = kThreads / kLanes;  // state rows per pass
constexpr int kBatch = 16;             // tokens staged together

// V columns per thread (4: vdim % 4 == 0), NP passes of kRows state rows
template <DT T, int V, int NP>
__global__ __launch_bounds__(kThreads) void step_kernel(Args a) {
  using S = typename dt_traits<T>::storage;
  constexpr int VT = kLanes * V;
  extern __shared__ float sm[];
  const int s = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * VT;
  const int n = a.q_len[s], t0 = a.q_start[s], slot = a.slots[s];
  if (n <= 0 || slot < 0 || slot >= a.nslots || t0 < 0 || t0 + n > a.T) return;
  const int dim = a.dim, vdim = a.vdim;
  float* sk = sm;                    // [kBatch][dim]
  float* sq = sk + kBatch * dim;     // [kBatch][dim]
  float* sv = sq + kBatch * dim;     // [kBatch][VT]
  float* red = sv + kBatch * VT;     // [kBatch][4][VT]
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int c = (threadIdx.x % kLanes) * V, r0 = threadIdx.x / kLanes;
  float* st = a.state + ((int64_t)slot * a.H + h) * dim * vdim;
  const bool fresh = a.kv_len[s] == n, cok = v0 + c < vdim;
  const float d = a.decay[h];
  float x[NP][V];
#pragma unroll
  for (int p = 0; p < NP; ++p) {
    const int r = p * kRows + r0;
#pragma unroll
    for (int j = 0; j < V; ++j) x[p][j] = 0.f;
    if (!fresh && r < dim && cok) {
      if constexpr (V == 4) {
        const f32x4 t = *reinterpret_cast<const f32x4*>(st + (int64_t)r * vdim + v0 + c);
#pragma unroll
        for (int j = 0; j < 4; ++j) x[p][j] = t[j];
      } else {
        x[p][0] = st[(int64_t)r * vdim + v0 + c];
      }
    }
  }
  const S* base = static_cast<const S*>(a.proj);
  S* out = static_cast<S*>(a.out);
  for (int b0 = 0; b0 < n; b0 += kBatch) {
    const int nb = min(kBatch, n - b0);
    for (int i = threadIdx.x; i < nb * dim; i += kThreads) {
      const int t = i / dim, r = i - t * dim;
      const S* row = base + (int64_t)(t0 + b0 + t) * a.ld + h * dim + r;
      sq[i] = fetch<T>(row, a.act);
      sk[i] = fetch<T>(row + a.H * dim, a.act);
    }
    for (int i = threadIdx.x; i < nb * VT; i += kThreads) {
      const int t = i / VT, j = i - t * VT;
      sv[i] = v0 + j < vdim ? fetch<T>(base + (int64_t)(t0 + b0 + t) * a.ld + 2 * a.H * dim + h * vdim + v0 + j, a.act) : 0.f;
    }
    __syncthreads();
    for (int t = 0; t < nb; ++t) {
      float o[V], vv[V];
#pragma unroll
      for (int j = 0; j < V; ++j) {
        o[j] = 0.f;
        vv[j] = sv[t * VT + c + j];
      }
#pragma unroll
      for (int p = 0; p < NP; ++p) {
        const int r = p * kRows + r0;
        const float kk = r < dim ? sk[t * dim + r] : 0.f, qq = r < dim ? sq[t * dim + r] : 0.f;
#pragma unroll
        for (int j = 0; j < V; ++j) {
          x[p][j] = d * x[p][j] + kk * vv[j];
          o[j] += qq * x[p][j];
        }
      }
#pragma unroll
      for (int j = 0; j < V; ++j) {
        o[j] += __shfl_xor(o[j], 8, 64);
        o[j] += __shfl_xor(o[j], 16, 64);
        o[j] += __shfl_xor(o[j], 32, 64);
      }
      if (lane < kLanes) {
#pragma unroll
        for (int j = 0; j < V; ++j) red[(t * 4 + wave) * VT + c + j] = o[j];
      }
    }
    __syncthreads();
    for (int i = threadIdx.x; i < nb * VT; i += kThreads) {
      const int t = i / VT, j = i - t * VT;
      const float* r = red + t * 4 * VT + j;
      if (v0 + j < vdim)
        out[(int64_t)(t0 + b0 + t) * a.H * vdim + h * vdim + v0 + j] = from_f32<T>(r[0] + r[VT] + r[2 * VT] + r[3 * VT]);
    }
    // the next batch writes sq / sk / sv only (their readers are past the barrier above) and red after
    // its own first barrier
  }
#pragma unroll
  for (int p = 0; p < NP; ++p) {
    const int r = p * kRows + r0;
    if (r < dim && cok) {
      if constexpr (V == 4) *reinterpret_cast<f32x4*>(st + (int64_t)r * vdim + v0 + c) = f32x4{x[p][0], x[p][1], x[p][2], x[p][3]};
      else st[(int64_t)r * vdim + v0 + c] = x[p][0];
    }
  }
}

// ----------------------------------------------------------------------------------------- chunk form
constexpr int kTile = 64;    // tokens staged together
constexpr int kChunk = 256;  // tokens of a chunk
constexpr int kOutWaves = kChunk / 32;

// weight decay^n, n >= 0
__device__ __forceinline__ float decay_pow(float lg, int n) { return fast_exp2(lg * (float)n); }

__device__ __forceinline__ bf16x8 load8b(const unsigned short* p, bool ok) {
  u32x4 z = {0u, 0u, 0u, 0u};
  if (ok) z = *reinterpret_cast<const u32x4*>(p);
  return __builtin_bit_cast(bf16x8, z);
}
__device__ __forceinline__ bf16x8 silu8(bf16x8 r) {
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const float x = (float)r[i];
    r[i] = (__bf16)(x * __builtin_amdgcn_rcpf(1.f + fast_exp2(-LOG2E * x)));
  }
  return r;
}

// DP, VP: dim and vdim padded to 64 / 128. grid (H, chunks); d_out [chunks, H, dim, vdim] fp32
template <int DP, int VP>
__global__ __launch_bounds__(kThreads, 2) void chunk_state_kernel(Args a, const int* __restrict chunks, float* __restrict d_out) {
  char *lh = tl::lds, *ll = lh + kTile * 2 * DP, *lv = ll + kTile * 2 * DP;
  const int c = blockIdx.y, h = blockIdx.x;
  const int row0 = chunks[3 * c + 1], n = chunks[3 * c + 2];
  unsigned short* kb = static_cast<unsigned short*>(const_cast<void*>(a.proj)) + (int64_t)row0 * a.ld + (a.H + h) * a.dim;
  unsigned short* vb = static_cast<unsigned short*>(const_cast<void*>(a.proj)) + (int64_t)row0 * a.ld + 2 * a.H * a.dim + h * a.vdim;
  const float lg = a.decay[a.H + h];
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, l32 = lane & 31, hh = lane >> 5;
  constexpr int DT_ = DP / 32, NV = VP / 32 * DT_ / 4;  // wave: one 32-row tile of dim, NV column tiles
  const int dt = w % DT_, vt0 = (w / DT_) * NV;
  f32x16 acc[NV];
#pragma unroll
  for (int j = 0; j < NV; ++j) acc[j] = zero16();
  constexpr int KC = DP / 8, VC = VP / 8, NK = kTile * KC / kThreads, NVL = kTile * VC / kThreads;
  int ok[2], ov[NV][2];  // the lane's transposed-read offsets
  {
    tl::LaneOffs<DP> k;
    tl::LaneOffs<VP> v;
    k.init(lane);
    v.init(lane);
#pragma unroll
    for (int e = 0; e < 2; ++e) {
#pragma unroll
      for (int t = 0; t < DT_; ++t)
        if (t == dt) ok[e] = k.tr[t][e];
#pragma unroll
      for (int t = 0; t < VP / 32; ++t)
#pragma unroll
        for (int j = 0; j < NV; ++j)
          if (t == vt0 + j) ov[j][e] = v.tr[t][e];
    }
  }
  bf16x8 rk[NK], rv[NVL];
  auto load = [&](int t0) {
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int x = threadIdx.x + i * kThreads, t = t0 + x / KC, ch = x % KC;
      rk[i] = load8b(kb + (int64_t)t * a.ld + ch * 8, t < n && ch * 8 < a.dim);
    }
#pragma unroll
    for (int i = 0; i < NVL; ++i) {
      const int x = threadIdx.x + i * kThreads, t = t0 + x / VC, ch = x % VC;
      rv[i] = load8b(vb + (int64_t)t * a.ld + ch * 8, t < n && ch * 8 < a.vdim);
    }
  };
  load(0);
  for (int t0 = 0; t0 < n; t0 += kTile) {
    if (t0) __syncthreads();
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int x = threadIdx.x + i * kThreads, t = x / KC, ch = x % KC;
      bf16x8 k8 = rk[i];
      if (a.act) {
        k8 = silu8(k8);
        if (t0 + t < n && ch * 8 < a.dim) *reinterpret_cast<bf16x8*>(kb + (int64_t)(t0 + t) * a.ld + ch * 8) = k8;
      }
      const float f = t0 + t < n ? decay_pow(lg, n - 1 - t0 - t) : 0.f;
      bf16x8 hi, lo;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float y = (float)k8[e] * f;
        hi[e] = (__bf16)y;
        lo[e] = (__bf16)(y - (float)hi[e]);
      }
      *reinterpret_cast<bf16x8*>(lh + tl::off<DP>(t, ch)) = hi;
      *reinterpret_cast<bf16x8*>(ll + tl::off<DP>(t, ch)) = lo;
    }
#pragma unroll
    for (int i = 0; i < NVL; ++i) {
      const int x = threadIdx.x + i * kThreads, t = x / VC, ch = x % VC;
      bf16x8 v8 = rv[i];
      if (a.act) {
        v8 = silu8(v8);
        if (t0 + t < n && ch * 8 < a.vdim) *reinterpret_cast<bf16x8*>(vb + (int64_t)(t0 + t) * a.ld + ch * 8) = v8;
      }
      *reinterpret_cast<bf16x8*>(lv + tl::off<VP>(t, ch)) = v8;
    }
    __syncthreads();
    if (t0 + kTile < n) load(t0 + kTile);
#pragma unroll
    for (int s = 0; s < kTile / 16; ++s) {
      const bf16x8 ah = tl::tr_at(lh + 16 * s * 2 * DP, ok), al = tl::tr_at(ll + 16 * s * 2 * DP, ok);
#pragma unroll
      for (int j = 0; j < NV; ++j) {
        const bf16x8 b = tl::tr_at(lv + 16 * s * 2 * VP, ov[j]);
        acc[j] = mfma(ah, b, acc[j]);
        acc[j] = mfma(al, b, acc[j]);
      }
    }
  }
  float* o = d_out + ((int64_t)c * a.H + h) * a.dim * a.vdim;
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int v = (vt0 + j) * 32 + l32;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int d = dt * 32 + acc_row(i, hh);
      if (d < a.dim && v < a.vdim) o[(int64_t)d * a.vdim + v] = acc[j][i];
    }
  }
}

// grid (sequences, H, ceil(dim * vdim / 1024)); buf: D on entry, the incoming state as (bf16 head << 16 | bf16
// remainder) on exit
__global__ __launch_bounds__(kThreads) void state_scan_kernel(Args a, const int* __restrict chunks, int nchunks, float* buf) {
  const int s = blockIdx.x, h = blockIdx.y, e = (blockIdx.z * kThreads + threadIdx.x) * 4, N = a.dim * a.vdim;
  const int n = a.q_len[s], slot = a.slots[s];
  if (n <= 0 || slot < 0 || slot >= a.nslots || e >= N) return;
  int c = 0;
  while (c < nchunks && chunks[3 * c] != s) ++c;
  float* st = a.state + ((int64_t)slot * a.H + h) * N + e;
  f32x4 x = {0.f, 0.f, 0.f, 0.f};
  if (a.kv_len[s] != n) x = *reinterpret_cast<const f32x4*>(st);
  const float lg = a.decay[a.H + h];
  int last = c;
  while (last < nchunks && chunks[3 * last] == s) ++last;
  constexpr int U = 4;  // chunks in flight
  const int64_t step = (int64_t)a.H * N;
  float* p = buf + ((int64_t)c * a.H + h) * N + e;
  for (; c < last; c += U, p += U * step) {
    f32x4 d[U];
#pragma unroll
    for (int i = 0; i < U; ++i)
      if (c + i < last) d[i] = *reinterpret_cast<const f32x4*>(p + i * step);
#pragma unroll
    for (int i = 0; i < U; ++i) {
      if (c + i >= last) break;
      unsigned u[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const unsigned short hi = f32_to_bf16(x[j]), lo = f32_to_bf16(x[j] - bf16_to_f32(hi));
        u[j] = ((unsigned)hi << 16) | lo;
      }
      *reinterpret_cast<u32x4*>(p + i * step) = u32x4{u[0], u[1], u[2], u[3]};
      const float f = decay_pow(lg, chunks[3 * (c + i) + 2]);
#pragma unroll
      for (int j = 0; j < 4; ++j) x[j] = f * x[j] + d[i][j];
    }
  }
  *reinterpret_cast<f32x4*>(st) = x;
}

// grid (H, chunks): 8 waves of 32 queries each. k and v of proj hold activated values already.
template <int DP, int VP>
__global__ __launch_bounds__(64 * kOutWaves, 1) void chunk_out_kernel(Args a, const int* __restrict chunks,
                                                                      const float* __restrict buf) {
  constexpr int SLOT = kTile * (2 * DP + 2 * VP), NS = DP / 16, NV = VP / 32, VC = VP / 8;
  char *slot0 = tl::lds, *ls = tl::lds + SLOT;  // the second slot takes the state's place
  const int c = blockIdx.y, h = blockIdx.x;
  const int sq = chunks[3 * c], row0 = chunks[3 * c + 1], n = chunks[3 * c + 2], ntiles = (n + kTile - 1) / kTile;
  const bool empty = a.kv_len[sq] == a.q_len[sq] && row0 == a.q_start[sq];  // nothing comes in
  const unsigned short* base = static_cast<const unsigned short*>(a.proj) + (int64_t)row0 * a.ld;
  const unsigned short *qb = base + h * a.dim, *kb = base + (a.H + h) * a.dim, *vb = base + 2 * a.H * a.dim + h * a.vdim;
  const float lg = a.decay[a.H + h];
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, l32 = lane & 31, hh = lane >> 5;
  const int q0 = (w < kOutWaves / 2 ? w : kOutWaves + kOutWaves / 2 - 1 - w) * 32;  // a SIMD's two waves: one early, one late
  const int iq = q0 + l32;
  auto issue = [&](int t, char* slot) {
    auto row = [&](int r) { return (int64_t)min(t * kTile + r, n - 1) * a.ld; };
    tl::load_tile<kTile, DP, kOutWaves>(slot, a.dim / 8, [&](int r) { return kb + row(r); });
    tl::load_tile<kTile, VP, kOutWaves>(slot + kTile * 2 * DP, a.vdim / 8, [&](int r) { return vb + row(r); });
  };
  issue(0, slot0);
  bf16x8 qf[NS];
#pragma unroll
  for (int s = 0; s < NS; ++s) {
    qf[s] = load8b(qb + (int64_t)min(iq, n - 1) * a.ld + 16 * s + 8 * hh, 16 * s + 8 * hh < a.dim);
    if (a.act) qf[s] = silu8(qf[s]);
  }
  tl::LaneOffs<DP> ok;
  tl::LaneOffs<VP> ov;
  ok.init(lane);
  ov.init(lane);
  f32x16 acc[NV];
#pragma unroll
  for (int j = 0; j < NV; ++j) acc[j] = zero16();

  // ---- decay^(i+1) S_in^T q_i
  if (!empty) {
    char *lh = ls, *ll = ls + DP * 2 * VP;
    const unsigned* sp = reinterpret_cast<const unsigned*>(buf) + ((int64_t)c * a.H + h) * a.dim * a.vdim;
    for (int x = threadIdx.x; x < DP * VC; x += 64 * kOutWaves) {
      const int d = x / VC, ch = x % VC;
      u32x4 u0 = {0u, 0u, 0u, 0u}, u1 = {0u, 0u, 0u, 0u};
      if (d < a.dim && ch * 8 < a.vdim) {
        u0 = *reinterpret_cast<const u32x4*>(sp + (int64_t)d * a.vdim + ch * 8);
        u1 = *reinterpret_cast<const u32x4*>(sp + (int64_t)d * a.vdim + ch * 8 + 4);
      }
      u32x4 hi, lo;
      hi[0] = (u0[0] >> 16) | (u0[1] & 0xffff0000u);
      hi[1] = (u0[2] >> 16) | (u0[3] & 0xffff0000u);
      hi[2] = (u1[0] >> 16) | (u1[1] & 0xffff0000u);
      hi[3] = (u1[2] >> 16) | (u1[3] & 0xffff0000u);
      lo[0] = (u0[0] & 0xffffu) | (u0[1] << 16);
      lo[1] = (u0[2] & 0xffffu) | (u0[3] << 16);
      lo[2] = (u1[0] & 0xffffu) | (u1[1] << 16);
      lo[3] = (u1[2] & 0xffffu) | (u1[3] << 16);
      *reinterpret_cast<u32x4*>(lh + tl::off<VP>(d, ch)) = hi;
      *reinterpret_cast<u32x4*>(ll + tl::off<VP>(d, ch)) = lo;
    }
    __syncthreads();
#pragma unroll
    for (int s = 0; s < NS; ++s) {
      // the query fragment in the transposed reads' k order: lanes of the two halves exchange 8 bytes
      const u32x4 u = __builtin_bit_cast(u32x4, qf[s]);
      const auto x = __builtin_amdgcn_permlane32_swap(u[0], u[2], false, false);
      const auto y = __builtin_amdgcn_permlane32_swap(u[1], u[3], false, false);
      const bf16x8 q = __builtin_bit_cast(bf16x8, u32x4{x[0], y[0], x[1], y[1]});
#pragma unroll
      for (int j = 0; j < NV; ++j) {
        acc[j] = mfma(tl::tr_at(lh + 16 * s * 2 * VP, ov.tr[j]), q, acc[j]);
        acc[j] = mfma(tl::tr_at(ll + 16 * s * 2 * VP, ov.tr[j]), q, acc[j]);
      }
    }
    const float f = decay_pow(lg, iq + 1);
#pragma unroll
    for (int j = 0; j < NV; ++j)
#pragma unroll
      for (int i = 0; i < 16; ++i) acc[j][i] *= f;
  }
  float fk[16];  // decay from a key of a 32-key block to the block's last key
#pragma unroll
  for (int i = 0; i < 16; ++i) fk[i] = decay_pow(lg, 31 - acc_row(i, hh));
  tl::wait_loads();
  __syncthreads();

  // ---- the chunk's keys up to the query
  auto step = [&](int t, auto slot) {
    constexpr int CUR = decltype(slot)::value;
    const char* lk = CUR ? ls : slot0;
    const char* lv = lk + kTile * 2 * DP;
    if (t + 1 < ntiles) issue(t + 1, CUR ? slot0 : ls);
#pragma unroll
    for (int kt = 0; kt < 2; ++kt) {
      const int j0 = t * kTile + kt * 32;
      if (j0 > q0) continue;  // wave-uniform
      f32x16 sc = zero16();
#pragma unroll
      for (int s = 0; s < NS; ++s) sc = mfma(tl::row_at(lk + kt * 32 * 2 * DP, ok.row[s]), qf[s], sc);
      if (j0 < q0) {
        const float f = decay_pow(lg, iq - j0 - 31);
#pragma unroll
        for (int i = 0; i < 16; ++i) sc[i] *= f * fk[i];
      } else {
#pragma unroll
        for (int i = 0; i < 16; ++i) {
          const int dist = l32 - acc_row(i, hh);
          sc[i] = dist >= 0 ? sc[i] * decay_pow(lg, dist) : 0.f;
        }
      }
#pragma unroll
      for (int x = 0; x < 2; ++x) {
        const bf16x8 p = acc_to_b(sc, x);
#pragma unroll
        for (int j = 0; j < NV; ++j) acc[j] = mfma(tl::tr_at(lv + (kt * 32 + 16 * x) * 2 * VP, ov.tr[j]), p, acc[j]);
      }
    }
    tl::wait_loads();
    __syncthreads();
  };
  for (int t = 0; t < ntiles; t += 2) {
    step(t, std::integral_constant<int, 0>{});
    if (t + 1 < ntiles) step(t + 1, std::integral_constant<int, 1>{});
  }
  if (iq < n) {
    unsigned short* o = static_cast<unsigned short*>(a.out) + (int64_t)(row0 + iq) * a.H * a.vdim + h * a.vdim;
#pragma unroll
    for (int j = 0; j < NV; ++j)
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        const int v = j * 32 + 8 * g + 4 * hh;
        if (v < a.vdim) {
          u16x4 r;
#pragma unroll
          for (int e = 0; e < 4; ++e) r[e] = f32_to_bf16(acc[j][4 * g + e]);
          *reinterpret_cast<u16x4*>(o + v) = r;
        }
      }
  }
}

template <DT D, int V, typename F>
void dispatch_step(int np, F go) {
  if (np <= 1) go(step_kernel<D, V, 1>);
  else if (np <= 2) go(step_kernel<D, V, 2>);
  else if (np <= 4) go(step_kernel<D, V, 4>);
  else if (np <= 8) go(step_kernel<D, V, 8>);
  else go(step_kernel<D, V, 16>);
}

Args check_args(const at::Tensor& proj, at::Tensor& state, const at::Tensor& decay, const at::Tensor& q_start,
                const at::Tensor& q_len, const at::Tensor& kv_len, const at::Tensor& slots, int64_t H, int64_t dim,
                int64_t vdim, bool act, at::Tensor& out) {
  SXE_CHECK_CUDA(proj);
  SXE_CHECK(proj.dim() == 2 && proj.stride(1) == 1 && proj.size(1) >= H * (2 * dim + vdim), "decay_attention: proj [T, q | k | v]");
  SXE_CHECK(state.is_cuda() && state.is_contiguous() && state.scalar_type() == at::kFloat && state.dim() == 4 &&
                state.size(1) == H && state.size(2) == dim && state.size(3) == vdim,
            "decay_attention: state fp32 [slots, heads, dim, vdim]");
  SXE_CHECK(decay.is_cuda() && decay.is_contiguous() && decay.scalar_type() == at::kFloat && decay.numel() == 2 * H,
            "decay_attention: decay fp32 [2, heads]");
  const int64_t S = q_start.numel();
  for (const auto* t : {&q_start, &q_len, &kv_len, &slots})
    SXE_CHECK(t->is_cuda() && t->is_contiguous() && t->scalar_type() == at::kInt && t->numel() == S,
              "decay_attention: int32 [sequences]");
  out = at::empty({proj.size(0), H * vdim}, proj.options());
  return Args{proj.data_ptr(), proj.stride(0), state.data_ptr<float>(), decay.data_ptr<float>(), q_start.data_ptr<int>(),
              q_len.data_ptr<int>(), kv_len.data_ptr<int>(), slots.data_ptr<int>(), out.data_ptr(), (int)H, (int)dim,
              (int)vdim, (int)state.size(0), (int)proj.size(0), act};
}

}  // namespace la

at::Tensor decay_attention_step(const at::Tensor& proj, at::Tensor state, const at::Tensor& decay, const at::Tensor& q_start,
                                const at::Tensor& q_len, const at::Tensor& kv_len, const at::Tensor& slots, int64_t H,
                                int64_t dim, int64_t vdim, bool act) {
  at::Tensor out;
  c10::DeviceGuard g(proj.device());
  const la::Args a = la::check_args(proj, state, decay, q_start, q_len, kv_len, slots, H, dim, vdim, act, out);
  const int64_t S = q_start.numel();
  if (S == 0 || proj.size(0) == 0) return out;
  SXE_CHECK(dim <= 16 * la::kRows, "decay_attention: head size ", dim, " above ", 16 * la::kRows);
  SXE_CHECK(H <= 65535 && vdim <= 65535, "decay_attention: sizes");
  const int V = vdim % 4 == 0 ? 4 : 1, VT = la::kLanes * V, np = (int)((dim + la::kRows - 1) / la::kRows);
  const size_t lds = sizeof(float) * (la::kBatch * (2 * dim + VT) + la::kBatch * 4 * VT);
  const dim3 grid(S, H, (vdim + VT - 1) / VT);
  auto go = [&](auto kern) {
    SXE_HIP_CHECK(hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    hipLaunchKernelGGL(kern, grid, dim3(la::kThreads), lds, cur_stream(), a);
  };
  SXE_CHECK(proj.scalar_type() == at::kFloat || proj.scalar_type() == at::kBFloat16, "decay_attention: fp32 or bf16");
  if (proj.scalar_type() == at::kFloat) {
    if (V == 4) la::dispatch_step<DT::F32, 4>(np, go);
    else la::dispatch_step<DT::F32, 1>(np, go);
  } else {
    if (V == 4) la::dispatch_step<DT::BF16, 4>(np, go);
    else la::dispatch_step<DT::BF16, 1>(np, go);
  }
  SXE_LAUNCH_CHECK();
  return out;
}

// chunks int32 [n, 3]: (sequence, first row, rows <= kChunk), a sequence's chunks in order and side by side. With an
// activation, the k and v columns of proj are replaced by their activated values.
at::Tensor decay_attention_chunk(at::Tensor proj, at::Tensor state, const at::Tensor& decay, const at::Tensor& q_start,
                                 const at::Tensor& q_len, const at::Tensor& kv_len, const at::Tensor& slots,
                                 const at::Tensor& chunks, int64_t size, int64_t H, int64_t dim, int64_t vdim, bool act) {
  at::Tensor out;
  c10::DeviceGuard g(proj.device());
  const la::Args a = la::check_args(proj, state, decay, q_start, q_len, kv_len, slots, H, dim, vdim, act, out);
  SXE_CHECK(proj.scalar_type() == at::kBFloat16 && dim % 8 == 0 && vdim % 8 == 0 && dim <= 128 && vdim <= 128 &&
                proj.stride(0) % 8 == 0 && reinterpret_cast<uintptr_t>(proj.data_ptr()) % 16 == 0,
            "decay_attention: chunk form takes bf16, sizes up to 128 in multiples of 8");
  SXE_CHECK(chunks.is_cuda() && chunks.scalar_type() == at::kInt && chunks.is_contiguous() && chunks.dim() == 2 &&
                chunks.size(1) == 3 && size == la::kChunk, "decay_attention: chunks int32 [n, 3] of up to ", la::kChunk, " rows");
  const int64_t S = q_start.numel(), nc = chunks.size(0);
  if (S == 0 || nc == 0) return out;
  SXE_CHECK(H <= 65535 && nc <= 65535, "decay_attention: sizes");
  auto buf = at::empty({nc, H, dim, vdim}, proj.options().dtype(at::kFloat));
  auto go = [&](auto ks, auto ko, int DP, int VP) {
    const size_t l1 = la::kTile * (4 * DP + 2 * VP), slot = la::kTile * (2 * DP + 2 * VP);
    const size_t l3 = slot + std::max<size_t>(slot, 4 * DP * VP);
    SXE_HIP_CHECK(hipFuncSetAttribute((const void*)ks, hipFuncAttributeMaxDynamicSharedMemorySize, (int)l1));
    SXE_HIP_CHECK(hipFuncSetAttribute((const void*)ko, hipFuncAttributeMaxDynamicSharedMemorySize, (int)l3));
    hipLaunchKernelGGL(ks, dim3(H, nc), dim3(la::kThreads), l1, cur_stream(), a, chunks.data_ptr<int>(), buf.data_ptr<float>());
    hipLaunchKernelGGL(la::state_scan_kernel, dim3(S, H, (dim * vdim + 4 * la::kThreads - 1) / (4 * la::kThreads)),
                       dim3(la::kThreads), 0, cur_stream(), a, chunks.data_ptr<int>(), (int)nc, buf.data_ptr<float>());
    hipLaunchKernelGGL(ko, dim3(H, nc), dim3(64 * la::kOutWaves), l3, cur_stream(), a, chunks.data_ptr<int>(), buf.data_ptr<float>());
  };
  if (dim <= 64 && vdim <= 64) go(la::chunk_state_kernel<64, 64>, la::chunk_out_kernel<64, 64>, 64, 64);
  else if (dim <= 64) go(la::chunk_state_kernel<64, 128>, la::chunk_out_kernel<64, 128>, 64, 128);
  else if (vdim <= 64) go(la::chunk_state_kernel<128, 64>, la::chunk_out_kernel<128, 64>, 128, 64);
  else go(la::chunk_state_kernel<128, 128>, la::chunk_out_kernel<128, 128>, 128, 128);
  SXE_LAUNCH_CHECK();
  return out;
}

}  // namespace sxe

TORCH_LIBRARY_FRAGMENT(sxe, m) {
  m.def("decay_attention_step(Tensor proj, Tensor(a!) state, Tensor decay, Tensor q_start, Tensor q_len, Tensor kv_len, "
        "Tensor slots, int H, int dim, int vdim, bool act) -> Tensor");
  m.def("decay_attention_chunk(Tensor(b!) proj, Tensor(a!) state, Tensor decay, Tensor q_start, Tensor q_len, Tensor kv_len, "
        "Tensor slots, Tensor chunks, int size, int H, int dim, int vdim, bool act) -> Tensor");
}
TORCH_LIBRARY_IMPL(sxe, CUDA, m) {
  m.impl("decay_attention_step", &sxe::decay_attention_step);
  m.impl("decay_attention_chunk", &sxe::decay_attention_chunk);
}
