// LDS tiles of [rows][D] bf16 (D = 64 or 128) for kernels whose tiles arrive by direct-to-LDS loads: XOR
// swizzle, hoisted per-lane read offsets and the loader. Read forms and lane maps are those of sxe_mfma.h
// (ds_read_b128 of a row, ds_read_b64_tr_b16 for a transposed operand).
#pragma once
#include "sxe_mfma.h"

namespace sxe {
namespace tl {
using namespace mf;

// swizzle of a row: position c of row r holds chunk c ^ swz(r)
template <int D>
__device__ __forceinline__ int swz(int row) {
  return (((row & 3) << 2) | ((row >> 2) & 3)) & (D >= 128 ? 15 : D / 8 - 1);
}
template <int D>
__device__ __forceinline__ int off(int row, int ch) {
  return row * (2 * D) + 16 * (ch ^ swz<D>(row));
}

// Byte offsets of a lane's reads, for tile rows that start at a multiple of 16:
//   row[s]: row (lane & 31), chunk 2 s + (lane >> 5) -- operand of k-step s
//   tr[t]:  the transposed operand of columns 32 t .., 16 rows (k order of an accumulator used as B operand)
template <int D>
struct LaneOffs {
  int row[D / 16], tr[D / 32][2];
  __device__ __forceinline__ void init(int lane) {
    const int r = lane & 31, h = lane >> 5;
#pragma unroll
    for (int s = 0; s < D / 16; ++s) row[s] = off<D>(r, 2 * s + h);
    const int g = lane >> 4, i = lane & 15, q = i >> 2, p = i & 3, hh = g >> 1;
#pragma unroll
    for (int t = 0; t < D / 32; ++t) {
      const int ch = 4 * t + 2 * (g & 1) + (p >> 1);
      tr[t][0] = off<D>(4 * hh + q, ch) + 8 * (p & 1);
      tr[t][1] = off<D>(4 * hh + q + 8, ch) + 8 * (p & 1);
    }
  }
};
__device__ __forceinline__ bf16x8 row_at(const char* base, int o) { return *reinterpret_cast<const bf16x8*>(base + o); }
__device__ __forceinline__ bf16x8 tr_at(const char* base, const int (&o)[2]) {
  const i16x4 lo = lds_tr(base, o[0]), hi = lds_tr(base, o[1]);
  return __builtin_bit_cast(bf16x8, __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7));
}

extern __shared__ __attribute__((aligned(16))) char lds[];  // a kernel's dynamic LDS

// 16 bytes per lane from `src` to lane-linear LDS at the wave-uniform `dst`. Inline asm, so that the compiler's
// wait counts do not tie it to the LDS reads in between: consumers run wait_loads() and a barrier.
__device__ __forceinline__ void glds16(const void* src, char* dst) {
  const unsigned a = __builtin_amdgcn_readfirstlane((unsigned)(uintptr_t)(__attribute__((address_space(3))) char*)lds +
                                                    (unsigned)(dst - lds));
  asm volatile("s_mov_b32 m0, %0\n\tglobal_load_lds_dwordx4 %1, off" ::"s"(a), "v"(src) : "memory", "m0");
}
__device__ __forceinline__ void wait_loads() { __builtin_amdgcn_s_waitcnt(0x0F70); }

// ROWS rows of a tile by NW waves; row_ptr(r): global start of tile row r, of which `chunks` 16-byte chunks exist
// (positions beyond them repeat the last chunk: they meet zeros of the other operand or unused outputs)
template <int ROWS, int D, int NW, typename F>
__device__ __forceinline__ void load_tile(char* dst, int chunks, F row_ptr) {
  constexpr int CH = D / 8, RPK = 64 / CH;
  static_assert(ROWS % (RPK * NW) == 0, "rows split evenly over the waves");
  const int lane = threadIdx.x & 63, w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
#pragma unroll
  for (int i = 0; i < ROWS / RPK / NW; ++i) {
    const int n = i * NW + w, row = RPK * n + lane / CH, ch = min((lane % CH) ^ swz<D>(row), chunks - 1);
    glds16(row_ptr(row) + ch * 8, dst + n * 1024);
  }
}

}  // namespace tl
}  // namespace sxe
