// Tile loops of the mixer library's own "NT" products (both operands contiguous along the reduction): fp32 -- true
// fp32, no reduced-precision matrix mode -- on LDS-tiled vector FMAs, bf16 on the matrix cores.  Workgroups of
// kTileThreads; row r of A begins at element a_off(r), row n of B at b_off + n * K.
#pragma once

#include "mixers_common.cuh"

namespace swm {

constexpr int TM = 32, TN = 64, TK = 32, kTileThreads = 256;

// acc[2][4] of thread (ty, tx): rows 2 * ty + {0, 1}, columns tx + 16 * {0..3} of the tile
template <typename T, typename OffOf>
__device__ __forceinline__ void tile_gemm(float (&acc)[2][4], const void* __restrict__ a, OffOf a_off, int rows,
                                          const void* __restrict__ b, int64_t b_off, int n0, int N, int K,
                                          float (*As)[TK + 1], float (*Bs)[TK + 1]) {
  const int tid = threadIdx.x, ty = tid >> 4, tx = tid & 15;
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = 0.0f;
  for (int k0 = 0; k0 < K; k0 += TK) {
    // A tile: 32 x 32 = 1024 values, 4 per thread; B tile: 64 x 32 = 2048 values, 8 per thread
#pragma unroll
    for (int it = 0; it < 4; ++it) {
      const int e = tid + it * kTileThreads, r = e >> 5, k = e & 31;
      float v = 0.0f;
      if (r < rows && k0 + k < K) v = ld<T>(a, a_off(r) + k0 + k);
      As[r][k] = v;
    }
#pragma unroll
    for (int it = 0; it < 8; ++it) {
      const int e = tid + it * kTileThreads, r = e >> 5, k = e & 31;
      float v = 0.0f;
      if (n0 + r < N && k0 + k < K) v = ld<T>(b, b_off + (int64_t)(n0 + r) * K + k0 + k);
      Bs[r][k] = v;
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < TK; ++k) {
      const float a0 = As[2 * ty][k], a1 = As[2 * ty + 1][k];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float bv = Bs[tx + 16 * j][k];
        acc[0][j] += a0 * bv;
        acc[1][j] += a1 * bv;
      }
    }
    __syncthreads();
  }
}

// bf16 on the matrix cores:
// 64 x 64 output tile per workgroup, one 32 x 32 quadrant per wave (v_mfma_f32_32x32x16_bf16, fp32 accumulation);
// stages of 64 reduction steps go global -> LDS as 16-byte vectors.  Both operands are contiguous along the
// reduction and are read with the SAME lane -> k mapping (8 consecutive k per lane, the wave's halves 8 apart),
// so only the accumulator's layout matters: element i of lane l is row 8 * (i / 4) + 4 * (l / 32) + i % 4,
// column l % 32.  VEC: the reduction size and every row's first element are multiples of 8 elements; otherwise elements are
// fetched one by one.
constexpr int MM = 64, MN = 64, MK = 64, MPAD = 8;
using bf16x8 = __attribute__((ext_vector_type(8))) __bf16;
using f32x16 = __attribute__((ext_vector_type(16))) float;

// elements [k, k + 8) of a row of K bf16 numbers, zeros beyond
__device__ __forceinline__ uint4 load8(const uint16_t* __restrict__ row, int k, int K) {
  uint32_t w[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const uint32_t lo = k + 2 * j < K ? row[k + 2 * j] : 0u, hi = k + 2 * j + 1 < K ? row[k + 2 * j + 1] : 0u;
    w[j] = lo | (hi << 16);
  }
  return make_uint4(w[0], w[1], w[2], w[3]);
}

template <bool VEC, typename OffOf>
__device__ __forceinline__ void tile_gemm_mfma(f32x16& acc, const uint16_t* __restrict__ a, OffOf a_off, int rows,
                                               const uint16_t* __restrict__ b, int64_t b_off, int n0, int N, int K,
                                               uint16_t (*As)[MK + MPAD], uint16_t (*Bs)[MK + MPAD]) {
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int wm = wave >> 1, wn = wave & 1;
#pragma unroll
  for (int i = 0; i < 16; ++i) acc[i] = 0.0f;
  for (int k0 = 0; k0 < K; k0 += MK) {
#pragma unroll
    for (int it = 0; it < 2; ++it) {
      const int e = tid + it * kTileThreads, r = e >> 3, k = (e & 7) * 8;
      uint4 va = make_uint4(0u, 0u, 0u, 0u), vb = make_uint4(0u, 0u, 0u, 0u);
      if constexpr (VEC) {
        if (r < rows && k0 + k < K) va = *reinterpret_cast<const uint4*>(a + a_off(r) + k0 + k);
        if (n0 + r < N && k0 + k < K) vb = *reinterpret_cast<const uint4*>(b + b_off + (int64_t)(n0 + r) * K + k0 + k);
      } else {
        if (r < rows) va = load8(a + a_off(r), k0 + k, K);
        if (n0 + r < N) vb = load8(b + b_off + (int64_t)(n0 + r) * K, k0 + k, K);
      }
      *reinterpret_cast<uint4*>(&As[r][k]) = va;
      *reinterpret_cast<uint4*>(&Bs[r][k]) = vb;
    }
    __syncthreads();
#pragma unroll
    for (int ks = 0; ks < MK; ks += 16) {
      const bf16x8 av = *reinterpret_cast<const bf16x8*>(&As[wm * 32 + (lane & 31)][ks + 8 * (lane >> 5)]);
      const bf16x8 bv = *reinterpret_cast<const bf16x8*>(&Bs[wn * 32 + (lane & 31)][ks + 8 * (lane >> 5)]);
      acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(av, bv, acc, 0, 0, 0);
    }
    __syncthreads();
  }
}

// calls f(row in tile, column in tile, value) for the 16 accumulator elements of this lane
template <typename F>
__device__ __forceinline__ void for_each_acc(const f32x16& acc, F&& f) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int wm = wave >> 1, wn = wave & 1;
#pragma unroll
  for (int i = 0; i < 16; ++i) f(wm * 32 + 8 * (i / 4) + 4 * (lane >> 5) + (i % 4), wn * 32 + (lane & 31), acc[i]);
}

}  // namespace swm
