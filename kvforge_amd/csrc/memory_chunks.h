// What the kernels that take a matrix memory over chunks of tokens share: staging rows into LDS, and
// matrix products in true fp32.
//
// The matrix products of the chunks run on v_mfma_f32_16x16x4_f32 (true fp32): D[i][j] += sum_k
// A[i][k] B[k][j], k = 0..3; lane l gives A[l % 16][l / 16], B[l / 16][l % 16] and holds
// D[4 (l / 16) + v][l % 16].  The four lane groups stand for four *neighbouring* k each (group g
// takes k = k0 + 4 g + e in instruction e of four): a lane's operands for four instructions are 16
// consecutive bytes, and a product's result lies in the lanes as the next product's B operand.
#pragma once
#include "common.h"

namespace {
typedef float f32x4 __attribute__((ext_vector_type(4)));
__device__ __forceinline__ f32x4 zero4() { return f32x4{0.f, 0.f, 0.f, 0.f}; }
__device__ __forceinline__ float softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float sigmoidf(float z) { return 1.f / (1.f + expf(-z)); }

// Loads on their way into LDS are never predicated: a lane without an element of its own reads the
// rows' first one and the value is cleared when it is put down, so that no load waits for another.
//
// Four neighbouring elements e .. e + 3 of a head's row p; VEC: heads and rows start on 16 bytes and dk
// is a multiple of four, so that they are one load and lie inside the row or outside it together.
template <bool VEC>
__device__ __forceinline__ f32x4 load_four(const float* __restrict__ safe, const float* p, int e, int dk, bool ok) {
  if constexpr (VEC) {
    return *reinterpret_cast<const f32x4*>(ok && e < dk ? p + e : safe);
  } else {
    f32x4 v;
#pragma unroll
    for (int y = 0; y < 4; ++y) v[y] = *(ok && e + y < dk ? p + e + y : safe);
    return v;
  }
}
__device__ __forceinline__ f32x4 clear_past(f32x4 v, int e, int dk, bool ok) {
#pragma unroll
  for (int y = 0; y < 4; ++y) v[y] = ok && e + y < dk ? v[y] : 0.f;
  return v;
}

// Rows tb .. tb + cnt - 1 of a head of q or k (columns off .. off + dk - 1) on their way from memory into
// LDS, [CL][DKP + 4], by NT threads: all loads are asked for (`ask`) before the first is put down
// (`put`).  Zeros past the tokens and past dk.
template <int DKP, int CL, int NT, bool VEC> struct StagedRows {
  static constexpr int N = CL * (DKP / 4) / NT;
  static constexpr int ROWS = NT / (DKP / 4);     // a round's rows; a thread has the same elements in every round
  static_assert(N >= 1 && N * NT == CL * (DKP / 4) && ROWS * (DKP / 4) == NT, "whole rounds of threads");
  f32x4 v[N];
  template <typename Args>   // with the rows' stride `ld` and the head size `dk`
  __device__ __forceinline__ void ask(const float* __restrict__ rows, const Args& a, int off, int tb, int cnt) {
    const int t0 = threadIdx.x / (DKP / 4), e = 4 * (threadIdx.x % (DKP / 4));
    const float* p = rows + static_cast<size_t>(tb + t0) * a.ld + off;
    const size_t step = static_cast<size_t>(ROWS) * a.ld;
#pragma unroll
    for (int x = 0; x < N; ++x, p += step) v[x] = load_four<VEC>(rows, p, e, a.dk, t0 + ROWS * x < cnt);
  }
  __device__ __forceinline__ void put(float* dst, int cnt, int dk) const {
    const int t0 = threadIdx.x / (DKP / 4), e = 4 * (threadIdx.x % (DKP / 4));
    float* d = dst + t0 * (DKP + 4) + e;
#pragma unroll
    for (int x = 0; x < N; ++x)
      *reinterpret_cast<f32x4*>(d + x * ROWS * (DKP + 4)) = clear_past(v[x], e, dk, t0 + ROWS * x < cnt);
  }
};

// COLS columns of R rows of `ld` floats from p on, on their way into LDS turned round, [COLS][LLD]:
// element (r, c) lies at c * LLD + r.  Zeros past `rows_ok` rows and `cols_ok` columns (both at least one).
template <int R, int COLS, int NT, int LLD> struct StagedTurned {
  static constexpr int N = R * COLS / NT, ROWS = NT / COLS;
  static_assert(N >= 1 && N * NT == R * COLS && ROWS * COLS == NT, "whole rounds of threads");
  float v[N];
  __device__ __forceinline__ void ask(const float* __restrict__ p, size_t ld, int rows_ok, int cols_ok) {
    const int r0 = threadIdx.x / COLS, c = threadIdx.x % COLS;
    const float* q = p + static_cast<size_t>(r0) * ld + c;
#pragma unroll
    for (int x = 0; x < N; ++x, q += static_cast<size_t>(ROWS) * ld)
      v[x] = *(r0 + ROWS * x < rows_ok && c < cols_ok ? q : p);
  }
  __device__ __forceinline__ void put(float* dst, int rows_ok, int cols_ok) const {
    const int r0 = threadIdx.x / COLS, c = threadIdx.x % COLS;
    float* d = dst + c * LLD + r0;
#pragma unroll
    for (int x = 0; x < N; ++x) d[x * ROWS] = r0 + ROWS * x < rows_ok && c < cols_ok ? v[x] : 0.f;
  }
};

// acc += A B^T over k = 0 .. K - 1 (K a multiple of 16): `ra` and `rb` point at the lane's row of
// either operand, at element 4 (l / 16)
__device__ __forceinline__ f32x4 mma16(const float* ra, const float* rb, f32x4 acc) {
  const f32x4 a4 = *reinterpret_cast<const f32x4*>(ra), b4 = *reinterpret_cast<const f32x4*>(rb);
#pragma unroll
  for (int e = 0; e < 4; ++e) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a4[e], b4[e], acc, 0, 0, 0);
  return acc;
}
template <int K> __device__ __forceinline__ f32x4 mma_rows(const float* ra, const float* rb, f32x4 acc) {
  constexpr int AHEAD = K < 128 ? K / 16 : 8;      // steps whose operands are asked for together
#pragma unroll
  for (int k0 = 0; k0 < K; k0 += 16 * AHEAD) {
    f32x4 a4[AHEAD], b4[AHEAD];
#pragma unroll
    for (int u = 0; u < AHEAD; ++u) {
      a4[u] = *reinterpret_cast<const f32x4*>(ra + k0 + 16 * u);
      b4[u] = *reinterpret_cast<const f32x4*>(rb + k0 + 16 * u);
    }
#pragma unroll
    for (int u = 0; u < AHEAD; ++u)
#pragma unroll
      for (int e = 0; e < 4; ++e) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a4[u][e], b4[u][e], acc, 0, 0, 0);
  }
  return acc;
}
__device__ __forceinline__ f32x4 mma_rows(const float* ra, const float* rb, int K, f32x4 acc) {
  for (int k0 = 0; k0 < K; k0 += 16) acc = mma16(ra + k0, rb + k0, acc);
  return acc;
}

// more LDS than a kernel gets unasked is asked for once per kernel
template <typename F> hipError_t allow_lds(F* kernel, size_t bytes) {
  return hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize,
                             static_cast<int>(bytes));
}
}  // namespace
