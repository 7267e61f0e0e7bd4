// The matrix-core tile that a product per head is made of (heads_linear.hip, latent.hip): 16 tokens x NT
// tiles of 16 output columns, bfloat16 operands straight from memory (a head's matrix is small and stays
// in L2 for all its tokens), float32 sums.
#pragma once

#include "common.h"

namespace psamd {

typedef __attribute__((ext_vector_type(8))) __bf16 head_bf16x8;
typedef __attribute__((ext_vector_type(4))) float head_f32x4;

// Operand layout of v_mfma_f32_16x16x32_bf16: lane l supplies row l % 16, k = 8 * (l / 16) + [0, 8) of both
// operands and receives C[4 * (l / 16) + v][l % 16]; C's rows are rows of w, its columns tokens. `x` and
// `w[nt]` are this lane's rows, without the lane's k offset; K is a multiple of 8 (a piece of 8 is inside or
// outside as a whole: outside, the tokens' piece is zeros and the matrix's any piece of its row). The loads of
// U steps are in flight together.
template <int NT, int U>
__device__ __forceinline__ void head_tile(const bf16_t* __restrict__ x, const bf16_t* const (&w)[NT], int K, int g,
                                          head_f32x4 (&acc)[NT]) {
  head_bf16x8 zero;
#pragma unroll
  for (int i = 0; i < 8; ++i) zero[i] = static_cast<__bf16>(0.f);
#pragma unroll
  for (int nt = 0; nt < NT; ++nt) acc[nt] = head_f32x4{0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < K; k0 += 32 * U) {
    head_bf16x8 a[U][NT], b[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = k0 + 32 * u + 8 * g;
      const int at = k < K ? k : 0;
      b[u] = *reinterpret_cast<const head_bf16x8*>(x + at);
#pragma unroll
      for (int nt = 0; nt < NT; ++nt) a[u][nt] = *reinterpret_cast<const head_bf16x8*>(w[nt] + at);
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const head_bf16x8 bu = k0 + 32 * u + 8 * g < K ? b[u] : zero;
#pragma unroll
      for (int nt = 0; nt < NT; ++nt) acc[nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[u][nt], bu, acc[nt], 0, 0, 0);
    }
  }
}

// Where a wave's tile lies. Up to 16 tokens (FEW) the four waves of a workgroup take 16 columns each of
// the same tokens, otherwise 16 tokens each of the same NT * 16 columns.
template <int NT, bool FEW>
struct HeadPlace {
  int64_t m0;
  int n0;
  __device__ __forceinline__ HeadPlace(int wave)
      : m0(FEW ? 0 : (static_cast<int64_t>(blockIdx.y) * 4 + wave) * 16),
        n0(FEW ? (static_cast<int>(blockIdx.x) * 4 + wave) * 16 : static_cast<int>(blockIdx.x) * NT * 16) {}
};

}  // namespace psamd
