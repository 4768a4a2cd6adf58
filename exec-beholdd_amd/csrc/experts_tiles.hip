// The routed experts' products of a step of few rows on the matrix cores, from weights in the tiles layout (gemm_bf16.hip: blocks of
// 16 weight rows x 64 k in operand order), all experts in one launch.
//   experts_tiles   what experts_rows (experts.hip) computes, for bfloat16, K a multiple of 64 and N of 16
// A workgroup owns 16 outputs of one expert (gated: their gate rows and their up rows); its waves split K in 64-wide chunks and feed
// v_mfma_f32_16x16x32_bf16 with the weights as the row operand and up to 16 of the expert's pairs as columns; the waves' sums are
// added in a fixed order through LDS.  An expert's matrix is read once for every 16 of its pairs, as it lies (1 KB of contiguous
// memory a load), four chunks on their way per wave.  A pair's result does not depend on which other pairs the expert has.
#include "common.h"

typedef __bf16 et_bf16x8_t __attribute__((ext_vector_type(8)));
typedef float et_f32x4_t __attribute__((ext_vector_type(4)));
typedef uint32_t et_u32x4_t __attribute__((ext_vector_type(4)));

#define ET_AHEAD 4      // chunks a wave asks for together

__device__ inline et_bf16x8_t et_operand(et_u32x4_t v) { return __builtin_bit_cast(et_bf16x8_t, v); }

// grid (N / 16, E).  in [*][K]: the input of pair p is row p / in_div.  w [E][GATED ? 2 N : N][K] in tiles.
template <bool GATED, int WAVES>
__global__ __launch_bounds__(WAVES * BH_WAVE) void experts_tiles_kernel(const uint16_t* __restrict__ in, int in_div, const int32_t* __restrict__ list,
                                                                       int capacity, const int32_t* __restrict__ counts,
                                                                       const uint16_t* __restrict__ w, void* __restrict__ out_raw, int K, int N,
                                                                       float limit, float alpha, float shift,
                                                                       const float* __restrict__ in_weights) {
  constexpr int SIDES = GATED ? 2 : 1;
  __shared__ float partial[WAVES][SIDES][256];
  const int expert = blockIdx.y, count = counts[expert];
  if (count == 0) return;      // the whole workgroup
  const int lane = threadIdx.x % BH_WAVE, wave = threadIdx.x / BH_WAVE, i = lane % 16, g = lane / 16;
  const int chunks = K / 64, blocks = N / 16;
  const int32_t* mine = list + (size_t)expert * capacity;
  const uint16_t* from_w[SIDES];
#pragma unroll
  for (int t = 0; t < SIDES; ++t)
    from_w[t] = w + ((size_t)expert * SIDES * blocks + blockIdx.x + (size_t)t * blocks) * chunks * 1024 + lane * 8;
  for (int p0 = 0; p0 < count; p0 += 16) {
    const int column = p0 + i < count ? p0 + i : count - 1;      // a column beyond the last pair is computed again and not stored
    const uint16_t* x = in + (size_t)(mine[column] / in_div) * K + 16 * g;
    et_f32x4_t acc[SIDES];
#pragma unroll
    for (int t = 0; t < SIDES; ++t) acc[t] = et_f32x4_t{0.f, 0.f, 0.f, 0.f};
    for (int c0 = wave; c0 < chunks; c0 += WAVES * ET_AHEAD) {
      et_u32x4_t wv[SIDES][ET_AHEAD][2], xv[ET_AHEAD][2];
#pragma unroll
      for (int d = 0; d < ET_AHEAD; ++d) {
        const int c = c0 + d * WAVES < chunks ? c0 + d * WAVES : c0;
#pragma unroll
        for (int t = 0; t < SIDES; ++t)
#pragma unroll
          for (int u = 0; u < 2; ++u)
            wv[t][d][u] = __builtin_nontemporal_load(reinterpret_cast<const et_u32x4_t*>(from_w[t] + (size_t)c * 1024 + u * 512));
      }
#pragma unroll
      for (int d = 0; d < ET_AHEAD; ++d) {
        const int c = c0 + d * WAVES < chunks ? c0 + d * WAVES : c0;
#pragma unroll
        for (int u = 0; u < 2; ++u) xv[d][u] = *reinterpret_cast<const et_u32x4_t*>(x + (size_t)c * 64 + 8 * u);
      }
#pragma unroll
      for (int d = 0; d < ET_AHEAD; ++d) {
        if (c0 + d * WAVES >= chunks) break;      // the same for the whole wave
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
          for (int t = 0; t < SIDES; ++t)
            acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(et_operand(wv[t][d][u]), et_operand(xv[d][u]), acc[t], 0, 0, 0);
      }
    }
    // lane (i, g) holds column (pair) i, weight rows 4 g .. 4 g + 3
    if (p0) __syncthreads();      // the columns before have been read
#pragma unroll
    for (int t = 0; t < SIDES; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) partial[wave][t][i * 16 + 4 * g + r] = acc[t][r];
    __syncthreads();
    for (int e = threadIdx.x; e < 256; e += WAVES * BH_WAVE) {
      const int m = e / 16, n = blockIdx.x * 16 + e % 16;
      if (p0 + m >= count) continue;
      float sum[SIDES];
#pragma unroll
      for (int t = 0; t < SIDES; ++t) {
        sum[t] = 0.f;
#pragma unroll
        for (int v = 0; v < WAVES; ++v) sum[t] += partial[v][t][e];
      }
      const int pair = mine[p0 + m];
      const size_t at = (size_t)pair * N + n;
      if (GATED) {
        const float weight = in_weights ? in_weights[pair] : 1.0f;
        const float gate = fminf(sum[0] * weight, limit), up = fminf(fmaxf(sum[SIDES - 1] * weight, -limit), limit);
        reinterpret_cast<bf16_t*>(out_raw)[at] = from_f32<bf16_t>(gate / (1.0f + expf(-alpha * gate)) * (up + shift));
      } else {
        reinterpret_cast<float*>(out_raw)[at] = sum[0];
      }
    }
  }
}

// Whether this form takes products of these sizes.
extern "C" int bh_experts_tiles_takes(int K, int N) { return K >= 64 && N >= 16 && K % 64 == 0 && N % 16 == 0; }

extern "C" int bh_experts_tiles(const void* in, int in_div, const int32_t* list, int capacity, const int32_t* counts, const void* w, void* out,
                                int E, int K, int N, int gated, float limit, float alpha, float shift, const float* in_weights, hipStream_t stream) {
  BH_REQUIRE(E > 0 && in_div > 0 && capacity > 0 && bh_experts_tiles_takes(K, N), "experts_tiles: K must be a multiple of 64 and N of 16, got %d and %d", K, N);
  BH_REQUIRE(E <= 65535, "experts_tiles: too many experts");
  BH_REQUIRE(((uintptr_t)in | (uintptr_t)w) % 16 == 0, "experts_tiles: operands must be 16-byte aligned");
  const dim3 grid(N / 16, E);
  const bool wide = K >= 8 * 64 * ET_AHEAD;      // enough chunks that eight waves have four each
#define BH_ET(GATED, WAVES)                                                                                                          \
  experts_tiles_kernel<GATED, WAVES><<<grid, WAVES * BH_WAVE, 0, stream>>>((const uint16_t*)in, in_div, list, capacity, counts, (const uint16_t*)w, \
                                                                          out, K, N, limit, alpha, shift, in_weights)
  if (gated) {
    if (wide) BH_ET(true, 8);
    else BH_ET(true, 4);
  } else {
    if (wide) BH_ET(false, 8);
    else BH_ET(false, 4);
  }
#undef BH_ET
  return bh_check_launch("experts_tiles");
}
