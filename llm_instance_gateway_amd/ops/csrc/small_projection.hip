// A few output columns per row, kept in fp32, gfx950:
//   out[r, n] = sum_c h[r, c] * w[n, c]      h [R, C] bf16, w [N, C] bf16
// for router logits and recurrence gates, which are computed in fp32 from the
// bf16 rows the big GEMMs read (the products of two bf16 numbers are exact in
// fp32, the sums are fp32).
//
// A workgroup owns 16 rows and up to 64 columns; its 8 waves split the inner
// dimension (32 entries a step, wave after wave) on mfma_f32_16x16x32_bf16
// and meet in LDS once at the end.  Memory-bound: every row is read once, the
// weights stay in L2.

#include "elem_types.h"

typedef __bf16 sp_bf16x8 __attribute__((ext_vector_type(8)));

#define SP_WAVES 8

LIG_DEVICE sp_bf16x8 sp_load(const uint16_t* __restrict__ p, bool ok) {
  u16x8 raw = {0, 0, 0, 0, 0, 0, 0, 0};
  if (ok) raw = *reinterpret_cast<const u16x8*>(p);
  return __builtin_bit_cast(sp_bf16x8, raw);
}

template <int NT>  // 16-column tiles
__global__ __launch_bounds__(SP_WAVES * WAVE_SIZE) void small_projection_kernel(
    float* __restrict__ out, const uint16_t* __restrict__ h, const uint16_t* __restrict__ w,
    int R, int N, int C) {
  __shared__ float part[SP_WAVES][NT][16][17];
  const int wave = threadIdx.x / WAVE_SIZE, lane = threadIdx.x % WAVE_SIZE;
  const int li = lane & 15, lg = lane >> 4;
  const long r0 = (long)blockIdx.x * 16;
  const int n0 = blockIdx.y * NT * 16;
  const bool row_ok = r0 + li < R;
  const uint16_t* hp = h + (row_ok ? r0 + li : r0) * (long)C;
  f32x4 acc[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) acc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int k0 = wave * 32; k0 < C; k0 += SP_WAVES * 32) {
    const int c = k0 + lg * 8;
    const sp_bf16x8 a = sp_load(hp + c, row_ok && c < C);
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const int n = n0 + t * 16 + li;
      const sp_bf16x8 b = sp_load(w + (long)n * C + c, n < N && c < C);
      acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, acc[t], 0, 0, 0);
    }
  }
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int e = 0; e < 4; ++e) part[wave][t][lg * 4 + e][li] = acc[t][e];
  __syncthreads();
  for (int e = threadIdx.x; e < 16 * NT * 16; e += SP_WAVES * WAVE_SIZE) {
    const int row = e / (NT * 16), col = e - row * (NT * 16);
    float s = 0.f;
#pragma unroll
    for (int v = 0; v < SP_WAVES; ++v) s += part[v][col / 16][row][col % 16];
    if (r0 + row < R && n0 + col < N) out[(r0 + row) * N + n0 + col] = s;
  }
}

// Returns 0 when launched, 1 when the shape or alignment is not served.
extern "C" int lig_small_projection(float* out, const void* h, const void* w, int R, int N,
                                    int C, hipStream_t s) {
  if (C <= 0 || C % 8 != 0 || N <= 0 || !aligned16(h) || !aligned16(w)) return 1;
  if (R <= 0) return 0;
  const int rows = (R + 15) / 16;
#define LIG_SP(NT)                                                                             \
  hipLaunchKernelGGL(small_projection_kernel<NT>, dim3(rows, (N + NT * 16 - 1) / (NT * 16)),   \
                     dim3(SP_WAVES * WAVE_SIZE), 0, s, out, (const uint16_t*)h,                \
                     (const uint16_t*)w, R, N, C)
  // few rows (decode steps): narrower column tiles, so that a wave has fewer
  // loads in its chain and more workgroups share the columns
  if (N <= 16 || (long)rows * ((N + 31) / 32) < 256) LIG_SP(1);
  else if (N <= 32 || (long)rows * ((N + 63) / 64) < 256) LIG_SP(2);
  else LIG_SP(4);
#undef LIG_SP
  return 0;
}
