// Layer norms (centred, weight, no bias) over an fp32 residual, gfx950, fused
// with what enters the residual ahead of them.  One workgroup per row, fp32
// arithmetic, bf16 or fp32 storage (T) for tables, weights and outputs.
//
//   embed_layer_norm : x = scale * table[token];              h = LN(x) * w
//   add_layer_norm   : x += y / sqrt(mean(y^2) + eps) * w_y;  h = LN(x) * w
//
// LN(x) = (x - mean) / sqrt(mean((x - mean)^2) + eps); the deviations are
// squared after the mean is known (two reductions, no cancellation).  Without
// y the second form is the norm alone.  The row waits in LDS between the
// passes, every thread re-reading only what it wrote itself, so each operand
// crosses HBM once; h may be absent (only the residual is updated).

#include "elem_types.h"

#define LN_THREADS 256

template <typename T, int N, bool EMBED>
__global__ __launch_bounds__(LN_THREADS) void layer_norm_kernel(
    float* __restrict__ x, T* __restrict__ h, const T* __restrict__ table,
    const int64_t* __restrict__ tokens, float scale, const T* __restrict__ y,
    const T* __restrict__ w_y, const T* __restrict__ w, float eps, int H) {
  extern __shared__ __align__(16) float row_s[];  // [H]
  __shared__ float red[3][17];
  const long r = blockIdx.x;
  float* xr = x + r * H;
  const float inv_n = 1.0f / (float)H;
  float sum = 0.f;
  if (EMBED) {
    const T* src = table + tokens[r] * (long)H;
    for (int c = threadIdx.x * N; c < H; c += LN_THREADS * N) {
      float t[N];
      ldn<N>(src + c, t);
#pragma unroll
      for (int i = 0; i < N; ++i) {
        t[i] *= scale;
        sum += t[i];
      }
      stn<N>(xr + c, t);
      stn<N>(row_s + c, t);
    }
  } else {
    float inv_y = 0.f;
    if (y != nullptr) {
      float ss = 0.f;
      for (int c = threadIdx.x * N; c < H; c += LN_THREADS * N) {
        float t[N];
        ldn<N>(y + r * H + c, t);
#pragma unroll
        for (int i = 0; i < N; ++i) ss += t[i] * t[i];
        stn<N>(row_s + c, t);
      }
      ss = block_reduce_sum(ss, red[0]);
      inv_y = 1.0f / sqrtf(ss * inv_n + eps);
    }
    for (int c = threadIdx.x * N; c < H; c += LN_THREADS * N) {
      float t[N];
      ldn<N>(xr + c, t);
      if (y != nullptr) {
        float u[N], g[N];
        ldn<N>(row_s + c, u);
        ldn<N>(w_y + c, g);
#pragma unroll
        for (int i = 0; i < N; ++i) t[i] += u[i] * inv_y * g[i];
        stn<N>(xr + c, t);
      }
#pragma unroll
      for (int i = 0; i < N; ++i) sum += t[i];
      stn<N>(row_s + c, t);
    }
  }
  if (h == nullptr) return;  // uniform across the workgroup
  const float mean = block_reduce_sum(sum, red[1]) * inv_n;
  float var = 0.f;
  for (int c = threadIdx.x * N; c < H; c += LN_THREADS * N) {
    float t[N];
    ldn<N>(row_s + c, t);
#pragma unroll
    for (int i = 0; i < N; ++i) var += (t[i] - mean) * (t[i] - mean);
  }
  var = block_reduce_sum(var, red[2]) * inv_n;
  const float inv = 1.0f / sqrtf(var + eps);
  for (int c = threadIdx.x * N; c < H; c += LN_THREADS * N) {
    float t[N], g[N];
    ldn<N>(row_s + c, t);
    ldn<N>(w + c, g);
#pragma unroll
    for (int i = 0; i < N; ++i) t[i] = (t[i] - mean) * inv * g[i];
    stn<N>(h + r * H + c, t);
  }
}

extern "C" {

// tokens != null: the embedding form.  Returns 0 when launched, 1 when a row
// is wider than the workgroup's LDS.
int lig_layer_norm(float* x, void* h, const void* table, const int64_t* tokens, float scale,
                   const void* y, const void* w_y, const void* w, float eps, int R, int H,
                   int is_f32, hipStream_t s) {
  if (H <= 0 || H > 15 * 1024) return 1;
  if (R <= 0) return 0;
  const size_t smem = (size_t)H * sizeof(float);
  const bool v4 = H % 4 == 0 && aligned16(x) && aligned16(h) && aligned16(table) &&
                  aligned16(y) && aligned16(w_y) && aligned16(w);
#define LIG_LN(T, N, E)                                                             \
  hipLaunchKernelGGL((layer_norm_kernel<T, N, E>), dim3(R), dim3(LN_THREADS), smem, s, x, \
                     (T*)h, (const T*)table, tokens, scale, (const T*)y, (const T*)w_y,   \
                     (const T*)w, eps, H)
#define LIG_LN_T(T)                                            \
  if (tokens != nullptr) {                                     \
    if (v4) LIG_LN(T, 4, true); else LIG_LN(T, 1, true);       \
  } else {                                                     \
    if (v4) LIG_LN(T, 4, false); else LIG_LN(T, 1, false);     \
  }
  if (is_f32) {
    LIG_LN_T(float)
  } else {
    LIG_LN_T(bf16s)
  }
#undef LIG_LN_T
#undef LIG_LN
  return 0;
}

}  // extern "C"
