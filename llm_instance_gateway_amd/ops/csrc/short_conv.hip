// Short causal convolution over time, one filter per channel, then silu,
// gfx950:
//     y[t, c] = silu(sum_j w[j, c] x[t - (taps - 1) + j, c])
// over the segments of a flat batch; ahead of a segment's first row stand the
// sequence's last taps - 1 inputs, kept fp32 in a state row [taps - 1, C] per
// slot (zeros when the sequence starts here), which then takes the segment's
// last inputs.  bf16 or fp32 storage, fp32 arithmetic.
//
// A thread owns N neighbouring channels of one block of TB tokens of a
// segment and walks the block with the last taps - 1 inputs in registers, so
// an input row is read once (plus taps - 1 rows ahead of a block); the walk is
// cut into groups of four tokens whose loads are in flight together.  Only a
// segment's first block reads the state, and the same threads write it after
// their walk, so no other workgroup can see a half-updated row.  TAPS 0 takes
// the filter length at run time and re-reads the inputs per tap.

#include "elem_types.h"

#define SC_THREADS 256

template <int N, typename T>
LIG_DEVICE void sc_load(const T* p, float* v) {
  if (N == 8) ld8(p, v);
  else v[0] = ld(p);
}
template <int N, typename T>
LIG_DEVICE void sc_store(T* p, const float* v) {
  if (N == 8) st8(p, v);
  else st(p, v[0]);
}

template <typename T, int N, int TAPS>
__global__ __launch_bounds__(SC_THREADS) void short_conv_silu_kernel(
    T* __restrict__ out,                      // [R, C]
    const T* __restrict__ x, long x_stride,   // [R, C] column block
    const T* __restrict__ w,                  // [taps, C]
    float* __restrict__ state, long state_stride, const int* __restrict__ seg_start,
    const int* __restrict__ seg_len, const int* __restrict__ seg_slot,
    const int* __restrict__ seg_fresh, int C, int taps_rt, int TB) {
  const int taps = TAPS > 0 ? TAPS : taps_rt;
  const int seg = blockIdx.y;
  const int n = seg_len[seg];
  const int t0 = blockIdx.x * TB;
  const int c = (blockIdx.z * SC_THREADS + threadIdx.x) * N;
  if (t0 >= n || c >= C) return;  // no barrier below
  const int t1 = min(n, t0 + TB);
  const long r0 = seg_start[seg];
  const T* xs = x + r0 * x_stride + c;
  T* os = out + r0 * (long)C + c;
  float* srow = state + (long)seg_slot[seg] * state_stride + c;
  const bool resume = seg_fresh[seg] == 0;

  // input at segment offset t (negative: the state's rows)
  auto input = [&](int t, float* v) __attribute__((always_inline)) {
    if (t >= 0) {
      sc_load<N>(xs + t * x_stride, v);
    } else if (resume) {
      sc_load<N>(srow + (long)(t + taps - 1) * C, v);
    } else {
#pragma unroll
      for (int i = 0; i < N; ++i) v[i] = 0.f;
    }
  };

  if (TAPS > 0) {
    float wr[TAPS > 0 ? TAPS : 1][N], win[TAPS > 1 ? TAPS - 1 : 1][N];
#pragma unroll
    for (int j = 0; j < TAPS; ++j) sc_load<N>(w + (long)j * C + c, wr[j]);
#pragma unroll
    for (int j = 0; j < TAPS - 1; ++j) input(t0 - (TAPS - 1) + j, win[j]);
    for (int tg = t0; tg < t1; tg += 4) {
      float v[4][N];
#pragma unroll
      for (int u = 0; u < 4; ++u)
        if (tg + u < t1) sc_load<N>(xs + (tg + u) * x_stride, v[u]);
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        if (tg + u >= t1) break;
        float y[N];
#pragma unroll
        for (int i = 0; i < N; ++i) {
          float a = wr[TAPS - 1][i] * v[u][i];
#pragma unroll
          for (int j = 0; j < TAPS - 1; ++j) a += wr[j][i] * win[j][i];
          y[i] = a * sigmoid_for<T>(a);
#pragma unroll
          for (int j = 0; j + 1 < TAPS - 1; ++j) win[j][i] = win[j + 1][i];
          if (TAPS > 1) win[TAPS > 1 ? TAPS - 2 : 0][i] = v[u][i];
        }
        sc_store<N>(os + (long)(tg + u) * C, y);
      }
    }
  } else {
    for (int t = t0; t < t1; ++t) {
      float y[N];
#pragma unroll
      for (int i = 0; i < N; ++i) y[i] = 0.f;
      for (int j = 0; j < taps; ++j) {
        float v[N], wj[N];
        input(t - (taps - 1) + j, v);
        sc_load<N>(w + (long)j * C + c, wj);
#pragma unroll
        for (int i = 0; i < N; ++i) y[i] += wj[i] * v[i];
      }
#pragma unroll
      for (int i = 0; i < N; ++i) y[i] = y[i] * sigmoid_for<T>(y[i]);
      sc_store<N>(os + (long)t * C, y);
    }
  }
  if (t0 == 0) {
    // the segment's last taps - 1 inputs; a segment shorter than that keeps
    // the youngest old ones (row j takes old row n + j: ascending order never
    // overwrites a row that is still to be read)
    for (int j = 0; j < taps - 1; ++j) {
      float v[N];
      input(n - (taps - 1) + j, v);
      sc_store<N>(srow + (long)j * C, v);
    }
  }
}

// Returns 0 when launched, 1 when the launch is not possible.
extern "C" int lig_short_conv_silu(void* out, const void* x, long x_stride, const void* w,
                                   float* state, long state_stride, const int* seg_start,
                                   const int* seg_len, const int* seg_slot,
                                   const int* seg_fresh, int S, int max_len, int C, int taps,
                                   int is_f32, hipStream_t s) {
  if (C <= 0 || taps < 1 || S > 65535) return 1;
  if (S <= 0 || max_len <= 0) return 0;
  const bool v8 = C % 8 == 0 && x_stride % 8 == 0 && state_stride % 4 == 0 && aligned16(out) &&
                  aligned16(x) && aligned16(w) && aligned16(state);
  // every token whose window reaches ahead of the segment lies in block 0
  const int TB = taps - 1 > 16 ? taps - 1 : 16;
  const int threads_c = v8 ? C / 8 : C;
  const dim3 grid((max_len + TB - 1) / TB, S, (threads_c + SC_THREADS - 1) / SC_THREADS);
#define LIG_SC(T, N, TAPS)                                                                     \
  hipLaunchKernelGGL((short_conv_silu_kernel<T, N, TAPS>), grid, dim3(SC_THREADS), 0, s,       \
                     (T*)out, (const T*)x, x_stride, (const T*)w, state, state_stride,         \
                     seg_start, seg_len, seg_slot, seg_fresh, C, taps, TB)
#define LIG_SC_K(T, N)                     \
  if (taps == 2) LIG_SC(T, N, 2);          \
  else if (taps == 3) LIG_SC(T, N, 3);     \
  else if (taps == 4) LIG_SC(T, N, 4);     \
  else LIG_SC(T, N, 0)
  if (is_f32) {
    if (v8) { LIG_SC_K(float, 8); } else { LIG_SC_K(float, 1); }
  } else {
    if (v8) { LIG_SC_K(bf16s, 8); } else { LIG_SC_K(bf16s, 1); }
  }
#undef LIG_SC_K
#undef LIG_SC
  return 0;
}
