// Linear recurrences with a matrix state per head, gfx950: one [D, Dv] fp32
// matrix S per (sequence, head), scanned token by token in fp32.
//
//   bonus form (u, per-token per-channel decay):
//       o_t = (S + diag(u) k_t v_t^T)^T q_t
//       S  <- diag(w_t) S + k_t v_t^T,   w_t = exp(-exp(decay_pre_t))
//   constant-decay form (one d per head):
//       S  <- d S + k_t v_t^T
//       o_t = S^T q_t
//   gated form (one log input gate i and log forget gate f per head and
//   token, both squashed by cap * tanh(. / cap), f through log-sigmoid):
//       m_t = max(f + m_{t-1}, i)            (m starts at 0)
//       S_t = exp(f + m_{t-1} - m_t) S_{t-1} + exp(i - m_t) k_t v_t^T
//       n_t likewise with k_t alone
//       o_t = S_t^T q_t / (max(|n_t . q_t|, exp(-m_t)) + 1e-6)
//   delta form (a decay g and a write strength b per head and token; k and q
//   are unit vectors, several value heads may share a q/k head):
//       S  <- g S;  u = b (v - S^T k);  S <- S + k u^T
//       o_t = S^T q_t
//       g = exp(-exp(rate) softplus(z + bias)),  b = sigmoid(z_b)
//   optional on q and k as they are read: silu (also on v), a rotate-half
//   rotation by tabulated cosines and sines, a constant factor each.
//
// One workgroup per (segment, head, block of up to 64 value columns).  A
// thread owns value column j of the block and one SPLIT-th of the key
// channels (lane = SPLIT j + s, keys s*KPT .. s*KPT + KPT-1, KPT one of a few
// size classes; SPLIT is 8 for heads of 32 or more key channels, else 4),
// keeps its KPT state entries in registers for the whole segment, and the
// partial outputs of a column are summed with lane permutes.  In the gated
// form the vector n is one more column of every block whose value is 1, so
// n . q falls out of the same walk; outputs wait in LDS until the tile ends
// and are divided on their way out.  The segment is walked serially, TT (8
// to 32) tokens staged into LDS at a time (q, k, decays and gates already
// exponentiated, v), so a prompt portion and a single decoded token take the
// same arithmetic path in the same order: results do not depend on how a
// sequence is cut into steps.  (The running maximum inside a tile comes from
// a prefix sum and a prefix maximum over the lanes; it is only the scale S
// and n are kept at, and both decays are taken from the very values of m
// that are stored.)
//
// The state row of a sequence is stored in the order the threads hold it,
// [head][block][ii][thread] with D padded to SPLIT*KPT: loads and stores are
// coalesced; in the gated form the running maxima [head][block] follow
// (ops.matrix_state_width mirrors this).
// A segment that starts its sequence ignores what the slot held.
//
// The delta form's dot of k with the state is one more sum over the lanes of a
// column ahead of the update.  The unit norms stay outside the vectors: with
// k = kr / |kr| and raw kr in LDS, S^T k and k u^T take the factor as a scalar.
//
// Long bf16 portions of the constant-decay, gated and delta forms are handed
// to the chunked MFMA kernels, which read and write the same state rows.

#include "matrix_state.h"

#include <climits>


// Sum over the 4 or 8 neighbouring lanes that share a value column, through
// the data-parallel lane permutes of the vector ALU (no trip through LDS):
// swaps inside pairs, then pairs inside quads, then the two quads of a group
// of 8 mirrored onto each other.
template <int CTRL>
LIG_DEVICE float lane_permute(float v) {
  return __builtin_bit_cast(
      float, __builtin_amdgcn_mov_dpp(__builtin_bit_cast(int, v), CTRL, 0xF, 0xF, true));
}
template <int SPLIT>
LIG_DEVICE float split_sum(float o) {
  o += lane_permute<0xB1>(o);   // quad_perm [1, 0, 3, 2]
  o += lane_permute<0x4E>(o);   // quad_perm [2, 3, 0, 1]
  if (SPLIT == 8) o += lane_permute<0x141>(o);  // row_half_mirror: lane i <-> 7 - i
  return o;
}

// Entry i of a query or key head as the recurrence sees it: silu, rotation
// (entry i paired with i +- nf), constant factor; fp32 throughout.
template <typename T>
LIG_DEVICE float ms_prep(const T* __restrict__ x, int i, const float* __restrict__ cs, int nf,
                         float scale, int act_silu) {
  float a = ld(x + i);
  if (act_silu) a = a * sigmoid_f32(a);
  if (i < 2 * nf) {
    const bool lower = i < nf;
    const int p = lower ? i : i - nf;
    float b = ld(x + (lower ? i + nf : i - nf));
    if (act_silu) b = b * sigmoid_f32(b);
    const float c = cs[p], s = cs[nf + p];
    a = lower ? a * c - b * s : a * c + b * s;
  }
  return a * scale;
}

// KPT: key channels per thread (D is padded to SPLIT * KPT; padded channels carry
// q = k = w = 0 and stay zero).  MAXT bounds the workgroup size (SPLIT times
// the block's columns rounded up to whole waves) so the compiler may use the
// register file a small workgroup leaves it.
template <typename T, int MS_SPLIT, int KPT, int FORM, int MAXT>
__global__ __launch_bounds__(MAXT) void matrix_state_scan_kernel(const MsArgs A) {
  extern __shared__ __align__(16) float sm[];
  constexpr bool BONUS = FORM == MS_BONUS, GATED = FORM == MS_GATED, DELTA = FORM == MS_DELTA;
  constexpr int Dp = MS_SPLIT * KPT;
  const int H = A.H, D = A.D, Dv = A.Dv, TT = A.TT;
  const int CBw = GATED ? A.CB + 1 : A.CB;  // columns that own state
  float* q_s = sm;                 // [TT][Dp]
  float* k_s = q_s + TT * Dp;      // [TT][Dp]
  float* w_s = k_s + TT * Dp;      // [TT][Dp] (BONUS only)
  float* v_s = BONUS ? w_s + TT * Dp : w_s;  // [TT][CBw]
  float* o_s = v_s + TT * CBw;     // [TT][CBw] (GATED), then
  float* a_s = GATED ? o_s + TT * CBw : o_s;  // [TT] kept share of the state,
  float* b_s = a_s + TT;           // [TT] weight of the new key (DELTA: write strength),
  float* e_s = b_s + TT;           // [TT] exp(-m); DELTA: 1 / |k|,
  float* f_s = e_s + TT;           // [TT] DELTA: q_scale / |q|

  const int seg = blockIdx.x, h = blockIdx.y, blk = blockIdx.z;
  const int n = A.seg_len[seg];
  if (n <= 0 || n < A.len_min || n > A.len_max) return;
  const int r0 = A.seg_start[seg];
  const int tid = threadIdx.x, nt = blockDim.x;
  const int j = tid / MS_SPLIT, s = tid % MS_SPLIT;
  const bool owner = j < CBw;
  const int nthr = CBw * MS_SPLIT;  // threads that own state
  const int c0 = blk * A.CB, ncol = min(A.CB, Dv - c0);
  const int hk = DELTA ? h / A.rep : h;
  const T* q = (const T*)A.q + hk * D;
  const T* k = (const T*)A.k + hk * D;
  const T* v = (const T*)A.v + h * Dv + c0;

  float S[KPT], U[KPT];
  float* slot = A.state + (long)A.seg_slot[seg] * A.state_stride;
  float* srow = slot + (long)(h * A.NB + blk) * KPT * nthr;
  float* mrow = slot + (long)H * A.NB * KPT * nthr + h * A.NB + blk;  // (GATED)
  const bool resume = A.seg_fresh[seg] == 0;
#pragma unroll
  for (int ii = 0; ii < KPT; ++ii) {
    S[ii] = (owner && resume) ? srow[(long)ii * nthr + tid] : 0.f;
    const int i = s * KPT + ii;
    U[ii] = (BONUS && i < D) ? A.bonus[h * D + i] : 0.f;
  }
  const float dconst = FORM == MS_CONST ? A.head_decay[h] : 0.f;
  float m_run = (GATED && resume) ? *mrow : 0.f;  // wave 0 carries it along

#pragma nounroll
  for (int t0 = 0; t0 < n; t0 += TT) {
    const int nt_tok = min(TT, n - t0);
    __syncthreads();  // the previous tile's readers are done
#pragma nounroll
    for (int e = tid; e < nt_tok * Dp; e += nt) {
      const int t = e / Dp, i = e - t * Dp;
      const long r = r0 + t0 + t;
      float qv = 0.f, kv = 0.f, wv = 0.f;
      if (i < D) {
        const float* cs = A.cs + r * 2 * A.nf;
        // (delta form: the scale joins the unit norm's factor)
        qv = ms_prep(q + r * A.q_stride, i, cs, A.nf, DELTA ? 1.0f : A.q_scale, A.act_silu);
        kv = ms_prep(k + r * A.k_stride, i, cs, A.nf, A.k_scale, A.act_silu);
        if (BONUS) wv = expf(-expf(A.decay_pre[r * (long)(H * D) + h * D + i]));
      }
      q_s[e] = qv;
      k_s[e] = kv;
      if (BONUS) w_s[e] = wv;
    }
#pragma nounroll
    for (int e = tid; e < nt_tok * CBw; e += nt) {
      const int t = e / CBw, c = e - t * CBw;
      float vv = (GATED && c == A.CB) ? 1.0f : 0.f;
      if (c < ncol) {
        vv = ld(v + (long)(r0 + t0 + t) * A.v_stride + c);
        if (A.act_silu) vv = vv * sigmoid_f32(vv);
      }
      v_s[e] = vv;
    }
    if (DELTA && tid < nt_tok) {
      const long r = (long)(r0 + t0 + tid) * A.gate_stride + h;
      a_s[tid] = expf(ms_log_decay(A.gate_f[r], A.bias_i[h], A.bias_f[h]));
      b_s[tid] = sigmoid_f32(A.gate_i[r]);
    }
    if (GATED && tid < WAVE_SIZE) {
      // lane t: gates of token t, prefix sum of the log forget gates, prefix
      // maximum of (i - that sum)
      float gi = -INFINITY, gf = 0.f;
      if (tid < nt_tok) {
        const long r = (long)(r0 + t0 + tid) * A.gate_stride + h;
        gi = A.gate_cap * tanhf((A.gate_i[r] + A.bias_i[h]) / A.gate_cap);
        gf = A.gate_cap * tanhf((A.gate_f[r] + A.bias_f[h]) / A.gate_cap);
        gf = fminf(gf, 0.f) - log1pf(expf(-fabsf(gf)));
      }
      float F = gf;
#pragma unroll
      for (int d = 1; d < 32; d <<= 1) {
        const float u = __shfl_up(F, d, WAVE_SIZE);
        if (tid >= d) F += u;
      }
      float G = gi - F;
#pragma unroll
      for (int d = 1; d < 32; d <<= 1) {
        const float u = __shfl_up(G, d, WAVE_SIZE);
        if (tid >= d) G = fmaxf(G, u);
      }
      const float m = F + fmaxf(m_run, G);
      float m_prev = __shfl_up(m, 1, WAVE_SIZE);
      if (tid == 0) m_prev = m_run;
      if (tid < nt_tok) {
        a_s[tid] = expf(gf + m_prev - m);
        b_s[tid] = expf(gi - m);
        e_s[tid] = expf(-m);
      }
      m_run = __shfl(m, nt_tok - 1, WAVE_SIZE);
    }
    __syncthreads();
    if (DELTA) {
      // lengths of the staged q and k, a wave per token
      for (int t = tid / WAVE_SIZE; t < nt_tok; t += nt / WAVE_SIZE) {
        float sq = 0.f, sk = 0.f;
        for (int i = tid % WAVE_SIZE; i < Dp; i += WAVE_SIZE) {
          sq += q_s[t * Dp + i] * q_s[t * Dp + i];
          sk += k_s[t * Dp + i] * k_s[t * Dp + i];
        }
        sq = wave_reduce_sum(sq);
        sk = wave_reduce_sum(sk);
        if (tid % WAVE_SIZE == 0) {
          e_s[t] = 1.0f / sqrtf(sk + A.unit_eps);
          f_s[t] = A.q_scale / sqrtf(sq + A.unit_eps);
        }
      }
      __syncthreads();
    }
    // every wave of the workgroup walks the tile (idle lanes of the last
    // wave take part in the lane permutes with zeros)
    // one token: read its q, k, decay and v from LDS, output, state update
    auto step = [&](int t) __attribute__((always_inline)) {
      float vj = owner ? v_s[t * CBw + j] : 0.f;
      const float keep = GATED ? a_s[t] : dconst;
      if (GATED) vj *= b_s[t];
      const float* qt = q_s + t * Dp + s * KPT;
      const float* kt = k_s + t * Dp + s * KPT;
      const float* wt = w_s + t * Dp + s * KPT;
      float o = 0.f;
      if (DELTA) {
        const float g = a_s[t], ik = e_s[t];
        float held = 0.f;
#pragma unroll
        for (int i4 = 0; i4 < KPT; i4 += 4) {
          const f32x4 k4 = *reinterpret_cast<const f32x4*>(kt + i4);
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            S[i4 + e] *= g;
            held += k4[e] * S[i4 + e];
          }
        }
        held = split_sum<MS_SPLIT>(held);
        const float u = b_s[t] * (vj - held * ik) * ik;
#pragma unroll
        for (int i4 = 0; i4 < KPT; i4 += 4) {
          const f32x4 k4 = *reinterpret_cast<const f32x4*>(kt + i4);
          const f32x4 q4 = *reinterpret_cast<const f32x4*>(qt + i4);
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            S[i4 + e] += k4[e] * u;
            o += q4[e] * S[i4 + e];
          }
        }
        o = split_sum<MS_SPLIT>(o) * f_s[t];
        if (owner && s == 0 && j < ncol)
          A.out[(long)(r0 + t0 + t) * (H * Dv) + h * Dv + c0 + j] = o;
        return;
      }
#pragma unroll
      for (int i4 = 0; i4 < KPT; i4 += 4) {
        const f32x4 k4 = *reinterpret_cast<const f32x4*>(kt + i4);
        const f32x4 q4 = *reinterpret_cast<const f32x4*>(qt + i4);
        f32x4 w4 = {0.f, 0.f, 0.f, 0.f};
        if (BONUS) w4 = *reinterpret_cast<const f32x4*>(wt + i4);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int ii = i4 + e;
          const float kv = k4[e] * vj;
          if (BONUS) {
            o += q4[e] * (S[ii] + U[ii] * kv);
            S[ii] = w4[e] * S[ii] + kv;
          } else {
            S[ii] = keep * S[ii] + kv;
            o += q4[e] * S[ii];
          }
        }
      }
      o = split_sum<MS_SPLIT>(o);
      if (owner && s == 0) {
        if (GATED) o_s[t * CBw + j] = o;
        else if (j < ncol) A.out[(long)(r0 + t0 + t) * (H * Dv) + h * Dv + c0 + j] = o;
      }
    };
    // two tokens per trip: the second token's LDS reads overlap the first
    // token's arithmetic (the state update itself stays in order)
    int t = 0;
#pragma nounroll
    for (; t + 1 < nt_tok; t += 2) {
      step(t);
      step(t + 1);
    }
    if (t < nt_tok) step(t);
    if (GATED) {
      __syncthreads();
#pragma nounroll
      for (int e = tid; e < nt_tok * ncol; e += nt) {
        const int tt = e / ncol, c = e - tt * ncol;
        const float den = fmaxf(fabsf(o_s[tt * CBw + A.CB]), e_s[tt]) + 1e-6f;
        A.out[(long)(r0 + t0 + tt) * (H * Dv) + h * Dv + c0 + c] = o_s[tt * CBw + c] / den;
      }
    }
  }
  if (owner) {
#pragma unroll
    for (int ii = 0; ii < KPT; ++ii) srow[(long)ii * nthr + tid] = S[ii];
  }
  if (GATED && tid == 0) *mrow = m_run;
}

template <typename T, int SPLIT, int KPT, int FORM>
static void ms_launch(const MsArgs& a, dim3 grid, int threads, size_t smem, hipStream_t stream) {
  if (threads <= 256)
    hipLaunchKernelGGL((matrix_state_scan_kernel<T, SPLIT, KPT, FORM, 256>), grid,
                       dim3(threads), smem, stream, a);
  else
    hipLaunchKernelGGL((matrix_state_scan_kernel<T, SPLIT, KPT, FORM, 576>), grid,
                       dim3(threads), smem, stream, a);
}

template <typename T, int FORM>
static void ms_dispatch(const MsArgs& a, int split, int kpt, dim3 grid, int threads,
                        size_t smem, hipStream_t st) {
  if (split == 4) {
    if (kpt == 4) ms_launch<T, 4, 4, FORM>(a, grid, threads, smem, st);
    else ms_launch<T, 4, 8, FORM>(a, grid, threads, smem, st);
    return;
  }
  switch (kpt) {
    case 4: ms_launch<T, 8, 4, FORM>(a, grid, threads, smem, st); break;
    case 8: ms_launch<T, 8, 8, FORM>(a, grid, threads, smem, st); break;
    case 12: ms_launch<T, 8, 12, FORM>(a, grid, threads, smem, st); break;
    case 16: ms_launch<T, 8, 16, FORM>(a, grid, threads, smem, st); break;
    case 24: ms_launch<T, 8, 24, FORM>(a, grid, threads, smem, st); break;
    case 32: ms_launch<T, 8, 32, FORM>(a, grid, threads, smem, st); break;
    case 48: ms_launch<T, 8, 48, FORM>(a, grid, threads, smem, st); break;
    default: ms_launch<T, 8, 64, FORM>(a, grid, threads, smem, st); break;
  }
}

// Portions of at least this many tokens go through the chunked kernel where
// it serves the shape (bf16, constant-decay or gated form).
#define MS_CHUNK_MIN 16

// max_seg_len: the longest segment of the step (0: walk every segment).
// The form follows from the pointers: bonus -> bonus form, gate_i -> gated
// form, else the constant-decay form.  Returns 0 when launched, 1 when a head
// is wider than the kernel holds.
extern "C" int lig_matrix_state_scan(
    float* out, const void* q, long q_stride, const void* k, long k_stride,
    const void* v, long v_stride, const float* decay_pre, const float* head_decay,
    const float* bonus, const float* gate_i, const float* gate_f, long gate_stride,
    const float* bias_i, const float* bias_f, float gate_cap, const float* cs, int nf,
    float q_scale, float k_scale, float* state, long state_stride, const int* seg_start,
    const int* seg_len, const int* seg_slot, const int* seg_fresh, int S, int H,
    int D, int Dv, int act_silu, int max_seg_len, int is_f32, hipStream_t stream) {
  int split = 4, kpt = 0;
  if (D > 0) ms_shape(D, &split, &kpt);
  if (kpt == 0 || Dv <= 0 || 2 * nf > D) return 1;
  const int CB = Dv < MS_COLS ? Dv : MS_COLS;
  const int NB = (Dv + CB - 1) / CB;
  if (H > 65535 || NB > 65535) return 1;
  if (S <= 0) return 0;
  const int form = bonus != nullptr ? MS_BONUS : (gate_i != nullptr ? MS_GATED : MS_CONST);
  const int CBw = form == MS_GATED ? CB + 1 : CB;
  const int Dp = kpt * split;
  const int per_tok = (form == MS_BONUS ? 3 : 2) * Dp + (form == MS_GATED ? 2 * CBw + 3 : CBw);
  // tokens staged per tile: as many as 40 KB of LDS hold, 8 to 32
  const int TT = per_tok * 32 * 4 <= 40 * 1024 ? 32 : (per_tok * 16 * 4 <= 48 * 1024 ? 16 : 8);
  const size_t smem = (size_t)per_tok * TT * sizeof(float);
  const int threads = ((CBw * split + WAVE_SIZE - 1) / WAVE_SIZE) * WAVE_SIZE;
  MsArgs a{out, q, k, v, q_stride, k_stride, v_stride, decay_pre, head_decay, bonus,
                 gate_i, gate_f, gate_stride, bias_i, bias_f, gate_cap, cs, nf, q_scale,
                 k_scale, state, state_stride, seg_start, seg_len, seg_slot, seg_fresh,
                 H, D, Dv, CB, NB, TT, act_silu, split, kpt, 1, INT_MAX, 1, 0.f};
  const dim3 grid(S, H, NB);
  if (max_seg_len >= MS_CHUNK_MIN && !is_f32 && !act_silu && form != MS_BONUS &&
      ms_chunks_served(a, form)) {
    // long portions in chunks, the step's short ones by the walk
    a.len_min = MS_CHUNK_MIN;
    ms_chunks_launch(a, form, S, stream);
    if (S == 1) return 0;
    a.len_min = 1;
    a.len_max = MS_CHUNK_MIN - 1;
  }
#define LIG_MS_FORM(T)                                                                        \
  if (form == MS_BONUS) ms_dispatch<T, MS_BONUS>(a, split, kpt, grid, threads, smem, stream); \
  else if (form == MS_GATED)                                                                  \
    ms_dispatch<T, MS_GATED>(a, split, kpt, grid, threads, smem, stream);                     \
  else ms_dispatch<T, MS_CONST>(a, split, kpt, grid, threads, smem, stream)
  if (is_f32) {
    LIG_MS_FORM(float);
  } else {
    LIG_MS_FORM(bf16s);
  }
#undef LIG_MS_FORM
  return 0;
}

// The delta form.  gate_b: write-strength logits, gate_a: decay logits (fp32
// [R, H] views with one row stride); log_rate, bias: fp32 [H].  q and k hold
// KH heads, value head h reads head h / (H / KH).  scratch (chunked portions,
// may be null: everything is walked) holds lig_gated_delta_scratch bytes.
// Segments lie in row order.  Returns 0 when launched, 1 when a head is wider
// than the kernel holds or the heads do not divide.
extern "C" int lig_gated_delta_scan(
    float* out, const void* q, long q_stride, const void* k, long k_stride, const void* v,
    long v_stride, const float* gate_b, const float* gate_a, long gate_stride,
    const float* log_rate, const float* bias, float q_scale, float unit_eps, float* state,
    long state_stride, const int* seg_start, const int* seg_len, const int* seg_slot,
    const int* seg_fresh, int S, int H, int KH, int D, int Dv, int max_seg_len, void* scratch,
    int is_f32, hipStream_t stream) {
  int split = 4, kpt = 0;
  if (D > 0) ms_shape(D, &split, &kpt);
  if (kpt == 0 || Dv <= 0 || KH <= 0 || H % KH != 0) return 1;
  const int CB = Dv < MS_COLS ? Dv : MS_COLS;
  const int NB = (Dv + CB - 1) / CB;
  if (H > 65535 || NB > 65535) return 1;
  if (S <= 0) return 0;
  const int Dp = kpt * split;
  const int per_tok = 2 * Dp + CB + 4;
  const int TT = per_tok * 32 * 4 <= 40 * 1024 ? 32 : (per_tok * 16 * 4 <= 48 * 1024 ? 16 : 8);
  const size_t smem = (size_t)per_tok * TT * sizeof(float);
  const int threads = ((CB * split + WAVE_SIZE - 1) / WAVE_SIZE) * WAVE_SIZE;
  MsArgs a{out, q, k, v, q_stride, k_stride, v_stride, nullptr, nullptr, nullptr,
           gate_b, gate_a, gate_stride, log_rate, bias, 1.0f, nullptr, 0, q_scale,
           1.0f, state, state_stride, seg_start, seg_len, seg_slot, seg_fresh,
           H, D, Dv, CB, NB, TT, 0, split, kpt, 1, INT_MAX, H / KH, unit_eps};
  const dim3 grid(S, H, NB);
  if (max_seg_len >= MS_CHUNK_MIN && !is_f32 && scratch != nullptr && ms_delta_chunks_served(a)) {
    a.len_min = MS_CHUNK_MIN;
    ms_delta_chunks_launch(a, S, max_seg_len, scratch, stream);
    if (S == 1) return 0;
    a.len_min = 1;
    a.len_max = MS_CHUNK_MIN - 1;
  }
  if (is_f32) ms_dispatch<float, MS_DELTA>(a, split, kpt, grid, threads, smem, stream);
  else ms_dispatch<bf16s, MS_DELTA>(a, split, kpt, grid, threads, smem, stream);
  return 0;
}
