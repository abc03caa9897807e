// Matrix-state recurrences with one decay per head and token, in chunks of 64
// tokens on MFMA tiles, gfx950 (bf16 q, k, v; fp32 state).  The same
// recurrences, arguments and state rows as matrix_state_scan.hip; this kernel
// takes the long portions.
//
// With w_ts the factor that token s's key/value product has decayed by at
// token t, and c_t the factor of the state S the chunk starts from:
//     o_t = c_t (q_t . S) + sum_{s <= t} w_ts (q_t . k_s) v_s
//     S  <- c_end S + sum_s w_end,s k_s v_s^T
//   constant decay d:  w_ts = d^(t-s),  c_t = d^(t+1)
//   gated: F = prefix sum of the log forget gates, g_s = i_s - F_s,
//          M_t = max(m, max_{s <= t} g_s):  w_ts = exp(g_s - M_t),
//          c_t = exp(m - M_t),  m_t = F_t + M_t;  every exponent is <= 0.
//          The normaliser n follows the same sums with v = 1.
//
// One workgroup (4 waves) per (segment, head, block of up to 64 value
// columns); wave w owns 16 columns of the state, [Dp, 16] fp32 in MFMA
// accumulators for the whole segment.  Per chunk: q, k and v go to LDS (k and
// v also transposed), wave w scores token rows 16 w .. 16 w + 15 against the
// chunk's keys and leaves the weighted scores in LDS, every wave multiplies
// its state with all 64 queries, then the weighted scores with its values,
// writes the outputs, and adds the keys' products to its state.  The state
// enters the product with q straight from the accumulators: an MFMA
// contraction may visit its inner index in any order as long as both
// operands agree, so the queries are read from LDS in the order the
// accumulators hold the key channels.
//
// Precision: products of bf16 numbers are exact in fp32 and sums are fp32.
// fp32 operands (state, weighted scores, weighted values; q and k after a
// rotation) are split into two bf16 halves, x = hi + lo, and multiplied half
// by half (the lo * lo product is left out): about 16 mantissa bits.  Gates,
// weights, normaliser and running maximum are fp32 throughout.
//
// The chunk after the current one is fetched into registers during the
// arithmetic (unrotated form).

#include "matrix_state.h"
#include "matrix_state_mfma.h"

#define MC_THREADS 256

// DP: key channels padded to a multiple of 32.  ROT: q and k are rotated (and
// kept as two halves).
template <int DP, bool GATED, bool ROT>
__global__ __launch_bounds__(MC_THREADS) void matrix_state_chunk_kernel(const MsArgs A) {
  constexpr int KB = DP / 32, DT = DP / 16, NS = ROT ? 2 : 1, DROW = DP + 8;
  constexpr int NCH = DP / 32;  // 16-byte chunks of a q or k row per thread
  struct Shared {
    uint16_t q[NS][MC_T][DROW];
    uint16_t k[NS][MC_T][DROW];
    uint16_t kt[NS][DP][MC_TP];
    uint16_t vt[64][MC_TP];
    uint16_t p[2][MC_T][MC_TP];
    float n[DP];       // normaliser
    float qn[MC_T];    // q_t . n
    float rs[MC_T];    // row sums of the weighted scores
    float c[MC_T];     // c_t, times q_scale
    float w[MC_T];     // w_end,s, times k_scale
    float g[MC_T];     // gated: g_s
    float M[MC_T];     // gated: M_t
    float em[MC_T];    // gated: exp(-m_t)
    float pw[MC_T + 1];  // constant decay: d^i
    float c_end;
  };
  __shared__ Shared sm;

  const int seg = blockIdx.x, h = blockIdx.y, blk = blockIdx.z;
  const int n = A.seg_len[seg];
  if (n <= 0 || n < A.len_min || n > A.len_max) return;
  const int H = A.H, D = A.D, Dv = A.Dv, CB = A.CB;
  const long r0 = A.seg_start[seg];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int li = lane & 15, lg = lane >> 4;
  const int c0 = blk * CB, ncol = min(CB, Dv - c0);
  const uint16_t* q = (const uint16_t*)A.q + h * D;
  const uint16_t* k = (const uint16_t*)A.k + h * D;
  const uint16_t* v = (const uint16_t*)A.v + h * Dv + c0;

  // ---- state row: [head][block][entry][column * split + key lane], maxima behind ----
  const int CBw = GATED ? CB + 1 : CB;
  const int nthr = CBw * A.split, Dst = A.split * A.kpt;
  float* slot = A.state + (long)A.seg_slot[seg] * A.state_stride;
  float* srow = slot + (long)(h * A.NB + blk) * A.kpt * nthr;
  float* mrow = slot + (long)H * A.NB * A.kpt * nthr + h * A.NB + blk;
  const bool resume = A.seg_fresh[seg] == 0;
  const int col = wave * 16 + li;  // the state column this lane holds
  auto at = [&](int i, int j) { return (long)(i % A.kpt) * nthr + j * A.split + i / A.kpt; };
  f32x4 S[DT];
#pragma unroll
  for (int dt = 0; dt < DT; ++dt) {
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = dt * 16 + lg * 4 + r;
      S[dt][r] = (resume && i < Dst && col < CB) ? srow[at(i, col)] : 0.f;
    }
  }
  float m_run = 0.f;  // wave 0 carries it along
  if (GATED) {
    if (resume) m_run = *mrow;
    for (int i = tid; i < DP; i += MC_THREADS)
      sm.n[i] = (resume && i < Dst) ? srow[at(i, CB)] : 0.f;
  } else if (tid <= MC_T) {
    sm.pw[tid] = powf(A.head_decay[h], (float)tid);
  }
  const float qk_scale = A.q_scale * A.k_scale;

  // a thread stages token `lane` of the chunk, 16-byte chunks wave, wave + 4, ...
  u16x8 qr[NCH], kr[NCH], vr[2];
  const u16x8 zero8 = {0, 0, 0, 0, 0, 0, 0, 0};
  auto fetch = [&](int t0) __attribute__((always_inline)) {
    const bool ok = t0 + lane < n;
    const long r = r0 + t0 + lane;
    if (!ROT) {
#pragma unroll
      for (int j = 0; j < NCH; ++j) {
        const int d = (wave + 4 * j) * 8;
        const bool in = ok && d < D;
        qr[j] = in ? mc_ld16(q + r * A.q_stride + d) : zero8;
        kr[j] = in ? mc_ld16(k + r * A.k_stride + d) : zero8;
      }
    }
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int d = (wave + 4 * j) * 8;
      vr[j] = (ok && d < ncol) ? mc_ld16(v + r * A.v_stride + d) : zero8;
    }
  };
  fetch(0);

#pragma nounroll
  for (int t0 = 0; t0 < n; t0 += MC_T) {
    const int cnt = min(MC_T, n - t0);
    __syncthreads();  // the previous chunk's readers are done
    // ---- staging -------------------------------------------------------------------
    if (!ROT) {
#pragma unroll
      for (int j = 0; j < NCH; ++j) {
        const int d = (wave + 4 * j) * 8;
        *reinterpret_cast<u16x8*>(&sm.q[0][lane][d]) = qr[j];
        *reinterpret_cast<u16x8*>(&sm.k[0][lane][d]) = kr[j];
#pragma unroll
        for (int e = 0; e < 8; ++e) sm.kt[0][d + e][lane] = kr[j][e];
      }
    } else {
      // pairs (i, i + nf) lie in chunks nf / 8 apart: both at once
      const bool ok = t0 + lane < n;
      const long r = ok ? r0 + t0 + lane : r0;
      const int nf = A.nf, nfc = nf / 8;
      const float* cs = A.cs + r * 2 * nf;
      auto put = [&](uint16_t (*dst)[DROW], uint16_t (*lo)[DROW], bool key, int d, const float* x)
                     __attribute__((always_inline)) {
        u16x8 a, b;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          uint16_t hi, l;
          mc_split(ok ? x[e] : 0.f, hi, l);
          a[e] = hi;
          b[e] = l;
        }
        *reinterpret_cast<u16x8*>(&dst[lane][d]) = a;
        *reinterpret_cast<u16x8*>(&lo[lane][d]) = b;
        if (key) {
#pragma unroll
          for (int e = 0; e < 8; ++e) {
            sm.kt[0][d + e][lane] = a[e];
            sm.kt[NS - 1][d + e][lane] = b[e];
          }
        }
      };
      const int tasks = DP / 8 - nfc;  // pairs first, then the chunks that pass through
      for (int c = wave; c < tasks; c += 4) {
        const bool pair = c < nfc;
        const int d = (pair ? c : c + nfc) * 8;
#pragma unroll
        for (int which = 0; which < 2; ++which) {
          const uint16_t* src = which ? k + r * A.k_stride : q + r * A.q_stride;
          float a[8] = {0, 0, 0, 0, 0, 0, 0, 0}, b[8];
          if (d < D) {
            const u16x8 raw = mc_ld16(src + d);
#pragma unroll
            for (int e = 0; e < 8; ++e) a[e] = bf16_to_f32(raw[e]);
          }
          if (pair) {
            const u16x8 raw = mc_ld16(src + d + nf);
            float co[8], si[8];
            ld8(cs + d, co);
            ld8(cs + nf + d, si);
#pragma unroll
            for (int e = 0; e < 8; ++e) {
              const float u = a[e], w = bf16_to_f32(raw[e]);
              a[e] = u * co[e] - w * si[e];
              b[e] = w * co[e] + u * si[e];
            }
          }
          auto hi = which ? sm.k[0] : sm.q[0];
          auto lo = which ? sm.k[NS - 1] : sm.q[NS - 1];
          put(hi, lo, which == 1, d, a);
          if (pair) put(hi, lo, which == 1, d + nf, b);
        }
      }
    }
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int d = (wave + 4 * j) * 8;
#pragma unroll
      for (int e = 0; e < 8; ++e) sm.vt[d + e][lane] = vr[j][e];
    }
    // ---- decay factors: lane t of wave 0 owns token t ----------------------------------
    if (wave == 0) {
      const int t = lane;
      if (GATED) {
        float gi = -INFINITY, gf = 0.f;
        if (t < cnt) {
          const long r = (r0 + t0 + t) * A.gate_stride + h;
          gi = A.gate_cap * tanhf((A.gate_i[r] + A.bias_i[h]) / A.gate_cap);
          gf = A.gate_cap * tanhf((A.gate_f[r] + A.bias_f[h]) / A.gate_cap);
          gf = fminf(gf, 0.f) - log1pf(expf(-fabsf(gf)));
        }
        float F = gf;
#pragma unroll
        for (int d = 1; d < MC_T; d <<= 1) {
          const float u = __shfl_up(F, d, WAVE_SIZE);
          if (t >= d) F += u;
        }
        const float g = gi - F;
        float G = g;
#pragma unroll
        for (int d = 1; d < MC_T; d <<= 1) {
          const float u = __shfl_up(G, d, WAVE_SIZE);
          if (t >= d) G = fmaxf(G, u);
        }
        const float M = fmaxf(m_run, G);
        const float M_end = __shfl(M, cnt - 1, WAVE_SIZE);
        sm.c[t] = expf(m_run - M) * A.q_scale;
        sm.w[t] = expf(g - M_end) * A.k_scale;  // 0 past the portion's end
        sm.g[t] = g;
        sm.M[t] = M;
        sm.em[t] = expf(-(F + M));
        if (t == 0) sm.c_end = expf(m_run - M_end);
        m_run = __shfl(F, cnt - 1, WAVE_SIZE) + M_end;
      } else {
        sm.c[t] = sm.pw[t + 1] * A.q_scale;
        sm.w[t] = t < cnt ? sm.pw[cnt - 1 - t] * A.k_scale : 0.f;
        if (t == 0) sm.c_end = sm.pw[cnt];
      }
    }
    __syncthreads();
    if (t0 + MC_T < n) fetch(t0 + MC_T);

    // ---- weighted scores: wave's 16 tokens against keys up to them ---------------------
    {
      const int t = wave * 16 + li;
      const float Mt = GATED ? sm.M[t] : 0.f;
      float rowsum = 0.f;
      for (int st = 0; st <= wave; ++st) {
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kb = 0; kb < KB; ++kb) {
          const int d = kb * 32 + lg * 8;
          const u16x8 a = mc_ld16(&sm.k[0][st * 16 + li][d]), b = mc_ld16(&sm.q[0][t][d]);
          acc = mc_mfma(a, b, acc);
          if (ROT) {
            acc = mc_mfma(a, mc_ld16(&sm.q[NS - 1][t][d]), acc);
            acc = mc_mfma(mc_ld16(&sm.k[NS - 1][st * 16 + li][d]), b, acc);
          }
        }
        u16x4 hi, lo;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int s = st * 16 + lg * 4 + r;
          float p = 0.f;
          if (s <= t) p = acc[r] * qk_scale * (GATED ? __expf(sm.g[s] - Mt) : sm.pw[t - s]);
          rowsum += p;
          uint16_t a, b;
          mc_split(p, a, b);
          hi[r] = a;
          lo[r] = b;
        }
        *reinterpret_cast<u16x4*>(&sm.p[0][t][st * 16 + lg * 4]) = hi;
        *reinterpret_cast<u16x4*>(&sm.p[1][t][st * 16 + lg * 4]) = lo;
      }
      if ((wave & 1) == 0) {  // the other half of this wave's last 32 keys
        const u16x4 z = {0, 0, 0, 0};
        *reinterpret_cast<u16x4*>(&sm.p[0][t][(wave + 1) * 16 + lg * 4]) = z;
        *reinterpret_cast<u16x4*>(&sm.p[1][t][(wave + 1) * 16 + lg * 4]) = z;
      }
      if (GATED) {
        rowsum = stride_reduce_sum<16, 4>(rowsum);
        if (lg == 0) sm.rs[t] = rowsum;
        // q_t . n, four lanes per token
        const int tq = tid >> 2, part = tid & 3;
        float dot = 0.f;
        for (int d = part * 8; d < DP; d += 32) {
          float x[8];
          const u16x8 raw = mc_ld16(&sm.q[0][tq][d]);
#pragma unroll
          for (int e = 0; e < 8; ++e) x[e] = bf16_to_f32(raw[e]) * sm.n[d + e];
#pragma unroll
          for (int e = 0; e < 8; ++e) dot += x[e];
        }
        dot += __shfl_xor(dot, 1, WAVE_SIZE);
        dot += __shfl_xor(dot, 2, WAVE_SIZE);
        if (part == 0) sm.qn[tq] = dot;
      }
    }
    // ---- the chunk's starting state with all queries -------------------------------------
    f32x4 o[4];
#pragma unroll
    for (int tt = 0; tt < 4; ++tt) o[tt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int u = 0; u < KB; ++u) {
      u16x8 hi, lo;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        uint16_t a, b;
        mc_split(S[2 * u][r], a, b);
        hi[r] = a;
        lo[r] = b;
        mc_split(S[2 * u + 1][r], a, b);
        hi[4 + r] = a;
        lo[4 + r] = b;
      }
      const int d = u * 32 + lg * 4;
#pragma unroll
      for (int tt = 0; tt < 4; ++tt) {
        const uint16_t* qp = sm.q[0][tt * 16 + li];
        const u16x8 b = mc_ld8x2(qp + d, qp + d + 16);
        o[tt] = mc_mfma(hi, b, o[tt]);
        o[tt] = mc_mfma(lo, b, o[tt]);
        if (ROT) {
          const uint16_t* ql = sm.q[NS - 1][tt * 16 + li];
          o[tt] = mc_mfma(hi, mc_ld8x2(ql + d, ql + d + 16), o[tt]);
        }
      }
    }
    __syncthreads();
    // ---- weighted scores with the wave's values; outputs -----------------------------------
    u16x8 vf[2];
#pragma unroll
    for (int sb = 0; sb < 2; ++sb) vf[sb] = mc_ld16(&sm.vt[col][sb * 32 + lg * 8]);
#pragma unroll
    for (int tt = 0; tt < 4; ++tt) {
      const int t = tt * 16 + li;
      const float ct = sm.c[t];
      o[tt] *= ct;
#pragma unroll
      for (int sb = 0; sb <= tt / 2; ++sb) {
        o[tt] = mc_mfma(vf[sb], mc_ld16(&sm.p[0][t][sb * 32 + lg * 8]), o[tt]);
        o[tt] = mc_mfma(vf[sb], mc_ld16(&sm.p[1][t][sb * 32 + lg * 8]), o[tt]);
      }
      if (t < cnt && wave * 16 + lg * 4 < ncol) {
        if (GATED) {
          const float den = fmaxf(fabsf(sm.rs[t] + ct * sm.qn[t]), sm.em[t]) + 1e-6f;
          o[tt] *= 1.0f / den;
        }
        *reinterpret_cast<f32x4*>(A.out + (r0 + t0 + t) * (long)(H * Dv) + h * Dv + c0 +
                                  wave * 16 + lg * 4) = o[tt];
      }
    }
    // ---- the keys' products join the state ---------------------------------------------------
    const float c_end = sm.c_end;
    u16x8 wh[2], wl[2];
#pragma unroll
    for (int sb = 0; sb < 2; ++sb) {
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        uint16_t a, b;
        mc_split(bf16_to_f32(vf[sb][e]) * sm.w[sb * 32 + lg * 8 + e], a, b);
        wh[sb][e] = a;
        wl[sb][e] = b;
      }
    }
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      S[dt] *= c_end;
#pragma unroll
      for (int sb = 0; sb < 2; ++sb) {
        const u16x8 a = mc_ld16(&sm.kt[0][dt * 16 + li][sb * 32 + lg * 8]);
        S[dt] = mc_mfma(a, wh[sb], S[dt]);
        S[dt] = mc_mfma(a, wl[sb], S[dt]);
        if (ROT)
          S[dt] = mc_mfma(mc_ld16(&sm.kt[NS - 1][dt * 16 + li][sb * 32 + lg * 8]), wh[sb], S[dt]);
      }
    }
    if (GATED) {
      for (int d = tid; d < DP; d += MC_THREADS) {
        float acc = sm.n[d] * c_end;
        for (int s = 0; s < MC_T; s += 8) {
          const u16x8 raw = mc_ld16(&sm.kt[0][d][s]);
#pragma unroll
          for (int e = 0; e < 8; ++e) acc += bf16_to_f32(raw[e]) * sm.w[s + e];
        }
        sm.n[d] = acc;
      }
    }
  }

#pragma unroll
  for (int dt = 0; dt < DT; ++dt) {
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = dt * 16 + lg * 4 + r;
      if (i < Dst && col < CB) srow[at(i, col)] = S[dt][r];
    }
  }
  if (GATED) {
    for (int i = tid; i < Dst; i += MC_THREADS) srow[at(i, CB)] = i < DP ? sm.n[i] : 0.f;
    if (tid == 0) *mrow = m_run;
  }
}

bool ms_chunks_served(const MsArgs& a, int form) {
  const bool rot = a.nf > 0;
  return a.D % 8 == 0 && a.Dv % 8 == 0 && a.D <= (rot ? 128 : 256) && a.nf % 8 == 0 &&
         !(rot && form == MS_GATED) && a.q_stride % 8 == 0 && a.k_stride % 8 == 0 &&
         a.v_stride % 8 == 0 && aligned16(a.q) && aligned16(a.k) && aligned16(a.v) &&
         aligned16(a.out) && aligned16(a.cs);
}

void ms_chunks_launch(const MsArgs& a, int form, int S, hipStream_t st) {
  const dim3 grid(S, a.H, a.NB);
#define LIG_MC(DP, G, R) \
  hipLaunchKernelGGL((matrix_state_chunk_kernel<DP, G, R>), grid, dim3(MC_THREADS), 0, st, a)
#define LIG_MC_D(G)                          \
  do {                                       \
    if (a.D <= 32) LIG_MC(32, G, false);     \
    else if (a.D <= 64) LIG_MC(64, G, false); \
    else if (a.D <= 128) LIG_MC(128, G, false); \
    else if (a.D <= 192) LIG_MC(192, G, false); \
    else LIG_MC(256, G, false);              \
  } while (0)
  if (a.nf > 0) {
    if (a.D <= 32) LIG_MC(32, false, true);
    else if (a.D <= 64) LIG_MC(64, false, true);
    else LIG_MC(128, false, true);
  } else if (form == MS_GATED) {
    LIG_MC_D(true);
  } else {
    LIG_MC_D(false);
  }
#undef LIG_MC_D
#undef LIG_MC
}
