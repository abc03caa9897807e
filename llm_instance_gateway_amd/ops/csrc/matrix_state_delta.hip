// The gated delta rule in chunks of 64 tokens on MFMA tiles, gfx950 (bf16 q,
// k, v; fp32 state): the delta form of matrix_state_scan.hip, same arguments
// and state rows; these kernels take the long portions.
//
// Inside a chunk, with G_t the sum of the log decays up to token t, unit
// vectors k, q and S the state the chunk starts from, the corrections u solve
// a unit lower triangular system:
//     u_t + b_t sum_{s<t} e^(G_t-G_s) (k_t . k_s) u_s = b_t (v_t - e^(G_t) S^T k_t)
//     o_t = e^(G_t) S^T q_t + sum_{s<=t} e^(G_t-G_s) (q_t . k_s) u_s
//     S  <- e^(G_end) S + sum_s e^(G_end-G_s) k_s u_s^T
// (the WY form of the chunked delta rule).  The system's matrix does not
// depend on S, so its inverse is computed for all chunks of the step at once:
//
// delta_chunk_inverse_kernel, one workgroup (4 waves) per (chunk, segment,
// head): k . k by MFMA on bf16 rows (exact products), fp32 from there on.
// The four 16 x 16 diagonal blocks are inverted by substitution, a column per
// lane; the blocks below them follow level by level,
//     T_ij = -T_ii sum_{j<=m<i} A_im T_mj,
// with fp32 MFMA (16x16x4).  The inverse times diag(b) leaves as two bf16
// halves, with the token factors the second kernel needs.  The log decays are
// summed in double: a token that decays nearly everything must not cost the
// differences after it their precision.
//
// delta_chunk_scan_kernel, one workgroup per (segment, head, one or two
// blocks of 64 value columns), walks the chunks; wave w owns 16 columns of
// the state, [D, 16] fp32 in MFMA accumulators for the whole segment.  The
// state, the right-hand sides and the corrections go from accumulators
// straight into the next product as an operand: a contraction may visit its
// inner index in any order as long as both operands agree, so the other
// operand is read from LDS in the order the accumulators hold it.  Per chunk
// the waves share only the staged q, k, k transposed, the inverse and the
// weighted scores.  The next chunk's rows are fetched into registers during
// the arithmetic.
//
// Precision: products of bf16 numbers are exact in fp32, sums are fp32, fp32
// operands are split into two bf16 halves (lo * lo left out).  The unit norms
// stay fp32 scalars outside the bf16 vectors.

#include "matrix_state.h"
#include "matrix_state_mfma.h"

// What the first kernel leaves for one (chunk, head).
struct DeltaChunk {
  uint16_t t_hi[MC_T][MC_T];  // inverse * diag(b); blocks above the diagonal unwritten
  uint16_t t_lo[MC_T][MC_T];
  double G[MC_T];     // summed log decays
  float ik[MC_T];     // 1 / |k|
  float ek[MC_T];     // e^G / |k|
  float eg[MC_T];     // e^G
  float wk[MC_T];     // e^(G_end - G) / |k|, 0 past the portion's end
};

// Chunk c of segment seg (first row r0): segments lie in row order, so these
// places are distinct and below R / 64 + S + 1.
LIG_DEVICE long delta_chunk_slot(long r0, int c, int seg) { return r0 / MC_T + c + seg; }

extern "C" long lig_gated_delta_scratch(int R, int S, int H) {
  return ((long)R / MC_T + S + 1) * H * (long)sizeof(DeltaChunk);
}

#define DI_THREADS 256
#define DI_ROW 68  // padded fp32 LDS row

template <int DP>
__global__ __launch_bounds__(DI_THREADS) void delta_chunk_inverse_kernel(
    const MsArgs A, DeltaChunk* __restrict__ scratch) {
  constexpr int KB = DP / 32;
  // One square holds both triangles in 16 x 16 blocks: the system's block (i,
  // j) at its own place, the inverse's block (i, j) at place (j, i), each in
  // row order; a diagonal block of the inverse replaces the system's.
  __shared__ __align__(16) float a_s[MC_T][DI_ROW];
  __shared__ double g_s[MC_T];
  __shared__ __align__(16) float b_s[MC_T];
  __shared__ float ik_s[MC_T];

  const int seg = blockIdx.y, h = blockIdx.z;
  const int n = A.seg_len[seg];
  const int c0 = blockIdx.x * MC_T;
  if (c0 >= n || n < A.len_min) return;
  const int cnt = min(MC_T, n - c0);
  const long r0 = A.seg_start[seg];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int li = lane & 15, lg = lane >> 4;
  const uint16_t* k = (const uint16_t*)A.k + (h / A.rep) * A.D + (r0 + c0) * A.k_stride;
  DeltaChunk* out = scratch + delta_chunk_slot(r0, blockIdx.x, seg) * A.H + h;

  if (wave == 0) {
    float b = 0.f, lgd = 0.f;
    if (lane < cnt) {
      const long r = (r0 + c0 + lane) * A.gate_stride + h;
      b = sigmoid_f32(A.gate_i[r]);
      lgd = ms_log_decay(A.gate_f[r], A.bias_i[h], A.bias_f[h]);
    }
    double G = (double)lgd;
#pragma unroll
    for (int d = 1; d < MC_T; d <<= 1) {
      const double u = __shfl_up(G, d, WAVE_SIZE);
      if (lane >= d) G += u;
    }
    g_s[lane] = G;
    b_s[lane] = b;
  }

  // ---- k . k: wave's 16 tokens against the tokens up to them -------------------------
  auto row = [&](int t, int kb) __attribute__((always_inline)) {
    const int d = kb * 32 + lg * 8;
    u16x8 z = {0, 0, 0, 0, 0, 0, 0, 0};
    return (t < cnt && d < A.D) ? mc_ld16(k + t * A.k_stride + d) : z;
  };
  u16x8 af[KB];
#pragma unroll
  for (int kb = 0; kb < KB; ++kb) af[kb] = row(wave * 16 + li, kb);
  f32x4 acc[4];
#pragma unroll
  for (int st = 0; st < 4; ++st) {
    acc[st] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (st <= wave) {
#pragma unroll
      for (int kb = 0; kb < KB; ++kb) acc[st] = mc_mfma(af[kb], row(st * 16 + li, kb), acc[st]);
      if (st == wave) {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (lg * 4 + r == li) ik_s[wave * 16 + li] = 1.0f / sqrtf(acc[st][r] + A.unit_eps);
      }
    }
  }
  __syncthreads();
  // ---- the system's strictly lower part --------------------------------------------------
#pragma unroll
  for (int st = 0; st < 4; ++st) {
    if (st <= wave) {
      const int s = st * 16 + li;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = wave * 16 + lg * 4 + r;
        float a = 0.f;
        if (s < t)
          a = b_s[t] * ik_s[t] * ik_s[s] * __expf((float)(g_s[t] - g_s[s])) * acc[st][r];
        a_s[t][s] = a;
      }
    }
  }
  __syncthreads();
  // ---- diagonal blocks: lane li solves for column li of the inverse ------------------------
  {
    const int b = wave * 16;
    float x[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float v = i == li ? 1.f : 0.f;
#pragma unroll
      for (int m = 0; m < i; ++m) v -= a_s[b + i][b + m] * x[m];
      x[i] = v;
    }
    if (lg == 0) {
#pragma unroll
      for (int i = 0; i < 16; ++i) a_s[b + i][b + li] = x[i];
    }
  }
  __syncthreads();
  // ---- blocks below the diagonal, one level of distance at a time --------------------------
#pragma unroll
  for (int lvl = 1; lvl < 4; ++lvl) {
    if (wave + lvl < 4) {
      const int bi = (wave + lvl) * 16, bj = wave * 16;
      f32x4 x = {0.f, 0.f, 0.f, 0.f}, y = {0.f, 0.f, 0.f, 0.f};
      for (int m = bj; m < bi; m += 16) {
#pragma unroll
        for (int e = 0; e < 16; e += 4)
          x = __builtin_amdgcn_mfma_f32_16x16x4f32(a_s[bi + li][m + e + lg], a_s[bj + e + lg][m + li],
                                                   x, 0, 0, 0);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r)  // x's rows lg * 4 + r are this lane's share of the contraction
        y = __builtin_amdgcn_mfma_f32_16x16x4f32(a_s[bi + li][bi + lg * 4 + r], x[r], y, 0, 0, 0);
#pragma unroll
      for (int r = 0; r < 4; ++r) a_s[bj + lg * 4 + r][bi + li] = -y[r];
    }
    __syncthreads();
  }
  // ---- write out ------------------------------------------------------------------------------
  {
    const int t = tid >> 2, s0 = (tid & 3) * 16;
    if (s0 <= t) {
      const float* src = &a_s[s0 + (t & 15)][t & ~15];  // row t of block (t / 16, s0 / 16)
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        u32x4 hi, lo;
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          const int s = half * 8 + e * 4;
          mc_split4(*reinterpret_cast<const f32x4*>(src + s) *
                        *reinterpret_cast<const f32x4*>(&b_s[s0 + s]), e, hi, lo);
        }
        *reinterpret_cast<u32x4*>(&out->t_hi[t][s0 + half * 8]) = hi;
        *reinterpret_cast<u32x4*>(&out->t_lo[t][s0 + half * 8]) = lo;
      }
    }
  }
  if (tid < MC_T) {
    const double G = g_s[tid], G_end = g_s[MC_T - 1];  // tokens past the end decay nothing
    const float ik = ik_s[tid], eg = expf((float)G);
    out->G[tid] = G;
    out->ik[tid] = ik;
    out->eg[tid] = eg;
    out->ek[tid] = eg * ik;
    out->wk[tid] = tid < cnt ? expf((float)(G_end - G)) * ik : 0.f;
  }
}

// NW waves: 4 walk one block of 64 value columns, 8 walk two that share q, k,
// the inverse and the weighted scores.
template <int DP, int NW>
__global__ __launch_bounds__(NW * WAVE_SIZE) void delta_chunk_scan_kernel(
    const MsArgs A, const DeltaChunk* __restrict__ scratch) {
  // LDS rows advance by 2 banks (mod 32), so that the 8-byte operand reads of
  // 16 rows spread over all of them
  constexpr int KB = DP / 32, DT = DP / 16, DROW = DP + 4, TROW = MC_T + 4;
  constexpr int CC = DP / 8;                  // 16-byte chunks of a q or k row
  constexpr int NCH = (CC + NW - 1) / NW;     // of them per thread
  constexpr int NT = 2 * MC_T * MC_T / 8 / (NW * WAVE_SIZE);  // inverse chunks per thread
  struct Shared {
    uint16_t q[MC_T][DROW];
    uint16_t k[MC_T][DROW];
    uint16_t kt[DP][TROW];
    uint16_t t[2][MC_T][TROW];
    uint16_t p[2][MC_T][TROW];
    double G[MC_T];
    float ik[MC_T], ek[MC_T], wk[MC_T], eg[MC_T];
    float c[MC_T];        // e^G * q_scale / |q|
    float qs[NW][MC_T];   // shares of |q|^2
  };
  __shared__ __align__(16) Shared sm;

  const int seg = blockIdx.x, h = blockIdx.y;
  const int n = A.seg_len[seg];
  if (n <= 0 || n < A.len_min) return;
  const int H = A.H, D = A.D, Dv = A.Dv, CB = A.CB;
  const long r0 = A.seg_start[seg];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int li = lane & 15, lg = lane >> 4;
  const int blk = blockIdx.z * (NW / 4) + (wave >> 2);
  const bool active = blk < A.NB;  // uniform over the wave; others stage and score only
  const int c0 = blk * CB, ncol = active ? min(CB, Dv - c0) : 0;
  const int col = (wave & 3) * 16 + li;  // the state column this lane holds
  const uint16_t* q = (const uint16_t*)A.q + (h / A.rep) * D;
  const uint16_t* k = (const uint16_t*)A.k + (h / A.rep) * D;
  const uint16_t* v = (const uint16_t*)A.v + h * Dv + (active ? c0 : 0);
  const DeltaChunk* ch = scratch + delta_chunk_slot(r0, 0, seg) * H + h;

  // ---- state row: [head][block][entry][column * split + key lane] ----------------------
  const int nthr = CB * A.split, Dst = A.split * A.kpt;
  float* srow = A.state + (long)A.seg_slot[seg] * A.state_stride + (long)(h * A.NB + blk) * A.kpt * nthr;
  const bool resume = A.seg_fresh[seg] == 0;
  auto at = [&](int i, int j) { return (long)(i % A.kpt) * nthr + j * A.split + i / A.kpt; };
  f32x4 S[DT];
#pragma unroll
  for (int dt = 0; dt < DT; ++dt) {
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = dt * 16 + lg * 4 + r;
      S[dt][r] = (active && resume && i < Dst && col < CB) ? srow[at(i, col)] : 0.f;
    }
  }
  // the blocks above the diagonal are never written: zero for the whole walk
  for (int e = tid; e < 2 * MC_T * TROW / 8; e += NW * WAVE_SIZE) {
    const u16x8 z = {0, 0, 0, 0, 0, 0, 0, 0};
    reinterpret_cast<u16x8*>(&sm.t[0][0][0])[e] = z;
    reinterpret_cast<u16x8*>(&sm.p[0][0][0])[e] = z;
  }

  // A thread stages token `lane`, 16-byte chunks wave, wave + NW, ...  Rows past
  // the portion's end read its last token instead: their write strength and
  // their weight in the state are zero and their outputs are not stored.
  u16x8 qr[NCH], kr[NCH], tr[NT];
  uint16_t vr[16];
  double Gr = 0.0;
  float sr[4] = {0.f, 0.f, 0.f, 0.f};
  const u16x8 zero8 = {0, 0, 0, 0, 0, 0, 0, 0};
  const int q_stride = (int)A.q_stride, k_stride = (int)A.k_stride, v_stride = (int)A.v_stride;
  const int q_off = lane * q_stride, k_off = lane * k_stride;
  const bool col_ok = col < ncol;
  const int v_off = lg * 4 * v_stride + (col_ok ? col : 0);
  auto fetch = [&](int t0) __attribute__((always_inline)) {
    const uint16_t* qb = q + (r0 + t0) * A.q_stride;
    const uint16_t* kb = k + (r0 + t0) * A.k_stride;
    const int last = n - 1 - t0;
    const int qo = last < MC_T - 1 ? min(lane, last) * q_stride : q_off;
    const int ko = last < MC_T - 1 ? min(lane, last) * k_stride : k_off;
#pragma unroll
    for (int j = 0; j < NCH; ++j) {
      const int d = (wave + NW * j) * 8;
      const bool in = d < D;  // uniform over the wave
      qr[j] = in ? mc_ld16(qb + qo + d) : zero8;
      kr[j] = in ? mc_ld16(kb + ko + d) : zero8;
    }
    const DeltaChunk* c = ch + (long)(t0 / MC_T) * H;
#pragma unroll
    for (int j = 0; j < NT; ++j) {
      const int e = tid + j * NW * WAVE_SIZE;
      const int t = (e / 8) % MC_T, s0 = (e % 8) * 8;
      const uint16_t* src = e < MC_T * MC_T / 8 ? &c->t_hi[t][s0] : &c->t_lo[t][s0];
      if (s0 / 16 <= t / 16) tr[j] = mc_ld16(src);
    }
    if (tid < MC_T) {
      Gr = c->G[tid];
      sr[0] = c->ik[tid];
      sr[1] = c->ek[tid];
      sr[2] = c->wk[tid];
      sr[3] = c->eg[tid];
    }
  };
  // values of token tt * 16 + lg * 4 + i, column col
  auto fetch_v = [&](int t0) __attribute__((always_inline)) {
    const uint16_t* vb = v + (r0 + t0) * A.v_stride;
    const int last = n - 1 - t0;
    if (last >= MC_T - 1) {
#pragma unroll
      for (int e = 0; e < 16; ++e) vr[e] = vb[v_off + ((e >> 2) * 16 + (e & 3)) * v_stride];
    } else {
#pragma unroll
      for (int e = 0; e < 16; ++e)
        vr[e] = vb[min((e >> 2) * 16 + lg * 4 + (e & 3), last) * v_stride + (col_ok ? col : 0)];
    }
  };
  fetch(0);
  fetch_v(0);

#pragma nounroll
  for (int t0 = 0; t0 < n; t0 += MC_T) {
    const int cnt = min(MC_T, n - t0);
    __syncthreads();  // the previous chunk's readers are done
    // ---- staging -------------------------------------------------------------------------
    float sq = 0.f;
#pragma unroll
    for (int j = 0; j < NCH; ++j) {
      const int d = (wave + NW * j) * 8;
      if (d < DP) {
        mc_st8x2(&sm.q[lane][d], qr[j]);
        mc_st8x2(&sm.k[lane][d], kr[j]);
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          sm.kt[d + e][lane] = kr[j][e];
          const float x = bf16_to_f32(qr[j][e]);
          sq += x * x;
        }
      }
    }
    sm.qs[wave][lane] = sq;
#pragma unroll
    for (int j = 0; j < NT; ++j) {
      const int e = tid + j * NW * WAVE_SIZE;
      const int half = e / (MC_T * MC_T / 8), t = (e / 8) % MC_T, s0 = (e % 8) * 8;
      if (s0 / 16 <= t / 16) mc_st8x2(&sm.t[half][t][s0], tr[j]);
    }
    if (tid < MC_T) {
      sm.G[tid] = Gr;
      sm.ik[tid] = sr[0];
      sm.ek[tid] = sr[1];
      sm.wk[tid] = sr[2];
      sm.eg[tid] = sr[3];
    }
    __syncthreads();
    if (t0 + MC_T < n) fetch(t0 + MC_T);

    // ---- weighted scores: 16 tokens against keys up to them ---------------------------------
    {
      const int tile = wave & 3, t = tile * 16 + li;
      float qq = 0.f;
#pragma unroll
      for (int w = 0; w < (CC < NW ? CC : NW); ++w) qq += sm.qs[w][t];
      const float iq = A.q_scale / sqrtf(qq + A.unit_eps);
      const double Gt = sm.G[t];
      if (wave < 4 && lg == 0) sm.c[t] = sm.eg[t] * iq;
      for (int st = wave >> 2; st <= tile; st += NW / 4) {
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kb = 0; kb < KB; ++kb) {
          const int d = kb * 32 + lg * 8;
          const uint16_t *kp = &sm.k[st * 16 + li][d], *qp = &sm.q[t][d];
          acc = mc_mfma(mc_ld8x2(kp, kp + 4), mc_ld8x2(qp, qp + 4), acc);
        }
        f32x4 p;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int s = st * 16 + lg * 4 + r;
          p[r] = s <= t ? acc[r] * iq * sm.ik[s] * __expf((float)(Gt - sm.G[s])) : 0.f;
        }
        uint32_t h0, h1, l0, l1;
        mc_split2(p[0], p[1], h0, l0);
        mc_split2(p[2], p[3], h1, l1);
        *reinterpret_cast<u32x2*>(&sm.p[0][t][st * 16 + lg * 4]) = u32x2{h0, h1};
        *reinterpret_cast<u32x2*>(&sm.p[1][t][st * 16 + lg * 4]) = u32x2{l0, l1};
      }
    }
    f32x4 o[4];
    u32x4 uh[2], ul[2], wh[2], wl[2];
    if (active) {
      // ---- the chunk's starting state with all keys and all queries ---------------------------
      f32x4 x[4];
#pragma unroll
      for (int tt = 0; tt < 4; ++tt) x[tt] = o[tt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int u = 0; u < KB; ++u) {
        u32x4 sh, sl;
        mc_split4(S[2 * u], 0, sh, sl);
        mc_split4(S[2 * u + 1], 1, sh, sl);
#pragma unroll
        for (int tt = 0; tt < 4; ++tt) {
          const uint16_t* kp = &sm.k[tt * 16 + li][u * 32 + lg * 4];
          const uint16_t* qp = &sm.q[tt * 16 + li][u * 32 + lg * 4];
          const u16x8 a = mc_ld8x2(kp, kp + 16), b = mc_ld8x2(qp, qp + 16);
          x[tt] = mc_mfma(a, sh, x[tt]);
          o[tt] = mc_mfma(sh, b, o[tt]);
          x[tt] = mc_mfma(a, sl, x[tt]);
          o[tt] = mc_mfma(sl, b, o[tt]);
        }
      }
      // ---- right-hand sides: v - e^G S^T k ---------------------------------------------------
      u32x4 rh[2], rl[2];
#pragma unroll
      for (int tt = 0; tt < 4; ++tt) {
        const f32x4 ek = *reinterpret_cast<const f32x4*>(&sm.ek[tt * 16 + lg * 4]);
        f32x4 val;
#pragma unroll
        for (int i = 0; i < 4; ++i) val[i] = col_ok ? bf16_to_f32(vr[tt * 4 + i]) : 0.f;
        mc_split4(val - ek * x[tt], tt & 1, rh[tt / 2], rl[tt / 2]);
      }
      if (t0 + MC_T < n) fetch_v(t0 + MC_T);
      // ---- corrections u = inverse * right-hand sides ----------------------------------------
#pragma unroll
      for (int tt = 0; tt < 4; ++tt) {
        f32x4 c = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int u = 0; u <= tt / 2; ++u) {
          const uint16_t* th = &sm.t[0][tt * 16 + li][u * 32 + lg * 4];
          const uint16_t* tl = &sm.t[1][tt * 16 + li][u * 32 + lg * 4];
          const u16x8 a = mc_ld8x2(th, th + 16);
          c = mc_mfma(a, rh[u], c);
          c = mc_mfma(a, rl[u], c);
          c = mc_mfma(mc_ld8x2(tl, tl + 16), rh[u], c);
        }
        const f32x4 wk = *reinterpret_cast<const f32x4*>(&sm.wk[tt * 16 + lg * 4]);
        mc_split4(c, tt & 1, uh[tt / 2], ul[tt / 2]);
        mc_split4(c * wk, tt & 1, wh[tt / 2], wl[tt / 2]);
      }
    }
    __syncthreads();
    if (active) {
      // ---- weighted scores with the corrections; outputs -----------------------------------------
#pragma unroll
      for (int tt = 0; tt < 4; ++tt) {
        const int t = tt * 16 + li;
        o[tt] *= sm.c[t];
#pragma unroll
        for (int u = 0; u <= tt / 2; ++u) {
          const uint16_t* ph = &sm.p[0][t][u * 32 + lg * 4];
          const uint16_t* pl = &sm.p[1][t][u * 32 + lg * 4];
          const u16x8 b = mc_ld8x2(ph, ph + 16);
          o[tt] = mc_mfma(uh[u], b, o[tt]);
          o[tt] = mc_mfma(ul[u], b, o[tt]);
          o[tt] = mc_mfma(uh[u], mc_ld8x2(pl, pl + 16), o[tt]);
        }
        const int vc = (wave & 3) * 16 + lg * 4;
        if (t < cnt && vc < ncol)
          *reinterpret_cast<f32x4*>(A.out + (r0 + t0 + t) * (long)(H * Dv) + h * Dv + c0 + vc) = o[tt];
      }
      // ---- the keys' products join the state --------------------------------------------------------
      const float g_end = sm.eg[MC_T - 1];
#pragma unroll
      for (int dt = 0; dt < DT; ++dt) {
        S[dt] *= g_end;
#pragma unroll
        for (int u = 0; u < 2; ++u) {
          const uint16_t* kp = &sm.kt[dt * 16 + li][u * 32 + lg * 4];
          const u16x8 a = mc_ld8x2(kp, kp + 16);
          S[dt] = mc_mfma(a, wh[u], S[dt]);
          S[dt] = mc_mfma(a, wl[u], S[dt]);
        }
      }
    }
  }

  if (active) {
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = dt * 16 + lg * 4 + r;
        if (i < Dst && col < CB) srow[at(i, col)] = S[dt][r];
      }
    }
  }
}

bool ms_delta_chunks_served(const MsArgs& a) {
  // offsets inside a chunk are 32-bit
  const long lim = 2147483647L / MC_T;
  return a.q_stride <= lim && a.k_stride <= lim && a.v_stride <= lim && a.D % 8 == 0 &&
         a.Dv % 8 == 0 && a.D <= 256 && a.q_stride % 8 == 0 &&
         a.k_stride % 8 == 0 && aligned16(a.q) && aligned16(a.k) && aligned16(a.out);
}

void ms_delta_chunks_launch(const MsArgs& a, int S, int max_seg_len, void* scratch,
                            hipStream_t st) {
  DeltaChunk* sc = (DeltaChunk*)scratch;
  const dim3 gi((max_seg_len + MC_T - 1) / MC_T, S, a.H);
  // two value blocks per workgroup share the staged operands where the
  // registers of eight waves hold the state
#define LIG_DC(DP)                                                                            \
  do {                                                                                        \
    hipLaunchKernelGGL(delta_chunk_inverse_kernel<DP>, gi, dim3(DI_THREADS), 0, st, a, sc);   \
    constexpr int NW = DP <= 128 ? 8 : 4;                                                     \
    if (a.NB > 1)                                                                             \
      hipLaunchKernelGGL((delta_chunk_scan_kernel<DP, NW>),                                   \
                         dim3(S, a.H, (a.NB + NW / 4 - 1) / (NW / 4)), dim3(NW * WAVE_SIZE),  \
                         0, st, a, sc);                                                       \
    else                                                                                      \
      hipLaunchKernelGGL((delta_chunk_scan_kernel<DP, 4>), dim3(S, a.H, 1),                   \
                         dim3(4 * WAVE_SIZE), 0, st, a, sc);                                  \
  } while (0)
  if (a.D <= 32) LIG_DC(32);
  else if (a.D <= 64) LIG_DC(64);
  else if (a.D <= 128) LIG_DC(128);
  else if (a.D <= 192) LIG_DC(192);
  else LIG_DC(256);
#undef LIG_DC
}
