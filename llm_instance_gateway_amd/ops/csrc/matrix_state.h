// What the kernels of the matrix-state recurrences share: the arguments, the
// layout of a sequence's state row and the delta form's gates.
#pragma once

#include "elem_types.h"

#define MS_COLS 64  // value columns per workgroup

enum { MS_CONST = 0, MS_BONUS = 1, MS_GATED = 2, MS_DELTA = 3 };

struct MsArgs {
  float* out;  // [R, H*Dv]
  const void *q, *k, *v;
  long q_stride, k_stride, v_stride;
  const float* decay_pre;   // [R, H*D]   (bonus form)
  const float* head_decay;  // [H]        (constant form)
  const float* bonus;       // [H*D]      (bonus form)
  const float *gate_i, *gate_f;  // [R, H] views, row stride gate_stride (gated form;
                                 // delta form: write strength and decay logits)
  long gate_stride;
  const float *bias_i, *bias_f;  // [H] (delta form: logarithm of the decay rate, decay bias)
  float gate_cap;
  const float* cs;  // nullable: [R, 2*nf] cosines | sines of the rotation
  int nf;
  float q_scale, k_scale;
  float* state;
  long state_stride;
  const int *seg_start, *seg_len, *seg_slot, *seg_fresh;
  int H, D, Dv, CB, NB, TT, act_silu;
  int split, kpt;        // key channel i of a state column sits in lane i / kpt, entry i % kpt
  int len_min, len_max;  // segments of other lengths belong to the other kernel
  int rep;               // value heads per query/key head (delta form; 1 elsewhere)
  float unit_eps;        // inside the root of the unit norms (delta form)
};

// Key split and key channels per thread for a head of D key channels: the
// smallest size class that holds ceil(D / split); kpt 0 when D is too wide.
static inline void ms_shape(int D, int* split, int* kpt) {
  static const int classes[] = {4, 8, 12, 16, 24, 32, 48, 64};
  *split = D >= 32 ? 8 : 4;
  const int need = (D + *split - 1) / *split;
  *kpt = 0;
  for (int c : classes)
    if (c >= need) {
      *kpt = c;
      break;
    }
}

// Delta form, one head of one token: the logarithm of the decay,
// -exp(log_rate) * softplus(z + bias), bounded where exp() of it is zero in
// fp32 terms anyway so that sums of it stay finite.
LIG_DEVICE float ms_log_decay(float z, float log_rate, float bias) {
  const float y = z + bias;
  const float sp = fmaxf(y, 0.f) + log1pf(expf(-fabsf(y)));
  return fmaxf(-expf(log_rate) * sp, -100.f);
}

// Chunked form on MFMA tiles (matrix_state_chunks.hip); false when the shape
// or alignment is not served.
bool ms_chunks_served(const MsArgs& a, int form);
void ms_chunks_launch(const MsArgs& a, int form, int S, hipStream_t stream);
// Chunked delta form (matrix_state_delta.hip); scratch holds
// ms_delta_scratch_bytes(R, S, H).
bool ms_delta_chunks_served(const MsArgs& a);
void ms_delta_chunks_launch(const MsArgs& a, int S, int max_seg_len, void* scratch,
                            hipStream_t stream);
