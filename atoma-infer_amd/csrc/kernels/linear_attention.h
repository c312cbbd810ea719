// Linear attention with a decaying state, no softmax and no denominator.  Per head, with q, k [dim] and v [vdim] of a
// token's projections,
//
//   S <- diag(alpha) S + k v^T,        o = S^T q,        y = o / sqrt(mean(o^2) + eps) * w * silu(g),
//
// S [dim, vdim] float32 per request and head, the mean over a head's vdim columns, w [vdim] shared by the heads or absent.
// Two kinds of decay:
//   * fixed: alpha is one number a head;
//   * gated: a number per key channel and token, alpha = sigmoid(z)^(1 / tau), z = W_2 l + b with l, a few numbers a
//     token, columns of the projection (the first half of a low-rank map).
// q and k may be rotated: column i < rot / 2 of a head with column i + rot / 2 by the angle position * freq[i] (float32,
// no table); q and k are multiplied by q_scale and k_scale.  State row layout: [heads][vdim][dim].
//
//   la_scan      token by token: a workgroup owns (entry, head) and up to 256 columns of S, a column in the registers of
//                16 neighbouring lanes, four neighbouring rows a lane at a time.  Where a workgroup holds all of a head's
//                columns the norm and the gate are in the same kernel, which then is the whole step of a decoded token
//                between two projections; else o leaves in float32 for la_out.
//   la_out       norm and gate of the entries that la_scan left unfinished, a wave a (token, head).
//   la_prepare,  entries of many tokens, in chunks of 64 tokens that are all worked on side by side
//   la_pass,     (linear_attention_chunks.hip).
//   la_finish
// State rows are read before an entry's first token and written behind its last, so prompts, portions and decoded tokens
// may be cut anywhere.  All sums, decays and the state are float32.
#pragma once
#include "common.h"

namespace atoma {

struct LinearAttention {
  const float* proj;            // [T, ld]
  int ld, off_q, off_k, off_v, off_g;
  const float* decay;           // [heads]: fixed decays; null: gated
  int off_low, rank;            // gated: columns of l, and how many
  const float* w2;              // [heads dim, rank]
  const float* b2;              // [heads dim]
  float inv_tau;
  const int32_t* positions;     // [T], read if rot > 0
  const float* freq;            // [rot / 2]
  const float* angles;          // [T, rot]: cosines, then sines of a token's pairs; read by the chunked kernels
  int rot;
  float q_scale, k_scale;
  const float* norm_w;          // [vdim] or null
  float eps;
  const int32_t* q_start;
  const int32_t* state_slots;
  float* state;
  int heads, dim, vdim;
};

constexpr int kMaxRot = 256;

__device__ __forceinline__ float silu(float x) { return x / (1.0f + expf(-x)); }

// sum over the 16 lanes of a DPP row; every lane gets it
__device__ __forceinline__ float row16_sum(float x) {
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0xB1, 0xf, 0xf, false));    // lanes i ^ 1
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x4E, 0xf, 0xf, false));    // lanes i ^ 2
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x141, 0xf, 0xf, false));   // the other quad of 8
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x140, 0xf, 0xf, false));   // the other half of 16
  return x;
}

// sigmoid(z)^(1 / tau) = exp(log sigmoid(z) / tau), log sigmoid(z) = min(z, 0) - log(1 + exp(-|z|)).  The logarithm's
// argument lies between 1 and 2, so its absolute error is that of a float near one, and with it the decay's relative
// error; v_exp_f32 and v_log_f32 (base 2) are good to about one unit in the last place.
__device__ __forceinline__ float gated_decay(float z, float inv_tau) {
  constexpr float kLog2e = 1.4426950408889634f;
  const float l = __builtin_amdgcn_logf(1.0f + __builtin_amdgcn_exp2f(-fabsf(z) * kLog2e));
  return __builtin_amdgcn_exp2f((fminf(z, 0.f) * kLog2e - l) * inv_tau);
}

// column r of a head's rotated q or k; cs, sn: cosines and sines of the token's pairs
__device__ __forceinline__ float rotated(const float* __restrict__ x, int r, int rot, const float* cs, const float* sn) {
  if (r >= rot) return x[r];
  const int half = rot >> 1;
  return r < half ? x[r] * cs[r] - x[r + half] * sn[r] : x[r] * cs[r - half] + x[r - half] * sn[r - half];
}

inline bool linear_attention_ok(const LinearAttention& a) {
  if (a.heads <= 0 || a.dim <= 0 || a.dim > 256 || a.vdim <= 0 || a.rot < 0 || a.rot % 2 || a.rot > a.dim ||
      a.rot > kMaxRot || a.off_q < 0 || a.off_k < 0 || a.off_v < 0 || a.off_g < 0 || a.ld < a.off_q + a.heads * a.dim ||
      a.ld < a.off_k + a.heads * a.dim || a.ld < a.off_v + a.heads * a.vdim || a.ld < a.off_g + a.heads * a.vdim)
    return false;
  if (a.decay == nullptr)
    return a.rot == 0 && a.rank > 0 && a.off_low >= 0 && a.ld >= a.off_low + a.rank && a.w2 && a.b2 && a.inv_tau > 0.f;
  return a.rot == 0 || (a.positions && a.freq);
}

inline LinearAttention linear_attention_args(const float* proj, const int32_t* at, const float* decay, const float* w2,
                                            const float* b2, float inv_tau, const int32_t* positions, const float* freq,
                                            const float* angles, int rot, float q_scale, float k_scale,
                                            const float* norm_w, float eps, const int32_t* q_start,
                                            const int32_t* state_slots, float* state, int heads, int dim, int vdim) {
  LinearAttention a;
  a.proj = proj, a.ld = at[0], a.off_q = at[1], a.off_k = at[2], a.off_v = at[3], a.off_g = at[4];
  a.decay = decay, a.off_low = at[5], a.rank = at[6], a.w2 = w2, a.b2 = b2, a.inv_tau = inv_tau;
  a.positions = positions, a.freq = freq, a.angles = angles, a.rot = rot, a.q_scale = q_scale, a.k_scale = k_scale;
  a.norm_w = norm_w, a.eps = eps, a.q_start = q_start, a.state_slots = state_slots, a.state = state;
  a.heads = heads, a.dim = dim, a.vdim = vdim;
  return a;
}

}  // namespace atoma
