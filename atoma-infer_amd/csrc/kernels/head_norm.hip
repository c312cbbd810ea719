// Queries and keys normed head by head, and the cache write, in one pass.
//
// Per token, from the float32 result of the fused q, k, v projection [T, >= nh hd + nkv hd + nkv vd]:
//   q_h <- q_h / sqrt(mean(q_h^2) + eps) * wq over the hd columns of every query head, to q_out [T, nh hd_out];
//   k_g <- k_g / sqrt(mean(k_g^2) + eps) * wk over those of every key head, into the key tiles;
//   v_g as it is, into the value tiles.
// wq and wk hold one number a column, shared by all heads.  Heads may leave wider than they came (hd_out >= hd, vd_out
// >= vd, zeros beyond): zeros add nothing to a score, and a value's zero columns meet zero columns of the output
// projection.  The tiles' element order is the attention kernels' (cache_layout.h).
//
// A head of a token is a unit of LANES lanes, four neighbouring columns a lane; units lie token by token (all query
// heads, key heads, value heads of a token, then the next token's).  VEC: rows whose pieces of four columns may be
// read and written with one instruction.
#include "common.h"
#include "cache_layout.h"

using namespace atoma;

__device__ __forceinline__ void put4(float* p, const float (&v)[4]) {
  *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
}
__device__ __forceinline__ void put4(bf16_t* p, const float (&v)[4]) {
  uint2 o;
  o.x = (uint32_t)f32_to_bf16_bits(v[0]) | ((uint32_t)f32_to_bf16_bits(v[1]) << 16);
  o.y = (uint32_t)f32_to_bf16_bits(v[2]) | ((uint32_t)f32_to_bf16_bits(v[3]) << 16);
  *reinterpret_cast<uint2*>(p) = o;
}

template <typename TQ, typename TC, int LANES, bool VEC>
__global__ void __launch_bounds__(256)
head_norm_kernel(const float* __restrict__ proj, int ld, const int32_t* __restrict__ slot_mapping, int n_units, int units,
                 int nh, int nkv, int hd, int vd, const float* __restrict__ wq, const float* __restrict__ wk, float eps,
                 TQ* __restrict__ q_out, TC* __restrict__ kcache, TC* __restrict__ vcache, int page_size, int hd_out,
                 int vd_out) {
  const int u = (blockIdx.x * 256 + threadIdx.x) / LANES, lane = threadIdx.x % LANES;
  if (u >= n_units) return;          // (whole units leave: the sums below stay inside a unit)
  const int t = u / units, h = u % units;
  const bool is_v = h >= nh + nkv, is_k = !is_v && h >= nh;
  const int size = is_v ? vd : hd, size_out = is_v ? vd_out : hd_out;
  const float* x = proj + (size_t)t * ld + (is_v ? (nh + nkv) * hd + (h - nh - nkv) * vd : h * hd);
  const float* w = is_k ? wk : wq;
  const int slot = h >= nh ? slot_mapping[t] : 0;
  const int d = lane * 4;
  float v[4] = {0.f, 0.f, 0.f, 0.f}, wt[4] = {1.f, 1.f, 1.f, 1.f};
  if (VEC) {
    if (d < size) {
      const float4 a = *reinterpret_cast<const float4*>(x + d);
      v[0] = a.x, v[1] = a.y, v[2] = a.z, v[3] = a.w;
      if (!is_v) {
        const float4 b = *reinterpret_cast<const float4*>(w + d);
        wt[0] = b.x, wt[1] = b.y, wt[2] = b.z, wt[3] = b.w;
      }
    }
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (d + i < size) {
        v[i] = x[d + i];
        if (!is_v) wt[i] = w[d + i];
      }
  }
  float ss = v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
#pragma unroll
  for (int o = LANES / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, LANES);
  if (!is_v) {
    const float inv = 1.0f / sqrtf(ss / (float)hd + eps);
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = v[i] * inv * wt[i];
  }
  if (d >= size_out) return;
  // (size_out is a multiple of 4, so a lane's four columns are all inside; a run of eight columns of a key tile too)
  if (h < nh) {
    put4(q_out + ((size_t)t * nh + h) * hd_out + d, v);
    return;
  }
  if (slot < 0) return;
  const int page = slot / page_size, off = slot % page_size;
  if (is_k) {
    TC* tile = kcache + ((size_t)page * nkv + (h - nh)) * page_size * hd_out;
    put4(tile + key_offset(off, d, page_size), v);
  } else {
    TC* tile = vcache + ((size_t)page * nkv + (h - nh - nkv)) * page_size * vd_out;
#pragma unroll
    for (int i = 0; i < 4; ++i) tile[value_offset(d + i, off, vd_out, page_size)] = from_f32<TC>(v[i]);
  }
}

extern "C" int atoma_head_norm(const float* proj, int ld, const int32_t* slot_mapping, const float* wq, const float* wk,
                               float eps, void* q_out, void* kcache, void* vcache, int dtype, int page_size, int n_tokens,
                               int nh, int nkv, int hd, int vd, int hd_out, int vd_out, hipStream_t stream) {
  if (n_tokens <= 0) return 0;
  if (nh <= 0 || nkv <= 0 || hd <= 0 || vd <= 0 || hd_out < hd || vd_out < vd || hd_out > 256 || vd_out > 256 ||
      hd_out % 8 || vd_out % 8 || page_size <= 0 || ld < (nh + nkv) * hd + nkv * vd ||
      (((uintptr_t)q_out | (uintptr_t)kcache | (uintptr_t)vcache) & 15))
    return ATOMA_ERR_SHAPE;
  const int units = nh + 2 * nkv, widest = hd_out > vd_out ? hd_out : vd_out;
  if ((int64_t)n_tokens * units > (int64_t)1 << 30) return ATOMA_ERR_SHAPE;
  const int n_units = n_tokens * units;
  const bool vec = hd % 4 == 0 && vd % 4 == 0 && ld % 4 == 0 && (((uintptr_t)proj | (uintptr_t)wq | (uintptr_t)wk) & 15) == 0;
  const int lanes = widest <= 64 ? 16 : widest <= 128 ? 32 : 64;
  const dim3 grid((unsigned)(((int64_t)n_units * lanes + 255) / 256)), block(256);
#define ATOMA_HN(T, L, V)                                                                                          \
  hipLaunchKernelGGL((head_norm_kernel<T, T, L, V>), grid, block, 0, stream, proj, ld, slot_mapping, n_units, units, nh, \
                     nkv, hd, vd, wq, wk, eps, (T*)q_out, (T*)kcache, (T*)vcache, page_size, hd_out, vd_out)
#define ATOMA_HN_L(T, V)                    \
  do {                                      \
    if (lanes == 16) ATOMA_HN(T, 16, V);    \
    else if (lanes == 32) ATOMA_HN(T, 32, V); \
    else ATOMA_HN(T, 64, V);                \
  } while (0)
  if (dtype == kF32) { if (vec) ATOMA_HN_L(float, true); else ATOMA_HN_L(float, false); }
  else if (dtype == kBF16) { if (vec) ATOMA_HN_L(bf16_t, true); else ATOMA_HN_L(bf16_t, false); }
  else return ATOMA_ERR_DTYPE;
#undef ATOMA_HN_L
#undef ATOMA_HN
  ATOMA_LAUNCH_CHECK();
  return 0;
}
