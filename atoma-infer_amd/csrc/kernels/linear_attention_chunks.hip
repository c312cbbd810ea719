// Linear attention with a decaying state (linear_attention.h) for entries of many tokens: chunks of 64 tokens on the matrix cores, all chunks of all entries side by side.  With B_i the
// product of the decays of a chunk's tokens up to i (per channel), S0 the state before the chunk and n its tokens,
//
//   o_i = S0^T (B_i q_i) + sum_(j <= i) P_ij v_j,   P_ij = sum_c q_ic k_jc prod_(j < m <= i) alpha_mc,
//   S_n = diag(B_n) S0 + U,                         U = sum_j (prod_(j < m < n) alpha_m k_j) v_j^T.
//
// Every factor is a product of decays, never an inverse of one, so decays of any strength neither overflow nor lose
// digits: P of two tokens in the same 16 is summed channel by channel with the running product, P of tokens in different
// 16s splits at the boundary between them (what decays q from the start of its 16, what decays k to the end of its own,
// and the whole 16s between).
//   la_prepare   a workgroup a (chunk, head): P, B q, B_n and U of the chunk, none of which needs the state;
//   la_pass      elementwise over the state, chunk after chunk: keeps every chunk's S0, writes the last state;
//   la_finish    a workgroup a (chunk, head): o of the chunk from S0, P and v, then norm and gate.
// Operands of the matrix instructions (v_mfma_f32_16x16x32_bf16) that are float32 by nature, all of them here, are split
// into two bfloat16 terms hi + lo (16 bits of mantissa), products take hi hi + hi lo + lo hi, sums are float32; the
// low-rank product of the decays runs on v_mfma_f32_16x16x4_f32, in float32 throughout.
// The instruction as used here: D[m][n] += sum_k A[m][k] B[n][k]; a lane hands in A[m = lane % 16][8 values of k from
// (lane / 16) * 8] and B[n = lane % 16][the same k], and holds D[m = (lane / 16) * 4 + r][n = lane % 16].
// Compiled per padded key size: ATOMA_LA_DP, dim rounded up to a multiple of 32.
#include "linear_attention.h"

using namespace atoma;

#ifndef ATOMA_LA_DP
#define ATOMA_LA_DP 64
#endif
static_assert(ATOMA_LA_DP % 32 == 0 && ATOMA_LA_DP >= 32 && ATOMA_LA_DP <= 256, "padded key sizes 32 to 256");

typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 bf16x8;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float f32x4;

constexpr int kChunk = 64, kPad = 8, kTS = kChunk + kPad, kPElems = kChunk * kChunk;

__device__ __forceinline__ uint16_t hi_of(float x) { return __builtin_bit_cast(uint16_t, static_cast<__bf16>(x)); }
__device__ __forceinline__ uint16_t lo_of(float x, uint16_t hi) { return hi_of(x - bf16_bits_to_f32(hi)); }
__device__ __forceinline__ bf16x8 frag(const uint16_t* p) { return *reinterpret_cast<const bf16x8*>(p); }
__device__ __forceinline__ uint32_t pair(uint16_t a, uint16_t b) { return a | ((uint32_t)b << 16); }
__device__ __forceinline__ float pow_int(float l2, int n) { return n == 0 ? 1.0f : __builtin_amdgcn_exp2f(l2 * (float)n); }

// acc += A B with both operands in two terms
__device__ __forceinline__ f32x4 mfma3(bf16x8 ah, bf16x8 al, bf16x8 bh, bf16x8 bl, f32x4 acc) {
  acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(al, bh, acc, 0, 0, 0);
  acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ah, bl, acc, 0, 0, 0);
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(ah, bh, acc, 0, 0, 0);
}

// a fragment (hi, lo) times a float per value, split again
__device__ __forceinline__ void scale_frag(bf16x8& fh, bf16x8& fl, const float* f) {
#pragma unroll
  for (int x = 0; x < 8; ++x) {
    const float v = ((float)fh[x] + (float)fl[x]) * f[x];
    const __bf16 h = (__bf16)v;
    fh[x] = h;
    fl[x] = (__bf16)(v - (float)h);
  }
}

// 8 values as two pieces of rows of bfloat16 terms
__device__ __forceinline__ void store8(uint16_t* hi, uint16_t* lo, const float* v) {
  uint16_t h[8], l[8];
#pragma unroll
  for (int x = 0; x < 8; ++x) h[x] = hi_of(v[x]), l[x] = lo_of(v[x], h[x]);
  *reinterpret_cast<uint4*>(hi) = make_uint4(pair(h[0], h[1]), pair(h[2], h[3]), pair(h[4], h[5]), pair(h[6], h[7]));
  *reinterpret_cast<uint4*>(lo) = make_uint4(pair(l[0], l[1]), pair(l[2], l[3]), pair(l[4], l[5]), pair(l[6], l[7]));
}

// four values of a row of P as two terms: P is [2][64][64] per (chunk, head)
__device__ __forceinline__ void store_p4(uint16_t* p, int i, int j, const float* v) {
  uint16_t h[4], l[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) h[r] = hi_of(v[r]), l[r] = lo_of(v[r], h[r]);
  *reinterpret_cast<uint2*>(p + i * kChunk + j) = make_uint2(pair(h[0], h[1]), pair(h[2], h[3]));
  *reinterpret_cast<uint2*>(p + kPElems + i * kChunk + j) = make_uint2(pair(l[0], l[1]), pair(l[2], l[3]));
}

// What the chunked kernels hand each other, per (chunk, head) = chunk * heads + head.
struct ChunkBuffers {
  uint16_t* p;      // [2][64][64]
  uint16_t* q;      // [2][64][DP]: B q
  float* d;         // [DP]: B_n
  float* u;         // [VP][DP]
  uint16_t* s;      // [2][VP][DP]: S0 transposed
};
// chunks: [n][4] = (entry, first token, tokens, 0)

template <int DP>
constexpr int prepare_words() {      // LDS of la_prepare in floats, without the chunk's products T [4][DP]
  constexpr int a = 2 * kChunk * (DP + 4);                     // decays and q
  constexpr int b = 4 * kChunk * (DP + kPad) / 2;              // q and k in two terms
  constexpr int c = (2 * DP * kTS + 2 * 128 * kTS) / 2;        // k transposed and 128 columns of v transposed, in two terms
  return a > b ? (a > c ? a : c) : (b > c ? b : c);
}

constexpr int kPrepThreads = 512;

// P of the keys j = 4 m + kg, m = M0 and M1, of the wave's 16 tokens against the later ones of the same 16: 16 lanes share
// the channels (pairs c = 2 r16 + 32 i), a key's product with the decays since runs along in registers.
template <int DP, int M0, int M1>
__device__ __forceinline__ void scores_within(const float* A, const float* Q, const float (*key)[DP / 32][2], int r16, int kg,
                                              int row0, uint16_t* P) {
  constexpr int CI = DP / 32;
  float wk[2][CI][2], pd[2] = {0.f, 0.f};
#pragma unroll
  for (int y = 0; y < 2; ++y)
#pragma unroll
    for (int i = 0; i < CI; ++i) wk[y][i][0] = key[y][i][0], wk[y][i][1] = key[y][i][1];
#pragma unroll
  for (int i = 0; i < 16; ++i) {
    float2 al[CI], q2[CI];
#pragma unroll
    for (int c = 0; c < CI; ++c) {
      al[c] = *reinterpret_cast<const float2*>(A + (row0 + i) * (DP + 4) + 2 * r16 + 32 * c);
      q2[c] = *reinterpret_cast<const float2*>(Q + (row0 + i) * (DP + 4) + 2 * r16 + 32 * c);
    }
#pragma unroll
    for (int y = 0; y < 2; ++y) {
      const int m = y ? M1 : M0;
      if (4 * m > i) continue;
      const bool past = 4 * m + 3 < i || 4 * m + kg < i;      // the key lies before token i: its product goes on
      float dot = 0.f;
#pragma unroll
      for (int c = 0; c < CI; ++c) {
        wk[y][c][0] *= past ? al[c].x : 1.0f;
        wk[y][c][1] *= past ? al[c].y : 1.0f;
        dot = fmaf(wk[y][c][0], q2[c].x, dot);
        dot = fmaf(wk[y][c][1], q2[c].y, dot);
      }
      dot = row16_sum(dot);
      if (r16 == i && 4 * m + kg <= i) pd[y] = dot;
    }
  }
#pragma unroll
  for (int y = 0; y < 2; ++y) {
    const uint16_t hh = hi_of(pd[y]);
    uint16_t* dst = P + (row0 + r16) * kChunk + row0 + 4 * (y ? M1 : M0) + kg;
    dst[0] = hh;
    dst[kPElems] = lo_of(pd[y], hh);
  }
}

template <int DP, bool GATED>
__global__ void __launch_bounds__(kPrepThreads, DP <= 128 ? 4 : 2)
la_prepare_kernel(LinearAttention a, const int32_t* __restrict__ chunks, ChunkBuffers buf, int vp) {
  extern __shared__ float lds[];
  constexpr int QS = DP + kPad;                  // row stride of q and k in LDS, in elements
  constexpr int NT = kPrepThreads;
  constexpr int NP = (4 * DP + NT - 1) / NT;     // items of 16 values of q and k a thread
  constexpr int CT = DP / 16, CI = DP / 32;
  float* T = lds + prepare_words<DP>();          // [4][DP]: the product of the decays of each 16 tokens
  const int h = blockIdx.x, ck = blockIdx.y, tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  const int r16 = lane & 15, kg = lane >> 4, wq = w & 3, wh = w >> 2;
  const int tk = chunks[4 * ck + 1], n = chunks[4 * ck + 2];
  const size_t idx0 = (size_t)ck * a.heads + h;
  uint16_t* P = buf.p + idx0 * 2 * kPElems;
  const float* proj = a.proj + (size_t)tk * a.ld;      // token j of the chunk: proj + j * ld
  const int hd = h * a.dim;
  const float zero4[4] = {0.f, 0.f, 0.f, 0.f};
  // P above the diagonal of the blocks of 32 tokens that la_finish takes whole
  if (w < 2) store_p4(P, 32 * w + r16, 32 * w + 16 + 4 * kg, zero4);

  // A thread's items: gated, 16 tokens of one channel; fixed, 8 tokens of the two channels of a pair (those that are
  // rotated together, or two neighbours behind the rotated ones).  Value x of an item: token tok(x), channel col(x).
  const int half = a.rot >> 1;
  auto c0_of = [&](int p) { const int item = tid + NT * p;
                            if (GATED) return item % DP;
                            const int i = item % (DP / 2);
                            return i < half ? i : 2 * i; };
  auto b_of = [&](int p) { const int item = tid + NT * p; return GATED ? item / DP : item / (DP / 2); };
  auto live_item = [&](int p) { return b_of(p) < (GATED ? 4 : 8); };
  auto col = [&](int p, int x) { return GATED || x < 8 ? c0_of(p) : c0_of(p) + (c0_of(p) < half ? half : 1); };
  auto tok = [&](int p, int x) { return GATED ? 16 * b_of(p) + x : 8 * b_of(p) + (x & 7); };
  float qv[NP][16], kv[NP][16];
#pragma unroll
  for (int p = 0; p < NP; ++p) {
    if (!live_item(p)) continue;
#pragma unroll
    for (int x = 0; x < 16; ++x) {
      const int t = tok(p, x), c = col(p, x);
      const bool in = t < n && c < a.dim;
      const float* row = proj + (size_t)t * a.ld + hd + c;
      qv[p][x] = in ? row[a.off_q] : 0.f;
      kv[p][x] = in ? row[a.off_k] : 0.f;
    }
  }
  float dec = 1.0f, l2 = 0.f;
  if constexpr (GATED) {
    constexpr int AS = DP + 4;                    // (rows four apart fall into different banks)
    float* A = lds;                               // [64][AS] decays
    float* Q = lds + kChunk * AS;                 // [64][AS]
    float key[2][CI][2];                          // the wave's keys of scores_within
#pragma unroll
    for (int y = 0; y < 2; ++y) {
      const int j = 16 * wq + 4 * (y ? 3 - wh : wh) + kg;      // m = 0, 3 or 1, 2: equal work
#pragma unroll
      for (int i = 0; i < CI; ++i)
#pragma unroll
        for (int x = 0; x < 2; ++x) {
          const int c = 2 * r16 + 32 * i + x;
          key[y][i][x] = (j < n && c < a.dim) ? proj[(size_t)j * a.ld + a.off_k + hd + c] * a.k_scale : 0.f;
        }
    }
    // decays: z = low w2^T + b, 16 tokens against half of the channels
    {
      const int j = 16 * wq + r16, jc = j < n ? j : n - 1;
      f32x4 acc[CT / 2];
#pragma unroll
      for (int ct = 0; ct < CT / 2; ++ct) acc[ct] = f32x4{0.f, 0.f, 0.f, 0.f};
      constexpr int KU = CT <= 8 ? 2 : 1;      // steps of 4 low-rank values whose operands are asked for together
      for (int k0 = 0; k0 < a.rank; k0 += 4 * KU) {
        float lv[KU], wv[KU][CT / 2];
#pragma unroll
        for (int u = 0; u < KU; ++u) {
          const int k = k0 + 4 * u + kg;
          lv[u] = k < a.rank ? proj[(size_t)jc * a.ld + a.off_low + k] : 0.f;
#pragma unroll
          for (int ct = 0; ct < CT / 2; ++ct) {
            const int c = (wh * (CT / 2) + ct) * 16 + r16;
            wv[u][ct] = (k < a.rank && c < a.dim) ? a.w2[(hd + c) * a.rank + k] : 0.f;
          }
        }
#pragma unroll
        for (int u = 0; u < KU; ++u)
#pragma unroll
          for (int ct = 0; ct < CT / 2; ++ct) acc[ct] = __builtin_amdgcn_mfma_f32_16x16x4f32(lv[u], wv[u][ct], acc[ct], 0, 0, 0);
      }
#pragma unroll
      for (int ct = 0; ct < CT / 2; ++ct) {
        const int c = (wh * (CT / 2) + ct) * 16 + r16;
        const float b = c < a.dim ? a.b2[hd + c] : 0.f;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int t = 16 * wq + 4 * kg + r;
          A[t * AS + c] = (t < n && c < a.dim) ? gated_decay(acc[ct][r] + b, a.inv_tau) : 1.0f;
        }
      }
    }
#pragma unroll
    for (int p = 0; p < NP; ++p) {
      if (!live_item(p)) continue;
#pragma unroll
      for (int x = 0; x < 16; ++x) {
        qv[p][x] *= a.q_scale;
        kv[p][x] *= a.k_scale;
        Q[tok(p, x) * AS + col(p, x)] = qv[p][x];
      }
    }
    __syncthreads();
    if (wh == 0) scores_within<DP, 0, 3>(A, Q, key, r16, kg, 16 * wq, P);
    else scores_within<DP, 1, 2>(A, Q, key, r16, kg, 16 * wq, P);
    // q decayed from the start of its 16, k decayed to the end of its own
#pragma unroll
    for (int p = 0; p < NP; ++p) {
      if (!live_item(p)) continue;
      const int c = c0_of(p), b = b_of(p);
      float al[16], run = 1.0f;
#pragma unroll
      for (int x = 0; x < 16; ++x) {
        al[x] = A[(16 * b + x) * AS + c];
        run *= al[x];
        qv[p][x] *= run;
      }
      T[b * DP + c] = run;
      run = 1.0f;
#pragma unroll
      for (int x = 15; x >= 0; --x) {
        kv[p][x] *= run;
        run *= al[x];
      }
    }
    __syncthreads();      // decays and q in LDS have been read; T is complete
  } else {
    dec = a.decay[h], l2 = log2f(dec);
#pragma unroll
    for (int p = 0; p < NP; ++p) {
      if (!live_item(p)) continue;
      const int i = c0_of(p);
#pragma unroll
      for (int x = 0; x < 8; ++x) {
        float cs = 1.0f, sn = 0.f;
        if (i < half && tok(p, x) < n) {
          const float* ang = a.angles + (size_t)(tk + tok(p, x)) * a.rot;
          cs = ang[i], sn = ang[half + i];
        }
        const float q0 = qv[p][x], q1 = qv[p][x + 8], k0 = kv[p][x], k1 = kv[p][x + 8];
        qv[p][x] = (q0 * cs - q1 * sn) * a.q_scale, qv[p][x + 8] = (q1 * cs + q0 * sn) * a.q_scale;
        kv[p][x] = (k0 * cs - k1 * sn) * a.k_scale, kv[p][x + 8] = (k1 * cs + k0 * sn) * a.k_scale;
      }
    }
  }

  uint16_t* qh = (uint16_t*)lds;                  // [64][QS]
  uint16_t* ql = qh + kChunk * QS;
  uint16_t* kh = ql + kChunk * QS;
  uint16_t* kl = kh + kChunk * QS;
#pragma unroll
  for (int p = 0; p < NP; ++p) {
    if (!live_item(p)) continue;
#pragma unroll
    for (int x = 0; x < 16; ++x) {
      const int at = tok(p, x) * QS + col(p, x);
      const uint16_t q0 = hi_of(qv[p][x]), k0 = hi_of(kv[p][x]);
      qh[at] = q0, ql[at] = lo_of(qv[p][x], q0);
      kh[at] = k0, kl[at] = lo_of(kv[p][x], k0);
    }
    // k decayed on to the chunk's end
    if constexpr (GATED) {
      const int c = c0_of(p), b = b_of(p);
      float f = 1.0f, whole = 1.0f;
#pragma unroll
      for (int y = 0; y < 4; ++y) {
        const float t = T[y * DP + c];
        f *= y > b ? t : 1.0f;
        whole *= t;
      }
      if (b == 3) buf.d[idx0 * DP + c] = whole;
#pragma unroll
      for (int x = 0; x < 16; ++x) kv[p][x] *= f;
    } else {
#pragma unroll
      for (int x = 0; x < 8; ++x) {
        const float f = tok(p, x) < n ? pow_int(l2, n - 1 - tok(p, x)) : 0.f;
        kv[p][x] *= f, kv[p][x + 8] *= f;
      }
      if (b_of(p) == 0) buf.d[idx0 * DP + col(p, 0)] = buf.d[idx0 * DP + col(p, 8)] = pow_int(l2, n);
    }
  }
  // v of the first columns is on its way while the scores are made
  float vv[16];
  auto ask_v = [&](int v0) {
    const int v = v0 + (tid & 127);
#pragma unroll
    for (int x = 0; x < 16; ++x) {
      const int t = 16 * (tid >> 7) + x;
      vv[x] = (t < n && v < a.vdim) ? proj[(size_t)t * a.ld + a.off_v + h * a.vdim + v] : 0.f;
    }
  };
  ask_v(0);
  __syncthreads();

  // P between different 16s (gated), or all of P on and below the diagonal (fixed): D[j][i] with A = k, B = q
  for (int job = w; job < (GATED ? 6 : 10); job += 8) {
    int I, J;
    if constexpr (GATED) {
      I = job == 0 ? 3 : job == 1 ? 2 : job == 2 ? 3 : job == 3 ? 1 : job == 4 ? 2 : 3;
      J = job == 0 ? 0 : job == 1 ? 0 : job == 2 ? 1 : job == 3 ? 0 : job == 4 ? 1 : 2;
    } else {
      I = job < 4 ? 3 : job < 7 ? 2 : job < 9 ? 1 : 0;
      J = job < 4 ? job : job < 7 ? job - 4 : job < 9 ? job - 7 : 0;
    }
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < DP / 32; ++ks) {
      const int at = ks * 32 + kg * 8;
      bf16x8 bh = frag(qh + (16 * I + r16) * QS + at), bl = frag(ql + (16 * I + r16) * QS + at);
      if (GATED && I - J > 1) {      // the whole 16s between the two
        float f[8];
#pragma unroll
        for (int x = 0; x < 8; ++x) f[x] = T[(J + 1) * DP + at + x] * (I - J > 2 ? T[(J + 2) * DP + at + x] : 1.0f);
        scale_frag(bh, bl, f);
      }
      acc = mfma3(frag(kh + (16 * J + r16) * QS + at), frag(kl + (16 * J + r16) * QS + at), bh, bl, acc);
    }
    const int i = 16 * I + r16, j0 = 16 * J + 4 * kg;
    float pv[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) pv[r] = GATED ? acc[r] : (j0 + r <= i ? acc[r] * pow_int(l2, i - j0 - r) : 0.f);
    store_p4(P, i, j0, pv);
  }
  // B q for la_finish, 8 channels at a time: what is in LDS, decayed from the chunk's start
  uint16_t* qg = buf.q + idx0 * 2 * kChunk * DP;
  for (int idx = tid; idx < kChunk * DP / 8; idx += NT) {
    const int t = idx / (DP / 8), c = idx % (DP / 8) * 8;
    bf16x8 fh = frag(qh + t * QS + c), fl = frag(ql + t * QS + c);
    if (!GATED || t >= 16) {
      float f[8];
      if constexpr (GATED) {
#pragma unroll
        for (int x = 0; x < 8; ++x)
          f[x] = T[c + x] * (t >= 32 ? T[DP + c + x] : 1.0f) * (t >= 48 ? T[2 * DP + c + x] : 1.0f);
      } else {
        const float g = pow_int(l2, t + 1);
#pragma unroll
        for (int x = 0; x < 8; ++x) f[x] = g;
      }
      scale_frag(fh, fl, f);
    }
    *reinterpret_cast<bf16x8*>(qg + t * DP + c) = fh;
    *reinterpret_cast<bf16x8*>(qg + kChunk * DP + t * DP + c) = fl;
  }
  __syncthreads();      // q and k in LDS have been read

  // U: k decayed to the chunk's end, transposed, against v, 128 columns of it at a time
  uint16_t* kth = (uint16_t*)lds;                 // [DP][kTS]
  uint16_t* ktl = kth + DP * kTS;
  uint16_t* vth = ktl + DP * kTS;                 // [128][kTS]
  uint16_t* vtl = vth + 128 * kTS;
#pragma unroll
  for (int p = 0; p < NP; ++p) {
    if (!live_item(p)) continue;
    const int t = tok(p, 0);
    store8(kth + col(p, 0) * kTS + t, ktl + col(p, 0) * kTS + t, kv[p]);
    if constexpr (GATED) store8(kth + col(p, 0) * kTS + t + 8, ktl + col(p, 0) * kTS + t + 8, kv[p] + 8);
    else store8(kth + col(p, 8) * kTS + t, ktl + col(p, 8) * kTS + t, kv[p] + 8);
  }
  float* U = buf.u + idx0 * (size_t)vp * DP;
  for (int v0 = 0; v0 < vp; v0 += 128) {
    if (v0) __syncthreads();
    {
      const int at = (tid & 127) * kTS + 16 * (tid >> 7);
      store8(vth + at, vtl + at, vv);
      store8(vth + at + 8, vtl + at + 8, vv + 8);
    }
    __syncthreads();
    if (v0 + 128 < vp) ask_v(v0 + 128);
    const int vt = v0 + 16 * w;
    if (vt < vp) {
      bf16x8 bh[2], bl[2];
#pragma unroll
      for (int s = 0; s < 2; ++s)
        bh[s] = frag(vth + (16 * w + r16) * kTS + s * 32 + kg * 8), bl[s] = frag(vtl + (16 * w + r16) * kTS + s * 32 + kg * 8);
#pragma unroll
      for (int ct = 0; ct < CT; ++ct) {
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < 2; ++s)
          acc = mfma3(frag(kth + (ct * 16 + r16) * kTS + s * 32 + kg * 8), frag(ktl + (ct * 16 + r16) * kTS + s * 32 + kg * 8),
                      bh[s], bl[s], acc);
        *reinterpret_cast<f32x4*>(U + (size_t)(vt + r16) * DP + ct * 16 + 4 * kg) = acc;
      }
    }
  }
}

// A thread owns four neighbouring channels of one column of a head's state and walks the entry's chunks.
// entries: [n][4] = (entry, first chunk, chunks, 0)
__global__ void __launch_bounds__(256)
la_pass_kernel(LinearAttention a, const int32_t* __restrict__ entries, ChunkBuffers buf, int vp, int dp) {
  constexpr int AHEAD = 8;
  const int le = blockIdx.y;
  const int e = entries[4 * le], c0 = entries[4 * le + 1], nc = entries[4 * le + 2];
  const size_t per_head = (size_t)vp * dp, all = per_head * a.heads;
  const size_t at = ((size_t)blockIdx.x * 256 + threadIdx.x) * 4;
  if (at >= all) return;
  const int h = (int)(at / per_head), v = (int)(at % per_head) / dp, c = (int)(at % dp);
  float* srow = a.state + (((size_t)a.state_slots[e] * a.heads + h) * a.vdim + v) * (size_t)a.dim + c;
  float s[4];
#pragma unroll
  for (int x = 0; x < 4; ++x) s[x] = (v < a.vdim && c + x < a.dim) ? srow[x] : 0.f;
  const float* u = buf.u + (size_t)c0 * all + at;
  const float* d = buf.d + ((size_t)c0 * a.heads + h) * dp + c;
  uint16_t* sh = buf.s + 2 * (size_t)c0 * all + (size_t)h * 2 * per_head + (at - h * per_head);
  for (int k0 = 0; k0 < nc; k0 += AHEAD) {
    float4 uu[AHEAD], dd[AHEAD];
#pragma unroll
    for (int k = 0; k < AHEAD; ++k) {
      const int kk = k0 + k < nc ? k0 + k : nc - 1;
      uu[k] = *reinterpret_cast<const float4*>(u + (size_t)kk * all);
      dd[k] = *reinterpret_cast<const float4*>(d + (size_t)kk * a.heads * dp);
    }
#pragma unroll
    for (int k = 0; k < AHEAD; ++k) {
      if (k0 + k >= nc) break;
      uint16_t hh[4], ll[4];
#pragma unroll
      for (int x = 0; x < 4; ++x) hh[x] = hi_of(s[x]), ll[x] = lo_of(s[x], hh[x]);
      uint16_t* dst = sh + 2 * (size_t)(k0 + k) * all;
      *reinterpret_cast<uint2*>(dst) = make_uint2(pair(hh[0], hh[1]), pair(hh[2], hh[3]));
      *reinterpret_cast<uint2*>(dst + per_head) = make_uint2(pair(ll[0], ll[1]), pair(ll[2], ll[3]));
      s[0] = fmaf(dd[k].x, s[0], uu[k].x), s[1] = fmaf(dd[k].y, s[1], uu[k].y);
      s[2] = fmaf(dd[k].z, s[2], uu[k].z), s[3] = fmaf(dd[k].w, s[3], uu[k].w);
    }
  }
  if (v < a.vdim) {
#pragma unroll
    for (int x = 0; x < 4; ++x)
      if (c + x < a.dim) srow[x] = s[x];
  }
}

// VT: tiles of 16 columns a wave owns (tile w + 4 x), against all 64 tokens of the chunk
template <int DP, int VT>
__global__ void __launch_bounds__(256)
la_finish_kernel(LinearAttention a, const int32_t* __restrict__ chunks, ChunkBuffers buf, int vp,
                 uint16_t* __restrict__ y) {
  extern __shared__ float lds[];
  constexpr int QS = DP + kPad;
  uint16_t* qh = (uint16_t*)lds;                  // [64][QS]
  uint16_t* ql = qh + kChunk * QS;
  uint16_t* ph = ql + kChunk * QS;                // [64][kTS]
  uint16_t* pl = ph + kChunk * kTS;
  __shared__ float sums[4][kChunk];
  const int h = blockIdx.x, ck = blockIdx.y, tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  const int r16 = lane & 15, kg = lane >> 4;
  const int tk = chunks[4 * ck + 1], n = chunks[4 * ck + 2];
  const size_t idx0 = (size_t)ck * a.heads + h;
  const uint16_t* qg = buf.q + idx0 * 2 * kChunk * DP;
  const uint16_t* P = buf.p + idx0 * 2 * kPElems;
  const uint16_t* S = buf.s + idx0 * 2 * (size_t)vp * DP;
  const float* proj = a.proj + (size_t)tk * a.ld;
  for (int idx = tid; idx < kChunk * DP / 8; idx += 256) {
    const int t = idx / (DP / 8), c = idx % (DP / 8) * 8;
    *reinterpret_cast<uint4*>(qh + t * QS + c) = *reinterpret_cast<const uint4*>(qg + t * DP + c);
    *reinterpret_cast<uint4*>(ql + t * QS + c) = *reinterpret_cast<const uint4*>(qg + kChunk * DP + t * DP + c);
  }
  // (a block of P above the diagonal that is not read was not written either: rows 0 .. 31 end at column 32)
  for (int idx = tid; idx < kPElems / 8; idx += 256) {
    const int t = idx / 8, j = idx % 8 * 8;
    if (t < 32 && j >= 32) continue;
    *reinterpret_cast<uint4*>(ph + t * kTS + j) = *reinterpret_cast<const uint4*>(P + t * kChunk + j);
    *reinterpret_cast<uint4*>(pl + t * kTS + j) = *reinterpret_cast<const uint4*>(P + kPElems + t * kChunk + j);
  }
  f32x4 acc[VT][4];
#pragma unroll
  for (int x = 0; x < VT; ++x)
#pragma unroll
    for (int it = 0; it < 4; ++it) acc[x][it] = f32x4{0.f, 0.f, 0.f, 0.f};
  // v of the wave's columns, in two terms: a lane takes 8 tokens of one column
  bf16x8 vh[VT][2], vl[VT][2];
#pragma unroll
  for (int x = 0; x < VT; ++x) {
    const int v = (w + 4 * x) * 16 + r16;
#pragma unroll
    for (int s = 0; s < 2; ++s)
#pragma unroll
      for (int y8 = 0; y8 < 8; ++y8) {
        const int t = s * 32 + kg * 8 + y8;
        const float f = (t < n && v < a.vdim) ? proj[(size_t)t * a.ld + a.off_v + h * a.vdim + v] : 0.f;
        const __bf16 hb = (__bf16)f;
        vh[x][s][y8] = hb;
        vl[x][s][y8] = (__bf16)(f - (float)hb);
      }
  }
  // the state's first fragments are on their way before the tiles above have arrived
  bf16x8 sh[2][VT], sl[2][VT];
  auto ask_s = [&](int ks) {
#pragma unroll
    for (int x = 0; x < VT; ++x) {
      const int v0 = (w + 4 * x) * 16;
      const uint16_t* p = S + (size_t)((v0 < vp ? v0 : 0) + r16) * DP + ks * 32 + kg * 8;
      sh[ks & 1][x] = frag(p), sl[ks & 1][x] = frag(p + (size_t)vp * DP);
    }
  };
  ask_s(0);
  __syncthreads();
  // D[v][i]: S0^T (B q), then v^T P^T
#pragma unroll
  for (int ks = 0; ks < DP / 32; ++ks) {
    const int at = ks * 32 + kg * 8;
    if (ks + 1 < DP / 32) ask_s(ks + 1);
    bf16x8 bh[4], bl[4];
#pragma unroll
    for (int it = 0; it < 4; ++it)
      bh[it] = frag(qh + (it * 16 + r16) * QS + at), bl[it] = frag(ql + (it * 16 + r16) * QS + at);
#pragma unroll
    for (int x = 0; x < VT; ++x)      // (columns beyond vdim are computed from others' state and never stored)
#pragma unroll
      for (int it = 0; it < 4; ++it) acc[x][it] = mfma3(sh[ks & 1][x], sl[ks & 1][x], bh[it], bl[it], acc[x][it]);
  }
#pragma unroll
  for (int s = 0; s < 2; ++s)
#pragma unroll
    for (int it = 2 * s; it < 4; ++it) {
      const bf16x8 bh = frag(ph + (it * 16 + r16) * kTS + s * 32 + kg * 8), bl = frag(pl + (it * 16 + r16) * kTS + s * 32 + kg * 8);
#pragma unroll
      for (int x = 0; x < VT; ++x) acc[x][it] = mfma3(vh[x][s], vl[x][s], bh, bl, acc[x][it]);
    }
  // norm over a token's columns: over the lane's rows, the lane groups, the waves
#pragma unroll
  for (int it = 0; it < 4; ++it) {
    float ss = 0.f;
#pragma unroll
    for (int x = 0; x < VT; ++x)
#pragma unroll
      for (int r = 0; r < 4; ++r) ss = (w + 4 * x) * 16 < vp ? fmaf(acc[x][it][r], acc[x][it][r], ss) : ss;
    ss += __shfl_xor(ss, 16, 64);
    ss += __shfl_xor(ss, 32, 64);
    if (kg == 0) sums[w][it * 16 + r16] = ss;
  }
  __syncthreads();
  const bool vec = (a.vdim & 3) == 0 && ((a.ld | a.off_g) & 3) == 0;
#pragma unroll
  for (int it = 0; it < 4; ++it) {
    const int i = it * 16 + r16;
    if (i >= n) continue;
    const float ss = sums[0][i] + sums[1][i] + sums[2][i] + sums[3][i];
    const float inv = 1.0f / sqrtf(ss / (float)a.vdim + a.eps);
    const float* g = proj + (size_t)i * a.ld + a.off_g + h * a.vdim;
    uint16_t* dst = y + (size_t)(tk + i) * a.heads * a.vdim + h * a.vdim;
#pragma unroll
    for (int x = 0; x < VT; ++x) {
      const int v = (w + 4 * x) * 16 + 4 * kg;
      if (v >= a.vdim) continue;
      if (vec) {
        const float4 g4 = *reinterpret_cast<const float4*>(g + v);
        const float gv[4] = {g4.x, g4.y, g4.z, g4.w};
        float o[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) o[r] = acc[x][it][r] * inv * (a.norm_w ? a.norm_w[v + r] : 1.0f) * silu(gv[r]);
        *reinterpret_cast<uint2*>(dst + v) = make_uint2(pair(hi_of(o[0]), hi_of(o[1])), pair(hi_of(o[2]), hi_of(o[3])));
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (v + r < a.vdim)
            dst[v + r] = hi_of(acc[x][it][r] * inv * (a.norm_w ? a.norm_w[v + r] : 1.0f) * silu(g[v + r]));
      }
    }
  }
}

template <int DP, int VT>
static void launch_finish(const LinearAttention& a, const int32_t* chunks, const ChunkBuffers& buf, int vp, void* y,
                          int n_chunks, hipStream_t stream) {
  const size_t lds = (size_t)(2 * kChunk * (DP + kPad) + 2 * kChunk * kTS) * sizeof(uint16_t);
  (void)hipFuncSetAttribute((const void*)la_finish_kernel<DP, VT>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
  hipLaunchKernelGGL((la_finish_kernel<DP, VT>), dim3(a.heads, n_chunks), dim3(256), lds, stream, a, chunks, buf, vp,
                     (uint16_t*)y);
}

template <int DP, bool GATED>
static void launch_prepare(const LinearAttention& a, const int32_t* chunks, const ChunkBuffers& buf, int vp, int n_chunks,
                           hipStream_t stream) {
  const size_t lds = (size_t)(prepare_words<DP>() + 4 * DP) * sizeof(float);
  (void)hipFuncSetAttribute((const void*)la_prepare_kernel<DP, GATED>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
  hipLaunchKernelGGL((la_prepare_kernel<DP, GATED>), dim3(a.heads, n_chunks), dim3(kPrepThreads), lds, stream, a, chunks, buf,
                     vp);
}

// The columns of S as these kernels pad them, and the most they take.
extern "C" int atoma_linear_attention_padded_dim() { return ATOMA_LA_DP; }
extern "C" int atoma_linear_attention_padded_vdim(int vdim) { return (vdim + 15) / 16 * 16; }

// chunks [n_chunks][4] = (entry, first token, tokens, 0), entries [n_long][4] = (entry, first chunk, chunks, 0): device
// memory.  y is bfloat16.  Workspaces per (chunk, head), DP and VP the padded sizes: wp 2 x 64 x 64 bfloat16, wq
// 2 x 64 x DP bfloat16, wd DP float32, wu VP x DP float32, ws 2 x VP x DP bfloat16.  Other arguments as for
// atoma_linear_attention_scan.
extern "C" int atoma_linear_attention_chunked(const float* proj, const int32_t* at, const float* decay, const float* w2,
                                              const float* b2, float inv_tau, const int32_t* positions, const float* freq,
                                              const float* angles, int rot, float q_scale, float k_scale, const float* norm_w, float eps,
                                              const int32_t* q_start, const int32_t* state_slots, float* state,
                                              int heads, int dim, int vdim, void* y, const int32_t* chunks,
                                              int n_chunks, const int32_t* entries, int n_long, void* wp, void* wq,
                                              float* wd, float* wu, void* ws, hipStream_t stream) {
  if (n_chunks <= 0 || n_long <= 0) return 0;
  const LinearAttention a = linear_attention_args(proj, at, decay, w2, b2, inv_tau, positions, freq, angles, rot, q_scale,
                                                  k_scale, norm_w, eps, q_start, state_slots, state, heads, dim, vdim);
  constexpr int DP = ATOMA_LA_DP;
  if (!linear_attention_ok(a) || (rot > 0 && angles == nullptr) || (dim + 31) / 32 * 32 != DP || vdim > 512 || n_chunks > 65535 || n_long > 65535)
    return ATOMA_ERR_SHAPE;
  const ChunkBuffers buf{(uint16_t*)wp, (uint16_t*)wq, wd, wu, (uint16_t*)ws};
  const int vp = atoma_linear_attention_padded_vdim(vdim);
  if (decay == nullptr) launch_prepare<DP, true>(a, chunks, buf, vp, n_chunks, stream);
  else launch_prepare<DP, false>(a, chunks, buf, vp, n_chunks, stream);
  const size_t quads = (size_t)a.heads * vp * DP / 4;
  hipLaunchKernelGGL(la_pass_kernel, dim3((unsigned)((quads + 255) / 256), n_long), dim3(256), 0, stream, a, entries, buf,
                     vp, DP);
  const int vt = (vp + 63) / 64;
  if (vt <= 1) launch_finish<DP, 1>(a, chunks, buf, vp, y, n_chunks, stream);
  else if (vt <= 2) launch_finish<DP, 2>(a, chunks, buf, vp, y, n_chunks, stream);
  else if (vt <= 4) launch_finish<DP, 4>(a, chunks, buf, vp, y, n_chunks, stream);
  else launch_finish<DP, 8>(a, chunks, buf, vp, y, n_chunks, stream);
  ATOMA_LAUNCH_CHECK();
  return 0;
}
