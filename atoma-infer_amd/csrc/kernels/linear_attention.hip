// Linear attention with a decaying state, token by token (the mechanism: linear_attention.h).
#include "linear_attention.h"

using namespace atoma;

constexpr int kScanThreads = 512, kScanCols = kScanThreads / 16;

// MR: groups of 64 rows of S (4 a lane); MC: groups of 32 columns; GATED: a decay per channel; FUSED: the workgroup holds
// all columns of the head and finishes the token.  tb: tokens staged in LDS at a time.  Entries of `below` tokens and more
// are left alone (below > 0): they are the chunked kernels'.
// A decoded token's time is its chain of trips to memory, so an entry of one token asks for everything it needs (its
// columns of the projection, the low-rank matrix, the state) in one go.
template <int MR, int MC, bool GATED, bool FUSED, typename TO>
__global__ void __launch_bounds__(kScanThreads, MR * MC <= 8 ? 4 : 2)
la_scan_kernel(LinearAttention a, void* __restrict__ out, int tb, int below) {
  extern __shared__ float lds[];
  constexpr int DS = MR * 64, VS = MC * kScanCols;
  float* qs = lds;                            // [tb][DS]
  float* ks = qs + tb * DS;                   // [tb][DS]
  float* as = ks + tb * DS;                   // [tb][DS] (gated)
  float* vs = as + (GATED ? tb * DS : 0);     // [tb][VS]
  float* os = vs + tb * VS;                   // [tb][VS] (fused)
  float* gs = os + (FUSED ? tb * VS : 0);     // [tb][VS] (fused): silu of the gates, times the norm's weight
  float* cs = gs + (FUSED ? tb * VS : 0);     // [tb][rot / 2]
  float* sn = cs + tb * (a.rot >> 1);
  const int e = blockIdx.y, tid = threadIdx.x;
  const int vblocks = (a.vdim + VS - 1) / VS;
  const int h = blockIdx.x / vblocks, v0 = (blockIdx.x % vblocks) * VS;
  const int t0 = a.q_start[e], t1 = a.q_start[e + 1];
  if (t1 <= t0 || (below > 0 && t1 - t0 >= below)) return;
  const int part = tid & 15, cg = tid >> 4, half = a.rot >> 1, hd = h * a.dim;
  float* srow = a.state + ((size_t)a.state_slots[e] * a.heads + h) * (size_t)a.vdim * a.dim;
  const bool vec = (a.dim & 3) == 0 && (((uintptr_t)a.state) & 15) == 0;
  float s[MC][MR][4];
  // (the state's places are worked out anew for the stores, so that they need no registers in between)
  uint32_t at0 = (uint32_t)(v0 + cg) * a.dim + 4 * part;
  auto load_state = [&]() {
#pragma unroll
    for (int m = 0; m < MC; ++m) {
      const int j = v0 + cg + kScanCols * m;
#pragma unroll
      for (int i = 0; i < MR; ++i) {
        const int r = 64 * i + 4 * part;
        const float* p = srow + (at0 + (uint32_t)(kScanCols * m) * a.dim + 64 * i);
        if (vec) {
          float4 x = make_float4(0.f, 0.f, 0.f, 0.f);
          if (j < a.vdim && r < a.dim) x = *reinterpret_cast<const float4*>(p);
          s[m][i][0] = x.x, s[m][i][1] = x.y, s[m][i][2] = x.z, s[m][i][3] = x.w;
        } else {
#pragma unroll
          for (int x = 0; x < 4; ++x) s[m][i][x] = (j < a.vdim && r + x < a.dim) ? p[x] : 0.f;
        }
      }
    }
  };
  const float dec = GATED ? 1.0f : a.decay[h];
  // four lanes a channel share the sum over the low-rank columns
  auto low_sum = [&](int t, int r, int part4) {
    float z = 0.f;
    if (r < a.dim) {
      const float* l = a.proj + (size_t)t * a.ld + a.off_low;
      const float* w = a.w2 + (size_t)(hd + r) * a.rank;
#pragma unroll 4
      for (int x = part4; x < a.rank; x += 4) z = fmaf(l[x], w[x], z);
    }
    z += __shfl_xor(z, 1, 64);
    z += __shfl_xor(z, 2, 64);
    return z;
  };
  const bool one = t1 - t0 == 1;
  if (one) {
    const float* row = a.proj + (size_t)t0 * a.ld;
    float q = 0.f, k = 0.f, q2 = 0.f, k2 = 0.f, v = 0.f, g = 0.f, nw = 1.0f, f = 0.f;
    int pos = 0;
    const bool turns = tid < a.rot;
    if (tid < a.dim) {
      q = row[a.off_q + hd + tid], k = row[a.off_k + hd + tid];
      if (turns) {
        const int o = tid < half ? tid + half : tid - half;
        q2 = row[a.off_q + hd + o], k2 = row[a.off_k + hd + o];
        f = a.freq[tid < half ? tid : o], pos = a.positions[t0];
      }
    }
    if (tid < VS && v0 + tid < a.vdim) {
      v = row[a.off_v + h * a.vdim + v0 + tid];
      if constexpr (FUSED) {
        g = row[a.off_g + h * a.vdim + tid];
        if (a.norm_w != nullptr) nw = a.norm_w[tid];
      }
    }
    constexpr int NZ = (DS * 4 + kScanThreads - 1) / kScanThreads;
    float z[NZ];
    if constexpr (GATED) {
#pragma unroll
      for (int y = 0; y < NZ; ++y) {
        const int idx = tid + y * kScanThreads, r = idx >> 2;
        const float b = r < a.dim ? a.b2[hd + r] : 0.f;
        z[y] = low_sum(t0, r, idx & 3) + b;
      }
    }
    load_state();
    if (turns) {
      float c, sv;
      sincosf((float)pos * f, &sv, &c);
      q = tid < half ? q * c - q2 * sv : q * c + q2 * sv;
      k = tid < half ? k * c - k2 * sv : k * c + k2 * sv;
    }
    if (tid < DS) qs[tid] = q * a.q_scale, ks[tid] = k * a.k_scale;
    if (tid < VS) {
      vs[tid] = v;
      if constexpr (FUSED) gs[tid] = silu(g) * nw;
    }
    if constexpr (GATED) {
#pragma unroll
      for (int y = 0; y < NZ; ++y) {
        const int idx = tid + y * kScanThreads, r = idx >> 2;
        if ((idx & 3) == 0 && r < DS) as[r] = r < a.dim ? gated_decay(z[y], a.inv_tau) : 0.f;
      }
    }
  } else {
    load_state();
  }
  for (int tk = t0; tk < t1; tk += tb) {
    const int n = t1 - tk < tb ? t1 - tk : tb;
    if (!one) {
      __syncthreads();
      if (half) {
        for (int idx = tid; idx < n * half; idx += kScanThreads) {
          const int tt = idx / half, i = idx % half;
          sincosf((float)a.positions[tk + tt] * a.freq[i], &sn[tt * half + i], &cs[tt * half + i]);
        }
        __syncthreads();
      }
#pragma unroll 1      // (registers: the state is in them)
      for (int idx = tid; idx < n * DS; idx += kScanThreads) {
        const int tt = idx / DS, r = idx % DS;
        const float* row = a.proj + (size_t)(tk + tt) * a.ld + hd;
        float q = 0.f, k = 0.f;
        if (r < a.dim) {
          q = rotated(row + a.off_q, r, a.rot, cs + tt * half, sn + tt * half) * a.q_scale;
          k = rotated(row + a.off_k, r, a.rot, cs + tt * half, sn + tt * half) * a.k_scale;
        }
        qs[idx] = q, ks[idx] = k;
      }
#pragma unroll 1
      for (int idx = tid; idx < n * VS; idx += kScanThreads) {
        const int tt = idx / VS, j = v0 + idx % VS;
        const float* row = a.proj + (size_t)(tk + tt) * a.ld + h * a.vdim + j;
        vs[idx] = j < a.vdim ? row[a.off_v] : 0.f;
        if constexpr (FUSED) gs[idx] = j < a.vdim ? silu(row[a.off_g]) * (a.norm_w ? a.norm_w[j] : 1.0f) : 0.f;
      }
      if constexpr (GATED) {
#pragma unroll 1
        for (int idx = tid; idx < n * DS * 4; idx += kScanThreads) {
          const int c = idx >> 2, tt = c / DS, r = c % DS;
          const float z = low_sum(tk + tt, r, idx & 3);
          if ((idx & 3) == 0) as[c] = r < a.dim ? gated_decay(z + a.b2[hd + r], a.inv_tau) : 0.f;
        }
      }
    }
    __syncthreads();
#pragma unroll 1
    for (int tt = 0; tt < n; ++tt) {
      float v[MC], acc[MC];
#pragma unroll
      for (int m = 0; m < MC; ++m) v[m] = vs[tt * VS + cg + kScanCols * m], acc[m] = 0.f;
#pragma unroll
      for (int i = 0; i < MR; ++i) {
        const int r = tt * DS + 64 * i + 4 * part;
        const float4 q4 = *reinterpret_cast<const float4*>(qs + r), k4 = *reinterpret_cast<const float4*>(ks + r);
        float4 a4 = make_float4(dec, dec, dec, dec);
        if constexpr (GATED) a4 = *reinterpret_cast<const float4*>(as + r);
        const float qv[4] = {q4.x, q4.y, q4.z, q4.w}, kv[4] = {k4.x, k4.y, k4.z, k4.w}, av[4] = {a4.x, a4.y, a4.z, a4.w};
#pragma unroll
        for (int m = 0; m < MC; ++m)
#pragma unroll
          for (int x = 0; x < 4; ++x) {
            s[m][i][x] = fmaf(av[x], s[m][i][x], kv[x] * v[m]);
            acc[m] = fmaf(s[m][i][x], qv[x], acc[m]);
          }
      }
#pragma unroll
      for (int m = 0; m < MC; ++m) {
        const float o = row16_sum(acc[m]);
        const int j = cg + kScanCols * m;
        if (part == 0) {
          if constexpr (FUSED) os[tt * VS + j] = o;
          else if (v0 + j < a.vdim) ((float*)out)[(size_t)(tk + tt) * a.heads * a.vdim + h * a.vdim + v0 + j] = o;
        }
      }
    }
    // the state leaves while the last tokens are finished
    if (tk + tb >= t1) {
      asm volatile("" : "+v"(at0));
#pragma unroll
      for (int m = 0; m < MC; ++m) {
        const int j = v0 + cg + kScanCols * m;
        if (j >= a.vdim) continue;
#pragma unroll
        for (int i = 0; i < MR; ++i) {
          const int r = 64 * i + 4 * part;
          float* p = srow + (at0 + (uint32_t)(kScanCols * m) * a.dim + 64 * i);
          if (vec) {
            if (r < a.dim) *reinterpret_cast<float4*>(p) = make_float4(s[m][i][0], s[m][i][1], s[m][i][2], s[m][i][3]);
          } else {
#pragma unroll
            for (int x = 0; x < 4; ++x)
              if (r + x < a.dim) p[x] = s[m][i][x];
          }
        }
      }
    }
    if constexpr (FUSED) {
      __syncthreads();
      const int lane = tid & 63;
      for (int tt = tid >> 6; tt < n; tt += kScanThreads / 64) {
        float ss = 0.f;
        for (int j = lane; j < a.vdim; j += 64) ss = fmaf(os[tt * VS + j], os[tt * VS + j], ss);
        ss = wave_sum(ss);
        const float inv = 1.0f / sqrtf(ss / (float)a.vdim + a.eps);
        TO* y = (TO*)out + (size_t)(tk + tt) * a.heads * a.vdim + h * a.vdim;
        for (int j = lane; j < a.vdim; j += 64) y[j] = from_f32<TO>(os[tt * VS + j] * inv * gs[tt * VS + j]);
      }
    }
  }
}

// out[t] = cosines, then sines of the angles positions[t] * freq[i]
__global__ void __launch_bounds__(256)
la_angles_kernel(const int32_t* __restrict__ positions, const float* __restrict__ freq, int half, float* __restrict__ out,
                 int n) {
  const int idx = blockIdx.x * 256 + threadIdx.x;
  if (idx >= n * half) return;
  const int t = idx / half, i = idx % half;
  float s, c;
  sincosf((float)positions[t] * freq[i], &s, &c);
  out[(size_t)t * 2 * half + i] = c;
  out[(size_t)t * 2 * half + half + i] = s;
}

template <typename TO>
__global__ void __launch_bounds__(256)
la_out_kernel(LinearAttention a, const float* __restrict__ o, TO* __restrict__ y, int below) {
  const int e = blockIdx.y, h = blockIdx.x, lane = threadIdx.x & 63;
  const int t0 = a.q_start[e], t1 = a.q_start[e + 1];
  if (below > 0 && t1 - t0 >= below) return;
  for (int t = t0 + (threadIdx.x >> 6); t < t1; t += 4) {
    const size_t at = (size_t)t * a.heads * a.vdim + h * a.vdim;
    float ss = 0.f;
    for (int j = lane; j < a.vdim; j += 64) ss = fmaf(o[at + j], o[at + j], ss);
    ss = wave_sum(ss);
    const float inv = 1.0f / sqrtf(ss / (float)a.vdim + a.eps);
    const float* g = a.proj + (size_t)t * a.ld + a.off_g + h * a.vdim;
    for (int j = lane; j < a.vdim; j += 64)
      y[at + j] = from_f32<TO>(o[at + j] * inv * (a.norm_w ? a.norm_w[j] : 1.0f) * silu(g[j]));
  }
}

template <int MR, int MC, bool GATED, bool FUSED, typename TO>
static int launch_scan(const LinearAttention& a, void* out, int n_entries, int tb, int below, hipStream_t stream) {
  constexpr int DS = MR * 64, VS = MC * kScanCols;
  const int per_token = (GATED ? 3 : 2) * DS + (FUSED ? 3 : 1) * VS + a.rot;
  const size_t lds = (size_t)tb * per_token * sizeof(float);
  if (lds > 32 * 1024)
    (void)hipFuncSetAttribute((const void*)la_scan_kernel<MR, MC, GATED, FUSED, TO>,
                              hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
  dim3 grid(a.heads * ((a.vdim + VS - 1) / VS), n_entries);
  hipLaunchKernelGGL((la_scan_kernel<MR, MC, GATED, FUSED, TO>), grid, dim3(kScanThreads), lds, stream, a, out, tb, below);
  ATOMA_LAUNCH_CHECK();
  return 0;
}

template <int MR, bool GATED, typename TO>
static int scan_cols(const LinearAttention& a, void* y, float* o, int n_entries, int tb, int below, hipStream_t stream) {
  if (a.vdim <= 32) return launch_scan<MR, 1, GATED, true, TO>(a, y, n_entries, tb, below, stream);
  if (a.vdim <= 64) return launch_scan<MR, 2, GATED, true, TO>(a, y, n_entries, tb, below, stream);
  if (a.vdim <= 128) return launch_scan<MR, 4, GATED, true, TO>(a, y, n_entries, tb, below, stream);
  if constexpr (MR <= 2)      // (more rows of so many columns do not fit a workgroup's registers)
    if (a.vdim <= 256) return launch_scan<MR, 8, GATED, true, TO>(a, y, n_entries, tb, below, stream);
  if (o == nullptr) return ATOMA_ERR_SHAPE;
  const int rc = launch_scan<MR, 4, GATED, false, float>(a, o, n_entries, tb, below, stream);
  if (rc) return rc;
  hipLaunchKernelGGL((la_out_kernel<TO>), dim3(a.heads, n_entries), dim3(256), 0, stream, a, o, (TO*)y, below);
  ATOMA_LAUNCH_CHECK();
  return 0;
}

template <bool GATED, typename TO>
static int scan_rows(const LinearAttention& a, void* y, float* o, int n_entries, int tb, int below, hipStream_t stream) {
  if (a.dim <= 64) return scan_cols<1, GATED, TO>(a, y, o, n_entries, tb, below, stream);
  if (a.dim <= 128) return scan_cols<2, GATED, TO>(a, y, o, n_entries, tb, below, stream);
  if (a.dim <= 192) return scan_cols<3, GATED, TO>(a, y, o, n_entries, tb, below, stream);
  return scan_cols<4, GATED, TO>(a, y, o, n_entries, tb, below, stream);
}

// whether la_scan needs the float32 buffer o [T, heads vdim] between the recurrence and the norm
extern "C" int atoma_linear_attention_needs_o(int dim, int vdim) { return vdim > 256 || (vdim > 128 && dim > 128); }

// at: ld, off_q, off_k, off_v, off_g, off_low, rank (host memory).  tb: tokens staged at a time (1 to 16).
extern "C" int atoma_linear_attention_scan(const float* proj, const int32_t* at, const float* decay, const float* w2,
                                           const float* b2, float inv_tau, const int32_t* positions, const float* freq,
                                           int rot, float q_scale, float k_scale, const float* norm_w, float eps,
                                           const int32_t* q_start, const int32_t* state_slots, float* state, int heads,
                                           int dim, int vdim, void* y, int y_dtype, float* o, int n_entries, int tb,
                                           int below, hipStream_t stream) {
  if (n_entries <= 0) return 0;
  const LinearAttention a = linear_attention_args(proj, at, decay, w2, b2, inv_tau, positions, freq, nullptr, rot, q_scale,
                                                  k_scale, norm_w, eps, q_start, state_slots, state, heads, dim, vdim);
  if (!linear_attention_ok(a) || n_entries > 65535 || tb < 1 || tb > 16 || below < 0) return ATOMA_ERR_SHAPE;
  if (y_dtype == kF32)
    return decay ? scan_rows<false, float>(a, y, o, n_entries, tb, below, stream)
                 : scan_rows<true, float>(a, y, o, n_entries, tb, below, stream);
  if (y_dtype == kBF16)
    return decay ? scan_rows<false, bf16_t>(a, y, o, n_entries, tb, below, stream)
                 : scan_rows<true, bf16_t>(a, y, o, n_entries, tb, below, stream);
  return ATOMA_ERR_DTYPE;
}

extern "C" int atoma_linear_attention_angles(const int32_t* positions, const float* freq, int half, float* out, int n_tokens,
                                             hipStream_t stream) {
  if (n_tokens <= 0 || half <= 0) return 0;
  if (half > kMaxRot / 2 || (long)n_tokens * half > 2147483000L) return ATOMA_ERR_SHAPE;
  hipLaunchKernelGGL(la_angles_kernel, dim3((unsigned)(((long)n_tokens * half + 255) / 256)), dim3(256), 0, stream, positions,
                     freq, half, out, n_tokens);
  ATOMA_LAUNCH_CHECK();
  return 0;
}
