// Recurrences whose decay differs per state row: the selective state space with a step size per channel and a decay per
// (channel, state), and gated linear attention with a data-dependent decay per key channel.  Packed variable-length
// sequences, float state per slot; one token is the decode step.  Like the scans of seq_scan.hip these walk the tokens
// of a step in order with the state in registers and stage 16 tokens at a time through LDS; here a lane owns a small
// TILE of the state (rows x columns), so that a row vector read from LDS serves several columns and a column value
// several rows: the reads, not the arithmetic, bound a scan whose lanes own one column each.
#include "seq_common.h"

using namespace lipa;

namespace {

constexpr int CT = 16;      // tokens staged per chunk

// ln(1 + e^-a) for a >= 0 as 2 atanh(e / (2 + e)), e = e^-a: the argument stays below 1/3, so eight terms of the odd series
// reach float accuracy without a table or a branch (the staging of a chunk evaluates one per element).
__device__ __forceinline__ float log1p_exp_neg(float a) {
  const float e = __builtin_amdgcn_exp2f(a * -1.4426950408889634f), s = e * __builtin_amdgcn_rcpf(2.f + e), q = s * s;
  float p = 1.f / 17.f;
  p = p * q + 1.f / 15.f;
  p = p * q + 1.f / 13.f;
  p = p * q + 1.f / 11.f;
  p = p * q + 1.f / 9.f;
  p = p * q + 1.f / 7.f;
  p = p * q + 1.f / 5.f;
  p = p * q + 1.f / 3.f;
  return 2.f * s * (p * q + 1.f);
}
__device__ __forceinline__ float softplus_fast(float x) { return fmaxf(x, 0.f) + log1p_exp_neg(fabsf(x)); }
__device__ __forceinline__ float silu_fast(float z) {
  return z * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(z * -1.4426950408889634f));
}

// Lane layout of a wave: R lanes (4, 8 or 16) share a column; they differ in lane bits 4 and 5 (the wave's rows of 16
// lanes) and, above four, in bits 0 and 1.  The other bits tell the wave's 64 / R column groups apart.
template <int R>
__device__ __forceinline__ int lane_part(int lane) {
  return (lane >> 4) | (R >= 8 ? (lane & 1) << 2 : 0) | (R >= 16 ? (lane & 2) << 2 : 0);
}
template <int R>
__device__ __forceinline__ int lane_group(int lane) {
  return R == 4 ? lane & 15 : R == 8 ? (lane & 15) >> 1 : (lane & 15) >> 2;
}
// Four values summed over a column's R lanes at once: after exchanging halves of the wave and rows of 16 lanes, row i of
// the wave holds value i (in all lanes of its group): two exchanges and an exchange of sums instead of four butterflies.
__device__ __forceinline__ float dpp_quad_add(float v, int which) {
  const int o = which == 0 ? __builtin_amdgcn_mov_dpp(__float_as_int(v), 0xB1, 0xF, 0xF, true)     // quad_perm [1, 0, 3, 2]
                           : __builtin_amdgcn_mov_dpp(__float_as_int(v), 0x4E, 0xF, 0xF, true);    // quad_perm [2, 3, 0, 1]
  return v + __int_as_float(o);
}
__device__ __forceinline__ float swap32_add(float a, float b) {       // lanes 0-31: sum of a, lanes 32-63: sum of b
  const auto r = __builtin_amdgcn_permlane32_swap(__float_as_uint(a), __float_as_uint(b), false, false);
  return __uint_as_float(r[0]) + __uint_as_float(r[1]);
}
__device__ __forceinline__ float swap16_add(float a, float b) {       // even rows: sum of a over a pair of rows, odd: of b
  const auto r = __builtin_amdgcn_permlane16_swap(__float_as_uint(a), __float_as_uint(b), false, false);
  return __uint_as_float(r[0]) + __uint_as_float(r[1]);
}
template <int R>
__device__ __forceinline__ float sum_four(float v0, float v1, float v2, float v3) {
  float v = swap16_add(swap32_add(v0, v2), swap32_add(v1, v3));
  if (R >= 8) v = dpp_quad_add(v, 0);
  if (R >= 16) v = dpp_quad_add(v, 1);
  return v;
}

// NR contiguous entries of a state row of `len`, starting at i0 (past the row's end: 0); 16-byte accesses where they fit
template <int NR>
__device__ __forceinline__ void load_state(const float* p, int i0, int len, bool on, float (&r)[NR]) {
#pragma unroll
  for (int i4 = 0; i4 < NR / 4; ++i4) {
    f32x4 v = {0.f, 0.f, 0.f, 0.f};
    const int i = i0 + 4 * i4;
    if (on && (len & 3) == 0) {
      if (i < len) v = *reinterpret_cast<const f32x4*>(p + i);
    } else if (on) {
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (i + j < len) v[j] = p[i + j];
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) r[4 * i4 + j] = v[j];
  }
}
template <int NR>
__device__ __forceinline__ void store_state(float* p, int i0, int len, const float (&r)[NR]) {
#pragma unroll
  for (int i4 = 0; i4 < NR / 4; ++i4) {
    const int i = i0 + 4 * i4;
    if ((len & 3) == 0) {
      if (i < len) *reinterpret_cast<f32x4*>(p + i) = f32x4{r[4 * i4], r[4 * i4 + 1], r[4 * i4 + 2], r[4 * i4 + 3]};
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (i + j < len) p[i + j] = r[4 * i4 + j];
    }
  }
}

// ------------------------------------------------------------------------------------------------ selective scan
// dt = softplus(dt_pre + bias);  S[c, n] <- exp(-dt_c e^{A_log[c, n]}) S[c, n] + dt_c x_c B_n;
// y_c = sum_n S[c, n] C_n + D_c x_c;  out = scale * y * silu(z).
// A lane owns NS states of CH = 2 channels; R >= N / NS lanes share those channels, a block of 256 threads owns
// NC = 256 / R * CH channels of one sequence.  dt and dt x of the chunk go through LDS, a thread keeps the x and z it
// fetched for the read-out of the same (token, channel) pairs.  Two tokens per turn: their four read-outs are summed over
// the lanes together, and the next pair's inputs are read while the current pair is computed.
constexpr int CH = 2;

template <typename T, int NS, int R>
__global__ __launch_bounds__(256) void k_selective_scan(const T* __restrict__ x, int ldx, const float* __restrict__ dtp,
                                                        const float* __restrict__ dtb, const T* __restrict__ bm, int ldb,
                                                        const T* __restrict__ cm, int ldc, const float* __restrict__ a_log,
                                                        const float* __restrict__ dskip, const T* __restrict__ z, int ldz,
                                                        float* __restrict__ S, T* __restrict__ out, int ldo, float scale,
                                                        int C, int N, SeqDesc d) {
  constexpr int NC = 256 / R * CH, PER = CT * NC / 256, NP = NS * R, PB = (CT * NP + 255) / 256;
  __shared__ __attribute__((aligned(16))) float sdt[CT * NC];
  __shared__ __attribute__((aligned(16))) float sdx[CT * NC];     // dt x
  __shared__ __attribute__((aligned(16))) float sy[CT * NC];      // the tokens' read-outs
  __shared__ __attribute__((aligned(16))) float sB[CT * NP];
  __shared__ __attribute__((aligned(16))) float sC[CT * NP];
  const int s = blockIdx.x, tid = threadIdx.x;
  const int lane = tid & 63, grp = (tid >> 6) * (64 / R) + lane_group<R>(lane), row = lane >> 4;
  const int cb = blockIdx.y * NC, c0 = cb + grp * CH, n0 = lane_part<R>(lane) * NS;
  if (d.live && !d.live[s]) return;
  const int t0 = d.seq_off[s], t1 = d.seq_off[s + 1], p0 = d.pos0[s], slot = d.slots[s];
  float Sr[CH][NS], A[CH][NS];
#pragma unroll
  for (int h = 0; h < CH; ++h) {
    const bool ok = c0 + h < C;
    const size_t ch = ok ? c0 + h : 0;
    load_state<NS>(a_log + ch * N, n0, N, ok, A[h]);
    load_state<NS>(S + ((size_t)slot * C + ch) * N, n0, N, ok && p0 > 0, Sr[h]);
#pragma unroll
    for (int i = 0; i < NS; ++i) A[h][i] = -expf(A[h][i]) * 1.4426950408889634f;    // decays as powers of two
  }
  // A chunk's inputs are fetched without branches (addresses clamped to the step's last token and the last channel, values
  // past them dropped when they are staged), so that all of a thread's loads are in flight together; a thread's channel
  // is the same for all of its tokens.
  static_assert(256 % NC == 0 && 256 % NP == 0, "a thread keeps its column");
  const int fc = cb + tid % NC, ft = tid / NC, fcc = min(fc, C - 1), br = tid % NP, bt = tid / NP, brc = min(br, N - 1);
  const float bias = dtb[fcc], skip = dskip[fcc];
  T fx[PER], fz[PER], gx[PER], gz[PER], fB[PB], fC[PB];
  float fd[PER];
  auto fetch = [&](int tb) {
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const size_t t = min(tb + ft + 256 / NC * i, t1 - 1);
      fx[i] = x[t * ldx + fcc];
      fz[i] = z[t * ldz + fcc];
      fd[i] = dtp[t * C + fcc];
    }
#pragma unroll
    for (int i = 0; i < PB; ++i) {
      const size_t t = min(tb + bt + 256 / NP * i, t1 - 1);
      fB[i] = bm[t * ldb + brc];
      fC[i] = cm[t * ldc + brc];
    }
  };
  if (t0 < t1) fetch(t0);
  for (int tb = t0; tb < t1; tb += CT) {
    const int n = min(CT, t1 - tb);
    __syncthreads();
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const float dt = softplus_fast(fd[i] + bias);
      sdt[tid + 256 * i] = dt;
      sdx[tid + 256 * i] = dt * (float)fx[i];
      gx[i] = fx[i];
      gz[i] = fz[i];
    }
#pragma unroll
    for (int i = 0; i < PB; ++i)
      if (CT * NP >= 256 || tid < CT * NP) {
        sB[tid + 256 * i] = br < N ? (float)fB[i] : 0.f;          // a padded state never leaves zero
        sC[tid + 256 * i] = br < N ? (float)fC[i] : 0.f;
      }
    __syncthreads();
    if (tb + CT < t1) fetch(tb + CT);
    struct In {
      f32x4 B[NS / 4], C[NS / 4];
      float dt[CH], dx[CH];
    };
    auto load = [&](int tt, In& in) {
#pragma unroll
      for (int i4 = 0; i4 < NS / 4; ++i4) {
        in.B[i4] = *reinterpret_cast<const f32x4*>(sB + tt * NP + n0 + 4 * i4);
        in.C[i4] = *reinterpret_cast<const f32x4*>(sC + tt * NP + n0 + 4 * i4);
      }
#pragma unroll
      for (int h = 0; h < CH; ++h) {
        in.dt[h] = sdt[tt * NC + grp * CH + h];
        in.dx[h] = sdx[tt * NC + grp * CH + h];
      }
    };
    auto step = [&](const In& in, float (&y)[CH]) {
#pragma unroll
      for (int h = 0; h < CH; ++h) {
        float p[2] = {0.f, 0.f};
#pragma unroll
        for (int i = 0; i < NS; ++i) {
          Sr[h][i] = __builtin_amdgcn_exp2f(in.dt[h] * A[h][i]) * Sr[h][i] + in.dx[h] * in.B[i >> 2][i & 3];
          p[i & 1] += Sr[h][i] * in.C[i >> 2][i & 3];
        }
        y[h] = p[0] + p[1];
      }
    };
    In a0, a1;
    float ya[CH], yb[CH] = {0.f, 0.f};
    load(0, a0);
    int tt = 0;
    for (; tt + 1 < n; tt += 2) {
      load(tt + 1, a1);
      step(a0, ya);
      load(min(tt + 2, n - 1), a0);
      step(a1, yb);
      const float v = sum_four<R>(ya[0], ya[1], yb[0], yb[1]);     // row i of the wave: token tt + i / 2, channel i % 2
      if (R == 4 || (lane & (R == 8 ? 1 : 3)) == 0) sy[(tt + (row >> 1)) * NC + grp * CH + (row & 1)] = v;
    }
    if (tt < n) {
      step(a0, ya);
      const float v = sum_four<R>(ya[0], ya[1], yb[0], yb[1]);
      if ((R == 4 || (lane & (R == 8 ? 1 : 3)) == 0) && row < 2) sy[tt * NC + grp * CH + row] = v;
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int tt = ft + 256 / NC * i;
      if (tt < n && fc < C) {
        const float v = (sy[tid + 256 * i] + skip * (float)gx[i]) * silu_fast((float)gz[i]) * scale;
        out[(size_t)(tb + tt) * ldo + fc] = (T)v;
      }
    }
  }
#pragma unroll
  for (int h = 0; h < CH; ++h)
    if (c0 + h < C) store_state<NS>(S + ((size_t)slot * C + c0 + h) * N, n0, N, Sr[h]);
}

// ------------------------------------------------------------------------------------------ gated linear attention
// a = sigmoid(z + bias)^(1 / tau) per key channel;  S <- diag(a) S + k v^T;  o = S^T (qscale q).  S [slots, H, dv, dk].
// A lane owns RR rows of CC = 4 columns; R lanes share those columns, a block of 256 threads owns NC = 256 / R * 4 columns
// of one (sequence, head).  The decays are finished in float when a chunk is staged; the next token's vectors are read
// from LDS while the current token is computed.
constexpr int CC = 4;

template <typename T, int RR, int R>
__global__ __launch_bounds__(256) void k_gla_scan(const T* __restrict__ q, int ldq, const T* __restrict__ k, int ldk,
                                                  const T* __restrict__ v, int ldv, const float* __restrict__ z,
                                                  const float* __restrict__ zb, float inv_tau, float qscale,
                                                  float* __restrict__ S, float* __restrict__ out, int H, int dk, int dv,
                                                  SeqDesc d) {
  constexpr int DKP = RR * R, NC = 256 / R * CC, PR = CT * DKP / 256 > 0 ? CT * DKP / 256 : 1, PV = CT * NC / 256;
  __shared__ __attribute__((aligned(16))) float sk[CT * DKP];
  __shared__ __attribute__((aligned(16))) float sq[CT * DKP];
  __shared__ __attribute__((aligned(16))) float sa[CT * DKP];
  __shared__ __attribute__((aligned(16))) float sv[CT * NC];
  __shared__ __attribute__((aligned(16))) float so[CT * NC];       // the tokens' read-outs
  const int s = blockIdx.x / H, hd = blockIdx.x % H, cb = blockIdx.y * NC, tid = threadIdx.x;
  if (d.live && !d.live[s]) return;
  const int lane = tid & 63, grp = (tid >> 6) * (64 / R) + lane_group<R>(lane), row = lane >> 4;
  const int c0 = cb + grp * CC, r0 = lane_part<R>(lane) * RR;
  const int t0 = d.seq_off[s], t1 = d.seq_off[s + 1], p0 = d.pos0[s], slot = d.slots[s];
  float* Sh = S + ((size_t)slot * H + hd) * dv * dk;
  float Sr[CC][RR];
#pragma unroll
  for (int c = 0; c < CC; ++c)
    load_state<RR>(Sh + (size_t)(c0 + c < dv ? c0 + c : 0) * dk, r0, dk, p0 > 0 && c0 + c < dv, Sr[c]);
  static_assert(256 % NC == 0 && 256 % DKP == 0 && CT * DKP >= 256, "a thread keeps its row and its column");
  const int fr = tid % DKP, frt = tid / DKP, frc = hd * dk + min(fr, dk - 1);
  const int fc = cb + tid % NC, fct = tid / NC, fcc = hd * dv + min(fc, dv - 1);
  const float bias = zb[frc];
  T fk[PR], fq[PR], fv[PV];
  float fz[PR];
  auto fetch = [&](int tb) {                             // without branches, as in the selective scan
#pragma unroll
    for (int i = 0; i < PR; ++i) {
      const size_t t = min(tb + frt + 256 / DKP * i, t1 - 1);
      fk[i] = k[t * ldk + frc];
      fq[i] = q[t * ldq + frc];
      fz[i] = z[t * ((size_t)H * dk) + frc];
    }
#pragma unroll
    for (int i = 0; i < PV; ++i) {
      const size_t t = min(tb + fct + 256 / NC * i, t1 - 1);
      fv[i] = v[t * ldv + fcc];
    }
  };
  if (t0 < t1) fetch(t0);
  for (int tb = t0; tb < t1; tb += CT) {
    const int n = min(CT, t1 - tb);
    __syncthreads();
#pragma unroll
    for (int i = 0; i < PR; ++i) {
      sk[tid + 256 * i] = fr < dk ? (float)fk[i] : 0.f;       // a padded row never leaves zero
      sq[tid + 256 * i] = fr < dk ? (float)fq[i] * qscale : 0.f;
      const float zt = fz[i] + bias;                           // ln sigmoid(z) = min(z, 0) - ln(1 + e^-|z|)
      sa[tid + 256 * i] = __builtin_amdgcn_exp2f((fminf(zt, 0.f) - log1p_exp_neg(fabsf(zt))) * (inv_tau * 1.4426950408889634f));
    }
#pragma unroll
    for (int i = 0; i < PV; ++i) sv[tid + 256 * i] = (float)fv[i];
    __syncthreads();
    if (tb + CT < t1) fetch(tb + CT);
    struct In {
      f32x4 k[RR / 4], a[RR / 4], q[RR / 4], v;
    };
    auto load = [&](int tt, In& in) {
#pragma unroll
      for (int i4 = 0; i4 < RR / 4; ++i4) {
        in.k[i4] = *reinterpret_cast<const f32x4*>(sk + tt * DKP + r0 + 4 * i4);
        in.a[i4] = *reinterpret_cast<const f32x4*>(sa + tt * DKP + r0 + 4 * i4);
        in.q[i4] = *reinterpret_cast<const f32x4*>(sq + tt * DKP + r0 + 4 * i4);
      }
      in.v = *reinterpret_cast<const f32x4*>(sv + tt * NC + grp * CC);
    };
    auto step = [&](int tt, const In& in) {
      float o[CC] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < RR; ++i)
#pragma unroll
        for (int c = 0; c < CC; ++c) {
          Sr[c][i] = in.a[i >> 2][i & 3] * Sr[c][i] + in.k[i >> 2][i & 3] * in.v[c];
          o[c] += Sr[c][i] * in.q[i >> 2][i & 3];
        }
      const float v = sum_four<R>(o[0], o[1], o[2], o[3]);          // row c of the wave: column c
      if (R == 4 || (lane & (R == 8 ? 1 : 3)) == 0) so[tt * NC + grp * CC + row] = v;
    };
    In a0, a1;
    load(0, a0);
    int tt = 0;
    for (; tt + 1 < n; tt += 2) {
      load(tt + 1, a1);
      step(tt, a0);
      load(min(tt + 2, n - 1), a0);
      step(tt + 1, a1);
    }
    if (tt < n) step(tt, a0);
    __syncthreads();
#pragma unroll
    for (int i = 0; i < PV; ++i) {
      const int tt = fct + 256 / NC * i;
      if (tt < n && fc < dv) out[((size_t)(tb + tt) * H + hd) * dv + fc] = so[tid + 256 * i];
    }
  }
#pragma unroll
  for (int c = 0; c < CC; ++c)
    if (c0 + c < dv) store_state<RR>(Sh + (size_t)(c0 + c) * dk, r0, dk, Sr[c]);
}

}  // namespace

int seq_selective_max_states() { return 256; }
int seq_gla_max_dk() { return 256; }

void seq_selective_scan(int code, const void* x, int ldx, const float* dtp, const float* dtb, const void* b, int ldb,
                        const void* c, int ldc, const float* a_log, const float* dskip, const void* z, int ldz, float* S,
                        void* out, int ldo, float scale, int C, int N, SeqDesc d, hipStream_t st) {
  if (d.B == 0) return;
#define SEL_LAUNCH(NS_, R_)                                                                                           \
  hipLaunchKernelGGL((k_selective_scan<T, NS_, R_>), dim3(d.B, (C + 256 / R_ * CH - 1) / (256 / R_ * CH)), dim3(256), \
                     0, st, (const T*)x, ldx, dtp, dtb, (const T*)b, ldb, (const T*)c, ldc, a_log, dskip, (const T*)z, ldz, \
                     S, (T*)out, ldo, scale, C, N, d)
  SEQ_DISPATCH_T(code, {
    if (N <= 16)
      SEL_LAUNCH(4, 4);
    else if (N <= 32)
      SEL_LAUNCH(4, 8);
    else if (N <= 64)
      SEL_LAUNCH(4, 16);
    else if (N <= 128)
      SEL_LAUNCH(8, 16);
    else
      SEL_LAUNCH(16, 16);
  });
#undef SEL_LAUNCH
  LIPA_CHECK_LAUNCH();
}

void seq_gla_scan(int code, const void* q, int ldq, const void* k, int ldk, const void* v, int ldv, const float* z,
                  const float* zb, float inv_tau, float qscale, float* S, float* out, int H, int dk, int dv, SeqDesc d,
                  hipStream_t st) {
  if (d.B == 0) return;
#define GLA_LAUNCH(RR_, R_)                                                                                              \
  hipLaunchKernelGGL((k_gla_scan<T, RR_, R_>), dim3(d.B * H, (dv + 256 / R_ * CC - 1) / (256 / R_ * CC)), dim3(256), 0, st, \
                     (const T*)q, ldq, (const T*)k, ldk, (const T*)v, ldv, z, zb, inv_tau, qscale, S, out, H, dk, dv, d)
  SEQ_DISPATCH_T(code, {
    if (dk <= 16)
      GLA_LAUNCH(4, 4);
    else if (dk <= 32)
      GLA_LAUNCH(4, 8);
    else if (dk <= 64)
      GLA_LAUNCH(4, 16);
    else if (dk <= 128)
      GLA_LAUNCH(8, 16);
    else
      GLA_LAUNCH(16, 16);
  });
#undef GLA_LAUNCH
  LIPA_CHECK_LAUNCH();
}
