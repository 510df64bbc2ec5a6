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

template <int CTRL>
__device__ __forceinline__ float dpp_add_(float v) {
  return v + __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), CTRL, 0xF, 0xF, true));
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

// sum over R adjacent lanes (R <= 16, aligned): the sum ends in every lane
template <int R>
__device__ __forceinline__ float lanes_sum(float v) {
  if (R >= 2) v = dpp_add_<0xB1>(v);    // quad_perm [1, 0, 3, 2]
  if (R >= 4) v = dpp_add_<0x4E>(v);    // quad_perm [2, 3, 0, 1]
  if (R >= 8) v = dpp_add_<0x141>(v);   // row_half_mirror
  if (R >= 16) v = dpp_add_<0x140>(v);  // row_mirror
  return v;
}

// ------------------------------------------------------------------------------------------------ selective scan
// dt = softplus(dt_pre + bias);  S[c, n] <- exp(-dt_c e^{A_log[c, n]}) S[c, n] + dt_c x_c B_n;
// y_c = sum_n S[c, n] C_n + D_c x_c;  out = scale * y * silu(z).
// A lane owns NS states of CH channels; R = ceil(N / NS) lanes (a power of two <= 16) share those channels, a block of
// 256 threads owns NC = 256 / R * CH channels of one sequence.  dt and dt x of the chunk go through LDS, a thread keeps
// the x and z it fetched for the read-out of the same (token, channel) pairs.
template <typename T, int NS, int R, int CH>
__global__ __launch_bounds__(256) void k_selective_scan(const T* __restrict__ x, int ldx, const float* __restrict__ dtp,
                                                        const float* __restrict__ dtb, const T* __restrict__ bm, int ldb,
                                                        const T* __restrict__ cm, int ldc, const float* __restrict__ a_log,
                                                        const float* __restrict__ dskip, const T* __restrict__ z, int ldz,
                                                        float* __restrict__ S, T* __restrict__ out, int ldo, float scale,
                                                        int C, int N, SeqDesc d) {
  constexpr int NC = 256 / R * CH, PER = CT * NC / 256, NP = NS * R, PB = (CT * NP + 255) / 256;
  __shared__ __attribute__((aligned(16))) float sdt[CT * NC];
  __shared__ __attribute__((aligned(16))) float sdx[CT * NC];     // dt x; the tokens' read-outs replace it
  __shared__ __attribute__((aligned(16))) float sB[CT * NP];
  __shared__ __attribute__((aligned(16))) float sC[CT * NP];
  const int s = blockIdx.x, tid = threadIdx.x;
  const int rg = tid % R, grp = tid / R, cb = blockIdx.y * NC, c0 = cb + grp * CH, n0 = rg * NS;
  if (d.live && !d.live[s]) return;
  const int t0 = d.seq_off[s], t1 = d.seq_off[s + 1], p0 = d.pos0[s], slot = d.slots[s];
  float Sr[CH][NS], A[CH][NS];
#pragma unroll
  for (int h = 0; h < CH; ++h) {
    const bool ok = c0 + h < C;
    const size_t row = ok ? c0 + h : 0;
    load_state<NS>(a_log + row * N, n0, N, ok, A[h]);
    load_state<NS>(S + ((size_t)slot * C + row) * N, n0, N, ok && p0 > 0, Sr[h]);
#pragma unroll
    for (int i = 0; i < NS; ++i) A[h][i] = -expf(A[h][i]) * 1.4426950408889634f;    // decays as powers of two
  }
  float fx[PER], fz[PER], fd[PER], gx[PER], gz[PER], fB[PB], fC[PB];
  auto fetch = [&](int tb) {
    const int n = min(CT, t1 - tb);
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int e = tid + 256 * i, tt = e / NC, c = cb + e % NC;
      const bool ok = tt < n && c < C;
      fx[i] = ok ? (float)x[(size_t)(tb + tt) * ldx + c] : 0.f;
      fz[i] = ok ? (float)z[(size_t)(tb + tt) * ldz + c] : 0.f;
      fd[i] = ok ? dtp[(size_t)(tb + tt) * C + c] + dtb[c] : 0.f;
    }
#pragma unroll
    for (int i = 0; i < PB; ++i) {
      const int e = tid + 256 * i, tt = e / NP, r = e % NP;
      const bool ok = e < CT * NP && tt < n && r < N;
      fB[i] = ok ? (float)bm[(size_t)(tb + tt) * ldb + r] : 0.f;
      fC[i] = ok ? (float)cm[(size_t)(tb + tt) * ldc + r] : 0.f;
    }
  };
  if (t0 < t1) fetch(t0);
  for (int tb = t0; tb < t1; tb += CT) {
    const int n = min(CT, t1 - tb);
    __syncthreads();
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const float dt = softplusf_(fd[i]);
      sdt[tid + 256 * i] = dt;
      sdx[tid + 256 * i] = dt * fx[i];
      gx[i] = fx[i];
      gz[i] = fz[i];
    }
#pragma unroll
    for (int i = 0; i < PB; ++i)
      if (tid + 256 * i < CT * NP) {
        sB[tid + 256 * i] = fB[i];
        sC[tid + 256 * i] = fC[i];
      }
    __syncthreads();
    if (tb + CT < t1) fetch(tb + CT);
    for (int tt = 0; tt < n; ++tt) {
      float dt[CH], dx[CH], y[CH];
#pragma unroll
      for (int h = 0; h < CH; ++h) {
        dt[h] = sdt[tt * NC + grp * CH + h];
        dx[h] = sdx[tt * NC + grp * CH + h];
        y[h] = 0.f;
      }
#pragma unroll
      for (int i4 = 0; i4 < NS / 4; ++i4) {
        const f32x4 B = *reinterpret_cast<const f32x4*>(sB + tt * NP + n0 + 4 * i4);
        const f32x4 Cv = *reinterpret_cast<const f32x4*>(sC + tt * NP + n0 + 4 * i4);
#pragma unroll
        for (int h = 0; h < CH; ++h)
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            const int i = 4 * i4 + j;
            Sr[h][i] = __builtin_amdgcn_exp2f(dt[h] * A[h][i]) * Sr[h][i] + dx[h] * B[j];
            y[h] += Sr[h][i] * Cv[j];
          }
      }
#pragma unroll
      for (int h = 0; h < CH; ++h) y[h] = lanes_sum<R>(y[h]);
      // (a channel's dt x is read only by the R lanes of its group, which run in lockstep: its place takes the read-out)
      if (rg == 0)
#pragma unroll
        for (int h = 0; h < CH; ++h) sdx[tt * NC + grp * CH + h] = y[h];
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int e = tid + 256 * i, tt = e / NC, c = cb + e % NC;
      if (tt < n && c < C) {
        const float v = (sdx[e] + dskip[c] * gx[i]) * (gz[i] * sigmoidf_(gz[i])) * scale;
        out[(size_t)(tb + tt) * ldo + c] = (T)v;
      }
    }
  }
#pragma unroll
  for (int h = 0; h < CH; ++h)
    if (c0 + h < C) store_state<NS>(S + ((size_t)slot * C + c0 + h) * N, n0, N, Sr[h]);
}

// ------------------------------------------------------------------------------------------ gated linear attention
// a = sigmoid(z + bias)^(1 / tau) per key channel;  S <- diag(a) S + k v^T;  o = S^T (qscale q).  S [slots, H, dv, dk].
// A lane owns RR rows of CC = 4 columns; R lanes (a power of two <= 16) share those columns, a block of 256 threads owns
// NC = 256 / R * 4 columns of one (sequence, head).  The decays are finished in float when a chunk is staged.
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
  __shared__ __attribute__((aligned(16))) float sv[CT * NC];       // values; the tokens' read-outs replace them
  const int s = blockIdx.x / H, hd = blockIdx.x % H, cb = blockIdx.y * NC, tid = threadIdx.x;
  if (d.live && !d.live[s]) return;
  const int rg = tid % R, grp = tid / R, c0 = cb + grp * CC, r0 = rg * RR;
  const int t0 = d.seq_off[s], t1 = d.seq_off[s + 1], p0 = d.pos0[s], slot = d.slots[s];
  float* Sh = S + ((size_t)slot * H + hd) * dv * dk;
  float Sr[CC][RR];
#pragma unroll
  for (int c = 0; c < CC; ++c)
    load_state<RR>(Sh + (size_t)(c0 + c < dv ? c0 + c : 0) * dk, r0, dk, p0 > 0 && c0 + c < dv, Sr[c]);
  float fk[PR], fq[PR], fz[PR], fv[PV];
  auto fetch = [&](int tb) {
    const int n = min(CT, t1 - tb);
#pragma unroll
    for (int i = 0; i < PR; ++i) {
      const int e = tid + 256 * i, tt = e / DKP, r = e % DKP;
      const bool ok = tt < n && r < dk;
      fk[i] = ok ? (float)k[(size_t)(tb + tt) * ldk + hd * dk + r] : 0.f;
      fq[i] = ok ? (float)q[(size_t)(tb + tt) * ldq + hd * dk + r] * qscale : 0.f;
      fz[i] = ok ? z[(size_t)(tb + tt) * ((size_t)H * dk) + hd * dk + r] + zb[hd * dk + r] : 0.f;
    }
#pragma unroll
    for (int i = 0; i < PV; ++i) {
      const int e = tid + 256 * i, tt = e / NC, c = cb + e % NC;
      fv[i] = tt < n && c < dv ? (float)v[(size_t)(tb + tt) * ldv + hd * dv + c] : 0.f;
    }
  };
  if (t0 < t1) fetch(t0);
  for (int tb = t0; tb < t1; tb += CT) {
    const int n = min(CT, t1 - tb);
    __syncthreads();
#pragma unroll
    for (int i = 0; i < PR; ++i)
      if (tid + 256 * i < CT * DKP) {
        sk[tid + 256 * i] = fk[i];
        sq[tid + 256 * i] = fq[i];
        sa[tid + 256 * i] = expf(logsigmoidf_(fz[i]) * inv_tau);
      }
#pragma unroll
    for (int i = 0; i < PV; ++i) sv[tid + 256 * i] = fv[i];
    __syncthreads();
    if (tb + CT < t1) fetch(tb + CT);
    for (int tt = 0; tt < n; ++tt) {
      const f32x4 vv = *reinterpret_cast<const f32x4*>(sv + tt * NC + grp * CC);
      float o[CC] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i4 = 0; i4 < RR / 4; ++i4) {
        const f32x4 kk = *reinterpret_cast<const f32x4*>(sk + tt * DKP + r0 + 4 * i4);
        const f32x4 aa = *reinterpret_cast<const f32x4*>(sa + tt * DKP + r0 + 4 * i4);
        const f32x4 qq = *reinterpret_cast<const f32x4*>(sq + tt * DKP + r0 + 4 * i4);
#pragma unroll
        for (int c = 0; c < CC; ++c)
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            const int i = 4 * i4 + j;
            Sr[c][i] = aa[j] * Sr[c][i] + kk[j] * vv[c];
            o[c] += Sr[c][i] * qq[j];
          }
      }
#pragma unroll
      for (int c = 0; c < CC; ++c) o[c] = lanes_sum<R>(o[c]);
      // (the four values are read only by this group of lanes, which run in lockstep: their place takes the read-out)
      if (rg == 0) *reinterpret_cast<f32x4*>(sv + tt * NC + grp * CC) = f32x4{o[0], o[1], o[2], o[3]};
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < PV; ++i) {
      const int e = tid + 256 * i, tt = e / NC, c = cb + e % NC;
      if (tt < n && c < dv) out[((size_t)(tb + tt) * H + hd) * dv + c] = sv[e];
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
#define SEL_LAUNCH(NS_, R_, CH_)                                                                                           \
  hipLaunchKernelGGL((k_selective_scan<T, NS_, R_, CH_>), dim3(d.B, (C + 256 / R_ * CH_ - 1) / (256 / R_ * CH_)), dim3(256), \
                     0, st, (const T*)x, ldx, dtp, dtb, (const T*)b, ldb, (const T*)c, ldc, a_log, dskip, (const T*)z, ldz, \
                     S, (T*)out, ldo, scale, C, N, d)
  SEQ_DISPATCH_T(code, {
    if (N <= 4)
      SEL_LAUNCH(4, 1, 1);
    else if (N <= 8)
      SEL_LAUNCH(4, 2, 1);
    else if (N <= 16)
      SEL_LAUNCH(4, 4, 2);
    else if (N <= 32)
      SEL_LAUNCH(4, 8, 2);
    else if (N <= 64)
      SEL_LAUNCH(4, 16, 2);
    else if (N <= 128)
      SEL_LAUNCH(8, 16, 1);
    else
      SEL_LAUNCH(16, 16, 1);
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
