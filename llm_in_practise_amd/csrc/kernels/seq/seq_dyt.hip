// Residual blocks whose norm is a Dynamic Tanh (element-wise: no statistics over a row) and whose sublayers read a short
// causal convolution of the normed residual.  Because nothing is reduced over the row, one kernel does a sublayer's exit
// and the next one's entry for a run of tokens: weighted residual add, average over depth, tanh, convolution over time.
#include "seq_common.h"

using namespace lipa;

namespace {

constexpr int RUN = 16;       // tokens per block; two blocks per attention tile of 32 tokens
constexpr int MAXTAPS = 8;    // convolution taps (RUN >= MAXTAPS - 1: only a sequence's first run reads carried rows)

template <int V> struct Vec { float v[V]; };

template <int V>
__device__ __forceinline__ Vec<V> ldv(const float* p) {
  Vec<V> r;
  if constexpr (V == 4) {
    const f32x4 x = *reinterpret_cast<const f32x4*>(p);
    r.v[0] = x[0]; r.v[1] = x[1]; r.v[2] = x[2]; r.v[3] = x[3];
  } else {
    r.v[0] = p[0];
  }
  return r;
}
template <int V>
__device__ __forceinline__ Vec<V> ldv(const bf16* p) {
  Vec<V> r;
  if constexpr (V == 4) {
    const bf16x4 x = *reinterpret_cast<const bf16x4*>(p);
#pragma unroll
    for (int i = 0; i < 4; ++i) r.v[i] = (float)x[i];
  } else {
    r.v[0] = (float)p[0];
  }
  return r;
}
template <int V>
__device__ __forceinline__ void stv(float* p, const Vec<V>& r) {
  if constexpr (V == 4)
    *reinterpret_cast<f32x4*>(p) = f32x4{r.v[0], r.v[1], r.v[2], r.v[3]};
  else
    p[0] = r.v[0];
}
template <int V>
__device__ __forceinline__ void stv(bf16* p, const Vec<V>& r) {
  if constexpr (V == 4)
    *reinterpret_cast<bf16x4*>(p) = bf16x4{(bf16)r.v[0], (bf16)r.v[1], (bf16)r.v[2], (bf16)r.v[3]};
  else
    p[0] = (bf16)r.v[0];
}

struct DytArgs {
  int ldy;
  float mult;
  size_t sstride;        // T * W: a stream's stride
  int n;                 // this exit's stream
  const float *w, *b;    // [W]
  float alpha;
  const float* conv;     // [taps, W] or null
  int taps;
  const float* sin;      // [slots, taps - 1, W] carried rows, read
  float* sout;           // the same, written
  int W;
  const int *tile_seq, *tile_t0;
  int run;               // tokens per block without a convolution
};

// r of token t, columns [c, c + V): x + mult y, then the average over depth (the streams before this one are read, this
// one is written to sn).  r is kept in rout unless that is null (nothing was added: r is x).
template <typename YT, int V, bool STORE>
__device__ __forceinline__ Vec<V> residual_at(const DytArgs& a, const float* __restrict__ x, const YT* __restrict__ y,
                                              const float* __restrict__ streams, const float* __restrict__ depth,
                                              float* __restrict__ sn, float* __restrict__ rout, size_t t, int c) {
  const size_t o = t * a.W + c;
  Vec<V> r = ldv<V>(x + o);
  if (y != nullptr) {
    const Vec<V> yv = ldv<V>(y + t * a.ldy + c);
#pragma unroll
    for (int i = 0; i < V; ++i) r.v[i] += a.mult * yv.v[i];
  }
  if (depth != nullptr) {
    if (STORE) stv<V>(sn + o, r);
    const float dn = depth[a.n];
#pragma unroll
    for (int i = 0; i < V; ++i) r.v[i] *= dn;
#pragma unroll 4
    for (int j = 0; j < a.n; ++j) {
      const Vec<V> s = ldv<V>(streams + (size_t)j * a.sstride + o);
      const float dj = depth[j];
#pragma unroll
      for (int i = 0; i < V; ++i) r.v[i] += dj * s.v[i];
    }
  }
  if (STORE && rout != nullptr) stv<V>(rout + o, r);
  return r;
}

// One wave per (run of RUN tokens of one sequence, 64 * V columns); a thread walks its columns through the run and keeps
// the last TP - 1 normed inputs in registers (TP: taps rounded up, missing taps have weight zero).  The TP - 1 tokens
// before the run are recomputed (x and the streams before this one are not written by this launch), before the step's
// first token they come from the slot.  The block that holds a sequence's last token carries the last rows into the slot.
template <typename T, typename YT, int V, int TP>
__global__ __launch_bounds__(64) void k_residual_dyt(DytArgs a, const float* __restrict__ x, const YT* __restrict__ y,
                                                     const float* __restrict__ streams, const float* __restrict__ depth,
                                                     float* __restrict__ sn, float* __restrict__ rout, T* __restrict__ h,
                                                     SeqDesc d) {
  const int c = (blockIdx.y * 64 + threadIdx.x) * V;
  if (c >= a.W) return;
  const Vec<V> w = ldv<V>(a.w + c), b = ldv<V>(a.b + c);
  auto normed = [&](const Vec<V>& r) {
    Vec<V> o;
#pragma unroll
    for (int i = 0; i < V; ++i) o.v[i] = tanhf(a.alpha * r.v[i]) * w.v[i] + b.v[i];
    return o;
  };
  if constexpr (TP == 1) {
    const int t0 = blockIdx.x * a.run, t1 = min(t0 + a.run, d.Ttot);
    for (int t = t0; t < t1; ++t) stv<V>(h + (size_t)t * a.W + c, normed(residual_at<YT, V, true>(a, x, y, streams, depth, sn, rout, t, c)));
  } else {
    const int tile = blockIdx.x >> 1, s = a.tile_seq[tile], s0 = d.seq_off[s], s1 = d.seq_off[s + 1];
    const int t0 = a.tile_t0[tile] + RUN * (blockIdx.x & 1), t1 = min(t0 + RUN, s1);
    if (t0 >= t1) return;
    const int slot = d.slots[s], p0 = d.pos0[s], keep = a.taps - 1;
    Vec<V> cw[TP], win[TP - 1];
#pragma unroll
    for (int j = 0; j < TP; ++j) {
      if (j >= TP - a.taps)
        cw[j] = ldv<V>(a.conv + (size_t)(j - (TP - a.taps)) * a.W + c);
      else
#pragma unroll
        for (int i = 0; i < V; ++i) cw[j].v[i] = 0.f;
    }
#pragma unroll
    for (int j = 0; j < TP - 1; ++j) {
      const int li = t0 - s0 - (TP - 1) + j;              // place in this step's tokens of the sequence
#pragma unroll
      for (int i = 0; i < V; ++i) win[j].v[i] = 0.f;
      if (j >= TP - 1 - keep) {
        if (li >= 0)
          win[j] = normed(residual_at<YT, V, false>(a, x, y, streams, depth, sn, rout, s0 + li, c));
        else if (p0 > 0)
          win[j] = ldv<V>(a.sin + ((size_t)slot * keep + keep + li) * a.W + c);
      }
    }
    for (int t = t0; t < t1; ++t) {
      const Vec<V> hv = normed(residual_at<YT, V, true>(a, x, y, streams, depth, sn, rout, t, c));
      Vec<V> o;
#pragma unroll
      for (int i = 0; i < V; ++i) {
        float v = hv.v[i] + cw[TP - 1].v[i] * hv.v[i];
#pragma unroll
        for (int j = 0; j < TP - 1; ++j) v += cw[j].v[i] * win[j].v[i];
        o.v[i] = v;
      }
      stv<V>(h + (size_t)t * a.W + c, o);
#pragma unroll
      for (int j = 0; j < TP - 2; ++j) win[j] = win[j + 1];
      win[TP - 2] = hv;
    }
    if (t1 == s1 && keep > 0 && !(d.live != nullptr && !d.live[s])) {
#pragma unroll
      for (int j = 0; j < TP - 1; ++j)
        if (j >= TP - 1 - keep) stv<V>(a.sout + ((size_t)slot * keep + j - (TP - 1 - keep)) * a.W + c, win[j]);
    }
  }
}

// cap * tanh(z / cap) in place
__global__ __launch_bounds__(256) void k_softcap(float* __restrict__ z, size_t n, float cap, float inv) {
  for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (size_t)gridDim.x * 256) z[i] = cap * tanhf(z[i] * inv);
}

template <typename T, typename YT>
void launch_dyt(const DytArgs& a, const float* x, const void* y, float* streams, const float* depth, float* r, void* h,
                int ntiles, bool vec, SeqDesc d, hipStream_t st) {
  float* sn = depth != nullptr ? streams + (size_t)a.n * a.sstride : nullptr;
  const int V = vec ? 4 : 1;
  const unsigned gy = (unsigned)((a.W + 64 * V - 1) / (64 * V));
  const dim3 grid(a.conv != nullptr ? 2 * ntiles : (d.Ttot + a.run - 1) / a.run, gy);
#define DYT_LAUNCH(V_, TP_) \
  hipLaunchKernelGGL((k_residual_dyt<T, YT, V_, TP_>), grid, dim3(64), 0, st, a, x, (const YT*)y, \
                     streams, depth, sn, r, (T*)h, d)
  if (a.conv == nullptr) {
    if (vec) DYT_LAUNCH(4, 1); else DYT_LAUNCH(1, 1);
  } else if (a.taps <= 4) {
    if (vec) DYT_LAUNCH(4, 4); else DYT_LAUNCH(1, 4);
  } else {
    if (vec) DYT_LAUNCH(4, 8); else DYT_LAUNCH(1, 8);
  }
#undef DYT_LAUNCH
}

}  // namespace

int seq_dyt_max_taps() { return MAXTAPS; }

// y: null, float (y_f32) or the activation type; tiles only with a convolution
void seq_residual_dyt(int code, int y_f32, const float* x, const void* y, int ldy, float mult, float* streams, int n,
                      const float* depth, float* r, const float* w, const float* b, float alpha, const float* conv, int taps,
                      const float* sin, float* sout, void* h, int W, const int* tile_seq, const int* tile_t0, int ntiles,
                      SeqDesc d, hipStream_t st) {
  if (d.Ttot == 0) return;
  const DytArgs a{ldy, mult, (size_t)d.Ttot * W, n, w, b, alpha, conv, taps, sin, sout, W, tile_seq, tile_t0,
                  d.Ttot < 1024 ? 1 : RUN};
  const bool vec = W % 4 == 0 && (y == nullptr || (ldy % 4 == 0 && ((uintptr_t)y & 15) == 0));   // the rest: whole tensors
  SEQ_DISPATCH_T(code, {
    if (y_f32)
      launch_dyt<T, float>(a, x, y, streams, depth, r, h, ntiles, vec, d, st);
    else
      launch_dyt<T, T>(a, x, y, streams, depth, r, h, ntiles, vec, d, st);
  });
  LIPA_CHECK_LAUNCH();
}

void seq_softcap(float* z, size_t n, float cap, hipStream_t st) {
  if (n == 0) return;
  const size_t blocks = (n + 255) / 256;
  hipLaunchKernelGGL(k_softcap, dim3((unsigned)(blocks < 8192 ? blocks : 8192)), dim3(256), 0, st, z, n, cap, 1.f / cap);
  LIPA_CHECK_LAUNCH();
}
