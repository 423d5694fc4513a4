// Row-wise kernels of layer-listed (hybrid) models on gfx950: the multi-stream
// residual ("hyper-connections") update fused with the next sublayer's
// read-in and RMS norm, the embedding gather into fp32 streams, gated
// feed-forward activations, per-head q/k normalisation fused with the paged
// cache write, the two-map (differential) attention combine, and the
// single-residual step of parallel blocks (several sublayer outputs and a
// unit-RMS addend joined in one pass with the next RMS or layer norm).
//
// Every kernel is a template over the activation element (bf16 bits or
// float); reductions, norms, the residual streams and every scale are fp32
// whatever the element is.  Sizes are run-time arguments: nothing here is
// specialised for one model's widths.
#include "../kernels/common.h"

namespace {

constexpr int kThreads = 256;
constexpr int kMaxStreams = 8;

template <typename T> __device__ __forceinline__ float ldf(const T* p, int64_t i);
template <> __device__ __forceinline__ float ldf<bf16_t>(const bf16_t* p, int64_t i) { return bf16_to_f32(p[i]); }
template <> __device__ __forceinline__ float ldf<float>(const float* p, int64_t i) { return p[i]; }
template <typename T> __device__ __forceinline__ void stf(T* p, int64_t i, float v);
template <> __device__ __forceinline__ void stf<bf16_t>(bf16_t* p, int64_t i, float v) { p[i] = f32_to_bf16(v); }
template <> __device__ __forceinline__ void stf<float>(float* p, int64_t i, float v) { p[i] = v; }

// V consecutive elements as floats (V = 4: one 8-byte / 16-byte access; V = 1: scalar)
template <typename T, int V> __device__ __forceinline__ void ldv(const T* p, float* o) {
  if constexpr (V == 1) {
    o[0] = ldf<T>(p, 0);
  } else if constexpr (sizeof(T) == 2) {
    const uint2 w = *reinterpret_cast<const uint2*>(p);
    o[0] = bf16lo(w.x), o[1] = bf16hi(w.x), o[2] = bf16lo(w.y), o[3] = bf16hi(w.y);
  } else {
    const f32x4 w = *reinterpret_cast<const f32x4*>(p);
    o[0] = w[0], o[1] = w[1], o[2] = w[2], o[3] = w[3];
  }
}
template <typename T, int V> __device__ __forceinline__ void stv(T* p, const float* v) {
  if constexpr (V == 1) {
    stf<T>(p, 0, v[0]);
  } else if constexpr (sizeof(T) == 2) {
    uint2 w;
    w.x = pack_bf16x2(v[0], v[1]);
    w.y = pack_bf16x2(v[2], v[3]);
    *reinterpret_cast<uint2*>(p) = w;
  } else {
    *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]};
  }
}

template <typename T, int V> __device__ __forceinline__ void cpv(T* dst, const T* src) {  // raw copy of V elements
  if constexpr (V == 1) {
    dst[0] = src[0];
  } else if constexpr (sizeof(T) == 2) {
    *reinterpret_cast<uint2*>(dst) = *reinterpret_cast<const uint2*>(src);
  } else {
    *reinterpret_cast<f32x4*>(dst) = *reinterpret_cast<const f32x4*>(src);
  }
}

// One residual step of a model with S parallel residual streams X [rows, S, W]
// (fp32, updated in place).  With y (the previous sublayer's output):
//     X_t <- sum_s mix[s, t] X_s + gain[t] * y          for every stream t
// then, with read-in weights rin [S]:  u = sum_s rin[s] X_s  and
//     out = u / sqrt(mean(u^2) + eps) * nw              (nw fp32 [W]; nw == null: out = u)
// S = 1, mix = [1], gain = [1], rin = [1] is the ordinary pre-norm residual.
template <typename T, int V>
__global__ void __launch_bounds__(kThreads) stream_step_kernel(float* __restrict__ X, const T* __restrict__ y,
                                                               int64_t y_stride, const float* __restrict__ mix,
                                                               const float* __restrict__ gain,
                                                               const float* __restrict__ rin,
                                                               const float* __restrict__ nw, float eps,
                                                               T* __restrict__ out, int64_t out_stride, int S, int W) {
  __shared__ float red[16];
  __shared__ float sm[kMaxStreams * kMaxStreams + 2 * kMaxStreams];
  const int64_t row = blockIdx.x;
  float* x = X + row * (int64_t)S * W;
  float* s_mix = sm;
  float* s_gain = sm + kMaxStreams * kMaxStreams;
  float* s_in = s_gain + kMaxStreams;
  if (threadIdx.x < S * S && y) s_mix[threadIdx.x] = mix[threadIdx.x];
  if (threadIdx.x < S) {
    s_gain[threadIdx.x] = y ? gain[threadIdx.x] : 0.f;
    s_in[threadIdx.x] = rin ? rin[threadIdx.x] : 0.f;
  }
  __syncthreads();
  float ss = 0.f;
  for (int c = threadIdx.x * V; c < W; c += kThreads * V) {
    float v[kMaxStreams][V];
#pragma unroll
    for (int s = 0; s < kMaxStreams; ++s)
      if (s < S) ldv<float, V>(x + (int64_t)s * W + c, v[s]);
    if (y) {
      float yv[V], n[kMaxStreams][V];
      ldv<T, V>(y + row * y_stride + c, yv);
#pragma unroll
      for (int t = 0; t < kMaxStreams; ++t) {
        if (t < S) {
#pragma unroll
          for (int e = 0; e < V; ++e) {
            float a = s_gain[t] * yv[e];
#pragma unroll
            for (int s = 0; s < kMaxStreams; ++s)
              if (s < S) a += s_mix[s * S + t] * v[s][e];
            n[t][e] = a;
          }
          stv<float, V>(x + (int64_t)t * W + c, n[t]);
        }
      }
#pragma unroll
      for (int t = 0; t < kMaxStreams; ++t)
        if (t < S) {
#pragma unroll
          for (int e = 0; e < V; ++e) v[t][e] = n[t][e];
        }
    }
    if (rin) {
#pragma unroll
      for (int e = 0; e < V; ++e) {
        float uu = 0.f;
#pragma unroll
        for (int s = 0; s < kMaxStreams; ++s)
          if (s < S) uu += s_in[s] * v[s][e];
        ss += uu * uu;
      }
    }
  }
  if (!rin) return;
  const float tot = block_reduce_sum(ss, red);
  const float r = nw ? rsqrtf(tot / (float)W + eps) : 1.f;
  // second pass: this thread re-reads the stream values it wrote itself
  for (int c = threadIdx.x * V; c < W; c += kThreads * V) {
    float u[V], o[V], xv[V], wv[V];
#pragma unroll
    for (int e = 0; e < V; ++e) u[e] = 0.f;
    for (int s = 0; s < S; ++s) {
      ldv<float, V>(x + (int64_t)s * W + c, xv);
#pragma unroll
      for (int e = 0; e < V; ++e) u[e] += s_in[s] * xv[e];
    }
    if (nw) ldv<float, V>(nw + c, wv);
#pragma unroll
    for (int e = 0; e < V; ++e) o[e] = nw ? u[e] * r * wv[e] : u[e];
    stv<T, V>(out + row * out_stride + c, o);
  }
}

// X[t, s, :] = table[ids[t], :] * scale (+ ptab[pos[t], :], a learned vector per position)
// for every stream s (fp32 streams; product and sum are fp32); with nw [W] the row is then
// divided by its root mean square (eps inside the root) and multiplied by nw
constexpr int kResChunks = 8;
template <typename T, int V>
__global__ void __launch_bounds__(kThreads) embed_streams_kernel(float* __restrict__ X, const T* __restrict__ table,
                                                                 const int64_t* __restrict__ ids, int S, int W,
                                                                 int64_t vocab, const T* __restrict__ ptab,
                                                                 const int64_t* __restrict__ pos, int64_t n_pos,
                                                                 float scale, const float* __restrict__ nw, float eps) {
  __shared__ float red[16];
  const int64_t t = blockIdx.x;
  const int64_t id = ids[t];
  const bool ok = id >= 0 && id < vocab;
  const int64_t p = ptab ? pos[t] : -1;
  const bool pok = p >= 0 && p < n_pos;
  auto value = [&](int c, float* v) {
    if (ok) ldv<T, V>(table + id * (int64_t)W + c, v);
#pragma unroll
    for (int i = 0; i < V; ++i) v[i] = ok ? v[i] * scale : 0.f;
    if (pok) {
      float q[V];
      ldv<T, V>(ptab + p * (int64_t)W + c, q);
#pragma unroll
      for (int i = 0; i < V; ++i) v[i] += q[i];
    }
  };
  float r = 1.f;
  float v[kResChunks][V];  // the row, as far as it fits
#pragma unroll
  for (int k = 0; k < kResChunks; ++k) {
    const int c = (threadIdx.x + k * kThreads) * V;
    if (c < W) value(c, v[k]);
  }
  if (nw) {
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < kResChunks; ++k)
      if ((int)(threadIdx.x + k * kThreads) * V < W) {
#pragma unroll
        for (int i = 0; i < V; ++i) ss += v[k][i] * v[k][i];
      }
    for (int c = (threadIdx.x + kResChunks * kThreads) * V; c < W; c += kThreads * V) {
      float u[V];
      value(c, u);
#pragma unroll
      for (int i = 0; i < V; ++i) ss += u[i] * u[i];
    }
    r = rsqrtf(block_reduce_sum(ss, red) / (float)W + eps);
  }
  auto put = [&](int c, float* u) {
    if (nw) {
      float w[V];
      ldv<float, V>(nw + c, w);
#pragma unroll
      for (int i = 0; i < V; ++i) u[i] *= r * w[i];
    }
    for (int s = 0; s < S; ++s) stv<float, V>(X + (t * S + s) * (int64_t)W + c, u);
  };
#pragma unroll
  for (int k = 0; k < kResChunks; ++k) {
    const int c = (threadIdx.x + k * kThreads) * V;
    if (c < W) put(c, v[k]);
  }
  for (int c = (threadIdx.x + kResChunks * kThreads) * V; c < W; c += kThreads * V) {
    float u[V];
    value(c, u);
    put(c, u);
  }
}

// out[t, :] = table[ids[t], :] (zeros for ids outside the table)
template <typename T>
__global__ void __launch_bounds__(kThreads) gather_rows_kernel(T* __restrict__ out, const T* __restrict__ table,
                                                               const int64_t* __restrict__ ids, int W, int64_t vocab) {
  const int64_t t = blockIdx.x;
  const int64_t id = ids[t];
  const bool ok = id >= 0 && id < vocab;
  for (int c = threadIdx.x; c < W; c += kThreads) out[t * (int64_t)W + c] = ok ? table[id * (int64_t)W + c] : (T)0;
}

// One step of a single fp32 residual x [rows, W], in place:
//     x <- x + a + b + c / sqrt(mean(c^2) + eps) * cw        (a, b, c optional)
// then  xc = x in T (when xc), and the norm that follows (when out):
//     norm 1 (RMS):    out = x / sqrt(mean(x^2) + eps) * nw
//     norm 2 (layer):  out = (x - mean) / sqrt(mean((x - mean)^2) + eps) * nw + nb
// The row stays in registers between the passes (W <= kThreads * V * kResChunks)
// or is re-read from x by the thread that wrote it.
// EXT (further addends, all optional; ResExt below): a second normed addend d,
// an fp32 addend e, a constant row `bias`, the weighted sum of a mixture of
// experts, and a list of rows: then row r of out is the result for row rows[r],
// and x itself is left as it was.
template <typename T> struct ResExt {
  const T* d;         // + d / sqrt(mean(d^2) + eps) * dw
  int64_t d_stride;
  const float* dw;
  const float* e;     // + e, [rows, W] fp32
  const float* bias;  // + bias, [W]
  // + sum_k mw[row, k] * src_k: my[row * top + k] (expert outputs in slot order), or the row of mh
  // where the choice midx[row, k] is no expert (>= experts: an identity output)
  const T* my;
  const float* mw;
  const int* midx;
  int experts, top;
  const T* mh;
  int64_t mh_stride;
  const int64_t* rows;
};
// sum over the workgroup (4 waves); every call of a kernel has an area `red` of its own: one barrier
__device__ __forceinline__ float sum_all(float v, float* red) {
  v = wave_reduce_sum(v);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  return red[0] + red[1] + red[2] + red[3];
}

// KC: chunks of a row in registers.  F: which addends there are (bits below), or kAny: asked of the pointers.  With
// known addends nothing stands between the loads of a row: all of them are issued before the first is used.
constexpr int kHasA = 1, kHasB = 2, kHasC = 4, kHasD = 8, kHasBias = 16, kHasExperts = 32, kAny = -1;
template <typename T, int V, bool EXT, int KC, int F>
__global__ void __launch_bounds__(kThreads) residual_step_kernel(
    float* __restrict__ X, const T* __restrict__ a, int64_t a_stride, const T* __restrict__ b, int64_t b_stride,
    const T* __restrict__ c, int64_t c_stride, const float* __restrict__ cw, const T* __restrict__ cg,
    int64_t cg_stride, const float* __restrict__ cgb, float eps, int norm, const float* __restrict__ nw,
    const float* __restrict__ nb, T* __restrict__ out, T* __restrict__ xc, int W, ResExt<T> g) {
  static_assert(kThreads == 256, "sum_all adds four waves");
  __shared__ float red[4][4];
  const int64_t row = EXT && g.rows ? g.rows[blockIdx.x] : (int64_t)blockIdx.x, orow = blockIdx.x;
  float* x = X + row * (int64_t)W;
  const bool has_a = F == kAny ? a != nullptr : F & kHasA, has_b = F == kAny ? b != nullptr : F & kHasB,
             has_c = F == kAny ? c != nullptr : F & kHasC, has_d = EXT && (F == kAny ? g.d != nullptr : F & kHasD),
             has_bias = EXT && (F == kAny ? g.bias != nullptr : F & kHasBias),
             has_my = EXT && (F == kAny ? g.my != nullptr : F & kHasExperts), has_e = EXT && F == kAny && g.e;
  // the addend c at columns e .. e + V - 1, gated by sigmoid(cg + cgb) when a gate is given
  auto load_c = [&](int e, float* v) {
    ldv<T, V>(c + row * c_stride + e, v);
    if (F == kAny && cg) {
      float gt[V], gb[V];
      ldv<T, V>(cg + row * cg_stride + e, gt);
      if (cgb) ldv<float, V>(cgb + e, gb);
#pragma unroll
      for (int i = 0; i < V; ++i) v[i] *= 1.f / (1.f + expf(-(gt[i] + (cgb ? gb[i] : 0.f))));
    }
  };
  auto load_d = [&](int e, float* v) { ldv<T, V>(g.d + row * g.d_stride + e, v); };
  // the experts' weighted sum, two choices at a time
  auto load_experts = [&](int e, float* m) {
#pragma unroll
    for (int i = 0; i < V; ++i) m[i] = 0.f;
    for (int k = 0; k < g.top; k += 2) {
      const int64_t s0 = row * g.top + k, s1 = k + 1 < g.top ? s0 + 1 : s0;
      const float w0 = g.mw[s0], w1 = k + 1 < g.top ? g.mw[s1] : 0.f;
      const T* ident = g.mh + row * g.mh_stride;
      float t0[V], t1[V];
      ldv<T, V>((g.midx && g.midx[s0] >= g.experts ? ident : g.my + s0 * (int64_t)W) + e, t0);
      ldv<T, V>((g.midx && g.midx[s1] >= g.experts ? ident : g.my + s1 * (int64_t)W) + e, t1);
#pragma unroll
      for (int i = 0; i < V; ++i) m[i] += w0 * t0[i];
      if (k + 1 < g.top) {
#pragma unroll
        for (int i = 0; i < V; ++i) m[i] += w1 * t1[i];
      }
    }
  };
  // x and everything added to it as it is
  auto load_x = [&](int e, float* v) {
    float t[V];
    ldv<float, V>(x + e, v);
    if (has_a) {
      ldv<T, V>(a + row * a_stride + e, t);
#pragma unroll
      for (int i = 0; i < V; ++i) v[i] += t[i];
    }
    if (has_b) {
      ldv<T, V>(b + row * b_stride + e, t);
#pragma unroll
      for (int i = 0; i < V; ++i) v[i] += t[i];
    }
    if constexpr (EXT) {
      if (has_bias) {
        ldv<float, V>(g.bias + e, t);
#pragma unroll
        for (int i = 0; i < V; ++i) v[i] += t[i];
      }
      if (has_my) {
        load_experts(e, t);
#pragma unroll
        for (int i = 0; i < V; ++i) v[i] += t[i];
      }
      if (has_e) {
        ldv<float, V>(g.e + row * (int64_t)W + e, t);
#pragma unroll
        for (int i = 0; i < V; ++i) v[i] += t[i];
      }
    }
  };
  float r[KC][V], cv[KC][V], dv[EXT ? KC : 1][V], cs = 0.f, ds = 0.f;
  if constexpr (F == kAny) {
#pragma unroll
    for (int k = 0; k < KC; ++k) {
      const int e = (threadIdx.x + k * kThreads) * V;
      if (e < W) {
        if (has_c) load_c(e, cv[k]);
        if constexpr (EXT) {
          if (has_d) load_d(e, dv[k]);
        }
        load_x(e, r[k]);
      }
    }
  } else {  // columns past the row: the last ones again (nothing of them is used)
    float y[(F & kHasExperts) ? KC : 1][V], av[(F & kHasA) ? KC : 1][V], bv[(F & kHasB) ? KC : 1][V],
        cb[(F & kHasBias) ? KC : 1][V];
#pragma unroll
    for (int k = 0; k < KC; ++k) {
      const int e = min((int)(threadIdx.x + k * kThreads) * V, W - V);
      ldv<float, V>(x + e, r[k]);
      if constexpr ((F & kHasC) != 0) load_c(e, cv[k]);
      if constexpr ((F & kHasD) != 0) load_d(e, dv[k]);
      if constexpr ((F & kHasA) != 0) ldv<T, V>(a + row * a_stride + e, av[k]);
      if constexpr ((F & kHasB) != 0) ldv<T, V>(b + row * b_stride + e, bv[k]);
      if constexpr ((F & kHasBias) != 0) ldv<float, V>(g.bias + e, cb[k]);
    }
    if constexpr ((F & kHasExperts) != 0) {
#pragma unroll
      for (int k = 0; k < KC; ++k)
#pragma unroll
        for (int i = 0; i < V; ++i) y[k][i] = 0.f;
      for (int c0 = 0; c0 < g.top; c0 += 2) {  // two choices at a time over all chunks
        const int64_t s0 = row * g.top + c0, s1 = c0 + 1 < g.top ? s0 + 1 : s0;
        const float w0 = g.mw[s0], w1 = c0 + 1 < g.top ? g.mw[s1] : 0.f;
        const T* ident = g.mh + row * g.mh_stride;
        const bool i0 = g.midx && g.midx[s0] >= g.experts, i1 = g.midx && g.midx[s1] >= g.experts;
        const T *p0 = i0 ? ident : g.my + s0 * (int64_t)W, *p1 = i1 ? ident : g.my + s1 * (int64_t)W;
        float t0[KC][V], t1[KC][V];
#pragma unroll
        for (int k = 0; k < KC; ++k) {
          const int e = min((int)(threadIdx.x + k * kThreads) * V, W - V);
          ldv<T, V>(p0 + e, t0[k]);
          ldv<T, V>(p1 + e, t1[k]);
        }
#pragma unroll
        for (int k = 0; k < KC; ++k)
#pragma unroll
          for (int i = 0; i < V; ++i) {
            y[k][i] += w0 * t0[k][i];
            if (c0 + 1 < g.top) y[k][i] += w1 * t1[k][i];
          }
      }
    }
#pragma unroll
    for (int k = 0; k < KC; ++k)
#pragma unroll
      for (int i = 0; i < V; ++i) {
        if constexpr ((F & kHasA) != 0) r[k][i] += av[k][i];
        if constexpr ((F & kHasB) != 0) r[k][i] += bv[k][i];
        if constexpr ((F & kHasBias) != 0) r[k][i] += cb[k][i];
        if constexpr ((F & kHasExperts) != 0) r[k][i] += y[k][i];
      }
  }
#pragma unroll
  for (int k = 0; k < KC; ++k) {
    const int e = (threadIdx.x + k * kThreads) * V;
    if (e < W) {
#pragma unroll
      for (int i = 0; i < V; ++i) {
        if (has_c) cs += cv[k][i] * cv[k][i];
        if constexpr (EXT) {
          if (has_d) ds += dv[k][i] * dv[k][i];
        }
      }
    }
  }
  const int tail = (threadIdx.x + KC * kThreads) * V;  // wide rows: columns from here on are read when they are needed
  for (int e = tail; e < W; e += kThreads * V) {
    float v[V];
    if (has_c) {
      load_c(e, v);
#pragma unroll
      for (int i = 0; i < V; ++i) cs += v[i] * v[i];
    }
    if (has_d) {
      load_d(e, v);
#pragma unroll
      for (int i = 0; i < V; ++i) ds += v[i] * v[i];
    }
  }
  float rc = 0.f, rd = 0.f;
  if (has_d) {
    ds = wave_reduce_sum(ds);
    if ((threadIdx.x & 63) == 0) red[1][threadIdx.x >> 6] = ds;
  }
  if (has_c) rc = rsqrtf(sum_all(cs, red[0]) / (float)W + eps);
  else if (has_d) __syncthreads();
  if (has_d) rd = rsqrtf((red[1][0] + red[1][1] + red[1][2] + red[1][3]) / (float)W + eps);
  // the normed addends at columns e .. e + V - 1; ct, dt: the values of c and d there
  auto add = [&](int e, float* v, const float* ct, const float* dt) {
    float w[V];
    if (has_c) {
      ldv<float, V>(cw + e, w);
#pragma unroll
      for (int i = 0; i < V; ++i) v[i] += ct[i] * rc * w[i];
    }
    if (has_d) {
      ldv<float, V>(g.dw + e, w);
#pragma unroll
      for (int i = 0; i < V; ++i) v[i] += dt[i] * rd * w[i];
    }
  };
  // a wide row's tail: x and its addends from memory
  auto wide = [&](int e, float* v) {
    float ct[V], dt[V];
    load_x(e, v);
    if (has_c) load_c(e, ct);
    if (has_d) load_d(e, dt);
    add(e, v, ct, dt);
  };
  bool touch = has_a || has_b || has_c;
  if constexpr (EXT) touch = !g.rows && (touch || has_d || has_e || has_bias || has_my);
  float sum = 0.f;
#pragma unroll
  for (int k = 0; k < KC; ++k) {
    const int e = (threadIdx.x + k * kThreads) * V;
    if (e < W) {
      add(e, r[k], cv[k], dv[EXT ? k : 0]);
      if (touch) stv<float, V>(x + e, r[k]);
      if (xc) stv<T, V>(xc + orow * (int64_t)W + e, r[k]);
#pragma unroll
      for (int i = 0; i < V; ++i) sum += r[k][i];
    }
  }
  for (int e = tail; e < W; e += kThreads * V) {
    float v[V];
    wide(e, v);
    if (touch) stv<float, V>(x + e, v);
    if (xc) stv<T, V>(xc + orow * (int64_t)W + e, v);
#pragma unroll
    for (int i = 0; i < V; ++i) sum += v[i];
  }
  if (!norm) return;
  // a wide row's tail once more: as this thread wrote it, or (x left as it was) summed again
  auto again = [&](int e, float* v) {
    if (touch || !EXT || !g.rows) ldv<float, V>(x + e, v);
    else wide(e, v);
  };
  float mean = 0.f;
  if (norm == 2) mean = sum_all(sum, red[2]) / (float)W;
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < KC; ++k) {
    const int e = (threadIdx.x + k * kThreads) * V;
    if (e < W) {
#pragma unroll
      for (int i = 0; i < V; ++i) ss += (r[k][i] - mean) * (r[k][i] - mean);
    }
  }
  for (int e = tail; e < W; e += kThreads * V) {
    float v[V];
    again(e, v);
#pragma unroll
    for (int i = 0; i < V; ++i) ss += (v[i] - mean) * (v[i] - mean);
  }
  const float rs = rsqrtf(sum_all(ss, red[3]) / (float)W + eps);
  auto put = [&](int e, const float* v) {
    float w[V], bb[V], o[V];
    ldv<float, V>(nw + e, w);
    if (norm == 2) ldv<float, V>(nb + e, bb);
#pragma unroll
    for (int i = 0; i < V; ++i) o[i] = (v[i] - mean) * rs * w[i] + (norm == 2 ? bb[i] : 0.f);
    stv<T, V>(out + orow * (int64_t)W + e, o);
  };
#pragma unroll
  for (int k = 0; k < KC; ++k) {
    const int e = (threadIdx.x + k * kThreads) * V;
    if (e < W) put(e, r[k]);
  }
  for (int e = tail; e < W; e += kThreads * V) {
    float v[V];
    again(e, v);
    put(e, v);
  }
}

// Weighted sum over the results of all layers so far (a depth average):
//     dst[r, :] = sum_{j < n} w[j] * stack[j][row(r), :]        row(r) = rows ? rows[r] : r
// stack [>= n, T, W] fp32, one [T, W] plane per layer result; dst fp32 [n_rows, W] (it may be a
// later plane of the same stack); then, when out: out = dst / sqrt(mean(dst^2) + eps) * nw in T
// (nw one weight per column).  With c (the last sublayer's output, [T, c_stride] in T) the newest
// plane n - 1 first takes its closing addend, plane <- plane + c / sqrt(mean(c^2) + eps) * cw, and
// is written back (without `rows`; with them the sum alone uses it, a row may be listed twice).
// Sums in the order j = 0, 1, ..., all fp32.  The row stays in registers between the sum and the
// norm (W <= kThreads * V * kResChunks) or is re-read from dst.
template <typename T, int V>
__global__ void __launch_bounds__(kThreads) depth_mix_kernel(float* __restrict__ dst, float* __restrict__ stack,
                                                             int64_t plane, int n, const float* __restrict__ w,
                                                             const int64_t* __restrict__ rows, float eps,
                                                             const float* __restrict__ nw, T* __restrict__ out,
                                                             const T* __restrict__ c, int64_t c_stride,
                                                             const float* __restrict__ cw, int W) {
  __shared__ float red[16];
  const int64_t r = blockIdx.x;
  const int64_t row = rows ? rows[r] : r;
  float* src = stack + row * (int64_t)W;
  float* x = dst + r * (int64_t)W;
  float rc = 0.f;
  if (c) {
    float cs = 0.f;
    for (int e = threadIdx.x * V; e < W; e += kThreads * V) {
      float t[V];
      ldv<T, V>(c + row * c_stride + e, t);
#pragma unroll
      for (int i = 0; i < V; ++i) cs += t[i] * t[i];
    }
    rc = rsqrtf(block_reduce_sum(cs, red) / (float)W + eps);
    __syncthreads();
  }
  // the weighted sum of columns e .. e + V - 1 over the planes
  auto mix = [&](int e, float* a) {
#pragma unroll
    for (int i = 0; i < V; ++i) a[i] = 0.f;
    for (int j = 0; j < n; ++j) {
      float t[V];
      ldv<float, V>(src + j * plane + e, t);
      if (c && j == n - 1) {
        float cv[V], g[V];
        ldv<T, V>(c + row * c_stride + e, cv);
        ldv<float, V>(cw + e, g);
#pragma unroll
        for (int i = 0; i < V; ++i) t[i] += cv[i] * rc * g[i];
        if (!rows) stv<float, V>(src + j * plane + e, t);
      }
      const float wj = w[j];
#pragma unroll
      for (int i = 0; i < V; ++i) a[i] += wj * t[i];
    }
  };
  float acc[kResChunks][V];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < kResChunks; ++k) {
    const int e = (threadIdx.x + k * kThreads) * V;
    if (e < W) {
      mix(e, acc[k]);
      stv<float, V>(x + e, acc[k]);
#pragma unroll
      for (int i = 0; i < V; ++i) ss += acc[k][i] * acc[k][i];
    }
  }
  for (int e = (threadIdx.x + kResChunks * kThreads) * V; e < W; e += kThreads * V) {
    float a[V];
    mix(e, a);
    stv<float, V>(x + e, a);
#pragma unroll
    for (int i = 0; i < V; ++i) ss += a[i] * a[i];
  }
  if (!out) return;
  const float rs = rsqrtf(block_reduce_sum(ss, red) / (float)W + eps);
#pragma unroll
  for (int k = 0; k < kResChunks; ++k) {
    const int e = (threadIdx.x + k * kThreads) * V;
    if (e < W) {
      float g[V], o[V];
      ldv<float, V>(nw + e, g);
#pragma unroll
      for (int i = 0; i < V; ++i) o[i] = acc[k][i] * rs * g[i];
      stv<T, V>(out + r * (int64_t)W + e, o);
    }
  }
  for (int e = (threadIdx.x + kResChunks * kThreads) * V; e < W; e += kThreads * V) {
    float a[V], g[V], o[V];
    ldv<float, V>(x + e, a);  // written by this thread above
    ldv<float, V>(nw + e, g);
#pragma unroll
    for (int i = 0; i < V; ++i) o[i] = a[i] * rs * g[i];
    stv<T, V>(out + r * (int64_t)W + e, o);
  }
}

// out [rows, n] = x / sqrt(mean(x^2) + eps) * w over a column section x [rows, n] of wider rows
// (a low-rank latent between its two projections): one wave per row, fp32 sums
template <typename T>
__global__ void __launch_bounds__(kThreads) section_norm_kernel(T* __restrict__ out, const T* __restrict__ x,
                                                                int64_t x_stride, const float* __restrict__ w,
                                                                int rows, int n, float eps) {
  const int lane = threadIdx.x & 63;
  const int64_t row = (int64_t)blockIdx.x * (kThreads / 64) + (threadIdx.x >> 6);
  if (row >= rows) return;
  const T* xr = x + row * x_stride;
  float ss = 0.f;
  for (int e = lane; e < n; e += 64) {
    const float v = ldf<T>(xr, e);
    ss += v * v;
  }
  const float rs = rsqrtf(wave_reduce_sum(ss) / (float)n + eps);
  for (int e = lane; e < n; e += 64) stf<T>(out, row * n + e, ldf<T>(xr, e) * rs * (w ? w[e] : 1.f));
}

__device__ __forceinline__ float act_fn(float z, int act) {
  if (act == 5) return tanhf(z);
  if (act == 0) return fmaxf(z, 0.f);           // relu
  if (act == 1) return z / (1.f + __expf(-z));  // silu
  if (act == 3) return 1.f / (1.f + __expf(-z));  // sigmoid
  if (act == 4) {                                 // relu squared
    const float r = fmaxf(z, 0.f);
    return r * r;
  }
  // gelu, tanh form: 0.5 (1 + tanh u) = 1 / (1 + e^(-2 u)), u = sqrt(2 / pi) (z + 0.044715 z^3)
  return z * __builtin_amdgcn_rcpf(1.f + __expf(-1.5957691216057308f * (z + 0.044715f * z * z * z)));
}

// out [rows, F] = act(gate + gate_b) * (up + up_b) * row_scale[row] * post  (up null: act(gate) alone); gate and
// up are column sections of wider rows (a gated feed-forward's [gate | up], an output gate that is part of a
// fused projection).  u_dv > 0: up is head-major, column c of row r at up[(c / u_dv) * u_head + r * u_stride + c % u_dv].
// ROWS: rows per workgroup (with biases, so that they are read once for several rows).
template <typename T, int V, int ROWS>
__global__ void __launch_bounds__(kThreads) act_mul_kernel(T* __restrict__ out, const T* __restrict__ gate,
                                                           int64_t g_stride, const T* __restrict__ up,
                                                           int64_t u_stride, int F, int64_t out_stride, int act,
                                                           float limit, float alpha, float post,
                                                           const float* __restrict__ gate_b,
                                                           const float* __restrict__ up_b,
                                                           const float* __restrict__ row_scale, int u_dv,
                                                           int64_t u_head, int rows) {
  const int r0 = blockIdx.y * ROWS, n = ROWS == 1 ? 1 : min(ROWS, rows - r0);
  for (int c = (blockIdx.x * kThreads + threadIdx.x) * V; c < F; c += gridDim.x * kThreads * V) {
    float gb[V], ub[V];  // biases serve all rows of the workgroup
    if (gate_b) ldv<float, V>(gate_b + c, gb);
    if (up_b) ldv<float, V>(up_b + c, ub);
    for (int i = 0; i < n; ++i) {
      const int64_t r = r0 + i;
      float g[V], u[V], o[V];
      ldv<T, V>(gate + r * g_stride + c, g);
      if (up) ldv<T, V>(up + r * u_stride + (u_dv ? c / u_dv * u_head + c % u_dv : (int64_t)c), u);
      const float scale = row_scale ? post * row_scale[r] : post;
#pragma unroll
      for (int e = 0; e < V; ++e) {
        if (gate_b) g[e] += gb[e];
        if (up && up_b) u[e] += ub[e];
        if (act == 6) {  // clamped gated unit: g sigmoid(alpha g) (u + 1), g <= limit, |u| <= limit
          const float gc = fminf(g[e], limit), uc = fminf(fmaxf(u[e], -limit), limit);
          o[e] = gc / (1.f + __expf(-alpha * gc)) * (uc + 1.f);
        } else {
          o[e] = act_fn(g[e], act) * (up ? u[e] : 1.f);
        }
        o[e] *= scale;
      }
      stv<T, V>(out + r * out_stride + c, o);
    }
  }
}

// Per token row of a fused projection output x = [q | k | v]:
//   q: n_q vectors of d; with qw: unit RMS times qw [d]; with temp_coef != 0 a
//      position-dependent gain 1 + coef * ln(floor((p + 1) / every) + 1); in place
//   k: n_k vectors of d at column k_off; with kw: unit RMS times kw; written to
//      the K cache row of the token's slot (kc [slots, n_k * d])
//   v: v_mode 0: no V cache (V is the K cache); 1: the k section as projected
//      (before its norm) is the value; 2: v_w columns at v_off are the value,
//      mixed with an earlier layer's values of the same token when v_first is
//      given: (1 - v_lambda) v + v_lambda v_first, in fp32
// slot < 0: nothing is cached for the row.
template <typename T, int V>
__global__ void __launch_bounds__(kThreads) headprep_cache_kernel(
    T* __restrict__ x, int64_t x_stride, const int64_t* __restrict__ pos, const int64_t* __restrict__ slots,
    int n_q, int n_k, int d, int k_off, const float* __restrict__ qw, const float* __restrict__ kw, float eps,
    float temp_coef, double temp_every, T* __restrict__ kc, T* __restrict__ vc, int v_mode, int v_off, int v_w,
    const T* __restrict__ v_first, int64_t vf_stride, float v_lambda, int lpv) {
  // lpv lanes (a power of two) share one head vector, so a wave works on 64 / lpv
  // vectors at once and their loads overlap; the sum of squares is reduced inside the group
  const int64_t t = blockIdx.x;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, nw = kThreads / 64;
  const int per_wave = 64 / lpv, grp = lane / lpv, gl = lane - grp * lpv;
  T* row = x + t * x_stride;
  const int64_t slot = slots[t];
  const int k_w = n_k * d;
  float gain = 1.f;
  if (temp_coef != 0.f) {
    const double k = floor((double)(pos[t] + 1) / temp_every);
    gain = 1.f + temp_coef * logf((float)k + 1.f);
  }
  const bool q_work = qw != nullptr || temp_coef != 0.f;
  for (int v = wid * per_wave + grp; v < n_q + n_k; v += nw * per_wave) {
    const bool is_q = v < n_q;
    if (is_q && !q_work) continue;
    if (!is_q && slot < 0) continue;
    T* src = is_q ? row + (int64_t)v * d : row + k_off + (int64_t)(v - n_q) * d;
    const float* w = is_q ? qw : kw;
    float r = 1.f;
    if (w) {
      float ss = 0.f;
      for (int e = gl * V; e < d; e += lpv * V) {
        float a[V];
        ldv<T, V>(src + e, a);
#pragma unroll
        for (int i = 0; i < V; ++i) ss += a[i] * a[i];
      }
      for (int o = lpv >> 1; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
      r = rsqrtf(ss / (float)d + eps);
    }
    T* kd = is_q ? src : kc + slot * (int64_t)k_w + (int64_t)(v - n_q) * d;
    T* vd = (!is_q && v_mode == 1) ? vc + slot * (int64_t)k_w + (int64_t)(v - n_q) * d : nullptr;
    const float g = is_q ? gain : 1.f;
    for (int e = gl * V; e < d; e += lpv * V) {
      float a[V], wv[V];
      ldv<T, V>(src + e, a);
      if (vd) cpv<T, V>(vd + e, src + e);
      if (w) ldv<float, V>(w + e, wv);
#pragma unroll
      for (int i = 0; i < V; ++i) a[i] = a[i] * (w ? r * wv[i] : 1.f) * g;
      stv<T, V>(kd + e, a);
    }
  }
  if (v_mode == 2 && slot >= 0) {
    const T* vs = row + v_off;
    T* vd = vc + slot * (int64_t)v_w;
    if (v_first) {
      const T* vf = v_first + t * vf_stride;
      for (int e = threadIdx.x * V; e < v_w; e += kThreads * V) {
        float a[V], f[V];
        ldv<T, V>(vs + e, a);
        ldv<T, V>(vf + e, f);
#pragma unroll
        for (int i = 0; i < V; ++i) a[i] = (1.f - v_lambda) * a[i] + v_lambda * f[i];
        stv<T, V>(vd + e, a);
      }
    } else {
      for (int e = threadIdx.x * V; e < v_w; e += kThreads * V) cpv<T, V>(vd + e, vs + e);
    }
  }
}

// Two-map attention combine: a [rows, H, 2, dv] fp32 (map outputs over the
// same values)  ->  out [rows, H, dv] = unit_rms(a1 - lam * a2) * post, times
// sigmoid(gate[row, head]) when gate (logits [rows, gate_stride], one per head) is given.
// One wave per (row, head).
template <typename T>
__global__ void __launch_bounds__(kThreads) diff_combine_kernel(T* __restrict__ out, const float* __restrict__ a,
                                                                int64_t n_vec, int dv, float lam, float post,
                                                                float eps, const T* __restrict__ gate,
                                                                int64_t gate_stride, int H) {
  const int lane = threadIdx.x & 63;
  const int64_t v = (int64_t)blockIdx.x * (kThreads / 64) + (threadIdx.x >> 6);
  if (v >= n_vec) return;
  const float* a1 = a + v * 2 * (int64_t)dv;
  const float* a2 = a1 + dv;
  float ss = 0.f;
  for (int e = lane; e < dv; e += 64) {
    const float o = a1[e] - lam * a2[e];
    ss += o * o;
  }
  float r = rsqrtf(wave_reduce_sum(ss) / (float)dv + eps) * post;
  if (gate) r /= 1.f + expf(-ldf<T>(gate, v / H * gate_stride + v % H));
  for (int e = lane; e < dv; e += 64) stf<T>(out, v * dv + e, (a1[e] - lam * a2[e]) * r);
}

}  // namespace

#define DISPATCH_T(f32, ...)          \
  if (f32) {                          \
    using T = float;                  \
    __VA_ARGS__;                      \
  } else {                            \
    using T = bf16_t;                 \
    __VA_ARGS__;                      \
  }

extern "C" {

int dxm_stream_step(float* X, const void* y, int64_t y_stride, const float* mix, const float* gain, const float* rin,
                    const float* nw, float eps, void* out, int64_t out_stride, int rows, int S, int W, int f32,
                    hipStream_t st) {
  if (S < 1 || S > kMaxStreams || W < 1) return 1;
  if (rows <= 0) return 0;
  if (y && (!mix || !gain)) return 2;
  if (rin && !out) return 3;
  const int esz = f32 ? 4 : 2;
  const bool vec = W % 4 == 0 && y_stride % 4 == 0 && out_stride % 4 == 0 && (uintptr_t)X % 16 == 0 &&
                   (uintptr_t)y % (4 * esz) == 0 && (uintptr_t)out % (4 * esz) == 0 && (uintptr_t)nw % 16 == 0;
  if (vec) {
    DISPATCH_T(f32, hipLaunchKernelGGL((stream_step_kernel<T, 4>), dim3(rows), dim3(kThreads), 0, st, X, (const T*)y,
                                       y_stride, mix, gain, rin, nw, eps, (T*)out, out_stride, S, W));
  } else {
    DISPATCH_T(f32, hipLaunchKernelGGL((stream_step_kernel<T, 1>), dim3(rows), dim3(kThreads), 0, st, X, (const T*)y,
                                       y_stride, mix, gain, rin, nw, eps, (T*)out, out_stride, S, W));
  }
  DX_CHECK_LAUNCH();
  return 0;
}

int dxm_embed_streams(float* X, const void* table, const int64_t* ids, int rows, int S, int W, int64_t vocab,
                      const void* ptab, const int64_t* pos, int64_t n_pos, float scale, const float* nw, float eps, int f32,
                      hipStream_t st) {
  if (rows <= 0) return 0;
  if (ptab && !pos) return 1;
  const int by = f32 ? 16 : 8;
  const bool vec = W % 4 == 0 && (uintptr_t)X % 16 == 0 && (uintptr_t)table % by == 0 && (uintptr_t)ptab % by == 0 &&
                   (uintptr_t)nw % 16 == 0;
#define EMBED(V)                                                                                                         \
  DISPATCH_T(f32, hipLaunchKernelGGL((embed_streams_kernel<T, V>), dim3(rows), dim3(kThreads), 0, st, X, (const T*)table, \
                                     ids, S, W, vocab, (const T*)ptab, pos, n_pos, scale, nw, eps))
  if (vec) { EMBED(4) }
  else { EMBED(1) }
#undef EMBED
  DX_CHECK_LAUNCH();
  return 0;
}

int dxm_gather_rows(void* out, const void* table, const int64_t* ids, int rows, int W, int64_t vocab, int f32,
                    hipStream_t st) {
  if (rows <= 0) return 0;
  DISPATCH_T(f32, hipLaunchKernelGGL(gather_rows_kernel<T>, dim3(rows), dim3(kThreads), 0, st, (T*)out,
                                     (const T*)table, ids, W, vocab));
  DX_CHECK_LAUNCH();
  return 0;
}

int dxm_residual_step(float* X, const void* a, int64_t a_stride, const void* b, int64_t b_stride, const void* c,
                      int64_t c_stride, const float* cw, const void* cg, int64_t cg_stride, const float* cgb, float eps,
                      int norm, const float* nw, const float* nb, void* out, void* xc, int rows, int W, const void* d,
                      int64_t d_stride, const float* dw, const float* e, const float* bias, const void* my,
                      const float* mw, const int* midx, int experts, int top, const void* mh, int64_t mh_stride,
                      const int64_t* pick, int f32, hipStream_t st) {
  if (rows <= 0) return 0;
  if (W < 1 || norm < 0 || norm > 2) return 1;
  if ((c && !cw) || (norm && (!nw || !out)) || (norm == 2 && !nb) || (cg && !c) || (d && !dw)) return 2;
  if (my && (!mw || top < 1 || (midx && !mh))) return 3;
  const int esz = f32 ? 4 : 2;
  auto al = [&](const void* p, int by) { return (uintptr_t)p % by == 0; };
  const bool vec = W % 4 == 0 && a_stride % 4 == 0 && b_stride % 4 == 0 && c_stride % 4 == 0 && cg_stride % 4 == 0 &&
                   d_stride % 4 == 0 && mh_stride % 4 == 0 && al(X, 16) && al(a, 4 * esz) && al(b, 4 * esz) &&
                   al(c, 4 * esz) && al(cg, 4 * esz) && al(cgb, 16) && al(cw, 16) && al(nw, 16) && al(nb, 16) &&
                   al(out, 4 * esz) && al(xc, 4 * esz) && al(d, 4 * esz) && al(dw, 16) && al(e, 16) && al(bias, 16) &&
                   al(my, 4 * esz) && al(mh, 4 * esz);
  const bool ext = d || e || bias || my || pick;
#define RES(V, EXT, KC, F)                                                                                              \
  DISPATCH_T(f32, hipLaunchKernelGGL((residual_step_kernel<T, V, EXT, KC, F>), dim3(rows), dim3(kThreads), 0, st, X,           \
                                     (const T*)a, a_stride, (const T*)b, b_stride, (const T*)c, c_stride, cw,           \
                                     (const T*)cg, cg_stride, cgb, eps, norm, nw, nb, (T*)out, (T*)xc, W,               \
                                     (ResExt<T>{(const T*)d, d_stride, dw, e, bias, (const T*)my, mw, midx, experts,    \
                                                top, (const T*)mh, mh_stride, pick})))
  const bool narrow = W <= 4 * kThreads * 4;  // four chunks hold the row: fewer registers, more workgroups per CU
  // the steps of parallel layers with known addends (a re-entering addend or a list of rows: any)
  const int f = e || pick || cg || W < 4 * kThreads ? kAny
                : (a ? kHasA : 0) | (b ? kHasB : 0) | (c ? kHasC : 0) | (d ? kHasD : 0) | (bias ? kHasBias : 0) |
                      (my ? kHasExperts : 0);
#define RES_KNOWN(F) \
  if (f == (F)) {    \
    if (narrow) { RES(4, true, 4, F) } else { RES(4, true, 8, F) } \
    DX_CHECK_LAUNCH(); \
    return 0;        \
  }
  if (vec && ext) {
    RES_KNOWN(kHasB | kHasC | kHasD | kHasExperts)
    RES_KNOWN(kHasA | kHasExperts)
    RES_KNOWN(kHasB | kHasC | kHasD | kHasBias)
    RES_KNOWN(kHasA | kHasBias)
  }
#undef RES_KNOWN
  if (vec && ext && narrow) { RES(4, true, 4, kAny) }
  else if (vec && ext) { RES(4, true, 8, kAny) }
  else if (vec && narrow) { RES(4, false, 4, kAny) }
  else if (vec) { RES(4, false, 8, kAny) }
  else if (ext) { RES(1, true, 8, kAny) }
  else { RES(1, false, 8, kAny) }
#undef RES
  DX_CHECK_LAUNCH();
  return 0;
}

int dxm_act_mul(void* out, const void* gate, int64_t g_stride, const void* up, int64_t u_stride, int rows, int F,
                int64_t out_stride, int act, float limit, float alpha, float post, const float* gate_b,
                const float* up_b, const float* row_scale, int u_dv, int64_t u_head, int f32, hipStream_t st) {
  if (rows <= 0 || F <= 0) return 0;
  if (act < 0 || act > 6 || (act == 6 && (!up || !(limit > 0.f)))) return 1;
  if (u_dv < 0 || (u_dv && (!up || F % u_dv))) return 2;
  const int esz = f32 ? 4 : 2;
  const bool vec = F % 4 == 0 && g_stride % 4 == 0 && u_stride % 4 == 0 && out_stride % 4 == 0 && u_dv % 4 == 0 &&
                   u_head % 4 == 0 && (uintptr_t)gate % (4 * esz) == 0 && (uintptr_t)up % (4 * esz) == 0 &&
                   (uintptr_t)out % (4 * esz) == 0 && (uintptr_t)gate_b % 16 == 0 && (uintptr_t)up_b % 16 == 0;
  const int per = kThreads * (vec ? 4 : 1);
  const int gx = (F + per - 1) / per;
  constexpr int kRowsPer = 8;
  const bool many = (gate_b || up_b) && rows >= 2048;
  const int rows_per = many ? kRowsPer : 1;
  for (int r0 = 0; r0 < rows; r0 += 65535 * rows_per) {
    const int nr = rows - r0 < 65535 * rows_per ? rows - r0 : 65535 * rows_per, gy = (nr + rows_per - 1) / rows_per;
#define ACT_MUL(V, ROWS)                                                                                               \
  DISPATCH_T(f32, hipLaunchKernelGGL((act_mul_kernel<T, V, ROWS>), dim3(gx, gy), dim3(kThreads), 0, st,                \
                                     (T*)out + r0 * out_stride, (const T*)gate + r0 * g_stride, g_stride,              \
                                     up ? (const T*)up + r0 * u_stride : nullptr, u_stride, F, out_stride, act, limit, \
                                     alpha, post, gate_b, up_b, row_scale ? row_scale + r0 : nullptr, u_dv, u_head, nr))
    if (vec && many) { ACT_MUL(4, kRowsPer) }
    else if (vec) { ACT_MUL(4, 1) }
    else if (many) { ACT_MUL(1, kRowsPer) }
    else { ACT_MUL(1, 1) }
#undef ACT_MUL
  }
  DX_CHECK_LAUNCH();
  return 0;
}

int dxm_headprep_cache(void* x, int64_t x_stride, const int64_t* pos, const int64_t* slots, int rows, int n_q, int n_k,
                       int d, int k_off, const float* qw, const float* kw, float eps, float temp_coef,
                       double temp_every, void* kc, void* vc, int v_mode, int v_off, int v_w, const void* v_first,
                       int64_t vf_stride, float v_lambda, int f32, hipStream_t st) {
  if (rows <= 0) return 0;
  if (n_q < 0 || n_k < 0 || d < 1 || v_mode < 0 || v_mode > 2) return 1;
  if (n_k > 0 && !kc) return 2;
  if (v_mode != 0 && !vc) return 3;
  if (temp_coef != 0.f && !(temp_every > 0)) return 4;
  if (v_first && v_mode != 2) return 5;
  const int esz = f32 ? 4 : 2;
  const bool vec = d % 4 == 0 && k_off % 4 == 0 && x_stride % 4 == 0 && v_off % 4 == 0 && v_w % 4 == 0 &&
                   vf_stride % 4 == 0 && (uintptr_t)v_first % (4 * esz) == 0 &&
                   (uintptr_t)x % (4 * esz) == 0 && (uintptr_t)kc % (4 * esz) == 0 && (uintptr_t)vc % (4 * esz) == 0 &&
                   (uintptr_t)qw % 16 == 0 && (uintptr_t)kw % 16 == 0;
  // lanes per head vector: about two chunks of V elements per lane
  const int chunks = (d + (vec ? 4 : 1) - 1) / (vec ? 4 : 1);
  int lpv = 1;
  while (lpv < 64 && lpv * 2 < chunks) lpv <<= 1;
  if (vec) {
    DISPATCH_T(f32, hipLaunchKernelGGL((headprep_cache_kernel<T, 4>), dim3(rows), dim3(kThreads), 0, st, (T*)x,
                                       x_stride, pos, slots, n_q, n_k, d, k_off, qw, kw, eps, temp_coef, temp_every,
                                       (T*)kc, (T*)vc, v_mode, v_off, v_w, (const T*)v_first, vf_stride, v_lambda,
                                       lpv));
  } else {
    DISPATCH_T(f32, hipLaunchKernelGGL((headprep_cache_kernel<T, 1>), dim3(rows), dim3(kThreads), 0, st, (T*)x,
                                       x_stride, pos, slots, n_q, n_k, d, k_off, qw, kw, eps, temp_coef, temp_every,
                                       (T*)kc, (T*)vc, v_mode, v_off, v_w, (const T*)v_first, vf_stride, v_lambda,
                                       lpv));
  }
  DX_CHECK_LAUNCH();
  return 0;
}

int dxm_depth_mix(float* dst, float* stack, int64_t plane, int n, const float* w, const int64_t* rows, int n_rows,
                  float eps, const float* nw, void* out, const void* c, int64_t c_stride, const float* cw, int W,
                  int f32, hipStream_t st) {
  if (n_rows <= 0) return 0;
  if (n < 1 || W < 1 || !dst || !stack || !w || (out && !nw) || (c && !cw)) return 1;
  const int esz = f32 ? 4 : 2;
  auto al = [&](const void* p, int by) { return (uintptr_t)p % by == 0; };
  const bool vec = W % 4 == 0 && plane % 4 == 0 && c_stride % 4 == 0 && al(dst, 16) && al(stack, 16) && al(nw, 16) &&
                   al(out, 4 * esz) && al(c, 4 * esz) && al(cw, 16);
  if (vec) {
    DISPATCH_T(f32, hipLaunchKernelGGL((depth_mix_kernel<T, 4>), dim3(n_rows), dim3(kThreads), 0, st, dst, stack, plane,
                                       n, w, rows, eps, nw, (T*)out, (const T*)c, c_stride, cw, W));
  } else {
    DISPATCH_T(f32, hipLaunchKernelGGL((depth_mix_kernel<T, 1>), dim3(n_rows), dim3(kThreads), 0, st, dst, stack, plane,
                                       n, w, rows, eps, nw, (T*)out, (const T*)c, c_stride, cw, W));
  }
  DX_CHECK_LAUNCH();
  return 0;
}

int dxm_section_norm(void* out, const void* x, int64_t x_stride, const float* w, int rows, int n, float eps, int f32,
                     hipStream_t st) {
  if (rows <= 0) return 0;
  if (n < 1 || !out || !x) return 1;
  const int blocks = (rows + kThreads / 64 - 1) / (kThreads / 64);
  DISPATCH_T(f32, hipLaunchKernelGGL(section_norm_kernel<T>, dim3(blocks), dim3(kThreads), 0, st, (T*)out, (const T*)x,
                                     x_stride, w, rows, n, eps));
  DX_CHECK_LAUNCH();
  return 0;
}

int dxm_diff_combine(void* out, const float* a, int64_t n_vec, int dv, float lam, float post, float eps,
                     const void* gate, int64_t gate_stride, int H, int f32, hipStream_t st) {
  if (n_vec <= 0) return 0;
  if (gate && (H < 1 || n_vec % H)) return 1;
  const int64_t blocks = (n_vec + kThreads / 64 - 1) / (kThreads / 64);
  DISPATCH_T(f32, hipLaunchKernelGGL(diff_combine_kernel<T>, dim3((unsigned)blocks), dim3(kThreads), 0, st, (T*)out, a,
                                     n_vec, dv, lam, post, eps, (const T*)gate, gate_stride, H > 0 ? H : 1));
  DX_CHECK_LAUNCH();
  return 0;
}

}  // extern "C"
