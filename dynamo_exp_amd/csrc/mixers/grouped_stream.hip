// Grouped GEMM of few rows per expert (a decode step of a mixture of experts), for gfx950: the experts'
// weights stream from HBM once, straight into matrix-core fragments; the handful of activation rows comes
// from L2.  Same meaning as grouped_gemm (moe.hip): for expert e, rows r of its run offsets[e] ..
// offsets[e + 1],
//     out[dst(r), :] = a[src(r), :] @ w[e]^T        src(r) = order[r] / top (gather) or r, dst(r) = order[r] (scatter) or r
// and with glu (weights in blocks of 32 gate rows and their 32 up rows) out = silu(gate) * up, [R, N / 2].
//
// A workgroup (4 waves) takes 32 weight rows of one expert -- 16 gate and their 16 up rows with glu -- and
// all rows of the expert, 32 at a time; the waves share the width in pieces of 64 and their partial
// sums are added in LDS in wave order.  v_mfma_f32_16x16x32_bf16 with the weights as A (lane: one weight row,
// 32 contiguous bytes of each piece: four lanes read a whole line) and the activations as B in the same
// order, so nothing is shuffled; D pieces are in flight per wave.
#include "../kernels/common.h"

namespace {

typedef uint32_t gs_raw4 __attribute__((ext_vector_type(4)));
typedef __bf16 gs_bf16x8 __attribute__((ext_vector_type(8)));

struct StreamGemmArgs {
  bf16_t* out;
  const bf16_t* a;
  int64_t a_stride;
  const bf16_t* w;  // [E, N, K]
  const int* order;
  const int* offsets;
  int N, K, top, gather, scatter;
};

// MT: 16-row activation tiles, D: pieces in flight
template <int MT, int D, bool GLU>
__device__ __forceinline__ void stream_pass(const StreamGemmArgs& g, int e, int lo, int rows, int j, f32x4* red) {
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, c16 = lane & 15, g4 = lane >> 4;
  // first weight rows of the two 16-row tiles
  const int n0 = GLU ? 64 * (j >> 1) + 16 * (j & 1) : 32 * j;
  const int n1 = GLU ? n0 + 32 : n0 + 16;
  const bf16_t* wp[2];
#pragma unroll
  for (int t = 0; t < 2; ++t) {
    const int n = (t ? n1 : n0) + c16;
    wp[t] = g.w + ((int64_t)e * g.N + (n < g.N ? n : 0)) * g.K + 16 * g4 + 64 * wave;
  }
  const bf16_t* ap[MT];
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    const int r = lo + min(16 * m + c16, rows - 1);  // rows past the last repeat it and are not stored
    ap[m] = g.a + (int64_t)(g.gather ? g.order[r] / g.top : r) * g.a_stride + 16 * g4 + 64 * wave;
  }
  f32x4 C[2][MT];
#pragma unroll
  for (int t = 0; t < 2; ++t)
#pragma unroll
    for (int m = 0; m < MT; ++m) C[t][m] = f32x4{0.f, 0.f, 0.f, 0.f};
  gs_raw4 W[D][2][2], A[D][MT][2];
  const int np = (g.K / 64 - wave + 3) / 4;  // this wave's pieces: wave, wave + 4, ...
  auto fetch = [&](int s, int p) {
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int h = 0; h < 2; ++h)
        W[s][t][h] = __builtin_nontemporal_load(reinterpret_cast<const gs_raw4*>(wp[t] + (int64_t)p * 256 + 8 * h));
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int h = 0; h < 2; ++h) A[s][m][h] = *reinterpret_cast<const gs_raw4*>(ap[m] + (int64_t)p * 256 + 8 * h);
  };
  auto use = [&](int s) {
#pragma unroll
    for (int h = 0; h < 2; ++h)
#pragma unroll
      for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int m = 0; m < MT; ++m)
          C[t][m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(gs_bf16x8, W[s][t][h]),
                                                            __builtin_bit_cast(gs_bf16x8, A[s][m][h]), C[t][m], 0, 0, 0);
  };
  if (np > 0) {
    // workgroups start at different pieces: rows a power of two apart would otherwise meet on the same channels
    const int skew = (j * 5 + e * 3) % np;
    auto at = [&](int p) {
      p = min(p, np - 1) + skew;
      return p < np ? p : p - np;
    };
#pragma unroll
    for (int s = 0; s < D; ++s) fetch(s, at(s));
    for (int p = 0; p < np; p += D) {  // a slot is refilled as it is used (at the end: with the last piece again)
#pragma unroll
      for (int s = 0; s < D; ++s) {
        if (p + s < np) use(s);
        fetch(s, at(p + D + s));
      }
    }
  }
  // C[t][m]: weight rows n_t + 4 g4 .. + 3 of activation row 16 m + c16
#pragma unroll
  for (int t = 0; t < 2; ++t)
#pragma unroll
    for (int m = 0; m < MT; ++m) red[((wave * 2 + t) * MT + m) * 64 + lane] = C[t][m];
  __syncthreads();
  constexpr int kFrags = GLU ? MT : 2 * MT;
  for (int f = wave; f < kFrags; f += 4) {
    const int t = GLU ? 0 : f / MT, m = GLU ? f : f - t * MT;
    auto total = [&](int tt) {
      f32x4 s = red[(tt * MT + m) * 64 + lane];
#pragma unroll
      for (int wv = 1; wv < 4; ++wv) s += red[((wv * 2 + tt) * MT + m) * 64 + lane];
      return s;
    };
    f32x4 v = total(t);
    int n = (t ? n1 : n0) + 4 * g4, No = g.N;
    if constexpr (GLU) {
      const f32x4 u = total(1);
#pragma unroll
      for (int i = 0; i < 4; ++i) v[i] = v[i] / (1.f + __expf(-v[i])) * u[i];
      n = 16 * j + 4 * g4;
      No = g.N / 2;
    }
    const int r = 16 * m + c16;
    if (r >= rows || n >= No) continue;
    const int64_t dst = g.scatter ? g.order[lo + r] : lo + r;
    *reinterpret_cast<uint2*>(g.out + dst * No + n) = uint2{pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3])};
  }
  __syncthreads();  // (red is free again)
}

constexpr int kMT = 2, kDepth = 2;
template <bool GLU>
__global__ void __launch_bounds__(256, 4) stream_grouped_gemm_kernel(StreamGemmArgs g) {
  __shared__ __attribute__((aligned(16))) f32x4 red[4 * 2 * kMT * 64];
  const int e = blockIdx.y, j = blockIdx.x;
  const int lo = g.offsets[e], hi = g.offsets[e + 1];
  for (int r = lo; r < hi; r += 16 * kMT) stream_pass<kMT, kDepth, GLU>(g, e, r, min(hi - r, 16 * kMT), j, red);
}

}  // namespace

extern "C" {

// 1 when stream_grouped_gemm takes the shape: whole 64-wide pieces, whole 32-row blocks of weights
int dxm_stream_grouped_ok(int N, int K) { return N >= 32 && N % 32 == 0 && K >= 64 && K % 64 == 0; }

int dxm_stream_grouped_gemm(void* out, const void* a, int64_t a_stride, const void* w, const int* order,
                            const int* offsets, int R, int E, int N, int K, int top, int gather, int scatter, int glu,
                            hipStream_t st) {
  if (R <= 0) return 0;
  if (E < 1 || E > 65535 || top < 1 || !dxm_stream_grouped_ok(N, K) || (glu && N % 64)) return 1;
  if (!out || !a || !w || !order || !offsets || a_stride % 8 || (uintptr_t)a % 16 || (uintptr_t)w % 16 ||
      (uintptr_t)out % 8)
    return 2;
  const StreamGemmArgs g{(bf16_t*)out, (const bf16_t*)a, a_stride, (const bf16_t*)w, order, offsets, N, K, top, gather, scatter};
  const dim3 grid((unsigned)(N / 32), (unsigned)E);
  if (glu) hipLaunchKernelGGL(stream_grouped_gemm_kernel<true>, grid, dim3(256), 0, st, g);
  else hipLaunchKernelGGL(stream_grouped_gemm_kernel<false>, grid, dim3(256), 0, st, g);
  DX_CHECK_LAUNCH();
  return 0;
}

}  // extern "C"
