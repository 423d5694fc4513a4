// Decode attention of plain grouped-query heads (softmax weights, causal or
// window mask, no score terms, up to 16 heads per key/value head) for gfx950:
// the same partition and workspace as group_decode (tile_attention.hip: one wave
// per row, K head and key part; merge_parts joins the parts), with the key loop
// laid out to keep loads in flight:
//   * tiles are the 64-key pieces of the pages (pages are multiples of 64 keys),
//     so a tile's rows are one scalar base plus lane constants;
//   * a tile's K rows go from memory straight into MFMA A fragments (a lane
//     reads 16 bytes of its key), its V rows through registers into a transposed,
//     swizzled LDS image;
//   * each half's registers are refilled with the next tile as soon as they are
//     free: K after the score products, V after it is written to LDS;
//   * masks apply to the first and last tile only; weights are the sum of two
//     bf16 numbers in the value product, scores and sums are fp32.
#include "recurrent.h"

namespace {

struct StreamArgs {
  const bf16_t* q;
  int64_t q_stride;
  const bf16_t* kc;
  const bf16_t* vc;
  float* ws;  // [rows, n_qh, parts, 2 + dv]
  const int64_t* pos;
  const int* seq;  // null: row i is sequence i
  const int* bt;
  int bt_stride, bs_shift;
  int n_qh, maps, group;
  int Wk, Wv;
  float scale_log2;
  int size;  // window (0: causal)
  int parts;
};

// element offset of 16-byte piece pc of row r in the [dv][64 keys] image
__device__ __forceinline__ int voff(int r, int pc) { return r * 64 + ((pc ^ ((r >> 1) & 7)) << 3); }

template <int D, int DV>
__global__ void __launch_bounds__(64, 2) stream_decode_kernel(StreamArgs a) {
  constexpr int NK = D / 32, NC = DV / 16, CH = DV / 8, VI = 16 * CH / 64;  // VI: V items (4 keys x 8 columns) per lane
  static_assert(D % 32 == 0 && 16 * CH % 64 == 0, "whole fragments, whole V items");
  __shared__ __attribute__((aligned(16))) bf16_t Vt[DV * 64];
  const int lane = threadIdx.x, c16 = lane & 15, g4 = lane >> 4;
  const int gm = blockIdx.x, row = blockIdx.y, part = blockIdx.z;
  const int g = gm / a.maps, m = gm - g * a.maps;
  const int p = __builtin_amdgcn_readfirstlane((int)a.pos[row]);
  const int lo = a.size && p - a.size + 1 > 0 ? p - a.size + 1 : 0;
  const int first = lo >> 6, n_tiles = (p >> 6) - first + 1;
  const int tpp = (n_tiles + a.parts - 1) / a.parts;
  const int t0 = first + part * tpp, t1 = min(t0 + tpp, first + n_tiles);
  const int* bt = a.bt + (int64_t)__builtin_amdgcn_readfirstlane(a.seq ? a.seq[row] : row) * a.bt_stride;
  const bool okh = c16 < a.group;
  const int qh = (g * a.group + (okh ? c16 : 0)) * a.maps + m;
  bf16x8_t qf[NK];
#pragma unroll
  for (int ks = 0; ks < NK; ++ks) {
    const raw_u32x4 zero{0u, 0u, 0u, 0u};
    qf[ks] = __builtin_bit_cast(bf16x8_t, okh ? *reinterpret_cast<const raw_u32x4*>(
        a.q + (int64_t)row * a.q_stride + (int64_t)qh * D + 32 * ks + 8 * g4) : zero);
  }
  // lane constants inside a tile: the K fragment of key c16, the V item (keys 4 vk .. + 3, columns 8 vc8 .. + 7)
  const int vk = lane / CH, vc8 = lane % CH;
  const bf16_t* kl = a.kc + (int64_t)gm * D + (int64_t)c16 * a.Wk + 8 * g4;
  const bf16_t* vl = a.vc + (int64_t)g * DV + (int64_t)(4 * vk) * a.Wv + 8 * vc8;
  raw_u32x4 kr[4][NK], vr[VI][4];
  auto slot = [&](int t) -> int64_t {
    const int j = t << 6;
    return ((int64_t)bt[j >> a.bs_shift] << a.bs_shift) + (j & ((1 << a.bs_shift) - 1));
  };
  auto fetch_k = [&](int64_t base) {
    const bf16_t* src = kl + base * a.Wk;
#pragma unroll
    for (int kb = 0; kb < 4; ++kb)
#pragma unroll
      for (int ks = 0; ks < NK; ++ks)
        kr[kb][ks] = __builtin_nontemporal_load(reinterpret_cast<const raw_u32x4*>(src + (int64_t)kb * 16 * a.Wk + 32 * ks));
  };
  auto fetch_v = [&](int64_t base) {
    const bf16_t* src = vl + base * a.Wv;
#pragma unroll
    for (int i = 0; i < VI; ++i)
#pragma unroll
      for (int k = 0; k < 4; ++k)
        vr[i][k] = __builtin_nontemporal_load(
            reinterpret_cast<const raw_u32x4*>(src + (int64_t)(4 * (64 / CH) * i + k) * a.Wv));
  };
  float mx = -INFINITY, lsum = 0.f;  // log2 units
  f32x4 O[NC];
#pragma unroll
  for (int cb = 0; cb < NC; ++cb) O[cb] = f32x4{0.f, 0.f, 0.f, 0.f};
  int64_t next = 0;
  if (t0 < t1) {
    const int64_t base = slot(t0);
    fetch_k(base);
    fetch_v(base);
    next = slot(min(t0 + 1, t1 - 1));
  }
  for (int t = t0; t < t1; ++t) {
    const bool more = t + 1 < t1;
    f32x4 S[4];
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) {
      S[kb] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < NK; ++ks)
        S[kb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, kr[kb][ks]), qf[ks], S[kb], 0, 0, 0);
    }
    if (more) fetch_k(next);
    if (t == (p >> 6)) {  // the page's rows behind the query: stale values must not meet a zero weight
#pragma unroll
      for (int i = 0; i < VI; ++i)
#pragma unroll
        for (int k = 0; k < 4; ++k)
          if ((t << 6) + 4 * (vk + 64 / CH * i) + k > p) vr[i][k] = raw_u32x4{0u, 0u, 0u, 0u};
    }
    __syncthreads();  // (one wave: orders the image's reads and writes)
#pragma unroll
    for (int i = 0; i < VI; ++i) {
      const int kg = vk + 64 / CH * i;  // keys of a 32-key half are stored in the order the weights' fragments have them
      const int pc = 4 * (kg >> 3) + (kg & 3), hf = 4 * ((kg >> 2) & 1);
#pragma unroll
      for (int w = 0; w < 4; ++w) {
        uint2 ev, od;
        ev.x = (vr[i][0][w] & 0xffffu) | (vr[i][1][w] << 16);
        ev.y = (vr[i][2][w] & 0xffffu) | (vr[i][3][w] << 16);
        od.x = (vr[i][0][w] >> 16) | (vr[i][1][w] & 0xffff0000u);
        od.y = (vr[i][2][w] >> 16) | (vr[i][3][w] & 0xffff0000u);
        *reinterpret_cast<uint2*>(Vt + voff(8 * vc8 + 2 * w, pc) + hf) = ev;
        *reinterpret_cast<uint2*>(Vt + voff(8 * vc8 + 2 * w + 1, pc) + hf) = od;
      }
    }
    if (more) {
      fetch_v(next);
      next = slot(min(t + 2, t1 - 1));
    }
    // scores in log2 units: lane column = head, rows = keys 16 kb + 4 g4 + r
#pragma unroll
    for (int kb = 0; kb < 4; ++kb)
#pragma unroll
      for (int r = 0; r < 4; ++r) S[kb][r] *= a.scale_log2;
    if (t == first || t == (p >> 6)) {
#pragma unroll
      for (int kb = 0; kb < 4; ++kb)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int j = (t << 6) + 16 * kb + 4 * g4 + r;
          if (j < lo || j > p) S[kb][r] = -INFINITY;
        }
    }
    float mloc = S[0][0];
#pragma unroll
    for (int kb = 0; kb < 4; ++kb)
#pragma unroll
      for (int r = 0; r < 4; ++r) mloc = fmaxf(mloc, S[kb][r]);
    mloc = fmaxf(mloc, __shfl_xor(mloc, 16, 64));
    mloc = fmaxf(mloc, __shfl_xor(mloc, 32, 64));
    const float mn = fmaxf(mx, mloc);  // finite: every visited tile holds a visible key
    if (__any(mn > mx)) {
      const float alpha = fast_exp2(mx - mn);
      mx = mn;
      lsum *= alpha;
#pragma unroll
      for (int cb = 0; cb < NC; ++cb)
#pragma unroll
        for (int r = 0; r < 4; ++r) O[cb][r] *= alpha;
    }
    bf16x8_t Ph[2], Pl[2];
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      float w8[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        w8[e] = fast_exp2(S[2 * kk + e / 4][e % 4] - mn);
        lsum += w8[e];
      }
      raw_u32x4 hi, lw;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        hi[e] = pack_bf16x2(w8[2 * e], w8[2 * e + 1]);
        lw[e] = pack_bf16x2(w8[2 * e] - bf16lo(hi[e]), w8[2 * e + 1] - bf16hi(hi[e]));
      }
      Ph[kk] = __builtin_bit_cast(bf16x8_t, hi);
      Pl[kk] = __builtin_bit_cast(bf16x8_t, lw);
    }
    __syncthreads();
#pragma unroll
    for (int kk = 0; kk < 2; ++kk)
#pragma unroll
      for (int cb = 0; cb < NC; ++cb) {
        const bf16x8_t vf = __builtin_bit_cast(bf16x8_t, *reinterpret_cast<const raw_u32x4*>(Vt + voff(16 * cb + c16, 4 * kk + g4)));
        O[cb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, Ph[kk], O[cb], 0, 0, 0);
        O[cb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, Pl[kk], O[cb], 0, 0, 0);
      }
  }
  lsum += __shfl_xor(lsum, 16, 64);
  lsum += __shfl_xor(lsum, 32, 64);
  if (!okh) return;
  float* w = a.ws + (((int64_t)row * a.n_qh + qh) * a.parts + part) * (2 + DV);
  if (g4 == 0) {
    w[0] = mx * 0.6931471805599453f;
    w[1] = lsum;
  }
#pragma unroll
  for (int cb = 0; cb < NC; ++cb)
#pragma unroll
    for (int r = 0; r < 4; ++r) w[2 + cb * 16 + 4 * g4 + r] = O[cb][r];
}

}  // namespace

extern "C" {

// 1 when the kernel takes these heads: widths it is instantiated for, pages of whole 64-key tiles
int dxm_stream_decode_ok(int d, int dv, int group, int bs, int mask) {
  return ((d == 128 && dv == 128) || (d == 64 && dv == 64)) && group >= 1 && group <= 16 && bs >= 64 &&
         (bs & (bs - 1)) == 0 && (mask == 0 || mask == 1);
}

int dxm_stream_decode(float* ws, const void* q, int64_t q_stride, const void* kc, const void* vc, const int64_t* pos,
                      const int* seq, const int* bt, int bt_stride, int bs, int rows, int n_qh, int maps, int group, int d,
                      int dv, int Wk, int Wv, float scale, int mask, int size, int parts, hipStream_t st) {
  if (rows <= 0) return 0;
  if (!dxm_stream_decode_ok(d, dv, group, bs, mask)) return 2;
  if (n_qh < 1 || maps < 1 || n_qh % maps || (n_qh / maps) % group || rows > 65535) return 1;
  if ((mask && size < 1) || parts < 1 || parts > 65535 || !(scale > 0.f)) return 3;
  if (!ws || Wk % 8 || Wv % 8 || q_stride % 8 || (uintptr_t)q % 16 || (uintptr_t)kc % 16 || (uintptr_t)vc % 16) return 4;
  StreamArgs a{(const bf16_t*)q, q_stride, (const bf16_t*)kc, (const bf16_t*)vc, ws, pos, seq, bt, bt_stride,
               __builtin_ctz((unsigned)bs), n_qh, maps, group, Wk, Wv, scale * 1.4426950408889634f, mask ? size : 0, parts};
  const dim3 grid(n_qh / group, rows, parts);
  if (d == 128) hipLaunchKernelGGL((stream_decode_kernel<128, 128>), grid, dim3(64), 0, st, a);
  else hipLaunchKernelGGL((stream_decode_kernel<64, 64>), grid, dim3(64), 0, st, a);
  DX_CHECK_LAUNCH();
  return 0;
}

}  // extern "C"
