// Chunked, matrix-core form of the linear recurrences for prompt portions in
// bf16 (the token-by-token form and the definitions: linear_scan.hip).  One
// workgroup walks a sequence's rows of one (head, 64 columns) chunk by chunk;
// each of its four product waves owns 16 columns p of the running matrix, which
// stays in fp32 accumulators for the whole walk.  With E(a, b) the decay from token a to
// token b, a chunk is three products,
//     o_t = E(start, t) S^T q_t + sum_(s <= t) (q_t . E(s, t) k_s) u_s v_s,
//     S  <- E(start, end) S + sum_s (E(s, end) u_s k_s) v_s^T.
// q, k, v are bf16 as projected; whatever carries a decay, a step size or the
// state enters its product as the sum of two bf16 numbers (hi + lo, 16 bits of
// mantissa), and all sums are fp32.
//
// v_mfma_f32_16x16x32_bf16: lane l = 16 g + c holds row (column) c of A (B) at
// eight k-slots of its group g, and of the result column c, rows 4 g .. 4 g + 3.
// Which k a slot stands for is free as long as A and B agree: with slots {4 g +
// 0..3, 16 + 4 g + 0..3} a pair of result tiles of S is an A operand as it lies in
// the registers.
#include "linear_scan.h"

namespace {

__device__ __forceinline__ bf16x8_t as_bf16x8(const raw_u32x4& v) { return __builtin_bit_cast(bf16x8_t, v); }

// eight k-slots from one 16-byte run / from two 8-byte runs 16 elements apart
__device__ __forceinline__ bf16x8_t frag8(const bf16_t* p) { return as_bf16x8(*reinterpret_cast<const raw_u32x4*>(p)); }
__device__ __forceinline__ bf16x8_t frag4_4(const bf16_t* p, const bf16_t* p16) {
  const uint2 a = *reinterpret_cast<const uint2*>(p), b = *reinterpret_cast<const uint2*>(p16);
  return as_bf16x8(raw_u32x4{a.x, a.y, b.x, b.y});
}

// hi + lo bf16 parts of four floats
__device__ __forceinline__ void split4(const float* v, uint2& hi, uint2& lo) {
  hi.x = pack_bf16x2(v[0], v[1]);
  hi.y = pack_bf16x2(v[2], v[3]);
  lo.x = pack_bf16x2(v[0] - bf16lo(hi.x), v[1] - bf16hi(hi.x));
  lo.y = pack_bf16x2(v[2] - bf16lo(hi.y), v[3] - bf16hi(hi.y));
}
__device__ __forceinline__ void split8(const float* v, raw_u32x4& hi, raw_u32x4& lo) {
  uint2 h0, l0, h1, l1;
  split4(v, h0, l0);
  split4(v + 4, h1, l1);
  hi = raw_u32x4{h0.x, h0.y, h1.x, h1.y};
  lo = raw_u32x4{l0.x, l0.y, l1.x, l1.y};
}

// four rows of eight elements each -> element e of all four rows, 8 bytes
__device__ __forceinline__ uint2 column4(const raw_u32x4* r, int e) {
  const int w = e >> 1;
  if (e & 1)
    return uint2{(r[0][w] >> 16) | (r[1][w] & 0xffff0000u), (r[2][w] >> 16) | (r[3][w] & 0xffff0000u)};
  return uint2{(r[0][w] & 0xffffu) | (r[1][w] << 16), (r[2][w] & 0xffffu) | (r[3][w] << 16)};
}

__device__ __forceinline__ f32x4 mfma32(bf16x8_t a, bf16x8_t b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}

// inclusive sums over the 64 lanes: within rows of 16, then the last lane of a row (of a half) into the next
template <int CTRL, int ROWS> __device__ __forceinline__ float dpp_rows(float v) {
  return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, ROWS, 0xf, false));
}
__device__ __forceinline__ float row_scan_sum(float v) {
  v += dpp_f<0x111>(v);
  v += dpp_f<0x112>(v);
  v += dpp_f<0x114>(v);
  v += dpp_f<0x118>(v);
  return v;
}
__device__ __forceinline__ float wave_scan_sum(float v) {
  v = row_scan_sum(v);
  v += dpp_rows<0x142, 0xa>(v);
  v += dpp_rows<0x143, 0xc>(v);
  return v;
}

constexpr float kLog2e = 1.4426950408889634f;
constexpr int kPB = 64;  // columns of a workgroup

// the workgroup's sequence: its rows and slot; false: nothing to do
struct Walk {
  int r0, n, h, hq, col0, slot;
  bool fresh;
};
__device__ __forceinline__ bool open_walk(const ScanArgs& g, Walk& w) {
  const int s = blockIdx.z;
  w.h = blockIdx.y;
  w.hq = w.h / g.qk_rep;
  w.col0 = blockIdx.x * kPB;
  w.r0 = g.seq_rows[s];
  w.n = g.seq_rows[s + 1] - w.r0;
  if (w.n < g.min_rows || w.r0 < 0 || w.r0 + w.n > g.T) return false;
  w.slot = g.slots[s];
  if (w.slot < 0 || w.slot >= g.n_slots) {  // padding: zeros out, no state touched
    for (int i = threadIdx.x; i < w.n * kPB; i += blockDim.x)
      g.out[(int64_t)(w.r0 + i / kPB) * g.H * g.dv + (int64_t)w.h * g.dv + w.col0 + i % kPB] = 0.f;
    return false;
  }
  w.fresh = g.pos[w.r0] == 0;
  return true;
}

// ---------------------------------------------------------------------------
// One decay per token and head (kFixed, kStep): chunks of 64 tokens.  The decays
// between the chunk's tokens form a [64, 64] matrix of their own, which
// multiplies the q k^T products element by element.  Four waves (the upper ones)
// stage a chunk's rows and form these weights, 16 token rows each (only the tiles
// on and below the diagonal), one chunk ahead, in the other half of the
// double-buffered LDS; the lower four form the outputs and walk the state.
// LDS rows are cut into 16-byte pieces that an XOR with row bits moves around, so that the 16 rows a fragment
// read touches (whichever lane groups the hardware serves together) and the staging writes (rows 4 apart) lie on
// different banks: element offset of piece pc of row r in a [..][DK] and in a [..][64] image.
template <int DK> __device__ __forceinline__ int koff(int r, int pc) {
  if constexpr (DK == 128) return r * 128 + ((pc ^ ((r & 12) | ((r & 3) ^ (r >> 4)))) << 3);
  return r * (DK + 8) + (pc << 3);  // (narrow rows: padding)
}
__device__ __forceinline__ int soff(int r, int pc) { return r * 64 + ((pc ^ ((r >> 1) & 7)) << 3); }

template <int DK> struct ChunkBuf {
  bf16_t q[64 * (DK == 128 ? DK : DK + 8)];  // [t][n]
  bf16_t kT[DK * 64];                        // k [n][s]
  bf16_t vT[kPB * 64];                       // v [p][s]
  bf16_t m[2][64 * 64];                      // hi, lo of the pair weights [t][s]
  float L[64], u[64], w[64];  // log2 decay since the start, step, step x decay to the end
};

template <int DK, int MODE>
__global__ void __launch_bounds__(512, 2) chunk_scan_kernel(ScanArgs g) {
  constexpr int Q = 64;                       // tokens per chunk
  constexpr int NO = DK / 8, NI = 16 * NO;    // staged items of q / k: 4 tokens x 8 channels
  constexpr int NM = DK / 16, NK = DK / 32;
  static_assert(NI <= 256 && DK % 32 == 0, "one staged item per thread");
  __shared__ __attribute__((aligned(16))) ChunkBuf<DK> bufs[2];
  __shared__ __attribute__((aligned(16))) bf16_t ks[sizeof(bufs[0].q) / sizeof(bf16_t)];  // k [s][n]
  Walk w;
  if (!open_walk(g, w)) return;
  const bool former = threadIdx.x >= 256;
  const int tid = threadIdx.x & 255, wave = tid >> 6, c16 = tid & 15, g4 = (tid & 63) >> 4;

  if (former) {  // ---- stage the chunks' rows; form the pair weights
    const int sq = tid & 15, oc = tid >> 4;  // token quad, channel octet
    // the thread's first row of the chunk being fetched
    const bf16_t* q = (const bf16_t*)g.q + (int64_t)(w.r0 + 4 * sq) * g.qs + (int64_t)w.hq * DK + 8 * oc;
    const bf16_t* k = (const bf16_t*)g.k + (int64_t)(w.r0 + 4 * sq) * g.ks + (int64_t)w.hq * DK + 8 * oc;
    const bf16_t* v = (const bf16_t*)g.v + (int64_t)(w.r0 + 4 * sq) * g.vs + (int64_t)w.h * g.dv + w.col0 + 8 * oc;
    const float skip = g.skip ? g.skip[w.h] : 0.f, qsc = g.q_scale;
    const float fixed_l2 = MODE == kFixed ? fmaxf(log2f(g.decay[w.h]), -1e6f) : 0.f;
    bf16_t rg = 0;  // step logit of token tid (first wave)
    const bf16_t* gl = MODE == kStep ? (const bf16_t*)g.g + (int64_t)w.r0 * g.gs + w.h : nullptr;
    const float g_bias = MODE == kStep && g.g_bias ? g.g_bias[w.h] : 0.f;
    const float rate_l2 = MODE == kStep ? -g.rate[w.h] * kLog2e : 0.f;
    raw_u32x4 rq[4], rk[4], rv[4];
    auto fetch = [&](int t0) {
      const raw_u32x4 zero{0u, 0u, 0u, 0u};
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const bool ok = t0 + 4 * sq + i < w.n;
        rq[i] = (NI == 256 || tid < NI) && ok ? *reinterpret_cast<const raw_u32x4*>(q + i * g.qs) : zero;
        rk[i] = (NI == 256 || tid < NI) && ok ? *reinterpret_cast<const raw_u32x4*>(k + i * g.ks) : zero;
        rv[i] = tid < 128 && ok ? *reinterpret_cast<const raw_u32x4*>(v + i * g.vs) : zero;
      }
      q += Q * g.qs;
      k += Q * g.ks;
      v += Q * g.vs;
      if (MODE == kStep && tid < Q && t0 + tid < w.n) rg = gl[(int64_t)(t0 + tid) * g.gs];
    };
    auto stage = [&](ChunkBuf<DK>& b, int t0) {
      if (NI == 256 || tid < NI) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          *reinterpret_cast<raw_u32x4*>(b.q + koff<DK>(4 * sq + i, oc)) = rq[i];
          *reinterpret_cast<raw_u32x4*>(ks + koff<DK>(4 * sq + i, oc)) = rk[i];
        }
#pragma unroll
        for (int e = 0; e < 8; ++e)
          *reinterpret_cast<uint2*>(b.kT + soff(8 * oc + e, sq >> 1) + 4 * (sq & 1)) = column4(rk, e);
      }
      if (tid < 128) {
#pragma unroll
        for (int e = 0; e < 8; ++e)
          *reinterpret_cast<uint2*>(b.vT + soff(8 * oc + e, sq >> 1) + 4 * (sq & 1)) = column4(rv, e);
      }
      if (tid < Q) {  // one wave: log decays since the chunk's start (inclusive scan)
        const bool ok = t0 + tid < w.n;
        float u = ok ? 1.f : 0.f, L = ok ? fixed_l2 : 0.f;
        if (MODE == kStep && ok) {
          u = softplusf_(bf16_to_f32(rg) + g_bias);
          L = rate_l2 * u;
        }
        L = wave_scan_sum(L);
        u *= g.k_scale;
        b.L[tid] = L;
        b.u[tid] = u;
        const float Lend = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, L), 63));
        b.w[tid] = u * fast_exp2(Lend - L);
      }
    };
    auto weigh = [&](ChunkBuf<DK>& b) {  // 16 query tokens per wave: (q_t . k_s) E(s, t) u_s
      const int t = 16 * wave + c16;
      bf16x8_t cq[NK];
#pragma unroll
      for (int kk = 0; kk < NK; ++kk) cq[kk] = frag8(b.q + koff<DK>(t, 4 * kk + g4));
      const float Lt = b.L[t];
      for (int j = 0; j <= (wave | 1); ++j) {  // (an even wave's last half fragment is zero)
        float m4[4] = {0.f, 0.f, 0.f, 0.f};
        const int s0 = 16 * j + 4 * g4;
        if (j <= wave) {
          f32x4 a{0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int kk = 0; kk < NK; ++kk) a = mfma32(frag8(ks + koff<DK>(16 * j + c16, 4 * kk + g4)), cq[kk], a);
          const f32x4 L4 = *reinterpret_cast<const f32x4*>(b.L + s0), u4 = *reinterpret_cast<const f32x4*>(b.u + s0);
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            if (s0 + r <= t) m4[r] = a[r] * fast_exp2(Lt - L4[r]) * u4[r] * qsc;
            if (s0 + r == t) m4[r] += skip;
          }
        }
        uint2 hi, lo;
        split4(m4, hi, lo);
        *reinterpret_cast<uint2*>(b.m[0] + soff(t, s0 >> 3) + (s0 & 7)) = hi;
        *reinterpret_cast<uint2*>(b.m[1] + soff(t, s0 >> 3) + (s0 & 7)) = lo;
      }
    };
    fetch(0);
    stage(bufs[0], 0);
    __syncthreads();  // chunk 0 is staged
    fetch(Q);
    weigh(bufs[0]);
    for (int t0 = 0, cur = 0; t0 < w.n; t0 += Q, cur ^= 1) {
      const bool more = t0 + Q < w.n;
      __syncthreads();  // chunk t0 is weighed; the other half is consumed
      if (more) stage(bufs[cur ^ 1], t0 + Q);
      __syncthreads();  // chunk t0 + Q is staged
      if (more) {
        fetch(t0 + 2 * Q);
        weigh(bufs[cur ^ 1]);
      }
    }
    return;
  }

  // ---- outputs and state.  (The barriers of the two roles pair up: one in front, two per chunk.)
  float* sp = g.state + (((int64_t)w.slot * g.H + w.h) * g.dv + w.col0 + 16 * wave + c16) * DK + 4 * g4;
  f32x4 S[NM];
#pragma unroll
  for (int m = 0; m < NM; ++m) S[m] = w.fresh ? f32x4{0.f, 0.f, 0.f, 0.f} : *reinterpret_cast<const f32x4*>(sp + 16 * m);
  const float qsc = g.q_scale;
  const int p = 16 * wave + c16;
  __syncthreads();
  for (int t0 = 0, cur = 0; t0 < w.n; t0 += Q, cur ^= 1) {
    __syncthreads();
    const ChunkBuf<DK>& b = bufs[cur];
    bf16x8_t xf[2], Sh[NK], Sl[NK];
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) xf[kk] = frag8(b.vT + soff(p, 4 * kk + g4));
#pragma unroll
    for (int kk = 0; kk < NK; ++kk) {
      float s8[8];
#pragma unroll
      for (int e = 0; e < 4; ++e) s8[e] = S[2 * kk][e], s8[4 + e] = S[2 * kk + 1][e];
      raw_u32x4 hi, lo;
      split8(s8, hi, lo);
      Sh[kk] = as_bf16x8(hi);
      Sl[kk] = as_bf16x8(lo);
    }
    auto output = [&](int tt) {  // 16 tokens x the wave's 16 columns
      if (t0 + 16 * tt >= w.n) return;
      const int t = 16 * tt + c16;
      f32x4 a{0.f, 0.f, 0.f, 0.f}, a1{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < NK; ++kk) {
        const bf16x8_t cf = frag4_4(b.q + koff<DK>(t, 4 * kk + (g4 >> 1)) + 4 * (g4 & 1),
                                    b.q + koff<DK>(t, 4 * kk + 2 + (g4 >> 1)) + 4 * (g4 & 1));
        a = mfma32(Sh[kk], cf, a);
        a1 = mfma32(Sl[kk], cf, a1);
      }
      const float e = fast_exp2(b.L[t]) * qsc;
#pragma unroll
      for (int r = 0; r < 4; ++r) a[r] = (a[r] + a1[r]) * e, a1[r] = 0.f;
#pragma unroll
      for (int kk = 0; kk <= tt / 2; ++kk) {
        a = mfma32(xf[kk], frag8(b.m[0] + soff(t, 4 * kk + g4)), a);
        a1 = mfma32(xf[kk], frag8(b.m[1] + soff(t, 4 * kk + g4)), a1);
      }
      if (t0 + t < w.n)
        *reinterpret_cast<f32x4*>(g.out + ((int64_t)(w.r0 + t0 + t) * g.H + w.h) * g.dv + w.col0 + 16 * wave + 4 * g4) =
            f32x4{a[0] + a1[0], a[1] + a1[1], a[2] + a1[2], a[3] + a1[3]};
    };
    output(0);
    output(1);
    __syncthreads();
    output(2);
    output(3);
    const float eq = fast_exp2(b.L[Q - 1]);
    bf16x8_t xh[2], xl[2];
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      float x8[8];
      chunk_to_f32<bf16_t>(__builtin_bit_cast(raw_u32x4, xf[kk]), x8);
#pragma unroll
      for (int e = 0; e < 8; ++e) x8[e] *= b.w[32 * kk + 8 * g4 + e];
      raw_u32x4 hi, lo;
      split8(x8, hi, lo);
      xh[kk] = as_bf16x8(hi);
      xl[kk] = as_bf16x8(lo);
    }
#pragma unroll
    for (int m = 0; m < NM; ++m) {
#pragma unroll
      for (int r = 0; r < 4; ++r) S[m][r] *= eq;
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) {
        const bf16x8_t kf = frag8(b.kT + soff(16 * m + c16, 4 * kk + g4));
        S[m] = mfma32(kf, xh[kk], S[m]);
        S[m] = mfma32(kf, xl[kk], S[m]);
      }
    }
  }
#pragma unroll
  for (int m = 0; m < NM; ++m) *reinterpret_cast<f32x4*>(sp + 16 * m) = S[m];
}

// ---------------------------------------------------------------------------
// A decay per token and key channel (kChannel): chunks of 32 tokens.  With L the
// log decays summed from the chunk's start, the decay of a pair factors per channel
// into e^L of the query token and e^-L of the key token, and
//     S <- e^L(end) (S + sum_s (k_s e^-L(s)) v_s^T)
// takes the same scaled keys.  Where a channel decays so far inside a chunk that
// e^-L would leave the number range, the pairs are summed one by one with
// exponent differences, and the scaled keys carry e^(L(end) - L(s)) instead, with
// e^L(end) on S alone.
// Eight waves (the upper ones) form a chunk's operands, one chunk ahead, in the
// other half of the double-buffered LDS; the lower four run the matrix products.
// The lanes of half an upper wave hold the 32 tokens of the same eight channels,
// so the running log decays are DPP scans.  Channels and tokens are stored in the
// order of the k-slots (slot_of32), so that every fragment is one 16-byte read.
template <int DK> struct ChannelBuf {
  static constexpr int KP = DK + 8, SP = 40;
  bf16_t qi[2][32 * KP];  // hi, lo of q e^L                  [t][n]
  bf16_t km[2][32 * KP];  //           k e^-L                 [s][n]
  bf16_t ke[2][DK * SP];  //           the same, transposed   [n][s]
  bf16_t vT[kPB * SP];    // v [p][s]
  float eq[DK];           // e^L(end)
  int far[8];             // per forming wave (16 channels): e^-L would leave the number range
};

constexpr float kFarLog2 = 96.f;  // log2 of the largest e^-L used as a factor
constexpr int kFormThreads = 512, kProdThreads = 256;

// place of element i of a run of 32: group g's slots are {4 g .. + 3, 16 + 4 g .. + 3}
__device__ __forceinline__ int slot_of32(int i) { return 8 * ((i >> 2) & 3) + 4 * (i >> 4) + (i & 3); }

// log2 of sigmoid(z)^(1 / tau)
__device__ __forceinline__ float channel_log2(float z, float inv_tau) {
  const float y = z * kLog2e;
  return -(fmaxf(-y, 0.f) + __builtin_amdgcn_logf(1.f + fast_exp2(-fabsf(y)))) * inv_tau;
}

template <int DK>
__global__ void __launch_bounds__(kFormThreads + kProdThreads, 3) channel_chunk_kernel(ScanArgs g) {
  using Buf = ChannelBuf<DK>;
  constexpr int Q = 32, KP = Buf::KP, SP = Buf::SP, NM = DK / 16, NK = DK / 32;
  static_assert(DK % 32 == 0 && DK <= 128, "one staged item per thread");
  __shared__ __attribute__((aligned(16))) Buf bufs[2];
  Walk w;
  if (!open_walk(g, w)) return;
  const bool former = threadIdx.x >= kProdThreads;
  const int tid = former ? threadIdx.x - kProdThreads : threadIdx.x;
  const int wave = tid >> 6, lane = tid & 63;
  const bf16_t* q = (const bf16_t*)g.q + (int64_t)w.r0 * g.qs + (int64_t)w.hq * DK;
  const bf16_t* k = (const bf16_t*)g.k + (int64_t)w.r0 * g.ks + (int64_t)w.hq * DK;
  const bf16_t* z = (const bf16_t*)g.g + (int64_t)w.r0 * g.gs + (int64_t)w.h * DK;
  const bf16_t* v = (const bf16_t*)g.v + (int64_t)w.r0 * g.vs + (int64_t)w.h * g.dv + w.col0;
  const float* zb = g.g_bias ? g.g_bias + w.h * DK : nullptr;

  if (former) {  // ---- operands of the chunks
    const int tok = lane & 31, oc = 2 * wave + (lane >> 5);  // token, channels 8 oc .. + 7 (q, k, decays)
    const bool has_k = oc < DK / 8;
    const int ov = oc - (16 - kPB / 8);  // ... columns 8 ov .. + 7 (v, the last waves)
    const bool has_v = ov >= 0;
    const int ts = slot_of32(tok);
    const int n0 = (8 * oc & ~31) + slot_of32(8 * oc & 31), n1 = (8 * oc & ~31) + slot_of32((8 * oc & 31) + 4);
    float bias[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) bias[e] = zb && has_k ? zb[8 * oc + e] : 0.f;
    raw_u32x4 rq, rk, rz, rv;
    bool live = false;
    auto fetch = [&](int t0) {
      const raw_u32x4 zero{0u, 0u, 0u, 0u};
      const int64_t t = t0 + tok;
      live = t < w.n;
      rz = live && has_k ? *reinterpret_cast<const raw_u32x4*>(z + t * g.gs + 8 * oc) : zero;
      rq = live && has_k ? *reinterpret_cast<const raw_u32x4*>(q + t * g.qs + 8 * oc) : zero;
      rk = live && has_k ? *reinterpret_cast<const raw_u32x4*>(k + t * g.ks + 8 * oc) : zero;
      rv = live && has_v ? *reinterpret_cast<const raw_u32x4*>(v + t * g.vs + 8 * ov) : zero;
    };
    auto form = [&](Buf& b) {
      bool far = false;
      float L[8], x[8];
      if (has_k) {
        chunk_to_f32<bf16_t>(rz, x);
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const float l = row_scan_sum(live ? channel_log2(x[e] + bias[e], g.inv_tau) : 0.f);
          L[e] = l + dpp_rows<0x142, 0xa>(l);  // the second row of 16 goes on from the first one's end
          far |= L[e] < -kFarLog2;
        }
      }
      const bool any = __any(far);
      if (lane == 0) b.far[wave] = any;
      if (has_k) {
        float y[8];
        raw_u32x4 hi, lo;
        chunk_to_f32<bf16_t>(rq, x);
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          y[e] = fast_exp2(L[e]);
          x[e] *= y[e];
        }
        if (tok == 31) {
          *reinterpret_cast<f32x4*>(b.eq + 8 * oc) = f32x4{y[0], y[1], y[2], y[3]};
          *reinterpret_cast<f32x4*>(b.eq + 8 * oc + 4) = f32x4{y[4], y[5], y[6], y[7]};
        }
        auto put = [&](bf16_t(*dst)[32 * KP]) {
          split8(x, hi, lo);
          *reinterpret_cast<uint2*>(dst[0] + tok * KP + n0) = uint2{hi[0], hi[1]};
          *reinterpret_cast<uint2*>(dst[0] + tok * KP + n1) = uint2{hi[2], hi[3]};
          *reinterpret_cast<uint2*>(dst[1] + tok * KP + n0) = uint2{lo[0], lo[1]};
          *reinterpret_cast<uint2*>(dst[1] + tok * KP + n1) = uint2{lo[2], lo[3]};
        };
        put(b.qi);
        chunk_to_f32<bf16_t>(rk, x);
        if (any) {  // (a wave with a far channel: relative to the chunk's end, for S; its pairs are summed one by one)
#pragma unroll
          for (int e = 0; e < 8; ++e) L[e] -= __shfl(L[e], lane | 31, 64);
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] *= g.k_scale * fast_exp2(-L[e]);
        put(b.km);
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const int i = (8 * oc + e) * SP + ts;
          b.ke[0][i] = (bf16_t)(e & 1 ? hi[e >> 1] >> 16 : hi[e >> 1] & 0xffffu);
          b.ke[1][i] = (bf16_t)(e & 1 ? lo[e >> 1] >> 16 : lo[e >> 1] & 0xffffu);
        }
      }
      if (has_v) {
#pragma unroll
        for (int e = 0; e < 8; ++e) b.vT[(8 * ov + e) * SP + ts] = (bf16_t)(e & 1 ? rv[e >> 1] >> 16 : rv[e >> 1] & 0xffffu);
      }
    };
    fetch(0);
    form(bufs[0]);
    fetch(Q);
    for (int t0 = 0, cur = 0; t0 < w.n; t0 += Q, cur ^= 1) {
      __syncthreads();  // chunk t0 is formed; the other half is consumed
      if (t0 + Q < w.n) {
        form(bufs[cur ^ 1]);
        fetch(t0 + 2 * Q);
      }
    }
    return;
  }

  // ---- products.  (The barriers of the two loops pair up: one per chunk in each.)
  const int c16 = lane & 15, g4 = lane >> 4;
  float* sp = g.state + (((int64_t)w.slot * g.H + w.h) * g.dv + w.col0 + 16 * wave + c16) * DK + 4 * g4;
  f32x4 S[NM];
#pragma unroll
  for (int m = 0; m < NM; ++m) S[m] = w.fresh ? f32x4{0.f, 0.f, 0.f, 0.f} : *reinterpret_cast<const f32x4*>(sp + 16 * m);
  auto pair_by_pair = [&](int t0, int st, int tt, f32x4& a) {  // a[r] = sum_n q_t k_s E(s, t), s = 16 st + 4 g4 + r, t = 16 tt + c16
    a = f32x4{0.f, 0.f, 0.f, 0.f};
    const int tl = 16 * tt + c16, s_lo = 16 * st + 4 * g4;
    const int64_t t = t0 + tl;
    if (t >= w.n) return;
    for (int n = 0; n < DK; ++n) {
      const float qv = bf16_to_f32(q[t * g.qs + n]), zbn = zb ? zb[n] : 0.f;
      float E = 0.f;  // log2 decay from s to t, s walking down from t
      for (int s = tl; s >= s_lo; --s) {
        if (s < s_lo + 4) {
          const float x = qv * bf16_to_f32(k[(int64_t)(t0 + s) * g.ks + n]) * g.k_scale * fast_exp2(E);
#pragma unroll
          for (int r = 0; r < 4; ++r)
            if (s == s_lo + r) a[r] += x;
        }
        E += channel_log2(bf16_to_f32(z[(int64_t)(t0 + s) * g.gs + n]) + zbn, g.inv_tau);
      }
    }
  };
  for (int t0 = 0, cur = 0; t0 < w.n; t0 += Q, cur ^= 1) {
    __syncthreads();  // this chunk is formed
    const Buf& b = bufs[cur];
    int far[8], any_far = 0;
#pragma unroll
    for (int i = 0; i < 8; ++i) far[i] = b.far[i], any_far |= far[i];
    const bf16x8_t vf = frag8(b.vT + (16 * wave + c16) * SP + 8 * g4);
    // the chunk's pair weights [s][t] as three 16 x 16 tiles (every wave forms what it needs itself), and S^T q:
    // five sums, taken in turn so that dependent instructions are far apart
    const f32x4 zero{0.f, 0.f, 0.f, 0.f};
    f32x4 a00 = zero, a01 = zero, a11 = zero, y0 = zero, y1 = zero;
#pragma unroll
    for (int kk = 0; kk < NK; ++kk) {
      const int o0 = c16 * KP + 32 * kk + 8 * g4, o1 = o0 + 16 * KP;
      const bf16x8_t k0 = frag8(b.km[0] + o0), k1 = frag8(b.km[0] + o1), q0 = frag8(b.qi[0] + o0), q1 = frag8(b.qi[0] + o1);
      const bf16x8_t k0l = frag8(b.km[1] + o0), k1l = frag8(b.km[1] + o1), q0l = frag8(b.qi[1] + o0),
                     q1l = frag8(b.qi[1] + o1);
      float s8[8];
#pragma unroll
      for (int e = 0; e < 4; ++e) s8[e] = S[2 * kk][e], s8[4 + e] = S[2 * kk + 1][e];
      raw_u32x4 hi, lo;
      split8(s8, hi, lo);
      const bf16x8_t Sh = as_bf16x8(hi), Sl = as_bf16x8(lo);
      a00 = mfma32(k0, q0, a00);
      a01 = mfma32(k0, q1, a01);
      a11 = mfma32(k1, q1, a11);
      y0 = mfma32(Sh, q0, y0);
      y1 = mfma32(Sh, q1, y1);
      a00 = mfma32(k0, q0l, a00);
      a01 = mfma32(k0, q1l, a01);
      a11 = mfma32(k1, q1l, a11);
      y0 = mfma32(Sl, q0, y0);
      y1 = mfma32(Sl, q1, y1);
      a00 = mfma32(k0l, q0, a00);
      a01 = mfma32(k0l, q1, a01);
      a11 = mfma32(k1l, q1, a11);
      y0 = mfma32(Sh, q0l, y0);
      y1 = mfma32(Sh, q1l, y1);
    }
#pragma unroll
    for (int m = 0; m < NM; ++m) {
      // a forming wave's 16 channels: their keys are relative to the chunk's start, or (far) to its end
      const f32x4 e4 = *reinterpret_cast<const f32x4*>(b.eq + 16 * m + 4 * g4);
      const int o = (16 * m + c16) * SP + 8 * g4;
      const bf16x8_t kh = frag8(b.ke[0] + o), kl = frag8(b.ke[1] + o);
      if (far[m]) {
#pragma unroll
        for (int r = 0; r < 4; ++r) S[m][r] *= e4[r];
      }
      S[m] = mfma32(kh, vf, S[m]);
      S[m] = mfma32(kl, vf, S[m]);
      if (!far[m]) {
#pragma unroll
        for (int r = 0; r < 4; ++r) S[m][r] *= e4[r];
      }
    }
    if (any_far) {
      pair_by_pair(t0, 0, 0, a00);
      pair_by_pair(t0, 0, 1, a01);
      pair_by_pair(t0, 1, 1, a11);
    }
    float w0[8], w1[8];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const bool seen = 4 * g4 + r <= c16;
      w0[r] = seen ? a00[r] : 0.f;
      w0[4 + r] = 0.f;
      w1[r] = a01[r];
      w1[4 + r] = seen ? a11[r] : 0.f;
    }
    raw_u32x4 h0, l0, h1, l1;
    split8(w0, h0, l0);
    split8(w1, h1, l1);
    y0 = mfma32(vf, as_bf16x8(h0), y0);
    y1 = mfma32(vf, as_bf16x8(h1), y1);
    y0 = mfma32(vf, as_bf16x8(l0), y0);
    y1 = mfma32(vf, as_bf16x8(l1), y1);
    float* o = g.out + ((int64_t)(w.r0 + t0 + c16) * g.H + w.h) * g.dv + w.col0 + 16 * wave + 4 * g4;
#pragma unroll
    for (int r = 0; r < 4; ++r) y0[r] *= g.q_scale, y1[r] *= g.q_scale;
    if (t0 + c16 < w.n) *reinterpret_cast<f32x4*>(o) = y0;
    if (t0 + 16 + c16 < w.n) *reinterpret_cast<f32x4*>(o + (int64_t)16 * g.H * g.dv) = y1;
  }
#pragma unroll
  for (int m = 0; m < NM; ++m) *reinterpret_cast<f32x4*>(sp + 16 * m) = S[m];
}

}  // namespace

// sizes and alignment the chunked kernels take (bf16 rows as 16-byte runs, whole column blocks)
bool chunk_scan_ok(int mode, const ScanArgs& g) {
  auto al = [](const void* p) { return (uintptr_t)p % 16 == 0; };
  return (g.dk == 32 || g.dk == 64 || g.dk == 128) && g.dv % kPB == 0 && g.qs % 8 == 0 && g.ks % 8 == 0 &&
         g.vs % 8 == 0 && al(g.q) && al(g.k) && al(g.v) && al(g.state) && al(g.out) &&
         (mode != kChannel || (g.gs % 8 == 0 && al(g.g) && !g.skip));
}

#define CHUNK_DK(KERNEL, NT)                                                  \
  if (g.dk == 32) hipLaunchKernelGGL((KERNEL(32)), grid, NT, 0, st, g);       \
  else if (g.dk == 64) hipLaunchKernelGGL((KERNEL(64)), grid, NT, 0, st, g);  \
  else hipLaunchKernelGGL((KERNEL(128)), grid, NT, 0, st, g);

void launch_chunk_scan(int mode, const ScanArgs& g, int n_seq, hipStream_t st) {
  const dim3 grid(g.dv / kPB, g.H, n_seq);
#define FIXED_K(D) chunk_scan_kernel<D, kFixed>
#define STEP_K(D) chunk_scan_kernel<D, kStep>
#define CHANNEL_K(D) channel_chunk_kernel<D>
  if (mode == kFixed) { CHUNK_DK(FIXED_K, dim3(512)) }
  else if (mode == kStep) { CHUNK_DK(STEP_K, dim3(512)) }
  else { CHUNK_DK(CHANNEL_K, dim3(kFormThreads + kProdThreads)) }
}
