// Shared by the attention kernels that walk pages of whole 64-key tiles (stream_attention.hip,
// latent_attention.hip): masks, LDS images of a tile, matrix-core fragments.
#pragma once
#include "recurrent.h"

namespace {

// element offset of 16-byte piece pc of row r in the [dv][64 keys] image; the row bits that move the pieces
// keep both the fragment reads (16 neighbouring rows) and the transposed writes (rows 8 apart) on different banks
__device__ __forceinline__ int voff(int r, int pc) { return r * 64 + ((pc ^ ((r >> 1) & 7) ^ ((r >> 3) & 7)) << 3); }

// keys 4 kg .. + 3 (four rows of eight columns, in registers) into columns 8 ch .. + 7 of the image; the keys of
// a 32-key half are stored in the order of the k-slots: group g's slots are keys {4 g .. + 3, 16 + 4 g .. + 3}
__device__ __forceinline__ void put_v(bf16_t* Vt, const raw_u32x4* r, int kg, int ch) {
  const int pc = 4 * (kg >> 3) + (kg & 3), hf = 4 * ((kg >> 2) & 1);
#pragma unroll
  for (int w = 0; w < 4; ++w) {
    uint2 ev, od;
    ev.x = (r[0][w] & 0xffffu) | (r[1][w] << 16);
    ev.y = (r[2][w] & 0xffffu) | (r[3][w] << 16);
    od.x = (r[0][w] >> 16) | (r[1][w] & 0xffff0000u);
    od.y = (r[2][w] >> 16) | (r[3][w] & 0xffff0000u);
    *reinterpret_cast<uint2*>(Vt + voff(8 * ch + 2 * w, pc) + hf) = ev;
    *reinterpret_cast<uint2*>(Vt + voff(8 * ch + 2 * w + 1, pc) + hf) = od;
  }
}

__device__ __forceinline__ bf16x8_t frag16(const bf16_t* p) {
  return __builtin_bit_cast(bf16x8_t, *reinterpret_cast<const raw_u32x4*>(p));
}
// first key that the query at position p sees (mask 0: causal, 1: window, 2: chunk)
__device__ __forceinline__ int first_key(int p, int mask, int size) {
  if (mask == 1) return p - size + 1 > 0 ? p - size + 1 : 0;
  if (mask == 2) return (int)((unsigned)p / (unsigned)size) * size;
  return 0;
}
__device__ __forceinline__ f32x4 mma(bf16x8_t a, bf16x8_t b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}
// row of the caches of key 64 t of a sequence
__device__ __forceinline__ int64_t tile_slot(const int* bt, int shift, int t) {
  const int j = t << 6;
  return ((int64_t)bt[j >> shift] << shift) + (j & ((1 << shift) - 1));
}

// element offset of 16-byte piece pc of key r in the [64][D] image: an XOR with low bits of the row (rows of 8
// pieces: of its pair), as many as keep the piece inside the row, spreads a fragment's 16 rows over the banks
template <int D> __device__ __forceinline__ int kimg(int r, int pc) {
  constexpr int kLow = (D / 8) & -(D / 8);  // largest power of two that divides the pieces of a row
  constexpr int kMask = kLow > 16 ? 15 : kLow - 1;
  return r * D + ((pc ^ (D == 64 ? (r >> 1) & 7 : r & kMask)) << 3);
}

}  // namespace
