// What the kernels that write keys and values to the cache pages share: bfloat16 in pieces of
// eight, and the tile that turns values on their way into the pages.
#pragma once
#include "common.h"

constexpr int kRopeTokV = 16;
constexpr int kRopeVCols = 256;                // v columns per workgroup
constexpr int kRopeVRow = kRopeVCols + 8;      // padded: rows stay 16-byte aligned, banks spread

__device__ __forceinline__ void unpack8(const uint4 u, float (&v)[8]) {
  const uint32_t w[4] = {u.x, u.y, u.z, u.w};
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    v[2 * i] = __uint_as_float(w[i] << 16);
    v[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
  }
}
__device__ __forceinline__ uint4 pack8(const float (&v)[8]) {
  uint32_t w[4];
#pragma unroll
  for (int i = 0; i < 4; ++i)
    w[i] = (uint32_t)f32_to_bf16(v[2 * i]) | ((uint32_t)f32_to_bf16(v[2 * i + 1]) << 16);
  return make_uint4(w[0], w[1], w[2], w[3]);
}

// Values of the step's rows into v_pages[page][kv head][d][offset]: workgroup `vb` of those that
// do this takes a tile of kRopeTokV tokens times kRopeVCols columns (256 threads).
__device__ __forceinline__ void store_value_tile(
    const bf16_t* __restrict__ qkv, long long row_stride, int v_off, int T, int nkv, int d,
    const int* __restrict__ slots, bf16_t* __restrict__ v_pages, int page_size, int vb) {
  const int tid = threadIdx.x;
  __shared__ __attribute__((aligned(16))) bf16_t v_s[kRopeTokV * kRopeVRow];
  __shared__ long long page_s[kRopeTokV];                // -1: the token is not stored
  __shared__ int off_s[kRopeTokV];
  const int cols = nkv * d;
  const int chunks = (cols + kRopeVCols - 1) / kRopeVCols;
  const int t0 = (vb / chunks) * kRopeTokV, c0 = (vb % chunks) * kRopeVCols;
  if (tid < kRopeTokV) {
    const int slot = t0 + tid < T ? slots[t0 + tid] : -1;
    const int page = slot < 0 ? -1 : slot / page_size;
    page_s[tid] = page;
    off_s[tid] = slot < 0 ? 0 : slot - page * page_size;
  }
  const int nc = min(kRopeVCols, cols - c0), nc8 = nc / 8;
  for (int i = tid; i < kRopeTokV * nc8; i += blockDim.x) {
    const int tt = i / nc8, c = (i - tt * nc8) * 8;
    if (t0 + tt < T)
      *(uint4*)(v_s + tt * kRopeVRow + c) =
          *(const uint4*)(qkv + (long long)(t0 + tt) * row_stride + v_off + c0 + c);
  }
  __syncthreads();
  for (int i = tid; i < kRopeTokV * nc; i += blockDim.x) {
    const int tt = i % kRopeTokV, c = i / kRopeTokV;
    const long long page = page_s[tt];
    if (page < 0) continue;
    const int col = c0 + c, h = col / d, j = col - h * d;
    v_pages[((page * nkv + h) * d + j) * page_size + off_s[tt]] = v_s[tt * kRopeVRow + c];
  }
}

