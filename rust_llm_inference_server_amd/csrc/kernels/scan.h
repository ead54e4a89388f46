// What the scans over a matrix state share (recurrent.hip, channel_delta.hip): the activations of a
// recurrence in float32, sums over a wave by data-parallel adds, and the tile sizes of the forms
// for long runs of tokens.
#pragma once
#include "common.h"

#include <math.h>

__device__ __forceinline__ float sigmoidf_(float x) { return 1.0f / (1.0f + expf(-x)); }
__device__ __forceinline__ float siluf_(float x) { return x / (1.0f + expf(-x)); }
__device__ __forceinline__ float softplusf_(float x) { return x > 20.0f ? x : log1pf(expf(x)); }

// Sum over the 64 lanes of a wave, every lane gets it: four data-parallel-primitive adds inside
// rows of 16 lanes (neighbour, pair, the other quad, the other half-row) and the two half
// swaps; no trip through LDS.  The order of the additions is fixed.
template <int CTRL>
__device__ __forceinline__ float dpp_from(float v) {
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xF, 0xF, true));
}
__device__ __forceinline__ float lanes_sum(float v) {
  v += dpp_from<0xB1>(v);    // quad_perm [1, 0, 3, 2]
  v += dpp_from<0x4E>(v);    // quad_perm [2, 3, 0, 1]
  v += dpp_from<0x141>(v);   // row_half_mirror
  v += dpp_from<0x140>(v);   // row_mirror
  v = xor16_sum(v);
  return xor32_sum(v);
}

// Four sums over the wave at once, for values a wave holds per lane for four columns: lanes
// trade columns with their neighbour and their neighbour's neighbour, so that lane l carries on
// with column l % 4 alone, and the steps that follow (4 and 8 lanes round the row, the half
// swaps) keep that class.  Lane l ends with the whole sum of column l % 4: ten adds and moves
// for four sums where four separate sums take twenty-four.  The order of the additions is fixed.
__device__ __forceinline__ float lanes_sum4(const float (&p)[4], int lane) {
  const bool odd = lane & 1, high = lane & 2;
  float a01 = odd ? p[1] : p[0];
  a01 += dpp_from<0xB1>(odd ? p[0] : p[1]);
  float a23 = odd ? p[3] : p[2];
  a23 += dpp_from<0xB1>(odd ? p[2] : p[3]);
  float a = high ? a23 : a01;
  a += dpp_from<0x4E>(high ? a01 : a23);
  a += dpp_from<0x124>(a);   // row_ror 4
  a += dpp_from<0x128>(a);   // row_ror 8
  a = xor16_sum(a);
  return xor32_sum(a);
}

// The same for two columns: lane l ends with the whole sum of column l % 2.
__device__ __forceinline__ float lanes_sum2(const float (&p)[2], int lane) {
  const bool odd = lane & 1;
  float a = odd ? p[1] : p[0];
  a += dpp_from<0xB1>(odd ? p[0] : p[1]);
  a += dpp_from<0x4E>(a);    // two lanes on: the same column
  a += dpp_from<0x124>(a);
  a += dpp_from<0x128>(a);
  a = xor16_sum(a);
  return xor32_sum(a);
}
template <int NC>
__device__ __forceinline__ float lanes_sum_cols(const float (&p)[NC], int lane) {
  if constexpr (NC == 4) return lanes_sum4(p, lane);
  else return lanes_sum2(p, lane);
}

// Value channels a wave of the scans walks at a time, and the tokens and key channels of a tile.
constexpr int kCols = 4;
template <int KR>
struct ScanTile {
  static constexpr int kTokens = KR == 4 ? 16 : 32;
  static constexpr int kKeys = KR * kWave;
};

static inline int scan_compute_units() {
  static int units = 0;
  if (units == 0) {
    int dev = 0;
    hipDeviceProp_t prop;
    units = (hipGetDevice(&dev) == hipSuccess && hipGetDeviceProperties(&prop, dev) == hipSuccess)
                ? prop.multiProcessorCount : 256;
  }
  return units;
}

// Forms that cut every sequence's tokens of the step into chunks of `len` number the chunks of all
// sequences in order.  The `index`-th chunk's tokens [t0, t1) (false: there are fewer), and the
// number of chunks in front of a sequence.
__device__ __forceinline__ bool chunk_span(const int* cu, int num_seqs, int len, int index, int& t0,
                                           int& t1) {
  int left = index;
  for (int s = 0; s < num_seqs; ++s) {
    const int b = cu[s], e = cu[s + 1];
    const int chunks = (e - b + len - 1) / len;
    if (left < chunks) {
      t0 = b + left * len;
      t1 = min(e, t0 + len);
      return true;
    }
    left -= chunks;
  }
  return false;
}
__device__ __forceinline__ int chunks_before(const int* cu, int seq, int len) {
  int n = 0;
  for (int s = 0; s < seq; ++s) n += (cu[s + 1] - cu[s] + len - 1) / len;
  return n;
}
