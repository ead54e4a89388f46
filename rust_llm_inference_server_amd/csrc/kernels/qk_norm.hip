// Queries and keys that are rotated and then divided by their own root mean square, on their way
// from the fused projection to the attention kernels: per token and head
//   r = rotation of the head's first `rot` numbers by the token's position (halves: number j with
//       j + rot / 2; `interleaved`: 2j with 2j + 1), the rest as they are,
//   r / sqrt(mean(r^2) + eps), the mean over the head's `real` numbers (the rest of its D columns
//   is padding, zeros, and stays zeros).
// Queries stay in the row.  `keys` 1: keys go to k_pages[page][kv head][offset][D] and the values,
// as they are, to v_pages[page][kv head][D][offset]; 2: keys stay in the row too (for an attention
// kernel that writes the cache itself); 0: queries alone.  Angles, squares and quotients are float32, with one
// rounding at the store.
#include "common.h"
#include "kv_write.h"

#include <math.h>

// Any layout: a wave per head of a token, the four waves of a workgroup take the heads in turn.
template <typename TX, int DPL>
__global__ __launch_bounds__(256) void norm_rope_kv_write_kernel(
    TX* __restrict__ qkv, long long row_stride, int k_off, int v_off, int nh, int nkv, int D,
    int real, int rot, float eps, const float* __restrict__ cos_t, const float* __restrict__ sin_t,
    const int* __restrict__ positions, const int* __restrict__ slots, TX* __restrict__ k_pages,
    TX* __restrict__ v_pages, int page_size, int interleaved, int keys) {
  const int t = blockIdx.x, wave = threadIdx.x / kWave, lane = threadIdx.x % kWave;
  TX* row = qkv + (long long)t * row_stride;
  const int half = rot / 2;
  const long long angle = rot ? (long long)positions[t] * half : 0;
  const int slot = keys == 1 ? slots[t] : -1;
  const long long page = slot < 0 ? 0 : slot / page_size;
  const int off = slot < 0 ? 0 : slot - (int)page * page_size;
  const int heads = nh + (slot >= 0 || keys == 2 ? nkv : 0);
  for (int h = wave; h < heads; h += 4) {
    const bool is_k = h >= nh;
    const TX* src = row + (is_k ? k_off + (h - nh) * D : h * D);
    float v[DPL];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < DPL; ++i) {
      const int j = lane + kWave * i;
      v[i] = j < D ? ld(src + j) : 0.f;
      if (j < rot) {
        const int p = interleaved ? j / 2 : (j < half ? j : j - half);
        const bool first = interleaved ? j % 2 == 0 : j < half;
        const int d = interleaved ? 1 : half;
        const float w = ld(src + (first ? j + d : j - d));
        const float c = cos_t[angle + p], s = sin_t[angle + p];
        v[i] = first ? v[i] * c - w * s : v[i] * c + w * s;
      }
      ss += v[i] * v[i];
    }
    // (every lane's loads of the head lie in front of this sum, every store behind it)
    const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)real + eps);
    TX* dst = is_k && keys == 1 ? k_pages + ((page * nkv + (h - nh)) * page_size + off) * D
                                : row + (src - row);
#pragma unroll
    for (int i = 0; i < DPL; ++i) {
      const int j = lane + kWave * i;
      if (j < D) st(dst + j, v[i] * inv);
    }
  }
  if (slot < 0) return;
  for (int i = threadIdx.x; i < nkv * D; i += 256) {
    const int h = i / D, j = i - h * D;
    v_pages[((page * nkv + h) * D + j) * page_size + off] = row[v_off + h * D + j];
  }
}

// bfloat16 in pieces of eight: LPH lanes (a power of two) share a head, the partner of a rotated
// piece comes from the lane that holds it; a lane has its piece of HPL heads of one token, which
// share the angles.  The first `qk_blocks` workgroups turn q and k, the others move values as the
// plain cache write does.
template <int LPH, int HPL, bool INTERLEAVED>
__global__ __launch_bounds__(256) void norm_rope_kv_write_bf16x8_kernel(
    bf16_t* __restrict__ qkv, long long row_stride, int k_off, int v_off, int T, int nh, int nkv,
    int D, int real, int rot, float eps, const float* __restrict__ cos_t,
    const float* __restrict__ sin_t, const int* __restrict__ positions,
    const int* __restrict__ slots, bf16_t* __restrict__ k_pages, bf16_t* __restrict__ v_pages,
    int page_size, int keys, unsigned sets, int qk_blocks) {
  if ((int)blockIdx.x >= qk_blocks) {
    store_value_tile(qkv, row_stride, v_off, T, nkv, D, slots, v_pages, page_size,
                     (int)blockIdx.x - qk_blocks);
    return;
  }
  const unsigned set = (blockIdx.x * 256u + threadIdx.x) / LPH;
  const int sub = threadIdx.x % LPH;
  const int heads = nh + (keys ? nkv : 0), per_tok = (heads + HPL - 1) / HPL;
  // (lanes past the last set, a token's last head or the head's width work on a place that is
  // there and drop the result: the shuffles want every lane of the wave)
  const bool live = set < sets && sub * 8 < D;
  const int j0 = sub * 8 < D ? sub * 8 : 0;
  const unsigned own = set < sets ? set : sets - 1;
  const int t = (int)(own / (unsigned)per_tok);
  const int h0 = (int)(own - (unsigned)t * (unsigned)per_tok) * HPL;
  bf16_t* row = qkv + (long long)t * row_stride + j0;
  const int slot = keys == 1 ? slots[t] : 0;
  uint4 raw[HPL];
#pragma unroll
  for (int i = 0; i < HPL; ++i) {
    const int h = min(h0 + i, heads - 1);
    raw[i] = *(const uint4*)(row + (h < nh ? h * D : k_off + (h - nh) * D));
  }
  const int half = rot / 2;
  const bool turns = j0 < rot;
  const bool first = j0 < half;
  float c[8], s[8];
  if (rot) {                                      // (the same for the whole grid)
    const long long angle = (long long)positions[t] * half;
    const long long a = angle + (!turns ? 0 : INTERLEAVED ? j0 / 2 : first ? j0 : j0 - half);
    *(float4*)&c[0] = *(const float4*)(cos_t + a);
    *(float4*)&s[0] = *(const float4*)(sin_t + a);
    if constexpr (!INTERLEAVED) {
      *(float4*)&c[4] = *(const float4*)(cos_t + a + 4);
      *(float4*)&s[4] = *(const float4*)(sin_t + a + 4);
    }
  }
  const int lane = threadIdx.x % kWave;
  const int from = turns ? (first ? lane + half / 8 : lane - half / 8) : lane;
#pragma unroll
  for (int i = 0; i < HPL; ++i) {
    float r[8];
    unpack8(raw[i], r);
    if (rot) {
      if constexpr (INTERLEAVED) {
        if (turns) {
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const float u = r[2 * e], w = r[2 * e + 1];
            r[2 * e] = u * c[e] - w * s[e];
            r[2 * e + 1] = w * c[e] + u * s[e];
          }
        }
      } else {
        float w[8];
        uint4 other;
        other.x = __shfl(raw[i].x, from, kWave);
        other.y = __shfl(raw[i].y, from, kWave);
        other.z = __shfl(raw[i].z, from, kWave);
        other.w = __shfl(raw[i].w, from, kWave);
        unpack8(other, w);
        if (turns) {
#pragma unroll
          for (int e = 0; e < 8; ++e)
            r[e] = first ? r[e] * c[e] - w[e] * s[e] : r[e] * c[e] + w[e] * s[e];
        }
      }
    }
    float ss = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) ss += r[e] * r[e];
    if (!live) ss = 0.f;
#pragma unroll
    for (int o = LPH / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, kWave);
    const float inv = 1.0f / sqrtf(ss / (float)real + eps);
    const int h = h0 + i;
    const bool is_k = h >= nh;
    if (!live || h >= heads || (is_k && slot < 0)) continue;
#pragma unroll
    for (int e = 0; e < 8; ++e) r[e] *= inv;
    bf16_t* dst = row + (is_k ? k_off + (h - nh) * D : h * D);
    if (is_k && keys == 1) {
      const int page = slot / page_size;
      const int off = slot - page * page_size;
      dst = k_pages + (((long long)page * nkv + (h - nh)) * page_size + off) * D + j0;
    }
    *(uint4*)dst = pack8(r);
  }
}

RLIS_API int rlis_norm_rope_kv_write(void* qkv, int dtype, long long row_stride, int k_off, int v_off,
                                     int T, int nh, int nkv, int D, int real, int rot, float eps,
                                     const float* cos_t, const float* sin_t, const int* positions,
                                     const int* slots, void* k_pages, void* v_pages, int page_size,
                                     int interleaved, int keys, hipStream_t stream) {
  RLIS_REQUIRE(T >= 0 && nh > 0 && nkv > 0 && D > 0 && D <= 512 && real > 0 && real <= D,
               "norm_rope_kv_write: bad sizes (heads of %d)", D);
  RLIS_REQUIRE(rot >= 0 && rot <= real && rot % 2 == 0,
               "norm_rope_kv_write: %d rotated numbers of %d", rot, real);
  RLIS_REQUIRE(rot == 0 || (cos_t && sin_t && positions),
               "norm_rope_kv_write: a rotation needs its tables and positions");
  RLIS_REQUIRE(keys != 1 || (slots && k_pages && v_pages && page_size > 0),
               "norm_rope_kv_write: a cache write needs pages and slots");
  RLIS_REQUIRE(k_off >= nh * D && v_off >= k_off + nkv * D && row_stride >= v_off + (long long)nkv * D,
               "norm_rope_kv_write: rows of %lld do not hold the heads", row_stride);
  RLIS_REQUIRE(keys >= 0 && keys <= 2, "norm_rope_kv_write: unknown treatment of keys %d", keys);
  RLIS_REQUIRE(dtype == RLIS_F32 || dtype == RLIS_BF16, "norm_rope_kv_write: unknown dtype %d", dtype);
  if (T == 0) return 0;
  const int heads = nh + (keys ? nkv : 0);
  int lph = 2;
  while (lph * 8 < D) lph *= 2;
  // (few heads in all: one a lane, for more lanes at work)
  const bool four = (long long)T * heads * lph >= 1 << 16;
  const long long sets = (long long)T * (four ? ceil_div(heads, 4) : heads);
  const bool by8 = dtype == RLIS_BF16 && D % 8 == 0 && row_stride % 8 == 0 && k_off % 8 == 0 &&
                   v_off % 8 == 0 && rot % (interleaved ? 8 : 16) == 0 && (uintptr_t)qkv % 16 == 0 &&
                   (uintptr_t)cos_t % 16 == 0 && (uintptr_t)sin_t % 16 == 0 &&
                   (keys != 1 || (uintptr_t)k_pages % 16 == 0) && sets * lph < (1ll << 31) - 256;
  if (by8) {
    const int qk_blocks = (int)ceil_div_ll(sets * lph, 256);
    const int v_blocks = keys == 1 ? ceil_div(T, kRopeTokV) * ceil_div(nkv * D, kRopeVCols) : 0;
#define LAUNCH8(LPH, HPL, INTER)                                                                \
  norm_rope_kv_write_bf16x8_kernel<LPH, HPL, INTER><<<qk_blocks + v_blocks, 256, 0, stream>>>(  \
      (bf16_t*)qkv, row_stride, k_off, v_off, T, nh, nkv, D, real, rot, eps, cos_t, sin_t,      \
      positions, slots, (bf16_t*)k_pages, (bf16_t*)v_pages, page_size, keys, (unsigned)sets,    \
      qk_blocks)
#define BY_PAIRING(LPH)                                     \
  do {                                                      \
    if (interleaved && four) LAUNCH8(LPH, 4, true);         \
    else if (interleaved) LAUNCH8(LPH, 1, true);            \
    else if (four) LAUNCH8(LPH, 4, false);                  \
    else LAUNCH8(LPH, 1, false);                            \
  } while (0)
    if (lph == 2) BY_PAIRING(2);
    else if (lph == 4) BY_PAIRING(4);
    else if (lph == 8) BY_PAIRING(8);
    else if (lph == 16) BY_PAIRING(16);
    else if (lph == 32) BY_PAIRING(32);
    else BY_PAIRING(64);
#undef BY_PAIRING
#undef LAUNCH8
    RLIS_LAUNCH_CHECK("norm_rope_kv_write");
    return 0;
  }
#define LAUNCH(TX, DPL)                                                                            \
  norm_rope_kv_write_kernel<TX, DPL><<<T, 256, 0, stream>>>(                                        \
      (TX*)qkv, row_stride, k_off, v_off, nh, nkv, D, real, rot, eps, cos_t, sin_t, positions,      \
      slots, (TX*)k_pages, (TX*)v_pages, page_size, interleaved, keys)
#define BY_D(TX)                            \
  do {                                      \
    if (D <= 64) LAUNCH(TX, 1);             \
    else if (D <= 128) LAUNCH(TX, 2);       \
    else if (D <= 256) LAUNCH(TX, 4);       \
    else LAUNCH(TX, 8);                     \
  } while (0)
  if (dtype == RLIS_F32) BY_D(float);
  else BY_D(bf16_t);
#undef BY_D
#undef LAUNCH
  RLIS_LAUNCH_CHECK("norm_rope_kv_write");
  return 0;
}
