// Kernels around the residual stream of blocks whose norms stand behind their sublayers, and the
// inputs such a model takes from its tokens: the norm of a sublayer's result on its way into the
// stream, the rows of a table of token pairs, a layer's own token input, and the rows of queries
// and keys behind a norm over the whole row.
#include "common.h"

#include <math.h>

// ----------------------------------------------------------- norm, then into the stream
// x[t] += y[t] / sqrt(mean(y[t]^2) + eps) * weight in the float32 residual x (T, W); y is (T, W) in
// either dtype, or `parts` float32 partial sums (part_stride elements apart) that are added in
// order and, with round16, rounded to bfloat16 first.  The new row goes to `out` (T, W) in its
// dtype when out is given, or (next_w) the norm of the new row,
// x[t] / sqrt(mean(x[t]^2) + next_eps) * next_w, which is what a sublayer with a norm in front
// reads.  y null: x stays as it is and is copied to `out`.
//
// One workgroup per token.  A thread owns up to CH chunks of four consecutive elements; all of a
// row's loads (residual, weight, the parts eight at a time) are asked for before the sum of
// squares is waited for, and a chunk past the row reads the row's first elements and adds
// nothing.
template <typename TY, typename TW, typename TO, int NT, int CH, bool NEXT>
__global__ __launch_bounds__(NT) void norm_join_kernel(
    float* __restrict__ x, const TY* __restrict__ y, int parts, long long part_stride, int round16,
    const TW* __restrict__ weight, float eps, TO* __restrict__ out, int W,
    const TW* __restrict__ next_w, float next_eps) {
  __shared__ float red[NT / kWave];
  const long long base = (long long)blockIdx.x * W;
  int col[CH];
  bool live[CH];
  float4 xr[CH];
  TW wt[CH][4], nt[CH][4];
  float s[CH][4];
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int j = (threadIdx.x + c * NT) * 4;
    live[c] = j < W;
    col[c] = live[c] ? j : 0;
  }
  constexpr int AHEAD = sizeof(TY) == 2 ? 1 : (CH == 1 ? 8 : 4);
  for (int p = 0; p < parts; p += AHEAD) {
    TY a[CH][AHEAD][4];
#pragma unroll
    for (int c = 0; c < CH; ++c)
#pragma unroll
      for (int q = 0; q < AHEAD; ++q) {
        const TY* src = y + (long long)min(p + q, parts - 1) * part_stride + base + col[c];
        if constexpr (sizeof(TY) == 2) {
          const uint2 v = *(const uint2*)src;
          a[c][q][0] = (TY)(v.x & 0xffffu);
          a[c][q][1] = (TY)(v.x >> 16);
          a[c][q][2] = (TY)(v.y & 0xffffu);
          a[c][q][3] = (TY)(v.y >> 16);
        } else {
          const float4 v = *(const float4*)src;
          a[c][q][0] = v.x; a[c][q][1] = v.y; a[c][q][2] = v.z; a[c][q][3] = v.w;
        }
      }
    if (p == 0) {
      // (behind the first parts in the order of loads, ahead of everything that waits)
#pragma unroll
      for (int c = 0; c < CH; ++c) {
        xr[c] = *(const float4*)(x + base + col[c]);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          wt[c][e] = weight[col[c] + e];
          if constexpr (NEXT) nt[c][e] = next_w[col[c] + e];
        }
      }
    }
#pragma unroll
    for (int c = 0; c < CH; ++c)
#pragma unroll
      for (int q = 0; q < AHEAD; ++q)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float v = widen(a[c][q][e]);
          if (p == 0 && q == 0) s[c][e] = v;
          else if (p + q < parts) s[c][e] += v;
        }
  }
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < CH; ++c)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      if (round16) s[c][e] = bf16_to_f32(f32_to_bf16(s[c][e]));
      if (live[c]) ss += s[c][e] * s[c][e];
    }
  ss = block_sum<NT>(ss, red);
  const float inv = 1.0f / sqrtf(ss / (float)W + eps);
  if constexpr (NEXT) {
    float sn = 0.f;
#pragma unroll
    for (int c = 0; c < CH; ++c) {
      const float xs[4] = {xr[c].x, xr[c].y, xr[c].z, xr[c].w};
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        s[c][e] = xs[e] + s[c][e] * inv * widen(wt[c][e]);
        if (live[c]) sn += s[c][e] * s[c][e];
      }
      if (live[c])
        *(float4*)(x + base + col[c]) = make_float4(s[c][0], s[c][1], s[c][2], s[c][3]);
    }
    sn = block_sum<NT>(sn, red);
    const float next_inv = 1.0f / sqrtf(sn / (float)W + next_eps);
#pragma unroll
    for (int c = 0; c < CH; ++c) {
      if (!live[c]) continue;
      float r[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) r[e] = s[c][e] * next_inv * widen(nt[c][e]);
      if constexpr (sizeof(TO) == 2) {
        uint2 o;
        o.x = (uint32_t)f32_to_bf16(r[0]) | ((uint32_t)f32_to_bf16(r[1]) << 16);
        o.y = (uint32_t)f32_to_bf16(r[2]) | ((uint32_t)f32_to_bf16(r[3]) << 16);
        *(uint2*)(out + base + col[c]) = o;
      } else {
        *(float4*)(out + base + col[c]) = make_float4(r[0], r[1], r[2], r[3]);
      }
    }
    return;
  }
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    if (!live[c]) continue;
    float r[4];
    const float xs[4] = {xr[c].x, xr[c].y, xr[c].z, xr[c].w};
#pragma unroll
    for (int e = 0; e < 4; ++e) r[e] = xs[e] + s[c][e] * inv * widen(wt[c][e]);
    *(float4*)(x + base + col[c]) = make_float4(r[0], r[1], r[2], r[3]);
    if (out) {
      if constexpr (sizeof(TO) == 2) {
        uint2 o;
        o.x = (uint32_t)f32_to_bf16(r[0]) | ((uint32_t)f32_to_bf16(r[1]) << 16);
        o.y = (uint32_t)f32_to_bf16(r[2]) | ((uint32_t)f32_to_bf16(r[3]) << 16);
        *(uint2*)(out + base + col[c]) = o;
      } else {
        *(float4*)(out + base + col[c]) = make_float4(r[0], r[1], r[2], r[3]);
      }
    }
  }
}

// Any width: two passes over the row, the second reads it again.
template <typename TY, typename TW, typename TO>
__global__ __launch_bounds__(256) void norm_join_any_kernel(
    float* __restrict__ x, const TY* __restrict__ y, int parts, long long part_stride, int round16,
    const TW* __restrict__ weight, float eps, TO* __restrict__ out, int W,
    const TW* __restrict__ next_w, float next_eps) {
  __shared__ float red[4];
  const long long base = (long long)blockIdx.x * W;
  float ss = 0.f;
  for (int j = threadIdx.x; j < W; j += 256) {
    const float v = delta_sum(y + base + j, parts, part_stride, round16);
    ss += v * v;
  }
  ss = block_sum<256>(ss, red);
  const float inv = 1.0f / sqrtf(ss / (float)W + eps);
  float sn = 0.f;
  for (int j = threadIdx.x; j < W; j += 256) {
    const float v = delta_sum(y + base + j, parts, part_stride, round16);
    const float r = x[base + j] + v * inv * ld(weight + j);
    x[base + j] = r;
    if (out && !next_w) st(out + base + j, r);
    sn += r * r;
  }
  if (!next_w) return;
  // (a thread reads back the elements it has written itself)
  const float next_inv = 1.0f / sqrtf(block_sum<256>(sn, red) / (float)W + next_eps);
  for (int j = threadIdx.x; j < W; j += 256)
    st(out + base + j, x[base + j] * next_inv * ld(next_w + j));
}

template <typename TO>
__global__ void cast_rows_kernel(const float* __restrict__ x, TO* __restrict__ out, long long n) {
  long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x;
  const long long stride = (long long)gridDim.x * blockDim.x;
  for (; i < n; i += stride) st(out + i, x[i]);
}

template <typename TY, typename TW, typename TO>
static void launch_norm_join(float* x, const void* y, int parts, long long part_stride, int round16,
                             const void* w, float eps, void* out, int T, int W, bool vec,
                             const void* next_w, float next_eps, hipStream_t stream) {
#define RLIS_JOIN_AS(NT, CH, NEXT)                                                             \
  norm_join_kernel<TY, TW, TO, NT, CH, NEXT><<<T, NT, 0, stream>>>(                            \
      x, (const TY*)y, parts, part_stride, round16, (const TW*)w, eps, (TO*)out, W,            \
      (const TW*)next_w, next_eps)
#define RLIS_JOIN(NT, CH)                            \
  do {                                               \
    if (next_w) RLIS_JOIN_AS(NT, CH, true);          \
    else RLIS_JOIN_AS(NT, CH, false);                \
  } while (0)
  const int quads = W / 4;
  if (!vec || quads > 4096)
    norm_join_any_kernel<TY, TW, TO><<<T, 256, 0, stream>>>(x, (const TY*)y, parts, part_stride,
                                                            round16, (const TW*)w, eps, (TO*)out, W,
                                                            (const TW*)next_w, next_eps);
  else if (quads <= 64) RLIS_JOIN(64, 1);
  else if (quads <= 128) RLIS_JOIN(128, 1);
  else if (quads <= 256) RLIS_JOIN(256, 1);
  else if (quads <= 512 && T <= 64) RLIS_JOIN(512, 1);
  else if (quads <= 512) RLIS_JOIN(256, 2);
  else if (quads <= 1024) RLIS_JOIN(512, 2);
  else if (quads <= 2048) RLIS_JOIN(1024, 2);
  else RLIS_JOIN(1024, 4);
#undef RLIS_JOIN
#undef RLIS_JOIN_AS
}

RLIS_API int rlis_norm_join(float* x, const void* y, int y_dtype, int parts, long long part_stride,
                            int round16, const void* weight, int w_dtype, float eps, void* out,
                            int out_dtype, int T, int W, const void* next_w, float next_eps,
                            hipStream_t stream) {
  RLIS_REQUIRE(T >= 0 && W > 0, "norm_join: bad sizes T=%d W=%d", T, W);
  RLIS_REQUIRE(!next_w || (y && out), "norm_join: a norm behind the join needs a row and a result");
  RLIS_REQUIRE(y == nullptr || (weight && parts >= 1), "norm_join: a row to join needs a weight");
  RLIS_REQUIRE(parts == 1 || (y_dtype == RLIS_F32 && part_stride >= (long long)T * W),
               "norm_join: a stack of partial sums is float32 and whole");
  RLIS_REQUIRE(y_dtype == RLIS_F32 || y_dtype == RLIS_BF16, "norm_join: unknown dtype %d", y_dtype);
  RLIS_REQUIRE(w_dtype == RLIS_F32 || w_dtype == RLIS_BF16, "norm_join: unknown weight dtype %d", w_dtype);
  RLIS_REQUIRE(out_dtype == RLIS_F32 || out_dtype == RLIS_BF16, "norm_join: unknown result dtype %d", out_dtype);
  if (T == 0) return 0;
  if (y == nullptr) {
    RLIS_REQUIRE(out != nullptr, "norm_join: nothing to do");
    const long long n = (long long)T * W;
    const int blocks = (int)(ceil_div_ll(n, 256) < 8192 ? ceil_div_ll(n, 256) : 8192);
    if (out_dtype == RLIS_BF16)
      cast_rows_kernel<bf16_t><<<blocks, 256, 0, stream>>>(x, (bf16_t*)out, n);
    else
      cast_rows_kernel<float><<<blocks, 256, 0, stream>>>(x, (float*)out, n);
    RLIS_LAUNCH_CHECK("norm_join");
    return 0;
  }
  const bool vec = W % 4 == 0 && (uintptr_t)x % 16 == 0 && (uintptr_t)y % 16 == 0 &&
                   (!out || (uintptr_t)out % 16 == 0) && (parts == 1 || part_stride % 4 == 0);
#define RLIS_BY_OUT(TY, TW)                                                                      \
  do {                                                                                           \
    if (out && out_dtype == RLIS_F32)                                                            \
      launch_norm_join<TY, TW, float>(x, y, parts, part_stride, round16, weight, eps, out, T, W, \
                                      vec, next_w, next_eps, stream);                            \
    else                                                                                         \
      launch_norm_join<TY, TW, bf16_t>(x, y, parts, part_stride, round16, weight, eps, out, T, W, \
                                       vec, next_w, next_eps, stream);                           \
  } while (0)
  if (y_dtype == RLIS_F32 && w_dtype == RLIS_F32) RLIS_BY_OUT(float, float);
  else if (y_dtype == RLIS_F32) RLIS_BY_OUT(float, bf16_t);
  else if (w_dtype == RLIS_F32) RLIS_BY_OUT(bf16_t, float);
  else RLIS_BY_OUT(bf16_t, bf16_t);
#undef RLIS_BY_OUT
  RLIS_LAUNCH_CHECK("norm_join");
  return 0;
}

// ----------------------------------------------------------------- a layer's token input
// z[t][j] <- gelu(z[t][j]) * table[ids[t]][col0 + j] in place (tanh form, float32 arithmetic, one
// rounding); z rows ldz apart, table rows ldt apart.
template <typename TX>
__global__ void side_gate_kernel(TX* __restrict__ z, long long ldz, const TX* __restrict__ table,
                                 long long ldt, const int* __restrict__ ids, int dim,
                                 long long total) {
  const long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= total) return;
  const long long t = i / dim;
  const int j = (int)(i - t * dim);
  TX* p = z + t * ldz + j;
  st(p, gelu_tanh_f(ld(p)) * ld(table + (long long)ids[t] * ldt + j));
}

RLIS_API int rlis_side_gate(void* z, int dtype, long long ldz, const void* table, long long ldt,
                            const int* ids, int T, int dim, hipStream_t stream) {
  RLIS_REQUIRE(T >= 0 && dim > 0 && ldz >= dim && ldt >= dim, "side_gate: bad sizes");
  const long long total = (long long)T * dim;
  if (total == 0) return 0;
  const unsigned blocks = (unsigned)ceil_div_ll(total, 256);
  if (dtype == RLIS_F32)
    side_gate_kernel<float><<<blocks, 256, 0, stream>>>((float*)z, ldz, (const float*)table, ldt, ids,
                                                        dim, total);
  else if (dtype == RLIS_BF16)
    side_gate_kernel<bf16_t><<<blocks, 256, 0, stream>>>((bf16_t*)z, ldz, (const bf16_t*)table, ldt,
                                                         ids, dim, total);
  else
    RLIS_REQUIRE(false, "side_gate: unknown dtype %d", dtype);
  RLIS_LAUNCH_CHECK("side_gate");
  return 0;
}

// ------------------------------------------------------- embedding with a table of pairs
// out[t] = table[ids[t]] * scale + pairs[row], row = (previous * mul_prev + ids[t] * mul_cur) mod
// buckets, row `buckets` for a sequence's first token.  The token before a sequence's first one
// of the step is the slot's (last[slots[s] * last_stride], the token plus one; 0: there is none),
// which then becomes the last token of the step.  One workgroup per token: that of a sequence's
// first token reads the slot before it writes it, and no other touches it.
template <typename TW>
__global__ __launch_bounds__(256) void embed_pairs_kernel(
    float* __restrict__ out, const TW* __restrict__ table, const TW* __restrict__ pairs,
    const int* __restrict__ ids, int W, float scale, long long buckets, long long mul_prev,
    long long mul_cur, int* __restrict__ last, long long last_stride,
    const int* __restrict__ seq_of_token, const int* __restrict__ cu, const int* __restrict__ slots) {
  const int t = blockIdx.x;
  const int s = seq_of_token[t];
  const int t0 = cu[s], t1 = cu[s + 1];
  const int id = ids[t];
  int* slot = last + (long long)slots[s] * last_stride;
  const bool first = t == t0;
  const int before = first ? *slot : ids[t - 1] + 1;
  if (first) {
    __syncthreads();                     // (the same branch for the whole workgroup)
    if (threadIdx.x == 0) *slot = ids[t1 - 1] + 1;
  }
  const long long row =
      before == 0 ? buckets : ((long long)(before - 1) * mul_prev + (long long)id * mul_cur) % buckets;
  const TW* a = table + (long long)id * W;
  const TW* b = pairs + row * W;
  for (int j = threadIdx.x; j < W; j += 256)
    out[(long long)t * W + j] = ld(a + j) * scale + ld(b + j);
}

RLIS_API int rlis_embed_pairs(float* out, const void* table, const void* pairs, int dtype,
                              const int* ids, int T, int W, int buckets, float scale,
                              long long mul_prev, long long mul_cur, int* last,
                              long long last_stride, const int* seq_of_token, const int* cu,
                              const int* slots, hipStream_t stream) {
  RLIS_REQUIRE(T >= 0 && W > 0 && buckets > 0 && last_stride >= 1, "embed_pairs: bad sizes");
  RLIS_REQUIRE(mul_prev >= 0 && mul_prev < (1LL << 31) && mul_cur >= 0 && mul_cur < (1LL << 31),
               "embed_pairs: the multipliers must be in [0, 2^31)");
  if (T == 0) return 0;
  if (dtype == RLIS_F32)
    embed_pairs_kernel<float><<<T, 256, 0, stream>>>(out, (const float*)table, (const float*)pairs, ids,
                                                     W, scale, buckets, mul_prev, mul_cur, last,
                                                     last_stride, seq_of_token, cu, slots);
  else if (dtype == RLIS_BF16)
    embed_pairs_kernel<bf16_t><<<T, 256, 0, stream>>>(out, (const bf16_t*)table, (const bf16_t*)pairs,
                                                      ids, W, scale, buckets, mul_prev, mul_cur,
                                                      last, last_stride, seq_of_token, cu, slots);
  else
    RLIS_REQUIRE(false, "embed_pairs: unknown dtype %d", dtype);
  RLIS_LAUNCH_CHECK("embed_pairs");
  return 0;
}

// ------------------------------------------------- queries and keys behind whole-row norms
// A token's projection row p = [q heads | k heads | ...], heads D wide (the first `real` numbers
// of each are the model's, the rest zeros), becomes the row [q | k | v] the attention kernels
// take: v = k + bias as it is; q and k are biased, divided by the root mean square of all their
// heads' numbers together (eps inside the root), multiplied by a weight per column, and the first
// `rot` dims of every head turned by the token's position (cos/sin float32 (positions, rot / 2),
// null: no rotation; INTERLEAVED: dims 2i and 2i + 1 form a pair, else i and i + rot / 2).
// Float32 arithmetic, one rounding.  One workgroup per token, V consecutive dims a thread at a
// time; the second pass reads the row again (from the cache).
template <typename TX, int V>
__device__ __forceinline__ void load_dims(const TX* p, float (&v)[V]) {
  if constexpr (V == 8 && sizeof(TX) == 2) {
    const uint4 u = *(const uint4*)p;
    const uint32_t w[4] = {u.x, u.y, u.z, u.w};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      v[2 * i] = __uint_as_float(w[i] << 16);
      v[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
    }
  } else {
#pragma unroll
    for (int i = 0; i < V; ++i) v[i] = ld(p + i);
  }
}
template <typename TX, int V>
__device__ __forceinline__ void store_dims(TX* p, const float (&v)[V]) {
  if constexpr (V == 8 && sizeof(TX) == 2) {
    uint32_t w[4];
#pragma unroll
    for (int i = 0; i < 4; ++i)
      w[i] = (uint32_t)f32_to_bf16(v[2 * i]) | ((uint32_t)f32_to_bf16(v[2 * i + 1]) << 16);
    *(uint4*)p = make_uint4(w[0], w[1], w[2], w[3]);
  } else {
#pragma unroll
    for (int i = 0; i < V; ++i) st(p + i, v[i]);
  }
}

template <typename TX, int V, bool INTERLEAVED>
__global__ __launch_bounds__(256) void row_prepare_kernel(
    TX* __restrict__ out, const TX* __restrict__ p, long long ldp, int nh, int nkv, int D, int real,
    const float* __restrict__ bias, const float* __restrict__ q_weight,
    const float* __restrict__ k_weight, float eps, const float* __restrict__ cos_t,
    const float* __restrict__ sin_t, int rot, const int* __restrict__ positions) {
  __shared__ float red[8];
  const int t = blockIdx.x;
  const TX* row = p + (long long)t * ldp;
  const int q_cols = nh * D, cols = (nh + nkv) * D;
  TX* dst = out + (long long)t * (cols + nkv * D);
  float sq = 0.f, sk = 0.f;
  for (int c = threadIdx.x * V; c < cols; c += 256 * V) {
    float v[V];
    load_dims<TX, V>(row + c, v);
    float s = 0.f;
#pragma unroll
    for (int e = 0; e < V; ++e) {
      const float b = v[e] + (bias ? bias[c + e] : 0.f);
      s += b * b;
    }
    if (c < q_cols) sq += s;
    else sk += s;
  }
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  if (threadIdx.x % kWave == 0) {
    red[threadIdx.x / kWave] = sq;
    red[4 + threadIdx.x / kWave] = sk;
  }
  __syncthreads();
  const float q_inv = 1.0f / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / (float)(nh * real) + eps);
  const float k_inv = 1.0f / sqrtf(((red[4] + red[5]) + (red[6] + red[7])) / (float)(nkv * real) + eps);
  const int half = rot / 2;
  const long long angle = cos_t ? (long long)positions[t] * half : 0;
  for (int c = threadIdx.x * V; c < cols; c += 256 * V) {
    const bool is_q = c < q_cols;
    const float inv = is_q ? q_inv : k_inv;
    const float* weight = is_q ? q_weight + c : k_weight + (c - q_cols);
    float v[V], r[V];
    load_dims<TX, V>(row + c, v);
#pragma unroll
    for (int e = 0; e < V; ++e) {
      v[e] += bias ? bias[c + e] : 0.f;
      r[e] = v[e] * inv * weight[e];
    }
    if (!is_q) store_dims<TX, V>(dst + nkv * D + c, v);
    const int j = c % D;
    if (cos_t && j < rot) {
      if constexpr (INTERLEAVED) {
#pragma unroll
        for (int e = 0; e < V; e += 2) {
          if (j + e < rot) {
            const float cs = cos_t[angle + (j + e) / 2], sn = sin_t[angle + (j + e) / 2];
            const float a = r[e], b = r[e + 1];
            r[e] = a * cs - b * sn;
            r[e + 1] = b * cs + a * sn;
          }
        }
      } else {
        // (half is a multiple of V: a thread's dims lie on one side)
        const int d = j < half ? half : -half;
        float w[V];
        load_dims<TX, V>(row + c + d, w);
#pragma unroll
        for (int e = 0; e < V; ++e) {
          const int i = j < half ? j + e : j + e - half;
          const float cs = cos_t[angle + i], sn = sin_t[angle + i];
          const float other = (w[e] + (bias ? bias[c + d + e] : 0.f)) * inv * weight[d + e];
          r[e] = j < half ? r[e] * cs - other * sn : r[e] * cs + other * sn;
        }
      }
    }
    store_dims<TX, V>(dst + c, r);
  }
}

// The usual case (bfloat16, heads of a multiple of 8, neighbouring dims as pairs, a rotated width
// of a multiple of 8 or none): a thread owns CH pieces of eight dims and keeps them; everything
// it reads, the weights and angles too, is asked for before the sums are waited for.
template <int CH>
__global__ __launch_bounds__(1024) void row_prepare_bf16x8_kernel(
    bf16_t* __restrict__ out, const bf16_t* __restrict__ p, long long ldp, int nh, int nkv, int D,
    int real, const float* __restrict__ bias, const float* __restrict__ q_weight,
    const float* __restrict__ k_weight, float eps, const float* __restrict__ cos_t,
    const float* __restrict__ sin_t, int rot, const int* __restrict__ positions) {
  __shared__ float red[2][16];
  const int t = blockIdx.x, NT = blockDim.x;
  const bf16_t* row = p + (long long)t * ldp;
  const int q_cols = nh * D, cols = (nh + nkv) * D;
  bf16_t* dst = out + (long long)t * (cols + nkv * D);
  uint4 raw[CH];
  float4 b4[CH][2], w4[CH][2], c4[CH], s4[CH];
  int at[CH];
  const int half = rot / 2;
  const long long angle = cos_t ? (long long)positions[t] * half : 0;
#pragma unroll
  for (int i = 0; i < CH; ++i) {
    const int c = (threadIdx.x + i * NT) * 8;
    at[i] = c < cols ? c : 0;                // (past the end: the first piece again, not used)
    raw[i] = *(const uint4*)(row + at[i]);
    const float* w = at[i] < q_cols ? q_weight + at[i] : k_weight + (at[i] - q_cols);
    w4[i][0] = *(const float4*)w;
    w4[i][1] = *(const float4*)(w + 4);
    b4[i][0] = b4[i][1] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (bias) {                              // (the same for the whole grid)
      b4[i][0] = *(const float4*)(bias + at[i]);
      b4[i][1] = *(const float4*)(bias + at[i] + 4);
    }
    if (cos_t) {
      const int j = at[i] % D;
      const long long a = angle + (j < rot ? j / 2 : 0);
      c4[i] = *(const float4*)(cos_t + a);
      s4[i] = *(const float4*)(sin_t + a);
    }
  }
  float v[CH][8];
  float sq = 0.f, sk = 0.f;
#pragma unroll
  for (int i = 0; i < CH; ++i) {
    const uint32_t u[4] = {raw[i].x, raw[i].y, raw[i].z, raw[i].w};
    const float b[8] = {b4[i][0].x, b4[i][0].y, b4[i][0].z, b4[i][0].w,
                        b4[i][1].x, b4[i][1].y, b4[i][1].z, b4[i][1].w};
    float s = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      v[i][e] = __uint_as_float(e % 2 ? u[e / 2] & 0xffff0000u : u[e / 2] << 16) + b[e];
      s += v[i][e] * v[i][e];
    }
    const bool live = (int)(threadIdx.x + i * NT) * 8 < cols;
    sq += live && at[i] < q_cols ? s : 0.f;
    sk += live && at[i] >= q_cols ? s : 0.f;
  }
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  if (threadIdx.x % kWave == 0) {
    red[0][threadIdx.x / kWave] = sq;
    red[1][threadIdx.x / kWave] = sk;
  }
  __syncthreads();
  sq = sk = 0.f;
  for (int w = 0; w < NT / kWave; ++w) {
    sq += red[0][w];
    sk += red[1][w];
  }
  const float q_inv = 1.0f / sqrtf(sq / (float)(nh * real) + eps);
  const float k_inv = 1.0f / sqrtf(sk / (float)(nkv * real) + eps);
#pragma unroll
  for (int i = 0; i < CH; ++i) {
    const int c = (threadIdx.x + i * NT) * 8;
    if (c >= cols) continue;
    const bool is_q = c < q_cols;
    const float inv = is_q ? q_inv : k_inv;
    if (!is_q) store_dims<bf16_t, 8>(dst + nkv * D + c, v[i]);
    const float w[8] = {w4[i][0].x, w4[i][0].y, w4[i][0].z, w4[i][0].w,
                        w4[i][1].x, w4[i][1].y, w4[i][1].z, w4[i][1].w};
    float r[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) r[e] = v[i][e] * inv * w[e];
    if (cos_t && c % D < rot) {
      const float cs[4] = {c4[i].x, c4[i].y, c4[i].z, c4[i].w};
      const float sn[4] = {s4[i].x, s4[i].y, s4[i].z, s4[i].w};
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float a = r[2 * e], b = r[2 * e + 1];
        r[2 * e] = a * cs[e] - b * sn[e];
        r[2 * e + 1] = b * cs[e] + a * sn[e];
      }
    }
    store_dims<bf16_t, 8>(dst + c, r);
  }
}

RLIS_API int rlis_row_prepare(void* out, const void* p, int dtype, long long ldp, int T, int nh,
                              int nkv, int D, int real, const float* bias, const float* q_weight,
                              const float* k_weight, float eps, const float* cos, const float* sin,
                              int rot, const int* positions, int interleaved, hipStream_t stream) {
  RLIS_REQUIRE(T >= 0 && nh > 0 && nkv > 0 && D > 0 && real > 0 && real <= D,
               "row_prepare: bad sizes");
  RLIS_REQUIRE(ldp >= (long long)(nh + nkv) * D, "row_prepare: rows of %lld hold no %d heads of %d",
               ldp, nh + nkv, D);
  RLIS_REQUIRE(q_weight && k_weight, "row_prepare: both norms need a weight");
  RLIS_REQUIRE(!cos || (sin && positions && rot > 0 && rot % 2 == 0 && rot <= D),
               "row_prepare: a rotation of %d dims needs tables and positions", rot);
  RLIS_REQUIRE(dtype == RLIS_F32 || dtype == RLIS_BF16, "row_prepare: unknown dtype %d", dtype);
  if (T == 0) return 0;
  const bool wide = dtype == RLIS_BF16 && D % 8 == 0 && ldp % 8 == 0 && (uintptr_t)p % 16 == 0 &&
                    (uintptr_t)out % 16 == 0 && (!cos || interleaved || (rot / 2) % 8 == 0);
#define LAUNCH(TX, V, INTER)                                                                     \
  row_prepare_kernel<TX, V, INTER><<<T, 256, 0, stream>>>(                                        \
      (TX*)out, (const TX*)p, ldp, nh, nkv, D, real, bias, q_weight, k_weight, eps, cos, sin,     \
      cos ? rot : 0, positions)
  const int pieces = (nh + nkv) * D / 8;
  if (wide && interleaved && pieces <= 4096 && (!cos || (rot % 8 == 0 && (uintptr_t)cos % 16 == 0 &&
                                                         (uintptr_t)sin % 16 == 0)) &&
      (!bias || (uintptr_t)bias % 16 == 0) && (uintptr_t)q_weight % 16 == 0 && (uintptr_t)k_weight % 16 == 0) {
#define LAUNCH8(CH)                                                                                \
  row_prepare_bf16x8_kernel<CH><<<T, ceil_div(ceil_div(pieces, CH), 64) * 64, 0, stream>>>(         \
      (bf16_t*)out, (const bf16_t*)p, ldp, nh, nkv, D, real, bias, q_weight, k_weight, eps, cos,    \
      sin, cos ? rot : 0, positions)
    if (pieces <= 512) LAUNCH8(1);
    else if (pieces <= 1024) LAUNCH8(2);
    else LAUNCH8(4);
#undef LAUNCH8
    RLIS_LAUNCH_CHECK("row_prepare");
    return 0;
  }
  if (interleaved) {
    RLIS_REQUIRE(D % 2 == 0, "row_prepare: pairs of neighbouring dims need an even head size");
    if (wide) LAUNCH(bf16_t, 8, true);
    else if (dtype == RLIS_BF16) LAUNCH(bf16_t, 2, true);
    else LAUNCH(float, 2, true);
  } else {
    if (wide) LAUNCH(bf16_t, 8, false);
    else if (dtype == RLIS_BF16) LAUNCH(bf16_t, 1, false);
    else LAUNCH(float, 1, false);
  }
#undef LAUNCH
  RLIS_LAUNCH_CHECK("row_prepare");
  return 0;
}
