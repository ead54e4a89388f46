// The gated delta rule with a decay per head and key channel.  Per token and head, S being key
// channels x value channels:
//   S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q,
// g_i = exp(-exp(A_log) softplus(z_i + dt_bias_i)), beta = sigmoid(b), from the raw projections;
// all of it float32.  Column j of S is independent of the others.  With the decayed vectors
// g * k and g * q, d1 = S^T (g k) and d2 = S^T (g q) of the state in front of the token give
// u_j = beta (v_j - d1_j) and o_j = d2_j + (k . q) u_j, so both sums are over the old state.
//
// State layout, work split and tokens per tile as in recurrent.hip: [head][value channel][key
// channel] in the request's slot, a wave owns a few value channels of one (sequence, head), lane i
// holds S[i][j] (and i + 64, ... for more than 64 key channels).
#include "scan.h"
#include "tile_mma.h"

namespace {

struct ChannelDeltaArgs {
  float* out;
  long long ldo;
  const float *q, *k, *v;
  long long ldqkv;
  const float* b_raw;
  long long ldb;
  const float* z;
  long long ldz;
  const float *a_log, *dt_bias;
  float* state;
  long long state_stride;
  const int *cu, *slots;
  int heads, kv_heads, dk, dv;
};

// Decode and short portions: what does not depend on the state is made one token ahead.
template <int KR>
__global__ __launch_bounds__(256) void channel_delta_scan_kernel(const ChannelDeltaArgs a) {
  const int lane = threadIdx.x % kWave;
  const int wave = threadIdx.x / kWave;
  const int j0 = (blockIdx.x * (blockDim.x / kWave) + wave) * kCols;
  const int head = blockIdx.y;
  const int s = blockIdx.z;
  const int dk = a.dk, dv = a.dv;
  if (j0 >= dv) return;
  const int kh = head / (a.heads / a.kv_heads);
  const int t0 = a.cu[s], t1 = a.cu[s + 1];
  float* base = a.state + (long long)a.slots[s] * a.state_stride + (long long)head * dv * dk;
  int idx[KR];
  float live[KR], bias[KR];
#pragma unroll
  for (int r = 0; r < KR; ++r) {
    const int i = lane + r * kWave;
    idx[r] = i < dk ? i : dk - 1;
    live[r] = i < dk ? 1.f : 0.f;
    bias[r] = a.dt_bias[head * dk + idx[r]];
  }
  int col[kCols];
#pragma unroll
  for (int c = 0; c < kCols; ++c) col[c] = j0 + c < dv ? j0 + c : dv - 1;
  float S[kCols][KR];
#pragma unroll
  for (int c = 0; c < kCols; ++c)
#pragma unroll
    for (int r = 0; r < KR; ++r) S[c][r] = base[(long long)col[c] * dk + idx[r]] * live[r];
  const float neg_a = -expf(a.a_log[head]);
  float kn[KR], qn[KR], gn[KR], vn[kCols], betan = 0.f, kqn = 0.f;
  auto fetch = [&](int t) {
    const float* kt = a.k + (long long)t * a.ldqkv + kh * dk;
    const float* qt = a.q + (long long)t * a.ldqkv + kh * dk;
    const float* zt = a.z + (long long)t * a.ldz + head * dk;
    float kq = 0.f;
#pragma unroll
    for (int r = 0; r < KR; ++r) {
      kn[r] = kt[idx[r]] * live[r];
      qn[r] = qt[idx[r]] * live[r];
      gn[r] = expf(neg_a * softplusf_(zt[idx[r]] + bias[r]));
      kq += kn[r] * qn[r];
    }
#pragma unroll
    for (int c = 0; c < kCols; ++c) vn[c] = a.v[(long long)t * a.ldqkv + head * dv + col[c]];
    betan = sigmoidf_(a.b_raw[(long long)t * a.ldb + head]);
    kqn = lanes_sum(kq);
  };
  if (t0 < t1) fetch(t0);
  for (int t = t0; t < t1; ++t) {
    float kc[KR], gk[KR], gq[KR], g[KR], vc[kCols];
#pragma unroll
    for (int r = 0; r < KR; ++r) {
      g[r] = gn[r];
      kc[r] = kn[r];
      gk[r] = gn[r] * kn[r];
      gq[r] = gn[r] * qn[r];
    }
#pragma unroll
    for (int c = 0; c < kCols; ++c) vc[c] = vn[c];
    const float beta = betan, kq = kqn;
    fetch(t + 1 < t1 ? t + 1 : t);
    float d1[kCols], d2[kCols];
#pragma unroll
    for (int c = 0; c < kCols; ++c) {
      d1[c] = 0.f;
      d2[c] = 0.f;
#pragma unroll
      for (int r = 0; r < KR; ++r) {
        d1[c] += S[c][r] * gk[r];
        d2[c] += S[c][r] * gq[r];
      }
    }
#pragma unroll
    for (int c = 0; c < kCols; ++c) {
      d1[c] = lanes_sum(d1[c]);
      d2[c] = lanes_sum(d2[c]);
    }
#pragma unroll
    for (int c = 0; c < kCols; ++c) {
      const float u = beta * (vc[c] - d1[c]);
#pragma unroll
      for (int r = 0; r < KR; ++r) S[c][r] = g[r] * S[c][r] + kc[r] * u;
      if (lane == c && j0 + c < dv)
        a.out[(long long)t * a.ldo + head * dv + j0 + c] = d2[c] + kq * u;
    }
  }
#pragma unroll
  for (int c = 0; c < kCols; ++c)
    if (j0 + c < dv) {
#pragma unroll
      for (int r = 0; r < KR; ++r)
        if (lane + r * kWave < dk) base[(long long)(j0 + c) * dk + lane + r * kWave] = S[c][r];
    }
}

// Long runs: tiles of tokens go through LDS (the next tile waits in registers meanwhile), and
// tokens are walked in pairs whose sums over the wave are all over the state in front of the
// pair.  With decays g0, g1 of the two tokens:
//   u0 = beta0 (v0 - S^T (g0 k0)),            o0 = S^T (g0 q0) + (k0.q0) u0
//   u1 = beta1 (v1 - S^T (g0 g1 k1) - (g1 k0 . k1) u0)
//   o1 = S^T (g0 g1 q1) + (g1 k0 . q1) u0 + (k1.q1) u1
//   S <- g0 g1 S + (g1 k0) u0^T + k1 u1^T
// The four products of the tokens' own vectors are made once a tile by the four waves together.
// Tokens past the end carry k = q = 0, beta = 0 and g = 1.
template <int KR, int NC>
__global__ __launch_bounds__(256) void channel_delta_tiled_kernel(const ChannelDeltaArgs a) {
  constexpr int TT = KR == 4 ? 8 : 16, DK = KR * kWave, CB = 4 * NC, GROUP = kWave / NC;
  __shared__ float tk[TT][DK], tq[TT][DK], tg[TT][DK], tv[TT][CB], tb[TT];
  __shared__ __attribute__((aligned(16))) float tp[TT / 2][4];
  const int lane = threadIdx.x % kWave;
  const int wave = threadIdx.x / kWave;
  const int dk = a.dk, dv = a.dv;
  const int jb = blockIdx.x * CB;
  const int j0 = jb + wave * NC;
  const int head = blockIdx.y;
  const int s = blockIdx.z;
  const int kh = head / (a.heads / a.kv_heads);
  const int t0 = a.cu[s], t1 = a.cu[s + 1];
  float* base = a.state + (long long)a.slots[s] * a.state_stride + (long long)head * dv * dk;
  float S[NC][KR];
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int col = j0 + c < dv ? j0 + c : dv - 1;
#pragma unroll
    for (int r = 0; r < KR; ++r) {
      const int i = lane + r * kWave;
      S[c][r] = base[(long long)col * dk + (i < dk ? i : dk - 1)] * (i < dk ? 1.f : 0.f);
    }
  }
  const float neg_a = -expf(a.a_log[head]);
  constexpr int PER = TT * DK / 256, PERV = (TT * CB + 255) / 256;
  static_assert(TT * DK % 256 == 0 && TT <= 256, "tile sizes");
  float rk[PER], rq[PER], rz[PER], rv[PERV], rb = 0.f;
  auto ask = [&](int tile) {
    const int n = min(TT, t1 - tile);
#pragma unroll
    for (int p = 0; p < PER; ++p) {
      const int e = threadIdx.x + p * 256, tt = e / DK, i = e % DK;
      const int ic = i < dk ? i : dk - 1;
      const long long t = tile + (tt < n ? tt : n - 1);
      const long long row = t * a.ldqkv + kh * dk;
      const float keep = (tt < n && i < dk) ? 1.f : 0.f;
      rk[p] = a.k[row + ic] * keep;
      rq[p] = a.q[row + ic] * keep;
      rz[p] = a.z[t * a.ldz + head * dk + ic] + a.dt_bias[head * dk + ic];
    }
#pragma unroll
    for (int p = 0; p < PERV; ++p) {
      const int e = min((int)threadIdx.x + p * 256, TT * CB - 1), tt = e / CB, c = e % CB;
      const int col = jb + c < dv ? jb + c : dv - 1;
      rv[p] = a.v[(long long)(tile + (tt < n ? tt : n - 1)) * a.ldqkv + head * dv + col];
    }
    const int tt = threadIdx.x < TT ? threadIdx.x : TT - 1;
    rb = a.b_raw[(long long)(tile + (tt < n ? tt : n - 1)) * a.ldb + head];
  };
  if (t0 < t1) ask(t0);
  for (int tile = t0; tile < t1; tile += TT) {
    const int n = min(TT, t1 - tile);
    __syncthreads();                               // the tile before has been walked
#pragma unroll
    for (int p = 0; p < PER; ++p) {
      const int e = threadIdx.x + p * 256;
      tk[e / DK][e % DK] = rk[p];
      tq[e / DK][e % DK] = rq[p];
      tg[e / DK][e % DK] = e / DK < n ? expf(neg_a * softplusf_(rz[p])) : 1.f;
    }
#pragma unroll
    for (int p = 0; p < PERV; ++p) {
      const int e = threadIdx.x + p * 256;
      if (e < TT * CB) tv[e / CB][e % CB] = rv[p];
    }
    if (threadIdx.x < TT) tb[threadIdx.x] = (int)threadIdx.x < n ? sigmoidf_(rb) : 0.f;
    __syncthreads();
    ask(tile + TT < t1 ? tile + TT : tile);
    // entries of pair f: k0.q0, (g1 k0).k1, (g1 k0).q1, k1.q1
    for (int f = wave; f < TT / 2; f += 4) {
      float four[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int r = 0; r < KR; ++r) {
        const int i = lane + r * kWave;
        const float k0 = tk[2 * f][i], k1 = tk[2 * f + 1][i], q1 = tq[2 * f + 1][i];
        const float gk0 = tg[2 * f + 1][i] * k0;
        four[0] += k0 * tq[2 * f][i];
        four[1] += gk0 * k1;
        four[2] += gk0 * q1;
        four[3] += k1 * q1;
      }
      const float mine = lanes_sum4(four, lane);               // of entry lane % 4
      if (lane < 4) tp[f][lane] = mine;
    }
    __syncthreads();
    // Lane l gathers the read-out of token l / NC of a group for column l % NC and stores it when
    // the group is through: one store a group.
    float gathered = 0.f;
    for (int tb0 = 0; tb0 < n; tb0 += 2) {
      float k0[KR], k1[KR], g01[KR], s10[NC], s11[NC], s20[NC], s21[NC];
#pragma unroll
      for (int c = 0; c < NC; ++c) s10[c] = s11[c] = s20[c] = s21[c] = 0.f;
#pragma unroll
      for (int r = 0; r < KR; ++r) {
        const int i = lane + r * kWave;
        const float ga = tg[tb0][i], gb = tg[tb0 + 1][i];
        const float ka = tk[tb0][i];
        g01[r] = ga * gb;
        k0[r] = gb * ka;
        k1[r] = tk[tb0 + 1][i];
        const float xa = ga * ka, ya = ga * tq[tb0][i];
        const float xb = g01[r] * k1[r], yb = g01[r] * tq[tb0 + 1][i];
#pragma unroll
        for (int c = 0; c < NC; ++c) {
          s10[c] += S[c][r] * xa;
          s20[c] += S[c][r] * ya;
          s11[c] += S[c][r] * xb;
          s21[c] += S[c][r] * yb;
        }
      }
      float d10, d20, d11, d21;
      if constexpr (NC == 2) {
        const float fa[4] = {s10[0], s10[1], s20[0], s20[1]}, fb[4] = {s11[0], s11[1], s21[0], s21[1]};
        const float ma = lanes_sum4(fa, lane), mb = lanes_sum4(fb, lane);
        d10 = dpp_from<0x44>(ma);                              // quad_perm [0, 1, 0, 1]
        d20 = dpp_from<0xEE>(ma);                              // quad_perm [2, 3, 2, 3]
        d11 = dpp_from<0x44>(mb);
        d21 = dpp_from<0xEE>(mb);
      } else {
        d10 = lanes_sum_cols<NC>(s10, lane);
        d20 = lanes_sum_cols<NC>(s20, lane);
        d11 = lanes_sum_cols<NC>(s11, lane);
        d21 = lanes_sum_cols<NC>(s21, lane);
      }
      const float4 pair = *(const float4*)tp[tb0 / 2];
      const float v0 = tv[tb0][wave * NC + (lane & (NC - 1))];
      const float v1 = tv[tb0 + 1][wave * NC + (lane & (NC - 1))];
      const float u0 = tb[tb0] * (v0 - d10);
      const float u1 = tb[tb0 + 1] * (v1 - d11 - pair.y * u0);
      if (lane / NC == tb0 % GROUP) gathered = d20 + pair.x * u0;
      if (lane / NC == (tb0 + 1) % GROUP) gathered = d21 + pair.z * u0 + pair.w * u1;
      float c0[NC], c1[NC];
      c0[0] = dpp_from<0x00>(u0);
      c0[1] = dpp_from<0x55>(u0);
      c1[0] = dpp_from<0x00>(u1);
      c1[1] = dpp_from<0x55>(u1);
      if constexpr (NC == 4) {
        c0[2] = dpp_from<0xAA>(u0);
        c0[3] = dpp_from<0xFF>(u0);
        c1[2] = dpp_from<0xAA>(u1);
        c1[3] = dpp_from<0xFF>(u1);
      }
#pragma unroll
      for (int c = 0; c < NC; ++c)
#pragma unroll
        for (int r = 0; r < KR; ++r) S[c][r] = g01[r] * S[c][r] + k0[r] * c0[c] + k1[r] * c1[c];
      if ((tb0 + 2) % GROUP == 0 || tb0 + 2 >= n) {
        const int token = tb0 / GROUP * GROUP + lane / NC;
        if (token < n && token < tb0 + 2 && j0 + (lane & (NC - 1)) < dv)
          a.out[(long long)(tile + token) * a.ldo + head * dv + j0 + (lane & (NC - 1))] = gathered;
      }
    }
  }
#pragma unroll
  for (int c = 0; c < NC; ++c)
    if (j0 + c < dv) {
#pragma unroll
      for (int r = 0; r < KR; ++r)
        if (lane + r * kWave < dk) base[(long long)(j0 + c) * dk + lane + r * kWave] = S[c][r];
    }
}

// ------------------------------------------------------------------------ long portions
// Chunks of kChunk tokens on the matrix cores, float32 products (v_mfma_f32_16x16x4_f32).  With S0
// the state in front of a chunk and G(t, s) the products of the decays of tokens s + 1 .. t per
// key channel (G(t) from the chunk's start), the writes u_t of a chunk solve
//   u_t = beta_t (v_t - S0^T (G(t) k_t) - sum_{s<t} A[t][s] u_s),  A[t][s] = sum_i G(t,s) k_t k_s,
// a unit lower triangular system that does not depend on S0: with U0 its solution for the right
// hand side beta v and W that for beta (G k),  U = U0 - W S0, and
//   o_t = S0^T (G(t) q_t) + sum_{s<=t} B[t][s] u_s,          B[t][s] = sum_i G(t,s) q_t k_s,
//   S  <- G(n) S0 + sum_s (G(n, s) k_s) u_s^T.
// Three launches: what does not depend on the state, chunk by chunk and head by head side by
// side; the states, chunk after chunk, a workgroup per 16 value channels; the read-outs, side by
// side again.
//
// No decay is ever divided by: inside 16 tokens G(t, s) is formed by multiplying the decays up from s;
// between blocks of 16 it is split at the later block's start into two factors that are at most
// one, the exponentials of sums of logarithms that all have one sign.  So strong decays
// underflow to zero and nothing overflows or cancels.
constexpr int kChunk = 64, kSub = 16, kSubs = kChunk / kSub;

struct ChannelDeltaChunks {
  ChannelDeltaArgs a;
  int num_seqs, max_chunks, dvp;   // dvp: value channels rounded up to 16
  float *w, *qt, *kt, *u, *b, *gc, *s0;
};

// Per (chunk, head): w (64, DK), qt (64, DK) = G q, kt (DK, 64) = G(n, s) k, u (dvp, 64), b (64, 64),
// gc (DK) = G(n), s0 (dvp, DK).
template <int DK>
__host__ __device__ constexpr long long chunk_floats(int dvp) {
  return 3LL * kChunk * DK + (long long)dvp * kChunk + kChunk * kChunk + DK + (long long)dvp * DK;
}

template <int DK>
struct PrepLds {
  static constexpr int kStride = DK + 4;
  float k[kChunk][kStride], q[kChunk][kStride], g[kChunk][kStride], p[kChunk][kStride];
  float a[kChunk][kChunk + 4];
  float end[kSubs][DK];
  float beta[kChunk];
};

__device__ __forceinline__ float4 ld4(const float* p) { return *(const float4*)p; }
__device__ __forceinline__ void mfma4(const float4& a, const float4& b, mma_f32x4& acc) {
  acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x, b.x, acc, 0, 0, 0);
  acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.y, b.y, acc, 0, 0, 0);
  acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.z, b.z, acc, 0, 0, 0);
  acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.w, b.w, acc, 0, 0, 0);
}

template <int DK>
__global__ __launch_bounds__(256) void channel_delta_prepare_kernel(const ChannelDeltaChunks c) {
  extern __shared__ __attribute__((aligned(16))) char prep_smem[];
  PrepLds<DK>& L = *reinterpret_cast<PrepLds<DK>*>(prep_smem);
  const ChannelDeltaArgs& a = c.a;
  const int chunk = blockIdx.x, head = blockIdx.y;
  int t0, t1;
  if (!chunk_span(a.cu, c.num_seqs, kChunk, chunk, t0, t1)) return;   // (the whole workgroup)
  const int n = t1 - t0;
  const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave;
  const int kh = head / (a.heads / a.kv_heads);
  const int dk = a.dk, dv = a.dv;
  const long long at = (long long)chunk * a.heads + head;
  float* ws_w = c.w + at * kChunk * DK;
  float* ws_qt = c.qt + at * kChunk * DK;
  float* ws_kt = c.kt + at * kChunk * DK;
  float* ws_u = c.u + at * c.dvp * kChunk;
  float* ws_b = c.b + at * kChunk * kChunk;
  const float neg_a = -expf(a.a_log[head]);
  if (tid < kChunk) {
    const float raw = a.b_raw[(long long)(t0 + min(tid, n - 1)) * a.ldb + head];
    L.beta[tid] = tid < n ? sigmoidf_(raw) : 0.f;
  }
  // A thread owns (channel, block of 16 tokens) items: their inputs, the logarithms of the decays
  // (kept in registers), the running sums from the block's start.  Tokens past the end carry zero
  // keys and no decay.
  constexpr int ITEMS = DK * kSubs / 256;
  float lg[ITEMS][kSub];
#pragma unroll
  for (int it = 0; it < ITEMS; ++it) {
    const int id = tid + it * 256, ch = id % DK, sub = id / DK;
    const int ic = min(ch, dk - 1);
    const float bias = a.dt_bias[head * dk + ic];
    float kv[kSub], qv[kSub];
#pragma unroll
    for (int j = 0; j < kSub; ++j) {
      const long long t = t0 + min(sub * kSub + j, n - 1);
      lg[it][j] = a.z[t * a.ldz + head * dk + ic];
      kv[j] = a.k[t * a.ldqkv + kh * dk + ic];
      qv[j] = a.q[t * a.ldqkv + kh * dk + ic];
    }
    float sum = 0.f;
#pragma unroll
    for (int j = 0; j < kSub; ++j) {
      const int t = sub * kSub + j;
      const bool live = t < n && ch < dk;
      lg[it][j] = live ? neg_a * softplusf_(lg[it][j] + bias) : 0.f;
      sum += lg[it][j];
      L.k[t][ch] = live ? kv[j] : 0.f;
      L.q[t][ch] = live ? qv[j] : 0.f;
      L.g[t][ch] = expf(lg[it][j]);
      L.p[t][ch] = sum;
    }
    L.end[sub][ch] = sum;
  }
  __syncthreads();
  // Blocks of 16 x 16 on the diagonal: lane l carries column s = l % 16 for a quarter of the
  // channels; w = G(t, s) k_s is multiplied up as t goes on.  (For t <= s the entries of A mean
  // nothing and are not read; those of B are zero for t < s.)
  {
    const int s = lane % 16, gq = lane / 16, r0 = wave * kSub;
    float acc_a[kSub], acc_b[kSub];
#pragma unroll
    for (int j = 0; j < kSub; ++j) acc_a[j] = acc_b[j] = 0.f;
    for (int m = 0; m < DK / 16; ++m) {
      const int i = 16 * m + 4 * gq;
      const float4 ks = ld4(&L.k[r0 + s][i]);
      float4 w = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
      for (int j = 0; j < kSub; ++j) {
        const float4 g4 = ld4(&L.g[r0 + j][i]), k4 = ld4(&L.k[r0 + j][i]), q4 = ld4(&L.q[r0 + j][i]);
        const bool own = j == s;
        w.x = own ? ks.x : w.x * g4.x;
        w.y = own ? ks.y : w.y * g4.y;
        w.z = own ? ks.z : w.z * g4.z;
        w.w = own ? ks.w : w.w * g4.w;
        acc_a[j] += (k4.x * w.x + k4.y * w.y) + (k4.z * w.z + k4.w * w.w);
        acc_b[j] += (q4.x * w.x + q4.y * w.y) + (q4.z * w.z + q4.w * w.w);
      }
    }
#pragma unroll
    for (int j = 0; j < kSub; ++j) {
      acc_a[j] = xor32_sum(xor16_sum(acc_a[j]));
      acc_b[j] = xor32_sum(xor16_sum(acc_b[j]));
      if (j / 4 == gq) {
        L.a[r0 + j][r0 + s] = acc_a[j];
        ws_b[(r0 + j) * kChunk + r0 + s] = acc_b[j];
      }
    }
  }
  __syncthreads();
  // The decays make room for the sums of the logarithms behind a token, up to its block's end; on
  // the way, what the state's update and the read-out take: G(n, s) k and G q.
#pragma unroll
  for (int it = 0; it < ITEMS; ++it) {
    const int id = tid + it * 256, ch = id % DK, sub = id / DK;
    float before = 0.f, behind = 0.f;
    for (int r = 0; r < sub; ++r) before += L.end[r][ch];
    for (int r = sub + 1; r < kSubs; ++r) behind += L.end[r][ch];
    float suffix = 0.f, khat[kSub];
#pragma unroll
    for (int j = kSub - 1; j >= 0; --j) {
      const int t = sub * kSub + j;
      L.g[t][ch] = suffix;
      khat[j] = L.k[t][ch] * expf(suffix + behind);
      suffix += lg[it][j];
      ws_qt[t * DK + ch] = L.q[t][ch] * expf(before + L.p[t][ch]);
    }
#pragma unroll
    for (int j = 0; j < kSub; j += 4)
      *(float4*)(ws_kt + ch * kChunk + sub * kSub + j) =
          make_float4(khat[j], khat[j + 1], khat[j + 2], khat[j + 3]);
    if (sub == kSubs - 1) c.gc[at * DK + ch] = expf(before + L.end[sub][ch]);
  }
  __syncthreads();
  // Blocks below the diagonal: block ba against an earlier block bb, G(t, s) split at ba's start.
  for (int pair = wave; pair < kSubs * (kSubs - 1) / 2; pair += 4) {
    const int ba = pair < 1 ? 1 : (pair < 3 ? 2 : 3), bb = pair - ba * (ba - 1) / 2;
    const int row = ba * kSub + lane % 16, col = bb * kSub + lane % 16, g = lane / 16;
    mma_f32x4 acc_a = {0.f, 0.f, 0.f, 0.f}, acc_b = {0.f, 0.f, 0.f, 0.f};
    for (int m = 0; m < DK / 16; ++m) {
      const int i = 16 * m + 4 * g;
      float4 between = ld4(&L.g[col][i]);
      for (int r = bb + 1; r < ba; ++r) {
        const float4 e = ld4(&L.end[r][i]);
        between.x += e.x;
        between.y += e.y;
        between.z += e.z;
        between.w += e.w;
      }
      const float4 p = ld4(&L.p[row][i]);
      float4 kr = ld4(&L.k[row][i]), qr = ld4(&L.q[row][i]), kc = ld4(&L.k[col][i]);
      const float4 e = make_float4(expf(p.x), expf(p.y), expf(p.z), expf(p.w));
      kr.x *= e.x; kr.y *= e.y; kr.z *= e.z; kr.w *= e.w;
      qr.x *= e.x; qr.y *= e.y; qr.z *= e.z; qr.w *= e.w;
      kc.x *= expf(between.x); kc.y *= expf(between.y);
      kc.z *= expf(between.z); kc.w *= expf(between.w);
      mfma4(kr, kc, acc_a);
      mfma4(qr, kc, acc_b);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = ba * kSub + 4 * g + i;
      L.a[t][col] = acc_a[i];
      ws_b[t * kChunk + col] = acc_b[i];
    }
  }
  __syncthreads();
  // The triangular system, a thread per column: key channels (W) first, value channels (U0) behind.
  for (int col = tid; col < DK + c.dvp; col += 256) {
    float x[kChunk];
    if (col < DK) {
#pragma unroll
      for (int sub = 0; sub < kSubs; ++sub) {
        float before = 0.f;
        for (int r = 0; r < sub; ++r) before += L.end[r][col];
#pragma unroll
        for (int j = 0; j < kSub; ++j) {
          const int t = sub * kSub + j;
          x[t] = L.k[t][col] * expf(before + L.p[t][col]);
        }
      }
    } else {
      const float* v = a.v + (long long)t0 * a.ldqkv + head * dv + min(col - DK, dv - 1);
#pragma unroll
      for (int t = 0; t < kChunk; ++t) x[t] = v[(long long)min(t, n - 1) * a.ldqkv];
      const bool real = col - DK < dv;
#pragma unroll
      for (int t = 0; t < kChunk; ++t) x[t] = (real && t < n) ? x[t] : 0.f;
    }
#pragma unroll
    for (int t = 0; t < kChunk; ++t) {
      float s4[4] = {x[t], 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < t; s += 4) {
        const float4 r = ld4(&L.a[t][s]);
        s4[0] -= r.x * x[s];
        if (s + 1 < t) s4[1] -= r.y * x[s + 1];
        if (s + 2 < t) s4[2] -= r.z * x[s + 2];
        if (s + 3 < t) s4[3] -= r.w * x[s + 3];
      }
      x[t] = L.beta[t] * ((s4[0] + s4[1]) + (s4[2] + s4[3]));
    }
    if (col < DK) {
#pragma unroll
      for (int t = 0; t < kChunk; ++t) ws_w[t * DK + col] = x[t];
    } else {
#pragma unroll
      for (int t = 0; t < kChunk; t += 4)
        *(float4*)(ws_u + (long long)(col - DK) * kChunk + t) = make_float4(x[t], x[t + 1], x[t + 2], x[t + 3]);
    }
  }
}

// The states: a workgroup per (16 value channels, head, sequence) walks the sequence's chunks.  Wave
// w owns the key channels of its DK / 64 tiles of 16 (registers: rows 4 (lane / 16) + i, column
// lane % 16) and 16 tokens of U.  A chunk's operands are asked for one chunk ahead.
template <int DK>
__global__ __launch_bounds__(256) void channel_delta_states_kernel(const ChannelDeltaChunks c) {
  constexpr int KT = DK / 64, KM = DK / 16, TM = kChunk / 16;
  __shared__ __attribute__((aligned(16))) float ssm[16][DK + 4], usm[16][kChunk + 4];
  const ChannelDeltaArgs& a = c.a;
  const int head = blockIdx.y, s = blockIdx.z;
  const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
  const int l16 = lane % 16, g = lane / 16;
  const int col = blockIdx.x * 16 + l16;
  const int dk = a.dk, dv = a.dv;
  const int first = chunks_before(a.cu, s, kChunk);
  const int chunks = (a.cu[s + 1] - a.cu[s] + kChunk - 1) / kChunk;
  if (chunks == 0) return;
  float* base = a.state + (long long)a.slots[s] * a.state_stride + (long long)head * dv * dk;
  mma_f32x4 S[KT];
#pragma unroll
  for (int j = 0; j < KT; ++j) {
    const int key = (wave * KT + j) * 16 + 4 * g;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const bool live = key + i < dk && col < dv;
      const float v = base[live ? (long long)col * dk + key + i : 0];
      S[j][i] = live ? v : 0.f;
    }
    *(float4*)&ssm[l16][key] = make_float4(S[j][0], S[j][1], S[j][2], S[j][3]);
  }
  float4 wf[KM], kf[KT][TM], uf, gf[KT];
  auto ask = [&](int chunk) {
    const long long at = (long long)(first + chunk) * a.heads + head;
    const float* w = c.w + at * kChunk * DK + (wave * 16 + l16) * DK + 4 * g;
#pragma unroll
    for (int m = 0; m < KM; ++m) wf[m] = ld4(w + 16 * m);
    uf = ld4(c.u + (at * c.dvp + col) * kChunk + wave * 16 + 4 * g);
#pragma unroll
    for (int j = 0; j < KT; ++j) {
      const int tile = (wave * KT + j) * 16;
      const float* kt = c.kt + at * kChunk * DK + (tile + l16) * kChunk + 4 * g;
#pragma unroll
      for (int m = 0; m < TM; ++m) kf[j][m] = ld4(kt + 16 * m);
      gf[j] = ld4(c.gc + at * DK + tile + 4 * g);
    }
  };
  ask(0);
  __syncthreads();
  for (int k = 0; k < chunks; ++k) {
    const long long at = (long long)(first + k) * a.heads + head;
    float* s0 = c.s0 + (at * c.dvp + col) * DK;
#pragma unroll
    for (int j = 0; j < KT; ++j)
      *(float4*)(s0 + (wave * KT + j) * 16 + 4 * g) = make_float4(S[j][0], S[j][1], S[j][2], S[j][3]);
    mma_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int m = 0; m < KM; ++m) mfma4(wf[m], ld4(&ssm[l16][16 * m + 4 * g]), acc);
    const float4 u = make_float4(uf.x - acc[0], uf.y - acc[1], uf.z - acc[2], uf.w - acc[3]);
    *(float4*)&usm[l16][wave * 16 + 4 * g] = u;
    *(float4*)(c.u + (at * c.dvp + col) * kChunk + wave * 16 + 4 * g) = u;
    float4 kn[KT][TM];
#pragma unroll
    for (int j = 0; j < KT; ++j) {
#pragma unroll
      for (int m = 0; m < TM; ++m) kn[j][m] = kf[j][m];
      S[j][0] *= gf[j].x;
      S[j][1] *= gf[j].y;
      S[j][2] *= gf[j].z;
      S[j][3] *= gf[j].w;
    }
    ask(k + 1 < chunks ? k + 1 : k);          // (the last chunk's again: not used)
    __syncthreads();
#pragma unroll
    for (int m = 0; m < TM; ++m) {
      const float4 ub = ld4(&usm[l16][16 * m + 4 * g]);
#pragma unroll
      for (int j = 0; j < KT; ++j) mfma4(kn[j][m], ub, S[j]);
    }
#pragma unroll
    for (int j = 0; j < KT; ++j)
      *(float4*)&ssm[l16][(wave * KT + j) * 16 + 4 * g] = make_float4(S[j][0], S[j][1], S[j][2], S[j][3]);
    __syncthreads();
  }
#pragma unroll
  for (int j = 0; j < KT; ++j) {
    const int key = (wave * KT + j) * 16 + 4 * g;
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (key + i < dk && col < dv) base[(long long)col * dk + key + i] = S[j][i];
  }
}

// The read-outs: wave w takes 16 tokens of a chunk against up to 64 value channels.
template <int DK>
__global__ __launch_bounds__(256) void channel_delta_outputs_kernel(const ChannelDeltaChunks c) {
  constexpr int NB = 4;
  const ChannelDeltaArgs& a = c.a;
  const int chunk = blockIdx.x, head = blockIdx.y, c0 = blockIdx.z * 16 * NB;
  int t0, t1;
  if (!chunk_span(a.cu, c.num_seqs, kChunk, chunk, t0, t1)) return;
  const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
  const int l16 = lane % 16, g = lane / 16;
  if (t0 + wave * 16 >= t1) return;
  const long long at = (long long)chunk * a.heads + head;
  const float* q = c.qt + at * kChunk * DK + (wave * 16 + l16) * DK + 4 * g;
  const float* b = c.b + at * kChunk * kChunk + (wave * 16 + l16) * kChunk + 4 * g;
  const float *s[NB], *u[NB];
  mma_f32x4 acc[NB];
#pragma unroll
  for (int x = 0; x < NB; ++x) {
    const int col = min(c0 + x * 16, c.dvp - 16) + l16;      // (past the end: not stored)
    s[x] = c.s0 + (at * c.dvp + col) * DK + 4 * g;
    u[x] = c.u + (at * c.dvp + col) * kChunk + 4 * g;
    acc[x] = mma_f32x4{0.f, 0.f, 0.f, 0.f};
  }
#pragma unroll 4
  for (int m = 0; m < DK / 16; ++m) {
    const float4 qa = ld4(q + 16 * m);
#pragma unroll
    for (int x = 0; x < NB; ++x) mfma4(qa, ld4(s[x] + 16 * m), acc[x]);
  }
  for (int m = 0; m <= wave; ++m) {
    const float4 ba = ld4(b + 16 * m);
#pragma unroll
    for (int x = 0; x < NB; ++x) mfma4(ba, ld4(u[x] + 16 * m), acc[x]);
  }
#pragma unroll
  for (int x = 0; x < NB; ++x) {
    const int col = c0 + x * 16 + l16;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = t0 + wave * 16 + 4 * g + i;
      if (t < t1 && col < a.dv) a.out[(long long)t * a.ldo + head * a.dv + col] = acc[x][i];
    }
  }
}

template <int DK>
int launch_channel_delta_chunks(ChannelDeltaChunks c, float* ws, hipStream_t stream) {
  const long long n = (long long)c.max_chunks * c.a.heads;
  c.w = ws;
  c.qt = c.w + n * kChunk * DK;
  c.kt = c.qt + n * kChunk * DK;
  c.u = c.kt + n * kChunk * DK;
  c.b = c.u + n * c.dvp * kChunk;
  c.gc = c.b + n * kChunk * kChunk;
  c.s0 = c.gc + n * DK;
  static LdsGrant grant;
  constexpr int bytes = (int)sizeof(PrepLds<DK>);
  static_assert(bytes <= 160 * 1024, "the chunk does not fit the LDS");
  const hipError_t e = grant_lds(grant, (const void*)&channel_delta_prepare_kernel<DK>, bytes);
  RLIS_REQUIRE(e == hipSuccess, "channel_delta_chunks: %d bytes of LDS: %s", bytes, hipGetErrorString(e));
  channel_delta_prepare_kernel<DK><<<dim3(c.max_chunks, c.a.heads), 256, bytes, stream>>>(c);
  RLIS_LAUNCH_CHECK("channel_delta_chunks");
  channel_delta_states_kernel<DK><<<dim3(c.dvp / 16, c.a.heads, c.num_seqs), 256, 0, stream>>>(c);
  RLIS_LAUNCH_CHECK("channel_delta_chunks");
  channel_delta_outputs_kernel<DK><<<dim3(c.max_chunks, c.a.heads, ceil_div(c.dvp, 64)), 256, 0, stream>>>(c);
  RLIS_LAUNCH_CHECK("channel_delta_chunks");
  return 0;
}

}  // namespace

// Floats of workspace per (chunk, head) that rlis_channel_delta_chunks needs.
RLIS_API long long rlis_channel_delta_chunk_floats(int dk, int dv) {
  const int dvp = ceil_div(dv, 16) * 16;
  return dk <= 64 ? chunk_floats<64>(dvp) : chunk_floats<128>(dvp);
}

// rlis_channel_delta_scan for steps with long portions; max_chunks: at least the chunks of 64
// tokens of all sequences together; ws: max_chunks * heads * rlis_channel_delta_chunk_floats floats,
// 16-byte aligned.
RLIS_API int rlis_channel_delta_chunks(float* out, long long ldo, const float* q, const float* k,
                                       const float* v, long long ldqkv, const float* b_raw,
                                       long long ldb, const float* z, long long ldz,
                                       const float* a_log, const float* dt_bias, float* state,
                                       long long state_stride, const int* cu, const int* slots,
                                       int num_seqs, int heads, int kv_heads, int dk, int dv,
                                       int max_chunks, float* ws, hipStream_t stream) {
  RLIS_REQUIRE(heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && dk > 0 && dv > 0,
               "channel_delta_chunks: bad sizes heads=%d kv_heads=%d dk=%d dv=%d", heads, kv_heads, dk, dv);
  RLIS_REQUIRE(dk <= 128, "channel_delta_chunks: %d key channels, at most 128", dk);
  RLIS_REQUIRE(state_stride >= (long long)heads * dk * dv, "channel_delta_chunks: the state is too short");
  RLIS_REQUIRE(ldz >= (long long)heads * dk && ldb >= heads && ldo >= (long long)heads * dv,
               "channel_delta_chunks: rows shorter than the heads they hold");
  RLIS_REQUIRE(heads <= 65535 && num_seqs <= 65535 && max_chunks > 0 && ws && (uintptr_t)ws % 16 == 0,
               "channel_delta_chunks: %d chunks, or no aligned workspace", max_chunks);
  if (num_seqs <= 0) return 0;
  ChannelDeltaChunks c;
  c.a = ChannelDeltaArgs{out, ldo, q, k, v, ldqkv, b_raw, ldb, z, ldz, a_log, dt_bias, state,
                         state_stride, cu, slots, heads, kv_heads, dk, dv};
  c.num_seqs = num_seqs;
  c.max_chunks = max_chunks;
  c.dvp = ceil_div(dv, 16) * 16;
  return dk <= 64 ? launch_channel_delta_chunks<64>(c, ws, stream)
                  : launch_channel_delta_chunks<128>(c, ws, stream);
}

RLIS_API int rlis_channel_delta_scan(float* out, long long ldo, const float* q, const float* k,
                                     const float* v, long long ldqkv, const float* b_raw,
                                     long long ldb, const float* z, long long ldz,
                                     const float* a_log, const float* dt_bias, float* state,
                                     long long state_stride, const int* cu, const int* slots,
                                     int num_seqs, int heads, int kv_heads, int dk, int dv,
                                     int tiled, hipStream_t stream) {
  RLIS_REQUIRE(heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && dk > 0 && dv > 0,
               "channel_delta_scan: bad sizes heads=%d kv_heads=%d dk=%d dv=%d", heads, kv_heads, dk, dv);
  RLIS_REQUIRE(dk <= 256, "channel_delta_scan: %d key channels, at most 256", dk);
  RLIS_REQUIRE(state_stride >= (long long)heads * dk * dv, "channel_delta_scan: the state is too short");
  RLIS_REQUIRE(ldz >= (long long)heads * dk && ldb >= heads && ldo >= (long long)heads * dv,
               "channel_delta_scan: rows shorter than the heads they hold");
  RLIS_REQUIRE(heads <= 65535 && num_seqs <= 65535, "channel_delta_scan: grid too large");
  if (num_seqs <= 0) return 0;
  const ChannelDeltaArgs a{out, ldo, q, k, v, ldqkv, b_raw, ldb, z, ldz, a_log, dt_bias, state,
                           state_stride, cu, slots, heads, kv_heads, dk, dv};
  const dim3 grid(ceil_div(dv, 4 * kCols), heads, num_seqs);
  // few workgroups (a single prompt): two value channels a wave instead of four, twice the waves
  // (tiled 2 / 3: four / two channels a wave whatever the grid, for tests)
  const bool narrow = tiled == 3 || (tiled == 1 && (long long)grid.x * heads * num_seqs < 2 * scan_compute_units());
  const dim3 grid2(ceil_div(dv, 4 * 2), heads, num_seqs);
#define LAUNCH(KR)                                                                      \
  do {                                                                                  \
    if (!tiled) channel_delta_scan_kernel<KR><<<grid, 256, 0, stream>>>(a);              \
    else if (narrow) channel_delta_tiled_kernel<KR, 2><<<grid2, 256, 0, stream>>>(a);    \
    else channel_delta_tiled_kernel<KR, kCols><<<grid, 256, 0, stream>>>(a);             \
  } while (0)
  if (dk <= 64) LAUNCH(1);
  else if (dk <= 128) LAUNCH(2);
  else LAUNCH(4);
#undef LAUNCH
  RLIS_LAUNCH_CHECK("channel_delta_scan");
  return 0;
}
