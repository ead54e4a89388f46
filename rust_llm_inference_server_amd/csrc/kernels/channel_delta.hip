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

}  // namespace

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
