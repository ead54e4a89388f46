// A real-gated linear recurrent unit: one float32 number per channel and request.  Per token
//   r = sigmoid(gr + r_bias), i = sigmoid(gi + i_bias)
//   log a = rate r  (rate < 0),  S <- a S + sqrt(1 - a^2) i u,  out = S gelu(y + y_bias)
// with gr, gi, y raw float32 products and u, out in the activation dtype.  The gates of a block
// of n channels lie together, n numbers for r and n for i.  1 - a^2 is formed as -expm1(2 log a).
//
// A sequence's channels are independent of each other, so a thread owns a channel; what is
// sequential is the walk over the tokens.  Long portions are cut into chunks that walk side by
// side: every chunk from a zero state (its decay and its sum), the chunks joined in order, every
// chunk again from its true start state.
#include "scan.h"

namespace {

struct RglruArgs {
  void* out;
  const void* u;
  long long ldu;
  const float* gates;
  long long ldg;
  const float *r_bias, *i_bias, *rate;
  const float* y;
  long long ldy;
  const float* y_bias;
  float* state;
  long long state_stride;
  const int *cu, *slots;
  int num_seqs, C, n, chunk, max_chunks;
  float* ws;                       // (2, max_chunks, C): decay and sum of every chunk
};

struct RglruToken { float a, drive; };

// The token's decay and what it adds to the state.
__device__ __forceinline__ RglruToken rglru_token(float gr, float gi, float u, float rb, float ib,
                                                  float rate) {
  const float log_a = rate * sigmoidf_(gr + rb);
  return {expf(log_a), sqrtf(-expm1f(2.0f * log_a)) * sigmoidf_(gi + ib) * u};
}

constexpr int kAhead = 4;          // tokens whose inputs are asked for together

// Tokens t0 .. t1 of channel c from state S; OUT: results are stored, else the decays' product
// is returned in `decay`.
template <typename TX, bool OUT>
__device__ __forceinline__ float rglru_walk(const RglruArgs& a, int c, int t0, int t1, float S,
                                            float& decay) {
  const int g = (c / a.n) * 2 * a.n + c % a.n;
  const float rb = a.r_bias[c], ib = a.i_bias[c], rate = a.rate[c];
  const float yb = OUT ? a.y_bias[c] : 0.f;
  const TX* u = (const TX*)a.u + c;
  float sum_log = 0.f;
  for (int t = t0; t < t1; t += kAhead) {
    float gr[kAhead], gi[kAhead], yv[kAhead], uv[kAhead];
#pragma unroll
    for (int k = 0; k < kAhead; ++k) {
      const long long row = min(t + k, t1 - 1);       // (past the end: the last token again, unused)
      gr[k] = a.gates[row * a.ldg + g];
      gi[k] = a.gates[row * a.ldg + g + a.n];
      uv[k] = ld(u + row * a.ldu);
      if (OUT) yv[k] = a.y[row * a.ldy + c];
    }
#pragma unroll
    for (int k = 0; k < kAhead; ++k) {
      if (t + k >= t1) break;
      const RglruToken x = rglru_token(gr[k], gi[k], uv[k], rb, ib, rate);
      S = x.a * S + x.drive;
      if (OUT)
        st((TX*)a.out + (long long)(t + k) * a.C + c, S * gelu_tanh_f(yv[k] + yb));
      else
        sum_log += rate * sigmoidf_(gr[k] + rb);
    }
  }
  if (!OUT) decay = expf(sum_log);
  return S;
}

template <typename TX>
__global__ __launch_bounds__(256) void rglru_scan_kernel(const RglruArgs a) {
  const int c = blockIdx.x * blockDim.x + threadIdx.x;
  const int s = blockIdx.y;
  if (c >= a.C) return;
  float* slot = a.state + (long long)a.slots[s] * a.state_stride + c;
  float unused;
  *slot = rglru_walk<TX, true>(a, c, a.cu[s], a.cu[s + 1], *slot, unused);
}

template <typename TX, bool OUT>
__global__ __launch_bounds__(256) void rglru_chunk_kernel(const RglruArgs a) {
  const int c = blockIdx.x * blockDim.x + threadIdx.x;
  const int chunk = blockIdx.y;
  int t0, t1;
  if (c >= a.C || !chunk_span(a.cu, a.num_seqs, a.chunk, chunk, t0, t1)) return;
  float* decay_at = a.ws + (long long)chunk * a.C + c;
  float* sum_at = decay_at + (long long)a.max_chunks * a.C;
  float decay = 1.f;
  if (OUT) {
    rglru_walk<TX, true>(a, c, t0, t1, *sum_at, decay);
  } else {
    const float S = rglru_walk<TX, false>(a, c, t0, t1, 0.f, decay);
    *decay_at = decay;
    *sum_at = S;
  }
}

// A sequence's chunks in order: every chunk's start state takes the place of its sum.
__global__ __launch_bounds__(256) void rglru_join_kernel(const RglruArgs a) {
  const int c = blockIdx.x * blockDim.x + threadIdx.x;
  const int s = blockIdx.y;
  if (c >= a.C) return;
  const int first = chunks_before(a.cu, s, a.chunk);
  const int chunks = (a.cu[s + 1] - a.cu[s] + a.chunk - 1) / a.chunk;
  float* slot = a.state + (long long)a.slots[s] * a.state_stride + c;
  float S = *slot;
  const float* decay = a.ws + (long long)first * a.C + c;
  float* sum = a.ws + ((long long)a.max_chunks + first) * a.C + c;
  constexpr int U = 8;
  for (int k = 0; k < chunks; k += U) {
    float d[U], b[U];
#pragma unroll
    for (int i = 0; i < U; ++i) {
      const long long at = (long long)min(k + i, chunks - 1) * a.C;
      d[i] = decay[at];
      b[i] = sum[at];
    }
#pragma unroll
    for (int i = 0; i < U; ++i) {
      if (k + i >= chunks) break;
      sum[(long long)(k + i) * a.C] = S;
      S = d[i] * S + b[i];
    }
  }
  *slot = S;
}

}  // namespace

RLIS_API int rlis_rglru_scan(void* out, int dtype, const void* u, long long ldu, const float* gates,
                             long long ldg, const float* r_bias, const float* i_bias,
                             const float* rate, const float* y, long long ldy, const float* y_bias,
                             float* state, long long state_stride, const int* cu, const int* slots,
                             int num_seqs, int C, int n, int chunk, int max_chunks, float* ws,
                             hipStream_t stream) {
  RLIS_REQUIRE(C > 0 && n > 0 && C % n == 0, "rglru_scan: %d channels in blocks of %d", C, n);
  RLIS_REQUIRE(ldu >= C && ldy >= C && ldg >= 2LL * C && state_stride >= C,
               "rglru_scan: rows shorter than the channels");
  RLIS_REQUIRE(num_seqs <= 65535, "rglru_scan: %d sequences, at most 65535", num_seqs);
  RLIS_REQUIRE(dtype == RLIS_F32 || dtype == RLIS_BF16, "rglru_scan: unknown dtype %d", dtype);
  if (num_seqs <= 0) return 0;
  const RglruArgs a{out, u, ldu, gates, ldg, r_bias, i_bias, rate, y, ldy, y_bias, state,
                    state_stride, cu, slots, num_seqs, C, n, chunk, max_chunks, ws};
  if (max_chunks > 0) {
    RLIS_REQUIRE(ws && chunk > 0 && max_chunks <= 65535, "rglru_scan: %d chunks of %d tokens",
                 max_chunks, chunk);
    const dim3 grid(ceil_div(C, 256), max_chunks), join(ceil_div(C, 256), num_seqs);
    if (dtype == RLIS_F32) rglru_chunk_kernel<float, false><<<grid, 256, 0, stream>>>(a);
    else rglru_chunk_kernel<bf16_t, false><<<grid, 256, 0, stream>>>(a);
    RLIS_LAUNCH_CHECK("rglru_scan");
    rglru_join_kernel<<<join, 256, 0, stream>>>(a);
    RLIS_LAUNCH_CHECK("rglru_scan");
    if (dtype == RLIS_F32) rglru_chunk_kernel<float, true><<<grid, 256, 0, stream>>>(a);
    else rglru_chunk_kernel<bf16_t, true><<<grid, 256, 0, stream>>>(a);
    RLIS_LAUNCH_CHECK("rglru_scan");
    return 0;
  }
  const int threads = C >= 4096 ? 256 : 64;
  const dim3 grid(ceil_div(C, threads), num_seqs);
  if (dtype == RLIS_F32) rglru_scan_kernel<float><<<grid, threads, 0, stream>>>(a);
  else rglru_scan_kernel<bf16_t><<<grid, threads, 0, stream>>>(a);
  RLIS_LAUNCH_CHECK("rglru_scan");
  return 0;
}
