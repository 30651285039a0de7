// The selective scan of Mamba: a recurrence over the tokens with a state of N numbers per channel, whose step size, input
// and read-out the tokens choose.  Per channel c and state n, S [inner][N] (a new sequence starts with S = 0):
//     dt_c  = softplus(zdt_c + bias_c)
//     S[c, n] <- exp(dt_c A[c, n]) S[c, n] + dt_c x_c B_n;    y_c = sum_n S[c, n] C_n + D_c x_c;    out_c = y_c silu(z_c)
// Step sizes, decays, state and read-out are 32-bit.
//
// No channel meets another: a channel's states lie in TPC neighbouring lanes, SPT states a lane, whose parts of y meet through
// the vector unit's lane permutations (``group_sum``), and a workgroup of four waves owns 256 / TPC channels of one request.
// The next MS_TOKENS tokens' operands are fetched by the whole workgroup into registers while the current ones are worked
// through from LDS; four tokens are worked through together, so that only S passes from token to token and the exponentials
// lie beside the chain.  The read-outs of a block of tokens go through LDS, from where they are gated and stored.  A
// token's arithmetic is the same whatever portion it arrives in.
// A request's slot holds S [inner][N] (and behind it whatever its owner keeps there).
#include "common.h"

#define MS_THREADS 256
#define MS_TOKENS 16  // tokens a block

struct SelectiveScanParams {
  const float* x;  // [tokens][inner], behind the convolution
  const void* zdt;  // [tokens][..] step sizes ahead of bias and softplus, dt_stride apart
  const void* bc;   // [tokens][..] B at b_off, C at c_off, bc_stride apart
  const void* z;    // [tokens][..] gate, z_stride apart
  const float* dt_bias;  // [inner]
  const float* A;        // [inner][N], negative
  const float* Dskip;    // [inner]
  float* state;
  long long state_stride;
  const int* qo_indptr;
  const int* state_slots;
  void* out;  // [tokens][inner]
  int dt_stride, bc_stride, b_off, c_off, z_stride, inner, N;
};

template <typename T, int TPC, int SPT>
__global__ __launch_bounds__(MS_THREADS) void selective_scan_kernel(const SelectiveScanParams p) {
  constexpr int CPG = MS_THREADS / TPC;  // channels of a workgroup
  constexpr int NP = TPC * SPT;          // states of a channel as the lanes hold them (N padded)
  constexpr int TB = TPC * SPT >= 512 ? MS_TOKENS / 2 : MS_TOKENS;
  constexpr int XS = TB * CPG, BS = TB * NP;
  constexpr int XPER = (XS + MS_THREADS - 1) / MS_THREADS, BPER = (BS + MS_THREADS - 1) / MS_THREADS;
  __shared__ float x_s[XS], dt_s[XS], y_s[XS];
  __shared__ __attribute__((aligned(16))) float b_s[BS], c_s[BS];

  const int tid = threadIdx.x, b = blockIdx.y;
  const int t0 = p.qo_indptr[b], t1 = p.qo_indptr[b + 1];
  if (t1 <= t0) return;
  const int inner = p.inner, N = p.N, c0 = blockIdx.x * CPG;
  const int s = tid % TPC, cl = tid / TPC, ch = c0 + cl, n0 = s * SPT;
  const bool ch_ok = ch < inner;
  const T* zdt = (const T*)p.zdt;
  const T* bc = (const T*)p.bc;
  const T* z = (const T*)p.z;
  T* out = (T*)p.out;
  float* st = p.state + (long long)p.state_slots[b] * p.state_stride + (size_t)(ch_ok ? ch : 0) * N;
  float S[SPT], A[SPT];
#pragma unroll
  for (int j = 0; j < SPT; ++j) {
    const bool ok = ch_ok && n0 + j < N;
    S[j] = ok ? st[n0 + j] : 0.f;
    A[j] = ok ? p.A[(size_t)ch * N + n0 + j] : 0.f;
  }
  const float skip = ch_ok ? p.Dskip[ch] : 0.f;

  float px[XPER], pdt[XPER], pb[BPER], pc[BPER];
  auto fetch = [&](int t) {
#pragma unroll
    for (int i = 0; i < XPER; ++i) {
      const int idx = tid + i * MS_THREADS, tk = idx / CPG, c = c0 + idx % CPG;
      const bool live = idx < XS && t + tk < t1 && c < inner;
      px[i] = live ? p.x[(size_t)(t + tk) * inner + c] : 0.f;
      pdt[i] = live ? to_f(zdt[(size_t)(t + tk) * p.dt_stride + c]) + p.dt_bias[c] : -INFINITY;
    }
#pragma unroll
    for (int i = 0; i < BPER; ++i) {
      const int idx = tid + i * MS_THREADS, tk = idx / NP, n = idx % NP;
      const bool live = idx < BS && t + tk < t1 && n < N;
      const T* row = bc + (size_t)(t + (live ? tk : 0)) * p.bc_stride;
      pb[i] = live ? to_f(row[p.b_off + n]) : 0.f;
      pc[i] = live ? to_f(row[p.c_off + n]) : 0.f;
    }
  };
  auto stage = [&]() {
#pragma unroll
    for (int i = 0; i < XPER; ++i) {
      const int idx = tid + i * MS_THREADS;
      // (a token beyond the request's end has a step size of zero: it changes nothing)
      if (idx < XS) x_s[idx] = px[i], dt_s[idx] = softplus_f(pdt[i]);
    }
#pragma unroll
    for (int i = 0; i < BPER; ++i) {
      const int idx = tid + i * MS_THREADS;
      if (idx < BS) b_s[idx] = pb[i], c_s[idx] = pc[i];
    }
  };

  fetch(t0);
  stage();
  __syncthreads();
  constexpr int UN = 4;
  static_assert(TB % UN == 0, "a block of tokens is whole groups");
  for (int t = t0; t < t1; t += TB) {
    if (t + TB < t1) fetch(t + TB);
    const int nb = min(TB, t1 - t);
    for (int tk0 = 0; tk0 < nb; tk0 += UN) {
      float y[UN], xs[UN];
#pragma unroll
      for (int u = 0; u < UN; ++u) {
        const int tk = tk0 + u;
        const float dt = dt_s[tk * CPG + cl];
        xs[u] = x_s[tk * CPG + cl];
        const float dx = dt * xs[u];
        float sum = 0.f;
#pragma unroll
        for (int j = 0; j < SPT; ++j) {
          S[j] = fmaf(expf(dt * A[j]), S[j], dx * b_s[tk * NP + n0 + j]);
          sum = fmaf(S[j], c_s[tk * NP + n0 + j], sum);
        }
        y[u] = sum;
      }
#pragma unroll
      for (int u = 0; u < UN; ++u) y[u] = group_sum<TPC>(y[u]);
      if (s == 0) {
#pragma unroll
        for (int u = 0; u < UN; ++u) y_s[(tk0 + u) * CPG + cl] = fmaf(skip, xs[u], y[u]);
      }
    }
    __syncthreads();
    for (int idx = tid; idx < nb * CPG; idx += MS_THREADS) {
      const int tk = idx / CPG, c = c0 + idx % CPG;
      if (c < inner) {
        const float g = to_f(z[(size_t)(t + tk) * p.z_stride + c]);
        out[(size_t)(t + tk) * inner + c] = from_f<T>(y_s[idx] * g / (1.f + expf(-g)));
      }
    }
    if (t + TB < t1) stage();
    __syncthreads();
  }
  if (ch_ok) {
#pragma unroll
    for (int j = 0; j < SPT; ++j)
      if (n0 + j < N) st[n0 + j] = S[j];
  }
}

template <typename T>
static int selective_scan_launch(const SelectiveScanParams& p, int n_reqs, hipStream_t stream) {
  // few states: one a lane, so that a single request spreads over as many lanes as there are
  const int spt = p.N <= 16 ? 1 : (p.N <= 32 ? 2 : (p.N <= 128 ? 4 : 8));
  int tpc = 1;
  while (tpc * spt < p.N) tpc *= 2;
  const int cpg = MS_THREADS / tpc;
  const dim3 grid((p.inner + cpg - 1) / cpg, n_reqs);
#define MS_CASE(TPC, SPT) \
  if (tpc == TPC && spt == SPT) { selective_scan_kernel<T, TPC, SPT><<<grid, MS_THREADS, 0, stream>>>(p); return ns_launch_status(); }
  MS_CASE(1, 1) MS_CASE(2, 1) MS_CASE(4, 1) MS_CASE(8, 1) MS_CASE(16, 1)
  MS_CASE(16, 2) MS_CASE(16, 4) MS_CASE(32, 4) MS_CASE(32, 8) MS_CASE(64, 8)
#undef MS_CASE
  return NS_ERR_UNSUPPORTED;
}

extern "C" int ns_selective_scan(const float* x, const void* zdt, int dt_stride, const void* bc, int bc_stride, int b_off, int c_off, const void* z,
                                 int z_stride, const float* dt_bias, const float* A, const float* Dskip, float* state, long long state_stride,
                                 const int* qo_indptr, const int* state_slots, void* out, int n_reqs, int inner, int N, int dtype, hipStream_t stream) {
  if (n_reqs <= 0 || n_reqs > 65535 || inner <= 0 || N <= 0 || b_off < 0 || c_off < 0) return NS_ERR_BAD_ARG;
  if (N > 512) return NS_ERR_UNSUPPORTED;
  if (state_stride < (long long)inner * N) return NS_ERR_BAD_ARG;
  const SelectiveScanParams p{x, zdt, bc, z, dt_bias, A, Dskip, state, state_stride, qo_indptr, state_slots, out, dt_stride, bc_stride, b_off, c_off,
                              z_stride, inner, N};
  if (dtype == NS_DTYPE_F32) return selective_scan_launch<float>(p, n_reqs, stream);
  if (dtype == NS_DTYPE_BF16) return selective_scan_launch<bf16_t>(p, n_reqs, stream);
  return NS_ERR_UNSUPPORTED;
}
