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
//
// Long portions run in chunks of up to 64 tokens (few states only), because a single request's channels do not fill the GPU and
// its tokens are one chain.  What a chunk makes of the state in front of it is linear, S' = exp(A sum_t dt_t) S + U, with U what the
// chunk's tokens leave of a state of zero.  Three kernels: U and the sums of the step sizes, all chunks at once (the step sizes
// are kept for the third); the pass over a request's chunks, which leaves the state in front of each in U's place; every
// chunk again from there, for the read-outs.  A thread owns a channel with all of its states, so nothing meets across lanes and the
// chunk's B and C are read from LDS by all threads alike.
//
// Decays are 2^(dt A'), A' = A log2(e): the vector unit's own exponential, whose error is that of its rounded argument.
#include "common.h"

#define MS_LOG2E 1.4426950408889634f
__device__ __forceinline__ float decay_of(float dt, float a) { return __builtin_amdgcn_exp2f(dt * a); }

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
  int skip_from;  // > 0: requests that bring at least this many tokens are somebody else's
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
  if (t1 <= t0 || (p.skip_from > 0 && t1 - t0 >= p.skip_from)) return;
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
    A[j] = ok ? p.A[(size_t)ch * N + n0 + j] * MS_LOG2E : 0.f;
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
          S[j] = fmaf(decay_of(dt, A[j]), S[j], dx * b_s[tk * NP + n0 + j]);
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

// ------------------------------------------------------------------------------------------------ long portions in chunks
#define MC_TOKENS 64  // tokens of a chunk
#define MC_INTS 4     // a chunk: request, row of its first token, tokens (0: no chunk), chunks of the request if it is its first (else 0)
#define MC_UN 8       // tokens whose operands are fetched together

// B (and C) of a chunk's tokens in LDS, [tokens][NM], zeros beyond the last state
template <typename T, int NM>
__device__ __forceinline__ void chunk_rows(float* lds, const T* bc, int stride, int off, int row0, int nt, int N) {
  for (int i = threadIdx.x; i < nt * NM; i += blockDim.x) {
    const int t = i / NM, n = i % NM;
    lds[i] = n < N ? to_f(bc[(size_t)(row0 + t) * stride + off + n]) : 0.f;
  }
}

// U [chunk][N][inner], the sums of the step sizes [chunk][inner] and the step sizes [tokens][inner].  grid (blocks of channels, chunks)
template <typename T, int NM>
__global__ __launch_bounds__(MS_THREADS) void selective_chunk_state_kernel(const SelectiveScanParams p, const int* __restrict__ chunks,
                                                                           float* __restrict__ ws, float* __restrict__ sums, float* __restrict__ dts) {
  __shared__ __attribute__((aligned(16))) float b_s[MC_TOKENS * NM];
  const int* chk = chunks + (size_t)blockIdx.y * MC_INTS;
  const int row0 = chk[1], nt = chk[2];
  if (nt <= 0) return;
  chunk_rows<T, NM>(b_s, (const T*)p.bc, p.bc_stride, p.b_off, row0, nt, p.N);
  __syncthreads();
  const int c = blockIdx.x * MS_THREADS + threadIdx.x, inner = p.inner, N = p.N;
  if (c >= inner) return;
  float A[NM], S[NM], sum = 0.f;
#pragma unroll
  for (int n = 0; n < NM; ++n) S[n] = 0.f, A[n] = n < N ? p.A[(size_t)c * N + n] * MS_LOG2E : 0.f;
  const float bias = p.dt_bias[c];
  const T* zdt = (const T*)p.zdt + (size_t)row0 * p.dt_stride + c;
  const float* x = p.x + (size_t)row0 * inner + c;
  float* dto = dts + (size_t)row0 * inner + c;
  float px[MC_UN], pz[MC_UN];
  auto fetch = [&](int t0) {
#pragma unroll
    for (int u = 0; u < MC_UN; ++u) {
      const size_t t = min(t0 + u, nt - 1);
      px[u] = x[t * inner], pz[u] = to_f(zdt[t * p.dt_stride]);
    }
  };
  fetch(0);
  for (int t0 = 0; t0 < nt; t0 += MC_UN) {
    float xs[MC_UN], dt[MC_UN];
#pragma unroll
    for (int u = 0; u < MC_UN; ++u) xs[u] = px[u], dt[u] = softplus_f(pz[u] + bias);
    if (t0 + MC_UN < nt) fetch(t0 + MC_UN);
#pragma unroll
    for (int u = 0; u < MC_UN; ++u) {
      if (t0 + u >= nt) break;
      dto[(size_t)(t0 + u) * inner] = dt[u];
      sum += dt[u];
      const float dx = dt[u] * xs[u];
      const float4* bp = reinterpret_cast<const float4*>(b_s + (t0 + u) * NM);
#pragma unroll
      for (int n = 0; n < NM; n += 4) {
        const float4 b = bp[n / 4];
        S[n] = fmaf(decay_of(dt[u], A[n]), S[n], dx * b.x);
        S[n + 1] = fmaf(decay_of(dt[u], A[n + 1]), S[n + 1], dx * b.y);
        S[n + 2] = fmaf(decay_of(dt[u], A[n + 2]), S[n + 2], dx * b.z);
        S[n + 3] = fmaf(decay_of(dt[u], A[n + 3]), S[n + 3], dx * b.w);
      }
    }
  }
  sums[(size_t)blockIdx.y * inner + c] = sum;
  float* out = ws + (size_t)blockIdx.y * N * inner + c;
#pragma unroll
  for (int n = 0; n < NM; ++n)
    if (n < N) out[(size_t)n * inner] = S[n];
}

// The pass over a request's chunks, a state a thread.  grid (pieces of [N][inner], chunks): the workgroups of a request's first chunk
// walk all of its chunks.
__global__ __launch_bounds__(MS_THREADS) void selective_chunk_pass_kernel(const SelectiveScanParams p, const int* __restrict__ chunks,
                                                                          float* __restrict__ ws, const float* __restrict__ sums) {
  const int* chk = chunks + (size_t)blockIdx.y * MC_INTS;
  const int count = chk[3];
  if (chk[2] <= 0 || count <= 0) return;
  const int inner = p.inner, N = p.N;
  const size_t words = (size_t)inner * N, at = (size_t)blockIdx.x * MS_THREADS + threadIdx.x;
  if (at >= words) return;
  const int n = (int)(at / inner), c = (int)(at % inner);
  const float A = p.A[(size_t)c * N + n] * MS_LOG2E;
  float* st = p.state + (long long)p.state_slots[chk[0]] * p.state_stride + (size_t)c * N + n;
  float* u = ws + (size_t)blockIdx.y * words + at;
  const float* sp = sums + (size_t)blockIdx.y * inner + c;
  float S = *st, next = *u, next_sum = *sp;
  for (int i = 0; i < count; ++i) {
    const float cur = next, f = decay_of(next_sum, A);
    if (i + 1 < count) next = u[words], next_sum = sp[inner];
    *u = S;
    S = fmaf(f, S, cur);
    u += words, sp += inner;
  }
  *st = S;
}

// The gated read-outs of every chunk from the state in front of it.  grid (blocks of channels, chunks)
template <typename T, int NM>
__global__ __launch_bounds__(MS_THREADS) void selective_chunk_out_kernel(const SelectiveScanParams p, const int* __restrict__ chunks,
                                                                         const float* __restrict__ ws, const float* __restrict__ dts) {
  __shared__ __attribute__((aligned(16))) float b_s[MC_TOKENS * NM], c_s[MC_TOKENS * NM];
  const int* chk = chunks + (size_t)blockIdx.y * MC_INTS;
  const int row0 = chk[1], nt = chk[2];
  if (nt <= 0) return;
  chunk_rows<T, NM>(b_s, (const T*)p.bc, p.bc_stride, p.b_off, row0, nt, p.N);
  chunk_rows<T, NM>(c_s, (const T*)p.bc, p.bc_stride, p.c_off, row0, nt, p.N);
  __syncthreads();
  const int c = blockIdx.x * MS_THREADS + threadIdx.x, inner = p.inner, N = p.N;
  if (c >= inner) return;
  const float* in = ws + (size_t)blockIdx.y * N * inner + c;
  float A[NM], S[NM];
#pragma unroll
  for (int n = 0; n < NM; ++n) S[n] = n < N ? in[(size_t)n * inner] : 0.f, A[n] = n < N ? p.A[(size_t)c * N + n] * MS_LOG2E : 0.f;
  const float skip = p.Dskip[c];
  const T* z = (const T*)p.z + (size_t)row0 * p.z_stride + c;
  const float* x = p.x + (size_t)row0 * inner + c;
  const float* dti = dts + (size_t)row0 * inner + c;
  T* out = (T*)p.out + (size_t)row0 * inner + c;
  float px[MC_UN], pd[MC_UN], pz[MC_UN];
  auto fetch = [&](int t0) {
#pragma unroll
    for (int u = 0; u < MC_UN; ++u) {
      const size_t t = min(t0 + u, nt - 1);
      px[u] = x[t * inner], pd[u] = dti[t * inner], pz[u] = to_f(z[t * p.z_stride]);
    }
  };
  fetch(0);
  for (int t0 = 0; t0 < nt; t0 += MC_UN) {
    float xs[MC_UN], dt[MC_UN], g[MC_UN];
#pragma unroll
    for (int u = 0; u < MC_UN; ++u) xs[u] = px[u], dt[u] = pd[u], g[u] = pz[u];
    if (t0 + MC_UN < nt) fetch(t0 + MC_UN);
#pragma unroll
    for (int u = 0; u < MC_UN; ++u) {
      if (t0 + u >= nt) break;
      const float dx = dt[u] * xs[u];
      const float4* bp = reinterpret_cast<const float4*>(b_s + (t0 + u) * NM);
      const float4* cp = reinterpret_cast<const float4*>(c_s + (t0 + u) * NM);
      float y0 = skip * xs[u], y1 = 0.f;
#pragma unroll
      for (int n = 0; n < NM; n += 4) {
        const float4 b = bp[n / 4], cc = cp[n / 4];
        S[n] = fmaf(decay_of(dt[u], A[n]), S[n], dx * b.x);
        S[n + 1] = fmaf(decay_of(dt[u], A[n + 1]), S[n + 1], dx * b.y);
        S[n + 2] = fmaf(decay_of(dt[u], A[n + 2]), S[n + 2], dx * b.z);
        S[n + 3] = fmaf(decay_of(dt[u], A[n + 3]), S[n + 3], dx * b.w);
        y0 = fmaf(S[n], cc.x, y0), y1 = fmaf(S[n + 1], cc.y, y1);
        y0 = fmaf(S[n + 2], cc.z, y0), y1 = fmaf(S[n + 3], cc.w, y1);
      }
      out[(size_t)(t0 + u) * inner] = from_f<T>((y0 + y1) * g[u] / (1.f + expf(-g[u])));
    }
  }
}

template <typename T, int NM>
static int selective_chunks_launch(const SelectiveScanParams& p, const int* chunks, int n_chunks, float* ws, float* sums, float* dts, hipStream_t stream) {
  const dim3 grid((p.inner + MS_THREADS - 1) / MS_THREADS, n_chunks);
  selective_chunk_state_kernel<T, NM><<<grid, MS_THREADS, 0, stream>>>(p, chunks, ws, sums, dts);
  const size_t pieces = ((size_t)p.inner * p.N + MS_THREADS - 1) / MS_THREADS;
  selective_chunk_pass_kernel<<<dim3((int)pieces, n_chunks), MS_THREADS, 0, stream>>>(p, chunks, ws, sums);
  selective_chunk_out_kernel<T, NM><<<grid, MS_THREADS, 0, stream>>>(p, chunks, ws, dts);
  return ns_launch_status();
}

static int selective_check(const SelectiveScanParams& p) {
  if (p.inner <= 0 || p.N <= 0 || p.b_off < 0 || p.c_off < 0) return NS_ERR_BAD_ARG;
  return p.state_stride < (long long)p.inner * p.N ? NS_ERR_BAD_ARG : NS_OK;
}

extern "C" int ns_selective_scan(const float* x, const void* zdt, int dt_stride, const void* bc, int bc_stride, int b_off, int c_off, const void* z,
                                 int z_stride, const float* dt_bias, const float* A, const float* Dskip, float* state, long long state_stride,
                                 const int* qo_indptr, const int* state_slots, void* out, int n_reqs, int inner, int N, int skip_from, int dtype,
                                 hipStream_t stream) {
  const SelectiveScanParams p{x, zdt, bc, z, dt_bias, A, Dskip, state, state_stride, qo_indptr, state_slots, out, dt_stride, bc_stride, b_off, c_off,
                              z_stride, inner, N, skip_from};
  if (const int bad = selective_check(p)) return bad;
  if (n_reqs <= 0 || n_reqs > 65535) return NS_ERR_BAD_ARG;
  if (N > 512) return NS_ERR_UNSUPPORTED;
  if (dtype == NS_DTYPE_F32) return selective_scan_launch<float>(p, n_reqs, stream);
  if (dtype == NS_DTYPE_BF16) return selective_scan_launch<bf16_t>(p, n_reqs, stream);
  return NS_ERR_UNSUPPORTED;
}

// ``chunks``: int32 [n_chunks][MC_INTS]; ``ws``: float32 [n_chunks][N][inner]; ``sums``: float32 [n_chunks][inner]; ``dts``: float32 [tokens][inner]
extern "C" int ns_selective_chunks(const float* x, const void* zdt, int dt_stride, const void* bc, int bc_stride, int b_off, int c_off, const void* z,
                                   int z_stride, const float* dt_bias, const float* A, const float* Dskip, float* state, long long state_stride,
                                   const int* chunks, int n_chunks, const int* state_slots, float* ws, float* sums, float* dts, void* out, int inner,
                                   int N, int dtype, hipStream_t stream) {
  const SelectiveScanParams p{x, zdt, bc, z, dt_bias, A, Dskip, state, state_stride, nullptr, state_slots, out, dt_stride, bc_stride, b_off, c_off,
                              z_stride, inner, N, 0};
  if (const int bad = selective_check(p)) return bad;
  if (n_chunks <= 0 || n_chunks > 65535 || (size_t)inner * N / MS_THREADS >= 0x7fffffff) return NS_ERR_BAD_ARG;
  if (N > 32) return NS_ERR_UNSUPPORTED;
  if (dtype == NS_DTYPE_F32)
    return N <= 16 ? selective_chunks_launch<float, 16>(p, chunks, n_chunks, ws, sums, dts, stream)
                   : selective_chunks_launch<float, 32>(p, chunks, n_chunks, ws, sums, dts, stream);
  if (dtype == NS_DTYPE_BF16)
    return N <= 16 ? selective_chunks_launch<bf16_t, 16>(p, chunks, n_chunks, ws, sums, dts, stream)
                   : selective_chunks_launch<bf16_t, 32>(p, chunks, n_chunks, ws, sums, dts, stream);
  return NS_ERR_UNSUPPORTED;
}
