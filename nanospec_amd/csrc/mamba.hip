// The selective scan of Mamba: a recurrence over the tokens with a state of N numbers per channel, whose step size, input
// and read-out the tokens choose.  With S [inner][N] (a new sequence starts with S = 0), token by token, c a channel:
//     dt[c] = softplus(zdt[c] + bias[c])
//     S[c] <- S[c] * exp(dt[c] A[c]) + (dt[c] x[c]) B;    y[c] = S[c] . C + D[c] x[c];    out[c] = y[c] silu(z[c])
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
// chunk's tokens leave of a state of zero.  Three kernels: U and the sums of the step sizes, all chunks at once; the pass over a
// request's chunks, which leaves the state in front of each in U's place; every chunk again from there, for the read-outs.  A
// workgroup takes a chunk and 64 channels, four lanes a channel; step sizes, dt x, B and C of the whole chunk are made once into LDS
// before its tokens are worked through.
//
// Decays are 2^(dt A'), A' = A log2(e): the vector unit's own exponential, whose error is that of its rounded argument.
#include "common.h"

#define MS_LOG2E 1.4426950408889634f
__device__ __forceinline__ float decay_of(float dt, float a) { return __builtin_amdgcn_exp2f(dt * a); }

// softplus(z) = max(z, 0) + log(1 + u), u = exp(-|z|) in (0, 1]: up to a tenth by the logarithm's own series (1 + u would lose most of u),
// beyond that by the vector unit's logarithm.
__device__ __forceinline__ float softplus_unit(float z) {
  const float u = __builtin_amdgcn_exp2f(-fabsf(z) * MS_LOG2E);
  float q = 1.f / 9.f;
#pragma unroll
  for (int n = 8; n >= 1; --n) q = fmaf(-u, q, 1.f / (float)n);
  return fmaxf(z, 0.f) + (u < 0.1f ? u * q : __builtin_amdgcn_logf(1.f + u) * 0.6931471805599453f);
}

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
      if (idx < XS) x_s[idx] = px[i], dt_s[idx] = softplus_unit(pdt[i]);
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
#define MC_LANES 4    // lanes that share a channel's states
#define MC_CH (MS_THREADS / MC_LANES)  // channels of a workgroup

// What the tokens of a chunk bring to a workgroup's channels, in LDS: step sizes and dt x [tokens][MC_CH], B (and C) [tokens][NM] with
// zeros beyond the last state.
template <typename T, int NM>
__device__ __forceinline__ void chunk_operands(float* dt_s, float* dx_s, float* b_s, float* c_s, const SelectiveScanParams& p, int row0, int nt, int c0) {
  const T* zdt = (const T*)p.zdt;
  const T* bc = (const T*)p.bc;
#pragma unroll 4
  for (int i = threadIdx.x; i < nt * MC_CH; i += MS_THREADS) {
    const size_t t = row0 + i / MC_CH;
    const int c = c0 + i % MC_CH;
    const bool ok = c < p.inner;
    const float dt = ok ? softplus_unit(to_f(zdt[t * p.dt_stride + c]) + p.dt_bias[c]) : 0.f;
    dt_s[i] = dt;
    dx_s[i] = ok ? dt * p.x[t * p.inner + c] : 0.f;
  }
  for (int i = threadIdx.x; i < nt * NM; i += MS_THREADS) {
    const T* row = bc + (size_t)(row0 + i / NM) * p.bc_stride;
    const int n = i % NM;
    b_s[i] = n < p.N ? to_f(row[p.b_off + n]) : 0.f;
    if (c_s) c_s[i] = n < p.N ? to_f(row[p.c_off + n]) : 0.f;
  }
  __syncthreads();
}

// U [chunk][inner][N] and the sums of the step sizes [chunk][inner].  grid (blocks of channels, chunks)
template <typename T, int NM>
__global__ __launch_bounds__(MS_THREADS) void selective_chunk_state_kernel(const SelectiveScanParams p, const int* __restrict__ chunks,
                                                                           float* __restrict__ ws, float* __restrict__ sums) {
  constexpr int SPT = NM / MC_LANES;
  __shared__ float dt_s[MC_TOKENS * MC_CH], dx_s[MC_TOKENS * MC_CH];
  __shared__ __attribute__((aligned(16))) float b_s[MC_TOKENS * NM];
  const int* chk = chunks + (size_t)blockIdx.y * MC_INTS;
  const int row0 = chk[1], nt = chk[2], c0 = blockIdx.x * MC_CH;
  if (nt <= 0) return;
  chunk_operands<T, NM>(dt_s, dx_s, b_s, nullptr, p, row0, nt, c0);
  const int cl = threadIdx.x / MC_LANES, n0 = threadIdx.x % MC_LANES * SPT, c = c0 + cl, inner = p.inner, N = p.N;
  if (c >= inner) return;
  float A[SPT], S[SPT], sum = 0.f;
#pragma unroll
  for (int j = 0; j < SPT; ++j) S[j] = 0.f, A[j] = n0 + j < N ? p.A[(size_t)c * N + n0 + j] * MS_LOG2E : 0.f;
#pragma unroll 4
  for (int t = 0; t < nt; ++t) {
    const float dt = dt_s[t * MC_CH + cl], dx = dx_s[t * MC_CH + cl];
    sum += dt;
    const float4* bp = reinterpret_cast<const float4*>(b_s + t * NM + n0);
#pragma unroll
    for (int j = 0; j < SPT; j += 4) {
      const float4 b = bp[j / 4];
      S[j] = fmaf(decay_of(dt, A[j]), S[j], dx * b.x);
      S[j + 1] = fmaf(decay_of(dt, A[j + 1]), S[j + 1], dx * b.y);
      S[j + 2] = fmaf(decay_of(dt, A[j + 2]), S[j + 2], dx * b.z);
      S[j + 3] = fmaf(decay_of(dt, A[j + 3]), S[j + 3], dx * b.w);
    }
  }
  if (n0 == 0) sums[(size_t)blockIdx.y * inner + c] = sum;
  float* out = ws + ((size_t)blockIdx.y * inner + c) * N + n0;
#pragma unroll
  for (int j = 0; j < SPT; ++j)
    if (n0 + j < N) out[j] = S[j];
}

// The pass over a request's chunks, a state a thread.  grid (pieces of [inner][N], chunks): the workgroups of a request's first chunk
// walk all of its chunks.
__global__ __launch_bounds__(MS_THREADS) void selective_chunk_pass_kernel(const SelectiveScanParams p, const int* __restrict__ chunks,
                                                                          float* __restrict__ ws, const float* __restrict__ sums) {
  const int* chk = chunks + (size_t)blockIdx.y * MC_INTS;
  const int count = chk[3];
  if (chk[2] <= 0 || count <= 0) return;
  const int inner = p.inner;
  const size_t words = (size_t)inner * p.N, at = (size_t)blockIdx.x * MS_THREADS + threadIdx.x;
  if (at >= words) return;
  const float A = p.A[at] * MS_LOG2E;
  float* st = p.state + (long long)p.state_slots[chk[0]] * p.state_stride + at;
  float* u = ws + (size_t)blockIdx.y * words + at;
  const float* sp = sums + (size_t)blockIdx.y * inner + at / p.N;
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

// The gated read-outs of every chunk from the state in front of it.  grid (blocks of channels, chunks).  A token's y takes the place of
// its dt x in LDS (the lanes of a channel have read it by then), from where it is gated and stored row by row.
template <typename T, int NM>
__global__ __launch_bounds__(MS_THREADS) void selective_chunk_out_kernel(const SelectiveScanParams p, const int* __restrict__ chunks,
                                                                         const float* __restrict__ ws) {
  constexpr int SPT = NM / MC_LANES;
  __shared__ float dt_s[MC_TOKENS * MC_CH], dx_s[MC_TOKENS * MC_CH];
  __shared__ __attribute__((aligned(16))) float b_s[MC_TOKENS * NM], c_s[MC_TOKENS * NM];
  const int* chk = chunks + (size_t)blockIdx.y * MC_INTS;
  const int row0 = chk[1], nt = chk[2], c0 = blockIdx.x * MC_CH;
  if (nt <= 0) return;
  chunk_operands<T, NM>(dt_s, dx_s, b_s, c_s, p, row0, nt, c0);
  const int s = threadIdx.x % MC_LANES, cl = threadIdx.x / MC_LANES, n0 = s * SPT, c = c0 + cl, inner = p.inner, N = p.N;
  const bool ok = c < inner;
  const float* in = ws + ((size_t)blockIdx.y * inner + (ok ? c : 0)) * N + n0;
  float A[SPT], S[SPT];
#pragma unroll
  for (int j = 0; j < SPT; ++j) {
    const bool on = ok && n0 + j < N;
    S[j] = on ? in[j] : 0.f, A[j] = on ? p.A[(size_t)c * N + n0 + j] * MS_LOG2E : 0.f;
  }
#pragma unroll 4
  for (int t = 0; t < nt; ++t) {
    const float dt = dt_s[t * MC_CH + cl], dx = dx_s[t * MC_CH + cl];
    const float4* bp = reinterpret_cast<const float4*>(b_s + t * NM + n0);
    const float4* cp = reinterpret_cast<const float4*>(c_s + t * NM + n0);
    float y0 = 0.f, y1 = 0.f;
#pragma unroll
    for (int j = 0; j < SPT; j += 4) {
      const float4 b = bp[j / 4], cc = cp[j / 4];
      S[j] = fmaf(decay_of(dt, A[j]), S[j], dx * b.x);
      S[j + 1] = fmaf(decay_of(dt, A[j + 1]), S[j + 1], dx * b.y);
      S[j + 2] = fmaf(decay_of(dt, A[j + 2]), S[j + 2], dx * b.z);
      S[j + 3] = fmaf(decay_of(dt, A[j + 3]), S[j + 3], dx * b.w);
      y0 = fmaf(S[j], cc.x, y0), y1 = fmaf(S[j + 1], cc.y, y1);
      y0 = fmaf(S[j + 2], cc.z, y0), y1 = fmaf(S[j + 3], cc.w, y1);
    }
    const float y = group_sum<MC_LANES>(y0 + y1);
    if (s == 0) dx_s[t * MC_CH + cl] = y;
  }
  __syncthreads();
  const T* z = (const T*)p.z;
  T* out = (T*)p.out;
#pragma unroll 4
  for (int i = threadIdx.x; i < nt * MC_CH; i += MS_THREADS) {
    const size_t t = row0 + i / MC_CH;
    const int ch = c0 + i % MC_CH;
    if (ch >= inner) continue;
    const float g = to_f(z[t * p.z_stride + ch]);
    out[t * inner + ch] = from_f<T>(fmaf(p.Dskip[ch], p.x[t * inner + ch], dx_s[i]) * g / (1.f + expf(-g)));
  }
}

template <typename T, int NM>
static int selective_chunks_launch(const SelectiveScanParams& p, const int* chunks, int n_chunks, float* ws, float* sums, hipStream_t stream) {
  const dim3 grid((p.inner + MC_CH - 1) / MC_CH, n_chunks);
  selective_chunk_state_kernel<T, NM><<<grid, MS_THREADS, 0, stream>>>(p, chunks, ws, sums);
  const size_t pieces = ((size_t)p.inner * p.N + MS_THREADS - 1) / MS_THREADS;
  selective_chunk_pass_kernel<<<dim3((int)pieces, n_chunks), MS_THREADS, 0, stream>>>(p, chunks, ws, sums);
  selective_chunk_out_kernel<T, NM><<<grid, MS_THREADS, 0, stream>>>(p, chunks, ws);
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

// ``chunks``: int32 [n_chunks][MC_INTS]; ``ws``: float32 [n_chunks][inner][N]; ``sums``: float32 [n_chunks][inner]
extern "C" int ns_selective_chunks(const float* x, const void* zdt, int dt_stride, const void* bc, int bc_stride, int b_off, int c_off, const void* z,
                                   int z_stride, const float* dt_bias, const float* A, const float* Dskip, float* state, long long state_stride,
                                   const int* chunks, int n_chunks, const int* state_slots, float* ws, float* sums, void* out, int inner,
                                   int N, int dtype, hipStream_t stream) {
  const SelectiveScanParams p{x, zdt, bc, z, dt_bias, A, Dskip, state, state_stride, nullptr, state_slots, out, dt_stride, bc_stride, b_off, c_off,
                              z_stride, inner, N, 0};
  if (const int bad = selective_check(p)) return bad;
  if (n_chunks <= 0 || n_chunks > 65535 || (size_t)inner * N / MS_THREADS >= 0x7fffffff) return NS_ERR_BAD_ARG;
  if (N > 32) return NS_ERR_UNSUPPORTED;
  if (dtype == NS_DTYPE_F32)
    return N <= 16 ? selective_chunks_launch<float, 16>(p, chunks, n_chunks, ws, sums, stream)
                   : selective_chunks_launch<float, 32>(p, chunks, n_chunks, ws, sums, stream);
  if (dtype == NS_DTYPE_BF16)
    return N <= 16 ? selective_chunks_launch<bf16_t, 16>(p, chunks, n_chunks, ws, sums, stream)
                   : selective_chunks_launch<bf16_t, 32>(p, chunks, n_chunks, ws, sums, stream);
  return NS_ERR_UNSUPPORTED;
}
