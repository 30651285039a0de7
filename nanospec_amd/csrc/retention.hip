// Retention: linear attention with one fixed decay per head, no soft-max and no denominator, token by token in 32-bit.
// Per head, S [D][E] (a new sequence starts with S = 0):
//     S_t = decay_h S_(t-1) + k_t v_t^T;   o_t = S_t^T q_t
// q and k are rotated by their position and k is multiplied by ``k_scale`` first; with ``silu`` q, k and v pass a SiLU before that.
//
//   retention_prep   a token's row [.. q .. k .. v ..] of the layer's first product (the model's precision) -> 32-bit rows
//                    [q rotated | k rotated and scaled | v]: angles, cosine, sine and the rotation in 32-bit
//   retention_scan   the recurrence over every request's tokens of the step, in order, from the state in its slot
//   retention_chunks the same for long portions, in chunks of 64 tokens as matrix products (below)
//   log_decay_heads  decays per head that the input chooses (below), in the logarithm (those per channel: ``retention_prep``)
//   gate_mul         y = x * sigmoid(g) or x * g sigmoid(g), the gate formed in 32-bit (the soft-max attention's output gate)
//
// The scan is laid out like the matrix memory's (memory.hip): a column of S never meets another column, so a wave owns 64 / TPC
// columns and the TPC lanes of a column hold 8 key channels each; their partial sums meet through the vector unit's lane
// permutations (``group_sum``).  A workgroup is four waves that share the staged operands: the next block of tokens is
// fetched into registers while the current block is worked through from LDS; four tokens are worked through together, and
// only S passes from token to token.  A token's arithmetic is the same whatever portion it arrives in.
// State slot of a request: S as [H][E][D] (a column's key channels contiguous).
//
// The same two forms serve recurrences whose decay the input chooses (a kernel's ``KIND``), with the logarithms of the decays
// (at most 0) in memory per token:
//   0  one fixed decay per head                                            retention, lightning attention
//   1  one decay per token and head, log_decay [tokens][H]                 the state-space recurrence of Mamba-2
//   2  one decay per token, head and key channel, log_decay [tokens][H D]  gated linear attention
// Keys and queries may be shared by groups of neighbouring heads (G < H); q, k and v may lie anywhere in a row.  With KIND 1 a
// token's k v^T may be weighted by v_scale[t][h] and the read-out may get skip[h] v_t added.
//
// Long portions: with one fixed decay a the tokens of a chunk (l tokens, numbered 0 .. l - 1) meet the state in front of it
// and each other as matrix products weighted by powers of the decay, all of them at most 1:
//     U    = sum_j a^(l - 1 - j) k_j v_j^T                                       what the chunk adds to the state
//     S'   = a^l S + U
//     o_i  = a^(i + 1) S^T q_i + sum_(j <= i) a^(i - j) (q_i . k_j) v_j
// Three kernels: U of every chunk at once; the pass over a request's chunks (a multiply-add an element), which leaves the state
// in front of each chunk in U's place and the last one in the slot; the outputs of every chunk at once.  The products are the
// 32-bit matrix instruction (v_mfma_f32_16x16x4_f32: 32-bit operands and sums), so the recurrence stays 32-bit throughout.
#include "common.h"
#include "rope.h"

__device__ __forceinline__ float maybe_silu(float z, int silu) { return silu ? z / (1.f + expf(-z)) : z; }

// A few workgroups a token (grid.y), each a share of its columns.  With ``log_decay`` also the logarithms of the decays per key channel
// that the token chooses, log(sigmoid(z + z_bias)) / tau, in 32-bit.
template <typename T>
__global__ __launch_bounds__(256) void retention_prep_kernel(const T* __restrict__ proj, int stride, int q_off, int k_off, int v_off,
                                                             const int* __restrict__ positions, const float* __restrict__ inv_freq,
                                                             float* __restrict__ out, int H, int D, int E, RopeForm form, float k_scale,
                                                             int silu, const T* __restrict__ z, int z_stride,
                                                             const float* __restrict__ z_bias, float inv_tau, float* __restrict__ log_decay) {
  const int t = blockIdx.x;
  const T* row = proj + (size_t)t * stride;
  float* o = out + (size_t)t * H * (2 * D + E);
  const int pos = positions[t];
  const int half = form.rot / 2;
  const int first = blockIdx.y * blockDim.x + threadIdx.x, step = gridDim.y * blockDim.x;
  // rotated pairs of q and k: item = (which, head, pair)
  for (int i = first; i < 2 * H * half; i += step) {
    const int which = i / (H * half), h = (i / half) % H, j = i % half;
    int d1, d2;
    rope_pair_channels(form, j, d1, d2);
    const T* src = row + (which ? k_off : q_off) + (size_t)h * D;
    float c, s, a, b;
    rope_cos_sin(form, pos, inv_freq[j], c, s);
    rope_turn(maybe_silu(to_f(src[d1]), silu), maybe_silu(to_f(src[d2]), silu), c, s, a, b);
    const float m = which ? k_scale : 1.f;
    float* dst = o + (size_t)which * H * D + (size_t)h * D;
    dst[d1] = a * m;
    dst[d2] = b * m;
  }
  if (form.rot == 0) {  // nothing is rotated: q and k are copied as they lie
    for (int i = first; i < H * D; i += step) o[i] = maybe_silu(to_f(row[q_off + i]), silu);
    for (int i = first; i < H * D; i += step) o[(size_t)H * D + i] = maybe_silu(to_f(row[k_off + i]), silu) * k_scale;
  }
  const int rest = form.rot == 0 ? 0 : D - form.rot;
  for (int i = first; i < 2 * H * rest; i += step) {
    const int which = i / (H * rest), h = (i / rest) % H, d = form.rot + i % rest;
    o[(size_t)which * H * D + (size_t)h * D + d] =
        maybe_silu(to_f(row[(which ? k_off : q_off) + (size_t)h * D + d]), silu) * (which ? k_scale : 1.f);
  }
  for (int i = first; i < H * E; i += step) o[(size_t)2 * H * D + i] = maybe_silu(to_f(row[v_off + i]), silu);
  if (log_decay)
    for (int i = first; i < H * D; i += step)
      log_decay[(size_t)t * H * D + i] = -softplus_f(-(to_f(z[(size_t)t * z_stride + i]) + z_bias[i])) * inv_tau;
}

extern "C" int ns_retention_prep(const void* proj, int stride, int q_off, int k_off, int v_off, const int* positions, const float* inv_freq,
                                 float* out, int n_tokens, int H, int D, int E, int rot, int interleaved, float factor, float k_scale, int silu,
                                 const void* z, int z_stride, const float* z_bias, float inv_tau, float* log_decay, int dtype, hipStream_t stream) {
  if (n_tokens <= 0 || H <= 0 || D <= 0 || E <= 0 || rot < 0 || rot > D || rot % 2 || (rot > 0 && !inv_freq)) return NS_ERR_BAD_ARG;
  if (log_decay && (!z || !z_bias)) return NS_ERR_BAD_ARG;
  const RopeForm form{rot, interleaved, factor};
  const long long items = (long long)H * (2 * D + E);
  const dim3 grid(n_tokens, (int)(items <= 512 ? 1 : (items + 511) / 512 < 8 ? (items + 511) / 512 : 8));
  if (dtype == NS_DTYPE_F32)
    retention_prep_kernel<float><<<grid, 256, 0, stream>>>((const float*)proj, stride, q_off, k_off, v_off, positions, inv_freq, out, H, D, E, form, k_scale, silu,
                                                         (const float*)z, z_stride, z_bias, inv_tau, log_decay);
  else if (dtype == NS_DTYPE_BF16)
    retention_prep_kernel<bf16_t><<<grid, 256, 0, stream>>>((const bf16_t*)proj, stride, q_off, k_off, v_off, positions, inv_freq, out, H, D, E, form, k_scale, silu,
                                                         (const bf16_t*)z, z_stride, z_bias, inv_tau, log_decay);
  else
    return NS_ERR_UNSUPPORTED;
  return ns_launch_status();
}

#define RT_KPT 8  // key channels a lane holds of its column
#define RT_WAVES 4
#define RT_THREADS (RT_WAVES * NS_WAVE)

// where a recurrence finds its operands
struct DecayRows {
  const float* rows;  // [tokens][row_w]: q [G][D] at q_off, k [G][D] at k_off, v [H][E] at v_off
  int row_w, q_off, k_off, v_off;
  int H, G, D, E;  // head h reads q and k of head h / (H / G)
  const float* decay;      // KIND 0: [H]
  float* log_decay;        // KIND 1: [tokens][H], KIND 2: [tokens][H * D] (the chunked form leaves sums within chunks there)
  const float* v_scale;    // KIND 1: [tokens][H] or null
  const float* skip;       // KIND 1: [H] or null
};

struct RetentionParams {
  DecayRows r;
  float* state;  // [slots][state_stride]
  long long state_stride;
  const int* qo_indptr;
  const int* state_slots;
  float* out;  // [tokens][H * E]
  int vec_ok;  // 8 channels of q and k can be fetched with aligned vector loads
  int skip_from;  // > 0: requests that bring at least this many tokens are somebody else's (``retention_chunks``)
};

template <int TPC, int KIND>
__global__ __launch_bounds__(RT_THREADS) void retention_scan_kernel(const RetentionParams p) {
  constexpr int DP = RT_KPT * TPC;                           // key channels of a column as the lanes hold them (D padded)
  constexpr int CPW = NS_WAVE / TPC;                         // columns a wave owns
  constexpr int CPG = CPW * RT_WAVES;                        // columns a workgroup owns
  constexpr int TB = TPC <= 16 ? 16 : (TPC == 32 ? 8 : 4);   // tokens a block
  constexpr int NV = KIND == 2 ? 3 : 2;                      // vectors over the key channels per token: q, k and the decays
  constexpr int SLICES = TB * NV * TPC;                      // 8-channel pieces of them in a block
  constexpr int PER = (SLICES + RT_THREADS - 1) / RT_THREADS;  // pieces a thread fetches
  constexpr int VALS = TB * CPG;                             // values of v in a block
  constexpr int VPER = (VALS + RT_THREADS - 1) / RT_THREADS;
  __shared__ __attribute__((aligned(16))) float qk_s[TB * NV * DP];  // per token: q [DP], k [DP], decays [DP]
  __shared__ float v_s[VALS];
  __shared__ float a_s[TB], w_s[TB];  // KIND 1: a token's decay; the weight of its k v^T

  const int tid = threadIdx.x, lane = tid % NS_WAVE, wave = tid / NS_WAVE, h = blockIdx.y, b = blockIdx.z;
  const int t0 = p.qo_indptr[b], t1 = p.qo_indptr[b + 1];
  if (t1 <= t0 || (p.skip_from > 0 && t1 - t0 >= p.skip_from)) return;
  const int H = p.r.H, D = p.r.D, E = p.r.E;
  const size_t row_w = p.r.row_w;
  const int kh = h / (H / p.r.G);
  const int s = lane % TPC, cw = wave * CPW + lane / TPC, col = blockIdx.x * CPG + cw, d0 = s * RT_KPT;
  const bool col_ok = col < E;
  float* st_S = p.state + (long long)p.state_slots[b] * p.state_stride + ((size_t)h * E + (col_ok ? col : 0)) * D;
  const float a = KIND == 0 ? p.r.decay[h] : 1.f;
  const float skip = KIND == 1 && p.r.skip ? p.r.skip[h] : 0.f;

  float S[RT_KPT];
#pragma unroll
  for (int j = 0; j < RT_KPT; ++j) S[j] = (col_ok && d0 + j < D) ? st_S[d0 + j] : 0.f;

  float pre[PER][RT_KPT], vpre[VPER], apre = 0.f, wpre = 1.f;
  auto fetch = [&](int t) {
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int idx = tid + i * RT_THREADS;  // (token, vector, piece)
      const int tk = idx / (NV * TPC), which = (idx / TPC) % NV, piece = idx % TPC;
      const bool live = idx < SLICES && t + tk < t1;
      const size_t row = t + (live ? tk : 0);
      const float* src = (KIND == 2 && which == 2) ? p.r.log_decay + (row * H + h) * D + piece * RT_KPT
                                                   : p.r.rows + row * row_w + (which ? p.r.k_off : p.r.q_off) + (size_t)kh * D + piece * RT_KPT;
      if (live && p.vec_ok && piece * RT_KPT + RT_KPT <= D) {
        const float4 x = *reinterpret_cast<const float4*>(src), y = *reinterpret_cast<const float4*>(src + 4);
        pre[i][0] = x.x, pre[i][1] = x.y, pre[i][2] = x.z, pre[i][3] = x.w, pre[i][4] = y.x, pre[i][5] = y.y, pre[i][6] = y.z, pre[i][7] = y.w;
      } else {
#pragma unroll
        for (int j = 0; j < RT_KPT; ++j) pre[i][j] = (live && piece * RT_KPT + j < D) ? src[j] : 0.f;
      }
    }
#pragma unroll
    for (int i = 0; i < VPER; ++i) {
      const int idx = tid + i * RT_THREADS, tk = idx / CPG, c = blockIdx.x * CPG + idx % CPG;
      vpre[i] = (idx < VALS && t + tk < t1 && c < E) ? p.r.rows[(size_t)(t + tk) * row_w + p.r.v_off + (size_t)h * E + c] : 0.f;
    }
    if (KIND == 1 && tid < TB) {
      const bool live = t + tid < t1;
      apre = live ? p.r.log_decay[(size_t)(t + tid) * H + h] : 0.f;
      wpre = (live && p.r.v_scale) ? p.r.v_scale[(size_t)(t + tid) * H + h] : 1.f;
    }
  };
  auto stage = [&]() {
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int idx = tid + i * RT_THREADS;
      if (idx < SLICES) {
        if (KIND == 2 && (idx / TPC) % NV == 2) {  // (tokens beyond the request's end and channels beyond the last: a decay of 1)
#pragma unroll
          for (int j = 0; j < RT_KPT; ++j) pre[i][j] = expf(pre[i][j]);
        }
        float4* dst = reinterpret_cast<float4*>(qk_s + (size_t)idx * RT_KPT);
        dst[0] = make_float4(pre[i][0], pre[i][1], pre[i][2], pre[i][3]);
        dst[1] = make_float4(pre[i][4], pre[i][5], pre[i][6], pre[i][7]);
      }
    }
#pragma unroll
    for (int i = 0; i < VPER; ++i) {
      const int idx = tid + i * RT_THREADS;
      if (idx < VALS) v_s[idx] = vpre[i];
    }
    if (KIND == 1 && tid < TB) a_s[tid] = expf(apre), w_s[tid] = wpre;
  };

  fetch(t0);
  stage();
  __syncthreads();
  constexpr int UN = 4;  // tokens worked through together: only S passes from token to token
  static_assert(TB % UN == 0, "a block of tokens is whole groups");
  for (int t = t0; t < t1; t += TB) {
    if (t + TB < t1) fetch(t + TB);
    const int nb = min(TB, t1 - t);
    for (int tk0 = 0; tk0 < nb; tk0 += UN) {
      float num[UN];
#pragma unroll
      for (int u = 0; u < UN; ++u) {
        const bool on = tk0 + u < nb;
        const float au = on ? (KIND == 1 ? a_s[tk0 + u] : a) : 1.f;  // (tokens beyond the block's end change nothing: their k and v are zero)
        const float vv = v_s[(tk0 + u) * CPG + cw] * (KIND == 1 ? w_s[tk0 + u] : 1.f);
        const float4* qp = reinterpret_cast<const float4*>(qk_s + (size_t)((tk0 + u) * NV) * DP + d0);
        const float4* kp = reinterpret_cast<const float4*>(qk_s + (size_t)((tk0 + u) * NV + 1) * DP + d0);
        const float4 q0 = qp[0], q1 = qp[1], k0 = kp[0], k1 = kp[1];
        const float q[RT_KPT] = {q0.x, q0.y, q0.z, q0.w, q1.x, q1.y, q1.z, q1.w};
        const float k[RT_KPT] = {k0.x, k0.y, k0.z, k0.w, k1.x, k1.y, k1.z, k1.w};
        float g[RT_KPT];
        if constexpr (KIND == 2) {
          const float4* gp = reinterpret_cast<const float4*>(qk_s + (size_t)((tk0 + u) * NV + 2) * DP + d0);
          const float4 g0 = gp[0], g1 = gp[1];
          g[0] = g0.x, g[1] = g0.y, g[2] = g0.z, g[3] = g0.w, g[4] = g1.x, g[5] = g1.y, g[6] = g1.z, g[7] = g1.w;
        } else {
#pragma unroll
          for (int j = 0; j < RT_KPT; ++j) g[j] = au;
        }
        float p0 = 0.f, p1 = 0.f;  // two partial sums: shorter chains
#pragma unroll
        for (int j = 0; j < RT_KPT; j += 2) {
          S[j] = fmaf(g[j], S[j], k[j] * vv);
          S[j + 1] = fmaf(g[j + 1], S[j + 1], k[j + 1] * vv);
          p0 = fmaf(S[j], q[j], p0);
          p1 = fmaf(S[j + 1], q[j + 1], p1);
        }
        num[u] = p0 + p1;
      }
#pragma unroll
      for (int u = 0; u < UN; ++u) num[u] = group_sum<TPC>(num[u]);
      if (s == 0 && col_ok) {
#pragma unroll
        for (int u = 0; u < UN; ++u)
          if (tk0 + u < nb) p.out[(size_t)(t + tk0 + u) * H * E + (size_t)h * E + col] = KIND == 1 ? fmaf(skip, v_s[(tk0 + u) * CPG + cw], num[u]) : num[u];
      }
    }
    __syncthreads();
    if (t + TB < t1) stage();
    __syncthreads();
  }
  if (col_ok) {
#pragma unroll
    for (int j = 0; j < RT_KPT; ++j)
      if (d0 + j < D) st_S[d0 + j] = S[j];
  }
}

template <int KIND>
static void retention_scan_launch(int tpc, dim3 grid, hipStream_t stream, const RetentionParams& p) {
  switch (tpc) {
    case 1: retention_scan_kernel<1, KIND><<<grid, RT_THREADS, 0, stream>>>(p); break;
    case 2: retention_scan_kernel<2, KIND><<<grid, RT_THREADS, 0, stream>>>(p); break;
    case 4: retention_scan_kernel<4, KIND><<<grid, RT_THREADS, 0, stream>>>(p); break;
    case 8: retention_scan_kernel<8, KIND><<<grid, RT_THREADS, 0, stream>>>(p); break;
    case 16: retention_scan_kernel<16, KIND><<<grid, RT_THREADS, 0, stream>>>(p); break;
    case 32: retention_scan_kernel<32, KIND><<<grid, RT_THREADS, 0, stream>>>(p); break;
    default: retention_scan_kernel<64, KIND><<<grid, RT_THREADS, 0, stream>>>(p); break;
  }
}

static int decay_rows_check(const DecayRows& r, int kind) {
  if (!r.rows || r.H <= 0 || r.H > 65535 || r.G <= 0 || r.H % r.G || r.D <= 0 || r.E <= 0 || r.q_off < 0 || r.k_off < 0 || r.v_off < 0) return NS_ERR_BAD_ARG;
  if (r.q_off + r.G * r.D > r.row_w || r.k_off + r.G * r.D > r.row_w || r.v_off + r.H * r.E > r.row_w) return NS_ERR_BAD_ARG;
  if (kind != 1 && (r.v_scale || r.skip)) return NS_ERR_BAD_ARG;
  if (kind < 0 || kind > 2 || (kind == 0 ? !r.decay : !r.log_decay)) return NS_ERR_BAD_ARG;
  return NS_OK;
}

// ``kind``: see above; exactly one of ``decay`` and ``log_decay`` is read
extern "C" int ns_retention_scan(const float* rows, int row_w, int q_off, int k_off, int v_off, const float* decay, float* log_decay,
                                 const float* v_scale, const float* skip, int kind, float* state, long long state_stride, const int* qo_indptr,
                                 const int* state_slots, float* out, int n_reqs, int H, int G, int D, int E, int skip_from, hipStream_t stream) {
  RetentionParams p{{rows, row_w, q_off, k_off, v_off, H, G, D, E, decay, log_decay, v_scale, skip}, state, state_stride, qo_indptr, state_slots, out,
                    0, skip_from};
  if (const int bad = decay_rows_check(p.r, kind)) return bad;
  if (n_reqs <= 0 || n_reqs > 65535) return NS_ERR_BAD_ARG;
  int tpc = 1;
  while (tpc * RT_KPT < D) tpc *= 2;
  if (tpc > NS_WAVE) return NS_ERR_UNSUPPORTED;
  if (state_stride < (long long)H * E * D) return NS_ERR_BAD_ARG;
  p.vec_ok = D % 8 == 0 && row_w % 4 == 0 && q_off % 4 == 0 && k_off % 4 == 0 && ((uintptr_t)rows % 16) == 0 && ((uintptr_t)log_decay % 16) == 0;
  const int cpg = RT_WAVES * NS_WAVE / tpc;
  dim3 grid((E + cpg - 1) / cpg, H, n_reqs);
  if (kind == 0) retention_scan_launch<0>(tpc, grid, stream, p);
  else if (kind == 1) retention_scan_launch<1>(tpc, grid, stream, p);
  else retention_scan_launch<2>(tpc, grid, stream, p);
  return ns_launch_status();
}

// ------------------------------------------------------------------------------------------------ long portions in chunks
#define RC_TOKENS 64  // tokens of a chunk
#define RC_INTS 4     // a chunk: request, row of its first token, tokens (0: no chunk), chunks of the request if it is its first (else 0)
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float rc_f32x4;

// What weighs the tokens of a chunk, in LDS.  KIND 0: pw[n] = a^n, n = 0 .. RC_TOKENS.  KIND 1: pw[j] = the sum of the logarithms
// of tokens 0 .. j.
template <int KIND>
__device__ __forceinline__ void rc_powers(float* pw, const DecayRows& r, int h, int row0, int nt) {
  if (KIND == 0) {
    const float a = r.decay[h];
    for (int i = threadIdx.x; i <= RC_TOKENS; i += blockDim.x) pw[i] = powf(a, (float)i);
  } else if (KIND == 1) {
    for (int i = threadIdx.x; i <= RC_TOKENS; i += blockDim.x) pw[i] = r.log_decay[(size_t)(row0 + min(i, nt - 1)) * r.H + h];
  }
  __syncthreads();
}

// The logarithms of the decays of every chunk's tokens, in place, become their sums from the chunk's first token on.
__global__ __launch_bounds__(256) void retention_chunk_sums_kernel(float* __restrict__ log_decay, const int* __restrict__ chunks, int width) {
  const int* ch = chunks + (size_t)blockIdx.y * RC_INTS;
  const int row0 = ch[1], nt = ch[2], c = blockIdx.x * blockDim.x + threadIdx.x;
  if (nt <= 0 || c >= width) return;
  float* p = log_decay + (size_t)row0 * width + c;
  float sum = 0.f;
  for (int t0 = 0; t0 < nt; t0 += 16) {
    float v[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) v[i] = p[(size_t)min(t0 + i, nt - 1) * width];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      sum += v[i];
      if (t0 + i < nt) p[(size_t)(t0 + i) * width] = sum;
    }
  }
}

// U of every chunk, [chunk][H][E][D].  grid (groups of four 64 x 64 tiles, H, chunks); a wave a tile of 64 value by 64 key channels:
// A = values weighted by what is left of their tokens at the chunk's end, B = keys (KIND 2: the weights are the keys', per
// channel), both straight from the rows (16 lanes read 64 neighbouring bytes).
template <int KIND>
__global__ __launch_bounds__(256) void retention_chunk_state_kernel(const DecayRows r, const int* __restrict__ chunks, float* __restrict__ ws) {
  __shared__ float pw[RC_TOKENS + 1];
  const int* ch = chunks + (size_t)blockIdx.z * RC_INTS;
  const int row0 = ch[1], nt = ch[2], h = blockIdx.y;
  if (nt <= 0) return;
  rc_powers<KIND>(pw, r, h, row0, nt);
  const int H = r.H, D = r.D, E = r.E;
  const int lane = threadIdx.x % NS_WAVE, wave = __builtin_amdgcn_readfirstlane(threadIdx.x / NS_WAVE), c = lane % 16, g = lane / 16;
  const int d_tiles = (D + 63) / 64, tile = blockIdx.x * 4 + wave;
  const int e0 = (tile / d_tiles) * 64, d0 = (tile % d_tiles) * 64;
  if (e0 >= E) return;
  const size_t row_w = r.row_w;
  const float* kp = r.rows + (size_t)row0 * row_w + r.k_off + (size_t)(h / (H / r.G)) * D;
  const float* vp = r.rows + (size_t)row0 * row_w + r.v_off + (size_t)h * E;
  const float* lp = KIND == 2 ? r.log_decay + (size_t)row0 * H * D + (size_t)h * D : nullptr;
  const float* sp = KIND == 1 && r.v_scale ? r.v_scale + (size_t)row0 * H + h : nullptr;
  rc_f32x4 acc[4][4];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = rc_f32x4{0.f, 0.f, 0.f, 0.f};
  // (channels beyond the last repeat it and are not stored; tokens beyond the last weigh nothing)
  int ei[4], di[4];
  float last[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    ei[i] = min(e0 + 16 * i + c, E - 1), di[i] = min(d0 + 16 * i + c, D - 1);
    last[i] = KIND == 2 ? lp[(size_t)(nt - 1) * H * D + di[i]] : 0.f;
  }
  // sixteen tokens (four steps) are on their way while the sixteen before them are multiplied
  float a[4][4], b[4][4], l[KIND == 2 ? 4 : 1][4], vs[4];
  auto fetch = [&](int j0) {
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      const size_t j = min(j0 + 4 * s + g, nt - 1), row = j * row_w;
      vs[s] = KIND == 1 && sp ? sp[j * H] : 1.f;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        a[s][i] = vp[row + ei[i]], b[s][i] = kp[row + di[i]];
        if constexpr (KIND == 2) l[s][i] = lp[j * H * D + di[i]];
      }
    }
  };
  fetch(0);
  for (int j0 = 0; j0 < nt; j0 += 16) {
    float ca[4][4], cb[4][4];
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      const int j = j0 + 4 * s + g;
      float w = 0.f;
      if (j < nt) w = vs[s] * (KIND == 0 ? pw[nt - 1 - j] : (KIND == 1 ? expf(pw[nt - 1] - pw[j]) : 1.f));
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        ca[s][i] = a[s][i] * w;
        if constexpr (KIND == 2) cb[s][i] = b[s][i] * expf(last[i] - l[s][i]);
        else cb[s][i] = b[s][i];
      }
    }
    if (j0 + 16 < nt) fetch(j0 + 16);
#pragma unroll
    for (int s = 0; s < 4; ++s)
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int n = 0; n < 4; ++n) acc[i][n] = __builtin_amdgcn_mfma_f32_16x16x4f32(ca[s][i], cb[s][n], acc[i][n], 0, 0, 0);
  }
  float* out = ws + ((size_t)blockIdx.z * H + h) * E * D;
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      const int e = e0 + 16 * i + 4 * g + q;
      if (e >= E) continue;
#pragma unroll
      for (int n = 0; n < 4; ++n) {
        const int d = d0 + 16 * n + c;
        if (d < D) out[(size_t)e * D + d] = acc[i][n][q];
      }
    }
}

// The pass over a request's chunks, four elements of the state a thread: U's place receives the state in front of the chunk.
// grid (pieces, chunks): the workgroups of a request's first chunk walk all of its chunks.
template <int KIND>
__global__ __launch_bounds__(256) void retention_chunk_pass_kernel(const DecayRows r, const int* __restrict__ chunks,
                                                                   const int* __restrict__ state_slots, float* __restrict__ state,
                                                                   long long state_stride, float* __restrict__ ws) {
  const int* ch = chunks + (size_t)blockIdx.y * RC_INTS;
  const int count = ch[3];
  if (ch[2] <= 0 || count <= 0) return;
  const int H = r.H, D = r.D, E = r.E;
  const size_t words = (size_t)H * E * D, at = ((size_t)blockIdx.x * blockDim.x + threadIdx.x) * 4;
  if (at >= words) return;
  const size_t h = at / ((size_t)E * D), d = at % D;
  const float a = KIND == 0 ? r.decay[h] : 0.f;
  const float full = KIND == 0 ? powf(a, (float)RC_TOKENS) : 0.f;
  // what a chunk of ``nt`` tokens from row ``row0`` on leaves of the state in front of it
  auto left = [&](const int* c) {
    rc_f32x4 f;
    if (KIND == 0) {
      const float v = c[2] == RC_TOKENS ? full : powf(a, (float)c[2]);
      f = rc_f32x4{v, v, v, v};
    } else if (KIND == 1) {
      const float v = expf(r.log_decay[(size_t)(c[1] + c[2] - 1) * H + h]);
      f = rc_f32x4{v, v, v, v};
    } else {
      f = *reinterpret_cast<const rc_f32x4*>(r.log_decay + (size_t)(c[1] + c[2] - 1) * H * D + h * D + d);
#pragma unroll
      for (int e = 0; e < 4; ++e) f[e] = expf(f[e]);
    }
    return f;
  };
  float* sp = state + (long long)state_slots[ch[0]] * state_stride + at;
  float* u = ws + (size_t)blockIdx.y * words + at;
  rc_f32x4 S = *reinterpret_cast<const rc_f32x4*>(sp);
  rc_f32x4 next = *reinterpret_cast<const rc_f32x4*>(u), next_f = left(ch);
  for (int i = 0; i < count; ++i) {
    const rc_f32x4 cur = next, f = next_f;
    if (i + 1 < count) {
      next = *reinterpret_cast<const rc_f32x4*>(u + words);
      next_f = left(ch + (size_t)(i + 1) * RC_INTS);
    }
    *reinterpret_cast<rc_f32x4*>(u) = S;
#pragma unroll
    for (int e = 0; e < 4; ++e) S[e] = fmaf(f[e], S[e], cur[e]);
    u += words;
  }
  *reinterpret_cast<rc_f32x4*>(sp) = S;
}

// The outputs of every chunk.  grid (blocks of 16 * ET value channels, H, chunks); wave w takes tokens 16 w .. 16 w + 15 of the
// chunk.  The products q . k are kept transposed (rows j, columns i): what a lane then holds of them, j = 4 g + r in register r
// for token i = lane % 16, is the A operand of the product with the values, whose four steps take the rows j = 4 g + r in
// that order, so they never leave the registers.  Where both operands run along the key channels, a lane's four neighbouring
// channels (one 16-byte load) are those of four steps.
//
// KIND 2: with L_t the sum of the logarithms up to token t, the product of token i's query and token j's key carries
// exp(L_i - L_j) per channel.  Across the sixteens of a chunk it is split at the token in front of the query's sixteen, exp(L_i -
// L_ref) exp(L_ref - L_j), both at most 1.  Within a sixteen it is split at its eighth token, whose factors are bounded by what
// eight tokens forget; sixteens of channels in which that is more than exp(RC_SPLIT) form every pair's factor by itself.
#define RC_SPLIT 40.f
template <int KIND, int ET>
__global__ __launch_bounds__(256, 2) void retention_chunk_out_kernel(const DecayRows r, const int* __restrict__ chunks, const float* __restrict__ ws,
                                                                     float* __restrict__ out) {
  __shared__ float pw[RC_TOKENS + 1];
  const int* ch = chunks + (size_t)blockIdx.z * RC_INTS;
  const int row0 = ch[1], nt = ch[2], h = blockIdx.y;
  if (nt <= 0) return;
  rc_powers<KIND>(pw, r, h, row0, nt);
  const int H = r.H, D = r.D, E = r.E;
  const int lane = threadIdx.x % NS_WAVE, wave = __builtin_amdgcn_readfirstlane(threadIdx.x / NS_WAVE), c = lane % 16, g = lane / 16;
  const int i0 = 16 * wave, e0 = blockIdx.x * 16 * ET;
  if (i0 >= nt) return;
  const size_t row_w = r.row_w, lrow = (size_t)H * D;
  const float* base = r.rows + (size_t)row0 * row_w + (size_t)(h / (H / r.G)) * D;
  const float* lbase = KIND == 2 ? r.log_decay + (size_t)row0 * lrow + (size_t)h * D : nullptr;
  const int qi = min(i0 + c, nt - 1);
  const float* qp = base + (size_t)qi * row_w + r.q_off;
  const float* kp[4];
  const float* lk[4];
#pragma unroll
  for (int t = 0; t < 4; ++t) {
    kp[t] = base + (size_t)min(16 * t + c, nt - 1) * row_w + r.k_off;
    lk[t] = KIND == 2 ? lbase + (size_t)min(16 * t + c, nt - 1) * lrow : nullptr;
  }
  const float* sp[ET];
  int ei[ET];
#pragma unroll
  for (int t = 0; t < ET; ++t) {
    ei[t] = min(e0 + 16 * t + c, E - 1);
    sp[t] = ws + (((size_t)blockIdx.z * H + h) * E + ei[t]) * D;
  }
  const rc_f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  rc_f32x4 pt[4], acc[ET];
#pragma unroll
  for (int t = 0; t < 4; ++t) pt[t] = zero;
#pragma unroll
  for (int t = 0; t < ET; ++t) acc[t] = zero;
  // the next sixteen channels are on their way while these are multiplied
  rc_f32x4 nq, nk[4], ns[ET], nlk[KIND == 2 ? 4 : 1];
  rc_f32x4 nref = zero, nmid = zero, nfirst = zero, nlast = zero;  // L of the token in front of the sixteen, of its eighth, first and last
  auto load4 = [&](const float* p, bool ok) { return ok ? *reinterpret_cast<const rc_f32x4*>(p) : zero; };
  auto fetch = [&](int d0) {
    const int d = d0 + 4 * g;
    const bool ok = d < D;  // (D is a multiple of four: a lane's four channels are inside or outside together)
    nq = load4(qp + d, ok);
#pragma unroll
    for (int t = 0; t < 4; ++t)
      if (t <= wave) {
        nk[t] = load4(kp[t] + d, ok);
        if constexpr (KIND == 2) nlk[t] = load4(lk[t] + d, ok);
      }
#pragma unroll
    for (int t = 0; t < ET; ++t) ns[t] = load4(sp[t] + d, ok);
    if constexpr (KIND == 2) {
      if (i0 > 0) nref = load4(lbase + (size_t)(i0 - 1) * lrow + d, ok);
      nmid = load4(lbase + (size_t)min(i0 + 7, nt - 1) * lrow + d, ok);
      nfirst = load4(lbase + (size_t)i0 * lrow + d, ok);
      nlast = load4(lbase + (size_t)min(i0 + 15, nt - 1) * lrow + d, ok);
    }
  };
  fetch(0);
  for (int d0 = 0; d0 < D; d0 += 16) {
    rc_f32x4 q = nq;
    rc_f32x4 k[4], s[ET], qr = nq, qd = nq;  // the query as it meets the state, earlier sixteens, and its own
    bool split = true;                       // (wave-uniform)
#pragma unroll
    for (int t = 0; t < 4; ++t) k[t] = nk[t];
#pragma unroll
    for (int t = 0; t < ET; ++t) s[t] = ns[t];
    if constexpr (KIND == 2) {
      rc_f32x4 lq = zero;  // L of the query's own token: the key of the same token holds it
#pragma unroll
      for (int t = 0; t < 4; ++t)
        if (t == wave) lq = nlk[t];
      float widest = 0.f;
#pragma unroll
      for (int e = 0; e < 4; ++e) widest = fmaxf(widest, nfirst[e] - nlast[e]);
      split = !__any(!(widest <= RC_SPLIT));
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        q[e] *= expf(lq[e]), qr[e] *= expf(lq[e] - nref[e]);
        qd[e] *= split ? expf(lq[e] - nmid[e]) : 0.f;
      }
#pragma unroll
      for (int t = 0; t < 4; ++t) {
        if (t < wave) {
#pragma unroll
          for (int e = 0; e < 4; ++e) k[t][e] *= expf(nref[e] - nlk[t][e]);
        } else if (t == wave) {  // (not split: the pairs of this sixteen are formed below)
#pragma unroll
          for (int e = 0; e < 4; ++e) k[t][e] *= split ? expf(nmid[e] - nlk[t][e]) : 0.f;
        }
      }
    }
    if (d0 + 16 < D) fetch(d0 + 16);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
#pragma unroll
      for (int t = 0; t < 4; ++t)
        if (t <= wave) pt[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(k[t][e], KIND != 2 ? q[e] : (t < wave ? qr[e] : qd[e]), pt[t], 0, 0, 0);
#pragma unroll
      for (int t = 0; t < ET; ++t) acc[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(q[e], s[t][e], acc[t], 0, 0, 0);
    }
    if constexpr (KIND == 2) {
      if (!split) {
        const float* li = lbase + (size_t)qi * lrow;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int j = min(i0 + 4 * g + e, nt - 1);
          const float* kj = base + (size_t)j * row_w + r.k_off;
          const float* lj = lbase + (size_t)j * lrow;
          float sum = 0.f;
          for (int d = d0; d < min(d0 + 16, D); ++d) sum = fmaf(qp[d] * kj[d], expf(fminf(li[d] - lj[d], 0.f)), sum);
#pragma unroll
          for (int t = 0; t < 4; ++t)
            if (t == wave) pt[t][e] += sum;
        }
      }
    }
  }
  if (KIND != 2) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = i0 + 4 * g + e;
      const float f = KIND == 0 ? pw[min(i + 1, RC_TOKENS)] : expf(pw[i]);
#pragma unroll
      for (int t = 0; t < ET; ++t) acc[t][e] *= f;
    }
  }
  float v[4][ET], vs[4];
  auto values = [&](int t) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int j = row0 + min(16 * t + 4 * g + e, nt - 1);
      const float* vp = r.rows + (size_t)j * row_w + r.v_off + (size_t)h * E;
      vs[e] = KIND == 1 && r.v_scale ? r.v_scale[(size_t)j * H + h] : 1.f;
#pragma unroll
      for (int n = 0; n < ET; ++n) v[e][n] = vp[ei[n]];
    }
  };
  values(0);
#pragma unroll
  for (int t = 0; t < 4; ++t) {
    if (t > wave) continue;
    float cv[4][ET], cs[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      cs[e] = vs[e];
#pragma unroll
      for (int n = 0; n < ET; ++n) cv[e][n] = v[e][n];
    }
    if (t < wave) values(t + 1);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = i0 + c, j = 16 * t + 4 * g + e;
      const float p = j <= i ? pt[t][e] * cs[e] * (KIND == 0 ? pw[i - j] : (KIND == 1 ? expf(pw[i] - pw[j]) : 1.f)) : 0.f;
#pragma unroll
      for (int n = 0; n < ET; ++n) acc[n] = __builtin_amdgcn_mfma_f32_16x16x4f32(p, cv[e][n], acc[n], 0, 0, 0);
    }
  }
  const float skip = KIND == 1 && r.skip ? r.skip[h] : 0.f;
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const int i = i0 + 4 * g + e;
    if (i >= nt) continue;
    float* o = out + (size_t)(row0 + i) * H * E + (size_t)h * E;
    const float* vp = r.rows + (size_t)(row0 + i) * row_w + r.v_off + (size_t)h * E;
#pragma unroll
    for (int n = 0; n < ET; ++n) {
      const int at = e0 + 16 * n + c;
      if (at < E) o[at] = KIND == 1 && r.skip ? fmaf(skip, vp[at], acc[n][e]) : acc[n][e];
    }
  }
}

template <int KIND>
static void retention_chunks_launch(const DecayRows& r, float* state, long long state_stride, const int* chunks, int n_chunks, const int* state_slots,
                                    float* ws, float* out, hipStream_t stream) {
  const int tiles = ((r.D + 63) / 64) * ((r.E + 63) / 64);
  if (KIND != 0) {
    const int width = KIND == 1 ? r.H : r.H * r.D;
    retention_chunk_sums_kernel<<<dim3((width + 255) / 256, n_chunks), 256, 0, stream>>>(r.log_decay, chunks, width);
  }
  retention_chunk_state_kernel<KIND><<<dim3((tiles + 3) / 4, r.H, n_chunks), 256, 0, stream>>>(r, chunks, ws);
  const size_t pieces = ((size_t)r.H * r.E * r.D / 4 + 255) / 256;
  retention_chunk_pass_kernel<KIND><<<dim3((int)pieces, n_chunks), 256, 0, stream>>>(r, chunks, state_slots, state, state_stride, ws);
  if (KIND == 2 || r.E <= 64)  // (with decays per channel the registers hold no more than 64 value channels)
    retention_chunk_out_kernel<KIND, 4><<<dim3((r.E + 63) / 64, r.H, n_chunks), 256, 0, stream>>>(r, chunks, ws, out);
  else
    retention_chunk_out_kernel<KIND, KIND == 2 ? 4 : 8><<<dim3((r.E + 127) / 128, r.H, n_chunks), 256, 0, stream>>>(r, chunks, ws, out);
}

// ``chunks``: int32 [n_chunks][RC_INTS]; ``ws``: float32 [n_chunks][H * E * D]
extern "C" int ns_retention_chunks(const float* rows, int row_w, int q_off, int k_off, int v_off, const float* decay, float* log_decay,
                                   const float* v_scale, const float* skip, int kind, float* state, long long state_stride, const int* chunks,
                                   int n_chunks, const int* state_slots, float* ws, float* out, int H, int G, int D, int E, hipStream_t stream) {
  const DecayRows r{rows, row_w, q_off, k_off, v_off, H, G, D, E, decay, log_decay, v_scale, skip};
  if (const int bad = decay_rows_check(r, kind)) return bad;
  if (n_chunks <= 0 || n_chunks > 65535) return NS_ERR_BAD_ARG;
  if (D % 4 || state_stride % 4 || (uintptr_t)rows % 16 || (uintptr_t)state % 16 || (uintptr_t)ws % 16 || row_w % 4 || q_off % 4 || k_off % 4 ||
      (kind == 2 && (uintptr_t)log_decay % 16))
    return NS_ERR_UNSUPPORTED;
  if (state_stride < (long long)H * E * D || ((size_t)H * E * D / 4 + 255) / 256 > 0x7fffffff) return NS_ERR_BAD_ARG;
  if (kind == 0) retention_chunks_launch<0>(r, state, state_stride, chunks, n_chunks, state_slots, ws, out, stream);
  else if (kind == 1) retention_chunks_launch<1>(r, state, state_stride, chunks, n_chunks, state_slots, ws, out, stream);
  else retention_chunks_launch<2>(r, state, state_stride, chunks, n_chunks, state_slots, ws, out, stream);
  return ns_launch_status();
}

// The step sizes of a state-space recurrence and the logarithms of the decays per head that they make:
//   dt[t][h] = softplus(z[t][h] + bias[h]);  log_decay[t][h] = -exp(a_log[h]) dt[t][h]
// z in the model's precision (it may be a column slice of wider rows), everything else in 32-bit.
template <typename T>
__global__ void log_decay_heads_kernel(float* __restrict__ dt, float* __restrict__ log_decay, const T* __restrict__ z, int z_stride,
                                       const float* __restrict__ bias, const float* __restrict__ a_log, int H, size_t count) {
  const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= count) return;
  const size_t t = i / H, h = i % H;
  const float d = softplus_f(to_f(z[t * z_stride + h]) + bias[h]);
  dt[i] = d;
  log_decay[i] = -expf(a_log[h]) * d;
}

extern "C" int ns_log_decay_heads(float* dt, float* log_decay, const void* z, int z_stride, const float* bias, const float* a_log, int n, int H,
                                  int dtype, hipStream_t stream) {
  if (n <= 0 || H <= 0) return NS_ERR_BAD_ARG;
  const size_t count = (size_t)n * H, blocks = (count + 255) / 256;
  if (blocks > 0x7fffffff) return NS_ERR_BAD_ARG;
  if (dtype == NS_DTYPE_F32)
    log_decay_heads_kernel<float><<<(int)blocks, 256, 0, stream>>>(dt, log_decay, (const float*)z, z_stride, bias, a_log, H, count);
  else if (dtype == NS_DTYPE_BF16)
    log_decay_heads_kernel<bf16_t><<<(int)blocks, 256, 0, stream>>>(dt, log_decay, (const bf16_t*)z, z_stride, bias, a_log, H, count);
  else
    return NS_ERR_UNSUPPORTED;
  return ns_launch_status();
}

// y[t][i] = x[t][i] * sigmoid(z)  (silu = 0)  or  x[t][i] * z sigmoid(z)  (silu = 1), z = g[t][i / share]: ``share`` neighbouring
// channels (a head's) have one gate; g may be a column slice
template <typename T>
__global__ void gate_mul_kernel(T* __restrict__ out, const T* __restrict__ x, const T* __restrict__ g, int g_stride, int width, int share, size_t count,
                                int silu) {
  const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= count) return;
  const size_t t = i / width, c = i % width;
  const float z = to_f(g[t * g_stride + c / share]);
  const float gate = (silu ? z : 1.f) / (1.f + expf(-z));
  out[i] = from_f<T>(to_f(x[i]) * gate);
}

extern "C" int ns_gate_mul(void* out, const void* x, const void* g, int g_stride, int n, int width, int share, int silu, int dtype, hipStream_t stream) {
  if (n <= 0 || width <= 0 || share <= 0 || width % share) return NS_ERR_BAD_ARG;
  const size_t count = (size_t)n * width, blocks = (count + 255) / 256;
  if (blocks > 0x7fffffff) return NS_ERR_BAD_ARG;
  if (dtype == NS_DTYPE_F32)
    gate_mul_kernel<float><<<(int)blocks, 256, 0, stream>>>((float*)out, (const float*)x, (const float*)g, g_stride, width, share, count, silu);
  else if (dtype == NS_DTYPE_BF16)
    gate_mul_kernel<bf16_t><<<(int)blocks, 256, 0, stream>>>((bf16_t*)out, (const bf16_t*)x, (const bf16_t*)g, g_stride, width, share, count, silu);
  else
    return NS_ERR_UNSUPPORTED;
  return ns_launch_status();
}
