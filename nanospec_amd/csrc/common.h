// Shared device helpers of the nanospec_amd kernels (gfx950 / CDNA4, wave64).
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

typedef __bf16 bf16_t;

#define NS_DTYPE_F32 0
#define NS_DTYPE_BF16 1
#define NS_WAVE 64

// Error codes returned by every extern "C" entry point (0 = launched).
#define NS_OK 0
#define NS_ERR_BAD_ARG 1001
#define NS_ERR_UNSUPPORTED 1002
#define NS_ERR_SCRATCH_TOO_SMALL 1003

template <typename T> __device__ __forceinline__ float to_f(T v) { return (float)v; }
template <typename T> __device__ __forceinline__ T from_f(float v) { return (T)v; }
// Round a 32-bit value to the storage type and come back: what a store followed by a load does.
template <typename T> __device__ __forceinline__ float round_to(float v) { return (float)(T)v; }

// The activations a kernel may be asked for by number: 0 the tanh form of GELU, 0.5 z (1 + tanh(sqrt(2/pi) (z + 0.044715
// z^3))); 1 SiLU, z sigmoid(z); 2 the square of the ReLU.
#define NS_ACTIVATIONS 3
__device__ __forceinline__ float activation_of(float z, int act) {
  if (act == 0) return 0.5f * z * (1.f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
  if (act == 1) return z / (1.f + expf(-z));
  const float r = fmaxf(z, 0.f);
  return r * r;
}

__device__ __forceinline__ float softplus_f(float z) { return z > 20.f ? z : log1pf(expf(z)); }

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int o = NS_WAVE / 2; o > 0; o >>= 1) v += __shfl_xor(v, o, NS_WAVE);
  return v;
}
__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
  for (int o = NS_WAVE / 2; o > 0; o >>= 1) v = fmaxf(v, __shfl_xor(v, o, NS_WAVE));
  return v;
}

// The sum of a value over RGC neighbouring lanes (a power of two; the group starts at a multiple of RGC), in all of them.  Up to 16 lanes lie in one row of the
// wave, where a lane reads its partner through the data path of the vector unit itself (quad permutations, then the
// mirrored half row and row: any partner in the other half will do for a sum); wider groups go on through LDS's crossbar.
template <int CTRL>
__device__ __forceinline__ float dpp_read(float v) {
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xf, 0xf, true));
}
template <int RGC>
__device__ __forceinline__ float group_sum(float v) {
  if constexpr (RGC >= 2) v += dpp_read<0xB1>(v);   // quad_perm [1, 0, 3, 2]
  if constexpr (RGC >= 4) v += dpp_read<0x4E>(v);   // quad_perm [2, 3, 0, 1]
  if constexpr (RGC >= 8) v += dpp_read<0x141>(v);  // row_half_mirror
  if constexpr (RGC >= 16) v += dpp_read<0x140>(v); // row_mirror
#pragma unroll
  for (int o = 16; o < RGC; o <<= 1) v += __shfl_xor(v, o, NS_WAVE);
  return v;
}

// Block-wide reductions for blocks of up to 1024 threads; `scratch` holds >= 16 floats of LDS.
// Every thread gets the result.  The order of the additions is fixed by the thread layout only.
__device__ __forceinline__ float block_sum(float v, float* scratch) {
  const int lane = threadIdx.x & (NS_WAVE - 1), wave = threadIdx.x / NS_WAVE;
  const int nwaves = (blockDim.x + NS_WAVE - 1) / NS_WAVE;
  v = wave_sum(v);
  __syncthreads();
  if (lane == 0) scratch[wave] = v;
  __syncthreads();
  float r = 0.f;
  for (int i = 0; i < nwaves; ++i) r += scratch[i];
  return r;
}
__device__ __forceinline__ float block_max(float v, float* scratch) {
  const int lane = threadIdx.x & (NS_WAVE - 1), wave = threadIdx.x / NS_WAVE;
  const int nwaves = (blockDim.x + NS_WAVE - 1) / NS_WAVE;
  v = wave_max(v);
  __syncthreads();
  if (lane == 0) scratch[wave] = v;
  __syncthreads();
  float r = -INFINITY;
  for (int i = 0; i < nwaves; ++i) r = fmaxf(r, scratch[i]);
  return r;
}

static inline int ns_launch_status() {
  hipError_t e = hipGetLastError();
  return e == hipSuccess ? NS_OK : (int)e;
}
