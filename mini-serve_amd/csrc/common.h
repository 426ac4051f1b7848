// Shared device helpers for the gfx950 kernels: element types, conversions, wave and block reductions.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

typedef __bf16 bf16;

#define WAVE 64

// Error codes returned by every extern "C" entry point (0 = launched).
#define MS_OK 0
#define MS_BAD_ARG 1
#define MS_UNSUPPORTED 2
#define MS_LAUNCH_FAILED 3

__device__ __forceinline__ float to_f32(float x) { return x; }
__device__ __forceinline__ float to_f32(bf16 x) { return static_cast<float>(x); }

template <typename T> __device__ __forceinline__ T from_f32(float x);
template <> __device__ __forceinline__ float from_f32<float>(float x) { return x; }
template <> __device__ __forceinline__ bf16 from_f32<bf16>(float x) { return static_cast<bf16>(x); }

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int off = WAVE / 2; off > 0; off >>= 1) v += __shfl_xor(v, off, WAVE);
  return v;
}

__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
  for (int off = WAVE / 2; off > 0; off >>= 1) v = fmaxf(v, __shfl_xor(v, off, WAVE));
  return v;
}

// Maximum / sum over the four lanes l, l ^ 16, l ^ 32, l ^ 48 (one element of each 16-lane row), the
// same bits in all four: v_permlane16_swap and v_permlane32_swap hand a lane its partner's value
// without a trip through LDS. The sum is (row 0 + row 1) + (row 2 + row 3) for every lane.
__device__ __forceinline__ float rows4_max(float v) {
  auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  v = fmaxf(__uint_as_float(a[0]), __uint_as_float(a[1]));
  auto b = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  return fmaxf(__uint_as_float(b[0]), __uint_as_float(b[1]));
}
__device__ __forceinline__ float rows4_sum(float v) {
  auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  v = __uint_as_float(a[0]) + __uint_as_float(a[1]);
  auto b = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  return __uint_as_float(b[0]) + __uint_as_float(b[1]);
}

// Sum over a block of NT threads (NT a multiple of 64, at most 1024). `red` holds NT / 64 floats.
// Every thread receives the total; the order of additions is fixed by NT alone.
template <int NT> __device__ __forceinline__ float block_sum(float v, float* red) {
  v = wave_sum(v);
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
  __syncthreads();
  if (lane == 0) red[wave] = v;
  __syncthreads();
  float total = 0.f;
#pragma unroll
  for (int i = 0; i < NT / WAVE; ++i) total += red[i];
  return total;
}

// Sum of `splits` floats spaced `stride` apart, added in ascending order. Loads are issued eight at a
// time so that they overlap; absent splits contribute an exact zero.
__device__ __forceinline__ float sum_splits(const float* __restrict__ p, int splits, size_t stride) {
  float acc = 0.f;
  for (int s0 = 0; s0 < splits; s0 += 8) {
    float v[8];
#pragma unroll
    for (int u = 0; u < 8; ++u) v[u] = (s0 + u < splits) ? p[(size_t)(s0 + u) * stride] : 0.f;
#pragma unroll
    for (int u = 0; u < 8; ++u) acc += v[u];
  }
  return acc;
}

// acc += parts of splits s0 .. s0 + B - 1 (those below `splits`), four floats each, in ascending order;
// the B loads are issued before the first sum.
template <int B>
__device__ __forceinline__ void add_splits(float4& acc, const float* __restrict__ p, int s0, int splits, size_t split_stride) {
  float4 t[B];
#pragma unroll
  for (int u = 0; u < B; ++u) {
    const bool in = s0 + u < splits;
    t[u] = *reinterpret_cast<const float4*>(p + (size_t)(in ? s0 + u : 0) * split_stride);
    if (!in) t[u] = make_float4(0.f, 0.f, 0.f, 0.f);
  }
#pragma unroll
  for (int u = 0; u < B; ++u) {
    acc.x += t[u].x; acc.y += t[u].y; acc.z += t[u].z; acc.w += t[u].w;
  }
}

// Four consecutive weights in one load (w + i is aligned to four elements), kept as loaded: what uses
// them comes after the block's sum, and a conversion right after the load would wait for it there.
template <typename TW> struct Weights4;
template <> struct Weights4<float> {
  float4 v;
  __device__ __forceinline__ void load(const float* w) { v = *reinterpret_cast<const float4*>(w); }
  __device__ __forceinline__ float at(int e) const { return e == 0 ? v.x : e == 1 ? v.y : e == 2 ? v.z : v.w; }
};
template <> struct Weights4<bf16> {
  union { uint2 u; bf16 e[4]; } v;
  __device__ __forceinline__ void load(const bf16* w) { v.u = *reinterpret_cast<const uint2*>(w); }
  __device__ __forceinline__ float at(int e) const { return to_f32(v.e[e]); }
};

// The sum of `splits` slices, four floats each, in ascending order. The loads of a batch of splits go out together; few
// splits (a tile product's two to four) take a batch of their own size, so that no load is issued for nothing.
__device__ __forceinline__ float4 add_splits4(const float* __restrict__ p, int splits, size_t split_stride) {
  float4 acc = make_float4(0.f, 0.f, 0.f, 0.f);
  if (splits == 1) {
    add_splits<1>(acc, p, 0, splits, split_stride);
  } else if (splits <= 2) {
    add_splits<2>(acc, p, 0, splits, split_stride);
  } else if (splits <= 4) {
    add_splits<4>(acc, p, 0, splits, split_stride);
  } else if (splits <= 8) {
    add_splits<8>(acc, p, 0, splits, split_stride);
  } else {  // the products of a decode step leave 12 to 16: one round trip, not two
    for (int s0 = 0; s0 < splits; s0 += 16) add_splits<16>(acc, p, s0, splits, split_stride);
  }
  return acc;
}

// Which elements of a head make pair j of a rotary position encoding: (j, j + rot/2) or (2j, 2j + 1).
#define MS_ROPE_HALVES 0
#define MS_ROPE_ADJACENT 1

// Activations of the gated feed-forward, by the number the host passes: out = act(gate) * up, in float32.
#define MS_ACT_SILU 0
#define MS_ACT_GELU_TANH 1
// A gated feed-forward with bounded inputs: g = min(gate, limit), u = clamp(up, -limit, limit),
// out = g sigmoid(1.702 g) (u + 1). Not of the form act(gate) * up: it takes `limit` beside the number.
#define MS_ACT_SWIGLU_CLAMPED 2
#define MS_GATED_COUNT 3  // what a gated feed-forward may run: the matrix kernels' epilogues and the activation kernels know them
// The square of max(x, 0): only as the activation of a feed-forward without a gate.
#define MS_ACT_RELU_SQUARED 3
// The hyperbolic tangent: between the two steps of a small projection, never in a feed-forward's gate.
#define MS_ACT_TANH 4
static __host__ __device__ __forceinline__ bool ms_act_ungated_ok(int act) {
  return act == MS_ACT_SILU || act == MS_ACT_GELU_TANH || act == MS_ACT_RELU_SQUARED || act == MS_ACT_TANH;
}
__device__ __forceinline__ float activate(float x, int act) {
  if (act == MS_ACT_RELU_SQUARED) { const float r = fmaxf(x, 0.f); return r * r; }
  if (act == MS_ACT_TANH) return tanhf(x);
  if (act == MS_ACT_GELU_TANH) return 0.5f * x * (1.f + tanhf(0.7978845608028654f * (x + 0.044715f * x * x * x)));
  return x / (1.f + expf(-x));
}
// log(1 + exp(z)) without overflow.
__device__ __forceinline__ float softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
// What a gated feed-forward makes of one gate and one up value, float32.
__device__ __forceinline__ float gated_value(float gate, float up, int act, float limit) {
  if (act == MS_ACT_SWIGLU_CLAMPED) {
    const float g = fminf(gate, limit);
    const float u = fminf(fmaxf(up, -limit), limit);
    return g / (1.f + expf(-1.702f * g)) * (u + 1.f);
  }
  return activate(gate, act) * up;
}

static inline int launch_status() { return hipGetLastError() == hipSuccess ? MS_OK : MS_LAUNCH_FAILED; }
