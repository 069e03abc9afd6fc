// Shared definitions for the gfx950 kernels: element types, error codes, small device helpers.
// Every entry point is extern "C", takes raw device pointers and a hipStream_t, launches
// asynchronously on that stream and returns 0, or a negative code without launching anything.
#pragma once

#include <hip/hip_runtime.h>
#include <hip/hip_bf16.h>
#include <stdint.h>

#define CW_OK 0
#define CW_ERR_ARG -1      // a size or pointer the kernel does not take
#define CW_ERR_DTYPE -2    // unknown element type code
#define CW_ERR_LAUNCH -3   // the HIP runtime refused the launch
#define CW_ERR_SIZE -4     // beyond a stated maximum

#define CW_F32 0
#define CW_BF16 1

#define CW_EXPORT extern "C" __attribute__((visibility("default")))

typedef __hip_bfloat16 bf16_t;

__device__ __forceinline__ float cw_to_float(float x) { return x; }
__device__ __forceinline__ float cw_to_float(bf16_t x) { return __bfloat162float(x); }

template <typename T> __device__ __forceinline__ T cw_from_float(float x);
template <> __device__ __forceinline__ float cw_from_float<float>(float x) { return x; }
template <> __device__ __forceinline__ bf16_t cw_from_float<bf16_t>(float x) { return __float2bfloat16(x); }

// bfloat16 bits <-> float without going through the class type (for packed 16-byte loads)
__device__ __forceinline__ float cw_bf16_bits_to_float(uint16_t b) {
  return __uint_as_float(((uint32_t)b) << 16);
}
__device__ __forceinline__ uint16_t cw_float_to_bf16_bits(float f) {
  // round to nearest even; NaN stays NaN
  uint32_t u = __float_as_uint(f);
  if ((u & 0x7fffffffu) > 0x7f800000u) return (uint16_t)((u >> 16) | 0x40u);
  u += 0x7fffu + ((u >> 16) & 1u);
  return (uint16_t)(u >> 16);
}

// Maximum / sum over the four lanes l, l ^ 16, l ^ 32, l ^ 48 of a wave, on the vector unit: the
// swaps of 16-lane rows and of the wave's halves (v_permlane16_swap, v_permlane32_swap) hand every
// lane both values of its pair, so all four lanes end with the same result, summed as
// (l + l^16) + (l^32 + l^48). (A shuffle goes through the LDS unit and waits behind its queue.)
typedef __attribute__((ext_vector_type(2))) unsigned int cw_u32x2_t;
__device__ __forceinline__ float cw_quad_max(float v) {
  const cw_u32x2_t a = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  v = fmaxf(__uint_as_float(a[0]), __uint_as_float(a[1]));
  const cw_u32x2_t b = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  return fmaxf(__uint_as_float(b[0]), __uint_as_float(b[1]));
}
__device__ __forceinline__ float cw_quad_sum(float v) {
  const cw_u32x2_t a = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  v = __uint_as_float(a[0]) + __uint_as_float(a[1]);
  const cw_u32x2_t b = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  return __uint_as_float(b[0]) + __uint_as_float(b[1]);
}

// The clipped gated activation: g = min(gate, limit), u = up cut to [-limit, limit];
// g * logistic(1.702 g) * (u + 1).
__device__ __forceinline__ float cw_clipped_glu(float gate, float up, float limit) {
  const float g = fminf(gate, limit), u = fminf(fmaxf(up, -limit), limit);
  return g / (1.0f + expf(-1.702f * g)) * (u + 1.0f);
}
// What the kernels of gate/up products make of a gate and an up value: ``act`` > 0 the clipped gated
// activation of that limit, < 0 max(gate, 0) * up, else silu(gate) * up.
__device__ __forceinline__ float cw_gated(float g, float u, float act) {
  return act > 0.0f ? cw_clipped_glu(g, u, act) : act < 0.0f ? fmaxf(g, 0.0f) * u : g / (1.0f + expf(-g)) * u;
}
// The tanh form of GELU, 0.5 z (1 + tanh(y)) with y = sqrt(2 / pi) (z + 0.044715 z^3), through
// 0.5 (1 + tanh(y)) = 1 / (1 + exp(-2 y)).
__device__ __forceinline__ float cw_gelu_tanh(float z) {
  return z / (1.0f + expf(-1.5957691216057308f * (z + 0.044715f * z * z * z)));
}

// Functions from the bare exp2, log2 and reciprocal instructions: a few units in the last place, and a
// fraction of the code of the library's (a kernel that runs for microseconds waits for its own code).
__device__ __forceinline__ float cw_exp_quick(float z) { return __builtin_amdgcn_exp2f(1.44269504f * z); }
__device__ __forceinline__ float cw_logistic(float z) { return __builtin_amdgcn_rcpf(1.0f + cw_exp_quick(-z)); }
__device__ __forceinline__ float cw_silu(float z) { return z * cw_logistic(z); }
// tanh: a power series for small z, else (1 - e) / (1 + e) with e = exp(-2 |z|)
__device__ __forceinline__ float cw_tanh_quick(float z) {
  const float s = z * z, e = cw_exp_quick(-2.0f * fabsf(z));
  const float series = z * (1.0f + s * (-0.333333333f + s * (0.133333333f + s * (-0.053968254f + s * 0.021869489f))));
  const float direct = copysignf((1.0f - e) * __builtin_amdgcn_rcpf(1.0f + e), z);
  return s < 0.0625f ? series : direct;
}
// Sine and cosine of an angle in radians, |a| up to 2^20: quarter turns from a product with 2 / pi in two
// parts, then the Taylor series on [-pi/4, pi/4].
__device__ __forceinline__ void cw_sincos_quick(float a, float& s, float& c) {
  const float hi = a * 0.636619772f, lo = fmaf(a, 0.636619772f, -hi) + a * 2.56825533e-8f;
  const float n = rintf(hi);
  const float r = ((hi - n) + lo) * 1.57079633f, q = r * r;
  const float sn = r * (1.0f + q * (-0.166666667f + q * (8.33333333e-3f + q * (-1.98412698e-4f + q * 2.75573192e-6f))));
  const float cs = 1.0f + q * (-0.5f + q * (4.16666667e-2f + q * (-1.38888889e-3f + q * 2.48015873e-5f)));
  const int k = (int)n & 3;
  const float u = k & 1 ? cs : sn, v = k & 1 ? sn : cs;
  s = k & 2 ? -u : u;
  c = (k + 1) & 2 ? -v : v;
}
__device__ __forceinline__ float cw_softplus(float z) { return z > 0.0f ? z + log1pf(expf(-z)) : log1pf(expf(z)); }
// The same from the bare exp2 and log2 instructions: max(z, 0) + ln(1 + e), e = exp(-|z|). ln(1 + e) is a
// short power series for small e, where 1 + e would lose its digits, and else ln(u) e / (u - 1) with u = 1 + e
// as rounded, which takes back what the rounding of the sum took.
__device__ __forceinline__ float cw_softplus_quick(float z) {
  const float e = __builtin_amdgcn_exp2f(-1.44269504f * fabsf(z));
  const float u = 1.0f + e;
  const float series = e * (1.0f + e * (-0.5f + e * (0.333333333f + e * (-0.25f + e * (0.2f - e * 0.166666667f)))));
  const float direct = 0.693147181f * __builtin_amdgcn_logf(u) * e * __builtin_amdgcn_rcpf(u - 1.0f);
  return fmaxf(z, 0.0f) + (e < 0.06f ? series : direct);
}

template <typename T, int V> struct CwVec;   // V neighbouring elements as float32
template <typename T> struct CwVec<T, 1> {
  static __device__ __forceinline__ void load(const T* p, float (&o)[1]) { o[0] = cw_to_float(p[0]); }
  static __device__ __forceinline__ void store(T* p, const float (&v)[1]) { p[0] = cw_from_float<T>(v[0]); }
};
template <> struct CwVec<float, 4> {
  static __device__ __forceinline__ void load(const float* p, float (&o)[4]) {
    const float4 v = *reinterpret_cast<const float4*>(p);
    o[0] = v.x; o[1] = v.y; o[2] = v.z; o[3] = v.w;
  }
  static __device__ __forceinline__ void store(float* p, const float (&v)[4]) { *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]); }
};
template <> struct CwVec<bf16_t, 4> {
  static __device__ __forceinline__ void load(const bf16_t* p, float (&o)[4]) {
    const uint2 d = *reinterpret_cast<const uint2*>(p);
    o[0] = __uint_as_float(d.x << 16); o[1] = __uint_as_float(d.x & 0xffff0000u);
    o[2] = __uint_as_float(d.y << 16); o[3] = __uint_as_float(d.y & 0xffff0000u);
  }
  static __device__ __forceinline__ void store(bf16_t* p, const float (&v)[4]) {
    *reinterpret_cast<uint2*>(p) = make_uint2((uint32_t)cw_float_to_bf16_bits(v[0]) | ((uint32_t)cw_float_to_bf16_bits(v[1]) << 16),
                                              (uint32_t)cw_float_to_bf16_bits(v[2]) | ((uint32_t)cw_float_to_bf16_bits(v[3]) << 16));
  }
};

__device__ __forceinline__ float cw_wave_sum(float v) {
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) v += __shfl_xor(v, off, 64);
  return v;
}
__device__ __forceinline__ float cw_wave_max(float v) {
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) v = fmaxf(v, __shfl_xor(v, off, 64));
  return v;
}

// A workgroup barrier for data that waves hand each other through LDS: LDS writes made before it
// are visible after it. __syncthreads() also orders global memory, and for that it waits until
// every global store the wave has issued is done; the counter it waits on counts loads as well, in
// order, so a wave that has prefetched its next tile and then stored a result waits at the barrier
// for the prefetch too, and the loop loses the overlap it was built for. Kernels whose global
// stores nobody in the workgroup reads back use this barrier in such loops.
__device__ __forceinline__ void cw_lds_barrier() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "workgroup", "local");
  __builtin_amdgcn_s_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "workgroup", "local");
}

static inline int cw_launch_status() {
  return hipGetLastError() == hipSuccess ? CW_OK : CW_ERR_LAUNCH;
}
