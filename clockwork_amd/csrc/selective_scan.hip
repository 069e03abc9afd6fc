// A selective recurrence: a state a channel whose decay depends on the token, for gfx950:
//   S_t[c, n] = exp(d_t[c] A[c, n]) S_(t-1)[c, n] + d_t[c] x_t[c] B_t[n],   y_t[c] = sum_n S_t[c, n] C_t[n] + D[c] x_t[c],
//   d_t[c] = softplus(W_dt[c, :] . low_t + dt_bias[c]),   out_t[c] = y_t[c] * silu(z_t[c]) * out_scale,
// A = -exp(A_log). x comes out of a short convolution; B, C and low (``rank`` numbers) are rows of one
// projection of x.
//
// A request's slot of the state is float32 [state][inner] (a state's channels side by side), then what the
// short convolution keeps.
//
// Single tokens (every request of the step has one): ssc_step_kernel, one workgroup a (request, 64 channels).
// Any other step cuts every request's tokens into segments that are walked side by side:
//   ssc_dt_kernel      d of every token and channel, float32 (the products on the matrix cores),
//   ssc_walk_kernel 0  every segment from a zero state: what it adds to the state, and the sum of its d,
//   ssc_carry_kernel   segment after segment: start(s + 1) = exp(A sum_d(s)) start(s) + added(s),
//   ssc_walk_kernel 1  every segment again, from its start state: the outputs.
// In the walks a lane owns a channel and SS_N of its states in registers; a wave's lanes are 64 channels, and
// waves share a channel's states where there are more. B and C of the segment wait in LDS and are read by
// all lanes at one address. The sums are those of the token-by-token kernel with other parentheses.
// Decays, steps, state and outputs are float32 whatever the activation type T is.
#include "common.h"

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_t;
typedef __attribute__((ext_vector_type(4))) float f32x4_t;
typedef __attribute__((ext_vector_type(4))) unsigned int u32x4_t;

#define SSC_MAX_STATE 256
#define SSC_AHEAD 4         // tokens whose inputs a walk asks for at once
#define SSC_STEP_AHEAD 8    // state rows a wave of the step kernel asks for at once

struct SscParams {
  const void* x;           // [T, inner]
  const void* z;           // [T, z_stride] gates, from column z_off
  int64_t z_stride;
  int z_off;
  const void* p;           // [T, p_stride]: low (rank), B (N), C (N)
  int64_t p_stride;
  const void* w_dt;        // [inner, rank], type T
  const float* dt_bias;    // [inner]
  const float* a2;         // [N, inner]: -exp(A_log) log2(e), states first
  const float* skip;       // [inner]
  float* state;            // slots, state_stride floats apart
  int64_t state_stride;
  int n_slots;
  const int* state_slots;  // [R]
  const int* cu_q;         // [R + 1]
  const int* items;        // (request, first token, tokens, number in its request) of a segment
  const int* req_first;    // [R + 1] first segment of each request
  float* d;                // [T, inner]
  float* added;            // [segments, N, inner]
  float* d_sum;            // [segments, inner]
  void* out;               // [T, out_stride], the channels from column 0
  int64_t out_stride;
  float out_scale;
  int inner, N, rank, n_tokens, seg_tokens, slices;
};

__device__ __forceinline__ float ssc_exp2(float v) { return __builtin_amdgcn_exp2f(v); }

// ---------------------------------------------------------------- steps
// A wave: 16 tokens x 64 channels. The matrix is the first operand, so a lane ends with 4 neighbouring
// channels of one token.
template <typename T>
__global__ __launch_bounds__(256) void ssc_dt_kernel(SscParams p, int vec) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, i = lane & 15, kq = lane >> 4;
  const int t0 = blockIdx.x * 64 + wave * 16, c0 = blockIdx.y * 64;
  if (t0 >= p.n_tokens) return;
  const int tok = min(t0 + i, p.n_tokens - 1);
  const T* low = (const T*)p.p + (int64_t)tok * p.p_stride;
  f32x4_t acc[4];
  const T* w[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    acc[j] = (f32x4_t){0.0f, 0.0f, 0.0f, 0.0f};
    w[j] = (const T*)p.w_dt + (int64_t)min(c0 + j * 16 + i, p.inner - 1) * p.rank;
  }
  if constexpr (sizeof(T) == 2) {
#pragma unroll 2
    for (int k = 0; k < p.rank; k += 32) {
      const int kk = k + kq * 8;
      union { u32x4_t u; bf16x8_t v; uint16_t s[8]; } a, b[4];
      a.u = (u32x4_t){0u, 0u, 0u, 0u};
      if (vec) {
        if (kk < p.rank) a.u = *reinterpret_cast<const u32x4_t*>(low + kk);
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e) if (kk + e < p.rank) a.s[e] = *reinterpret_cast<const uint16_t*>(low + kk + e);
      }
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        b[j].u = (u32x4_t){0u, 0u, 0u, 0u};
        if (vec) {
          if (kk < p.rank) b[j].u = *reinterpret_cast<const u32x4_t*>(w[j] + kk);
        } else {
#pragma unroll
          for (int e = 0; e < 8; ++e) if (kk + e < p.rank) b[j].s[e] = *reinterpret_cast<const uint16_t*>(w[j] + kk + e);
        }
      }
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(b[j].v, a.v, acc[j], 0, 0, 0);
    }
  } else {
    for (int k = 0; k < p.rank; k += 4) {
      const bool in = k + kq < p.rank;
      const float a = in ? cw_to_float(low[k + kq]) : 0.0f;
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(in ? cw_to_float(w[j][k + kq]) : 0.0f, a, acc[j], 0, 0, 0);
    }
  }
  if (t0 + i >= p.n_tokens) return;
  float* out = p.d + (int64_t)(t0 + i) * p.inner;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int c = c0 + j * 16 + kq * 4 + e;
      if (c < p.inner) acc[j][e] = cw_softplus_quick(acc[j][e] + p.dt_bias[c]);
    }
    const int c = c0 + j * 16 + kq * 4;
    if (!(p.inner & 3)) {
      if (c < p.inner) *reinterpret_cast<f32x4_t*>(out + c) = acc[j];
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) if (c + e < p.inner) out[c + e] = acc[j][e];
    }
  }
}

// ---------------------------------------------------------------- walks
// Waves of a workgroup: ``slices`` share the states of 64 channels, the rest are further channels.
template <typename T, int SS_N, int MODE>
__global__ __launch_bounds__(1024) void ssc_walk_kernel(SscParams p) {
  extern __shared__ __align__(16) float ssc_lds[];   // B (and C) [seg_tokens][MODE + 1][Np], then parts [waves][AHEAD][64]
  const int* item = p.items + 4 * (int64_t)blockIdx.x;
  const int req = item[0], tok0 = item[1];
  const int row0 = p.cu_q[req], q_len = p.cu_q[req + 1] - row0;
  if (tok0 >= q_len) return;  // a segment past the request's tokens (a batch of fixed shape)
  const int nt = min(min(item[2], p.seg_tokens), q_len - tok0);
  const int slices = p.slices, Np = slices * SS_N;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, waves = blockDim.x >> 6;
  const int slice = wave % slices, group = wave / slices;
  const int c = (blockIdx.y * (waves / slices) + group) * 64 + lane;
  const bool live = c < p.inner;
  const int cc = live ? c : p.inner - 1;
  const int64_t row = row0 + tok0;
  constexpr int W = MODE + 1;
  for (int i = threadIdx.x; i < nt * W * Np; i += blockDim.x) {
    const int t = i / (W * Np), e = i - t * (W * Np), which = e / Np, n = e - which * Np;
    ssc_lds[i] = n < p.N ? cw_to_float(((const T*)p.p)[(row + t) * p.p_stride + p.rank + which * p.N + n]) : 0.0f;
  }
  float* parts = ssc_lds + p.seg_tokens * W * Np;
  float A[SS_N], S[SS_N];
  float* mine = p.added + (int64_t)blockIdx.x * p.N * p.inner;
#pragma unroll
  for (int n = 0; n < SS_N; ++n) {
    const int at = slice * SS_N + n;
    A[n] = at < p.N ? p.a2[(int64_t)at * p.inner + cc] : 0.0f;
    S[n] = (MODE == 1 && at < p.N) ? mine[(int64_t)at * p.inner + cc] : 0.0f;
  }
  const float* dr = p.d + row * p.inner + cc;
  const T* xr = (const T*)p.x + row * p.inner + cc;
  const T* zr = MODE == 1 ? (const T*)p.z + row * p.z_stride + p.z_off + cc : nullptr;
  const float skip = MODE == 1 ? p.skip[cc] : 0.0f;
  T* out = MODE == 1 ? (T*)p.out + row * p.out_stride + cc : nullptr;
  float total = 0.0f;
  __syncthreads();
  for (int t0 = 0; t0 < nt; t0 += SSC_AHEAD) {
    float d[SSC_AHEAD], x[SSC_AHEAD], y[SSC_AHEAD];
    T z[SSC_AHEAD];
#pragma unroll
    for (int u = 0; u < SSC_AHEAD; ++u) {
      const int t = min(t0 + u, nt - 1);
      d[u] = dr[(int64_t)t * p.inner];
      x[u] = cw_to_float(xr[(int64_t)t * p.inner]);
      if (MODE == 1 && slice == 0) z[u] = zr[(int64_t)t * p.z_stride];
    }
#pragma unroll
    for (int u = 0; u < SSC_AHEAD; ++u) {
      y[u] = 0.0f;
      if (t0 + u < nt) {
        const float* b = ssc_lds + (t0 + u) * W * Np + slice * SS_N;
        const float dx = d[u] * x[u];
        if (MODE == 0) total += d[u];
        float y1 = 0.0f;
#pragma unroll
        for (int n = 0; n < SS_N; ++n) {
          S[n] = ssc_exp2(d[u] * A[n]) * S[n] + dx * b[n];
          if (MODE == 1) { if (n & 1) y1 += S[n] * b[Np + n]; else y[u] += S[n] * b[Np + n]; }
        }
        y[u] += y1;
      }
    }
    if (MODE == 1) {
      if (slices > 1) {
        __syncthreads();   // the parts of the tokens before have been read
#pragma unroll
        for (int u = 0; u < SSC_AHEAD; ++u) parts[(wave * SSC_AHEAD + u) * 64 + lane] = y[u];
        __syncthreads();
        if (slice == 0) {
#pragma unroll
          for (int u = 0; u < SSC_AHEAD; ++u)
            for (int s = 1; s < slices; ++s) y[u] += parts[((wave + s) * SSC_AHEAD + u) * 64 + lane];
        }
      }
      if (slice == 0 && live) {
#pragma unroll
        for (int u = 0; u < SSC_AHEAD; ++u)
          if (t0 + u < nt)
            out[(int64_t)(t0 + u) * p.out_stride] = cw_from_float<T>((y[u] + skip * x[u]) * cw_silu(cw_to_float(z[u])) * p.out_scale);
      }
    }
  }
  if (MODE == 0 && live) {
#pragma unroll
    for (int n = 0; n < SS_N; ++n)
      if (slice * SS_N + n < p.N) mine[(int64_t)(slice * SS_N + n) * p.inner + c] = S[n];
    if (slice == 0) p.d_sum[(int64_t)blockIdx.x * p.inner + c] = total;
  }
}

// a thread a (request, channel, state): walk the request's segments in order; what a segment added becomes
// its start state
__global__ __launch_bounds__(256) void ssc_carry_kernel(SscParams p) {
  const int r = blockIdx.x, n = blockIdx.z;
  const int c = blockIdx.y * 256 + threadIdx.x;
  const int slot = p.state_slots[r];
  const int q_len = p.cu_q[r + 1] - p.cu_q[r];
  if (c >= p.inner || slot < 0 || slot >= p.n_slots || q_len <= 0) return;
  float* st = p.state + slot * p.state_stride + (int64_t)n * p.inner + c;
  const float a = p.a2[(int64_t)n * p.inner + c];
  float S = *st;
  const int begin = p.req_first[r];
  int end = p.req_first[r + 1];
  while (end > begin && p.items[4 * (end - 1) + 1] >= q_len) --end;   // segments past the request's tokens (a batch of fixed shape)
  constexpr int U = 8;   // segments whose loads are on their way at once
  for (int s0 = begin; s0 < end; s0 += U) {
    float add[U], dec[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int s = min(s0 + u, end - 1);
      add[u] = p.added[((int64_t)s * p.N + n) * p.inner + c];
      dec[u] = ssc_exp2(a * p.d_sum[(int64_t)s * p.inner + c]);
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (s0 + u < end) {
        p.added[((int64_t)(s0 + u) * p.N + n) * p.inner + c] = S;
        S = dec[u] * S + add[u];
      }
  }
  *st = S;
}

// ---------------------------------------------------------------- single tokens
// Four waves share 64 channels of one request's token: each a quarter of the step's product and every
// fourth state.
template <typename T>
__global__ __launch_bounds__(256) void ssc_step_kernel(SscParams p, int vec) {
  __shared__ float red[4][64];
  __shared__ float bc[2 * SSC_MAX_STATE];
  const int r = blockIdx.x, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int64_t row = p.cu_q[r];
  const int slot = p.state_slots[r];
  if (p.cu_q[r + 1] <= row || slot < 0 || slot >= p.n_slots) return;
  const int c = blockIdx.y * 64 + lane;
  const bool live = c < p.inner;
  const int cc = live ? c : p.inner - 1;
  float* st = p.state + slot * p.state_stride + cc;
  // the state's rows are asked for before the step's product is made
  float ahead[SSC_STEP_AHEAD], rate[SSC_STEP_AHEAD];
#pragma unroll
  for (int i = 0; i < SSC_STEP_AHEAD; ++i) {
    const int n = min(wave + 4 * i, p.N - 1);
    ahead[i] = st[(int64_t)n * p.inner];
    rate[i] = p.a2[(int64_t)n * p.inner + cc];
  }
  const float bias = p.dt_bias[cc], skip = p.skip[cc];
  const T z = ((const T*)p.z)[row * p.z_stride + p.z_off + cc];
  const T* pr = (const T*)p.p + row * p.p_stride;
  const float x = cw_to_float(((const T*)p.x)[row * p.inner + cc]);
  for (int i = threadIdx.x; i < 2 * p.N; i += 256) bc[i] = cw_to_float(pr[p.rank + i]);
  const T* w = (const T*)p.w_dt + (int64_t)cc * p.rank;
  float s = 0.0f;
  if (vec) {
    constexpr int E = 16 / (int)sizeof(T);
    for (int k = wave * E; k < p.rank; k += 4 * E) {
      const u32x4_t a = *reinterpret_cast<const u32x4_t*>(w + k);
      const u32x4_t b = *reinterpret_cast<const u32x4_t*>(pr + k);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        if constexpr (sizeof(T) == 2) {
          s += __uint_as_float(a[i] << 16) * __uint_as_float(b[i] << 16);
          s += __uint_as_float(a[i] & 0xffff0000u) * __uint_as_float(b[i] & 0xffff0000u);
        } else {
          s += __uint_as_float(a[i]) * __uint_as_float(b[i]);
        }
      }
    }
  } else {
    for (int k = wave; k < p.rank; k += 4) s += cw_to_float(w[k]) * cw_to_float(pr[k]);
  }
  red[wave][lane] = s;
  __syncthreads();
  const float d = cw_softplus_quick((red[0][lane] + red[1][lane]) + (red[2][lane] + red[3][lane]) + bias);
  const float dx = d * x;
  float acc = 0.0f;
#pragma unroll
  for (int i = 0; i < SSC_STEP_AHEAD; ++i) {
    const int n = wave + 4 * i;
    if (n < p.N) {
      const float S = ssc_exp2(d * rate[i]) * ahead[i] + dx * bc[n];
      if (live) st[(int64_t)n * p.inner] = S;
      acc += S * bc[p.N + n];
    }
  }
  for (int n = wave + 4 * SSC_STEP_AHEAD; n < p.N; n += 4) {
    const float S = ssc_exp2(d * p.a2[(int64_t)n * p.inner + cc]) * st[(int64_t)n * p.inner] + dx * bc[n];
    if (live) st[(int64_t)n * p.inner] = S;
    acc += S * bc[p.N + n];
  }
  __syncthreads();   // the product's parts have been read
  red[wave][lane] = acc;
  __syncthreads();
  if (wave == 0 && live) {
    const float y = (red[0][lane] + red[1][lane]) + (red[2][lane] + red[3][lane]) + skip * x;
    ((T*)p.out)[row * p.out_stride + c] = cw_from_float<T>(y * cw_silu(cw_to_float(z)) * p.out_scale);
  }
}

// ---------------------------------------------------------------- entry points
#define SSC_LDS_MOST (150 * 1024)
static int ssc_width(int N) { return N <= 8 ? 8 : 16; }   // states a lane holds
static size_t ssc_lds_bytes(int seg_tokens, int N, int mode) {
  const int w = ssc_width(N), slices = (N + w - 1) / w;
  const int waves = slices >= 4 ? slices : 4 / slices * slices;
  return ((size_t)seg_tokens * (mode + 1) * slices * w + (mode == 1 && slices > 1 ? (size_t)waves * SSC_AHEAD * 64 : 0)) * sizeof(float);
}

// The most tokens a segment may have with a state of N (0: beyond the kernels).
CW_EXPORT int cw_selective_scan_max_segment(int N) {
  if (N < 1 || N > SSC_MAX_STATE) return 0;
  for (int q = 64; q >= 16; q >>= 1)
    if (ssc_lds_bytes(q, N, 1) <= SSC_LDS_MOST) return q;
  return 0;
}
// floats: d [T, inner], added [segments, N, inner], d_sum [segments, inner]
CW_EXPORT int64_t cw_selective_scan_workspace_floats(int n_tokens, int n_segments, int inner, int N) {
  return ((int64_t)n_tokens + (int64_t)n_segments * (N + 1)) * inner;
}

static int ssc_fill(SscParams& s, int dtype, const void* x, const void* z, int64_t z_stride, int z_off, const void* p, int64_t p_stride,
                    const void* w_dt, const float* dt_bias, const float* a2, const float* skip, float* state, int64_t state_stride,
                    int n_slots, const int* state_slots, const int* cu_q, void* out, int64_t out_stride, float out_scale, int inner,
                    int N, int rank) {
  if (!x || !z || !p || !w_dt || !dt_bias || !a2 || !skip || !state || !state_slots || !cu_q || !out) return CW_ERR_ARG;
  if (dtype != CW_F32 && dtype != CW_BF16) return CW_ERR_DTYPE;
  if (inner < 1 || rank < 1 || n_slots < 1 || z_off < 0 || z_off + inner > z_stride || rank + 2 * N > p_stride || inner > out_stride ||
      state_stride < (int64_t)N * inner)
    return CW_ERR_ARG;
  if (!cw_selective_scan_max_segment(N) || (inner + 63) / 64 > 65535) return CW_ERR_SIZE;
  s.x = x; s.z = z; s.z_stride = z_stride; s.z_off = z_off; s.p = p; s.p_stride = p_stride; s.w_dt = w_dt; s.dt_bias = dt_bias;
  s.a2 = a2; s.skip = skip; s.state = state; s.state_stride = state_stride; s.n_slots = n_slots; s.state_slots = state_slots;
  s.cu_q = cu_q; s.out = out; s.out_stride = out_stride; s.out_scale = out_scale; s.inner = inner; s.N = N; s.rank = rank;
  s.items = nullptr; s.req_first = nullptr; s.d = nullptr; s.added = nullptr; s.d_sum = nullptr; s.n_tokens = 0; s.seg_tokens = 0; s.slices = 1;
  return CW_OK;
}
static int ssc_vec(int dtype, const void* p, int64_t p_stride, const void* w_dt, int rank) {
  const int e = dtype == CW_BF16 ? 8 : 4;
  return rank % e == 0 && p_stride % e == 0 && !(((uintptr_t)p | (uintptr_t)w_dt) & 15);
}

// One token a request.
CW_EXPORT int cw_selective_scan_step(int dtype, const void* x, const void* z, int64_t z_stride, int z_off, const void* p, int64_t p_stride,
                                     const void* w_dt, const float* dt_bias, const float* a2, const float* skip, float* state,
                                     int64_t state_stride, int n_slots, const int* state_slots, const int* cu_q, void* out,
                                     int64_t out_stride, float out_scale, int n_requests, int inner, int N, int rank, hipStream_t stream) {
  SscParams s;
  const int rc = ssc_fill(s, dtype, x, z, z_stride, z_off, p, p_stride, w_dt, dt_bias, a2, skip, state, state_stride, n_slots, state_slots,
                          cu_q, out, out_stride, out_scale, inner, N, rank);
  if (rc != CW_OK) return rc;
  if (n_requests < 0) return CW_ERR_ARG;
  if (n_requests == 0) return CW_OK;
  const int vec = ssc_vec(dtype, p, p_stride, w_dt, rank);
  dim3 grid(n_requests, (inner + 63) / 64), block(256);
  if (dtype == CW_F32) hipLaunchKernelGGL(ssc_step_kernel<float>, grid, block, 0, stream, s, vec);
  else hipLaunchKernelGGL(ssc_step_kernel<bf16_t>, grid, block, 0, stream, s, vec);
  return cw_launch_status();
}

// Portions (and single tokens beside them). items: segments of up to ``seg_tokens`` tokens, a request's in order
// and together, ``req_first`` [R + 1] where they begin.
CW_EXPORT int cw_selective_scan_segments(int dtype, const void* x, const void* z, int64_t z_stride, int z_off, const void* p,
                                         int64_t p_stride, const void* w_dt, const float* dt_bias, const float* a2, const float* skip,
                                         float* state, int64_t state_stride, int n_slots, const int* state_slots, const int* cu_q,
                                         void* out, int64_t out_stride, float out_scale, const int* items, int n_segments,
                                         int seg_tokens, const int* req_first, float* workspace, int n_requests, int n_tokens, int inner,
                                         int N, int rank, hipStream_t stream) {
  SscParams s;
  const int rc = ssc_fill(s, dtype, x, z, z_stride, z_off, p, p_stride, w_dt, dt_bias, a2, skip, state, state_stride, n_slots, state_slots,
                          cu_q, out, out_stride, out_scale, inner, N, rank);
  if (rc != CW_OK) return rc;
  if (n_requests < 0 || n_tokens < 0 || n_segments < 0 || !items || !req_first || !workspace) return CW_ERR_ARG;
  if (seg_tokens < 1 || seg_tokens > cw_selective_scan_max_segment(N)) return CW_ERR_SIZE;
  if (n_requests == 0 || n_tokens == 0 || n_segments == 0) return CW_OK;
  const int w = ssc_width(N);
  s.items = items; s.req_first = req_first; s.n_tokens = n_tokens; s.seg_tokens = seg_tokens; s.slices = (N + w - 1) / w;
  s.d = workspace;
  s.added = s.d + (int64_t)n_tokens * inner;
  s.d_sum = s.added + (int64_t)n_segments * N * inner;
  const int vec = ssc_vec(dtype, p, p_stride, w_dt, rank);
  const int groups = s.slices >= 4 ? 1 : 4 / s.slices, waves = groups * s.slices;
  const dim3 dt_grid((n_tokens + 63) / 64, (inner + 63) / 64), walk_grid(n_segments, (inner + groups * 64 - 1) / (groups * 64)), walk_block(waves * 64);
  const dim3 carry_grid(n_requests, (inner + 255) / 256, N);
  const size_t lds0 = ssc_lds_bytes(seg_tokens, N, 0), lds1 = ssc_lds_bytes(seg_tokens, N, 1);
#define CW_RAISE(F_, LDS_)                                                                                                    \
  if ((LDS_) > 48 * 1024 && hipFuncSetAttribute((const void*)F_, hipFuncAttributeMaxDynamicSharedMemorySize, (int)(LDS_)) != hipSuccess) \
    return CW_ERR_LAUNCH
#define CW_WALKS(T_, W_)                                                                              \
  do {                                                                                                \
    CW_RAISE((ssc_walk_kernel<T_, W_, 0>), lds0);                                                     \
    CW_RAISE((ssc_walk_kernel<T_, W_, 1>), lds1);                                                     \
    hipLaunchKernelGGL((ssc_dt_kernel<T_>), dt_grid, dim3(256), 0, stream, s, vec);                   \
    hipLaunchKernelGGL((ssc_walk_kernel<T_, W_, 0>), walk_grid, walk_block, lds0, stream, s);         \
    hipLaunchKernelGGL(ssc_carry_kernel, carry_grid, dim3(256), 0, stream, s);                        \
    hipLaunchKernelGGL((ssc_walk_kernel<T_, W_, 1>), walk_grid, walk_block, lds1, stream, s);         \
  } while (0)
  if (dtype == CW_F32) { if (w == 8) CW_WALKS(float, 8); else CW_WALKS(float, 16); }
  else { if (w == 8) CW_WALKS(bf16_t, 8); else CW_WALKS(bf16_t, 16); }
#undef CW_WALKS
#undef CW_RAISE
  return cw_launch_status();
}
