// A state-space recurrence with one decay a head and token, for gfx950:
//   S_t = exp(-exp(A_log_h) d_t) S_(t-1) + d_t B_t x_t^T,   y_t = S_t^T C_t + D_h x_t,   S float32 [N, P] a head,
// d_t = softplus(step_t + dt_bias_h). B and C [groups, N] are shared by the heads of a group; x, B and C come
// out of a causal convolution a channel with a bias and silu.
//
// A request's slot of the state is float32 [heads][N][P], then [taps][channels]: the convolution's
// latest inputs, the one of position p in row p mod taps. A token at position p reads the rows of the
// taps - 1 positions before it and writes its own row, which none of them is.
//
// Single tokens (every request of the step has one): ss_step_kernel makes the convolution, the state
// update and the output of one (request, head) in one launch. Any other step:
//   short_conv_kernel      the convolution of runs of a request's tokens, 16 a work item,
//   ss_chunk_state_kernel  per (chunk of tokens, head) what the chunk adds to the state,
//                          sum over t of exp(cum_last - cum_t) d_t B_t x_t^T, and its decay exp(cum_last),
//                          cum the running sum of the logarithms of the decays,
//   ss_carry_kernel        per request chunk after chunk: the chunks' start states, from and to the slot,
//   ss_chunk_out_kernel    per (chunk, head) y = exp(cum_t) C_t S_start + sum over s <= t of
//                          (C_t . B_s) exp(cum_t - cum_s) d_s x_s + D x_t.
// gated_parts_norm_kernel follows either: y silu(z), divided part by part by its root mean square, times a weight.
//
// Products run on the matrix cores: those of two bfloat16 operands (C . B of a bfloat16 step: exact
// products, float32 sums) as 16x16x32 bfloat16 instructions, all that meet a decay, a step or the
// state as 16x16x4 float32 ones. Steps, decays, their logarithms, the state and the norm are float32
// whatever the activation type T is.
#include "common.h"
#include "short_conv.h"

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_t;
typedef __attribute__((ext_vector_type(4))) float f32x4_t;
typedef __attribute__((ext_vector_type(4))) unsigned int u32x4_t;

#define SS_MAX_TAPS SHORT_CONV_MAX_TAPS
#define SS_MAX_DIM 256          // N and P
#define SS_STEP_AHEAD 8         // rows of the state a thread of ss_step_kernel asks for at once

struct SsParams {
  const void* proj;        // [T, stride]: a token's gate z (z_off), x | B | C (c_off), steps (d_off)
  int64_t stride;
  int z_off, c_off, d_off;
  void* xbc;               // [T, channels]: x | B | C after the convolution (not for single tokens)
  const float* conv_w;     // [channels, taps], the last column meets the token itself
  const float* conv_b;     // [channels]
  const float* dt_bias;    // [heads]
  const float* a_log;      // [heads]
  const float* skip;       // [heads]
  float* state;            // slots, state_stride floats apart
  int64_t state_stride;
  int n_slots;
  const int* state_slots;  // [R]
  const int* cu_q;         // [R + 1]
  const int* ctx_lens;     // [R]
  const int* items;        // conv: (request, first token, tokens, 0); chunks: the same with the chunk's number in its request
  const int* req_first;    // [R + 1] first chunk of each request
  float* added;            // [chunks, heads, N, P]
  float* chunk_decay;      // [chunks, heads]
  float* y;                // [T, heads * P]
  int heads, groups, N, P, taps, channels;
};


// ---------------------------------------------------------------- chunks
// Rows of a chunk's operand in LDS: ``width`` elements of T, zeros past the operand's ``n`` and past
// the chunk's ``nt`` tokens. The padding (8 bfloat16 or 4 float32 elements) spreads rows over the banks.
template <typename T> struct SsPad { static constexpr int V = sizeof(T) == 2 ? 8 : 4; };
__host__ __device__ inline int ss_round(int n, int to) { return (n + to - 1) / to * to; }

template <typename T, int THREADS>
__device__ __forceinline__ void ss_stage(T* dst, int dst_stride, int width, const T* src, int64_t src_stride, int n, int nt, int rows, bool vec) {
  constexpr int V = SsPad<T>::V;
  if (vec) {  // n and width are multiples of 16 bytes
    const int per = width / V;
    for (int i = threadIdx.x; i < rows * per; i += THREADS) {
      const int t = i / per, e = (i - t * per) * V;
      u32x4_t v = (u32x4_t){0u, 0u, 0u, 0u};
      if (t < nt && e < n) v = *reinterpret_cast<const u32x4_t*>(src + (int64_t)t * src_stride + e);
      *reinterpret_cast<u32x4_t*>(dst + t * dst_stride + e) = v;
    }
  } else {
    for (int i = threadIdx.x; i < rows * width; i += THREADS) {
      const int t = i / width, e = i - t * width;
      dst[t * dst_stride + e] = (t < nt && e < n) ? src[(int64_t)t * src_stride + e] : cw_from_float<T>(0.0f);
    }
  }
}

// The chunk's steps and the running sum of its decays' logarithms, by the first wave (a lane a token).
__device__ __forceinline__ void ss_steps(const SsParams& p, float raw, bool live, int h, float* dd, float* cum, int rows) {
  const int lane = threadIdx.x;
  const float d = live ? cw_softplus(raw + p.dt_bias[h]) : 0.0f;
  float c = -expf(p.a_log[h]) * d;
#pragma unroll
  for (int off = 1; off < 64; off <<= 1) {
    const float o = __shfl_up(c, off, 64);
    if (lane >= off) c += o;
  }
  if (lane < rows) {
    dd[lane] = d;
    cum[lane] = c;
  }
}

template <typename T, int Q>
__global__ __launch_bounds__(Q * 4) void ss_chunk_state_kernel(SsParams p, int vec) {
  extern __shared__ __align__(16) unsigned char smem[];
  __shared__ float dd[Q], cum[Q], wt[Q];
  constexpr int WAVES = Q / 16, THREADS = Q * 4;
  const int* item = p.items + 4 * (int64_t)blockIdx.x;
  const int h = blockIdx.y, req = item[0], tok0 = item[1];
  const int row0 = p.cu_q[req], q_len = p.cu_q[req + 1] - row0;
  if (tok0 >= q_len) return;
  const int nt = min(min(item[2], Q), q_len - tok0);
  const int N = p.N, P = p.P, g = h / (p.heads / p.groups);
  const int Np = ss_round(N, 16), Pp = ss_round(P, 16);
  const int SB = Np + SsPad<T>::V, SX = Pp + SsPad<T>::V;
  T* Bs = (T*)smem;                // [Q][SB]
  T* Xs = Bs + Q * SB;             // [Q][SX]
  const T* xbc = (const T*)p.xbc + (int64_t)(row0 + tok0) * p.channels;
  if (threadIdx.x < 64) {
    const int t = threadIdx.x;
    const bool live = t < nt;
    const float raw = live ? cw_to_float(((const T*)p.proj)[(int64_t)(row0 + tok0 + t) * p.stride + p.d_off + h]) : 0.0f;
    ss_steps(p, raw, live, h, dd, cum, Q);
  }
  ss_stage<T, THREADS>(Bs, SB, Np, xbc + (int64_t)p.heads * P + g * N, p.channels, N, nt, Q, vec);
  ss_stage<T, THREADS>(Xs, SX, Pp, xbc + (int64_t)h * P, p.channels, P, nt, Q, vec);
  __syncthreads();
  if (threadIdx.x < Q) wt[threadIdx.x] = expf(cum[Q - 1] - cum[threadIdx.x]) * dd[threadIdx.x];
  if (threadIdx.x == 0) p.chunk_decay[(int64_t)blockIdx.x * p.heads + h] = expf(cum[Q - 1]);
  __syncthreads();
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, i = lane & 15, kq = lane >> 4;
  float* out = p.added + ((int64_t)blockIdx.x * p.heads + h) * N * P;
  const int p_tiles = Pp / 16, k_end = ss_round(nt, 4);
  for (int tn = wave; tn < Np / 16; tn += WAVES) {
    for (int tp = 0; tp < p_tiles; tp += 4) {
      f32x4_t acc[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[j] = (f32x4_t){0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll 4
      for (int k = 0; k < k_end; k += 4) {
        const int t = k + kq;
        const float a = cw_to_float(Bs[t * SB + tn * 16 + i]) * wt[t];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int col = min(tp + j, p_tiles - 1) * 16 + i;
          acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, cw_to_float(Xs[t * SX + col]), acc[j], 0, 0, 0);
        }
      }
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int c = (tp + j) * 16 + i;
        if (c < P) {
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const int n = tn * 16 + kq * 4 + e;
            if (n < N) out[(int64_t)n * P + c] = acc[j][e];
          }
        }
      }
    }
  }
}

// per (request, head, 256 * V state elements): walk the request's chunks in order; what a chunk added
// becomes its start state
template <int V>
__global__ __launch_bounds__(256) void ss_carry_kernel(SsParams p) {
  const int r = blockIdx.x, h = blockIdx.y;
  const int64_t e = ((int64_t)blockIdx.z * 256 + threadIdx.x) * V;
  const int64_t NP = (int64_t)p.N * p.P;
  const int slot = p.state_slots[r];
  const int q_len = p.cu_q[r + 1] - p.cu_q[r];
  if (e >= NP || slot < 0 || slot >= p.n_slots || q_len <= 0) return;
  float* st = p.state + slot * p.state_stride + h * NP + e;
  float S[V];
  CwVec<float, V>::load(st, S);
  const int begin = p.req_first[r];
  int end = p.req_first[r + 1];
  while (end > begin && p.items[4 * (end - 1) + 1] >= q_len) --end;   // chunks past the request's tokens (a batch of fixed shape)
  for (int c0 = begin; c0 < end; c0 += 4) {
    // four chunks' loads side by side: the chain is one multiply-add a chunk
    float add[4][V], dec[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int c = min(c0 + u, end - 1);
      CwVec<float, V>::load(p.added + ((int64_t)c * p.heads + h) * NP + e, add[u]);
      dec[u] = p.chunk_decay[(int64_t)c * p.heads + h];
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      if (c0 + u < end) {
        CwVec<float, V>::store(p.added + ((int64_t)(c0 + u) * p.heads + h) * NP + e, S);
#pragma unroll
        for (int v = 0; v < V; ++v) S[v] = dec[u] * S[v] + add[u][v];
      }
    }
  }
  CwVec<float, V>::store(st, S);
}

// C . B of 16 tokens against 16 tokens
template <typename T>
__device__ __forceinline__ f32x4_t ss_scores(const T* c_row, const T* b_row, int NK, int kq) {
  f32x4_t acc = (f32x4_t){0.0f, 0.0f, 0.0f, 0.0f};
  if constexpr (sizeof(T) == 2) {
    for (int k = 0; k < NK; k += 32)
      acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8_t*>(c_row + k + kq * 8),
                                                    *reinterpret_cast<const bf16x8_t*>(b_row + k + kq * 8), acc, 0, 0, 0);
  } else {
#pragma unroll 4
    for (int k = 0; k < NK; k += 4) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(c_row[k + kq], b_row[k + kq], acc, 0, 0, 0);
  }
  return acc;
}

// SLDS: the start state waits in LDS, else it is read where it lies.
template <typename T, int Q, bool SLDS>
__global__ __launch_bounds__(Q * 4) void ss_chunk_out_kernel(SsParams p, int vec) {
  extern __shared__ __align__(16) unsigned char smem[];
  __shared__ float dd[Q], cum[Q];
  constexpr int THREADS = Q * 4, SM = Q + 4;
  const int* item = p.items + 4 * (int64_t)blockIdx.x;
  const int h = blockIdx.y, req = item[0], tok0 = item[1];
  const int row0 = p.cu_q[req], q_len = p.cu_q[req + 1] - row0;
  if (tok0 >= q_len) return;
  const int nt = min(min(item[2], Q), q_len - tok0);
  const int N = p.N, P = p.P, g = h / (p.heads / p.groups);
  const int NK = ss_round(N, 32), Pp = ss_round(P, 16);
  const int SC = NK + SsPad<T>::V, SX = Pp + SsPad<T>::V, SS = Pp + 4;
  T* Cs = (T*)smem;                                    // [Q][SC]
  T* Xs = Cs + Q * SC;                                 // [Q][SX]
  float* Ss = (float*)(Xs + Q * SX);                   // [NK][SS] with SLDS
  T* Bs = SLDS ? (T*)(Ss + NK * SS) : (T*)Ss;          // [Q][SC], then the weights of the tokens, float32 [Q][SM]
  float* Ms = (float*)Bs;
  const T* xbc = (const T*)p.xbc + (int64_t)(row0 + tok0) * p.channels;
  const float* start = p.added + ((int64_t)blockIdx.x * p.heads + h) * N * P;
  if (threadIdx.x < 64) {
    const int t = threadIdx.x;
    const bool live = t < nt;
    const float raw = live ? cw_to_float(((const T*)p.proj)[(int64_t)(row0 + tok0 + t) * p.stride + p.d_off + h]) : 0.0f;
    ss_steps(p, raw, live, h, dd, cum, Q);
  }
  const int64_t b_col = (int64_t)p.heads * P + g * N;
  ss_stage<T, THREADS>(Cs, SC, NK, xbc + b_col + (int64_t)p.groups * N, p.channels, N, nt, Q, vec);
  ss_stage<T, THREADS>(Bs, SC, NK, xbc + b_col, p.channels, N, nt, Q, vec);
  ss_stage<T, THREADS>(Xs, SX, Pp, xbc + (int64_t)h * P, p.channels, P, nt, Q, vec);
  if constexpr (SLDS) ss_stage<float, THREADS>(Ss, SS, Pp, start, P, P, N, NK, P % 4 == 0);
  __syncthreads();
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, i = lane & 15, kq = lane >> 4;
  const bool live_rows = wave * 16 < nt;
  f32x4_t m[Q / 16];
#pragma unroll
  for (int j = 0; j < Q / 16; ++j) {
    m[j] = (f32x4_t){0.0f, 0.0f, 0.0f, 0.0f};
    if (j <= wave && live_rows) {
      const f32x4_t sc = ss_scores<T>(Cs + (wave * 16 + i) * SC, Bs + (j * 16 + i) * SC, NK, kq);
      const int s = j * 16 + i;
      const float cs = cum[s], ds = dd[s];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int t = wave * 16 + kq * 4 + e;
        m[j][e] = t >= s ? sc[e] * expf(cum[t] - cs) * ds : 0.0f;
      }
    }
  }
  __syncthreads();   // every wave has read B
#pragma unroll
  for (int j = 0; j < Q / 16; ++j)
    if (j <= wave)
#pragma unroll
      for (int e = 0; e < 4; ++e) Ms[(wave * 16 + kq * 4 + e) * SM + j * 16 + i] = m[j][e];
  __syncthreads();
  if (!live_rows) return;
  const T* crow = Cs + (wave * 16 + i) * SC;
  const float* mrow = Ms + (wave * 16 + i) * SM;
  const int p_tiles = Pp / 16, k_end = (wave + 1) * 16;
  float grow[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) grow[e] = expf(cum[wave * 16 + kq * 4 + e]);
  const float skip = p.skip[h];
  for (int tp = 0; tp < p_tiles; tp += 4) {
    f32x4_t acc[4];
    int col[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      acc[j] = (f32x4_t){0.0f, 0.0f, 0.0f, 0.0f};
      col[j] = min(tp + j, p_tiles - 1) * 16 + i;
    }
    if constexpr (SLDS) {
#pragma unroll 4
      for (int k = 0; k < NK; k += 4) {
        const float a = cw_to_float(crow[k + kq]);
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, Ss[(k + kq) * SS + col[j]], acc[j], 0, 0, 0);
      }
    } else {
      for (int k = 0; k < N; k += 4) {
        const float a = k + kq < N ? cw_to_float(crow[k + kq]) : 0.0f;
        const float* srow = start + (int64_t)min(k + kq, N - 1) * P;
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, srow[min(col[j], P - 1)], acc[j], 0, 0, 0);
      }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
      for (int e = 0; e < 4; ++e) acc[j][e] *= grow[e];
#pragma unroll 4
    for (int k = 0; k < k_end; k += 4) {
      const float a = mrow[k + kq];
#pragma unroll
      for (int j = 0; j < 4; ++j)
        acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, cw_to_float(Xs[(k + kq) * SX + col[j]]), acc[j], 0, 0, 0);
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int c = (tp + j) * 16 + i;
      if (c < P) {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int t = wave * 16 + kq * 4 + e;
          if (t < nt)
            p.y[(int64_t)(row0 + tok0 + t) * (p.heads * P) + h * P + c] = acc[j][e] + skip * cw_to_float(Xs[t * SX + c]);
        }
      }
    }
  }
}

// ---------------------------------------------------------------- single tokens
// A workgroup takes one request's token, one head and PW of its P columns. A thread owns V columns of
// every (256 / (PW / V))-th row of the state.
template <typename T, int V>
__global__ __launch_bounds__(256) void ss_step_kernel(SsParams p, int PW) {
  __shared__ float Bs[SS_MAX_DIM], Cs[SS_MAX_DIM], Xs[SS_MAX_DIM];
  __shared__ float red[256 * V];
  const int r = blockIdx.x, h = blockIdx.y, p0 = blockIdx.z * PW, tid = threadIdx.x;
  const int row = p.cu_q[r];
  const int slot = p.state_slots[r];
  if (p.cu_q[r + 1] <= row || slot < 0 || slot >= p.n_slots) return;
  const int N = p.N, P = p.P, per_group = p.heads / p.groups, g = h / per_group, taps = p.taps;
  const int pw = min(PW, P - p0);
  const int pos = p.ctx_lens[r] - 1;
  float* slot_state = p.state + slot * p.state_stride;
  float* ring = slot_state + (int64_t)p.heads * N * P;
  const T* in = (const T*)p.proj + (int64_t)row * p.stride;
  float* st = slot_state + (int64_t)h * N * P + p0;
  // the state's rows are asked for before the convolution's inputs are waited for
  const int cols = PW / V, rows_at_once = 256 / cols;
  const int pc = (tid % cols) * V, n0 = tid / cols;
  const bool active = n0 < rows_at_once && pc < pw;
  float ahead[SS_STEP_AHEAD][V];
#pragma unroll
  for (int i = 0; i < SS_STEP_AHEAD; ++i)
    if (active && n0 + i * rows_at_once < N) CwVec<float, V>::load(st + (int64_t)(n0 + i * rows_at_once) * P + pc, ahead[i]);
  const float d = cw_softplus(cw_to_float(in[p.d_off + h]) + p.dt_bias[h]);
  const float decay = expf(-expf(p.a_log[h]) * d);
  for (int e = tid; e < pw + 2 * N; e += 256) {
    // channels: this workgroup's of x, then B and C of the group
    const int c = e < pw ? h * P + p0 + e : p.heads * P + (e < pw + N ? g * N + (e - pw) : p.groups * N + g * N + (e - pw - N));
    const bool mine = e < pw || (h == g * per_group && blockIdx.z == 0);   // who leaves the channel's input in the slot
    const float now = cw_to_float(in[p.c_off + c]);
    float s = p.conv_b[c];
    const float* w = p.conv_w + (int64_t)c * taps;
#pragma unroll 4
    for (int k = 1; k < taps; ++k) {
      const float before = ring[(int64_t)((pos - k + taps) % taps) * p.channels + c];
      if (pos - k >= 0) s += w[taps - 1 - k] * before;
    }
    s += w[taps - 1] * now;
    if (mine) ring[(int64_t)(pos % taps) * p.channels + c] = now;
    // rounded as the convolution of a portion stores it
    const float o = cw_to_float(cw_from_float<T>(cw_silu(s)));
    if (e < pw) Xs[e] = o;
    else if (e < pw + N) Bs[e - pw] = o;
    else Cs[e - pw - N] = o;
  }
  __syncthreads();
  float acc[V], x[V];
#pragma unroll
  for (int v = 0; v < V; ++v) {
    acc[v] = 0.0f;
    x[v] = active ? Xs[pc + v] * d : 0.0f;
  }
  if (active) {
#pragma unroll
    for (int i = 0; i < SS_STEP_AHEAD; ++i) {
      const int n = n0 + i * rows_at_once;
      if (n < N) {
        const float b = Bs[n], cc = Cs[n];
        float S[V];
#pragma unroll
        for (int v = 0; v < V; ++v) {
          S[v] = decay * ahead[i][v] + b * x[v];
          acc[v] += cc * S[v];
        }
        CwVec<float, V>::store(st + (int64_t)n * P + pc, S);
      }
    }
#pragma unroll 4
    for (int n = n0 + SS_STEP_AHEAD * rows_at_once; n < N; n += rows_at_once) {
      float S[V];
      float* at = st + (int64_t)n * P + pc;
      CwVec<float, V>::load(at, S);
      const float b = Bs[n], cc = Cs[n];
#pragma unroll
      for (int v = 0; v < V; ++v) {
        S[v] = decay * S[v] + b * x[v];
        acc[v] += cc * S[v];
      }
      CwVec<float, V>::store(at, S);
    }
  }
#pragma unroll
  for (int v = 0; v < V; ++v) red[tid * V + v] = acc[v];
  __syncthreads();
  for (int c = tid; c < pw; c += 256) {
    float s = 0.0f;
    for (int q = 0; q < rows_at_once; ++q) s += red[(q * cols + c / V) * V + c % V];
    p.y[(int64_t)row * (p.heads * P) + h * P + p0 + c] = s + p.skip[h] * Xs[c];
  }
}

// ---------------------------------------------------------------- gate and norm
// out[t, j] = v_j / sqrt(mean over j's part of v^2 + eps) * w[j] with v = y silu(z); the row's ``n``
// elements lie in ``parts`` equal parts. Parts of up to 512 elements are a wave's, larger ones the workgroup's.
// GATE_LAST: v = y, and what is normed and weighted is multiplied by the logistic function of z.
template <typename T, int V, bool GATE_LAST>
__global__ __launch_bounds__(256) void gated_parts_norm_kernel(const float* __restrict__ y, const T* __restrict__ z,
                                                               int64_t z_stride, const float* __restrict__ w, float eps,
                                                               T* __restrict__ out, int n, int parts) {
  __shared__ float scratch[4];
  const int64_t t = blockIdx.x;
  const int part = n / parts, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const bool by_wave = part <= 512 && parts > 1;
  const int first = by_wave ? wave : 0, step = by_wave ? 4 : 1;
  const int at = (by_wave ? lane : (int)threadIdx.x) * V, stride = (by_wave ? 64 : 256) * V;
  const float* yr = y + t * n;
  const T* zr = z + t * z_stride;
  auto value = [&](int j, float (&v)[V]) __attribute__((always_inline)) {
    CwVec<float, V>::load(yr + j, v);
    if (GATE_LAST) return;
    float g[V];
    CwVec<T, V>::load(zr + j, g);
#pragma unroll
    for (int i = 0; i < V; ++i) v[i] *= cw_silu(g[i]);
  };
  for (int q = first; q < parts; q += step) {
    float ss = 0.0f;
    for (int j = q * part + at; j < (q + 1) * part; j += stride) {
      float v[V];
      value(j, v);
#pragma unroll
      for (int i = 0; i < V; ++i) ss += v[i] * v[i];
    }
    ss = cw_wave_sum(ss);
    if (!by_wave) {
      __syncthreads();
      if (lane == 0) scratch[wave] = ss;
      __syncthreads();
      ss = (scratch[0] + scratch[1]) + (scratch[2] + scratch[3]);
    }
    const float inv = 1.0f / sqrtf(ss / (float)part + eps);
    for (int j = q * part + at; j < (q + 1) * part; j += stride) {
      float v[V];
      value(j, v);
#pragma unroll
      for (int i = 0; i < V; ++i) v[i] *= inv * w[j + i];
      if (GATE_LAST) {
        float g[V];
        CwVec<T, V>::load(zr + j, g);
#pragma unroll
        for (int i = 0; i < V; ++i) v[i] *= cw_logistic(g[i]);
      }
      CwVec<T, V>::store(out + t * n + j, v);
    }
  }
}

// ---------------------------------------------------------------- entry points
static size_t ss_state_lds(int elem, int Q, int N, int P) {
  const int pad = elem == 2 ? 8 : 4;
  return (size_t)Q * (ss_round(N, 16) + pad + ss_round(P, 16) + pad) * elem;
}
static size_t ss_out_lds(int elem, int Q, int N, int P, bool slds) {
  const int pad = elem == 2 ? 8 : 4, NK = ss_round(N, 32), Pp = ss_round(P, 16);
  size_t b = (size_t)Q * (NK + pad) * elem;
  if (b < (size_t)Q * (Q + 4) * 4) b = (size_t)Q * (Q + 4) * 4;
  return (size_t)Q * (NK + pad + Pp + pad) * elem + b + (slds ? (size_t)NK * (Pp + 4) * 4 : 0);
}
#define SS_LDS_MOST (150 * 1024)

// Tokens of a chunk for a state of N x P and elements of ``dtype`` (0: the state is beyond the kernels).
CW_EXPORT int cw_state_space_chunk(int dtype, int N, int P) {
  const int elem = dtype == CW_BF16 ? 2 : 4;
  if (N < 1 || P < 1 || N > SS_MAX_DIM || P > SS_MAX_DIM) return 0;
  for (int q = 64; q >= 32; q >>= 1)
    if (ss_out_lds(elem, q, N, P, false) <= SS_LDS_MOST && ss_state_lds(elem, q, N, P) <= SS_LDS_MOST) return q;
  return 0;
}
CW_EXPORT int cw_state_space_max_taps(void) { return SS_MAX_TAPS; }
CW_EXPORT int64_t cw_state_space_slot_floats(int heads, int groups, int N, int P, int taps) {
  return (int64_t)heads * N * P + (int64_t)taps * (heads * P + 2 * groups * N);
}
// floats: added [chunks, heads, N, P], decays [chunks, heads] (rounded up to 4 each)
CW_EXPORT int64_t cw_state_space_workspace_floats(int n_chunks, int heads, int N, int P) {
  return ((int64_t)n_chunks * heads * N * P + 3) / 4 * 4 + (int64_t)n_chunks * heads;
}

static int ss_fill(SsParams& p, int dtype, const void* proj, int64_t stride, int z_off, int c_off, int d_off, const float* conv_w,
                   const float* conv_b, const float* dt_bias, const float* a_log, const float* skip, float* state,
                   int64_t state_stride, int n_slots, const int* state_slots, const int* cu_q, const int* ctx_lens, float* y,
                   int heads, int groups, int N, int P, int taps) {
  if (!proj || !conv_w || !conv_b || !dt_bias || !a_log || !skip || !state || !state_slots || !cu_q || !ctx_lens || !y) return CW_ERR_ARG;
  if (dtype != CW_F32 && dtype != CW_BF16) return CW_ERR_DTYPE;
  if (heads < 1 || groups < 1 || heads % groups || n_slots < 1) return CW_ERR_ARG;
  if (!cw_state_space_chunk(dtype, N, P) || taps < 1 || taps > SS_MAX_TAPS || heads > 65535) return CW_ERR_SIZE;
  const int channels = heads * P + 2 * groups * N;
  if (z_off < 0 || c_off < 0 || d_off < 0 || z_off + heads * P > stride || c_off + channels > stride || d_off + heads > stride) return CW_ERR_ARG;
  if (state_stride < cw_state_space_slot_floats(heads, groups, N, P, taps)) return CW_ERR_ARG;
  p.proj = proj; p.stride = stride; p.z_off = z_off; p.c_off = c_off; p.d_off = d_off; p.conv_w = conv_w; p.conv_b = conv_b;
  p.dt_bias = dt_bias; p.a_log = a_log; p.skip = skip; p.state = state; p.state_stride = state_stride; p.n_slots = n_slots;
  p.state_slots = state_slots; p.cu_q = cu_q; p.ctx_lens = ctx_lens; p.y = y; p.heads = heads; p.groups = groups; p.N = N; p.P = P;
  p.taps = taps; p.channels = channels;
  p.xbc = nullptr; p.items = nullptr; p.req_first = nullptr; p.added = nullptr; p.chunk_decay = nullptr;
  return CW_OK;
}

// One token a request. ``split``: workgroups that share a head's columns.
CW_EXPORT int cw_state_space_step(int dtype, const void* proj, int64_t stride, int z_off, int c_off, int d_off,
                                  const float* conv_w, const float* conv_b, const float* dt_bias, const float* a_log,
                                  const float* skip, float* state, int64_t state_stride, int n_slots, const int* state_slots,
                                  const int* cu_q, const int* ctx_lens, float* y, int n_requests, int heads, int groups, int N,
                                  int P, int taps, int split, hipStream_t stream) {
  SsParams p;
  const int rc = ss_fill(p, dtype, proj, stride, z_off, c_off, d_off, conv_w, conv_b, dt_bias, a_log, skip, state, state_stride,
                         n_slots, state_slots, cu_q, ctx_lens, y, heads, groups, N, P, taps);
  if (rc != CW_OK) return rc;
  if (n_requests < 0 || split < 1) return CW_ERR_ARG;
  if (n_requests == 0) return CW_OK;
  const bool v4 = P % 4 == 0 && state_stride % 4 == 0 && !((uintptr_t)state & 15);
  int PW = (P + split - 1) / split;
  if (v4) PW = ss_round(PW, 4);
  dim3 grid(n_requests, heads, (P + PW - 1) / PW), block(256);
#define CW_LAUNCH(T_, V_) hipLaunchKernelGGL((ss_step_kernel<T_, V_>), grid, block, 0, stream, p, PW)
  if (dtype == CW_F32) { if (v4) CW_LAUNCH(float, 4); else CW_LAUNCH(float, 1); }
  else { if (v4) CW_LAUNCH(bf16_t, 4); else CW_LAUNCH(bf16_t, 1); }
#undef CW_LAUNCH
  return cw_launch_status();
}

// Portions (and single tokens beside them). conv_items: runs of up to 16 tokens; chunk_items: runs of up
// to cw_state_space_chunk tokens, a request's in order and together, ``req_first`` [R + 1] where they begin.
CW_EXPORT int cw_state_space_chunks(int dtype, const void* proj, int64_t stride, int z_off, int c_off, int d_off,
                                    const float* conv_w, const float* conv_b, const float* dt_bias, const float* a_log,
                                    const float* skip, float* state, int64_t state_stride, int n_slots, const int* state_slots,
                                    const int* cu_q, const int* ctx_lens, float* y, void* xbc, const int* conv_items,
                                    int n_conv_items, const int* chunk_items, int n_chunks, const int* req_first,
                                    float* workspace, int n_requests, int heads, int groups, int N, int P, int taps,
                                    hipStream_t stream) {
  SsParams p;
  const int rc = ss_fill(p, dtype, proj, stride, z_off, c_off, d_off, conv_w, conv_b, dt_bias, a_log, skip, state, state_stride,
                         n_slots, state_slots, cu_q, ctx_lens, y, heads, groups, N, P, taps);
  if (rc != CW_OK) return rc;
  if (n_requests < 0 || n_conv_items < 0 || n_chunks < 0 || !xbc || !conv_items || !chunk_items || !req_first || !workspace) return CW_ERR_ARG;
  if (n_requests == 0 || n_chunks == 0) return CW_OK;
  const int elem = dtype == CW_BF16 ? 2 : 4, Q = cw_state_space_chunk(dtype, N, P);
  p.xbc = xbc;
  {
    const ShortConv c = {proj, stride, c_off, xbc, p.channels, 0, conv_w, conv_b, 1, state, state_stride, (int64_t)heads * N * P,
                         n_slots, state_slots, cu_q, ctx_lens, conv_items, p.channels, taps};
    const int rc2 = short_conv_launch(c, dtype, n_conv_items, stream);
    if (rc2 != CW_OK) return rc2;
  }
  p.items = chunk_items;
  p.req_first = req_first;
  p.added = workspace;
  p.chunk_decay = workspace + ((int64_t)n_chunks * heads * N * P + 3) / 4 * 4;
  const int v = 16 / elem;
  const int vec = N % v == 0 && P % v == 0 && p.channels % v == 0 && !((uintptr_t)xbc & 15);
  const size_t lds_a = ss_state_lds(elem, Q, N, P);
  // the start state goes through LDS where two workgroups still share a compute unit with it (or where one alone fits anyway)
  const size_t with_s = ss_out_lds(elem, Q, N, P, true);
  const bool slds = with_s <= 78 * 1024 || (ss_out_lds(elem, Q, N, P, false) > 78 * 1024 && with_s <= SS_LDS_MOST);
  const size_t lds_c = slds ? with_s : ss_out_lds(elem, Q, N, P, false);
  const dim3 cgrid(n_chunks, heads), cblock(Q * 4);
  const bool nv4 = ((int64_t)N * P) % 4 == 0 && state_stride % 4 == 0 && !(((uintptr_t)state | (uintptr_t)workspace) & 15);
#define CW_RAISE(F_, LDS_)                                                                                                    \
  if ((LDS_) > 48 * 1024 && hipFuncSetAttribute((const void*)F_, hipFuncAttributeMaxDynamicSharedMemorySize, (int)(LDS_)) != hipSuccess) \
    return CW_ERR_LAUNCH
#define CW_CHUNKS(T_, Q_)                                                                                                     \
  do {                                                                                                                        \
    CW_RAISE((ss_chunk_state_kernel<T_, Q_>), lds_a);                                                                         \
    hipLaunchKernelGGL((ss_chunk_state_kernel<T_, Q_>), cgrid, cblock, lds_a, stream, p, vec);                                \
    if (nv4) hipLaunchKernelGGL((ss_carry_kernel<4>), dim3(n_requests, heads, (unsigned)(((int64_t)N * P + 1023) / 1024)), dim3(256), 0, stream, p); \
    else hipLaunchKernelGGL((ss_carry_kernel<1>), dim3(n_requests, heads, (unsigned)(((int64_t)N * P + 255) / 256)), dim3(256), 0, stream, p); \
    if (slds) {                                                                                                               \
      CW_RAISE((ss_chunk_out_kernel<T_, Q_, true>), lds_c);                                                                   \
      hipLaunchKernelGGL((ss_chunk_out_kernel<T_, Q_, true>), cgrid, cblock, lds_c, stream, p, vec);                          \
    } else {                                                                                                                  \
      CW_RAISE((ss_chunk_out_kernel<T_, Q_, false>), lds_c);                                                                  \
      hipLaunchKernelGGL((ss_chunk_out_kernel<T_, Q_, false>), cgrid, cblock, lds_c, stream, p, vec);                         \
    }                                                                                                                         \
  } while (0)
  if (dtype == CW_F32) { if (Q == 64) CW_CHUNKS(float, 64); else CW_CHUNKS(float, 32); }
  else { if (Q == 64) CW_CHUNKS(bf16_t, 64); else CW_CHUNKS(bf16_t, 32); }
#undef CW_CHUNKS
#undef CW_RAISE
  return cw_launch_status();
}

CW_EXPORT int cw_gated_parts_norm(const float* y, const void* z, int dtype, int64_t z_stride, int z_off, const float* w, float eps,
                                  void* out, int T, int n, int parts, int gate_last, hipStream_t stream) {
  if (T < 0 || n < 1 || parts < 1 || n % parts || !y || !z || !w || !out || z_off < 0 || z_off + n > z_stride) return CW_ERR_ARG;
  if (T == 0) return CW_OK;
  const int elem = dtype == CW_BF16 ? 2 : 4;
  const bool v4 = (n / parts) % 4 == 0 && z_stride % 4 == 0 && z_off % 4 == 0 && !(((uintptr_t)z | (uintptr_t)out) & (elem * 4 - 1)) &&
                  !((uintptr_t)y & 15);
  dim3 grid(T), block(256);
#define CW_LAUNCH(T_, V_)                                                                                                        \
  do {                                                                                                                           \
    if (gate_last)                                                                                                               \
      hipLaunchKernelGGL((gated_parts_norm_kernel<T_, V_, true>), grid, block, 0, stream, y, (const T_*)z + z_off, z_stride, w, eps, (T_*)out, n, parts); \
    else                                                                                                                         \
      hipLaunchKernelGGL((gated_parts_norm_kernel<T_, V_, false>), grid, block, 0, stream, y, (const T_*)z + z_off, z_stride, w, eps, (T_*)out, n, parts); \
  } while (0)
  if (dtype == CW_F32) { if (v4) CW_LAUNCH(float, 4); else CW_LAUNCH(float, 1); }
  else if (dtype == CW_BF16) { if (v4) CW_LAUNCH(bf16_t, 4); else CW_LAUNCH(bf16_t, 1); }
  else return CW_ERR_DTYPE;
#undef CW_LAUNCH
  return cw_launch_status();
}
