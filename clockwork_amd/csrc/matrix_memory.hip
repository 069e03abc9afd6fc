// A matrix memory with exponential gates and a running maximum (the recurrence of an mLSTM), for gfx950. A head
// keeps S [D, V], n [D] and m, zero at a request's start, and a token brings q, k [D], v [V] and two numbers:
//   i = cap tanh((w_i . h + b_i) / cap),   f = log logistic(cap tanh((w_f . h + b_f) / cap)),   h the mixer's input,
//   m' = max(f + m, i),   S <- e^(f + m - m') S + e^(i - m') k v^T,   n <- e^(f + m - m') n + e^(i - m') k,
//   o = S^T q / (max(|n . q|, e^(-m')) + 1e-6)   (q times q_scale).
//
// A request's slot of the state is float32 [heads][D][V], then two copies of [heads][D + 1] (n and m of a head):
// the token at position p writes copy p mod 2 and reads the other one, so that workgroups which share a
// head's columns need no order among them.
//
// Single tokens (every request of the step has one): mm_step_kernel makes gates, state and output of (a part of)
// one head's columns. Any other step cuts every request's tokens into chunks. With F the running sum of f
// in a chunk, b_t = i_t - F_t and M_t = max(m_start, b_1 .. b_t) the maximum is m_t = F_t + M_t, and
//   mm_gate_kernel         i and f of every token and head, float32 sums,
//   mm_chunk_state_kernel  what a chunk adds, sum over t of e^(b_t - max b) k_t v_t^T (and k_t), its maximum
//                          F_end + max b and its F_end,
//   mm_carry_kernel        chunk after chunk with the running maximum: the chunks' start states,
//   mm_chunk_out_kernel    o_t = [e^(m_start - M_t) q_t S_start + sum over s <= t of e^(b_s - M_t) (q_t . k_s) v_s] / (...),
//                          the same weights without v for n . q.
// No exponent is positive. The norm of the heads and the output gate follow in a kernel of their own.
//
// Products run on the matrix cores: q . k of a bfloat16 step as 16x16x32 bfloat16 instructions (exact
// products, float32 sums), all that meet a gate or the state as 16x16x4 float32 ones. Gates, maxima, state
// and outputs are float32 whatever the activation type T is.
#include "common.h"

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_t;
typedef __attribute__((ext_vector_type(4))) float f32x4_t;
typedef __attribute__((ext_vector_type(4))) unsigned int u32x4_t;

#define MM_MAX_DIM 256
#define MM_COLS 64          // value columns of a chunk kernel's workgroup
#define MM_STEP_AHEAD 8     // rows of the state a thread of the step kernel asks for at once
#define MM_EPS 1e-6f
#define MM_NONE (-3.0e38f)

struct MmParams {
  const void* proj;        // [T, stride]: q (heads * D from q_off), k (k_off), v (heads * V from v_off)
  int64_t stride;
  int q_off, k_off, v_off;
  const void* h;           // [T, width] the mixer's input
  const void* gate_w;      // [2 * heads, width]: the rows of i, then those of f
  const float* gate_b;     // [2 * heads]
  int width;
  float cap, inv_cap, q_scale;
  float* gates;            // [T, 2 * heads] i and f (not for single tokens)
  float* state;
  int64_t state_stride;
  int n_slots;
  const int* state_slots;  // [R]
  const int* cu_q;         // [R + 1]
  const int* ctx_lens;     // [R]
  const int* items;        // (request, first token, tokens, number in its request)
  const int* req_first;    // [R + 1] first chunk of each request
  float* added;            // [chunks, heads, D, V]
  float* added_n;          // [chunks, heads, D + 1]: n, then the maximum
  float* chunk_f;          // [chunks, heads]
  float* start_m;          // [chunks, heads] the maximum a chunk starts from
  float* last;             // [R, heads, D + 1] n and m behind a request's last chunk
  float* y;                // [T, heads * V]
  int heads, D, V, n_tokens;
};

// the capped logarithm of a gate: of the input gate as it is, of the forget gate through log logistic
__device__ __forceinline__ float mm_log_gate(float z, float cap, float inv_cap, bool forget) {
  const float u = cap * cw_tanh_quick(z * inv_cap);
  return forget ? -cw_softplus_quick(-u) : u;
}
__host__ __device__ inline int mm_round(int n, int to) { return (n + to - 1) / to * to; }
// n and m of a head as the token at position ``pos`` leaves them
__device__ __forceinline__ float* mm_norm_at(const MmParams& p, float* slot, int pos, int h) {
  return slot + (int64_t)p.heads * p.D * p.V + ((int64_t)(pos & 1) * p.heads + h) * (p.D + 1);
}

// ---------------------------------------------------------------- gates
// 16 tokens x 64 gate rows a workgroup, K shared among the eight waves, whose sums meet in LDS. The matrix is
// the first operand: a lane ends with 4 neighbouring gates of one token.
#define MM_GATE_WAVES 8
template <typename T>
__global__ __launch_bounds__(MM_GATE_WAVES * 64) void mm_gate_kernel(MmParams p, int vec) {
  __shared__ f32x4_t red[MM_GATE_WAVES][4][64];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, i = lane & 15, kq = lane >> 4;
  const int t0 = blockIdx.x * 16, g0 = blockIdx.y * 64, G = 2 * p.heads;
  const T* x = (const T*)p.h + (int64_t)min(t0 + i, p.n_tokens - 1) * p.width;
  f32x4_t acc[4];
  const T* w[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    acc[j] = (f32x4_t){0.0f, 0.0f, 0.0f, 0.0f};
    w[j] = (const T*)p.gate_w + (int64_t)min(g0 + j * 16 + i, G - 1) * p.width;
  }
  const int tiles = min(4, (G - g0 + 15) / 16);
  if constexpr (sizeof(T) == 2) {
#pragma unroll 3
    for (int k = wave * 32; k < p.width; k += MM_GATE_WAVES * 32) {
      const int kk = k + kq * 8;
      union { u32x4_t u; bf16x8_t v; uint16_t s[8]; } a, b[4];
      a.u = (u32x4_t){0u, 0u, 0u, 0u};
      if (vec) {
        if (kk < p.width) a.u = *reinterpret_cast<const u32x4_t*>(x + kk);
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e) if (kk + e < p.width) a.s[e] = *reinterpret_cast<const uint16_t*>(x + kk + e);
      }
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        b[j].u = (u32x4_t){0u, 0u, 0u, 0u};
        if (j >= tiles) continue;
        if (vec) {
          if (kk < p.width) b[j].u = *reinterpret_cast<const u32x4_t*>(w[j] + kk);
        } else {
#pragma unroll
          for (int e = 0; e < 8; ++e) if (kk + e < p.width) b[j].s[e] = *reinterpret_cast<const uint16_t*>(w[j] + kk + e);
        }
      }
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (j < tiles) acc[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(b[j].v, a.v, acc[j], 0, 0, 0);
    }
  } else {
    for (int k = wave * 4; k < p.width; k += MM_GATE_WAVES * 4) {
      const bool in = k + kq < p.width;
      const float a = in ? cw_to_float(x[k + kq]) : 0.0f;
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (j < tiles) acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(in ? cw_to_float(w[j][k + kq]) : 0.0f, a, acc[j], 0, 0, 0);
    }
  }
#pragma unroll
  for (int j = 0; j < 4; ++j) red[wave][j][lane] = acc[j];
  __syncthreads();
  const int j = wave;   // a wave finishes one tile
  if (j >= tiles || t0 + i >= p.n_tokens) return;
  f32x4_t sum = red[0][j][lane];
#pragma unroll
  for (int v = 1; v < MM_GATE_WAVES; ++v) sum += red[v][j][lane];
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const int g = g0 + j * 16 + kq * 4 + e;
    if (g < G) {
      const float z = sum[e] + p.gate_b[g];
      p.gates[(int64_t)(t0 + i) * G + g] = mm_log_gate(z, p.cap, p.inv_cap, g >= p.heads);
    }
  }
}

// ---------------------------------------------------------------- chunks
template <typename T> struct MmPad { static constexpr int V = sizeof(T) == 2 ? 8 : 4; };

// An operand's rows on their way to LDS: ``width`` elements, zeros past the operand's ``n`` and past the ``nt``
// tokens. LANES neighbouring threads share a row, U rows a thread make a batch. The first batches of all
// operands are asked for (``load``) before any of them is waited for (``store``, which also fetches what is
// left). Loads are never conditional: a clamped address, zeros chosen afterwards.
// ``ACROSS``: LDS holds the operand's columns side by side, each with its tokens (element e of row t at
// dst[e * dst_stride + t]), so that a lane reads four neighbouring tokens of a column at once.
template <typename T, int THREADS, int LANES, int U, bool ACROSS>
struct MmRows {
  static constexpr int V = MmPad<T>::V, ROWS = THREADS / LANES;
  u32x4_t v[U];
  __device__ __forceinline__ void load(const T* src, int64_t src_stride, int e, int t0, int n, int nt) {
    const T* at = src + min(e, n - V);
#pragma unroll
    for (int u = 0; u < U; ++u) v[u] = *reinterpret_cast<const u32x4_t*>(at + (int64_t)min(t0 + u * ROWS, nt - 1) * src_stride);
  }
  __device__ __forceinline__ void first(const T* src, int64_t src_stride, int n, int nt, bool vec) {
    if (vec) load(src, src_stride, (threadIdx.x % LANES) * V, threadIdx.x / LANES, n, nt);
  }
  __device__ __forceinline__ void put(T* dst, int dst_stride, int e, int t0, int n, int nt, int rows, int width) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int t = t0 + u * ROWS;
      if (t < rows && e < width) {
        const u32x4_t z = (t < nt && e < n) ? v[u] : (u32x4_t){0u, 0u, 0u, 0u};
        if constexpr (!ACROSS) {
          *reinterpret_cast<u32x4_t*>(dst + t * dst_stride + e) = z;
        } else {
          union { u32x4_t w; T x[V]; } parts;
          parts.w = z;
#pragma unroll
          for (int i = 0; i < V; ++i) dst[(e + i) * dst_stride + t] = parts.x[i];
        }
      }
    }
  }
  __device__ __forceinline__ void store(T* dst, int dst_stride, int width, const T* src, int64_t src_stride, int n, int nt, int rows, bool vec) {
    const int r = threadIdx.x / LANES, l = threadIdx.x % LANES;
    if (vec) {
      put(dst, dst_stride, l * V, r, n, nt, rows, width);
#pragma unroll 1
      for (int e = l * V; e < width; e += LANES * V)
#pragma unroll 1
        for (int t0 = r + (e == l * V ? U * ROWS : 0); t0 < rows; t0 += U * ROWS) {
          load(src, src_stride, e, t0, n, nt);
          put(dst, dst_stride, e, t0, n, nt, rows, width);
        }
    } else {
#pragma unroll 1
      for (int t = r; t < rows; t += ROWS)
#pragma unroll 1
        for (int e = l; e < width; e += LANES)
          dst[ACROSS ? e * dst_stride + t : t * dst_stride + e] = (t < nt && e < n) ? src[(int64_t)t * src_stride + e] : cw_from_float<T>(0.0f);
    }
  }
};

// A lane a token of the chunk (the first wave), from its i and f: F, the running sum of f, and b = i - F
// (MM_NONE past the chunk's tokens, where F stays what it was).
__device__ __forceinline__ void mm_gates(float gi, float gf, bool live, float& F, float& b) {
  const int lane = threadIdx.x;
  F = live ? gf : 0.0f;
#pragma unroll
  for (int off = 1; off < 64; off <<= 1) {
    const float o = __shfl_up(F, off, 64);
    if (lane >= off) F += o;
  }
  b = live ? gi - F : MM_NONE;
}

template <typename T, int Q>
__global__ __launch_bounds__(Q * 4) void mm_chunk_state_kernel(MmParams p, int vec) {
  extern __shared__ __align__(16) unsigned char smem[];
  __shared__ float wt[64];
  constexpr int WAVES = Q / 16, THREADS = Q * 4;
  const int* item = p.items + 4 * (int64_t)blockIdx.x;
  const int h = blockIdx.y, req = item[0], tok0 = item[1], v0 = blockIdx.z * MM_COLS;
  const int row0 = p.cu_q[req], q_len = p.cu_q[req + 1] - row0;
  if (tok0 >= q_len) return;  // a chunk past the request's tokens (a batch of fixed shape)
  const int nt = min(min(item[2], Q), q_len - tok0);
  const int D = p.D, V = min(MM_COLS, p.V - v0), Dp = mm_round(D, 16), Vp = mm_round(V, 16);
  constexpr int ST = Q + 4;
  T* Ks = (T*)smem;                // [Dp][ST]
  T* Vs = Ks + Dp * ST;            // [MM_COLS][ST]
  const T* rows = (const T*)p.proj + (int64_t)(row0 + tok0) * p.stride;
  const float* gates = p.gates + (int64_t)(row0 + tok0 + min((int)threadIdx.x, nt - 1)) * (2 * p.heads);
  const float gi = threadIdx.x < 64 ? gates[h] : 0.0f, gf = threadIdx.x < 64 ? gates[p.heads + h] : 0.0f;
  const T *k_rows = rows + p.k_off + h * D, *v_rows = rows + p.v_off + h * p.V + v0;
  MmRows<T, THREADS, 16, 4, true> ks;
  MmRows<T, THREADS, sizeof(T) == 2 ? 8 : 16, 2, true> vs;
  ks.first(k_rows, p.stride, D, nt, vec);
  vs.first(v_rows, p.stride, V, nt, vec);
  ks.store(Ks, ST, Dp, k_rows, p.stride, D, nt, Q, vec);
  vs.store(Vs, ST, Vp, v_rows, p.stride, V, nt, Q, vec);
  if (threadIdx.x < 64) {
    const int t = threadIdx.x;
    float F, b;
    mm_gates(gi, gf, t < nt, F, b);
    const float most = cw_wave_max(b);
    wt[t] = t < nt ? cw_exp_quick(b - most) : 0.0f;
    if (t == 63 && blockIdx.z == 0) {
      p.added_n[((int64_t)blockIdx.x * p.heads + h) * (D + 1) + D] = F + most;
      p.chunk_f[(int64_t)blockIdx.x * p.heads + h] = F;
    }
  }
  __syncthreads();
  if (blockIdx.z == 0) {
    float* an = p.added_n + ((int64_t)blockIdx.x * p.heads + h) * (D + 1);
    for (int d = threadIdx.x; d < D; d += THREADS) {
      float s = 0.0f;
#pragma unroll 4
      for (int t = 0; t < Q; t += 4) {   // zeros past the chunk's tokens
        float k[4];
        CwVec<T, 4>::load(Ks + d * ST + t, k);
#pragma unroll
        for (int u = 0; u < 4; ++u) s += wt[t + u] * k[u];
      }
      an[d] = s;
    }
  }
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, i = lane & 15, kq = lane >> 4;
  float* out = p.added + ((int64_t)blockIdx.x * p.heads + h) * D * p.V + v0;
  const int v_tiles = Vp / 16, k_end = mm_round(nt, 16);
  // a lane quarter takes four neighbouring tokens, one a product: which tokens meet in a product is all one
  for (int tn = wave; tn < Dp / 16; tn += WAVES) {
    f32x4_t acc[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[j] = (f32x4_t){0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll 2
    for (int k = 0; k < k_end; k += 16) {
      const int t = k + kq * 4;
      float a[4], b[4][4];
      CwVec<T, 4>::load(Ks + (tn * 16 + i) * ST + t, a);
#pragma unroll
      for (int j = 0; j < 4; ++j) CwVec<T, 4>::load(Vs + (min(j, v_tiles - 1) * 16 + i) * ST + t, b[j]);
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        a[u] *= wt[t + u];
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[u], b[j][u], acc[j], 0, 0, 0);
      }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int c = j * 16 + i;
      if (c < V) {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int d = tn * 16 + kq * 4 + e;
          if (d < D) out[(int64_t)d * p.V + c] = acc[j][e];
        }
      }
    }
  }
}

// per (request, head, 256 * N state elements): walk the request's chunks in order; what a chunk added becomes
// its start state. The last workgroup of a head takes n and the maximum, and leaves what stands behind the
// last chunk in ``last``: the slot's copies are still read by the others.
template <int N>
__global__ __launch_bounds__(256) void mm_carry_kernel(MmParams p) {
  const int r = blockIdx.x, h = blockIdx.y;
  const int slot = p.state_slots[r];
  const int q_len = p.cu_q[r + 1] - p.cu_q[r];
  if (slot < 0 || slot >= p.n_slots || q_len <= 0) return;
  const bool norm = blockIdx.z == gridDim.z - 1;
  const int64_t DV = (int64_t)p.D * p.V;
  const int64_t e = ((int64_t)blockIdx.z * 256 + threadIdx.x) * N;
  if (!norm && e >= DV) return;
  float* slot_state = p.state + slot * p.state_stride;
  const float* before = mm_norm_at(p, slot_state, p.ctx_lens[r] - q_len - 1, h);   // of position -1: copy 1, zero
  float m = before[p.D];
  const int begin = p.req_first[r];
  int end = p.req_first[r + 1];
  while (end > begin && p.items[4 * (end - 1) + 1] >= q_len) --end;   // chunks past the request's tokens (a batch of fixed shape)
  if (norm) {
    for (int d = threadIdx.x; d < mm_round(p.D + 1, 256); d += 256) {
      float n = d < p.D ? before[d] : 0.0f, mm = m;
      for (int c0 = begin; c0 < end; c0 += 16) {
        float add[16], f[16], most[16];   // sixteen chunks' loads side by side
#pragma unroll
        for (int u = 0; u < 16; ++u) {
          const int64_t ch = (int64_t)min(c0 + u, end - 1) * p.heads + h;
          add[u] = p.added_n[ch * (p.D + 1) + min(d, p.D)];
          most[u] = p.added_n[ch * (p.D + 1) + p.D];
          f[u] = p.chunk_f[ch];
        }
#pragma unroll
        for (int u = 0; u < 16; ++u) {
          if (c0 + u >= end) continue;
          const int64_t ch = (int64_t)(c0 + u) * p.heads + h;
          const float next = fmaxf(mm + f[u], most[u]);
          if (d < p.D) {
            p.added_n[ch * (p.D + 1) + d] = n;
            n = cw_exp_quick(mm + f[u] - next) * n + cw_exp_quick(most[u] - next) * add[u];
          } else if (d == p.D) {
            p.start_m[ch] = mm;
          }
          mm = next;
        }
      }
      float* last = p.last + ((int64_t)r * p.heads + h) * (p.D + 1);
      if (d < p.D) last[d] = n;
      else if (d == p.D) last[d] = mm;
    }
    return;
  }
  float* st = slot_state + h * DV + e;
  float S[N];
  CwVec<float, N>::load(st, S);
  constexpr int U = 8;   // chunks whose loads are on their way at once
  for (int c0 = begin; c0 < end; c0 += U) {
    float add[U][N], f[U], most[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int c = min(c0 + u, end - 1);
      CwVec<float, N>::load(p.added + ((int64_t)c * p.heads + h) * DV + e, add[u]);
      f[u] = p.chunk_f[(int64_t)c * p.heads + h];
      most[u] = p.added_n[((int64_t)c * p.heads + h) * (p.D + 1) + p.D];
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      if (c0 + u < end) {
        CwVec<float, N>::store(p.added + ((int64_t)(c0 + u) * p.heads + h) * DV + e, S);
        const float next = fmaxf(m + f[u], most[u]);
        const float keep = cw_exp_quick(m + f[u] - next), take = cw_exp_quick(most[u] - next);
#pragma unroll
        for (int v = 0; v < N; ++v) S[v] = keep * S[v] + take * add[u][v];
        m = next;
      }
    }
  }
  CwVec<float, N>::store(st, S);
}

// q . k of 16 tokens against 16 tokens
template <typename T>
__device__ __forceinline__ f32x4_t mm_scores(const T* q_row, const T* k_row, int NK, int kq) {
  f32x4_t acc = (f32x4_t){0.0f, 0.0f, 0.0f, 0.0f};
  if constexpr (sizeof(T) == 2) {
    for (int k = 0; k < NK; k += 32)
      acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8_t*>(q_row + k + kq * 8),
                                                    *reinterpret_cast<const bf16x8_t*>(k_row + k + kq * 8), acc, 0, 0, 0);
  } else {
#pragma unroll 4
    for (int k = 0; k < NK; k += 4) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(q_row[k + kq], k_row[k + kq], acc, 0, 0, 0);
  }
  return acc;
}

template <typename T, int Q>
__global__ __launch_bounds__(Q * 4) void mm_chunk_out_kernel(MmParams p, int vec) {
  extern __shared__ __align__(16) unsigned char smem[];
  __shared__ float Fs[64], bs[64], Ms[64], den[Q], ns[MM_MAX_DIM];
  constexpr int THREADS = Q * 4, SW = Q + 4, ST = Q + 4;
  const int* item = p.items + 4 * (int64_t)blockIdx.x;
  const int h = blockIdx.y, req = item[0], tok0 = item[1], v0 = blockIdx.z * MM_COLS;
  const int row0 = p.cu_q[req], q_len = p.cu_q[req + 1] - row0;
  if (tok0 >= q_len) return;
  const int nt = min(min(item[2], Q), q_len - tok0);
  const int D = p.D, V = min(MM_COLS, p.V - v0), NK = mm_round(D, 32), Vp = mm_round(V, 16);
  const int SK = NK + MmPad<T>::V, SS = NK + 4;
  T* Qs = (T*)smem;                         // [Q][SK]
  T* Vs = Qs + Q * SK;                      // [MM_COLS][ST]
  float* Ss = (float*)(Vs + MM_COLS * ST);  // [MM_COLS][SS]
  T* Ks = (T*)(Ss + MM_COLS * SS);          // [Q][SK], then the weights of the tokens, float32 [Q][SW]
  float* Ws = (float*)Ks;
  const T* rows = (const T*)p.proj + (int64_t)(row0 + tok0) * p.stride;
  const float* start = p.added + ((int64_t)blockIdx.x * p.heads + h) * D * p.V + v0;
  const float* start_n = p.added_n + ((int64_t)blockIdx.x * p.heads + h) * (D + 1);
  const int slot = p.state_slots[req];
  if (slot < 0 || slot >= p.n_slots) return;   // no start state was made
  const float m_start = p.start_m[(int64_t)blockIdx.x * p.heads + h];
  if (blockIdx.z == 0 && tok0 + nt == q_len) {
    // behind the request's last chunk: n and m to the slot
    float* to = mm_norm_at(p, p.state + slot * p.state_stride, p.ctx_lens[req] - 1, h);
    const float* last = p.last + ((int64_t)req * p.heads + h) * (D + 1);
    for (int d = threadIdx.x; d <= D; d += THREADS) to[d] = last[d];
  }
  const float* gates = p.gates + (int64_t)(row0 + tok0 + min((int)threadIdx.x, nt - 1)) * (2 * p.heads);
  const float gi = threadIdx.x < 64 ? gates[h] : 0.0f, gf = threadIdx.x < 64 ? gates[p.heads + h] : 0.0f;
  const T *q_rows = rows + p.q_off + h * D, *k_rows = rows + p.k_off + h * D, *v_rows = rows + p.v_off + h * p.V + v0;
  const bool vec_s = !((p.V | V) & 3);
  MmRows<T, THREADS, 16, 4, false> qs, ks;
  MmRows<T, THREADS, sizeof(T) == 2 ? 8 : 16, 2, true> vs;
  MmRows<float, THREADS, 16, 8, true> ss;
  qs.first(q_rows, p.stride, D, nt, vec);
  ks.first(k_rows, p.stride, D, nt, vec);
  vs.first(v_rows, p.stride, V, nt, vec);
  ss.first(start, p.V, V, D, vec_s);
  const float n_mine = start_n[min((int)threadIdx.x, D - 1)];
  if (threadIdx.x < NK) ns[threadIdx.x] = threadIdx.x < D ? n_mine : 0.0f;
  for (int d = threadIdx.x + THREADS; d < NK; d += THREADS) ns[d] = d < D ? start_n[d] : 0.0f;
  qs.store(Qs, SK, NK, q_rows, p.stride, D, nt, Q, vec);
  ks.store(Ks, SK, NK, k_rows, p.stride, D, nt, Q, vec);
  vs.store(Vs, ST, Vp, v_rows, p.stride, V, nt, Q, vec);
  ss.store(Ss, SS, MM_COLS, start, p.V, V, D, NK, vec_s);   // (a row of the start state is p.V floats)
  if (threadIdx.x < 64) {
    const int t = threadIdx.x;
    float F, b;
    mm_gates(gi, gf, t < nt, F, b);
    float M = fmaxf(m_start, b);
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
      const float o = __shfl_up(M, off, 64);
      if (t >= off) M = fmaxf(M, o);
    }
    Fs[t] = F;
    bs[t] = b;
    Ms[t] = M;
  }
  __syncthreads();
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, i = lane & 15, kq = lane >> 4;
  const bool live_rows = wave * 16 < nt;
  f32x4_t m[Q / 16];
#pragma unroll
  for (int j = 0; j < Q / 16; ++j) {
    m[j] = (f32x4_t){0.0f, 0.0f, 0.0f, 0.0f};
    if (j <= wave && live_rows) {
      const f32x4_t sc = mm_scores<T>(Qs + (wave * 16 + i) * SK, Ks + (j * 16 + i) * SK, NK, kq);
      const int s = j * 16 + i;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int t = wave * 16 + kq * 4 + e;
        m[j][e] = t >= s ? sc[e] * p.q_scale * cw_exp_quick(bs[s] - Ms[t]) : 0.0f;
      }
    }
  }
  __syncthreads();   // every wave has read the keys
#pragma unroll
  for (int j = 0; j < Q / 16; ++j)
#pragma unroll
    for (int e = 0; e < 4; ++e) Ws[(wave * 16 + kq * 4 + e) * SW + j * 16 + i] = m[j][e];
  __syncthreads();
  if (!live_rows) return;
  const T* qrow = Qs + (wave * 16 + i) * SK;
  const float* wrow = Ws + (wave * 16 + i) * SW;
  {
    // four lanes a token: n . q of the start and of the chunk's own tokens, and the denominator
    const int t = wave * 16 + i;
    float a = 0.0f, b = 0.0f;
#pragma unroll 4
    for (int d = kq * 4; d < NK; d += 16) {   // zeros past D
      float q[4];
      CwVec<T, 4>::load(qrow + d, q);
#pragma unroll
      for (int u = 0; u < 4; ++u) a += q[u] * ns[d + u];
    }
#pragma unroll
    for (int s = kq * 4; s < Q; s += 16) {    // zeros past the token's own group
      float w[4];
      CwVec<float, 4>::load(wrow + s, w);
      b += (w[0] + w[1]) + (w[2] + w[3]);
    }
    const float nq = cw_quad_sum(a * (p.q_scale * cw_exp_quick(m_start - Ms[t])) + b);
    if (kq == 0) den[t] = __builtin_amdgcn_rcpf(fmaxf(fabsf(nq), cw_exp_quick(-(Fs[t] + Ms[t]))) + MM_EPS);
  }
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront", "local");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront", "local");
  const int v_tiles = Vp / 16, k_end = (wave + 1) * 16;
  f32x4_t acc[4];
  int col[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    acc[j] = (f32x4_t){0.0f, 0.0f, 0.0f, 0.0f};
    col[j] = min(j, v_tiles - 1) * 16 + i;
  }
#pragma unroll 2
  for (int k = kq * 4; k < NK; k += 16) {   // (a lane quarter takes four neighbouring elements, one a product)
    float a[4], b[4][4];
    CwVec<T, 4>::load(qrow + k, a);
#pragma unroll
    for (int j = 0; j < 4; ++j) CwVec<float, 4>::load(Ss + col[j] * SS + k, b[j]);
#pragma unroll
    for (int u = 0; u < 4; ++u)
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[u], b[j][u], acc[j], 0, 0, 0);
  }
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const float g = p.q_scale * cw_exp_quick(m_start - Ms[wave * 16 + kq * 4 + e]);
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[j][e] *= g;
  }
#pragma unroll 1
  for (int k = kq * 4; k < k_end; k += 16) {
    float a[4], b[4][4];
    CwVec<float, 4>::load(wrow + k, a);
#pragma unroll
    for (int j = 0; j < 4; ++j) CwVec<T, 4>::load(Vs + col[j] * ST + k, b[j]);
#pragma unroll
    for (int u = 0; u < 4; ++u)
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[u], b[j][u], acc[j], 0, 0, 0);
  }
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const int t = wave * 16 + kq * 4 + e;
    if (t >= nt) continue;
    const float f = den[t];
    float* out = p.y + (int64_t)(row0 + tok0 + t) * (p.heads * p.V) + h * p.V + v0;
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (j * 16 + i < V) out[j * 16 + i] = acc[j][e] * f;
  }
}

// ---------------------------------------------------------------- single tokens
// A workgroup takes one request's token, one head and VW of its V columns. A thread owns N columns of every
// (256 / (VW / N))-th row of the state. Gates, n and its product with q are made by every workgroup.
template <typename T, int N>
__global__ __launch_bounds__(256) void mm_step_kernel(MmParams p, int VW, int vec) {
  __shared__ float qs[MM_MAX_DIM], ks[MM_MAX_DIM];
  __shared__ float red[256 * N];
  __shared__ float sums[3][4];
  const int r = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * VW, tid = threadIdx.x;
  const int row = p.cu_q[r];
  const int slot = p.state_slots[r];
  if (p.cu_q[r + 1] <= row || slot < 0 || slot >= p.n_slots) return;
  const int D = p.D, V = p.V, vw = min(VW, V - v0), pos = p.ctx_lens[r] - 1;
  float* slot_state = p.state + slot * p.state_stride;
  float* st = slot_state + (int64_t)h * D * V + v0;
  const int cols = VW / N, rows_at_once = 256 / cols;
  const int vc = (tid % cols) * N, d0 = tid / cols;
  const bool active = d0 < rows_at_once && vc < vw;
  // the state's rows are asked for before the gates are made
  float ahead[MM_STEP_AHEAD][N];
#pragma unroll
  for (int i = 0; i < MM_STEP_AHEAD; ++i)
    if (active && d0 + i * rows_at_once < D) CwVec<float, N>::load(st + (int64_t)(d0 + i * rows_at_once) * V + vc, ahead[i]);
  const T* in = (const T*)p.proj + (int64_t)row * p.stride;
  const float* before = mm_norm_at(p, slot_state, pos - 1, h);
  float* after = mm_norm_at(p, slot_state, pos, h);
  const float n_before = tid < D ? before[tid] : 0.0f, m = before[D];
  const T* x = (const T*)p.h + (int64_t)row * p.width;
  const T* wi = (const T*)p.gate_w + (int64_t)h * p.width;
  const T* wf = wi + (int64_t)p.heads * p.width;
  float zi = 0.0f, zf = 0.0f;
  if (vec) {
    constexpr int E = 16 / (int)sizeof(T);
    for (int k = tid * E; k < p.width; k += 256 * E) {
      const u32x4_t a = *reinterpret_cast<const u32x4_t*>(x + k);
      const u32x4_t b = *reinterpret_cast<const u32x4_t*>(wi + k);
      const u32x4_t c = *reinterpret_cast<const u32x4_t*>(wf + k);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        if constexpr (sizeof(T) == 2) {
          const float lo = __uint_as_float(a[i] << 16), hi = __uint_as_float(a[i] & 0xffff0000u);
          zi += lo * __uint_as_float(b[i] << 16) + hi * __uint_as_float(b[i] & 0xffff0000u);
          zf += lo * __uint_as_float(c[i] << 16) + hi * __uint_as_float(c[i] & 0xffff0000u);
        } else {
          zi += __uint_as_float(a[i]) * __uint_as_float(b[i]);
          zf += __uint_as_float(a[i]) * __uint_as_float(c[i]);
        }
      }
    }
  } else {
    for (int k = tid; k < p.width; k += 256) {
      const float a = cw_to_float(x[k]);
      zi += a * cw_to_float(wi[k]);
      zf += a * cw_to_float(wf[k]);
    }
  }
  float k_mine = 0.0f, q_mine = 0.0f;
  if (tid < D) {
    qs[tid] = q_mine = cw_to_float(in[p.q_off + h * D + tid]) * p.q_scale;
    ks[tid] = k_mine = cw_to_float(in[p.k_off + h * D + tid]);
  }
  zi = cw_wave_sum(zi);
  zf = cw_wave_sum(zf);
  if ((tid & 63) == 0) {
    sums[0][tid >> 6] = zi;
    sums[1][tid >> 6] = zf;
  }
  __syncthreads();
  const float gi = mm_log_gate((sums[0][0] + sums[0][1]) + (sums[0][2] + sums[0][3]) + p.gate_b[h], p.cap, p.inv_cap, false);
  const float gf = mm_log_gate((sums[1][0] + sums[1][1]) + (sums[1][2] + sums[1][3]) + p.gate_b[p.heads + h], p.cap, p.inv_cap, true);
  const float next = fmaxf(gf + m, gi), keep = cw_exp_quick(gf + m - next), take = cw_exp_quick(gi - next);
  const float n = keep * n_before + take * k_mine;
  if (blockIdx.z == 0) {
    if (tid < D) after[tid] = n;
    if (tid == 0) after[D] = next;
  }
  const float nq = cw_wave_sum(n * q_mine);
  if ((tid & 63) == 0) sums[2][tid >> 6] = nq;
  float acc[N], v[N];
#pragma unroll
  for (int u = 0; u < N; ++u) {
    acc[u] = 0.0f;
    v[u] = active ? take * cw_to_float(in[p.v_off + h * V + v0 + vc + u]) : 0.0f;
  }
  if (active) {
#pragma unroll
    for (int i = 0; i < MM_STEP_AHEAD; ++i) {
      const int d = d0 + i * rows_at_once;
      if (d < D) {
        const float kk = ks[d], qq = qs[d];
        float S[N];
#pragma unroll
        for (int u = 0; u < N; ++u) {
          S[u] = keep * ahead[i][u] + kk * v[u];
          acc[u] += qq * S[u];
        }
        CwVec<float, N>::store(st + (int64_t)d * V + vc, S);
      }
    }
#pragma unroll 4
    for (int d = d0 + MM_STEP_AHEAD * rows_at_once; d < D; d += rows_at_once) {
      float S[N];
      float* at = st + (int64_t)d * V + vc;
      CwVec<float, N>::load(at, S);
      const float kk = ks[d], qq = qs[d];
#pragma unroll
      for (int u = 0; u < N; ++u) {
        S[u] = keep * S[u] + kk * v[u];
        acc[u] += qq * S[u];
      }
      CwVec<float, N>::store(at, S);
    }
  }
#pragma unroll
  for (int u = 0; u < N; ++u) red[tid * N + u] = acc[u];
  __syncthreads();
  const float total = (sums[2][0] + sums[2][1]) + (sums[2][2] + sums[2][3]);
  const float inv = __builtin_amdgcn_rcpf(fmaxf(fabsf(total), cw_exp_quick(-next)) + MM_EPS);
  for (int c = tid; c < vw; c += 256) {
    float s = 0.0f;
    for (int q = 0; q < rows_at_once; ++q) s += red[(q * cols + c / N) * N + c % N];
    p.y[(int64_t)row * (p.heads * V) + h * V + v0 + c] = s * inv;
  }
}

// ---------------------------------------------------------------- entry points
#define MM_LDS_MOST (150 * 1024)
static size_t mm_state_lds(int elem, int Q, int D) {
  return (size_t)(mm_round(D, 16) + MM_COLS) * (Q + 4) * elem;
}
static size_t mm_out_lds(int elem, int Q, int D) {
  const int pad = elem == 2 ? 8 : 4, NK = mm_round(D, 32);
  size_t k = (size_t)Q * (NK + pad) * elem;
  if (k < (size_t)Q * (Q + 4) * 4) k = (size_t)Q * (Q + 4) * 4;
  return ((size_t)Q * (NK + pad) + (size_t)MM_COLS * (Q + 4)) * elem + (size_t)MM_COLS * (NK + 4) * 4 + k;
}

// Tokens of a chunk for keys of D elements of ``dtype`` (0: beyond the kernels).
CW_EXPORT int cw_matrix_memory_chunk(int dtype, int D) {
  const int elem = dtype == CW_BF16 ? 2 : 4;
  if (D < 1 || D > MM_MAX_DIM) return 0;
  for (int q = 64; q >= 16; q >>= 1)
    if (mm_out_lds(elem, q, D) <= MM_LDS_MOST && mm_state_lds(elem, q, D) <= MM_LDS_MOST) return q;
  return 0;
}
CW_EXPORT int64_t cw_matrix_memory_slot_floats(int heads, int D, int V) { return (int64_t)heads * D * V + 2 * (int64_t)heads * (D + 1); }
// floats: added [chunks, heads, D, V], added_n [chunks, heads, D + 1], chunk_f and start_m [chunks, heads],
// last [R, heads, D + 1], gates [T, 2 * heads]
CW_EXPORT int64_t cw_matrix_memory_workspace_floats(int n_tokens, int n_requests, int n_chunks, int heads, int D, int V) {
  return (int64_t)n_chunks * heads * ((int64_t)D * V + D + 3) + (int64_t)n_requests * heads * (D + 1) + (int64_t)n_tokens * 2 * heads;
}

static int mm_fill(MmParams& p, int dtype, const void* proj, int64_t stride, int q_off, int k_off, int v_off, const void* h,
                   const void* gate_w, const float* gate_b, int width, float cap, float q_scale, float* state, int64_t state_stride,
                   int n_slots, const int* state_slots, const int* cu_q, const int* ctx_lens, float* y, int heads, int D, int V) {
  if (!proj || !h || !gate_w || !gate_b || !state || !state_slots || !cu_q || !ctx_lens || !y) return CW_ERR_ARG;
  if (dtype != CW_F32 && dtype != CW_BF16) return CW_ERR_DTYPE;
  if (heads < 1 || V < 1 || width < 1 || n_slots < 1 || !(cap > 0.0f)) return CW_ERR_ARG;
  if (!cw_matrix_memory_chunk(dtype, D) || heads > 65535 || (V + MM_COLS - 1) / MM_COLS > 65535) return CW_ERR_SIZE;
  if (q_off < 0 || k_off < 0 || v_off < 0 || q_off + heads * D > stride || k_off + heads * D > stride || v_off + heads * V > stride) return CW_ERR_ARG;
  if (state_stride < cw_matrix_memory_slot_floats(heads, D, V)) return CW_ERR_ARG;
  p.proj = proj; p.stride = stride; p.q_off = q_off; p.k_off = k_off; p.v_off = v_off; p.h = h; p.gate_w = gate_w; p.gate_b = gate_b;
  p.width = width; p.cap = cap; p.inv_cap = 1.0f / cap; p.q_scale = q_scale; p.state = state; p.state_stride = state_stride; p.n_slots = n_slots;
  p.state_slots = state_slots; p.cu_q = cu_q; p.ctx_lens = ctx_lens; p.y = y; p.heads = heads; p.D = D; p.V = V;
  p.gates = nullptr; p.items = nullptr; p.req_first = nullptr; p.added = nullptr; p.added_n = nullptr; p.chunk_f = nullptr;
  p.start_m = nullptr; p.last = nullptr; p.n_tokens = 0;
  return CW_OK;
}
static int mm_rows16(int dtype, const void* h, const void* gate_w, int width) {
  return width % (dtype == CW_BF16 ? 8 : 4) == 0 && !(((uintptr_t)h | (uintptr_t)gate_w) & 15);
}

// One token a request. ``split``: workgroups that share a head's columns.
CW_EXPORT int cw_matrix_memory_step(int dtype, const void* proj, int64_t stride, int q_off, int k_off, int v_off, const void* h,
                                    const void* gate_w, const float* gate_b, int width, float cap, float q_scale, float* state,
                                    int64_t state_stride, int n_slots, const int* state_slots, const int* cu_q, const int* ctx_lens,
                                    float* y, int n_requests, int heads, int D, int V, int split, hipStream_t stream) {
  MmParams p;
  const int rc = mm_fill(p, dtype, proj, stride, q_off, k_off, v_off, h, gate_w, gate_b, width, cap, q_scale, state, state_stride, n_slots,
                         state_slots, cu_q, ctx_lens, y, heads, D, V);
  if (rc != CW_OK) return rc;
  if (n_requests < 0 || split < 1) return CW_ERR_ARG;
  if (n_requests == 0) return CW_OK;
  const bool v4 = V % 4 == 0 && state_stride % 4 == 0 && !((uintptr_t)state & 15);
  int VW = (V + split - 1) / split;
  if (v4) VW = mm_round(VW, 4);
  if (VW > (v4 ? 1024 : 256)) VW = v4 ? 1024 : 256;   // a row of a workgroup's columns is at most its threads'
  const dim3 grid(n_requests, heads, (V + VW - 1) / VW), block(256);
  const int vec = mm_rows16(dtype, h, gate_w, width);
#define CW_LAUNCH(T_, N_) hipLaunchKernelGGL((mm_step_kernel<T_, N_>), grid, block, 0, stream, p, VW, vec)
  if (dtype == CW_F32) { if (v4) CW_LAUNCH(float, 4); else CW_LAUNCH(float, 1); }
  else { if (v4) CW_LAUNCH(bf16_t, 4); else CW_LAUNCH(bf16_t, 1); }
#undef CW_LAUNCH
  return cw_launch_status();
}

// Portions (and single tokens beside them). items: runs of up to cw_matrix_memory_chunk tokens, a request's in
// order and together, ``req_first`` [R + 1] where they begin.
CW_EXPORT int cw_matrix_memory_chunks(int dtype, const void* proj, int64_t stride, int q_off, int k_off, int v_off, const void* h,
                                      const void* gate_w, const float* gate_b, int width, float cap, float q_scale, float* state,
                                      int64_t state_stride, int n_slots, const int* state_slots, const int* cu_q, const int* ctx_lens,
                                      float* y, const int* items, int n_chunks, const int* req_first, float* workspace, int n_requests,
                                      int n_tokens, int heads, int D, int V, hipStream_t stream) {
  MmParams p;
  const int rc = mm_fill(p, dtype, proj, stride, q_off, k_off, v_off, h, gate_w, gate_b, width, cap, q_scale, state, state_stride, n_slots,
                         state_slots, cu_q, ctx_lens, y, heads, D, V);
  if (rc != CW_OK) return rc;
  if (n_requests < 0 || n_tokens < 0 || n_chunks < 0 || !items || !req_first || !workspace) return CW_ERR_ARG;
  if (n_requests == 0 || n_tokens == 0 || n_chunks == 0) return CW_OK;
  const int elem = dtype == CW_BF16 ? 2 : 4, Q = cw_matrix_memory_chunk(dtype, D);
  p.n_tokens = n_tokens; p.items = items; p.req_first = req_first;
  p.added = workspace;
  p.added_n = p.added + (int64_t)n_chunks * heads * D * V;
  p.chunk_f = p.added_n + (int64_t)n_chunks * heads * (D + 1);
  p.start_m = p.chunk_f + (int64_t)n_chunks * heads;
  p.last = p.start_m + (int64_t)n_chunks * heads;
  p.gates = p.last + (int64_t)n_requests * heads * (D + 1);
  const int v = 16 / elem;
  const int vec = D % v == 0 && V % v == 0 && stride % v == 0 && q_off % v == 0 && k_off % v == 0 && v_off % v == 0 && !((uintptr_t)proj & 15);
  const bool n4 = ((int64_t)D * V) % 4 == 0 && state_stride % 4 == 0 && !(((uintptr_t)state | (uintptr_t)workspace) & 15);
  const size_t lds_a = mm_state_lds(elem, Q, D), lds_c = mm_out_lds(elem, Q, D);
  const dim3 gate_grid((n_tokens + 15) / 16, (2 * heads + 63) / 64), grid(n_chunks, heads, (V + MM_COLS - 1) / MM_COLS), block(Q * 4);
  // four elements a thread where there are threads enough without
  const bool n4_pays = n4 && (int64_t)n_requests * heads * D * V >= (int64_t)1024 * 1024;
  const int64_t per = n4_pays ? 1024 : 256;
  const dim3 carry_grid(n_requests, heads, (unsigned)(((int64_t)D * V + per - 1) / per) + 1);
  const int gate_vec = mm_rows16(dtype, h, gate_w, width);
#define CW_RAISE(F_, LDS_)                                                                                                               \
  if ((LDS_) > 48 * 1024 && hipFuncSetAttribute((const void*)F_, hipFuncAttributeMaxDynamicSharedMemorySize, (int)(LDS_)) != hipSuccess) \
    return CW_ERR_LAUNCH
#define CW_CHUNKS(T_, Q_)                                                                                  \
  do {                                                                                                     \
    CW_RAISE((mm_chunk_state_kernel<T_, Q_>), lds_a);                                                      \
    CW_RAISE((mm_chunk_out_kernel<T_, Q_>), lds_c);                                                        \
    hipLaunchKernelGGL((mm_gate_kernel<T_>), gate_grid, dim3(MM_GATE_WAVES * 64), 0, stream, p, gate_vec); \
    hipLaunchKernelGGL((mm_chunk_state_kernel<T_, Q_>), grid, block, lds_a, stream, p, vec);               \
    if (n4_pays) hipLaunchKernelGGL((mm_carry_kernel<4>), carry_grid, dim3(256), 0, stream, p);            \
    else hipLaunchKernelGGL((mm_carry_kernel<1>), carry_grid, dim3(256), 0, stream, p);                    \
    hipLaunchKernelGGL((mm_chunk_out_kernel<T_, Q_>), grid, block, lds_c, stream, p, vec);                 \
  } while (0)
  if (dtype == CW_F32) { if (Q == 64) CW_CHUNKS(float, 64); else if (Q == 32) CW_CHUNKS(float, 32); else CW_CHUNKS(float, 16); }
  else { if (Q == 64) CW_CHUNKS(bf16_t, 64); else if (Q == 32) CW_CHUNKS(bf16_t, 32); else CW_CHUNKS(bf16_t, 16); }
#undef CW_CHUNKS
#undef CW_RAISE
  return cw_launch_status();
}
