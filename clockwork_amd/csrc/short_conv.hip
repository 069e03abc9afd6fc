// Short causal convolutions over a request's tokens, for gfx950: of the columns of a projection
// (cw_short_conv), and of a fused query / key / value projection together with all that stands between it
// and attention (cw_qkv_conv_store).
#include "short_conv.h"

CW_EXPORT int cw_short_conv_tokens(void) { return SHORT_CONV_TOKENS; }
CW_EXPORT int cw_short_conv_max_taps(void) { return SHORT_CONV_MAX_TAPS; }

// out[t, c] = act(b[c] + sum over k of w[c, taps - 1 - k] * in[t - k, in_off + c]) for the step's tokens; items are
// runs of up to SHORT_CONV_TOKENS tokens of one request, every run but a request's last one full.
CW_EXPORT int cw_short_conv(int dtype, const void* in, int64_t in_stride, int in_off, void* out, int64_t out_stride, const float* w,
                            const float* b, int silu, float* state, int64_t state_stride, int64_t ring_off, int n_slots,
                            const int* state_slots, const int* cu_q, const int* ctx_lens, const int* items, int n_items, int channels,
                            int taps, hipStream_t stream) {
  if (!in || !out || !w || !state || !state_slots || !cu_q || !ctx_lens || !items || n_items < 0 || n_slots < 1) return CW_ERR_ARG;
  if (channels < 1 || in_off < 0 || in_off + channels > in_stride || channels > out_stride || ring_off < 0 ||
      ring_off + (int64_t)taps * channels > state_stride)
    return CW_ERR_ARG;
  const ShortConv p = {in, in_stride, in_off, out, out_stride, 0, w, b, silu, state, state_stride, ring_off,
                       n_slots, state_slots, cu_q, ctx_lens, items, channels, taps};
  return short_conv_launch(p, dtype, n_items, stream);
}

// ---------------------------------------------------------------- queries, keys and values of attention
// A row of proj holds a token's queries (nq elements), keys (nk) and values (nv) one behind the other from
// column ``off``. In this order: the convolution of every channel (no bias, no activation; taps 0: none);
// the query projection as one vector of nq elements divided by its root mean square (eps inside the root)
// and multiplied by qw, the key projection likewise with kw (qw null: no norm); the first rdims elements of
// every head of ``dim`` elements rotated by the token's position in half-split pairs (i, i + rdims / 2),
// angle = float(position) * freq[i], cosine and sine multiplied by rot_mult. Queries go to q_out[t, nq], keys
// to k_plane[slot, nk], values times v_scale to v_plane[slot, nv]; a negative slot writes no cache row.
//
// A workgroup takes an item (a run of up to ``run`` tokens of one request). A thread convolves V channels
// of all its tokens with the inputs in registers; the results wait in LDS, float32, until the norms' sums
// are there. The first item's workgroup alone reads the request's earlier inputs and leaves the
// portion's last ones, so taps - 1 <= run.
struct QkvConv {
  const void* proj;
  int64_t stride;
  int off, nq, nk, nv, dim;
  const float* w;          // [nq + nk + nv, taps]
  int taps;
  float* state;
  int64_t state_stride, ring_off;
  int n_slots;
  const int* state_slots;
  const int* cu_q;
  const int* ctx_lens;
  const int* items;
  int run;
  const float* qw;         // [nq] or null
  const float* kw;         // [nk] or null
  float eps;
  const int* positions;
  const float* freq;
  int rdims;
  float rot_mult, v_scale;
  const int* slots;
  void* q_out;
  void* k_plane;
  void* v_plane;
  int64_t cache_rows;
};

#define QKV_MAX_RUN SHORT_CONV_TOKENS
#define QKV_RUN 4   // tokens of an item in the unrolled form (at most 4 taps)

template <typename T, int V, int TAPS>
__global__ __launch_bounds__(1024) void qkv_conv_store_kernel(QkvConv p) {
  extern __shared__ __align__(16) float qkv_lds[];  // [run][nq + nk + nv], then cosines and sines [run][2][rdims / 2]
  __shared__ float inv[2 * QKV_MAX_RUN];
  __shared__ int slot_of[QKV_MAX_RUN];
  const int* item = p.items + 4 * (int64_t)blockIdx.x;
  const int req = item[0], tok0 = item[1];
  const int row0 = p.cu_q[req], q_len = p.cu_q[req + 1] - row0;
  if (tok0 >= q_len) return;  // an item past the request's tokens (a batch of fixed shape)
  const int ntok = min(min(item[2], p.run), q_len - tok0);
  const int tid = threadIdx.x, threads = blockDim.x;
  const int QK = p.nq + p.nk, C = QK + p.nv, half = p.rdims / 2;
  const int taps = TAPS ? TAPS : p.taps;
  // what the later steps need is asked for together with the rows
  const int t_angle = half ? min(tid / half, ntok - 1) : 0, e_angle = half ? tid % half : 0;
  const float pos_mine = half ? (float)p.positions[row0 + tok0 + t_angle] : 0.0f, freq_mine = half ? p.freq[e_angle] : 0.0f;
  const int slot_mine = p.slots ? p.slots[row0 + tok0 + min(tid, ntok - 1)] : -1;
  float* ring = nullptr;
  if (taps > 0) {
    const int slot = p.state_slots[req];
    if (slot >= 0 && slot < p.n_slots) ring = p.state + slot * p.state_stride + p.ring_off;
  }
  const int pos0 = p.ctx_lens[req] - q_len;
  for (int c = tid * V; c < C; c += threads * V) {
    const T* in = (const T*)p.proj + (int64_t)row0 * p.stride + p.off + c;
    auto input = [&](int i, float (&o)[V]) __attribute__((always_inline)) {
      if (i >= 0) {
        CwVec<T, V>::load(in + (int64_t)i * p.stride, o);
      } else {
        const int pos = pos0 + i;
        if (pos >= 0 && ring) {
          CwVec<float, V>::load(ring + (int64_t)(pos % taps) * C + c, o);
        } else {
#pragma unroll
          for (int v = 0; v < V; ++v) o[v] = 0.0f;
        }
      }
    };
    if constexpr (TAPS > 0) {
      float w[TAPS][V], win[TAPS][V];
#pragma unroll
      for (int v = 0; v < V; ++v)
#pragma unroll
        for (int k = 0; k < TAPS; ++k) w[k][v] = p.w[(int64_t)(c + v) * TAPS + k];
#pragma unroll
      for (int k = 0; k < TAPS - 1; ++k) input(tok0 - (TAPS - 1) + k, win[k + 1]);
      float x[QKV_RUN][V];   // the item's rows are asked for before the first is used
#pragma unroll
      for (int t = 0; t < QKV_RUN; ++t) CwVec<T, V>::load(in + (int64_t)(tok0 + min(t, ntok - 1)) * p.stride, x[t]);
#pragma unroll
      for (int t = 0; t < QKV_RUN; ++t) {
        if (t >= ntok) break;
#pragma unroll
        for (int k = 0; k < TAPS - 1; ++k)
#pragma unroll
          for (int v = 0; v < V; ++v) win[k][v] = win[k + 1][v];
        float o[V];
#pragma unroll
        for (int v = 0; v < V; ++v) {
          win[TAPS - 1][v] = x[t][v];
          o[v] = 0.0f;
#pragma unroll
          for (int k = 0; k < TAPS; ++k) o[v] += w[k][v] * win[k][v];
        }
        CwVec<float, V>::store(qkv_lds + t * C + c, o);
      }
    } else {
#pragma unroll 1
      for (int t = 0; t < ntok; ++t) {
        float o[V], u[V];
        if (taps == 0) {
          CwVec<T, V>::load(in + (int64_t)(tok0 + t) * p.stride, o);
        } else {
#pragma unroll
          for (int v = 0; v < V; ++v) o[v] = 0.0f;
          for (int k = 0; k < taps; ++k) {
            input(tok0 + t - (taps - 1) + k, u);
#pragma unroll
            for (int v = 0; v < V; ++v) o[v] += p.w[(int64_t)(c + v) * taps + k] * u[v];
          }
        }
        CwVec<float, V>::store(qkv_lds + t * C + c, o);
      }
    }
    if (tok0 == 0 && ring) {
#pragma unroll 1
      for (int i = max(0, q_len - (taps - 1)); i < q_len; ++i) {
        float u[V];
        CwVec<T, V>::load(in + (int64_t)i * p.stride, u);
        CwVec<float, V>::store(ring + (int64_t)((pos0 + i) % taps) * C + c, u);
      }
    }
  }
  if (tid < ntok) slot_of[tid] = (slot_mine >= 0 && slot_mine < p.cache_rows) ? slot_mine : -1;
  float* cosines = qkv_lds + p.run * C;
#pragma unroll 1
  for (int i = tid; i < ntok * half; i += threads) {
    const int t = i / half, e = i - t * half;
    float s, c;
    if (i == tid) cw_sincos_quick(pos_mine * freq_mine, s, c);
    else cw_sincos_quick((float)p.positions[row0 + tok0 + t] * p.freq[e], s, c);
    cosines[(2 * t) * half + e] = c * p.rot_mult;
    cosines[(2 * t + 1) * half + e] = s * p.rot_mult;
  }
  __syncthreads();
  const int wave = tid >> 6, lane = tid & 63, waves = threads >> 6;
  if (p.qw) {
    // a wave a projection of a token: the sum of its squares
    for (int u = wave; u < 2 * ntok; u += waves) {
      const int t = u >> 1, n = (u & 1) ? p.nk : p.nq;
      const float* row = qkv_lds + t * C + ((u & 1) ? p.nq : 0);
      float ss = 0.0f;
#pragma unroll 4
      for (int j = lane * V; j < n; j += 64 * V) {   // V divides both sizes
        float r[V];
        CwVec<float, V>::load(row + j, r);
#pragma unroll
        for (int v = 0; v < V; ++v) ss += r[v] * r[v];
      }
      ss = cw_wave_sum(ss);
      if (lane == 0) inv[u] = rsqrtf(ss / (float)n + p.eps);
    }
    __syncthreads();
  }
  // a thread keeps its channels for all tokens: their weights, and which elements turn together
  for (int c = tid * V; c < C; c += threads * V) {
    if (c >= QK) {
#pragma unroll 1
      for (int t = 0; t < ntok; ++t) {
        if (slot_of[t] < 0) continue;
        float o[V];
        CwVec<float, V>::load(qkv_lds + t * C + c, o);
#pragma unroll
        for (int v = 0; v < V; ++v) o[v] *= p.v_scale;
        CwVec<T, V>::store((T*)p.v_plane + (int64_t)slot_of[t] * p.nv + (c - QK), o);
      }
      continue;
    }
    const bool is_q = c < p.nq;
    const float* w = p.qw ? (is_q ? p.qw : p.kw - p.nq) : nullptr;
    const int d = (is_q ? c : c - p.nq) % p.dim;
    float wm[V], wp[V];
    int pc[V];   // the partner's channel (the element's own where nothing turns)
#pragma unroll
    for (int v = 0; v < V; ++v) {
      pc[v] = d + v < p.rdims ? (d + v < half ? c + v + half : c + v - half) : c + v;
      wm[v] = w ? w[c + v] : 1.0f;
      wp[v] = w ? w[pc[v]] : 1.0f;
    }
#pragma unroll 1
    for (int t = 0; t < ntok; ++t) {
      if (!is_q && slot_of[t] < 0) continue;
      const float* row = qkv_lds + t * C;
      const float iv = w ? inv[2 * t + (is_q ? 0 : 1)] : 1.0f;
      float o[V];
      CwVec<float, V>::load(row + c, o);
#pragma unroll
      for (int v = 0; v < V; ++v) {
        o[v] *= iv * wm[v];
        if (d + v < p.rdims) {
          const bool low = d + v < half;
          const float b = row[pc[v]] * iv * wp[v];
          const int e = low ? d + v : d + v - half;
          const float cs = cosines[(2 * t) * half + e], sn = cosines[(2 * t + 1) * half + e];
          o[v] = low ? o[v] * cs - b * sn : o[v] * cs + b * sn;
        }
      }
      if (is_q) CwVec<T, V>::store((T*)p.q_out + (int64_t)(row0 + tok0 + t) * p.nq + c, o);
      else CwVec<T, V>::store((T*)p.k_plane + (int64_t)slot_of[t] * p.nk + (c - p.nq), o);
    }
  }
}

#define QKV_LDS_MOST (150 * 1024)
static size_t qkv_lds_bytes(int run, int channels, int rdims) { return (size_t)run * (channels + rdims) * sizeof(float); }

// Tokens a work item may hold (0: beyond the kernel). Few, so that a portion fills the chip; at least taps - 1.
CW_EXPORT int cw_qkv_conv_run(int nq, int nk, int nv, int rdims, int taps) {
  if (nq < 1 || nk < 1 || nv < 1 || rdims < 0 || taps < 0 || taps > SHORT_CONV_MAX_TAPS) return 0;
  const int least = taps > 2 ? taps - 1 : 1;
  for (int run = least > QKV_RUN ? least : QKV_RUN; run >= least; --run)
    if (qkv_lds_bytes(run, nq + nk + nv, rdims) <= QKV_LDS_MOST) return run;
  return 0;
}

CW_EXPORT int cw_qkv_conv_store(int dtype, const void* proj, int64_t stride, int off, int nq, int nk, int nv, int dim, const float* w,
                                int taps, float* state, int64_t state_stride, int64_t ring_off, int n_slots, const int* state_slots,
                                const int* cu_q, const int* ctx_lens, const int* items, int n_items, const float* qw, const float* kw,
                                float eps, const int* positions, const float* freq, int rdims, float rot_mult, float v_scale,
                                const int* slots, void* q_out, void* k_plane, void* v_plane, int64_t cache_rows, hipStream_t stream) {
  if (!proj || !cu_q || !ctx_lens || !items || !q_out || n_items < 0 || off < 0 || nv < 1 || dim < 1) return CW_ERR_ARG;
  const int run = cw_qkv_conv_run(nq, nk, nv, rdims, taps);
  if (!run) return CW_ERR_SIZE;
  const int64_t C = (int64_t)nq + nk + nv;
  if (off + C > stride || nq % dim || nk % dim || rdims > dim || (rdims & 1) || (rdims && (!freq || !positions))) return CW_ERR_ARG;
  if (taps > 0 && (!w || !state || !state_slots || n_slots < 1 || ring_off < 0 || ring_off + taps * C > state_stride)) return CW_ERR_ARG;
  if ((qw == nullptr) != (kw == nullptr) || (slots && (!k_plane || !v_plane))) return CW_ERR_ARG;
  if (n_items == 0) return CW_OK;
  const QkvConv p = {proj, stride, off, nq, nk, nv, dim, w, taps, state, state_stride, ring_off, n_slots, state_slots, cu_q, ctx_lens, items,
                     run, qw, kw, eps, positions, freq, rdims, rot_mult, v_scale, slots, q_out, k_plane, v_plane, cache_rows};
  const int elem = dtype == CW_BF16 ? 2 : 4;
  const uintptr_t align = elem * 4 - 1;
  const bool v4 = !((nq | nk | nv | dim | off) & 3) && !(stride & 3) && !(((uintptr_t)proj | (uintptr_t)q_out | (uintptr_t)k_plane | (uintptr_t)v_plane) & align) &&
                  !((uintptr_t)state & 15) && !(state_stride & 3) && !(ring_off & 3);
  const size_t lds = qkv_lds_bytes(run, (int)C, rdims);
  int threads = (int)((C / (v4 ? 4 : 1) + 63) / 64 * 64);
  threads = threads < 256 ? 256 : threads > 1024 ? 1024 : threads;
#define CW_LAUNCH(T_, V_, K_)                                                                                          \
  do {                                                                                                                 \
    if (lds > 48 * 1024 && hipFuncSetAttribute((const void*)qkv_conv_store_kernel<T_, V_, K_>,                         \
                                               hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess)    \
      return CW_ERR_LAUNCH;                                                                                            \
    hipLaunchKernelGGL((qkv_conv_store_kernel<T_, V_, K_>), dim3(n_items), dim3(threads), lds, stream, p);             \
  } while (0)
#define CW_BY_TAPS(T_)                     \
  do {                                     \
    if (!v4) CW_LAUNCH(T_, 1, 0);          \
    else if (taps == 2) CW_LAUNCH(T_, 4, 2); \
    else if (taps == 3) CW_LAUNCH(T_, 4, 3); \
    else if (taps == 4) CW_LAUNCH(T_, 4, 4); \
    else CW_LAUNCH(T_, 4, 0);              \
  } while (0)
  if (dtype == CW_F32) CW_BY_TAPS(float);
  else if (dtype == CW_BF16) CW_BY_TAPS(bf16_t);
  else return CW_ERR_DTYPE;
#undef CW_BY_TAPS
#undef CW_LAUNCH
  return cw_launch_status();
}
