// A short causal convolution over a request's tokens, one filter a channel, for gfx950:
//   out_p[c] = act(bias[c] + sum over k < taps of w[c, taps - 1 - k] * in_(p - k)[c]),
// zeros before the request's first token, the bias and the activation (silu) optional; float32 inside.
//
// A request keeps its latest inputs in its slot of a state: float32 [taps][channels], the one of position p
// in row p mod taps. A token at position p reads the rows of the taps - 1 positions before it and
// writes its own row, which none of them is.
#pragma once
#include "common.h"

#define SHORT_CONV_TOKENS 16                       // tokens of a work item
#define SHORT_CONV_MAX_TAPS (SHORT_CONV_TOKENS + 1)
#define SHORT_CONV_RUN 8                           // tokens of a workgroup in the unrolled form (at least its taps - 1)

struct ShortConv {
  const void* in;          // [T, in_stride], the channels from column in_off
  int64_t in_stride;
  int in_off;
  void* out;               // [T, out_stride], the channels from column out_off
  int64_t out_stride;
  int out_off;
  const float* w;          // [channels, taps], the last column meets the token itself
  const float* b;          // [channels] or null
  int silu;
  float* state;            // slots, state_stride floats apart; the inputs begin ring_off floats into a slot
  int64_t state_stride, ring_off;
  int n_slots;
  const int* state_slots;  // [R]
  const int* cu_q;         // [R + 1]
  const int* ctx_lens;     // [R]
  const int* items;        // (request, first token, tokens, 0), runs of up to SHORT_CONV_TOKENS tokens
  int channels, taps;
};

// A thread owns V channels of an item's tokens. The workgroup of a request's first item alone reads
// the slot's inputs, and afterwards writes the portion's last taps - 1 ones there (a thread what it has
// read itself). TAPS 0: any number up to SHORT_CONV_MAX_TAPS, V = 1.
template <typename T, int V, int TAPS>
__global__ __launch_bounds__(256) void short_conv_kernel(ShortConv p) {
  const int* item = p.items + 4 * (int64_t)blockIdx.x;
  const int req = item[0];
  int tok0 = item[1];
  const int row0 = p.cu_q[req], q_len = p.cu_q[req + 1] - row0;
  if (tok0 >= q_len) return;  // an item past the request's tokens (a batch of fixed shape)
  int ntok = min(min(item[2], SHORT_CONV_TOKENS), q_len - tok0);
  if constexpr (TAPS > 0) {
    // the item's tokens in runs of SHORT_CONV_RUN, a workgroup each
    const int first = blockIdx.z * SHORT_CONV_RUN;
    if (first >= ntok) return;
    tok0 += first;
    ntok = min(ntok - first, SHORT_CONV_RUN);
  }
  const int c = (blockIdx.y * 256 + threadIdx.x) * V;
  if (c >= p.channels) return;
  const int slot = p.state_slots[req];
  const bool has_slot = slot >= 0 && slot < p.n_slots;
  float* ring = has_slot ? p.state + slot * p.state_stride + p.ring_off : nullptr;
  const int pos0 = p.ctx_lens[req] - q_len;
  const int taps = TAPS ? TAPS : p.taps;
  const T* in = (const T*)p.in + (int64_t)row0 * p.in_stride + p.in_off + c;
  T* out = (T*)p.out + (int64_t)row0 * p.out_stride + p.out_off + c;
  // the input of the request's token i of this portion (negative: before it, from the slot)
  auto input = [&](int i, float (&o)[V]) __attribute__((always_inline)) {
    if (i >= 0) {
      CwVec<T, V>::load(in + (int64_t)i * p.in_stride, o);
    } else {
      const int pos = pos0 + i;
#pragma unroll
      for (int v = 0; v < V; ++v) o[v] = (pos >= 0 && ring) ? ring[(int64_t)(pos % taps) * p.channels + c + v] : 0.0f;
    }
  };
  if constexpr (TAPS > 0) {
    float w[TAPS][V], b[V], win[TAPS][V];
#pragma unroll
    for (int v = 0; v < V; ++v) {
      b[v] = p.b ? p.b[c + v] : 0.0f;
#pragma unroll
      for (int k = 0; k < TAPS; ++k) w[k][v] = p.w[(int64_t)(c + v) * TAPS + k];
    }
#pragma unroll
    for (int k = 0; k < TAPS - 1; ++k) input(tok0 - (TAPS - 1) + k, win[k + 1]);
    // all of the item's rows are asked for before the first is used
    float x[SHORT_CONV_RUN][V];
#pragma unroll
    for (int i = 0; i < SHORT_CONV_RUN; ++i) CwVec<T, V>::load(in + (int64_t)(tok0 + min(i, ntok - 1)) * p.in_stride, x[i]);
#pragma unroll
    for (int i = 0; i < SHORT_CONV_RUN; ++i) {
      if (i >= ntok) break;
#pragma unroll
      for (int k = 0; k < TAPS - 1; ++k)
#pragma unroll
        for (int v = 0; v < V; ++v) win[k][v] = win[k + 1][v];
      float o[V];
#pragma unroll
      for (int v = 0; v < V; ++v) {
        win[TAPS - 1][v] = x[i][v];
        float s = b[v];
#pragma unroll
        for (int k = 0; k < TAPS; ++k) s += w[k][v] * win[k][v];
        o[v] = p.silu ? cw_silu(s) : s;
      }
      CwVec<T, V>::store(out + (int64_t)(tok0 + i) * p.out_stride, o);
    }
  } else {
    for (int i = 0; i < ntok; ++i) {
      float o[V];
      o[0] = p.b ? p.b[c] : 0.0f;
      for (int k = 0; k < taps; ++k) {
        float u[V];
        input(tok0 + i - (taps - 1) + k, u);
        o[0] += p.w[(int64_t)c * taps + k] * u[0];
      }
      if (p.silu) o[0] = cw_silu(o[0]);
      CwVec<T, V>::store(out + (int64_t)(tok0 + i) * p.out_stride, o);
    }
  }
  if (tok0 == 0 && ring) {
    for (int i = max(0, q_len - (taps - 1)); i < q_len; ++i) {
      float u[V];
      CwVec<T, V>::load(in + (int64_t)i * p.in_stride, u);
#pragma unroll
      for (int v = 0; v < V; ++v) ring[(int64_t)((pos0 + i) % taps) * p.channels + c + v] = u[v];
    }
  }
}

// Launches the convolution; the caller has checked that the columns and the slot's inputs exist.
static inline int short_conv_launch(const ShortConv& p, int dtype, int n_items, hipStream_t stream) {
  if (p.taps < 1 || p.taps > SHORT_CONV_MAX_TAPS) return CW_ERR_SIZE;
  if (n_items == 0) return CW_OK;
  const int elem = dtype == CW_BF16 ? 2 : 4;
  const uintptr_t align = elem * 4 - 1;
  const bool v4 = p.channels % 4 == 0 && p.in_stride % 4 == 0 && p.in_off % 4 == 0 && p.out_stride % 4 == 0 && p.out_off % 4 == 0 &&
                  !((uintptr_t)p.in & align) && !((uintptr_t)p.out & align) && p.taps >= 2 && p.taps <= 4;
  const int per = v4 ? 4 : 1;
  dim3 grid(n_items, (p.channels + 256 * per - 1) / (256 * per), v4 ? SHORT_CONV_TOKENS / SHORT_CONV_RUN : 1), block(256);
#define CW_CONV(T_, V_, K_) hipLaunchKernelGGL((short_conv_kernel<T_, V_, K_>), grid, block, 0, stream, p)
#define CW_BY_TAPS(T_)                      \
  do {                                      \
    if (!v4) CW_CONV(T_, 1, 0);             \
    else if (p.taps == 2) CW_CONV(T_, 4, 2); \
    else if (p.taps == 3) CW_CONV(T_, 4, 3); \
    else CW_CONV(T_, 4, 4);                 \
  } while (0)
  if (dtype == CW_F32) CW_BY_TAPS(float);
  else if (dtype == CW_BF16) CW_BY_TAPS(bf16_t);
  else return CW_ERR_DTYPE;
#undef CW_BY_TAPS
#undef CW_CONV
  return cw_launch_status();
}
