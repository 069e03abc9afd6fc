"""A plain, slow Tufevik: whole sequences, no cache, one function per mechanism.

Shares no code with ``clockwork_amd``: it reads config.json and the safetensors file itself and
runs on the CPU in ``dtype`` (float64 by default, so that all of an error is the engine's).

The design in this file's notation. Tokens t_p at positions p = 0, 1, ...; the stream x_p has
``width`` elements; U(x) = x / sqrt(mean(x^2) + eps); D(x; n) = tanh(n.alpha x) * n + n.b, a norm
without statistics (n.alpha one number, n and n.b of the width).

* input: x_p = embedding.scale * embed[t_p].
* a layer: x <- x + D(M(D(x; norm1)); norm1b), then x <- x + D(F(D(x; norm2)); norm2b); a layer
  without F ends after the first half.
* M "mlstm", h its input: q = W_q h / sqrt(dim), k = W_k h, v = W_v h, cut into heads; a head has two
  numbers a token, i = c tanh((W_i h + b_i) / c) and f = log(logistic(c tanh((W_f h + b_f) / c))), c =
  gate_cap. It keeps S [dim, vdim], n [dim] and m, all zero at first:
      m' = max(f + m, i),   S <- e^(f + m - m') S + e^(i - m') k v^T,   n <- e^(f + m - m') n + e^(i - m') k,
      o = S^T q / (max(|n . q|, e^(-m')) + 1e-6).
  Every head's o is U'd; side by side, times a weight, times logistic(W_g h), projected back.
* M "parallel": left_scale L(h) + right_scale R(h).
  L: grouped heads. q, k, v = W h each pass a causal convolution over positions a channel (the taps'
  last column meets the token itself, zeros before position 0, no bias); q and k are U'd as whole
  projections, times weights of that size; the first rot.dims elements of every head turn in half-split
  pairs (i, i + dims/2) by p g_i, and what turns is multiplied by 0.1 ln(factor) + 1. With f_i =
  base^(-2i/dims) and r_i = (i - lo) / (hi - lo) cut to [0, 1]: g_i = r_i f_i / factor + (1 - r_i) f_i;
  lo = floor of d(fast), at least 0, hi = ceil of d(slow), at most dims - 1, d(t) = dims ln(original /
  (2 pi t)) / (2 ln base). Scores scale * q . k, softmax over all j <= i, a head's result times
  logistic(W_g h)_head; output projection.
  R: W_in h gives x and z (``inner`` each); x <- silu(causal convolution with a bias); W_x x gives a
  step row of dt_rank, B and C of ``state``; d = softplus(W_dt step + b), one number a channel. Channel c
  keeps S_c [state], zero at first: S_cn <- exp(-exp(A_log_cn) d_c) S_cn + d_c x_c B_n, y_c = S_c . C +
  D_c x_c; times silu(z), output projection.
* F "dense": W_down (relu(W_gate h) * (W_up h)). F "moe": z = router h + bias; the ``top`` largest z (the
  lower index first among equals), weights = softmax over those; an expert is W_down (silu(W_gate h) *
  (W_up h)).
* output: D(x; final.norm) times embed (without the scale).
"""

from __future__ import annotations

import json
import math
from pathlib import Path

import torch
from safetensors.torch import load_file


# ------------------------------------------------------------------------------- small pieces
def unit_rms(y, eps):
    return y / torch.sqrt((y * y).mean(-1, keepdim=True) + eps)


def logistic(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * logistic(z)


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def tanh_norm(x, w, name):
    return torch.tanh(w[name + ".alpha"] * x) * w[name] + w[name + ".b"]


def causal_conv(u, taps, bias=None):
    """u [T, channels], taps [channels, n]: out_p = bias + sum_k taps[:, n - 1 - k] * u_(p - k)."""
    T, n = u.shape[0], taps.shape[1]
    rows = []
    for p in range(T):
        acc = torch.zeros_like(u[0]) if bias is None else bias.clone()
        for k in range(min(n, p + 1)):
            acc = acc + taps[:, n - 1 - k] * u[p - k]
        rows.append(acc)
    return torch.stack(rows)


# ------------------------------------------------------------------------------- mixer "mlstm"
def log_gates(h, w, pre, cap):
    """(i, f), [T, heads] each: the logarithms of the input and forget gates."""
    i = cap * torch.tanh((h @ w[pre + "i"].t() + w[pre + "i.b"]) / cap)
    f = -softplus(-(cap * torch.tanh((h @ w[pre + "f"].t() + w[pre + "f.b"]) / cap)))
    return i, f


def matrix_memory(q, k, v, i, f):
    """One head. q, k [T, dim], v [T, vdim], i, f [T] -> o [T, vdim]."""
    S = torch.zeros(q.shape[1], v.shape[1], dtype=q.dtype)
    n = torch.zeros(q.shape[1], dtype=q.dtype)
    m = torch.zeros((), dtype=q.dtype)
    out = []
    for p in range(q.shape[0]):
        new = torch.maximum(f[p] + m, i[p])
        keep, take = torch.exp(f[p] + m - new), torch.exp(i[p] - new)
        S = keep * S + take * k[p][:, None] * v[p][None, :]
        n = keep * n + take * k[p]
        m = new
        out.append((S.t() @ q[p]) / (torch.maximum((n @ q[p]).abs(), torch.exp(-m)) + 1e-6))
    return torch.stack(out)


def mlstm(h, w, pre, mx, eps):
    T, H, D, V = h.shape[0], int(mx["heads"]), int(mx["dim"]), int(mx["vdim"])
    q = (h @ w[pre + "q"].t()).view(T, H, D) / math.sqrt(D)
    k = (h @ w[pre + "k"].t()).view(T, H, D)
    v = (h @ w[pre + "v"].t()).view(T, H, V)
    i, f = log_gates(h, w, pre, float(mx["gate_cap"]))
    heads = [unit_rms(matrix_memory(q[:, a], k[:, a], v[:, a], i[:, a], f[:, a]), eps) for a in range(H)]
    return (torch.cat(heads, -1) * w[pre + "norm"] * logistic(h @ w[pre + "g"].t())) @ w[pre + "o"].t()


# ------------------------------------------------------------------------------- mixer "parallel", left
def rotation_frequencies(rot):
    """(frequencies [dims / 2], the factor of what turns)."""
    n, base, s = int(rot["dims"]), float(rot["base"]), rot.get("scaling")
    f = [base ** (-2.0 * i / n) for i in range(n // 2)]
    if s is None:
        return f, 1.0

    def dim(turns):
        return n * math.log(float(s["original"]) / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo, hi = max(math.floor(dim(float(s["fast"]))), 0), min(math.ceil(dim(float(s["slow"]))), n - 1)
    factor = float(s["factor"])
    out = []
    for i, x in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(x / factor * r + x * (1.0 - r))
    return out, 0.1 * math.log(factor) + 1.0


def rotate_halves(v, positions, rot):
    """v [T, heads, n]: elements i and i + dims/2 turn together; the rest stay."""
    freq, mult = rotation_frequencies(rot)
    half = int(rot["dims"]) // 2
    out = v.clone()
    for i, f in enumerate(freq):
        angle = torch.as_tensor([p * f for p in positions], dtype=v.dtype)[:, None]
        c, s = torch.cos(angle) * mult, torch.sin(angle) * mult
        out[..., i] = v[..., i] * c - v[..., i + half] * s
        out[..., i + half] = v[..., i + half] * c + v[..., i] * s
    return out


def grouped_attention(h, w, pre, m, eps):
    T, H, G, D, V = h.shape[0], int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q, k, v = (causal_conv(h @ w[pre + n].t(), w[pre + n + ".conv"]) for n in ("q", "k", "v"))
    q = unit_rms(q, eps) * w[pre + "q.norm"]
    k = unit_rms(k, eps) * w[pre + "k.norm"]
    q = rotate_halves(q.view(T, H, D), range(T), m["rot"])
    k = rotate_halves(k.view(T, G, D), range(T), m["rot"])
    v = v.view(T, G, V)
    gate = logistic(h @ w[pre + "g"].t())
    seen = torch.arange(T)[None, :] <= torch.arange(T)[:, None]
    heads = []
    for a in range(H):
        g = a // (H // G)
        s = q[:, a] @ k[:, g].t() * float(m["scale"])
        weights = torch.softmax(torch.where(seen, s, torch.full_like(s, float("-inf"))), dim=-1)
        heads.append((weights @ v[:, g]) * gate[:, a : a + 1])
    return torch.cat(heads, -1) @ w[pre + "o"].t()


# ------------------------------------------------------------------------------- mixer "parallel", right
def selective_recurrence(x, B, C, d, a_log, skip):
    """x, d [T, inner], B, C [T, state], a_log [inner, state] -> y [T, inner]."""
    S = torch.zeros_like(a_log)
    out = []
    for p in range(x.shape[0]):
        S = torch.exp(-torch.exp(a_log) * d[p][:, None]) * S + (d[p] * x[p])[:, None] * B[p][None, :]
        out.append(S @ C[p] + skip * x[p])
    return torch.stack(out)


def selective_scan(h, w, pre, m):
    inner, rank, N = int(m["inner"]), int(m["dt_rank"]), int(m["state"])
    xz = h @ w[pre + "in"].t()
    x = silu(causal_conv(xz[:, :inner], w[pre + "conv"], w[pre + "conv.b"]))
    p = x @ w[pre + "x"].t()
    d = softplus(p[:, :rank] @ w[pre + "dt"].t() + w[pre + "dt.b"])
    y = selective_recurrence(x, p[:, rank : rank + N], p[:, rank + N :], d, w[pre + "A_log"], w[pre + "D"])
    return (y * silu(xz[:, inner:])) @ w[pre + "o"].t()


def parallel(h, w, pre, m, eps):
    return (float(m["left_scale"]) * grouped_attention(h, w, pre + "left.", m["left"], eps)
            + float(m["right_scale"]) * selective_scan(h, w, pre + "right.", m["right"]))


# ------------------------------------------------------------------------------- feed-forward
def relu_feed_forward(h, w, pre):
    return (torch.clamp(h @ w[pre + "gate"].t(), min=0.0) * (h @ w[pre + "up"].t())) @ w[pre + "down"].t()


def silu_expert(h, w, pre):
    return (silu(h @ w[pre + "gate"].t()) * (h @ w[pre + "up"].t())) @ w[pre + "down"].t()


def routed_choice(h, w, pre, top):
    z = h @ w[pre + "router"].t() + w[pre + "router.b"]
    chosen = torch.sort(z, dim=-1, descending=True, stable=True).indices[:, :top]
    return chosen, torch.softmax(torch.gather(z, 1, chosen), dim=-1)


def routed_feed_forward(h, w, pre, mlp):
    chosen, weight = routed_choice(h, w, pre, int(mlp["router"]["top"]))
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, r in zip(chosen[t].tolist(), weight[t]):
            out[t] = out[t] + r * silu_expert(h[t], w, f"{pre}e{e}.")
    return out


def feed_forward(h, w, pre, mlp):
    if mlp["kind"] == "dense":
        return relu_feed_forward(h, w, pre)
    if mlp["kind"] == "moe":
        return routed_feed_forward(h, w, pre, mlp)
    raise ValueError(f"feed-forward kind {mlp['kind']!r}")


# ------------------------------------------------------------------------------- the model
def layer(x, w, i, entry, eps):
    p, m = f"l{i}.", entry["mixer"]
    h = tanh_norm(x, w, p + "norm1")
    if entry["type"] == "mlstm":
        y = mlstm(h, w, p + "mix.", m, eps)
    elif entry["type"] == "parallel":
        y = parallel(h, w, p + "mix.", m, eps)
    else:
        raise ValueError(f"layer type {entry['type']!r}")
    x = x + tanh_norm(y, w, p + "norm1b")
    if entry.get("mlp") is not None:
        x = x + tanh_norm(feed_forward(tanh_norm(x, w, p + "norm2"), w, p + "mlp.", entry["mlp"]), w, p + "norm2b")
    return x


class PlainTufevik:
    def __init__(self, model_dir, dtype=torch.float64):
        model_dir = Path(model_dir)
        self.cfg = json.loads((model_dir / "config.json").read_text())
        self.w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in load_file(str(model_dir / "model.safetensors")).items()}
        self.dtype = dtype

    def streams(self, tokens):
        """The stream after every layer, [layers, T, width]."""
        cfg, w = self.cfg, self.w
        x = w["embed"][torch.as_tensor(list(tokens), dtype=torch.long)] * float(cfg["embedding"]["scale"])
        out = []
        for i, entry in enumerate(cfg["layers"]):
            x = layer(x, w, i, entry, float(cfg["norm"]["eps"]))
            out.append(x)
        return torch.stack(out)

    def logits(self, tokens):
        return (tanh_norm(self.streams(tokens)[-1], self.w, "final.norm") @ self.w["embed"].t()).float()

    def greedy(self, prompt, n):
        tokens = list(prompt)
        for _ in range(n):
            tokens.append(int(self.logits(tokens)[-1].argmax()))
        return tokens[len(prompt):]
