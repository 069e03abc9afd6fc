"""State-space mixers: one with one decay a head and token (``StateSpaceSpec``), here first, and a selective
scan whose decay depends on channel, state and token (``SelectiveScanSpec``).

One product makes the gate, x, B, C and the step inputs of every token. A step of single tokens: one
kernel a (request, head) makes the convolution from the request's latest inputs, the state update
and the output. Any other step: the convolution of runs of a request's tokens, then chunks of tokens
side by side (what each adds to the state, the start states carried from chunk to chunk, each
chunk's outputs from its start state and from one another), products on the matrix cores. Then one
kernel for gate and norm, and the output product. A request's slot is float32
[heads * state_dim * head_dim + taps * channels]: the matrices, then the convolution's latest inputs
by position modulo ``conv_taps``.
"""

from __future__ import annotations

import math

import numpy as np
import torch

from clockwork_amd import ops
from clockwork_amd.config.spec import ParamSpec, StateSpec
from clockwork_amd.parts.base import EntryCache, Part
from clockwork_amd.parts.sink_attention import query_runs
from clockwork_amd.parts.specs import SelectiveScanSpec, StateSpaceSpec


def request_chunks(ctx, chunk: int):
    """The step's tokens in chunks of up to ``chunk`` of one request, (request, first token, tokens, number in its
    request) each, a request's in order and together: (items on the device, their number, the first chunk
    of each request). Made once a step, kept in ``ctx.plans``."""
    key = ("chunks of requests", chunk)
    plan = ctx.plans.get(key)
    if plan is None:
        items, first = [], [0]
        for r, q_len in enumerate(ctx.h_q_lens):
            tok0 = np.arange(0, q_len, chunk, dtype=np.int32)
            rows = np.zeros((tok0.size, 4), dtype=np.int32)
            rows[:, 0] = r
            rows[:, 1] = tok0
            rows[:, 2] = np.minimum(chunk, q_len - tok0)
            rows[:, 3] = np.arange(tok0.size)
            items.append(rows.reshape(-1))
            first.append(first[-1] + tok0.size)
        device_items, device_first = ctx.upload([np.concatenate(items), first])
        plan = ctx.plans[key] = (device_items, first[-1], device_first)
    return plan


class StateSpace(Part):
    graph_safe = True

    def __init__(self, spec: StateSpaceSpec) -> None:
        self.spec = spec
        self.inner = spec.num_heads * spec.head_dim
        self.channels = self.inner + 2 * spec.num_groups * spec.state_dim
        # columns of the input product: gate, then x, B and C, then the steps
        self.c_off, self.d_off = self.inner, self.inner + self.channels
        self.in_width = self.d_off + spec.num_heads

    def param_specs(self):
        s = self.spec
        return {
            "in_weight": ParamSpec((self.in_width, s.hidden_size)),
            "conv_weight": ParamSpec((self.channels, s.conv_taps), precision="float32", init=("normal", 0.5)),
            "conv_bias": ParamSpec((self.channels,), precision="float32", init=("normal", 0.1)),
            "dt_bias": ParamSpec((s.num_heads,), precision="float32", init=("uniform", -4.0, 0.5)),
            "a_log": ParamSpec((s.num_heads,), precision="float32", init=("uniform", -1.0, 2.0)),
            "skip": ParamSpec((s.num_heads,), precision="float32", init=("one_plus_uniform", 0.5)),
            "norm_weight": ParamSpec((self.inner,), precision="float32", init=("one_plus_uniform", 0.1)),
            "out_weight": ParamSpec((s.hidden_size, self.inner)),
        }

    def cache_need(self):
        s = self.spec
        return StateSpec((s.num_heads * s.state_dim * s.head_dim + s.conv_taps * self.channels,), "float32")

    def kernel_libraries(self) -> list:
        return [("state_space", None)]

    def bind(self, params, device, dtype) -> None:
        s = self.spec
        self.chunk = ops.state_space_chunk(dtype, s.state_dim, s.head_dim)
        if not self.chunk:
            raise ValueError(f"a state of {s.state_dim} x {s.head_dim} a head is beyond the state-space kernels (256 either way)")
        if s.conv_taps > ops.state_space_max_taps():
            raise ValueError(f"a convolution of {s.conv_taps} taps is beyond the kernel ({ops.state_space_max_taps()})")
        self.in_weight, self.out_weight = params["in_weight"], params["out_weight"]
        pad = (-self.in_width) % 8
        if pad and dtype == torch.bfloat16:
            # rows of the product that begin at multiples of 16 bytes (the step columns leave odd widths)
            self.in_weight = torch.cat([self.in_weight, self.in_weight.new_zeros((pad, s.hidden_size))])
        self.vectors = tuple(params[n] for n in ("conv_weight", "conv_bias", "dt_bias", "a_log", "skip"))
        self.norm_weight = params["norm_weight"]

    def _chunks(self, ctx):
        """None for a step of single tokens, else what ``ops.state_space`` takes as ``chunks``."""
        if max(ctx.h_q_lens, default=0) <= 1:
            return None
        items, n_chunks, first = request_chunks(ctx, self.chunk)
        return (*query_runs(ctx, ops.STATE_SPACE_CONV_TOKENS), items, n_chunks, first)

    def prepare(self, ctx) -> None:
        self._chunks(ctx)

    def shape_class(self, q_lens, ctx_lens):
        return "chunks" if max(q_lens, default=0) > 1 else "single tokens"

    def forward(self, x: torch.Tensor, ctx, cache: EntryCache) -> torch.Tensor:
        s = self.spec
        policy = getattr(ctx, "products", None)
        proj = ops.linear(x, self.in_weight, policy=policy)
        # single tokens: a head's columns are shared by workgroups while compute units are idle
        split = min(4, max(1, ctx.num_compute_units // max(1, ctx.num_requests * s.num_heads)))
        y = ops.state_space(proj, 0, self.c_off, self.d_off, *self.vectors, cache.state, ctx.state_slots, ctx.cu_q, ctx.ctx_lens,
                            ctx.num_requests, s.num_heads, s.num_groups, s.state_dim, s.head_dim, s.conv_taps,
                            chunks=self._chunks(ctx), split=split)
        out = ops.gated_parts_norm(y, proj, 0, self.norm_weight, s.norm_eps, s.norm_groups)
        return ops.linear(out, self.out_weight, policy=policy)


# tokens of a segment of a selective scan, by the step's tokens: short steps are cut finer, so that they
# have as many segments side by side
SCAN_SEGMENTS = ((1024, 32), (0, 16))


class SelectiveScan(Part):
    """A selective scan (``SelectiveScanSpec``). The input product; the convolution with silu; the product
    of x that makes the step's input, B and C; then a step of single tokens is one kernel a (request, 64
    channels) that makes the steps from that input, moves the state on and gates the output, and any other
    step is cut into segments that are walked side by side; output product. A request's slot is float32
    [state_dim * inner + taps * inner]: the states (a state's channels side by side), then the
    convolution's latest inputs by position modulo ``conv_taps``."""

    graph_safe = True
    partial_ok = False   # may the output come as ``ops.PartialSums``? A block whose next norm adds them up sets it

    def __init__(self, spec: SelectiveScanSpec) -> None:
        self.spec = spec

    def param_specs(self):
        s = self.spec
        return {
            "in_weight": ParamSpec((2 * s.inner, s.hidden_size)),
            "conv_weight": ParamSpec((s.inner, s.conv_taps), precision="float32", init=("normal", 0.5)),
            "conv_bias": ParamSpec((s.inner,), precision="float32", init=("normal", 0.1)),
            "low_weight": ParamSpec((s.dt_rank + 2 * s.state_dim, s.inner)),
            "dt_weight": ParamSpec((s.inner, s.dt_rank), init=("normal", 0.1)),
            "dt_bias": ParamSpec((s.inner,), precision="float32", init=("uniform", -4.0, 0.5)),
            "a_log": ParamSpec((s.inner, s.state_dim), precision="float32", init=("uniform", -1.0, 2.0)),
            "skip": ParamSpec((s.inner,), precision="float32", init=("one_plus_uniform", 0.5)),
            "out_weight": ParamSpec((s.hidden_size, s.inner)),
        }

    def cache_need(self):
        s = self.spec
        return StateSpec(((s.state_dim + s.conv_taps) * s.inner,), "float32")

    def kernel_libraries(self) -> list:
        return [("short_conv", None), ("selective_scan", None)]

    def bind(self, params, device, dtype) -> None:
        s = self.spec
        self.max_segment = ops.selective_scan_max_segment(s.state_dim)
        if not self.max_segment:
            raise ValueError(f"{s.state_dim} states a channel are beyond the selective-scan kernels (256)")
        if s.conv_taps > ops.short_conv_max_taps():
            raise ValueError(f"a convolution of {s.conv_taps} taps is beyond the kernel ({ops.short_conv_max_taps()})")
        self.in_weight, self.out_weight = params["in_weight"], params["out_weight"]
        self.conv_weight, self.conv_bias = params["conv_weight"], params["conv_bias"]
        self.low_weight, self.dt_weight = params["low_weight"], params["dt_weight"]
        pad = (-self.low_weight.shape[0]) % 8
        if pad and dtype == torch.bfloat16:
            # rows of the product that begin at multiples of 16 bytes
            self.low_weight = torch.cat([self.low_weight, self.low_weight.new_zeros((pad, s.inner))])
        self.dt_bias, self.skip = params["dt_bias"], params["skip"]
        # A log2(e), states first: neighbouring lanes are neighbouring channels
        self.a2 = (-torch.exp(params["a_log"].double()) * math.log2(math.e)).float().t().contiguous()

    def _segments(self, ctx):
        """None for a step of single tokens, else what ``ops.selective_scan`` takes as ``segments``."""
        if max(ctx.h_q_lens, default=0) <= 1:
            return None
        total = sum(ctx.h_q_lens)
        tokens = min(self.max_segment, next(n for least, n in SCAN_SEGMENTS if total >= least))
        items, n, first = request_chunks(ctx, tokens)
        return items, n, tokens, first

    def prepare(self, ctx) -> None:
        query_runs(ctx, ops.short_conv_tokens())
        self._segments(ctx)

    def shape_class(self, q_lens, ctx_lens):
        return "segments" if max(q_lens, default=0) > 1 else "single tokens"

    def forward(self, x: torch.Tensor, ctx, cache: EntryCache):
        policy = getattr(ctx, "products", None)
        proj = ops.linear(x, self.in_weight, policy=policy)
        out = torch.empty((x.shape[0], self.spec.inner), dtype=x.dtype, device=x.device)
        self.mix(proj, 0, out, x, ctx, cache)
        return ops.linear(out, self.out_weight, partial_ok=self.partial_ok, policy=policy)

    def joins(self) -> bool:
        """May a pair of mixers make this one's products together with the other's (``mix`` with an output scale)?"""
        return True

    def mix(self, proj: torch.Tensor, off: int, out: torch.Tensor, x, ctx, cache: EntryCache, scale: float = 1.0) -> None:
        """What stands between the two outer products: from the columns of ``proj`` that begin at ``off`` to
        ``out`` [T, inner], times ``scale``."""
        s = self.spec
        items, n_items = query_runs(ctx, ops.short_conv_tokens())
        xs = ops.short_conv(proj, off, s.inner, self.conv_weight, self.conv_bias, cache.state, s.state_dim * s.inner, ctx.state_slots,
                            ctx.cu_q, ctx.ctx_lens, items, n_items, ctx.num_requests)
        low = ops.linear(xs, self.low_weight, policy=getattr(ctx, "products", None))
        ops.selective_scan(xs, proj, off + s.inner, low, self.dt_weight, self.dt_bias, self.a2, self.skip, cache.state, ctx.state_slots,
                           ctx.cu_q, ctx.num_requests, out, scale, s.dt_rank, segments=self._segments(ctx))
