"""Two mixers side by side on the same input (``PairMixerSpec``).

With norms: the result is the mean of their outputs, each RMS-normed over the model width with a
weight of its own (one kernel, float32 statistics). With ``scales``: l * left + r * right. Mixers that
stand between two products (``joins``) then share them: one product makes both mixers' inputs, each
writes its own columns of one matrix, times its scale, and one product adds them up in its float32
sums. Each mixer keeps its own cache: the pair states the needs of both as ``CacheNeeds`` and hands
each mixer what belongs to it."""

from __future__ import annotations

import torch

from clockwork_amd import ops
from clockwork_amd.config.spec import CacheNeeds, ParamSpec
from clockwork_amd.parts.base import EntryCache, Part
from clockwork_amd.parts.specs import PairMixerSpec
from clockwork_amd.registry import build_part


class PairMixer(Part):
    SIDES = ("left", "right")
    partial_ok = False   # may the output come as ``ops.PartialSums``? A block whose next norm adds them up sets it

    def __init__(self, spec: PairMixerSpec) -> None:
        self.spec = spec
        self.left, self.right = build_part(spec.left), build_part(spec.right)
        self.joint = spec.scales is not None and all(getattr(m, "joins", lambda: False)() for m in (self.left, self.right))
        if spec.scales is not None and not self.joint:
            raise NotImplementedError("a scaled pair takes mixers that write their output between two products (joins)")

    @property
    def graph_safe(self) -> bool:
        return all(getattr(m, "graph_safe", False) for m in (self.left, self.right))

    def _sides(self):
        return zip(self.SIDES, (self.left, self.right))

    def param_specs(self):
        specs = {}
        for side, mixer in self._sides():
            for name, p in mixer.param_specs().items():
                specs[f"{side}.{name}"] = p
            if not self.joint:
                specs[f"{side}_out_norm"] = ParamSpec((self.spec.hidden_size,), precision="float32", init=("one_plus_uniform", 0.1))
        if self.joint:
            # both mixers' first products are one
            rows = [specs.pop(f"{side}.in_weight").shape[0] for side in self.SIDES]
            specs["in_weight"] = ParamSpec((sum(rows), self.spec.hidden_size))
        return specs

    def cache_need(self):
        kept, self._members_of = [], []   # per side: its members in the entry's cache, and are they several needs
        for m in (self.left, self.right):
            need = m.cache_need()
            own = [] if need is None else list(need.needs) if isinstance(need, CacheNeeds) else [need]
            self._members_of.append((range(len(kept), len(kept) + len(own)), isinstance(need, CacheNeeds)))
            kept += own
        return CacheNeeds(tuple(kept)) if kept else None

    def kernel_libraries(self) -> list:
        jobs = [("rowwise", None)]
        for m in (self.left, self.right):
            jobs += [j for j in getattr(m, "kernel_libraries", lambda: [])() if j not in jobs]
        return jobs

    def bind(self, params, device, dtype) -> None:
        own = {side: {k[len(side) + 1:]: v for k, v in params.items() if k.startswith(side + ".")} for side in self.SIDES}
        if self.joint:
            rows = self.left.param_specs()["in_weight"].shape[0]
            own["left"]["in_weight"], own["right"]["in_weight"] = params["in_weight"][:rows], params["in_weight"][rows:]
        for side, mixer in self._sides():
            mixer.bind(own[side], device, dtype)
        if self.joint:
            ins = [m.in_weight for m in (self.left, self.right)]
            # a mixer that pads its rows moves the other's columns
            padded = sum(w.shape[0] for w in ins) != params["in_weight"].shape[0]
            self.in_weight = torch.cat(ins) if padded else params["in_weight"]
            self.right_off = ins[0].shape[0]
            outs = [m.out_weight for m in (self.left, self.right)]
            self.split = outs[0].shape[1]
            self.width = self.split + outs[1].shape[1]
            # one matrix where its rows, and the second mixer's columns, begin at whole 16 bytes (or elements are floats)
            self.one_output = dtype == torch.float32 or (self.split % 8 == 0 and self.width % 8 == 0)
            self.out_weight = torch.cat(outs, dim=1).contiguous() if self.one_output else None
        else:
            self.left_norm, self.right_norm = params["left_out_norm"], params["right_out_norm"]
        if not hasattr(self, "_members_of"):
            self.cache_need()

    def prepare(self, ctx) -> None:
        for m in (self.left, self.right):
            prepare = getattr(m, "prepare", None)
            if prepare is not None:
                prepare(ctx)

    def shape_class(self, q_lens, ctx_lens):
        return tuple(getattr(m, "shape_class", lambda a, b: None)(q_lens, ctx_lens) for m in (self.left, self.right))

    def _caches(self, cache: EntryCache) -> list:
        """Each mixer's part of the entry's cache."""
        out = []
        for members, several in self._members_of:
            if several:
                out.append(EntryCache(writes=cache.writes, members=[cache.members[i] for i in members]))
            else:
                out.append(cache.members[members[0]] if len(members) else EntryCache(writes=False))
        return out

    def forward(self, x: torch.Tensor, ctx, cache: EntryCache):
        left, right = self._caches(cache)
        if not self.joint:
            return ops.rms_mean2(self.left.forward(x, ctx, left), self.right.forward(x, ctx, right), self.left_norm, self.right_norm,
                                 self.spec.eps)
        policy = getattr(ctx, "products", None)
        proj = ops.linear(x, self.in_weight, policy=policy)
        T, (l, r) = x.shape[0], self.spec.scales
        if self.one_output:
            both = torch.empty((T, self.width), dtype=x.dtype, device=x.device)
            a, b = both[:, : self.split], both[:, self.split :]
        else:
            a, b = (torch.empty((T, n), dtype=x.dtype, device=x.device) for n in (self.split, self.width - self.split))
        self.left.mix(proj, 0, a, x, ctx, left, scale=float(l))
        self.right.mix(proj, self.right_off, b, x, ctx, right, scale=float(r))
        if self.one_output:
            return ops.linear(both, self.out_weight, partial_ok=self.partial_ok, policy=policy)
        y = ops.linear(a, self.left.out_weight, policy=policy)
        return ops.moe_combine(y, 1, torch.empty_like(y), always=ops.linear(b, self.right.out_weight, policy=policy))
