"""Tufevik: config.json keys -> typed config -> parts -> weight names.

A decoder with a norm before and a norm behind each sublayer, x <- x + N1b(M(N1(x))), then
x <- x + N2b(F(N2(x))); every norm is a Dynamic Tanh, tanh(alpha x) * w + b. The stream starts as the
token's embedding times ``embedding.scale``; the output is the model's norm and the embedding table
itself, without that factor.

A layer's mixer is one of two kinds. "mlstm": a matrix memory a head with exponential gates and a
running maximum, every head's output divided by its root mean square, weighted and gated. "parallel":
two mixers on the same input, scaled and added: grouped attention whose query, key and value projections
pass a short convolution, with a norm over the whole query and key projection, rotation with YaRN
frequencies and a gate a head; beside a selective scan. The feed-forward is a dense one gated by a ReLU, a
routed one (a router with a bias whose weights are the softmax over the chosen logits) or absent.

Every size and every constant that can differ between models of the design is read from config.json:
``vocab``, ``width``, ``norm.eps``, ``embedding.scale`` and, per entry of ``layers``, ``type``, ``mixer``
("mlstm": ``heads``, ``dim``, ``vdim``, ``gate_cap``; "parallel": ``left_scale``, ``right_scale``, ``left`` with
``heads``, ``kv_heads``, ``dim``, ``vdim``, ``conv``, ``scale``, ``rot.base``, ``rot.dims``, ``rot.scaling`` (``factor``,
``original``, ``fast``, ``slow``; absent: unscaled) and ``right`` with ``inner``, ``state``, ``conv``, ``dt_rank``) and
``mlp`` (``kind`` "dense": ``ff``; "moe": ``expert.ff``, ``router.experts``, ``router.top``; null: no feed-forward).
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Optional

from clockwork_amd.config.spec import LayerSpec, ModelSpec, RunEntry, WeightTarget
from clockwork_amd.parts.specs import (DynamicTanhSpec, GatedAttentionSpec, GatedMLPSpec, LinearHeadSpec, MatrixMemorySpec, PairMixerSpec,
                                       PositionTableEmbeddingSpec, RopeNeoxSpec, RoutedExpertsSpec, SelectiveScanSpec, YarnSpec)
from clockwork_amd.registry import Architecture, register_architecture

NAME = "Tufevik"
MIXER_KINDS = ("mlstm", "parallel")


def _need(d: dict, key: str, where: str):
    if not isinstance(d, dict) or d.get(key) is None:
        raise ValueError(f"config.json lacks {where}{key}")
    return d[key]


@dataclass(frozen=True)
class MemoryConfig:
    heads: int
    dim: int
    vdim: int
    gate_cap: float


@dataclass(frozen=True)
class AttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int
    scale: float
    rot_base: float
    rot_dims: int
    yarn: Optional[tuple]   # (factor, original, fast, slow) or None


@dataclass(frozen=True)
class ScanConfig:
    inner: int
    state: int
    conv: int
    dt_rank: int


@dataclass(frozen=True)
class ParallelConfig:
    left: AttentionConfig
    right: ScanConfig
    left_scale: float
    right_scale: float


@dataclass(frozen=True)
class DenseConfig:
    ff: int


@dataclass(frozen=True)
class RoutedConfig:
    ff: int
    experts: int
    top: int


@dataclass(frozen=True)
class TufevikLayerConfig:
    kind: str      # "mlstm" or "parallel"
    mixer: Any     # MemoryConfig or ParallelConfig
    mlp: Any       # DenseConfig, RoutedConfig or None


def _mixer(kind: str, m: dict, where: str):
    if kind == "mlstm":
        return MemoryConfig(*(int(_need(m, key, where)) for key in ("heads", "dim", "vdim")), gate_cap=float(_need(m, "gate_cap", where)))
    a, aw = _need(m, "left", where), where + "left."
    r, rw = _need(m, "right", where), where + "right."
    rot = _need(a, "rot", aw)
    yarn = rot.get("scaling")
    left = AttentionConfig(*(int(_need(a, key, aw)) for key in ("heads", "kv_heads", "dim", "vdim", "conv")), scale=float(_need(a, "scale", aw)),
                           rot_base=float(_need(rot, "base", aw + "rot.")), rot_dims=int(_need(rot, "dims", aw + "rot.")),
                           yarn=None if yarn is None else tuple(float(_need(yarn, key, aw + "rot.scaling."))
                                                                for key in ("factor", "original", "fast", "slow")))
    right = ScanConfig(*(int(_need(r, key, rw)) for key in ("inner", "state", "conv", "dt_rank")))
    return ParallelConfig(left, right, float(_need(m, "left_scale", where)), float(_need(m, "right_scale", where)))


def _feed_forward(mlp: dict, where: str):
    kind = _need(mlp, "kind", where)
    if kind == "dense":
        return DenseConfig(int(_need(mlp, "ff", where)))
    if kind != "moe":
        raise NotImplementedError(f"{where}kind {kind!r} is not a feed-forward of this design ('dense', 'moe')")
    router = _need(mlp, "router", where)
    return RoutedConfig(ff=int(_need(_need(mlp, "expert", where), "ff", where + "expert.")),
                        experts=int(_need(router, "experts", where + "router.")), top=int(_need(router, "top", where + "router.")))


@dataclass(frozen=True)
class TufevikConfig:
    vocab: int
    width: int
    eps: float
    embedding_scale: float
    layers: tuple

    @classmethod
    def from_dict(cls, d: dict) -> "TufevikConfig":
        if d.get("architecture", NAME) != NAME and NAME not in (d.get("architectures") or []):
            raise ValueError(f"expected a {NAME} model, got architecture={d.get('architecture')!r}")
        entries = _need(d, "layers", "")
        if not isinstance(entries, list) or not entries:
            raise ValueError("config.json: 'layers' must be a list with at least one layer")
        layers = []
        for i, entry in enumerate(entries):
            where = f"layers[{i}]."
            kind = _need(entry, "type", where)
            if kind not in MIXER_KINDS:
                raise NotImplementedError(f"{where}type {kind!r} is not a layer of this design {MIXER_KINDS}")
            mlp = entry.get("mlp")
            layers.append(TufevikLayerConfig(kind, _mixer(kind, _need(entry, "mixer", where), where + "mixer."),
                                             None if mlp is None else _feed_forward(mlp, where + "mlp.")))
        cfg = cls(vocab=int(_need(d, "vocab", "")), width=int(_need(d, "width", "")),
                  eps=float(_need(_need(d, "norm", ""), "eps", "norm.")),
                  embedding_scale=float(_need(_need(d, "embedding", ""), "scale", "embedding.")), layers=tuple(layers))
        cfg.check()
        return cfg

    def check(self) -> None:
        for name in ("vocab", "width"):
            if getattr(self, name) <= 0:
                raise ValueError(f"{name} must be positive, got {getattr(self, name)}")
        if not self.eps > 0:
            raise ValueError("norm.eps must be positive")
        for i, layer in enumerate(self.layers):
            if layer.kind == "parallel":
                a, r = layer.mixer.left, layer.mixer.right
                if min(a.heads, a.kv_heads, a.dim, a.vdim, a.conv) <= 0:
                    raise ValueError(f"layers[{i}]: sizes must be positive")
                if a.heads % a.kv_heads:
                    raise ValueError(f"layers[{i}]: {a.heads} heads are not a multiple of {a.kv_heads} kv_heads")
                if a.rot_dims % 2 or not 0 <= a.rot_dims <= a.dim:
                    raise ValueError(f"layers[{i}]: rot.dims {a.rot_dims} must be even and at most dim {a.dim}")
                if min(r.inner, r.state, r.conv, r.dt_rank) <= 0:
                    raise ValueError(f"layers[{i}]: the scan's sizes must be positive")
            f = layer.mlp
            if f is not None and f.ff <= 0:
                raise ValueError(f"layers[{i}]: the feed-forward's inner width must be positive")
            if isinstance(f, RoutedConfig) and not 1 <= f.top <= f.experts:
                raise ValueError(f"layers[{i}]: router.top {f.top} of {f.experts} experts")


def with_checkpoint_shapes(config: dict, shapes: dict) -> dict:
    """``config`` with what it leaves out of a parallel mixer's sizes taken from the checkpoint's tensors
    (``shapes``: name -> shape): the convolutions' taps, and the scan's inner width, states and step rank."""
    out = dict(config)
    out["layers"] = []
    for i, entry in enumerate(config.get("layers") or []):
        entry = dict(entry)
        mixer = entry.get("mixer")
        if entry.get("type") == "parallel" and isinstance(mixer, dict):
            mixer = entry["mixer"] = dict(mixer)
            mix = f"l{i}.mix"
            for side, sizes in (("left", {"conv": (f"{mix}.left.q.conv", 1)}),
                                ("right", {"conv": (f"{mix}.right.conv", 1), "inner": (f"{mix}.right.A_log", 0),
                                           "state": (f"{mix}.right.A_log", 1), "dt_rank": (f"{mix}.right.dt", 1)})):
                if isinstance(mixer.get(side), dict):
                    half = mixer[side] = dict(mixer[side])
                    for key, (name, axis) in sizes.items():
                        if half.get(key) is None and len(shapes.get(name, ())) > axis:
                            half[key] = int(shapes[name][axis])
        out["layers"].append(entry)
    return out


def _mixer_spec(W: int, eps: float, kind: str, m):
    if kind == "mlstm":
        return MatrixMemorySpec(hidden_size=W, num_heads=m.heads, key_dim=m.dim, value_dim=m.vdim, gate_cap=m.gate_cap, norm_eps=eps)
    a, r = m.left, m.right
    rope = None
    if a.rot_dims:
        rope = RopeNeoxSpec(rotary_dim=a.rot_dims, theta=a.rot_base, scaling=YarnSpec(*a.yarn) if a.yarn is not None else None)
    left = GatedAttentionSpec(hidden_size=W, num_heads=a.heads, num_kv_heads=a.kv_heads, key_dim=a.dim, value_dim=a.vdim, scale=a.scale,
                              norm_eps=eps, qk_norm=True, qk_norm_over="projection", conv_taps=a.conv, position=rope, output_gate=True,
                              gate_per_head=True)
    right = SelectiveScanSpec(hidden_size=W, inner=r.inner, state_dim=r.state, dt_rank=r.dt_rank, conv_taps=r.conv)
    return PairMixerSpec(hidden_size=W, left=left, right=right, scales=(m.left_scale, m.right_scale))


def _feed_forward_spec(W: int, f):
    if f is None:
        return None
    if isinstance(f, DenseConfig):
        return GatedMLPSpec(W, f.ff, activation="relu")
    # the softmax over the chosen logits is that over all of them, divided by the chosen ones' sum
    return RoutedExpertsSpec(hidden_size=W, intermediate_size=f.ff, num_experts=f.experts, top_k=f.top, router="softmax", renormalize=True,
                             weight_on="output", router_bias=True)


def build_spec(cfg: TufevikConfig) -> ModelSpec:
    W = cfg.width
    norm = DynamicTanhSpec(size=W)
    layers = []
    for layer in cfg.layers:
        feed_forward = _feed_forward_spec(W, layer.mlp)
        behind = [("mixer_post_norm", norm)] + ([("ffn_post_norm", norm)] if feed_forward is not None else [])
        layers.append(LayerSpec(arrangement="sandwich", mixer=_mixer_spec(W, cfg.eps, layer.kind, layer.mixer), mixer_norm=norm,
                                feed_forward=feed_forward, ffn_norm=norm if feed_forward is not None else None, extra=tuple(behind)))
    spec = ModelSpec(
        architecture=NAME, vocab_size=cfg.vocab, hidden_size=W, layers=layers, run=[RunEntry(layer=i) for i in range(len(layers))],
        final_norm=norm, tie_embeddings=True,
        embedding=PositionTableEmbeddingSpec(cfg.vocab, W, scale=cfg.embedding_scale), head=LinearHeadSpec(cfg.vocab, W, tied=True),
        info={"layers": len(layers), "hidden": W, "vocab": cfg.vocab, "kinds": [l.kind for l in cfg.layers], "tied": True},
    )
    spec.validate()
    return spec


def _norm_plan(dst: str, src: str, W: int) -> list:
    return [WeightTarget(f"{dst}.weight", (src,), ((W,),)), WeightTarget(f"{dst}.bias", (f"{src}.b",), ((W,),)),
            WeightTarget(f"{dst}.alpha", (f"{src}.alpha",), ((),), transform=("as_vector",))]


def _memory_plan(dst: str, mix: str, W: int, m: MemoryConfig) -> list:
    qk, v = m.heads * m.dim, m.heads * m.vdim
    return [
        WeightTarget(f"{dst}.in_weight", tuple(f"{mix}.{n}" for n in ("q", "k", "v", "g")), ((qk, W), (qk, W), (v, W), (v, W))),
        WeightTarget(f"{dst}.gate_weight", (f"{mix}.i", f"{mix}.f"), ((m.heads, W),) * 2),
        WeightTarget(f"{dst}.gate_bias", (f"{mix}.i.b", f"{mix}.f.b"), ((m.heads,),) * 2),
        WeightTarget(f"{dst}.norm_weight", (f"{mix}.norm",), ((v,),)),
        WeightTarget(f"{dst}.out_weight", (f"{mix}.o",), ((W, v),)),
    ]


def _parallel_plan(dst: str, mix: str, W: int, m: ParallelConfig) -> list:
    """Everything both mixers make of the layer's input is one product: q, k, v and the gates of the left, x
    and z of the right."""
    a, r, left, right = m.left, m.right, f"{mix}.left", f"{mix}.right"
    nq, nk, nv = a.heads * a.dim, a.kv_heads * a.dim, a.kv_heads * a.vdim
    return [
        WeightTarget(f"{dst}.in_weight", tuple(f"{left}.{n}" for n in ("q", "k", "v", "g")) + (f"{right}.in",),
                     ((nq, W), (nk, W), (nv, W), (a.heads, W), (2 * r.inner, W))),
        WeightTarget(f"{dst}.left.conv_weight", tuple(f"{left}.{n}.conv" for n in ("q", "k", "v")), tuple((n, a.conv) for n in (nq, nk, nv))),
        WeightTarget(f"{dst}.left.q_norm", (f"{left}.q.norm",), ((nq,),)),
        WeightTarget(f"{dst}.left.k_norm", (f"{left}.k.norm",), ((nk,),)),
        WeightTarget(f"{dst}.left.out_weight", (f"{left}.o",), ((W, a.heads * a.vdim),)),
        WeightTarget(f"{dst}.right.conv_weight", (f"{right}.conv",), ((r.inner, r.conv),)),
        WeightTarget(f"{dst}.right.conv_bias", (f"{right}.conv.b",), ((r.inner,),)),
        WeightTarget(f"{dst}.right.low_weight", (f"{right}.x",), ((r.dt_rank + 2 * r.state, r.inner),)),
        WeightTarget(f"{dst}.right.dt_weight", (f"{right}.dt",), ((r.inner, r.dt_rank),)),
        WeightTarget(f"{dst}.right.dt_bias", (f"{right}.dt.b",), ((r.inner,),)),
        WeightTarget(f"{dst}.right.a_log", (f"{right}.A_log",), ((r.inner, r.state),)),
        WeightTarget(f"{dst}.right.skip", (f"{right}.D",), ((r.inner,),)),
        WeightTarget(f"{dst}.right.out_weight", (f"{right}.o",), ((W, r.inner),)),
    ]


def weight_plan(cfg: TufevikConfig, spec: ModelSpec) -> list[WeightTarget]:
    """Checkpoint names -> the model's parameters. Projections that read the same input are stacked; the
    experts' gate and up matrices lie expert by expert."""
    W = cfg.width
    plan = [WeightTarget("embed.weight", ("embed",), ((cfg.vocab, W),))]
    for i, layer in enumerate(cfg.layers):
        src, dst = f"l{i}", f"layers.{i}"
        plan += _norm_plan(f"{dst}.mixer_norm", f"{src}.norm1", W) + _norm_plan(f"{dst}.mixer_post_norm", f"{src}.norm1b", W)
        mixer = _memory_plan if layer.kind == "mlstm" else _parallel_plan
        plan += mixer(f"{dst}.mixer", f"{src}.mix", W, layer.mixer)
        f = layer.mlp
        if f is None:
            continue
        plan += _norm_plan(f"{dst}.ffn_norm", f"{src}.norm2", W) + _norm_plan(f"{dst}.ffn_post_norm", f"{src}.norm2b", W)
        ff, mlp = f"{dst}.feed_forward", f"{src}.mlp"
        if isinstance(f, DenseConfig):
            plan += [WeightTarget(f"{ff}.gate_up_weight", (f"{mlp}.gate", f"{mlp}.up"), ((f.ff, W),) * 2),
                     WeightTarget(f"{ff}.down_weight", (f"{mlp}.down",), ((W, f.ff),))]
            continue
        gate_up = tuple(f"{mlp}.e{e}.{n}" for e in range(f.experts) for n in ("gate", "up"))
        down = tuple(f"{mlp}.e{e}.down" for e in range(f.experts))
        plan += [WeightTarget(f"{ff}.router_weight", (f"{mlp}.router",), ((f.experts, W),)),
                 WeightTarget(f"{ff}.router_bias", (f"{mlp}.router.b",), ((f.experts,),)),
                 WeightTarget(f"{ff}.gate_up_weight", gate_up, ((f.ff, W),) * len(gate_up)),
                 WeightTarget(f"{ff}.down_weight", down, ((W, f.ff),) * len(down))]
    plan += _norm_plan("final_norm", "final.norm", W)
    # the output head is the embedding table; a checkpoint that names it apart must hold the same
    plan.append(WeightTarget("lm_head.weight", ("head",), ((cfg.vocab, W),), optional=True))
    return plan


ARCHITECTURE = Architecture(name=NAME, parse_config=TufevikConfig.from_dict, build_spec=build_spec, weight_plan=weight_plan,
                            sizes_from_checkpoint=with_checkpoint_shapes)
register_architecture([NAME], ARCHITECTURE)
