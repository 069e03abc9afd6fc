"""Tufevik without a GPU: the configuration reader and what it refuses, the weight plan against the
tensors a checkpoint of the design holds, cache groups (pages, two kinds of state for a parallel layer, one
for a matrix memory), YaRN frequencies, what the blocks refuse, and the plain implementation against
second ways of writing it (the matrix memory and the selective scan in closed form, the convolution through
torch, the router by brute force, attention through torch)."""

import copy
import itertools
import math
from types import SimpleNamespace

import pytest
import torch

from clockwork_amd.cache.manager import CacheManager, cache_needs_of, plan_groups
from clockwork_amd.config.spec import PagedRowsSpec, StateSpec
from clockwork_amd.parts.model import DecoderModel, model_param_specs
from clockwork_amd.parts.rope import rotary_frequencies
from clockwork_amd.parts.specs import (DynamicTanhSpec, GatedAttentionSpec, LatentAttentionSpec, PairMixerSpec, RMSNormSpec, RopeNeoxSpec,
                                       RopePairsSpec, YarnSpec)
from clockwork_amd.registry import build_arrangement, build_part, resolve_architecture
from clockwork_amd.weights.loader import check_plan
from clockwork_amd.weights.random_init import write_random_model
from tests.configs import TUFEVIK_A, TUFEVIK_B, TUFEVIK_C, TUFEVIK_D, random_tufevik_config
from tests.plain import tufevik_plain as plain


def _describe(config):
    arch = resolve_architecture(config)
    cfg = arch.parse_config(config)
    spec = arch.build_spec(cfg)
    return arch, cfg, spec, arch.weight_plan(cfg, spec)


def test_the_design_is_found_and_every_constant_is_read():
    arch, cfg, spec, _ = _describe(TUFEVIK_A)
    assert arch.name == "Tufevik" and spec.architecture == "Tufevik"
    assert (cfg.vocab, cfg.width, cfg.eps, cfg.embedding_scale) == (211, 96, 1e-5, 3.0)
    assert spec.embedding.scale == 3.0 and spec.embedding.max_positions is None and spec.head.tied and spec.head.scale is None
    assert spec.tie_embeddings and spec.final_norm == DynamicTanhSpec(96)
    assert all(l.arrangement == "sandwich" for l in spec.layers)
    a, b, c, d = spec.layers
    pair = a.mixer
    assert pair.scales == (0.6, 1.3)
    m = pair.left
    assert (m.num_heads, m.num_kv_heads, m.key_dim, m.value_dim, m.conv_taps, m.scale, m.norm_eps) == (6, 2, 24, 40, 3, 0.3, 1e-5)
    assert (m.qk_norm, m.qk_norm_over, m.qk_norm_weight, m.qk_norm_after_rotation) == (True, "projection", True, False)
    assert (m.output_gate, m.gate_per_head, m.window, m.softcap, m.qkv_bias, m.out_bias) == (True, True, None, None, False, False)
    assert m.position == RopeNeoxSpec(16, 500.0, YarnSpec(4.0, 64, 8.0, 1.0))
    r = pair.right
    assert (r.inner, r.state_dim, r.conv_taps, r.dt_rank) == (80, 12, 4, 10)
    assert c.mixer.left.position.scaling == YarnSpec(8.0, 256, 16.0, 2.0) and c.mixer.scales == (1.0, 0.5)
    s = b.mixer
    assert (s.num_heads, s.key_dim, s.value_dim, s.gate_cap, s.norm_eps) == (3, 24, 40, 9.0, 1e-5)
    f = a.feed_forward
    assert (f.intermediate_size, f.num_experts, f.top_k, f.router, f.renormalize, f.router_bias) == (40, 6, 3, "softmax", True, True)
    assert (f.weight_on, f.choice_correction, f.groups, f.shared_intermediate, f.renorm_eps, f.limit) == ("output", False, None, None, 0.0, 0.0)
    assert (b.feed_forward.intermediate_size, b.feed_forward.activation) == (120, "relu")
    assert c.feed_forward is None and c.ffn_norm is None and [n for n, _ in c.extra] == ["mixer_post_norm"]
    assert [n for n, _ in d.extra] == ["mixer_post_norm", "ffn_post_norm"]
    left = _describe(TUFEVIK_B)[2].layers[0].mixer.left
    assert left.position is None and left.conv_taps == 1
    assert _describe(TUFEVIK_B)[2].layers[2].mixer.left.position.scaling is None


@pytest.mark.parametrize("path, value, error", [
    (("architecture",), "Tufevikk", ValueError),
    (("layers", 0, "type"), "attention", NotImplementedError),
    (("layers", 0, "mlp", "kind"), "swiglu", NotImplementedError),
    (("layers", 0, "mlp", "expert", "ff"), 0, ValueError),
    (("layers", 0, "mlp", "router", "top"), 7, ValueError),
    (("layers", 0, "mlp", "router", "top"), 0, ValueError),
    (("layers", 0, "mlp", "router"), None, ValueError),
    (("layers", 1, "mlp", "ff"), None, ValueError),
    (("layers", 1, "mlp", "ff"), -3, ValueError),
    (("layers", 0, "mixer", "left", "heads"), 5, ValueError),
    (("layers", 0, "mixer", "left", "conv"), None, ValueError),
    (("layers", 0, "mixer", "left", "conv"), 0, ValueError),
    (("layers", 0, "mixer", "left", "scale"), None, ValueError),
    (("layers", 0, "mixer", "left", "rot"), None, ValueError),
    (("layers", 0, "mixer", "left", "rot", "dims"), 15, ValueError),
    (("layers", 0, "mixer", "left", "rot", "dims"), 26, ValueError),
    (("layers", 0, "mixer", "left", "rot", "scaling", "slow"), None, ValueError),
    (("layers", 0, "mixer", "left", "rot", "scaling", "factor"), 0.0, ValueError),
    (("layers", 0, "mixer", "right", "state"), 0, ValueError),
    (("layers", 0, "mixer", "right", "dt_rank"), None, ValueError),
    (("layers", 0, "mixer", "left_scale"), None, ValueError),
    (("layers", 0, "mixer", "right_scale"), None, ValueError),
    (("layers", 1, "mixer", "gate_cap"), None, ValueError),
    (("layers", 1, "mixer", "gate_cap"), 0.0, ValueError),
    (("layers", 1, "mixer", "vdim"), 0, ValueError),
    (("embedding",), None, ValueError),
    (("embedding", "scale"), None, ValueError),
    (("norm",), None, ValueError),
    (("norm", "eps"), 0.0, ValueError),
    (("layers",), [], ValueError),
    (("width",), 0, ValueError),
])
def test_what_the_configuration_reader_refuses(path, value, error):
    config = copy.deepcopy(TUFEVIK_A)
    at = config
    for key in path[:-1]:
        at = at[key]
    at[path[-1]] = value
    with pytest.raises(error):
        _describe(config)


def _tensor_names(config):
    """Names and shapes of a checkpoint of the design, written out from the layer list."""
    W = config["width"]
    names = {"embed": (config["vocab"], W)}

    def norm(name):
        names.update({name: (W,), name + ".b": (W,), name + ".alpha": ()})

    norm("final.norm")
    for i, entry in enumerate(config["layers"]):
        p, m, mlp = f"l{i}.", entry["mixer"], entry["mlp"]
        x = p + "mix."
        norm(p + "norm1")
        norm(p + "norm1b")
        if entry["type"] == "mlstm":
            H, qk, v = m["heads"], m["heads"] * m["dim"], m["heads"] * m["vdim"]
            names.update({x + "q": (qk, W), x + "k": (qk, W), x + "v": (v, W), x + "g": (v, W), x + "o": (W, v), x + "norm": (v,),
                          x + "i": (H, W), x + "i.b": (H,), x + "f": (H, W), x + "f.b": (H,)})
        else:
            a, r = m["left"], m["right"]
            for n, rows in (("q", a["heads"] * a["dim"]), ("k", a["kv_heads"] * a["dim"]), ("v", a["kv_heads"] * a["vdim"])):
                names.update({f"{x}left.{n}": (rows, W), f"{x}left.{n}.conv": (rows, a["conv"])})
                if n != "v":
                    names[f"{x}left.{n}.norm"] = (rows,)
            names.update({x + "left.g": (a["heads"], W), x + "left.o": (W, a["heads"] * a["vdim"])})
            n, s, k = r["inner"], r["state"], r["dt_rank"]
            names.update({x + "right.in": (2 * n, W), x + "right.conv": (n, r["conv"]), x + "right.conv.b": (n,), x + "right.x": (k + 2 * s, n),
                          x + "right.dt": (n, k), x + "right.dt.b": (n,), x + "right.A_log": (n, s), x + "right.D": (n,), x + "right.o": (W, n)})
        if mlp is None:
            continue
        norm(p + "norm2")
        norm(p + "norm2b")
        f = p + "mlp."
        if mlp["kind"] == "moe":
            E = mlp["router"]["experts"]
            names.update({f + "router": (E, W), f + "router.b": (E,)})
        for e in [f] if mlp["kind"] == "dense" else [f"{f}e{e}." for e in range(E)]:
            ff = mlp["ff"] if mlp["kind"] == "dense" else mlp["expert"]["ff"]
            names.update({e + "gate": (ff, W), e + "up": (ff, W), e + "down": (W, ff)})
    return names


@pytest.mark.parametrize("config", [TUFEVIK_A, TUFEVIK_B, TUFEVIK_C, TUFEVIK_D] + [random_tufevik_config(s) for s in range(8)])
def test_the_weight_plan_takes_every_tensor_of_the_design_and_no_other(config):
    _, _, spec, plan = _describe(config)
    names = _tensor_names(config)
    assert check_plan(names, plan) == ([], [], [])
    specs = model_param_specs(spec)
    assert {t.param for t in plan} == set(specs)
    for target in plan:
        if target.transform is None:
            rows = sum(s[0] for s in target.source_shapes)
            assert specs[target.param].shape == (rows, *target.source_shapes[0][1:])
    assert check_plan(dict(names, extra=(1,)), plan)[1] == ["extra"]


def test_sizes_that_the_configuration_leaves_to_the_checkpoint():
    config = copy.deepcopy(TUFEVIK_A)
    mixer = config["layers"][0]["mixer"]
    del mixer["left"]["conv"]
    for key in ("inner", "state", "conv", "dt_rank"):
        del mixer["right"][key]
    arch = resolve_architecture(config)
    filled = arch.sizes_from_checkpoint(config, _tensor_names(TUFEVIK_A))
    assert arch.parse_config(filled) == arch.parse_config(TUFEVIK_A)
    assert "conv" not in mixer["left"]


def test_cache_groups_and_slots():
    _, _, spec, _ = _describe(TUFEVIK_A)
    model = DecoderModel(spec)
    groups = plan_groups(cache_needs_of(spec, model.mixers(), model.own_caches()))
    assert [(type(g.need), g.entries) for g in groups] == [
        (PagedRowsSpec, ((0, 0),)), (StateSpec, ((0, 1),)), (StateSpec, ((0, 2),)), (StateSpec, (1,)),
        (PagedRowsSpec, ((2, 0),)), (StateSpec, ((2, 1),)), (StateSpec, ((2, 2),)), (StateSpec, (3,))]
    assert groups[0].need.planes == (("k", (2, 24)), ("v", (2, 40)))
    assert groups[1].need.shape == (3 * (144 + 48 + 80),)                 # the convolution's latest inputs
    assert groups[2].need.shape == ((12 + 4) * 80,)                       # the scan's states and its own inputs
    assert groups[3].need.shape == (3 * 24 * 40 + 2 * 3 * 25,)            # matrices, then sums and maxima twice
    manager = CacheManager(groups, 8, 10, max_num_seqs=2)
    assert not manager.supports_prefix_sharing
    manager.admit("a", 20)
    manager.admit("b", 5)
    assert not manager.can_admit(5)
    manager.free("a")
    assert manager.can_admit(5)
    for config, paged in ((TUFEVIK_C, 0), (TUFEVIK_D, 2)):
        spec = _describe(config)[2]
        model = DecoderModel(spec)
        groups = plan_groups(cache_needs_of(spec, model.mixers(), model.own_caches()))
        assert sum(g.is_kv for g in groups) == paged


def test_a_pair_hands_each_mixer_its_own_caches():
    pair = DecoderModel(_describe(TUFEVIK_A)[2]).layers[0].mixer
    need = pair.cache_need()
    assert len(need.needs) == 3
    members = ["pages", "inputs", "states"]
    left, right = pair._caches(SimpleNamespace(members=members, writes=True))
    assert left.members == ["pages", "inputs"] and right == "states"


# ------------------------------------------------------------------------------- what is refused
def test_parts_that_do_not_fit_are_refused():
    base = dict(hidden_size=32, num_heads=2, num_kv_heads=1, key_dim=8, value_dim=8, scale=1.0)
    for bad in (dict(values="keys"), dict(qkv_bias=True), dict(query_temperature=(1.0, 4)), dict(position=RopePairsSpec(8, 10.0)),
                dict(qk_norm_over="head"), dict(qk_norm_after_rotation=True), dict(qk_norm_weight=False)):
        with pytest.raises(ValueError):
            GatedAttentionSpec(**base, **dict(dict(conv_taps=3, qk_norm_over="projection"), **bad))
    with pytest.raises(ValueError):
        GatedAttentionSpec(**base, qk_norm_over="row")
    with pytest.raises(ValueError):
        YarnSpec(4.0, 0, 32.0, 1.0)
    with pytest.raises(NotImplementedError):
        build_part(RopeNeoxSpec(8, 10.0, YarnSpec(4.0, 64, 8.0, 1.0)))
    # a scaled pair takes mixers that write between two products: plain gated attention does not
    left = GatedAttentionSpec(**base)
    with pytest.raises(NotImplementedError):
        build_part(PairMixerSpec(32, left, left, scales=(1.0, 1.0)))
    latent = LatentAttentionSpec(hidden_size=32, num_heads=2, key_dim=8, rope_dim=8, value_dim=8, q_rank=8, kv_rank=8, scale=1.0, rope_base=10.0,
                                 rotary_dims=8, norm_eps=1e-5)
    with pytest.raises(NotImplementedError):
        build_part(PairMixerSpec(32, GatedAttentionSpec(**base, conv_taps=2, qk_norm_over="projection"), latent, scales=(1.0, 1.0)))
    tanh, rms = build_part(DynamicTanhSpec(32)), build_part(RMSNormSpec(32, 1e-5))
    with pytest.raises(TypeError):
        build_arrangement("sandwich", mixer=SimpleNamespace(), mixer_norm=rms, mixer_post_norm=tanh)
    with pytest.raises(ValueError):
        build_arrangement("sandwich", mixer=SimpleNamespace(), mixer_norm=tanh, mixer_post_norm=tanh, feed_forward=SimpleNamespace(), ffn_norm=tanh)


@pytest.mark.parametrize("dims, base, yarn", [(16, 500.0, (4.0, 64, 8.0, 1.0)), (64, 10000.0, (8.0, 4096, 32.0, 1.0)), (10, 50.0, (2.0, 4, 30.0, 0.01)),
                                              (32, 1e6, (1.0, 100, 2.0, 1.0)), (8, 10.0, None), (12, 100.0, (3.0, 50, 5.0, 5.0))])
def test_yarn_frequencies(dims, base, yarn):
    """Against the plain implementation; and the ends of the ramp: what turns fast keeps its frequency, what
    turns slowly is divided by the factor."""
    freq, mult = rotary_frequencies(RopeNeoxSpec(dims, base, YarnSpec(*yarn) if yarn else None))
    rot = {"base": base, "dims": dims}
    if yarn:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), yarn))
    want, want_mult = plain.rotation_frequencies(rot)
    torch.testing.assert_close(freq, torch.tensor(want, dtype=torch.float64), rtol=1e-12, atol=0)
    assert mult == pytest.approx(want_mult)
    plain_freq = [base ** (-2 * i / dims) for i in range(dims // 2)]
    if yarn is None:
        assert mult == 1.0 and freq.tolist() == pytest.approx(plain_freq)
    elif yarn[0] == 8.0:
        assert freq[0] == plain_freq[0] and freq[-1] == pytest.approx(plain_freq[-1] / 8.0)
        between = [f for f, p in zip(freq.tolist(), plain_freq) if p / 8 * 1.001 < f < p * 0.999]
        assert len(between) > 3


# ------------------------------------------------------------------------------- the plain implementation
def _gen(seed):
    return torch.Generator().manual_seed(seed)


def test_plain_matrix_memory_in_closed_form():
    """o_t = sum_s w_ts (q_t . k_s) v_s / (max(|sum_s w_ts (q_t . k_s)|, e^(-m_t)) + 1e-6) with w_ts = exp(f_(s+1) +
    ... + f_t + i_s - m_t), m_t the largest of the exponents and of f_1 + ... + f_t."""
    T, D, V = 11, 4, 3
    g = _gen(1)
    q, k, v = torch.randn(T, D, generator=g).double(), torch.randn(T, D, generator=g).double(), torch.randn(T, V, generator=g).double()
    for shift in (-6.0, 0.0, 6.0):
        i, f = torch.randn(T, generator=g).double() * 2 + shift, -torch.rand(T, generator=g).double() * 3
        got = plain.matrix_memory(q, k, v, i, f)
        for t in range(T):
            exponents = [float(f[s + 1 : t + 1].sum() + i[s]) for s in range(t + 1)]
            m = max(exponents + [float(f[: t + 1].sum())])
            w = [math.exp(e - m) * float(q[t] @ k[s]) for s, e in enumerate(exponents)]
            num = sum(x * v[s] for s, x in enumerate(w))
            torch.testing.assert_close(got[t], num / (max(abs(sum(w)), math.exp(-m)) + 1e-6), rtol=1e-9, atol=1e-12)


def test_plain_log_gates():
    g = _gen(2)
    w = {n: torch.randn(s, generator=g).double() * 4 for n, s in (("i", (3, 6)), ("f", (3, 6)), ("i.b", (3,)), ("f.b", (3,)))}
    h = torch.randn(5, 6, generator=g).double()
    i, f = plain.log_gates(h, w, "", 7.0)
    torch.testing.assert_close(i, 7 * torch.tanh((h @ w["i"].t() + w["i.b"]) / 7))
    torch.testing.assert_close(f, torch.nn.functional.logsigmoid(7 * torch.tanh((h @ w["f"].t() + w["f.b"]) / 7)))
    assert float(i.abs().max()) <= 7.0 and float(f.max()) < 0.0


def test_plain_selective_recurrence_in_closed_form():
    T, C, N = 8, 3, 4
    g = _gen(3)
    x, d = torch.randn(T, C, generator=g).double(), torch.rand(T, C, generator=g).double()
    B, Cc = torch.randn(T, N, generator=g).double(), torch.randn(T, N, generator=g).double()
    a_log, skip = torch.randn(C, N, generator=g).double(), torch.randn(C, generator=g).double()
    got = plain.selective_recurrence(x, B, Cc, d, a_log, skip)
    for t in range(T):
        for c in range(C):
            want = float(skip[c] * x[t, c])
            for s in range(t + 1):
                decay = torch.exp(-torch.exp(a_log[c]) * d[s + 1 : t + 1, c].sum())
                want += float((decay * d[s, c] * x[s, c] * B[s] * Cc[t]).sum())
            assert float(got[t, c]) == pytest.approx(want, rel=1e-9)


@pytest.mark.parametrize("taps", [1, 2, 4, 7])
@pytest.mark.parametrize("biased", [True, False])
def test_plain_convolution_through_torch(taps, biased):
    g = _gen(4)
    u, w, b = torch.randn(11, 6, generator=g).double(), torch.randn(6, taps, generator=g).double(), torch.randn(6, generator=g).double()
    padded = torch.nn.functional.pad(u.t()[None], (taps - 1, 0))
    want = torch.nn.functional.conv1d(padded, w[:, None], b if biased else None, groups=6)[0].t()
    torch.testing.assert_close(plain.causal_conv(u, w, b if biased else None), want)


def test_plain_attention_through_torch():
    m = {"heads": 6, "kv_heads": 2, "dim": 8, "vdim": 5, "scale": 0.4, "rot": {"base": 30.0, "dims": 4}}
    g, W, T, taps = _gen(5), 12, 9, 3
    shapes = {"q": (48, W), "k": (16, W), "v": (10, W), "g": (6, W), "o": (W, 30), "q.norm": (48,), "k.norm": (16,), "q.conv": (48, taps),
              "k.conv": (16, taps), "v.conv": (10, taps)}
    w = {k: torch.randn(s, generator=g).double() for k, s in shapes.items()}
    h = torch.randn(T, W, generator=g).double()
    conv = {n: torch.nn.functional.conv1d(torch.nn.functional.pad((h @ w[n].t()).t()[None], (taps - 1, 0)), w[n + ".conv"][:, None],
                                          groups=w[n].shape[0])[0].t() for n in "qkv"}
    q, k = (torch.nn.functional.rms_norm(conv[n], (conv[n].shape[1],), w[n + ".norm"], eps=1e-5) for n in "qk")
    angle = torch.arange(T).double()[:, None] * torch.tensor([1.0, 30.0 ** -0.5]).double()

    def turn(x):
        first = torch.complex(x[..., :2].contiguous(), x[..., 2:4].contiguous()) * torch.polar(torch.ones_like(angle), angle)[:, None]
        return torch.cat([first.real, first.imag, x[..., 4:]], -1)

    q, k, v = turn(q.view(T, 6, 8)), turn(k.view(T, 2, 8)), conv["v"].view(T, 2, 5)
    out = torch.nn.functional.scaled_dot_product_attention(q.transpose(0, 1), k.repeat_interleave(3, 1).transpose(0, 1),
                                                           v.repeat_interleave(3, 1).transpose(0, 1), is_causal=True, scale=0.4)
    want = (out.transpose(0, 1) * torch.sigmoid(h @ w["g"].t())[..., None]).reshape(T, 30) @ w["o"].t()
    torch.testing.assert_close(plain.grouped_attention(h, w, "", m, 1e-5), want)


def test_plain_rotation_with_yarn_scales_what_turns_only():
    rot = {"base": 100.0, "dims": 4, "scaling": {"factor": 5.0, "original": 16, "fast": 4.0, "slow": 1.0}}
    v = torch.randn(3, 2, 6, generator=_gen(6)).double()
    turned = plain.rotate_halves(v, [0, 7, 2], rot)
    assert torch.equal(turned[..., 4:], v[..., 4:])
    torch.testing.assert_close(turned[..., :4].norm(dim=-1), v[..., :4].norm(dim=-1) * (0.1 * math.log(5.0) + 1.0))
    torch.testing.assert_close(turned[0, :, :4], v[0, :, :4] * (0.1 * math.log(5.0) + 1.0))


def test_plain_router_by_brute_force():
    g = _gen(7)
    w = {"router": torch.randn(6, 5, generator=g).double(), "router.b": torch.randn(6, generator=g).double() * 2}
    h = torch.randn(30, 5, generator=g).double()
    chosen, weight = plain.routed_choice(h, w, "", 3)
    for t in range(30):
        z = w["router"] @ h[t] + w["router.b"]
        best = max(itertools.combinations(range(6), 3), key=lambda es: sum(float(z[e]) for e in es))
        assert sorted(chosen[t].tolist()) == sorted(best)
        torch.testing.assert_close(weight[t], torch.exp(z[chosen[t]]) / torch.exp(z[chosen[t]]).sum())
    assert float(weight.sum(1).sub(1).abs().max()) < 1e-12


def test_plain_feed_forwards():
    g = _gen(8)
    w = {n: torch.randn(s, generator=g).double() for n, s in (("gate", (3, 4)), ("up", (3, 4)), ("down", (4, 3)))}
    h = torch.randn(7, 4, generator=g).double()
    torch.testing.assert_close(plain.relu_feed_forward(h, w, ""), (torch.relu(h @ w["gate"].t()) * (h @ w["up"].t())) @ w["down"].t())
    torch.testing.assert_close(plain.silu_expert(h, w, ""), (torch.nn.functional.silu(h @ w["gate"].t()) * (h @ w["up"].t())) @ w["down"].t())


def test_plain_model_moves_with_earlier_tokens_only(tmp_path):
    model = plain.PlainTufevik(write_random_model(tmp_path / "m", TUFEVIK_A, 3))
    base = model.streams([1, 2, 3, 4, 5, 6])
    assert base.shape == (4, 6, 96)
    other = model.streams([1, 2, 9, 4, 5, 6])
    assert torch.equal(base[:, :2], other[:, :2]) and float((base[:, 2:] - other[:, 2:]).abs().amax(dim=(0, 2)).min()) > 0
