"""Tufevik on the GPU against the plain implementation (tests/plain/tufevik_plain.py): each new
mechanism alone (the matrix memory over many sizes whole, in portions down to two tokens and token by token,
under gates that push its maximum up, down and to the cap, its state carried over hundreds of tokens; the
selective scan likewise; attention behind a convolution with whole-projection norms and YaRN rotation, a far
key among hundreds, a loud token in the convolutions; the pair of mixers with and without shared products;
the ReLU-gated feed-forward in every product; the router's bias; a branch's Dynamic Tanh as it joins with
each kind of branch, and the block), then whole models of four small configurations replayed whole, as
prefill then single tokens, in portions and as mixed batches on tight page pools and few state slots, in
both dtypes; models drawn at random; long decoding as graph replays; forks; greedy generation through the
engine's entry point, the command line and the trace program."""

import json
import subprocess
import sys
from pathlib import Path
from types import SimpleNamespace

import pytest
import torch

from clockwork_amd import ops
from clockwork_amd.parts.base import EntryCache
from clockwork_amd.parts.specs import (DynamicTanhSpec, GatedAttentionSpec, GatedMLPSpec, MatrixMemorySpec, PairMixerSpec, RMSNormSpec,
                                       RopeNeoxSpec, RoutedExpertsSpec, SelectiveScanSpec, YarnSpec)
from clockwork_amd.registry import build_arrangement, build_part
from tests import replay
from tests.configs import TUFEVIK_CONFIGS, random_tufevik_config
from tests.plain import tufevik_plain as plain
from tests.test_gpu_fuvavik import _step_through, bind, close

pytestmark = pytest.mark.gpu
DEV = "cuda"
REPO = Path(__file__).resolve().parents[1]
EPS = 1e-5
BOTH = pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])


def close_rows(got, want, dtype, worst=5e-4):
    """For a mixer that divides by its own sums (the memory's denominator, a head's root mean square): where
    those nearly cancel a row is ill-conditioned, so the errors are held by their distribution over the
    rows, each row's largest error against the outputs' scale."""
    assert not torch.isnan(got).any()
    rows = (got - want).abs().amax(dim=1) / float(want.square().mean().sqrt())
    half, most, last = float(rows.quantile(0.5)), float(rows.quantile(0.9)), float(rows.max())
    if dtype == torch.float32:
        assert half < 1e-5 and most < 5e-5 and last < worst, (half, most, last)
    else:
        assert half < 4e-2 and most < 1e-1, (half, most, last)


def step_batches(part, xs, steps, dtype, block_size=8, num_blocks=60, slots=None):
    """Requests ``xs`` ({name: [T, hidden]}) through one mixer in steps of several requests each ({name: tokens}),
    NaN-poisoned pools, slots for ``slots`` of them at a time; returns {name: outputs}."""
    from clockwork_amd.cache import CacheManager, plan_groups
    from clockwork_amd.cache.pools import CachePools
    from clockwork_amd.engine.batch import StepEntry, build_context

    groups = plan_groups([part.cache_need()])
    slots = slots or len(xs)
    manager = CacheManager(groups, block_size, num_blocks, max_num_seqs=slots)
    pools = CachePools(groups, block_size, num_blocks, slots, dtype, torch.device(DEV), fill=float("nan"))
    cache = pools.entry_cache(0)
    at, got = {n: 0 for n in xs}, {n: [] for n in xs}
    for step in steps:
        entries = []
        for n, k in step.items():
            if at[n] == 0:
                manager.admit(n, k)
            manager.extend(n, at[n], at[n] + k)
            entries.append(StepEntry(n, at[n], [0] * k))
        ctx = build_context(entries, manager, torch.device(DEV), 10)
        if pools.state:
            pools.set_fresh_states(ctx.state_slots, ctx.starts, ctx.num_requests)
        out = part.forward(torch.cat([xs[n][at[n] : at[n] + k] for n, k in step.items()]).to(dtype).to(DEV), ctx, cache).double().cpu()
        row = 0
        for n, k in step.items():
            got[n].append(out[row : row + k])
            row += k
            at[n] += k
            if at[n] == len(xs[n]):
                manager.free(n)
    assert all(at[n] == len(xs[n]) for n in xs)
    return {n: torch.cat(g) for n, g in got.items()}


# unequal requests in one step, portions beside single tokens; "d" takes a slot that another one gave back
UNEQUAL = {"a": 140, "b": 90, "c": 33, "d": 70}
UNEQUAL_STEPS = [{"a": 70, "b": 1, "c": 2}, {"a": 1, "b": 66, "c": 30}, {"a": 1, "b": 1, "c": 1}, {"a": 2, "b": 20, "d": 1}, {"b": 2, "d": 65},
                 {"a": 64, "d": 1}, {"a": 2, "d": 3}]


def unequal_inputs(hidden, dtype, seed=10):
    gen = torch.Generator().manual_seed(seed)
    return {n: torch.randn(L, hidden, generator=gen).to(dtype) for n, L in UNEQUAL.items()}


# ------------------------------------------------------------------------------- the matrix memory
def _mm_spec(hidden, heads, dim, vdim, cap=15.0):
    return MatrixMemorySpec(hidden_size=hidden, num_heads=heads, key_dim=dim, value_dim=vdim, gate_cap=cap, norm_eps=EPS)


def _mm_names(w, s):
    qk, v, m = s.num_heads * s.key_dim, s.num_heads * s.value_dim, w["in_weight"]
    return {"q": m[:qk], "k": m[qk : 2 * qk], "v": m[2 * qk : 2 * qk + v], "g": m[2 * qk + v :], "i": w["gate_weight"][: s.num_heads],
            "f": w["gate_weight"][s.num_heads :], "i.b": w["gate_bias"][: s.num_heads], "f.b": w["gate_bias"][s.num_heads :],
            "norm": w["norm_weight"], "o": w["out_weight"]}


def _mm_sizes(s):
    return {"heads": s.num_heads, "dim": s.key_dim, "vdim": s.value_dim, "gate_cap": s.gate_cap}


def _mm_want(x, w, spec):
    return plain.mlstm(x.double(), _mm_names(w, spec), "", _mm_sizes(spec), EPS)


# hidden, heads, dim, vdim: odd sizes, more value columns than a workgroup's, keys of a whole tile and not,
# chunks of 64, (float32, long keys) 32 and 16 tokens, more heads than a tile of gate rows
MM_SHAPES = [(64, 4, 16, 24), (100, 3, 10, 7), (96, 2, 64, 128), (72, 5, 33, 65), (64, 1, 256, 80), (128, 2, 128, 256), (40, 40, 4, 3), (64, 2, 8, 300), (264, 3, 200, 20)]


@BOTH
@pytest.mark.parametrize("shape", MM_SHAPES)
def test_the_matrix_memory_whole_in_portions_and_token_by_token(dtype, shape):
    spec = _mm_spec(*shape)
    part = build_part(spec)
    w = bind(part, dtype, seed=shape[1] + shape[3], matrix_std=0.2)
    T = 150
    x = torch.randn(T, spec.hidden_size, generator=torch.Generator().manual_seed(7)).to(dtype)
    want = _mm_want(x, w, spec)
    for cuts in ([T], [5, 1, 1, 17, 2, 70, 2, 52], [100] + [1] * 50, [2] * 75, [64, 64, 22], [1] * 33 + [117]):
        close_rows(_step_through(part, part.cache_need(), x, cuts, dtype), want, dtype, worst=3e-3)


@pytest.mark.parametrize("split_units", [1, 8, 1000])
def test_single_tokens_with_a_heads_columns_shared_among_workgroups(split_units):
    spec = _mm_spec(64, 3, 40, 64)
    part = build_part(spec)
    w = bind(part, torch.float32, seed=2, matrix_std=0.2)
    x = torch.randn(40, 64, generator=torch.Generator().manual_seed(3))
    close_rows(_step_through(part, part.cache_need(), x, [1] * 40, torch.float32, compute_units=split_units), _mm_want(x, w, spec), torch.float32)


@pytest.mark.parametrize("i_bias, f_bias", [(-40.0, 3.0), (40.0, 3.0), (0.0, -40.0), (0.0, 40.0), (-40.0, -40.0), (40.0, -40.0), (3.0, -1.0)])
def test_the_running_maximum_under_gates_at_their_ends(i_bias, f_bias):
    """Input gates far below zero (the maximum is that of the start, falling with the forget gates, and e^(-m)
    is the denominator), far above (it is the input's), forget gates that keep or drop everything."""
    spec = _mm_spec(48, 2, 12, 10, cap=6.0)
    part = build_part(spec)

    def change(values):
        values["gate_bias"] = torch.tensor([i_bias] * 2 + [f_bias] * 2)

    w = bind(part, torch.float32, seed=4, matrix_std=0.3, change=change)
    T = 200
    x = torch.randn(T, 48, generator=torch.Generator().manual_seed(5))
    want = _mm_want(x, w, spec)
    for cuts in ([T], [64, 1, 1, 70, 2, 62], [100] + [1] * 100):
        close_rows(_step_through(part, part.cache_need(), x, cuts, torch.float32), want, torch.float32, worst=3e-3)


def test_an_early_token_with_a_strong_input_gate_stays_and_a_weak_forget_gate_drops_it():
    """Token 2 writes with the largest input gate; with forget gates near one it is read 400 tokens later, with
    small ones nothing of it is left."""
    moved = {}
    for f_bias in (12.0, -2.0):
        spec = _mm_spec(32, 1, 8, 8)
        part = build_part(spec)

        def change(values, f_bias=f_bias):
            values["gate_weight"] = torch.zeros_like(values["gate_weight"])
            values["gate_weight"][0, 0] = 8.0           # the input gate reads element 0
            values["gate_bias"] = torch.tensor([-4.0, f_bias])

        w = bind(part, torch.float32, seed=3, matrix_std=0.3, change=change)
        T = 420
        x = torch.randn(T, 32, generator=torch.Generator().manual_seed(8)) * 0.5
        x[:, 0] = 0.0
        x[2, 0] = 1.0
        want = _mm_want(x, w, spec)
        for cuts in ([T], [150, 2, 268], [300] + [1] * 120):
            close_rows(_step_through(part, part.cache_need(), x, cuts, torch.float32), want, torch.float32, worst=3e-3)
        other = x.clone()
        other[2, 1:] += 3.0
        moved[f_bias] = float((_mm_want(other, w, spec) - want)[410:].abs().max())
    assert moved[12.0] > 1e-2 and moved[-2.0] < 1e-9


@BOTH
def test_matrix_memories_of_unequal_requests_in_one_step_equal_each_alone(dtype):
    spec = _mm_spec(64, 4, 32, 48)
    part = build_part(spec)
    w = bind(part, dtype, seed=9, matrix_std=0.2)
    xs = unequal_inputs(64, dtype)
    got = step_batches(part, xs, UNEQUAL_STEPS, dtype, slots=3)
    for n, x in xs.items():
        close_rows(got[n], _mm_want(x, w, spec), dtype, worst=3e-3)


def test_keys_beyond_the_memorys_kernels_are_refused():
    with pytest.raises(ValueError):
        bind(build_part(_mm_spec(32, 1, 257, 8)), torch.float32)


# ------------------------------------------------------------------------------- the selective scan
def _scan_spec(hidden, inner, state, rank, taps):
    return SelectiveScanSpec(hidden_size=hidden, inner=inner, state_dim=state, dt_rank=rank, conv_taps=taps)


def _scan_names(w, pre=""):
    return {pre + n: w[k] for n, k in {"in": "in_weight", "conv": "conv_weight", "conv.b": "conv_bias", "x": "low_weight", "dt": "dt_weight",
                                       "dt.b": "dt_bias", "A_log": "a_log", "D": "skip", "o": "out_weight"}.items()}


def _scan_sizes(s):
    return {"inner": s.inner, "state": s.state_dim, "dt_rank": s.dt_rank, "conv": s.conv_taps}


def _scan_want(x, w, spec):
    return plain.selective_scan(x.double(), _scan_names(w), "", _scan_sizes(spec))


# hidden, inner, states, rank, taps: sizes of 1, odd ones, states that one wave holds and that two, three and
# sixteen share, channels that are no multiple of 64, ranks that are no multiple of 8
SCAN_SHAPES = [(64, 96, 16, 8, 4), (100, 33, 7, 3, 1), (48, 1, 1, 1, 2), (72, 130, 40, 24, 5), (64, 256, 32, 16, 3), (40, 70, 256, 10, 4), (64, 64, 100, 100, 17), (64, 512, 8, 40, 2)]


@BOTH
@pytest.mark.parametrize("shape", SCAN_SHAPES)
def test_the_selective_scan_whole_in_portions_and_token_by_token(dtype, shape):
    spec = _scan_spec(*shape)
    part = build_part(spec)
    w = bind(part, dtype, seed=shape[1] + shape[2], matrix_std=0.2)
    T = 150
    x = torch.randn(T, spec.hidden_size, generator=torch.Generator().manual_seed(7)).to(dtype)
    want = _scan_want(x, w, spec)
    for cuts in ([T], [5, 1, 1, 17, 2, 70, 2, 52], [100] + [1] * 50, [2] * 75, [64, 64, 22]):
        close_rows(_step_through(part, part.cache_need(), x, cuts, dtype), want, dtype)


def test_long_portions_of_the_scan_are_cut_into_longer_segments():
    spec = _scan_spec(32, 80, 16, 8, 4)
    part = build_part(spec)
    w = bind(part, torch.float32, seed=1, matrix_std=0.2)
    x = torch.randn(1200, 32, generator=torch.Generator().manual_seed(2))
    close_rows(_step_through(part, part.cache_need(), x, [1100, 40, 60], torch.float32), _scan_want(x, w, spec), torch.float32)


def test_the_scans_state_keeps_a_token_from_far_back_and_forgets_by_its_decay():
    moved = {}
    for a_log in (-12.0, 4.0):
        spec = _scan_spec(32, 24, 8, 6, 2)
        part = build_part(spec)

        def change(values, a_log=a_log):
            values["a_log"] = torch.full_like(values["a_log"], a_log)
            values["dt_bias"] = torch.full_like(values["dt_bias"], 0.5)

        w = bind(part, torch.float32, seed=3, matrix_std=0.3, change=change)
        T = 420
        x = torch.randn(T, 32, generator=torch.Generator().manual_seed(8))
        want = _scan_want(x, w, spec)
        for cuts in ([T], [150, 2, 268], [300] + [1] * 120):
            close_rows(_step_through(part, part.cache_need(), x, cuts, torch.float32), want, torch.float32)
        other = x.clone()
        other[2] += 3.0
        moved[a_log] = float((_scan_want(other, w, spec) - want)[410:].abs().max())
    assert moved[-12.0] > 1e-2 and moved[4.0] < 1e-9


def test_tiny_and_huge_steps_of_the_scan():
    """Steps from 1e-9 to hundreds: the softplus keeps its digits at both ends."""
    for bias in (-20.0, -8.0, 0.0, 90.0):
        spec = _scan_spec(32, 40, 4, 4, 2)
        part = build_part(spec)

        def change(values, bias=bias):
            values["dt_bias"] = torch.full_like(values["dt_bias"], bias)
            values["skip"] = torch.zeros_like(values["skip"])
            values["a_log"] = torch.full_like(values["a_log"], -6.0)

        w = bind(part, torch.float32, seed=6, matrix_std=0.3, change=change)
        x = torch.randn(60, 32, generator=torch.Generator().manual_seed(9))
        want = _scan_want(x, w, spec)
        for cuts in ([60], [1] * 60):
            got = _step_through(part, part.cache_need(), x, cuts, torch.float32)
            assert float((got - want).abs().max()) < 3e-5 * float(want.abs().max()), bias


@BOTH
def test_scans_of_unequal_requests_in_one_step_equal_each_alone(dtype):
    spec = _scan_spec(64, 96, 24, 8, 4)
    part = build_part(spec)
    w = bind(part, dtype, seed=9, matrix_std=0.2)
    xs = unequal_inputs(64, dtype)
    got = step_batches(part, xs, UNEQUAL_STEPS, dtype, slots=3)
    for n, x in xs.items():
        close_rows(got[n], _scan_want(x, w, spec), dtype)


def test_sizes_beyond_the_scans_kernels_are_refused_by_name():
    for bad in (_scan_spec(32, 8, 257, 2, 2), _scan_spec(32, 8, 4, 2, 18)):
        with pytest.raises(ValueError):
            bind(build_part(bad), torch.float32)


# ------------------------------------------------------------------------------- attention behind a convolution
def _attn_spec(hidden, heads, kv_heads, dim, vdim, taps, rot=0, base=100.0, yarn=None, scale=0.3, **kw):
    position = RopeNeoxSpec(rot, base, YarnSpec(*yarn) if yarn else None) if rot else None
    options = dict(qk_norm=True, qk_norm_over="projection", output_gate=True, gate_per_head=True)
    options.update(kw)
    return GatedAttentionSpec(hidden_size=hidden, num_heads=heads, num_kv_heads=kv_heads, key_dim=dim, value_dim=vdim, scale=scale, norm_eps=EPS,
                              conv_taps=taps, position=position, **options)


def _attn_names(w, s, pre=""):
    nq, nk, nv = s.num_heads * s.key_dim, s.num_kv_heads * s.key_dim, s.num_kv_heads * s.value_dim
    m = w["in_weight"]
    at = [0, nq, nq + nk, nq + nk + nv, nq + nk + nv + s.num_heads]
    names = {n: m[a:b] for n, a, b in zip("qkvg", at, at[1:])}
    c = w["conv_weight"] if s.conv_taps else torch.ones(at[3], 1, dtype=torch.float64)
    names.update({"q.conv": c[:nq], "k.conv": c[nq : nq + nk], "v.conv": c[nq + nk :], "o": w["out_weight"], "q.norm": w["q_norm"],
                  "k.norm": w["k_norm"]})
    return {pre + k: v for k, v in names.items()}


def _attn_sizes(s):
    rot = {"base": 10.0, "dims": 0}
    if s.position is not None:
        rot = {"base": s.position.theta, "dims": s.position.rotary_dim}
        y = s.position.scaling
        if y is not None:
            rot["scaling"] = {"factor": y.factor, "original": y.original, "fast": y.fast, "slow": y.slow}
    return {"heads": s.num_heads, "kv_heads": s.num_kv_heads, "dim": s.key_dim, "vdim": s.value_dim, "scale": s.scale, "rot": rot}


def _attn_want(x, w, spec):
    return plain.grouped_attention(x.double(), _attn_names(w, spec), "", _attn_sizes(spec), EPS)


YARN = (4.0, 32, 8.0, 1.0)
# hidden, heads, kv heads, dim, vdim, taps, rotated elements: heads of the kernels for plain grouped
# attention (with values of the keys' size), of the matrix-core kernel for paged rows, of neither; no
# convolution, one tap, more taps than a work item's tokens, rotation of a part, all and none
ATTN_SHAPES = [(64, 4, 2, 32, 32, 4, 32), (64, 8, 2, 64, 64, 3, 16), (96, 2, 1, 128, 128, 2, 128), (64, 4, 1, 64, 128, 4, 32), (100, 3, 3, 10, 7, 5, 6), (72, 6, 2, 24, 40, 1, 0),
               (64, 4, 4, 16, 16, 9, 16), (48, 1, 1, 1, 1, 3, 0), (64, 2, 2, 96, 96, 17, 48), (64, 6, 3, 48, 16, 0, 12)]


@BOTH
@pytest.mark.parametrize("shape", ATTN_SHAPES)
def test_convolved_attention_whole_in_portions_and_token_by_token(dtype, shape):
    spec = _attn_spec(*shape, yarn=YARN if shape[6] else None)
    part = build_part(spec)
    w = bind(part, dtype, seed=shape[1], matrix_std=0.15)
    T = 75
    x = torch.randn(T, spec.hidden_size, generator=torch.Generator().manual_seed(4)).to(dtype)
    want = _attn_want(x, w, spec)
    for cuts in ([T], [5, 1, 1, 17, 2, 1, 2, 46], [1] * T, [2] * 37 + [1]):
        close(_step_through(part, part.cache_need(), x, cuts, dtype), want, dtype)


@BOTH
@pytest.mark.parametrize("dim, vdim", [(64, 64), (24, 40)])
def test_convolved_attention_of_unequal_requests_in_one_step(dtype, dim, vdim):
    spec = _attn_spec(64, 4, 2, dim, vdim, 4, 16, yarn=YARN)
    part = build_part(spec)
    w = bind(part, dtype, seed=9, matrix_std=0.15)
    xs = unequal_inputs(64, dtype)
    got = step_batches(part, xs, UNEQUAL_STEPS, dtype, slots=3)
    for n, x in xs.items():
        close(got[n], _attn_want(x, w, spec), dtype)


def test_the_attention_options_each_matter():
    x = torch.randn(60, 64, generator=torch.Generator().manual_seed(6))
    base = dict(taps=3, rot=16, base=100.0, yarn=YARN, scale=0.6)
    variants = {"base": {}, "no yarn": {"yarn": None}, "factor": {"yarn": (2.0, 32, 8.0, 1.0)}, "original": {"yarn": (4.0, 500, 8.0, 1.0)},
                "slow": {"yarn": (4.0, 32, 8.0, 3.0)}, "fast": {"yarn": (4.0, 32, 2.0, 1.0)}, "rotated part": {"rot": 8}, "base of the rotation": {"base": 7.0},
                "scale": {"scale": 0.9}, "no gate": {"output_gate": False, "gate_per_head": False}}
    outs = {}
    for key, kw in variants.items():
        part = build_part(_attn_spec(64, 4, 2, 16, 16, **dict(base, **kw)))
        full = torch.randn(64 + 32 + 32 + 4, 64, generator=torch.Generator().manual_seed(1)) * 0.4

        def change(values):
            values["in_weight"] = full[: values["in_weight"].shape[0]].clone()

        bind(part, torch.float32, seed=1, matrix_std=0.4, change=change)
        outs[key] = _step_through(part, part.cache_need(), x, [60], torch.float32)
    for key in variants:
        if key != "base":
            assert float((outs[key] - outs["base"]).abs().max()) > 1e-3, key


@BOTH
@pytest.mark.parametrize("dim, vdim", [(64, 64), (64, 128), (12, 8)])
def test_a_far_key_among_hundreds(dtype, dim, vdim):
    """Position 3 holds a key that every query scores far above all others: its value is every later token's
    output, 600 tokens on, across page borders, whole, in portions and decoded."""
    spec = _attn_spec(32, 2, 1, dim, vdim, 2, 0, scale=6.0)
    part = build_part(spec)
    T = 603

    def change(v):
        for n in ("in_weight", "out_weight", "conv_weight"):
            v[n] = torch.zeros_like(v[n])
        v["conv_weight"][:, 1] = 1.0                              # the token itself
        v["q_norm"], v["k_norm"] = torch.ones_like(v["q_norm"]), torch.ones_like(v["k_norm"])
        nq = 2 * dim
        v["in_weight"][0, 0] = v["in_weight"][dim, 0] = 1.0       # every query the same direction
        v["in_weight"][nq + 1, 1] = 1.0                           # the silent tokens' key
        v["in_weight"][nq, 2] = 1.0                               # the loud token's
        for c in range(4):
            v["in_weight"][nq + dim + c, 2] = 0.25 * (c + 1)      # its value
        v["in_weight"][nq + dim + vdim :, 3] = 1.0                # gates wide open
        for a in range(2):
            for c in range(4):
                v["out_weight"][4 * a + c, a * vdim + c] = 1.0

    bind(part, dtype, change=change)
    x = torch.zeros(T, 32)
    x[:, 0], x[:, 1], x[:, 3] = 1.0, 1.0, 20.0
    x[3, 1], x[3, 2] = 0.0, 1.0
    value = 0.25 * torch.tensor([1.0, 2.0, 3.0, 4.0] * 2, dtype=torch.float64)
    for cuts in ([T], [400] + [1] * (T - 400), [100, 2, 200, 301]):
        got = _step_through(part, part.cache_need(), x, cuts, dtype, block_size=16, num_blocks=40)
        assert float(got[:3, :8].abs().max()) < 1e-6
        # (a score of 6 sqrt(dim) sqrt(2 dim) and more: the others' weight is below 1e-9)
        assert float((got[3:, :8] - value).abs().max()) < (1e-5 if dtype == torch.float32 else 2e-2)


@pytest.mark.parametrize("taps", [2, 3, 4, 5, 9])
@pytest.mark.parametrize("cuts", ["whole", "portions", "pairs", "single"])
def test_one_loud_token_in_the_convolutions_reaches_exactly_its_taps(taps, cuts):
    """The convolutions weigh only their oldest tap. In the scan (its state kept out by a strong decay) and in
    the values of an attention whose every token sees itself above all, a loud token shows taps - 1
    positions later and nowhere else."""
    T = 70
    how = {"whole": [T], "portions": [3, 9, 2, 16, 5, 2, 31, 2], "pairs": [2] * 35, "single": [1] * T}[cuts]
    scan = build_part(_scan_spec(32, 12, 4, 4, taps))

    def only_oldest(values):
        values["conv_weight"] = torch.zeros_like(values["conv_weight"])
        values["conv_weight"][:, 0] = 1.0
        if "conv_bias" in values:
            values["conv_bias"] = torch.zeros_like(values["conv_bias"])
            values["a_log"] = torch.full_like(values["a_log"], 5.0)
            values["dt_bias"] = torch.full_like(values["dt_bias"], 1.0)

    ws = bind(scan, torch.float32, seed=5, matrix_std=0.3, change=only_oldest)
    attn_spec = _attn_spec(32, 2, 1, 8, 8, taps, 8, base=2.0, scale=0.2)
    attn = build_part(attn_spec)
    wa = bind(attn, torch.float32, seed=6, matrix_std=0.3, change=only_oldest)
    quiet = torch.randn(32, generator=torch.Generator().manual_seed(1))
    for loud in (0, 1, 15, 40):
        x = torch.zeros(T, 32) + 0.01 * quiet
        x[loud] += torch.randn(32, generator=torch.Generator().manual_seed(loud)) * 5
        got = _step_through(scan, scan.cache_need(), x, how, torch.float32)
        want = _scan_want(x, ws, scan.spec)
        close(got, want, torch.float32)
        # (the gate reads the loud token itself: its own position changes too)
        changed = (want - want[-1]).abs().amax(dim=1) > 1e-3
        assert bool(changed[loud + taps - 1]) and not bool(changed[loud + taps : loud + 20].any())
        close(_step_through(attn, attn.cache_need(), x, how, torch.float32), _attn_want(x, wa, attn_spec), torch.float32)


def test_a_mixer_behind_a_convolution_does_not_borrow_a_cache():
    part = build_part(_attn_spec(64, 2, 1, 8, 8, 3, 8))
    bind(part, torch.float32)
    cache = EntryCache(members=[EntryCache(group=0, planes={}, writes=False), EntryCache()])
    with pytest.raises(NotImplementedError):
        part.forward(torch.zeros(1, 64, device=DEV), SimpleNamespace(), cache)


def test_the_short_convolution_alone_with_and_without_bias_and_silu():
    from clockwork_amd.cache import CacheManager, plan_groups
    from clockwork_amd.config.spec import StateSpec
    from clockwork_amd.engine.batch import StepEntry, build_context
    from clockwork_amd.parts.sink_attention import query_runs

    for channels, taps, off in ((8, 4, 4), (300, 3, 0), (7, 2, 3), (1, 1, 0), (2052, 4, 12), (40, 12, 8)):
        gen = torch.Generator().manual_seed(channels)
        x = torch.randn(45, off + channels + 4, generator=gen)
        weight, bias = torch.randn(channels, taps, generator=gen), torch.randn(channels, generator=gen)
        for b, silu in ((bias, True), (None, False), (bias, False), (None, True)):
            want = plain.causal_conv(x[:, off : off + channels].double(), weight.double(), None if b is None else b.double())
            want = plain.silu(want) if silu else want
            for cuts in ([45], [1] * 45, [2, 20, 1, 22]):
                manager = CacheManager(plan_groups([StateSpec((taps * channels + 5,))]), 8, 1, max_num_seqs=2)
                state = torch.zeros(3, taps * channels + 5, device=DEV)
                got, at = [], 0
                for n in cuts:
                    if at == 0:
                        manager.admit("s", n)
                    ctx = build_context([StepEntry("s", at, [0] * n)], manager, torch.device(DEV), 10)
                    items, n_items = query_runs(ctx, ops.short_conv_tokens())
                    got.append(ops.short_conv(x[at : at + n].to(DEV).contiguous(), off, channels, weight.to(DEV), None if b is None else b.to(DEV),
                                              state, 5, ctx.state_slots, ctx.cu_q, ctx.ctx_lens, items, n_items, 1, silu=silu))
                    at += n
                torch.testing.assert_close(torch.cat(got).double().cpu(), want, rtol=1e-5, atol=1e-5)
                assert float(state[:, :5].abs().max()) == 0.0   # what lies ahead of the inputs is not touched


# ------------------------------------------------------------------------------- the pair
def _pair_names(w, spec):
    left_rows = spec.left.num_heads * spec.left.key_dim + spec.left.num_kv_heads * (spec.left.key_dim + spec.left.value_dim) + spec.left.num_heads
    left = {k[5:]: v for k, v in w.items() if k.startswith("left.")}
    right = {k[6:]: v for k, v in w.items() if k.startswith("right.")}
    left["in_weight"], right["in_weight"] = w["in_weight"][:left_rows], w["in_weight"][left_rows:]
    return {**_attn_names(left, spec.left, "left."), **_scan_names(right, "right.")}


# attention sizes, scan sizes: one output product for both; columns that begin at no multiple of 16 bytes
# (two products); heads whose gates leave an odd width ahead of the scan's columns
PAIRS = [((64, 4, 2, 32, 32, 4, 32), (64, 96, 16, 8, 4)), ((64, 3, 1, 10, 7, 3, 6), (64, 33, 5, 3, 2)), ((96, 6, 2, 64, 128, 2, 64), (96, 128, 40, 12, 3)),
         ((72, 5, 5, 16, 16, 1, 0), (72, 64, 8, 8, 1))]


@BOTH
@pytest.mark.parametrize("left, right", PAIRS)
def test_the_pair_of_scaled_mixers(dtype, left, right):
    spec = PairMixerSpec(left[0], _attn_spec(*left, yarn=YARN if left[6] else None), _scan_spec(*right), scales=(0.6, 1.7))
    part = build_part(spec)
    w = bind(part, dtype, seed=7, matrix_std=0.15)
    assert part.joint and part.one_output == (dtype == torch.float32 or (left[1] * left[4] % 8 == 0 and right[1] % 8 == 0))
    sizes = {"left": _attn_sizes(spec.left), "right": _scan_sizes(spec.right), "left_scale": 0.6, "right_scale": 1.7}
    xs = unequal_inputs(left[0], dtype, seed=11)
    got = step_batches(part, xs, UNEQUAL_STEPS, dtype, slots=3)
    for n, x in xs.items():
        close(got[n], plain.parallel(x.double(), _pair_names(w, spec), "", sizes, EPS), dtype)
    x = xs["b"]
    want = plain.parallel(x.double(), _pair_names(w, spec), "", sizes, EPS)
    for cuts in ([90], [1] * 90, [30, 2, 2, 1, 55]):
        close(_step_through(part, part.cache_need(), x, cuts, dtype), want, dtype)


# ------------------------------------------------------------------------------- feed-forward
@BOTH
@pytest.mark.parametrize("hidden, ff, T", [(96, 100, 7), (100, 60, 33), (256, 512, 1), (512, 8192, 1100), (512, 4096, 40), (1536, 8960, 8), (256, 130, 300)])
def test_the_relu_gated_feed_forward(dtype, hidden, ff, T):
    """Few rows (the activation in the streaming product), some, and a long portion (in the wide-tile product)."""
    if dtype == torch.float32 and T * ff > 1000000:
        T = 90
    part = build_part(GatedMLPSpec(hidden, ff, activation="relu"))
    w = bind(part, dtype, seed=ff, matrix_std=1.5 / hidden ** 0.5)
    x = torch.randn(T, hidden, generator=torch.Generator().manual_seed(9)).to(dtype)
    names = {"gate": w["gate_up_weight"][:ff], "up": w["gate_up_weight"][ff:], "down": w["down_weight"]}
    want = plain.relu_feed_forward(x.double(), names, "")
    close(part.forward(x.to(DEV), SimpleNamespace()).double().cpu(), want, dtype)
    part.partial_ok = True
    y = part.forward(x.to(DEV), SimpleNamespace())
    close((y.sum() if isinstance(y, ops.PartialSums) else y).double().cpu(), want, dtype)


def test_the_tiled_products_with_the_relu_gate():
    x = torch.randn(200, 256, generator=torch.Generator().manual_seed(1)).to(torch.bfloat16)
    w = (torch.randn(768, 256, generator=torch.Generator().manual_seed(2)) * 0.1).to(torch.bfloat16)
    want = torch.clamp(x.double() @ w[:384].double().t(), min=0.0) * (x.double() @ w[384:].double().t())
    for wide in (None, True, False):
        got = ops.linear_tiled(x.to(DEV), w.to(DEV), swiglu=True, wide=wide, limit=ops.RELU_GATE)
        close(got.double().cpu(), want, torch.bfloat16)


def _routed_names(w, s):
    E, F, H = s.num_experts, s.intermediate_size, s.hidden_size
    gu, down = w["gate_up_weight"].view(E, 2, F, H), w["down_weight"].view(E, H, F)
    names = {"router": w["router_weight"], "router.b": w["router_bias"]}
    for e in range(E):
        names.update({f"e{e}.gate": gu[e, 0], f"e{e}.up": gu[e, 1], f"e{e}.down": down[e]})
    return names


ROUTED_SHAPES = [(96, 40, 6, 3, 61), (100, 50, 4, 4, 37), (64, 1, 1, 1, 9), (48, 24, 8, 1, 130), (128, 72, 16, 4, 3), (72, 33, 40, 6, 20), (256, 256, 2, 2, 600), (256, 320, 3, 2, 500)]


@BOTH
@pytest.mark.parametrize("shape", ROUTED_SHAPES)
def test_routed_experts_with_a_bias_on_the_router(dtype, shape):
    hidden, ff, experts, top, T = shape
    spec = RoutedExpertsSpec(hidden_size=hidden, intermediate_size=ff, num_experts=experts, top_k=top, router="softmax", renormalize=True,
                             weight_on="output", router_bias=True)
    part = build_part(spec)

    def change(values):
        # biases that decide: far apart, so that rounding flips no choice
        values["router_bias"] = torch.randperm(experts, generator=torch.Generator().manual_seed(1)).float() * 1.5 - 2.0
        values["router_weight"] *= 0.2 if dtype == torch.bfloat16 else 1.0
        if dtype == torch.bfloat16:
            values["router_weight"] *= 0.1

    w = bind(part, dtype, seed=experts, matrix_std=2.0 / hidden ** 0.5, change=change)
    x = torch.randn(T, hidden, generator=torch.Generator().manual_seed(9)).to(dtype)
    names = _routed_names(w, spec)
    chosen, weight = plain.routed_choice(x.double(), names, "", top)
    xd = x.to(DEV)
    choice, score = part.route(xd)
    assert torch.equal(choice.cpu().long(), chosen)
    torch.testing.assert_close(score.double().cpu(), weight, rtol=2e-2 if dtype == torch.bfloat16 else 1e-4, atol=1e-6)
    want = plain.routed_feed_forward(x.double(), names, "", {"router": {"top": top}})
    close(part.forward(xd, SimpleNamespace()).double().cpu(), want, dtype)
    pairs = part.forward_pairs(xd, SimpleNamespace())
    close(pairs.value().double().cpu(), want, dtype)
    # the bias is part of the choice
    part.router_bias = torch.zeros_like(part.router_bias)
    if experts > top:
        assert not torch.equal(part.route(xd)[0], choice)


# ------------------------------------------------------------------------------- a branch's norm as it joins, the block
def _tanh_pair(H, dtype, seed=3):
    a, b = build_part(DynamicTanhSpec(H)), build_part(DynamicTanhSpec(H))
    wa, wb = bind(a, dtype, seed=seed), bind(b, dtype, seed=seed + 1)
    return a, b, *({"n": w["weight"], "n.b": w["bias"], "n.alpha": w["alpha"]} for w in (wa, wb))


@BOTH
@pytest.mark.parametrize("H, T", [(96, 5), (100, 37), (1, 3), (1536, 9), (2052, 70), (5001, 4)])
def test_a_branch_is_normed_as_it_joins_and_the_stream_behind_it(dtype, H, T):
    """A plain branch, one in float32 parts, a routed one of one and of six experts a token, with and without
    an always-used row; all rows, and chosen rows that leave the stream alone."""
    post, pre, wp, wn = _tanh_pair(H, dtype)
    gen = torch.Generator().manual_seed(H)
    resid = torch.randn(T, H, generator=gen) * 2
    x, a = (torch.randn(T, H, generator=gen).to(dtype) for _ in range(2))
    planes = torch.randn(6, T, H, generator=gen)
    branches = [(a.to(DEV), a.double()), (ops.PartialSums(planes.to(DEV)), planes.double().sum(0)), (ops.PartialSums(planes[:1].contiguous().to(DEV)), planes[0].double())]
    for top in (1, 6):
        y = torch.randn(T * top, H, generator=gen).to(dtype)
        choice, score = torch.zeros(T, top, dtype=torch.int32), torch.ones(T, top)
        for always in (None, a):
            value = y.double().view(T, top, H).sum(1) + (0 if always is None else always.double())
            branches.append((ops.RoutedSum(x.to(DEV), y.to(DEV), choice.to(DEV), score.to(DEV), None if always is None else always.to(DEV), top, 9), value))
    tol = dict(rtol=2e-5, atol=2e-5) if dtype == torch.float32 else dict(rtol=2e-2, atol=2e-2)
    rows = torch.tensor([T - 1, 0, T // 2], dtype=torch.int32)
    for branch, value in branches:
        stream = resid.double() + plain.tanh_norm(value, wp, "n")
        want = plain.tanh_norm(stream, wn, "n")
        r = resid.to(DEV)
        out = pre.forward(r, ops.NormedBranch(branch, post), rows=rows.to(DEV))
        assert torch.equal(r.cpu(), resid)
        torch.testing.assert_close(out.double().cpu(), want[rows.long()], **tol)
        out = pre.forward(r, ops.NormedBranch(branch, post))
        torch.testing.assert_close(r.double().cpu(), stream, rtol=2e-5, atol=2e-5)
        torch.testing.assert_close(out.double().cpu(), want, **tol)
        r = resid.to(DEV)
        post.join(r, branch)
        torch.testing.assert_close(r.double().cpu(), stream, rtol=2e-5, atol=2e-5)


class _Times:
    """A mixer or feed-forward that multiplies its input: shows what a branch read."""

    def __init__(self, factor):
        self.factor = factor

    def forward(self, x, ctx, cache=None):
        return (x.float() * self.factor).to(x.dtype)


@BOTH
@pytest.mark.parametrize("with_ff", [True, False])
@pytest.mark.parametrize("lazy", [True, False])
def test_the_block_with_norms_before_and_behind_its_sublayers(dtype, with_ff, lazy):
    W, T = 96, 11
    n1b, n1, w1b, w1 = _tanh_pair(W, dtype, seed=1)
    n2b, n2, w2b, w2 = _tanh_pair(W, dtype, seed=5)
    parts = dict(mixer=_Times(2.0), mixer_norm=n1, mixer_post_norm=n1b)
    if with_ff:
        parts.update(feed_forward=_Times(-3.0), ffn_norm=n2, ffn_post_norm=n2b)
    block = build_arrangement("sandwich", **parts)
    assert set(block.parts()) == set(parts)
    x0 = torch.randn(T, W, generator=torch.Generator().manual_seed(14)) * 3
    d = torch.randn(T, W, generator=torch.Generator().manual_seed(15)).to(dtype)
    resid = x0.clone().to(DEV)
    out = block.forward(resid, ops.NormedBranch(d.to(DEV), n2b), SimpleNamespace(next_norm_accepts_normed=lazy), None)
    x = x0.double() + plain.tanh_norm(d.double(), w2b, "n")
    x = x + plain.tanh_norm(2.0 * plain.tanh_norm(x, w1, "n"), w1b, "n")
    if with_ff:
        x = x + plain.tanh_norm(-3.0 * plain.tanh_norm(x, w2, "n"), w2b, "n")
    assert (out is None) == (not lazy)
    if lazy:
        out.norm.join(resid, out.branch)
    close(resid.double().cpu(), x, dtype)


def test_a_stream_input_joins_behind_a_normed_branch():
    post, pre, wp, wn = _tanh_pair(64, torch.float32)
    gen = torch.Generator().manual_seed(2)
    resid, d, extra = (torch.randn(5, 64, generator=gen) for _ in range(3))
    r = resid.to(DEV)
    out = pre.forward(r, ops.WithStreamInput(ops.NormedBranch(d.to(DEV), post), extra.to(DEV)))
    stream = resid.double() + plain.tanh_norm(d.double(), wp, "n") + extra.double()
    close(r.double().cpu(), stream, torch.float32)
    close(out.double().cpu(), plain.tanh_norm(stream, wn, "n"), torch.float32)


def test_a_sandwich_norm_that_cannot_norm_a_branch_is_refused():
    tanh, rms = build_part(DynamicTanhSpec(8)), build_part(RMSNormSpec(8, 1e-5))
    with pytest.raises(TypeError):
        build_arrangement("sandwich", mixer=_Times(1.0), mixer_norm=rms, mixer_post_norm=tanh)


# ------------------------------------------------------------------------------- whole models
def _livelier(model_dir, settle):
    """Random weights at which the mechanisms show: peaked attention, inputs and steps of the recurrences of
    order one, branches on both sides of the tanh's bend. ``settle``: the routers scaled down and their biases
    spread far apart, so that the rounding of a bfloat16 router's input does not flip a choice (which a
    comparison of logits cannot tell from a fault)."""
    from safetensors.torch import load_file, save_file

    path = str(Path(model_dir) / "model.safetensors")
    tensors = load_file(path)
    for key, t in list(tensors.items()):
        factor = {"q": 4.0, "k": 4.0, "v": 4.0, "g": 6.0, "in": 4.0, "x": 4.0, "gate": 6.0, "up": 6.0, "down": 3.0, "o": 3.0, "embed": 20.0,
                  "router": 0.5}.get(key.split(".")[-1] if "." in key else key)
        if factor is not None:
            tensors[key] = (t.float() * factor).to(t.dtype)
        if settle and key.endswith("mlp.router"):
            tensors[key] = (tensors[key].float() * 0.1).to(t.dtype)
        if settle and key.endswith("router.b"):
            order = torch.randperm(t.numel(), generator=torch.Generator().manual_seed(t.numel())).float()
            tensors[key] = (order * 1.2 - 1.0).to(t.dtype)
    save_file(tensors, path)
    return model_dir


@pytest.fixture(scope="module")
def tufevik_dirs(tmp_path_factory):
    from clockwork_amd.weights.random_init import write_random_model

    root = tmp_path_factory.mktemp("tufevik")
    return {(name, dtype): _livelier(write_random_model(root / f"{name}_{dtype}", cfg, seed), dtype == "bfloat16")
            for name, (cfg, seed, _) in TUFEVIK_CONFIGS.items() for dtype in ("float32", "bfloat16")}


def _requests(vocab, lengths, seed):
    gen = torch.Generator().manual_seed(seed)
    return {f"q{i}": torch.randint(0, vocab, (n,), generator=gen).tolist() for i, n in enumerate(lengths)}


def _check(got, ref, dtype, float32_bound=1e-4):
    """float32: element by element, against the logits' scale. bfloat16: the distribution of the errors over
    the positions (a wrong key, state, slot or token before moves every position behind it by the scale
    itself)."""
    keys = sorted(got)
    want = torch.stack([ref[rid][pos] for rid, pos in keys]).float()
    rows = torch.stack([got[k] for k in keys])
    assert not bool(torch.isnan(rows).any()), "NaN in the logits"
    scale = float(want.square().mean().sqrt())
    per_row = (rows - want).abs().max(dim=1).values / scale
    half, most, last = float(per_row.quantile(0.5)), float(per_row.quantile(0.9)), float(per_row.max())
    text = f"errors against the scale: median {half:.2e}, nine in ten within {most:.2e}, largest {last:.2e} at {keys[int(per_row.argmax())]}"
    if dtype == "float32":
        assert last < float32_bound, text
    else:
        assert half < 8e-2 and most < 1.5e-1, text


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("mode", ["whole", "prefill_then_decode", "portions", "mixed"])
@pytest.mark.parametrize("name", list(TUFEVIK_CONFIGS))
def test_models_in_four_batching_modes(tufevik_dirs, name, mode, dtype):
    cfg, _, block_size = TUFEVIK_CONFIGS[name]
    model_dir = tufevik_dirs[(name, dtype)]
    requests = _requests(cfg["vocab"], [50, 9, 77, 30, 64, 1, 2], seed=11)
    # pages for the four longest requests and two more, four state slots: freed pages and slots are
    # used again (NaN-poisoned pools: a read outside a request's pages shows)
    runner = replay.make_runner(model_dir, dtype, block_size, replay.pages_needed(requests, 4, block_size) + 2)
    oracle = plain.PlainTufevik(model_dir)
    ref = {rid: oracle.logits(toks) for rid, toks in requests.items()}
    got = replay.run_trace(runner, getattr(replay, mode)(requests))
    assert len(got) == sum(len(t) for t in requests.values())
    _check(got, ref, dtype)
    assert not runner.manager.live_requests()
    assert all(p.num_free == runner.manager.num_blocks for p in runner.manager.pools)


@pytest.mark.parametrize("seed", range(5000, 5006))
def test_models_drawn_at_random(tmp_path, seed):
    """Models whose sizes, layer order and constants are drawn at random, six requests of 1 to 330 tokens on
    pages of 64 barely enough for four of them, as mixed batches, in portions and as prefill then single
    tokens; float32 as the model stands, bfloat16 with the experts' choice settled by the biases."""
    import random

    from clockwork_amd.weights.random_init import write_random_model

    cfg = random_tufevik_config(seed)
    rng = random.Random(seed)
    lengths = [rng.randint(100, 330), rng.randint(2, 90), rng.randint(150, 260), rng.randint(40, 200), 1, 65]
    for dtype in ("float32", "bfloat16"):
        model_dir = _livelier(write_random_model(tmp_path / dtype, cfg, seed), dtype == "bfloat16")
        requests = _requests(cfg["vocab"], lengths, seed)
        oracle = plain.PlainTufevik(model_dir)
        ref = {rid: oracle.logits(toks) for rid, toks in requests.items()}
        for mode in ("mixed", "portions", "prefill_then_decode"):
            runner = replay.make_runner(model_dir, dtype, 64, replay.pages_needed(requests, 4, 64) + 1)
            got = replay.run_trace(runner, getattr(replay, mode)(requests))
            assert len(got) == sum(len(t) for t in requests.values())
            _check(got, ref, dtype, float32_bound=3e-4)
            assert not runner.manager.live_requests()


def test_the_stream_after_every_layer(tufevik_dirs):
    cfg, _, block_size = TUFEVIK_CONFIGS["TA"]
    model_dir = tufevik_dirs[("TA", "float32")]
    runner = replay.make_runner(model_dir, "float32", block_size, 16)
    tokens = _requests(cfg["vocab"], [40], seed=2)["q0"]
    seen = []
    for layer in runner.model.layers:
        inner = layer.forward

        def forward(resid, delta, ctx, cache, inner=inner):
            out = inner(resid, delta, ctx, cache)
            x = resid.clone()
            out.norm.join(x, out.branch)
            seen.append(x.cpu())
            return out

        layer.forward = forward
    replay.run_trace(runner, replay.whole({"a": tokens}))
    want = plain.PlainTufevik(model_dir).streams(tokens)
    assert len(seen) == want.shape[0] == 4
    for got, ref in zip(seen, want):
        torch.testing.assert_close(got.double(), ref, rtol=5e-5, atol=5e-5)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["TA", "TD"])
def test_long_decoding_replays_graphs_and_equals_eager_steps(tufevik_dirs, name, dtype):
    """A prompt, then 150 single tokens, two requests side by side: with captured graphs, against the same
    steps run eagerly and against the plain implementation."""
    cfg, _, block_size = TUFEVIK_CONFIGS[name]
    model_dir = tufevik_dirs[(name, dtype)]
    requests = _requests(cfg["vocab"], [200, 170], seed=12)
    steps = [{"entries": [{"id": rid, "tokens": toks[:20], "want": [19]}], "end": []} for rid, toks in requests.items()]
    for p in range(20, 170):
        steps.append({"entries": [{"id": rid, "tokens": toks[p : p + 1], "want": [0]} for rid, toks in requests.items()], "end": []})
    steps[-1]["end"] = list(requests)
    oracle = plain.PlainTufevik(model_dir)
    ref = {rid: oracle.logits(toks[:170]) for rid, toks in requests.items()}
    results = {}
    for graphs in (True, False):
        runner = replay.make_runner(model_dir, dtype, block_size, 64, use_graphs=graphs)
        results[graphs] = replay.run_trace(runner, steps)
        if graphs:
            assert any(isinstance(v, tuple) for v in runner._graphs.values()), "no decode step was captured"
        _check(results[graphs], ref, dtype)
    # a captured step is planned for the longest context of its class and may cut the keys into other
    # runs than an eager one: in bfloat16 that moves roundings
    bound = (1e-5 if dtype == "float32" else 2e-2) * float(torch.stack(list(results[False].values())).square().mean().sqrt())
    for key, row in results[True].items():
        torch.testing.assert_close(row, results[False][key], rtol=1e-4 if dtype == "float32" else 2e-2, atol=bound)


@pytest.mark.parametrize("name", ["TA", "TC"])
def test_random_traces_with_forks(tufevik_dirs, name):
    """A fork copies matrices, sums, maxima, scan states and convolution inputs, and shares the pages; portions
    of 2 to 200 tokens and single tokens in any mix, requests left out of steps."""
    cfg = TUFEVIK_CONFIGS[name][0]
    model_dir = tufevik_dirs[(name, "float32")]
    oracle = plain.PlainTufevik(model_dir)
    for seed in range(4):
        steps, seqs = replay.random_trace(seed, cfg["vocab"], kinds=("fork",))
        block_size = (4, 8, 16)[seed % 3]
        longest = sorted((-(-len(t) // block_size) for t in seqs.values()), reverse=True)[:4]
        runner = replay.make_runner(model_dir, "float32", block_size, sum(longest) + len(seqs) + 2, max_model_len=1024)
        got = replay.run_trace(runner, steps)
        _check(got, {rid: oracle.logits(toks) for rid, toks in seqs.items()}, "float32")
        assert not runner.manager.live_requests()
        assert all(p.num_free == runner.manager.num_blocks for p in runner.manager.pools)


def test_greedy_generation_through_the_engine(tufevik_dirs):
    from clockwork_amd.config.engine import EngineConfig
    from clockwork_amd.engine.llm_engine import LLMEngine
    from clockwork_amd.engine.sequence import SamplingParams

    for name in ("TA", "TC"):
        model_dir = tufevik_dirs[(name, "float32")]
        vocab = TUFEVIK_CONFIGS[name][0]["vocab"]
        oracle = plain.PlainTufevik(model_dir)
        prompts = [[3, 14, 15, 92, 65], list(range(60, 120)), [7], list(range(40))]
        assert all(t < vocab for p in prompts for t in p)
        want = [oracle.greedy(p, 8) for p in prompts]
        cfg = EngineConfig.defaults(str(model_dir), dtype="float32", block_size=8, num_blocks=64, max_num_batched_tokens=24)
        engine = LLMEngine(cfg)
        outs = engine.generate(prompts, SamplingParams(max_tokens=8, temperature=0.0))
        assert [o.token_ids for o in outs] == want
        # once more on the same engine: pages and state slots of the first round are used again
        outs = engine.generate(prompts[::-1], SamplingParams(max_tokens=8, temperature=0.0))
        assert [o.token_ids for o in outs] == want[::-1]


def test_generation_with_preemption_starts_the_states_anew(tufevik_dirs):
    """Too few pages for all requests: some are put back and run again from their first token."""
    from clockwork_amd.config.engine import EngineConfig
    from clockwork_amd.engine.llm_engine import LLMEngine
    from clockwork_amd.engine.sequence import SamplingParams

    model_dir = tufevik_dirs[("TA", "float32")]
    oracle = plain.PlainTufevik(model_dir)
    prompts = [list(range(i, i + 20)) for i in range(0, 80, 20)]
    want = [oracle.greedy(p, 24) for p in prompts]
    cfg = EngineConfig.defaults(str(model_dir), dtype="float32", block_size=4, num_blocks=26, max_num_batched_tokens=64, watermark=0.0)
    engine = LLMEngine(cfg)
    outs = engine.generate(prompts, SamplingParams(max_tokens=24, temperature=0.0))
    assert [o.token_ids for o in outs] == want
    assert engine.stats()["num_preempted_total"] > 0


def test_the_command_line_and_the_trace_program(tufevik_dirs, tmp_path):
    model_dir = tufevik_dirs[("TB", "float32")]
    oracle = plain.PlainTufevik(model_dir)
    prompt = [5, 17, 3, 60, 1]
    out = subprocess.run([sys.executable, str(REPO / "bin" / "clockwork-generate"), "--model", str(model_dir),
                          "--set", "dtype=float32", "--prompt-ids", ",".join(map(str, prompt)), "--max-tokens", "5"],
                         capture_output=True, text=True, timeout=600)
    assert out.returncode == 0, out.stderr[-2000:]
    assert json.loads(out.stdout.splitlines()[-1])["token_ids"] == oracle.greedy(prompt, 5), out.stdout
    tokens = _requests(90, [45], seed=13)["q0"]
    lines = [json.dumps({"step": 0, "entries": [{"id": "a", "tokens": tokens[:30], "want": [0, 29]}], "end": []}),
             json.dumps({"step": 1, "entries": [{"id": "a", "tokens": tokens[30:32], "want": []}], "end": []}),
             json.dumps({"step": 2, "entries": [{"id": "a", "tokens": tokens[32:], "want": [12]}], "end": ["a"]})]
    run = subprocess.run([sys.executable, str(REPO / "bin" / "trace_run"), "--model", str(model_dir), "--dtype", "float32",
                          "--out", str(tmp_path / "out"), "--max-tokens", "64"], input="\n".join(lines) + "\n",
                         capture_output=True, text=True, timeout=600)
    assert run.returncode == 0, run.stderr[-2000:]
    assert [l for l in run.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    import numpy as np

    ref = oracle.logits(tokens)
    first = torch.from_numpy(np.fromfile(tmp_path / "out" / "0.f32", dtype="<f4").reshape(2, -1))
    last = torch.from_numpy(np.fromfile(tmp_path / "out" / "2.f32", dtype="<f4").reshape(1, -1))
    assert not (tmp_path / "out" / "1.f32").exists()
    scale = float(ref.square().mean().sqrt())
    torch.testing.assert_close(first, ref[[0, 29]], rtol=1e-4, atol=1e-4 * scale)
    torch.testing.assert_close(last, ref[[44]], rtol=1e-4, atol=1e-4 * scale)
