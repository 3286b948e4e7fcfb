"""Salolorn without a GPU: the configuration, the plain model's own mechanisms against closed forms, and the engine's host side
(parts, cache manager with pages and states for every pass of a loop, step function, scheduler) over CPU stand-ins for the
kernels, against the plain model."""
import json
import math

import pytest
import torch

import salolorn_util as U
from emulated_ops import EmulatedOps
from plain import salolorn_plain as P

from machserve_amd.config import ConfigError, SalolornConfig, config_from_dict
from machserve_amd.engine.loading import load_model

# The stand-ins leave a product of few rows as two partial sums, one of them noise of order one: 32-bit rounding of that
# noise, through sharpened softmaxes, is what this bound allows.  A key that is missing or one too many, a state that is
# lost or a sink left out is off by a hundred times more.
TOL = 5e-4
F64 = torch.float64


def loaded(model_dir, page_size=16, max_tokens=512, max_requests=4, num_pages=None):
    return load_model(model_dir, dtype="float32", device="cpu", ops=EmulatedOps(torch.float32), page_size=page_size,
                      max_tokens=max_tokens, max_requests=max_requests, use_graphs=False, num_pages=num_pages)


# ------------------------------------------------------------------ configuration
@pytest.mark.parametrize("name", sorted(U.CONFIGS_ALL))
def test_configuration_round_trip_and_plan(name):
    raw = U.CONFIGS_ALL[name]
    cfg = config_from_dict(raw)
    assert isinstance(cfg, SalolornConfig)
    assert config_from_dict(json.loads(json.dumps(cfg.to_dict()))) == cfg
    spec = cfg.to_spec()
    runs = P.runs(raw)
    assert list(spec.order) == [i for i, _ in runs]
    starts = [p for p, (_, opens) in enumerate(runs) if opens is not None]
    assert (spec.loop_steps is None and not starts) or list(spec.loop_steps.starts) == starts
    assert all(l.block == "sandwich" for l in spec.layers)
    names = [n for n, _, _ in cfg.random_tensor_plan()]
    assert len(set(names)) == len(names) and names[0] == "embed" and names[-1] == "final.norm"
    assert ("loop.step" in names) == ("loop" in raw)
    for i, layer in enumerate(raw["layers"]):
        has = lambda s: f"l{i}.{s}" in names
        assert has("norm1") and has("norm1b") and has("norm2") == has("norm2b") == has("mlp.gate") == (layer["mlp"] is not None)
        assert has("mix.q.conv") == has("mix.A_log") == (layer["type"] == "delta")
        assert has("mix.dkv.norm") == (layer["type"] == "latent_attention")
        assert has("mix.left.sink") == has("mix.right.a2.b") == (layer["type"] == "parallel")


def test_configuration_errors_name_the_key():
    def broken(change):
        raw = json.loads(json.dumps(U.CONFIGS["mixed"]))
        change(raw)
        return raw
    for match, change in [
            (r"layers\[0\]\.mixer\.conv", lambda r: r["layers"][0]["mixer"].pop("conv")),
            (r"layers\[0\]\.mixer\.heads", lambda r: r["layers"][0]["mixer"].update(kv_heads=3)),
            ("rot.dims", lambda r: r["layers"][1]["mixer"]["rot"].update(dims=6)),
            ("kv_rank", lambda r: r["layers"][1]["mixer"].update(kv_rank=0)),
            (r"mixer\.left\.mask", lambda r: r["layers"][2]["mixer"]["left"].pop("mask")),
            (r"left\.rot\.dims", lambda r: r["layers"][2]["mixer"]["left"]["rot"].update(dims=18)),
            (r"left\.heads", lambda r: r["layers"][2]["mixer"]["left"].update(kv_heads=3)),
            (r"right\.tau", lambda r: r["layers"][2]["mixer"]["right"].update(tau=0)),
            ("right_scale", lambda r: r["layers"][2]["mixer"].pop("right_scale")),
            ("mamba", lambda r: r["layers"][1].update(type="mamba")),
            (r"mlp\.kind", lambda r: r["layers"][1]["mlp"].update(kind="moe")),
            (r"mlp\.ff", lambda r: r["layers"][1]["mlp"].pop("ff")),
            ("loop.stop", lambda r: r["loop"].update(stop=6)),
            ("loop.start", lambda r: r["loop"].update(start=4)),
            ("loop.times", lambda r: r["loop"].update(times=0)),
            ("logit_scale", lambda r: r.pop("logit_scale")),
            ("norm", lambda r: r.pop("norm"))]:
        with pytest.raises(ConfigError, match=match):
            config_from_dict(broken(change))


# ------------------------------------------------------------------ the plain mechanisms against closed forms
def test_rotation_of_neighbours_and_of_halves():
    x = torch.randn(6, 2, 10, dtype=F64)
    p, i, dims = 4, 1, 6
    a = p * 100.0 ** (-2 * i / dims)
    for neighbours, (u, v) in ((True, (2, 3)), (False, (1, 4))):
        y = P.rotate(x, 100.0, dims, neighbours)
        assert torch.equal(y[..., dims:], x[..., dims:]) and torch.allclose(y[0], x[0])
        assert torch.allclose(y[..., :dims].pow(2).sum(-1), x[..., :dims].pow(2).sum(-1))
        assert torch.allclose(y[p, 1, u], x[p, 1, u] * math.cos(a) - x[p, 1, v] * math.sin(a))
        assert torch.allclose(y[p, 1, v], x[p, 1, v] * math.cos(a) + x[p, 1, u] * math.sin(a))


def test_chunks_and_sinks():
    see = P.chunk_visible(10, 4)
    assert see[3].tolist() == [True] * 4 + [False] * 6 and see[4].tolist() == [False] * 4 + [True] + [False] * 5
    s = torch.tensor([[1.0, 2.0, 50.0]], dtype=F64)
    w = P.sink_softmax(s, torch.tensor([[True, True, False]]), torch.tensor(0.5, dtype=F64))
    den = math.exp(1.0) + math.exp(2.0) + math.exp(0.5)
    assert torch.allclose(w, torch.tensor([[math.exp(1.0) / den, math.exp(2.0) / den, 0.0]], dtype=F64))


def test_the_linear_recurrence_is_a_decayed_sum_over_earlier_tokens():
    torch.manual_seed(0)
    n, H, d, dv = 7, 2, 3, 4
    q, k, v, alpha = torch.randn(n, H, d, dtype=F64), torch.randn(n, H, d, dtype=F64), torch.randn(n, H, dv, dtype=F64), torch.rand(n, H, d, dtype=F64)
    got = P.gated_linear_recurrence(q, k, v, alpha)
    for i in range(n):
        want = torch.zeros(H, dv, dtype=F64)
        for j in range(i + 1):
            decay = alpha[j + 1:i + 1].prod(0)                         # the token's own decay does not touch its own write
            want += (q[i] * decay * k[j]).sum(-1, keepdim=True) * v[j]
        assert torch.allclose(got[i], want)


def test_the_delta_rule_replaces_what_a_key_held():
    """With unit keys, no decay and step size one, reading a key back gives the value written last, whatever was there."""
    k = torch.zeros(4, 1, 3, dtype=F64)
    k[0, 0, 0] = k[1, 0, 1] = k[2, 0, 0] = k[3, 0, 2] = 1.0            # the third token writes the first one's key again
    v, one = torch.randn(4, 1, 5, dtype=F64), torch.ones(4, 1, dtype=F64)
    q = torch.zeros(4, 1, 3, dtype=F64)
    q[:, 0, 0] = 1.0
    o = P.delta_recurrence(q, k, v, one, one)
    assert torch.allclose(o[1], v[0]) and torch.allclose(o[2], v[2]) and torch.allclose(o[3], v[2])
    o = P.delta_recurrence(q, k, v, 0.25 * one, one)                   # a quarter of the way
    assert torch.allclose(o[2], 0.25 * v[0] + 0.25 * (v[2] - 0.25 * v[0]))
    o = P.delta_recurrence(q, k, v, one, 0.5 * one)                    # the decay comes before the write and the read
    assert torch.allclose(o[0], v[0]) and torch.allclose(o[1], 0.5 * v[0])


def test_convolution_ends_at_the_current_token_and_starts_from_zeros():
    x, w = torch.randn(5, 2, dtype=F64), torch.randn(2, 3, dtype=F64)
    y = P.causal_conv(x, w)
    assert torch.allclose(y[0], w[:, 2] * x[0]) and torch.allclose(y[1], w[:, 1] * x[0] + w[:, 2] * x[1])
    assert torch.allclose(y[4], w[:, 0] * x[2] + w[:, 1] * x[3] + w[:, 2] * x[4])


def test_unit_vectors_have_a_floor():
    assert torch.allclose(P.unit(torch.tensor([3.0, 4.0], dtype=F64)), torch.tensor([0.6, 0.8], dtype=F64), atol=1e-6)
    assert torch.allclose(P.unit(torch.tensor([1e-3, 0.0], dtype=F64)), torch.tensor([1 / math.sqrt(2), 0.0], dtype=F64))


def test_passes_of_a_loop_add_the_embedding_and_their_row():
    cfg = {"norm": {"eps": 1e-6}, "logit_scale": 1.0, "layers": [{}] * 3, "loop": {"start": 1, "stop": 2, "times": 3}}
    assert P.runs(cfg) == [(0, None), (1, 0), (1, 1), (1, 2), (2, None)]
    assert P.runs({"layers": [{}] * 2}) == [(0, None), (1, None)]
    # layers that leave nothing (their second norms are zeros): only the passes' own sums remain
    d = 8
    raw = U.model(d, 5, [(U.delta(1, 1, 2, 2, 2), None)], loop=(0, 1, 3))
    from machserve_amd.weights import random_tensor_dict
    t = random_tensor_dict(config_from_dict(raw), 0)
    t["l0.norm1b"] = torch.zeros(d)
    outs = []
    P.forward(t, raw, [3, 1], F64, outs)
    e, r = t["embed"][[3, 1]].double(), t["loop.step"].double()
    assert torch.allclose(outs[0], e + r[0]) and torch.allclose(outs[1], 2 * e + r[0] + r[1]) and torch.allclose(outs[2], 3 * e + r.sum(0))


def test_plain_model_whole_equals_its_prefixes(tmp_path):
    d = U.make_dir(tmp_path, "mixed", seed=1)
    w, cfg = U.read(d)
    toks = U.tokens_of(40, 97, 0)
    whole = P.forward(w, cfg, toks)
    for n in (1, 2, 7, 17, 39):
        assert torch.allclose(P.forward(w, cfg, toks[:n])[-1], whole[n - 1], atol=1e-9)


def test_mistakes_in_the_plain_model_would_show(tmp_path):
    """The tests' own power: the plain model with a mechanism changed a little is far from what it was."""
    d = U.make_dir(tmp_path, "mixed", seed=16)
    toks = U.tokens_of(60, 97, 9)
    w, cfg = U.read(d)
    want = P.forward(w, cfg, toks)

    def off(change_cfg=None, change_w=None):
        c, t = json.loads(json.dumps(cfg)), dict(w)
        if change_cfg:
            change_cfg(c)
        if change_w:
            change_w(t)
        return U.relative_error(P.forward(t, c, toks)[30:], want[30:])

    every = lambda end, f: lambda t: t.update({k: f(v) for k, v in t.items() if k.endswith(end)})
    assert off(lambda c: c["layers"][2]["mixer"]["left"]["mask"].update(size=17)) > 1e-2
    assert off(lambda c: c["layers"][2]["mixer"]["right"].update(tau=5.0)) > 1e-2
    assert off(lambda c: c["layers"][2]["mixer"].update(left_scale=0.75)) > 1e-2
    assert off(lambda c: c["layers"][1]["mixer"]["rot"].update(base=9000.0)) > 1e-4
    assert off(lambda c: c["loop"].update(times=2)) > 1e-2
    assert off(None, every(".sink", lambda v: v - 30.0)) > 1e-2
    assert off(None, every(".dt_bias", lambda v: v - 30.0)) > 1e-2          # no decay
    assert off(None, every("mix.q.conv", lambda v: torch.roll(v, 1, 1))) > 1e-2
    assert off(None, every("loop.step", lambda v: v[[0, 0, 0]])) > 1e-2
    # a state that is lost: what the last tokens see when the sequence starts later
    assert U.relative_error(P.forward(w, cfg, toks[20:])[-5:], want[-5:]) > 1e-2


# ------------------------------------------------------------------ the engine's host side over CPU stand-ins
@pytest.mark.parametrize("name", sorted(U.CONFIGS))
def test_any_cut_of_a_prompt_equals_the_plain_model(tmp_path, name):
    d = U.make_dir(tmp_path, name, seed=3)
    n = 60 if name != "wide" else 30
    toks = U.tokens_of(n, U.CONFIGS[name]["vocab"], 5)
    want = U.plain_logits(d, toks)
    lm = loaded(d)
    for what, schedule in {"whole": [[("a", n)]], "token by token": [[("a", 1)]] * n,
                           "portions down to two tokens": U.cut("a", n, [2, 17, 3, 2, 16, 1, 1, 15, 2])}.items():
        got = U.run_schedule(lm, {"a": toks}, schedule)["a"]
        assert U.relative_error(got, want) < TOL, what
    lm.cache.check()


def test_unequal_requests_side_by_side_with_pages_and_slots_used_again(tmp_path):
    d = U.make_dir(tmp_path, "mixed", seed=4)
    reqs = {"a": U.tokens_of(50, 97, 1), "b": U.tokens_of(1, 97, 2), "c": U.tokens_of(33, 97, 3), "d": U.tokens_of(40, 97, 4)}
    schedule = [[("b", 1), ("a", 17), ("c", 3)], [("a", 1), ("c", 30)], [("a", 2), ("d", 15)], [("a", 1), ("d", 1)], [("a", 29), ("d", 24)]]
    lm = loaded(d, max_requests=3, num_pages=8)
    got = U.run_schedule(lm, reqs, schedule)
    for i, toks in reqs.items():
        assert U.relative_error(got[i], U.plain_logits(d, toks)) < TOL, i
    lm.cache.check()
    assert all(g.pool.available() == g.pool.num_pages for g in lm.cache.groups.values())


def test_every_pass_of_a_loop_has_pages_and_states_of_its_own(tmp_path):
    lm = loaded(U.make_dir(tmp_path, "mixed", seed=6))
    assert lm.model.order == [0, 1, 2, 3, 1, 2, 3, 1, 2, 3, 4] and len(lm.model.blocks) == 5
    groups = {g.spec.window: sorted(run for run, _ in g.spec.layers) for g in lm.cache.groups.values()}
    assert groups == {None: [1, 4, 7, 10], 16: [2, 5, 8]}                   # all keys; a chunk of them
    at = lambda p, what: (lm.device_cache.binding(p)[1] if isinstance(lm.device_cache.binding(p), list) else lm.device_cache.binding(p)).tensors[what].data_ptr()
    assert len({at(p, "kv") for p in (0, 2, 3, 5, 6, 8, 9)}) == 7           # linear attention's and the delta rule's states
    assert len({at(p, "conv") for p in (0, 3, 6, 9)}) == 4


def test_a_rank_of_the_checkpoints_own(tmp_path):
    """config.json does not name the rank of the decays' bottleneck: it is that of the tensors, and the two must fit."""
    from safetensors.torch import load_file, save_file
    d = U.make_dir(tmp_path, "once", seed=5, rank=3)
    toks = U.tokens_of(25, 80, 1)
    got = U.run_schedule(loaded(d), {"a": toks}, [[("a", 20)]] + [[("a", 1)]] * 5)["a"]
    assert U.relative_error(got, U.plain_logits(d, toks)) < TOL
    path = d + "/model.safetensors"
    w = load_file(path)
    w["l2.mix.right.a1"] = torch.zeros(4, 64)
    save_file(w, path)
    with pytest.raises(ValueError, match="bottleneck"):
        loaded(d)


def test_greedy_generation_through_the_scheduler(tmp_path):
    from machserve_amd.engine import Engine
    d = U.make_dir(tmp_path, "mixed", seed=8)
    w, cfg = U.read(d)
    prompts = [U.tokens_of(n, 97, n) for n in (5, 19, 1, 30)]
    lm = loaded(d, max_requests=3, max_tokens=256)
    engine = Engine(lm, max_batch_tokens=24, chunk_size=8, max_running=3, freeze_gc=False)
    got = engine.generate(prompts, max_new=5)
    for p, g in zip(prompts, got):
        assert g == P.greedy_generate(w, cfg, p, 5, torch.float64)
    lm.cache.check()


def test_a_layer_without_feed_forward_may_bring_its_unused_norms(tmp_path):
    from safetensors.torch import load_file, save_file
    from machserve_amd.weights.loader import WeightsError
    d = U.make_dir(tmp_path, "mixed", seed=9)
    path = d + "/model.safetensors"
    w = load_file(path)
    w["l0.norm2"], w["l0.norm2b"] = torch.ones(64), torch.ones(64)
    save_file(w, path)
    toks = U.tokens_of(9, 97, 1)
    got = U.run_schedule(loaded(d), {"a": toks}, [[("a", 9)]])["a"]
    assert U.relative_error(got, U.plain_logits(d, toks)) < TOL
    w["l4.mix.g"] = torch.ones(2, 64)
    save_file(w, path)
    with pytest.raises(WeightsError, match="l4.mix.g"):
        loaded(d)


# ------------------------------------------------------------------ the new parts beyond this design's own combination
def test_weighted_branches_add_to_a_plain_stream():
    from machserve_amd.parts.base import ResidualStream
    torch.manual_seed(0)
    ops = EmulatedOps(torch.float32)
    x = torch.randn(3, 8)
    (a, wa), (b, wb) = (torch.randn(3, 5), torch.randn(8, 5)), (torch.randn(3, 4), torch.randn(8, 4))
    s = ResidualStream(x.clone(), ops)
    s.add_weighted([((a, wa), 0.5), ((b, wb), -2.0)])
    assert torch.allclose(s.value(), x + 0.5 * a @ wa.T - 2.0 * b @ wb.T, atol=1e-5)


def test_specs_that_do_not_fit_are_refused():
    from machserve_amd.config import GatedDeltaSpec, GatedLinearSpec, SideBySideSpec
    from machserve_amd.parts import MIXERS, Runtime
    rt = Runtime(torch.device("cpu"), torch.float32, EmulatedOps(torch.float32))
    with pytest.raises(ValueError, match="query/key heads"):
        MIXERS.build(GatedDeltaSpec("gated_delta", 16, 4, 3, 8, 8, 4), rt)
    with pytest.raises(ValueError, match="taps"):
        MIXERS.build(GatedDeltaSpec("gated_delta", 16, 4, 2, 8, 8, 17), rt)
    with pytest.raises(ValueError, match="300"):
        MIXERS.build(GatedLinearSpec("gated_linear", 16, 4, 8, 300), rt)
    one = GatedLinearSpec("gated_linear", 16, 4, 8, 8)
    with pytest.raises(ValueError, match="factors"):
        MIXERS.build(SideBySideSpec("side_by_side", 16, (one, one), factors=(1.0,)), rt)
    from dataclasses import replace
    spec = config_from_dict(U.CONFIGS["mixed"]).to_spec()
    with pytest.raises(ConfigError, match="passes begin"):
        replace(spec, loop_steps=replace(spec.loop_steps, starts=(1, 99))).validate()
