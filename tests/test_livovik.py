"""Livovik without a GPU: the configuration, the plain model's own mechanisms against closed forms, and the engine's host
side (parts, cache manager with a chunk of keys a layer run, step function, scheduler) over CPU stand-ins for the kernels,
against the plain model."""
import json
import math

import pytest
import torch

import livovik_util as U
from emulated_ops import EmulatedOps
from plain import livovik_plain as P

from machserve_amd.config import ConfigError, LivovikConfig, config_from_dict
from machserve_amd.engine.loading import load_model

# The stand-ins leave a product of few rows as two partial sums, one of them noise of order one: 32-bit rounding of that
# noise, through sharpened softmaxes, is what this bound allows.  A key that is missing or one too many or a sink left out
# is off by a hundred times more.
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
    assert isinstance(cfg, LivovikConfig)
    assert config_from_dict(json.loads(json.dumps(cfg.to_dict()))) == cfg
    spec = cfg.to_spec()
    own = [i for i, l in enumerate(raw["layers"]) if "weights_of" not in l]
    assert len(spec.layers) == len(own) and len(spec.order) == len(raw["layers"])
    assert [own[j] for j in spec.order] == [P.owner(raw["layers"], i) for i in range(len(raw["layers"]))]
    assert all(l.block == "sumnorm" and l.alpha == raw["postln_alpha"] for l in spec.layers)
    names = [n for n, _, _ in cfg.random_tensor_plan()]
    assert len(set(names)) == len(names) and names[0] == "embed" and names[-2:] == ["final.norm", "head"]
    for i, layer in enumerate(raw["layers"]):
        mlp = layer["mlp"]
        has = lambda s: f"l{i}.{s}" in names
        assert has("norm1") == has("mix.sink") == has("mix.g") == (i in own)
        assert has("norm2") == (i in own and mlp is not None)
        assert has("mlp.router") == (i in own and mlp is not None and mlp["kind"] == "moe")
        assert has("mlp.shared.sg") == (has("mlp.router") and "shared" in mlp)


def test_configuration_errors_name_the_key():
    def broken(change):
        raw = json.loads(json.dumps(U.CONFIGS["mixed"]))
        change(raw)
        return raw
    for match, change in [
            (r"layers\[1\]\.mixer\.kv_heads", lambda r: r["layers"][1]["mixer"].pop("kv_heads")),
            ("heads", lambda r: r["layers"][1]["mixer"].update(kv_heads=3)),
            ("rot.dims", lambda r: r["layers"][3]["mixer"].update(rot={"base": 10.0, "dims": 7})),
            ("rot.scaling.high", lambda r: r["layers"][5]["mixer"]["rot"]["scaling"].pop("high")),
            ("scaling.low", lambda r: r["layers"][5]["mixer"]["rot"]["scaling"].update(low=9.0)),
            ("mask.size", lambda r: r["layers"][5]["mixer"]["mask"].update(size=0)),
            ("latent", lambda r: r["layers"][1].update(type="latent")),
            ("top", lambda r: r["layers"][3]["mlp"]["router"].update(top=9)),
            ("kind", lambda r: r["layers"][3]["mlp"].update(kind="glu")),
            (r"shared\.ff", lambda r: (r["layers"][0]["mlp"]["shared"].pop("ff"))),
            ("weights_of", lambda r: r["layers"][2].update(weights_of=6)),
            ("weights_of", lambda r: r["layers"][2].update(weights_of=True)),
            ("weights_of", lambda r: r["layers"][0].update(weights_of=2)),          # the two would name each other
            ("weights_of", lambda r: r["layers"][3].update(weights_of=3)),
            (r"layers\[2\].*differ", lambda r: r["layers"][2]["mixer"].update(scale=0.31)),
            ("postln_alpha", lambda r: r.pop("postln_alpha")),
            ("norm", lambda r: r.pop("norm"))]:
        with pytest.raises(ConfigError, match=match):
            config_from_dict(broken(change))


# ------------------------------------------------------------------ the plain mechanisms against closed forms
def test_chunks_are_counted_from_position_zero():
    see = P.chunk_visible(10, 4)
    assert see[3].tolist() == [True] * 4 + [False] * 6
    assert see[4].tolist() == [False] * 4 + [True] + [False] * 5
    assert see[7].tolist() == [False] * 4 + [True] * 4 + [False] * 2
    assert see[9].tolist() == [False] * 8 + [True] * 2
    assert P.chunk_visible(5, None)[4].tolist() == [True] * 5


def test_a_sink_is_one_more_term_of_the_denominator():
    s = torch.tensor([[1.0, 2.0, 50.0]], dtype=F64)
    see = torch.tensor([[True, True, False]])
    w = P.sink_softmax(s, see, torch.tensor(0.5, dtype=F64))
    den = math.exp(1.0) + math.exp(2.0) + math.exp(0.5)
    assert torch.allclose(w, torch.tensor([[math.exp(1.0) / den, math.exp(2.0) / den, 0.0]], dtype=F64))
    w = P.sink_softmax(s, see, torch.tensor(800.0, dtype=F64))              # a sink far above every score takes everything
    assert torch.isfinite(w).all() and float(w.abs().max()) < 1e-9
    assert torch.allclose(P.sink_softmax(s, see, None).sum(), torch.ones((), dtype=F64))


def test_frequencies_below_between_and_above_the_bounds():
    rot = {"base": 100.0, "dims": 12, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 64.0}}
    plain = [100.0 ** (-2.0 * i / 12) for i in range(6)]
    turns = [64.0 * f / (2 * math.pi) for f in plain]
    got = P.frequencies(rot)
    kinds = set()
    for f, t, g in zip(plain, turns, got):
        if t > 4.0:
            want, kind = f, "kept"
        elif t < 1.0:
            want, kind = f / 8.0, "divided"
        else:
            s = (t - 1.0) / 3.0
            want, kind = (1 - s) * f / 8.0 + s * f, "mixed"
        kinds.add(kind)
        assert abs(g - want) < 1e-12
    assert kinds == {"kept", "mixed", "divided"}
    assert P.frequencies({"base": 100.0, "dims": 12}) == plain


def test_the_engines_table_of_frequencies_is_the_plain_models():
    from machserve_amd.config import RotarySpec, WavelengthScalingSpec
    from machserve_amd.parts import Runtime
    from machserve_amd.parts.registry import POSITION_ENCODINGS
    rt = Runtime(torch.device("cpu"), torch.float32, EmulatedOps(torch.float32))
    for base, dims, scaling in [(500.0, 8, (4.0, 1.0, 3.0, 64)), (1e6, 64, (8.0, 1.0, 4.0, 1000)), (100.0, 6, (3.0, 1.0, 1.0, 30)),
                                (50.0, 2, (2.0, 0.25, 4.0, 12.5)), (250000.0, 32, None)]:
        bands = WavelengthScalingSpec(*scaling) if scaling else None
        part = POSITION_ENCODINGS.build(RotarySpec("rotary", 64, base, rotary_dim=dims, table_precision="float64", wavelengths=bands), rt)
        rot = {"base": base, "dims": dims}
        if scaling:
            rot["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
        assert torch.allclose(part.rotary_inv_freq().double(), torch.tensor(P.frequencies(rot), dtype=F64), rtol=1e-6, atol=0)
        assert part.score_factor() == 1.0


def test_rotation_of_half_against_half_leaves_the_rest_and_keeps_lengths():
    x = torch.randn(6, 2, 10, dtype=F64)
    rot = {"base": 100.0, "dims": 6}
    p, i = 4, 1
    a = p * 100.0 ** (-2 * i / 6)
    y = P.rotate(x, rot)
    assert torch.equal(y[..., 6:], x[..., 6:]) and torch.allclose(y[0], x[0])
    assert torch.allclose(y[..., :6].pow(2).sum(-1), x[..., :6].pow(2).sum(-1))
    assert torch.allclose(y[p, 1, 1], x[p, 1, 1] * math.cos(a) - x[p, 1, 4] * math.sin(a))
    assert torch.allclose(y[p, 1, 4], x[p, 1, 4] * math.cos(a) + x[p, 1, 1] * math.sin(a))


def test_attention_of_one_token_is_its_gated_value_beside_the_sink():
    torch.manual_seed(0)
    w, m = 6, {"heads": 2, "kv_heads": 1, "dim": 4, "vdim": 3, "scale": 0.5, "mask": {"size": 4}}
    t = {s: torch.randn(n, w, dtype=F64) for s, n in (("q", 8), ("k", 4), ("v", 3), ("g", 2))}
    t.update({"q.norm": torch.randn(4, dtype=F64), "k.norm": torch.randn(4, dtype=F64), "sink": torch.tensor([0.3, -1.0], dtype=F64), "o": torch.eye(6, dtype=F64)})
    h = torch.randn(1, w, dtype=F64)
    got = P.attention(h, t, "", m, 1e-6)[0]
    k = (h @ t["k"].T)[0]
    k = k / torch.sqrt((k * k).mean() + 1e-6) * t["k.norm"]
    for a in range(2):
        q = (h @ t["q"].T)[0, 4 * a:4 * a + 4]
        q = q / torch.sqrt((q * q).mean() + 1e-6) * t["q.norm"]
        e = torch.exp((q @ k) * 0.5)
        want = e / (e + torch.exp(t["sink"][a])) * (h @ t["v"].T)[0] / (1 + torch.exp(-(h @ t["g"].T)[0, a]))
        assert torch.allclose(got[3 * a:3 * a + 3], want)


def test_an_experts_weight_multiplies_its_input():
    torch.manual_seed(1)
    w_ = 4
    t = {"router": torch.tensor([[1.0, 0, 0, 0], [0, 1.0, 0, 0], [0, 0, 1.0, 0]], dtype=F64)}
    for e in range(3):
        t.update({f"e{e}.gate": torch.randn(5, w_, dtype=F64), f"e{e}.up": torch.randn(5, w_, dtype=F64), f"e{e}.down": torch.randn(w_, 5, dtype=F64)})
    h = torch.tensor([[2.0, -1.0, 3.0, 0.7]], dtype=F64)
    mlp = {"router": {"experts": 3, "top": 2}, "expert": {"ff": 5}}
    want = torch.zeros(1, w_, dtype=F64)
    for e in (0, 2):                                                          # the two largest logits, weights not renormalised
        x = h / (1 + math.exp(-float(h[0, e])))
        g = x @ t[f"e{e}.gate"].T
        want += (g / (1 + torch.exp(-g)) * (x @ t[f"e{e}.up"].T)) @ t[f"e{e}.down"].T
    assert torch.allclose(P.moe(h, t, "", mlp), want)


def test_the_expert_for_every_token_is_gated():
    torch.manual_seed(2)
    w_ = 4
    t = {"router": torch.zeros(1, w_, dtype=F64)}
    for e in ("e0", "shared"):
        t.update({f"{e}.gate": torch.randn(3, w_, dtype=F64), f"{e}.up": torch.randn(3, w_, dtype=F64), f"{e}.down": torch.randn(w_, 3, dtype=F64)})
    h = torch.randn(2, w_, dtype=F64)
    mlp = {"router": {"experts": 1, "top": 1}, "expert": {"ff": 3}, "shared": {"ff": 3}}
    t["shared.sg"] = torch.zeros(1, w_, dtype=F64)
    half = P.moe(h, t, "", mlp)
    assert torch.allclose(half, P.expert(0.5 * h, t, "e0.") + 0.5 * P.expert(h, t, "shared."))


def test_the_norm_comes_after_the_sum():
    x, w = torch.randn(3, 8, dtype=F64), torch.randn(8, dtype=F64)
    cfg = {"norm": {"eps": 1e-5}, "postln_alpha": 3.0, "layers": [{"mixer": {"heads": 1, "kv_heads": 1, "dim": 2, "vdim": 2, "scale": 1.0}, "mlp": None}]}
    t = {"l0.mix." + s: torch.zeros(n, 8, dtype=F64) for s, n in (("q", 2), ("k", 2), ("v", 2), ("g", 1))}
    t.update({"l0.mix.q.norm": w[:2], "l0.mix.k.norm": w[:2], "l0.mix.sink": w[:1], "l0.mix.o": torch.zeros(8, 2, dtype=F64), "l0.norm1": w})
    v = 3.0 * x                                                               # a mixer that leaves nothing
    assert torch.allclose(P.layer(x, t, cfg, 0), v / torch.sqrt((v * v).mean(-1, keepdim=True) + 1e-5) * w)


def test_the_square_of_relu():
    t = {"up": torch.eye(3, dtype=F64), "down": torch.eye(3, dtype=F64)}
    assert P.dense(torch.tensor([[-2.0, 0.5, 3.0]], dtype=F64), t, "").tolist() == [[0.0, 0.25, 9.0]]


def test_plain_model_whole_equals_its_prefixes(tmp_path):
    d = U.make_dir(tmp_path, "mixed", seed=1)
    w, cfg = U.read(d)
    toks = U.tokens_of(40, 97, 0)
    whole = P.forward(w, cfg, toks)
    for n in (1, 2, 7, 17, 39):
        assert torch.allclose(P.forward(w, cfg, toks[:n])[-1], whole[n - 1], atol=1e-9)


# ------------------------------------------------------------------ the engine's host side over CPU stand-ins
def _cut(rid, n, sizes):
    out, at, k = [], 0, 0
    while at < n:
        c = min(sizes[k % len(sizes)], n - at)
        out.append([(rid, c)])
        at, k = at + c, k + 1
    return out


@pytest.mark.parametrize("name", sorted(U.CONFIGS))
def test_any_cut_of_a_prompt_equals_the_plain_model(tmp_path, name):
    d = U.make_dir(tmp_path, name, seed=3)
    n = 70 if name != "wide" else 40
    toks = U.tokens_of(n, U.CONFIGS[name]["vocab"], 5)
    want = U.plain_logits(d, toks)
    lm = loaded(d)
    for what, schedule in {"whole": [[("a", n)]], "token by token": [[("a", 1)]] * n,
                           "portions down to two tokens": _cut("a", n, [2, 17, 3, 2, 16, 1, 1, 15, 2])}.items():
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


def test_layers_that_share_tensors_have_caches_of_their_own(tmp_path):
    lm = loaded(U.make_dir(tmp_path, "mixed", seed=6))
    assert lm.model.order == [0, 1, 0, 2, 1, 3] and len(lm.model.blocks) == 4
    groups = {g.spec.window: sorted(run for run, _ in g.spec.layers) for g in lm.cache.groups.values()}
    assert groups == {16: [0, 2], 24: [1, 4], None: [3], 20: [5]}             # a chunk of keys each, all keys without chunks
    pools = [lm.device_cache.binding(p).kpool.data_ptr() for p in range(6)]
    assert len(set(pools)) == 6


def test_pages_behind_a_chunk_are_given_back(tmp_path):
    """A request of 90 tokens through layers that see chunks holds a few pages at a time, and its numbers stay right."""
    d = U.make_dir(tmp_path, "odd", seed=7)
    toks = U.tokens_of(90, 61, 2)
    lm = loaded(d, max_requests=1, num_pages={"window7": 2, "window33": 4, "window1": 2})
    got = U.run_schedule(lm, {"a": toks}, _cut("a", 90, [9, 1, 2, 8, 3]))["a"]
    assert U.relative_error(got, U.plain_logits(d, toks)) < TOL
    lm.cache.check()


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


def test_a_layer_without_feed_forward_may_bring_its_unused_norm(tmp_path):
    """The second norm of a layer that has no feed-forward is not used and not missed; a tensor of a layer that runs
    another's, or any other the model does not know, is refused by name."""
    from safetensors.torch import load_file, save_file
    from machserve_amd.weights.loader import WeightsError
    d = U.make_dir(tmp_path, "mixed", seed=9)
    path = d + "/model.safetensors"
    w = load_file(path)
    w["l5.norm2"] = torch.ones(64)
    save_file(w, path)
    toks = U.tokens_of(9, 97, 1)
    got = U.run_schedule(loaded(d), {"a": toks}, [[("a", 9)]])["a"]
    assert U.relative_error(got, U.plain_logits(d, toks)) < TOL
    w["l2.norm1"] = torch.ones(64)
    save_file(w, path)
    with pytest.raises(WeightsError, match="l2.norm1"):
        loaded(d)


# ------------------------------------------------------------------ the new variants of parts beyond this design's own combination
def test_chunked_attention_with_convolution_biases_and_gates_of_their_own_product():
    """Norms per head, a sink and a gate behind a convolution and biases: the variants of the mixer go together."""
    from machserve_amd.config import ChunkedAttentionSpec, RotarySpec
    from machserve_amd.parts import MIXERS, Runtime
    ops = EmulatedOps(torch.float32)
    rt = Runtime(torch.device("cpu"), torch.float32, ops)
    base = dict(hidden=16, heads=4, kv_heads=2, head_dim=8, v_head_dim=12, scale=0.5, norm_eps=1e-6, chunk=5)
    rot = RotarySpec("rotary", 8, 100.0, rotary_dim=4, table_precision="float64")
    m = MIXERS.build(ChunkedAttentionSpec("chunked_attention", position=rot, conv_taps=0, bias=True, qk_norm=False, head_norm=True, sink=True,
                                          head_gate=True, **base), rt)
    assert not m.fused and {d.name for d in m.tensor_decls()} >= {"q.bias", "q.norm", "sink", "g.weight"}
    m = MIXERS.build(ChunkedAttentionSpec("chunked_attention", position=rot, conv_taps=3, bias=False, qk_norm=False, head_norm=True, **base), rt)
    assert not m.fused and "sink" not in {d.name for d in m.tensor_decls()}
    with pytest.raises(ValueError, match="exclude"):
        MIXERS.build(ChunkedAttentionSpec("chunked_attention", position=rot, qk_norm=True, head_norm=True, **base), rt)


def test_combinations_of_routed_experts_that_are_not_built_are_refused():
    from machserve_amd.config import RoutedMlpSpec
    from machserve_amd.parts import FEED_FORWARDS, Runtime
    rt = Runtime(torch.device("cpu"), torch.float32, EmulatedOps(torch.float32))
    with pytest.raises(ValueError, match="input"):
        FEED_FORWARDS.build(RoutedMlpSpec("routed_mlp", 16, 4, 2, 8, "silu", weigh="input"), rt)
    with pytest.raises(ValueError, match="every token"):
        FEED_FORWARDS.build(RoutedMlpSpec("routed_mlp", 16, 4, 2, 8, "silu", 0, False, gated=True, shared_gate=True), rt)
    with pytest.raises(ValueError, match="scoring"):
        FEED_FORWARDS.build(RoutedMlpSpec("routed_mlp", 16, 4, 2, 8, "silu", scoring="softplus"), rt)
