"""Salolorn on the GPU: every new kernel alone against the CPU stand-in of the same entry point (written from the mechanisms'
equations), and the whole engine (cuts of prompts, decoding, mixed batches with pages and slots used again, captured steps,
generation) against the plain model."""
import json
import os
import subprocess
import sys

import pytest
import torch

import salolorn_util as U
from emulated_ops import EmulatedOps
from gpu_util import DEV
from plain import salolorn_plain as P

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]
F32 = 1e-4     # float32 against the plain model in 64-bit
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def ops_of(dtype):
    from machserve_amd.kernels import get_ops
    return get_ops(dtype, DEV)


def dev(t, dtype=None):
    return None if t is None else t.to(device=DEV, dtype=dtype or t.dtype).contiguous()


def i32(values):
    return torch.tensor(values, dtype=torch.int32)


def close(got, want, dtype, what="", bound32=1e-4):
    got, want = got.float().cpu().double(), want.double().cpu()
    assert torch.isfinite(got).all(), what
    bound = (bound32 if dtype == torch.float32 else 2e-2) * float(want.abs().max()) + 1e-6
    err = float((got - want).abs().max())
    assert err <= bound, f"{what}: error {err:.3e} over {bound:.3e}"


def sequences(lengths, slots):
    starts = [sum(lengths[:i]) for i in range(len(lengths))]
    return i32(starts), i32(lengths), i32(slots)


def batches(single):
    """Requests' rows of one step and their slots: decoded rows alone, or portions of every length about a chunk's and a
    segment's edges, unequal side by side."""
    if single:
        return [([1], [0]), ([1] * 5, [4, 0, 2, 5, 1])]
    return [([1], [1]), ([2], [0]), ([16, 1, 17], [2, 0, 5]), ([63], [3]), ([64], [0]), ([65, 3], [1, 4]), ([130, 1, 1, 64, 7], [5, 4, 3, 2, 1]),
            ([400], [2]), ([320, 300], [0, 3])]


# ------------------------------------------------------------------ gated linear attention
SIZES_LINEAR = [(2, 12, 20), (3, 10, 18), (1, 5, 7), (2, 32, 40), (4, 64, 32), (2, 128, 128), (2, 64, 256), (1, 256, 64), (1, 200, 130)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("single", [False, True])
@pytest.mark.parametrize("H,d,dv", SIZES_LINEAR)
def test_gated_linear_attention(dtype, single, H, d, dv):
    ops, ref = ops_of(dtype), EmulatedOps(dtype)
    torch.manual_seed(H * d + dv)
    dvp, cols, R = -(-dv // 4) * 4, -(-H * dv // 8) * 8, 11
    for lengths, slots in batches(single):
        for parts in (1, 3):
            T = sum(lengths)
            n = 2 * H * (d + dv) + R
            sums = torch.randn(parts, T, -(-n // 8) * 8) * parts ** -0.5
            a2t, b, norm = torch.randn(R, H * d) * 0.5, torch.randn(H * d) + 2.0, torch.rand(dv) + 0.5
            seqs = sequences(lengths, slots)
            state = torch.zeros(6, H, d, dvp)
            state[..., :dv] = torch.randn(6, H, d, dv)
            want_state, got_state = state.clone(), dev(state)
            for tau in (16.0, 1.0):
                want_alpha = ref.key_decay(sums, 2 * H * (d + dv), a2t, b, tau)
                got_alpha = ops.key_decay(dev(sums), 2 * H * (d + dv), dev(a2t), dev(b), tau)
                close(got_alpha, want_alpha, torch.float32, "decays", 1e-5)
            args = (norm, 1e-5, d ** -0.5)
            want = ref.gated_linear(sums, want_alpha, *args, want_state, *seqs, H, d, dv, cols, single=single)
            got = ops.gated_linear(dev(sums), dev(want_alpha), dev(norm), 1e-5, d ** -0.5, got_state, *[dev(s) for s in seqs], H, d, dv, cols, single=single)
            close(got, want, dtype, f"outputs of {lengths}")
            close(got_state, want_state, torch.float32, f"states after {lengths}")


# ------------------------------------------------------------------ the gated delta rule
SIZES_DELTA = [(4, 2, 16, 24), (5, 1, 10, 13), (2, 2, 9, 6), (4, 2, 32, 32), (2, 1, 64, 128), (2, 2, 96, 48), (4, 2, 128, 128), (2, 1, 64, 256), (1, 1, 256, 64), (2, 1, 200, 130)]


def delta_inputs(H, G, d, dv, T, parts, taps, seed):
    torch.manual_seed(seed)
    C = 2 * G * d + H * dv
    n = C + H * dv + 2 * H
    sums = torch.randn(parts, T, -(-n // 8) * 8) * parts ** -0.5
    return sums, torch.randn(C, taps) * 0.6, torch.log(1.0 + torch.arange(H).float()), torch.randn(H)


@pytest.mark.parametrize("single", [False, True])
@pytest.mark.parametrize("H,G,d,dv", SIZES_DELTA)
@pytest.mark.parametrize("taps", [4, 1, 2, 6, 16])
def test_delta_rows(single, H, G, d, dv, taps):
    ops, ref = ops_of(torch.float32), EmulatedOps(torch.float32)
    C = 2 * G * d + H * dv
    for lengths, slots in batches(single):
        for parts in (1, 3):
            T = sum(lengths)
            sums, conv, a_log, dt = delta_inputs(H, G, d, dv, T, parts, taps, T + taps)
            seqs = sequences(lengths, slots)
            state = torch.randn(6, taps - 1, C) if taps > 1 else None
            want_state, got_state = (None, None) if state is None else (state.clone(), dev(state))
            want = ref.delta_rows(sums, conv, want_state, a_log, dt, d ** -0.5, *seqs, H, G, d, dv, single=single)
            got = ops.delta_rows(dev(sums), dev(conv), got_state, dev(a_log), dev(dt), d ** -0.5, *[dev(s) for s in seqs], H, G, d, dv, single=single)
            for g, w, what in zip(got, want, ("q", "k", "v", "beta", "decay")):
                close(g, w, torch.float32, f"{what} of {lengths}", 1e-5)
            if taps > 1:
                close(got_state, want_state, torch.float32, f"convolution state after {lengths}", 1e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("single", [False, True])
@pytest.mark.parametrize("H,G,d,dv", SIZES_DELTA)
def test_delta_rule(dtype, single, H, G, d, dv):
    ops, ref = ops_of(dtype), EmulatedOps(dtype)
    dvp, cols = -(-dv // 4) * 4, -(-H * dv // 8) * 8
    for lengths, slots in batches(single):
        for parts, slow in ((1, False), (2, True)):
            T = sum(lengths)
            sums, conv, a_log, dt = delta_inputs(H, G, d, dv, T, parts, 1, T + d)
            seqs = sequences(lengths, slots)
            rows = list(EmulatedOps(torch.float32).delta_rows(sums, conv, None, a_log, dt - (6.0 if slow else 0.0), d ** -0.5, *seqs, H, G, d, dv))
            if slow:  # keys close to one another under slow decays: what a chunk's tokens take from each other is large
                rows[1] = torch.nn.functional.normalize(rows[1].view(T, G, d) + 1.5 * torch.nn.functional.normalize(torch.ones(d), dim=0), dim=-1).reshape(T, G * d)
            norm, gate_col = torch.rand(dv) + 0.5, 2 * G * d + H * dv
            state = torch.zeros(6, H, d, dvp)
            state[..., :dv] = torch.randn(6, H, d, dv)
            want_state, got_state = state.clone(), dev(state)
            want = ref.gated_delta(*rows, sums, gate_col, norm, 1e-5, want_state, *seqs, H, G, d, dv, cols, single=single)
            got = ops.gated_delta(*[dev(r) for r in rows], dev(sums), gate_col, dev(norm), 1e-5, got_state, *[dev(s) for s in seqs], H, G, d, dv, cols, single=single)
            close(got, want, dtype, f"outputs of {lengths}")
            close(got_state, want_state, torch.float32, f"states after {lengths}")


# ------------------------------------------------------------------ two weighted branches under a norm, the opening of a pass
@pytest.mark.parametrize("d,T", [(48, 5), (130, 37), (1028, 3), (2048, 9), (5120, 3)])
def test_norm_of_two_weighted_branches(d, T):
    ops, ref = ops_of(torch.bfloat16), EmulatedOps(torch.bfloat16)
    torch.manual_seed(d)
    w = torch.randn(d)
    for na, nb, fa, fb in ((1, 1, 1.2, 0.9), (3, 1, -0.5, 2.0), (2, 9, 1.0, 1.0), (17, 8, 0.3, -1.7)):
        x, pa, pb = torch.randn(T, d), torch.randn(na, T, d), torch.randn(nb, T, d)
        want, got = x.clone(), dev(x)
        ref.norm_add_weighted(want, pa, fa, pb, fb, w, 1e-5)
        ops.norm_add_weighted(got, dev(pa), fa, dev(pb), fb, dev(w), 1e-5)
        close(got, want, torch.float32, f"{na} and {nb} sums", 1e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("d,T", [(48, 5), (256, 70), (1024, 33), (1028, 3), (2048, 9), (4096, 5)])
def test_norm_behind_a_branch_and_ahead_of_the_next(dtype, d, T):
    ops, ref = ops_of(dtype), EmulatedOps(dtype)
    torch.manual_seed(d)
    w, w2 = torch.randn(d), torch.randn(d)
    taken = 0
    for counts, factors in (((1,), (1.0,)), ((2,), (1.0,)), ((3,), (1.0,)), ((8,), (1.0,)), ((9,), (1.0,)), ((1, 1), (1.2, -0.4)), ((2, 1), (0.5, 2.0)), ((3, 4), (1.0, 1.0)), ((1, 7), (2.0, 0.1))):
        x, branches = torch.randn(T, d) * 2, [(torch.randn(n, T, d), f) for n, f in zip(counts, factors)]
        if not ops.norm_add_norm_takes(d, branches):
            continue
        taken += 1
        want_x, got_x = x.clone(), dev(x)
        want = ref.norm_add_norm(want_x, branches, w, 1e-5, w2, 1e-4)
        got = ops.norm_add_norm(got_x, [(dev(p), f) for p, f in branches], dev(w), 1e-5, dev(w2), 1e-4)
        close(got_x, want_x, torch.float32, f"stream after {counts}", 1e-5)
        close(got, want, dtype, f"rows for the next branch after {counts}")
    assert taken >= 4
    assert not ops.norm_add_norm_takes(50, [(torch.zeros(1, 1, 50), 1.0)])


def test_the_opening_of_a_pass():
    ops = ops_of(torch.float32)
    torch.manual_seed(0)
    x, first, row = torch.randn(7, 50), torch.randn(7, 50), torch.randn(50)
    for f in (first, None):
        got = dev(x)
        ops.open_pass(got, dev(f), dev(row))
        close(got, x + row + (0 if f is None else f), torch.float32)


@pytest.mark.parametrize("rot", [16, 6])
def test_angles_of_the_latents_key_part_stay_exact_at_far_positions(rot):
    """Rows at positions up to a hundred thousand against a rotation in 64-bit by the same frequencies."""
    ops = ops_of(torch.float32)
    torch.manual_seed(rot)
    T, rank, hd, ps = 40, 24, 48, 64
    pos = torch.randint(50000, 100000, (T,), dtype=torch.int32)
    inv = 100.0 ** (-torch.arange(rot // 2, dtype=torch.float32) * 2 / rot)
    proj = torch.randn(1, T, 48)
    kpool, vpool = torch.zeros(1, 1, ps, hd, device=DEV), torch.zeros(1, 1, hd, ps, device=DEV)
    ops.latent_rows(dev(proj), None, dev(torch.ones(rank)), 1e-6, dev(pos), dev(inv), 1.0, dev(torch.arange(T, dtype=torch.int32)), kpool, vpool, 0, rank, rot, ps)
    k = proj[0, :, rank:rank + rot].double()
    a = pos.double()[:, None] * inv.double()
    u, v = k[:, 0::2], k[:, 1::2]
    want = torch.stack([u * torch.cos(a) - v * torch.sin(a), v * torch.cos(a) + u * torch.sin(a)], -1).reshape(T, rot)
    assert float((kpool[0, 0, :T, rank:rank + rot].cpu().double() - want).abs().max()) < 2e-5
    q = torch.randn(T, 2 * (8 + rot))
    _, att = ops.latent_query(dev(q), dev(pos), dev(inv), 1.0, 2, 8, rot, rank, hd)
    qr = q.double().view(T, 2, 8 + rot)[..., 8:]
    u, v, a = qr[..., 0::2], qr[..., 1::2], a[:, None, :]
    want = torch.stack([u * torch.cos(a) - v * torch.sin(a), v * torch.cos(a) + u * torch.sin(a)], -1).reshape(T, 2, rot)
    assert float((att[..., rank:rank + rot].cpu().double() - want).abs().max()) < 2e-5


# ------------------------------------------------------------------ keys that stand out, where this design's attention looks for them
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("decoded", [False, True])
@pytest.mark.parametrize("H,KV,hd,chunk,n,key,seen", [
    # every head over one key/value head (a latent and a rotated part), every earlier key seen: the first of all, page borders, itself
    (6, 1, 96, 0, 900, 0, True), (6, 1, 96, 0, 900, 15, True), (6, 1, 96, 0, 900, 16, True), (5, 1, 80, 0, 700, 699, True), (17, 1, 64, 0, 500, 3, True),
    (3, 1, 256, 0, 600, 255, True),
    # chunks with a sink and a gate: their first position, the one before it, the row that opens a chunk, a page's border within
    (6, 2, 64, 104, 624, 520, True), (6, 2, 64, 104, 624, 519, False), (6, 2, 64, 104, 625, 624, True), (6, 2, 64, 104, 625, 623, False),
    (4, 4, 48, 33, 330, 304, True), (4, 4, 48, 33, 330, 296, False), (9, 3, 128, 500, 400, 0, True)])
def test_a_key_that_stands_out_is_seen_where_it_should_be(dtype, decoded, H, KV, hd, chunk, n, key, seen):
    from test_livovik_gpu import _keys_case
    rows = 1 if decoded else n
    sinks, gate = (torch.full((H,), -9.0), torch.full((rows, H), 0.5)) if chunk else (None, None)
    top = float(_keys_case(dtype, H, KV, hd, 16, n - rows, rows, key, chunk, sinks, gate)[:hd].min())
    full = 25.0 if chunk else 50.0   # the key's value is 50 in every column; halved by the gate
    assert (top > 0.8 * full) if seen else top < 0.4 * full


# ------------------------------------------------------------------ the engine against the plain model
def loaded(model_dir, dtype, page_size=16, max_tokens=1024, max_requests=4, use_graphs=True, num_pages=None):
    from machserve_amd.engine.loading import load_model
    return load_model(model_dir, dtype=dtype, device=DEV, page_size=page_size, max_tokens=max_tokens, max_requests=max_requests,
                      use_graphs=use_graphs, num_pages=num_pages)


def plain_for(model_dir, dtype, tokens):
    """The plain model in 64-bit, on the weights as the run holds them."""
    return U.plain_logits(model_dir, tokens, torch.float64, weights_as=dtype)


def sharpen_for(dtype):
    """Softmaxes far from flat for the 32-bit runs, where a wrong key must show; milder for bfloat16, whose rounding a
    sharp softmax multiplies."""
    return 3.0 if dtype == torch.float32 else 1.0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(U.CONFIGS))
def test_prompts_cut_anywhere_and_decoding_equal_the_plain_model(tmp_path, name, dtype):
    d = U.make_dir(tmp_path, name, seed=7, sharpen=sharpen_for(dtype))
    n = 150
    toks = U.tokens_of(n, U.CONFIGS[name]["vocab"], 8)
    want = plain_for(d, dtype, toks)
    lm = loaded(d, dtype)
    schedules = {"whole": [[("a", n)]], "prompt, then token by token": [[("a", 60)]] + [[("a", 1)]] * (n - 60),
                 "portions down to two tokens": U.cut("a", n, [2, 33, 3, 16, 2, 47, 1, 1, 31, 2])}
    for what, schedule in schedules.items():
        got = U.run_schedule(lm, {"a": toks}, schedule)["a"]
        assert U.within(got, want, dtype), (what, U.relative_error(got, want))
    lm.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
def test_sizes_nearer_a_real_models(tmp_path, dtype):
    d = U.make_dir(tmp_path, "big", seed=17, sharpen=1.0)
    n = 330
    toks = U.tokens_of(n, 1000, 4)
    want = plain_for(d, dtype, toks)
    lm = loaded(d, dtype, page_size=64)
    for what, schedule in {"whole": [[("a", n)]], "portions, then token by token": U.cut("a", 290, [128, 2, 97, 63]) + [[("a", 1)]] * 40}.items():
        got = U.run_schedule(lm, {"a": toks}, schedule)["a"]
        assert U.within(got, want, dtype), (what, U.relative_error(got, want))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("graphs", [False, True])
def test_unequal_requests_side_by_side_equal_each_alone(tmp_path, dtype, graphs):
    name = "mixed"
    d = U.make_dir(tmp_path, name, seed=9, sharpen=sharpen_for(dtype))
    vocab = U.CONFIGS[name]["vocab"]
    reqs = {"a": U.tokens_of(90, vocab, 1), "b": U.tokens_of(1, vocab, 2), "c": U.tokens_of(41, vocab, 3),
            "d": U.tokens_of(70, vocab, 4), "e": U.tokens_of(35, vocab, 5)}
    schedule = [[("b", 1), ("a", 20), ("c", 5)], [("a", 1), ("c", 30)], [("a", 2), ("c", 2), ("d", 17)], [("a", 1), ("c", 1), ("d", 1)],
                [("a", 1), ("c", 1), ("d", 1)], [("a", 1), ("c", 1), ("d", 1)], [("a", 1), ("c", 1), ("d", 1)],
                [("d", 1), ("e", 16), ("a", 1)], [("a", 30), ("e", 1), ("d", 2)], [("a", 32), ("d", 46), ("e", 18)]]
    lm = loaded(d, dtype, max_requests=3, num_pages=16, use_graphs=graphs)
    got = U.run_schedule(lm, reqs, schedule)
    for i, toks in reqs.items():
        assert U.within(got[i], plain_for(d, dtype, toks), dtype), i
    if dtype == torch.float32:      # and the same numbers, beyond rounding, as each request alone in one step
        alone = loaded(d, dtype, use_graphs=False)
        for i, toks in reqs.items():
            assert U.relative_error(got[i], U.run_schedule(alone, {i: toks}, [[(i, len(toks))]])[i]) < 2e-5, i
    lm.cache.check()
    assert all(g.pool.available() == g.pool.num_pages for g in lm.cache.groups.values())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["odd", "mixed"])
def test_long_decoding_from_captured_steps(tmp_path, name, dtype):
    """Decoded tokens pass the edges of many chunks and leave pages behind; looped layers are in the captured steps with a
    cache or state of their own for every pass."""
    d = U.make_dir(tmp_path, name, seed=10, sharpen=sharpen_for(dtype))
    toks = U.tokens_of(330, U.CONFIGS[name]["vocab"], 3)
    lm = loaded(d, dtype, max_tokens=512)
    got = U.run_schedule(lm, {"a": toks}, [[("a", 10)]] + [[("a", 1)]] * 320)["a"]
    assert U.within(got, plain_for(d, dtype, toks), dtype)
    assert len(lm.step._graphs) > 0     # the single rows ran from captured steps


def test_captured_steps_replay_as_launched_ones(tmp_path):
    """The same decode steps from captured graphs and launched kernel by kernel, other work between the replays."""
    d = U.make_dir(tmp_path, "mixed", seed=22)
    reqs = {i: U.tokens_of(40, 97, k) for k, i in enumerate("abc")}
    schedule = [[("a", 9), ("b", 14), ("c", 2)]] + [[("a", 1), ("b", 1), ("c", 1)]] * 26
    schedule.append([("a", 5), ("c", 12)])
    runs = []
    for graphs in (True, False):
        lm = loaded(d, torch.float32, max_requests=3, use_graphs=graphs)
        runs.append(U.run_schedule(lm, reqs, schedule))
        torch.randn(64, 64, device=DEV).sum().item()
    for i in reqs:
        assert U.relative_error(*[r[i] for r in runs]) < 2e-5, i


def test_a_long_prompt_in_portions_behind_pages_of_64(tmp_path):
    d = U.make_dir(tmp_path, "mixed", seed=11)
    toks = U.tokens_of(700, 97, 6)
    want = plain_for(d, torch.float32, toks)
    lm = loaded(d, torch.float32, page_size=64, max_tokens=768)
    for what, schedule in {"whole": [[("a", 700)]], "portions": U.cut("a", 700, [500, 63, 2, 129, 6])}.items():
        got = U.run_schedule(lm, {"a": toks}, schedule)["a"]
        assert U.relative_error(got, want) < F32, (what, U.relative_error(got, want))


def test_long_portions_beside_decoded_tokens(tmp_path):
    d = U.make_dir(tmp_path, "mixed", seed=21, rank=5)
    reqs = {"a": U.tokens_of(500, 97, 1), "b": U.tokens_of(320, 97, 2), "c": U.tokens_of(9, 97, 3)}
    schedule = [[("a", 190), ("b", 200)], [("c", 7), ("b", 118)], [("b", 1), ("a", 305), ("c", 1)], [("b", 1), ("a", 5), ("c", 1)]]
    lm = loaded(d, torch.float32, page_size=64, max_tokens=1024, max_requests=3)
    got = U.run_schedule(lm, reqs, schedule)
    for i, toks in reqs.items():
        assert U.relative_error(got[i], plain_for(d, torch.float32, toks)) < F32, i


def test_first_tokens_of_a_sequence(tmp_path):
    for name in sorted(U.CONFIGS):
        d = U.make_dir(tmp_path, name, seed=12)
        toks = U.tokens_of(4, U.CONFIGS[name]["vocab"], 1)
        lm = loaded(d, torch.float32)
        for n in (1, 2, 3, 4):
            want = plain_for(d, torch.float32, toks[:n])
            assert U.relative_error(U.run_schedule(lm, {"a": toks[:n]}, [[("a", n)]])["a"], want) < F32, (name, n)
            assert U.relative_error(U.run_schedule(lm, {"a": toks[:n]}, [[("a", 1)]] * n)["a"], want) < F32, (name, n, "one by one")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_entry_point(tmp_path, dtype):
    import machserve_amd
    d = U.make_dir(tmp_path, "mixed", seed=13, sharpen=sharpen_for(torch.float32 if dtype == "float32" else torch.bfloat16))
    w, cfg = U.read(d)
    prompts = [U.tokens_of(n, 97, n) for n in (3, 21, 1, 40, 17)]
    got = machserve_amd.generate(d, prompts, max_new=8, dtype=dtype, page_size=16, capacity=3, max_batch_tokens=32, chunk_size=16)
    for p, g in zip(prompts, got):
        if dtype == "float32":
            assert g == P.greedy_generate(w, cfg, p, 8, torch.float64)
        else:   # bfloat16 may flip a near-tie: every token must be within rounding of the best
            seq = list(p)
            for t in g:
                logits = plain_for(d, torch.bfloat16, seq)[-1]
                assert logits[t] >= logits.max() - 5e-2 * (logits.max() - logits.min()), "a token that is not a maximum"
                seq.append(t)


def test_a_folder_of_this_layout_runs_through_the_trace_program(tmp_path):
    import numpy as np
    d = U.make_dir(tmp_path, "odd", seed=14)
    toks = U.tokens_of(50, 61, 2)
    out = tmp_path / "out"
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": toks[:33], "want": [0, 32]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": toks[33:], "want": [16]}, {"id": "y", "tokens": toks[:2], "want": []}], "end": ["x", "y"]}]
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", d, "--dtype", "float32", "--out", str(out),
                        "--max-tokens", "128", "--page-size", "16"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                       capture_output=True, text=True, timeout=600)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == ["done 0", "done 1"]
    want = plain_for(d, torch.float32, toks)
    got = torch.from_numpy(np.concatenate([np.fromfile(out / "0.f32", dtype="<f4"), np.fromfile(out / "1.f32", dtype="<f4")]).reshape(3, 61))
    assert U.relative_error(got, want[[0, 32, 49]]) < F32


def test_command_line_generates_from_a_folder(tmp_path):
    d = U.make_dir(tmp_path, "once", seed=15)
    w, cfg = U.read(d)
    prompt = U.tokens_of(9, 80, 4)
    cmd = [sys.executable, os.path.join(ROOT, "bin", "machserve"), "--max-new", "5", "--dtype", "f32", "--tpp", "16", "--prompt-ids"]
    r = subprocess.run(cmd + [",".join(map(str, prompt)), "--model", d], capture_output=True, text=True, timeout=600)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [int(t) for t in r.stdout.split()] == P.greedy_generate(w, cfg, prompt, 5, torch.float64)
