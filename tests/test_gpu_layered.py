"""Layered models on the GPU against their plain statement (layered_ref.py), through the engine and the C ABI.

fp32 models are held to a few 1e-5 of the logits' spread, which every mistake of test_layered_host.py exceeds; bf16 models to what
rounding costs.  Blocks of rows (prompt kernels), single rows (decode kernels) and mixtures of both see the same tokens."""
import os
import subprocess
import sys

import numpy as np
import pytest

import espresso_amd._lib as lib
import espresso_amd.engine as eng
import espresso_amd.layered as layered
import espresso_amd.llama as ll
import layered_ref as ref
import layered_util as lu

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
BOTH = pytest.mark.parametrize("precision", ["f32", "bf16"])

PARALLEL = lu.config([lu.latent(), lu.retention(), lu.latent(kv_from=0, window=7), lu.retention(ff=0), lu.retention(heads=3, dim=24, vdim=40, dims=10)])
SEQUENTIAL = lu.sequential([lu.mamba2(), lu.attention(factor=4.0), lu.mamba2(heads=6, vdim=20, state=40, groups=3, conv=3, norm_groups=4, kind="mamba2_2", ff=40),
                            lu.attention(kv_from=1, factor=4.0, window=7, ff=0), lu.mamba2(heads=2, groups=1, conv=6, norm_groups=1)])
# one mechanism at a time, and sizes at the borders of tiles, chunks, head groups and kernel variants
CONFIGS = {
    "retention alone": lu.config([lu.retention(ff=0)]),
    "one head, no decay and full decay": lu.config([lu.retention(heads=1, decay=[1.0]), lu.retention(heads=2, decay=[0.0, 0.25])], eps=0.05),   # (q . k) v over its own size alone is ill conditioned: a large eps
    "retention of uneven heads": lu.config([lu.retention(heads=5, dim=36, vdim=72, dims=20), lu.retention(heads=2, dim=130, vdim=33)], width=100),
    "latent attention alone": lu.config([lu.latent(ff=0)]),
    "latent attention without YaRN": lu.config([lu.latent(scaling=None, heads=1, dim=32, vdim=32, kv_rank=64, rot_dim=32)]),
    "sharp scores": lu.config([lu.latent(scale=2.0), lu.latent(scale=2.0, kv_from=0)]),
    "window of one": lu.config([lu.latent(window=1), lu.retention()]),
    "windows at tile borders": lu.config([lu.latent(window=w) for w in (31, 32, 33, 63, 64, 65)]),
    "window past the context": lu.config([lu.latent(window=100000)]),
    "shared latents, wider reader": lu.config([lu.latent(window=5), lu.latent(kv_from=0, window=90), lu.latent(window=9), lu.latent(kv_from=2)]),
    "many heads": lu.config([lu.latent(heads=37, dim=8, vdim=8, rot_dim=4)], width=120),
    "long query heads": lu.config([lu.latent(heads=2, dim=224, vdim=160, kv_rank=300, rot_dim=48), lu.latent(heads=2, dim=100, vdim=40, rot_dim=64)]),
    "wide latents": lu.config([lu.latent(heads=2, kv_rank=600, dim=64, vdim=64)]),
    "odd sizes": lu.config([lu.latent(ff=37), lu.retention(ff=101)], vocab=333, width=71, residual_mult=1.0, softcap=4.0),
    "no softcap": lu.config([lu.retention()], softcap=None),
    "Mamba-2 alone": lu.sequential([lu.mamba2()]),
    "Mamba-2 and a feed-forward": lu.sequential([lu.mamba2(ff=48), lu.mamba2(ff=33)]),
    "one head, one tap": lu.sequential([lu.mamba2(heads=1, groups=1, conv=1, norm_groups=1), lu.mamba2(heads=1, groups=1, conv=2, norm_groups=2)]),
    "a group per head": lu.sequential([lu.mamba2(heads=6, groups=6, norm_groups=6, vdim=32, state=32, conv=3)]),
    "parts of a norm that end within heads": lu.sequential([lu.mamba2(heads=4, vdim=9, norm_groups=3), lu.mamba2(heads=10, vdim=33, norm_groups=6, state=19, groups=5)]),
    "more parts than wavefronts": lu.sequential([lu.mamba2(heads=8, vdim=20, norm_groups=16, groups=4)]),
    "odd states and values": lu.sequential([lu.mamba2(heads=3, vdim=5, state=11, groups=3, norm_groups=1), lu.mamba2(heads=2, vdim=130, state=65, groups=1, conv=5)], width=71, vocab=333),
    "wide states, many taps": lu.sequential([lu.mamba2(heads=2, vdim=40, state=300, groups=2, conv=20, norm_groups=4)]),
    "more taps than a chunk": lu.sequential([lu.mamba2(conv=75)]),
    "attention alone": lu.sequential([lu.attention(ff=0)]),
    "attention and feed-forwards": lu.sequential([lu.attention(ff=37), lu.attention(ff=130)], width=71, vocab=97),
    "as many key heads as queries": lu.sequential([lu.attention(heads=3, kv_heads=3, dim=16, vdim=16, dims=16)]),
    "one key head for many": lu.sequential([lu.attention(heads=11, kv_heads=1, dim=8, vdim=40, dims=4), lu.attention(heads=6, kv_heads=2, dim=24, dims=2)]),
    "groups of eight": lu.sequential([lu.attention(heads=16, kv_heads=2, dim=32, vdim=32, dims=32, window=64)], width=100),
    "attention, odd heads": lu.sequential([lu.attention(heads=4, kv_heads=2, dim=30, vdim=33, dims=18), lu.attention(heads=2, kv_heads=2, dim=7, vdim=5, dims=6)]),
    "attention, long heads": lu.sequential([lu.attention(heads=2, kv_heads=1, dim=224, vdim=160, dims=56), lu.attention(heads=2, kv_heads=2, dim=130, vdim=300, dims=130)]),
    "linear scaling": lu.sequential([lu.attention(factor=8.0, base=500.0, dims=16), lu.attention(factor=0.5, base=100.0)]),
    "attention, sharp scores": lu.sequential([lu.attention(scale=1.5), lu.attention(scale=1.5, kv_from=0)]),
    "attention, window of one": lu.sequential([lu.attention(window=1), lu.mamba2()]),
    "attention, windows at tile borders": lu.sequential([lu.attention(window=w, ff=0) for w in (31, 32, 33, 63, 64, 65)]),
    "attention, window past the context": lu.sequential([lu.attention(window=100000)]),
    "shared keys, wider reader": lu.sequential([lu.attention(window=5), lu.attention(kv_from=0, window=90, scale=0.5), lu.attention(window=9), lu.attention(kv_from=2, ff=0)]),
    "a large eps": lu.sequential([lu.mamba2(), lu.attention()], eps=0.3),
    "wide stream": lu.sequential([lu.attention(), lu.mamba2()], width=2100),
}


@pytest.fixture(scope="module", params=["parallel", "sequential"])
def mixed(request, tmp_path_factory):
    return lu.Model(tmp_path_factory.mktemp("mixed"), {"parallel": PARALLEL, "sequential": SEQUENTIAL}[request.param], seed=11, gain=1.5)


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_mechanisms_and_sizes(tmp_path, name):
    """Whole prompt as a block, token by token, and the residual stream after every layer."""
    m = lu.Model(tmp_path, CONFIGS[name], seed=len(name), gain=1.5)
    t = lu.tokens(m.cfg, 150)
    streams = []
    want = m.logits(t, streams)
    for precision in ("f32", "bf16"):
        rt = m.runtime(precision)
        got = layered.trace_layers(rt, t, 0)
        for i, (g, w) in enumerate(zip(got, streams)):
            assert lu.error(g, w) < lu.limit(precision), (precision, "layer", i)
        assert lu.error(lu.feed(rt, t, [150], 1), want) < lu.limit(precision), (precision, "block")
        assert lu.error(lu.feed(rt, t, [1], 2), want) < lu.limit(precision), (precision, "steps")


@BOTH
@pytest.mark.parametrize("portions", [[2], [3], [5, 2, 31], [64], [63, 2, 65], [1, 100, 1], [33], [128, 7]])
def test_portions_of_any_size(mixed, precision, portions):
    t = lu.tokens(mixed.cfg, 170, 1)
    rt = mixed.runtime(precision)
    want = mixed.logits(t)
    for least in (1, 1000):        # every portion through the block kernels, down to one row; then every token through the decode kernels
        layered.set_min_block_rows(rt, least)
        assert lu.error(lu.feed(rt, t, portions, 0 if least == 1 else 1), want) < lu.limit(precision), least
    layered.set_min_block_rows(rt, 3)
    assert lu.error(lu.feed(rt, t, portions, 2), want) < lu.limit(precision)


@BOTH
def test_more_than_a_block_and_the_ring_comes_round(tmp_path, precision):
    """Prompts past the rows of one block, and positions past the cached ring, in prompts and in decoding."""
    m = lu.Model(tmp_path, lu.config([lu.latent(window=30), lu.retention(decay=[0.995, 1.0]), lu.latent(kv_from=0, window=9)]), seed=5, gain=1.5)
    t = lu.tokens(m.cfg, 1250, 2)
    want = m.logits(t)
    rt = m.runtime(precision, max_seq=1300)
    for s, portions in enumerate(([1200, 1], [511, 3, 700, 1], [600, 2])):
        got = lu.feed(rt, t, portions, s)
        assert lu.error(got, want) < lu.limit(precision), portions


@BOTH
def test_long_decoding(mixed, precision):
    t = lu.tokens(mixed.cfg, 400, 3)
    rt = mixed.runtime(precision, max_seq=400)
    assert lu.error(lu.feed(rt, t, [3, 1]), mixed.logits(t)) < lu.limit(precision)
    with pytest.raises(lib.EspressoError, match="exceeds context"):
        rt.append([1])


def edge_model(tmp_path, window, kv_from):
    """Queries and keys of the one attention layer that matters agree only for token 1, so a query looks at the places where token 1
    stands within its window, and nothing else competes with it but the sink."""
    layers = [lu.latent(window=window, ff=0, scale=1.0, scaling=None, rot_dim=2)]
    if kv_from:
        layers[0]["mixer"]["mask"]["size"] = 3
        layers.append(lu.latent(window=window, ff=0, scale=1.0, scaling=None, rot_dim=2, kv_from=0))
    cfg = lu.config(layers, residual_mult=1.0)
    m = lu.Model(tmp_path, cfg, seed=21)
    w, last = m.weights, f"l{len(layers) - 1}."
    # embeddings: dimension 0 marks token 1, dimension 1 is shared by all tokens
    e = w["embed"]
    e[:, 0], e[:, 1], e[1, 0] = 0.0, 4.0, 12.0
    w["l0.mix.dkv"][:2] = 0.0
    w["l0.mix.dkv"][0, 0] = 4.0                       # latent 0 = token 1 was here
    w["l0.mix.dkv"][m.cfg["layers"][0]["mixer"]["kv_rank"]:] = 0.0
    q, uk, dim, rot = w[last + "mix.q"], w[last + "mix.uk"], 16, 2
    uk[:] = 0.0
    q[:] = 0.0
    for h in range(3):
        q[h * (dim + rot), 1] = 6.0                   # every token asks for it
        uk[h * dim, 0] = 3.0
    w["l0.mix.dkv.norm"][:] = 1.0
    lu.write_model(m.dir, cfg, w)
    return m


@pytest.mark.parametrize("window,kv_from", [(17, False), (32, False), (33, True), (64, False), (65, True), (96, True)])
def test_a_key_just_inside_and_just_outside_the_window(tmp_path, window, kv_from):
    m = edge_model(tmp_path, window, kv_from)
    t = [2 + x % 90 for x in lu.tokens(m.cfg, 260, 9)]
    for place in (0, 31, 32, 100, 127):
        t[place] = 1
    want = m.logits(t)
    # the statement itself tells the places apart: without its key a query's logits move far beyond the limit
    other = list(t)
    other[100] = 5
    moved = np.abs(m.logits(other) - want).max(axis=1) / np.std(want)
    if window < 28:
        assert moved[100 + window - 1] > 1e-2 > 1e-9 > moved[100 + window]
    for precision in ("f32", "bf16"):
        rt = m.runtime(precision, max_seq=260)
        for s, portions in enumerate(([260], [100, 1], [99, 2, 30, 1], [7])):
            assert lu.error(lu.feed(rt, t, portions, s), want) < lu.limit(precision), (precision, portions)


@pytest.mark.parametrize("sink", [-20.0, 0.0, 6.0, 80.0])
def test_sinks_from_absent_to_dominant(tmp_path, sink):
    m = lu.Model(tmp_path, lu.config([lu.latent(window=25), lu.latent(window=70)]), seed=4, gain=1.5, sink=sink)
    t = lu.tokens(m.cfg, 90, 4)
    want = m.logits(t)
    for precision in ("f32", "bf16"):
        rt = m.runtime(precision)
        assert lu.error(lu.feed(rt, t, [90], 0), want) < lu.limit(precision)
        assert lu.error(lu.feed(rt, t, [1], 1), want) < lu.limit(precision)


def test_the_first_tokens(mixed):
    for n in (1, 2, 3, 4, 5):
        t = lu.tokens(mixed.cfg, n, 30 + n)
        want = mixed.logits(t)
        rt = mixed.runtime()
        assert lu.error(lu.feed(rt, t, [n], 0), want) < lu.F32_LIMIT
        assert lu.error(lu.feed(rt, t, [1], 1), want) < lu.F32_LIMIT
        if n > 1:
            layered.set_min_block_rows(rt, 1)
            assert lu.error(lu.feed(rt, t, [1, n - 1], 2), want) < lu.F32_LIMIT


@BOTH
def test_sequences_take_turns_and_slots_are_used_again(mixed, precision):
    """Requests of unequal lengths, interleaved in portions; each alone gives the same logits, whatever slot it has and whatever ran
    there before."""
    rt = mixed.runtime(precision, sequences=3)
    requests = [lu.tokens(mixed.cfg, n, 40 + n) for n in (70, 9, 131, 33, 2, 64)]
    want = [mixed.logits(t) for t in requests]
    waiting, live, got = list(range(6)), {}, {i: [] for i in range(6)}
    rng = np.random.default_rng(0)
    at = [0] * 6
    while waiting or live:
        while waiting and len(live) < 3:
            i = waiting.pop(0)
            live[i] = rt.acquire_sequence()
        if len(live) == 3:
            with pytest.raises(lib.EspressoError, match="slots are taken"):
                rt.acquire_sequence()
        i = list(live)[int(rng.integers(len(live)))]
        n = min(int(rng.choice([1, 1, 2, 7, 40])), len(requests[i]) - at[i])
        got[i].append(rt.append(requests[i][at[i]:at[i] + n], list(range(n)), sequence=live[i]))
        at[i] += n
        if at[i] == len(requests[i]):
            rt.release_sequence(live.pop(i))
    for i in range(6):
        assert lu.error(np.concatenate(got[i]), want[i]) < lu.limit(precision), i
    assert rt.acquire_sequence() == 0 and rt.visible(0) == 0


def test_recurrent_state_cannot_be_taken_back(mixed):
    rt = mixed.runtime()
    rt.append(lu.tokens(mixed.cfg, 9))
    with pytest.raises(lib.EspressoError, match="cannot go from token 9 to 5"):
        rt.set_visible(5)
    rt.set_visible(9)
    rt.set_visible(0)
    t = lu.tokens(mixed.cfg, 20, 3)
    assert lu.error(lu.feed(rt, t, [20]), mixed.logits(t)) < lu.F32_LIMIT


def test_wrong_calls_are_refused(mixed):
    rt = mixed.runtime(max_seq=20)
    for call, message in ((lambda: rt.append([1, 96]), "outside vocab"), (lambda: rt.append([1, 2], [1, 0]), "ascend"), (lambda: rt.append([1, 2], [2]), "ascend"),
                          (lambda: rt.append(list(range(21))), "exceeds context"), (lambda: rt.append([1], sequence=4), "sequence 4 of 4"),
                          (lambda: ll.generate_two_token(rt, rt, [1], 2), "needs a llama runtime"), (lambda: rt.set_weight(0, 0, 0, np.zeros(4)), "needs a llama runtime")):
        with pytest.raises(lib.EspressoError, match=message):
            call()
    assert rt.visible(0) == 0


@BOTH
def test_greedy_generation_through_the_engine(mixed, precision):
    """Captured step graphs (one and eight steps), the same tokens as the plain statement; a second prompt starts afresh."""
    e = mixed.engine(precision, max_seq=120)
    for n, seed in ((13, 1), (70, 2)):
        prompt = lu.tokens(mixed.cfg, n, seed)
        got, r = e.generate(prompt, 30)
        want = mixed.greedy(prompt, 30)
        if precision == "f32":
            assert got == want
        else:   # bf16: up to the first near-tie of the statement's logits
            same = next((i for i in range(30) if got[i] != want[i]), 30)
            if same < 30:
                top = np.sort(mixed.logits(prompt + want[:same])[-1])
                assert top[-1] - top[-2] < 0.1 * np.std(top)
        assert r["exact_head_backend"] == "hip_gemv_logits_argmax" and r["token_count"] == 30
    assert e.generate(prompt, 30)[0] == got
    rt = e.runtime()
    ll.set_graph_replay(rt, False)
    assert e.generate(prompt, 30)[0] == got
    ll.set_graph_replay(rt, True)
    for i in range(3):          # replays after other eager work and synchronisation
        rt.append(lu.tokens(mixed.cfg, 5, i), [4], sequence=1)
        rt.set_visible(0, 1)
        assert e.generate(prompt, 30)[0] == got


def test_generation_ends_with_the_stop_token(mixed):
    prompt = lu.tokens(mixed.cfg, 13, 1)
    free = mixed.greedy(prompt, 40)
    for stop in (free[5], free[11], free[0]):
        e = mixed.engine("f32", max_seq=120, eos=stop)
        want = free[:free.index(stop) + 1]
        for _ in range(2):
            assert e.generate(prompt, 40)[0] == want
        # what the replays past the stop left behind: the sequence goes on as if nothing had followed
        rt = e.runtime()
        seen = prompt + want[:-1]
        assert rt.visible(0) == len(seen)
        more = lu.tokens(mixed.cfg, 6, 8)
        got = rt.append(more, list(range(6)))
        assert lu.error(got, mixed.logits(seen + more)[len(seen):]) < lu.F32_LIMIT


def test_batches_of_unequal_prompts(mixed):
    rt = mixed.runtime("f32", max_seq=160, sequences=5)
    prompts = [lu.tokens(mixed.cfg, n, 60 + n) for n in (3, 41, 17, 90, 1)]
    got, _ = ll.generate_batch(rt, prompts, 20)
    for p, g in zip(prompts, got):
        assert g == mixed.greedy(p, 20)


def marked_attention(tmp_path, window, kv_from):
    """Grouped attention whose queries match only the keys of token 1, by far: a query's logits say whether token 1 stands in its window."""
    layers = [lu.attention(window=window, ff=0, scale=0.5, dims=4)]
    if kv_from:
        layers = [lu.attention(window=3, ff=0, scale=0.5, dims=4), lu.attention(window=window, ff=0, scale=0.5, dims=4, kv_from=0)]
    cfg = lu.sequential(layers)
    m = lu.Model(tmp_path, cfg, seed=23)
    w, last = m.weights, f"l{len(layers) - 1}."
    w["embed"][:, 0], w["embed"][:, 1], w["embed"][1, 0] = 0.0, 4.0, 12.0   # dimension 0 marks token 1, dimension 1 is shared by all
    k, q, dim = w["l0.mix.k"], w[last + "mix.q"], 16
    k[:], q[:] = 0.0, 0.0
    for g in range(2):
        k[g * dim + 10, 0], k[g * dim + 11, 1] = 1.0, 0.5                    # past the rotated dimensions
    for h in range(4):
        q[h * dim + 10, 1] = 1.0
    w["l0.mix.k.norm"][:], w[last + "mix.q.norm"][:] = 1.0, 1.0
    lu.write_model(m.dir, cfg, w)
    return m


@pytest.mark.parametrize("window,kv_from", [(17, False), (31, False), (32, True), (33, False), (64, True), (65, False), (96, False)])
def test_a_marked_key_just_inside_and_just_outside_the_window(tmp_path, window, kv_from):
    m = marked_attention(tmp_path, window, kv_from)
    t = [2 + x % 90 for x in lu.tokens(m.cfg, 260, 9)]
    for place in (0, 31, 100):
        t[place] = 1
    want = m.logits(t)
    other = list(t)
    other[100] = 5
    moved = np.abs(m.logits(other) - want).max(axis=1) / np.std(want)
    assert moved[100 + window - 1] > 1e-1 > 1e-9 > moved[100 + window]
    for precision in ("f32", "bf16"):
        rt = m.runtime(precision, max_seq=260)
        for s, portions in enumerate(([260], [100, 1], [99, 2, 30, 1], [7])):
            assert lu.error(lu.feed(rt, t, portions, s), want) < lu.limit(precision), (precision, portions)


@pytest.mark.parametrize("name,a_log,dt_bias,dt_gain", [("nothing is forgotten", -30.0, -1.0, 1.0), ("everything is forgotten", 5.0, 2.0, 1.0), ("now and then everything is forgotten", 3.5, -6.0, 9.0),
                                                        ("large steps", -8.0, 30.0, 1.0), ("steps of almost nothing", 0.0, -14.0, 0.1)])
def test_states_from_kept_to_forgotten(tmp_path, name, a_log, dt_bias, dt_gain):
    """Decays at their extremes, also beside each other in one chunk (differences of large sums of logarithms)."""
    m = lu.Model(tmp_path, lu.sequential([lu.mamba2(heads=4, conv=3)]), seed=6, gain=1.5)
    m.weights["l0.mix.A_log"][:] = lu.to_bf16(np.full(4, a_log))
    m.weights["l0.mix.dt_bias"][:] = lu.to_bf16(dt_bias + np.arange(4))
    m.weights["l0.mix.in"][-4:] = lu.to_bf16(m.weights["l0.mix.in"][-4:] * dt_gain)
    lu.write_model(m.dir, m.cfg, m.weights)
    t = lu.tokens(m.cfg, 230, 4)
    want = m.logits(t)
    for precision in ("f32", "bf16"):
        rt = m.runtime(precision)
        for s, portions in enumerate(([230], [1], [65, 1, 62, 2])):
            assert lu.error(lu.feed(rt, t, portions, s), want) < lu.limit(precision), (precision, portions)


@BOTH
def test_a_state_remembers_its_first_token(tmp_path, precision):
    """Without decay the first token, whose input stands out, shows hundreds of tokens later, through blocks, portions and steps."""
    m = lu.Model(tmp_path, lu.sequential([lu.mamba2()]), seed=8)
    m.weights["l0.mix.A_log"][:] = -30.0
    m.weights["embed"][1] *= 16.0
    lu.write_model(m.dir, m.cfg, m.weights)
    t = [1] + [2 + x % 90 for x in lu.tokens(m.cfg, 599, 5)]
    want = m.logits(t)
    moved = np.abs(m.logits([7] + t[1:]) - want).max(axis=1) / np.std(want)
    assert moved[599] > 2e-1
    rt = m.runtime(precision, max_seq=600)
    for s, portions in enumerate(([600], [530, 1], [2, 510, 3])):
        assert lu.error(lu.feed(rt, t, portions, s), want) < lu.limit(precision), portions


@BOTH
@pytest.mark.parametrize("taps", [2, 5, 9])
def test_portions_shorter_than_the_convolution(tmp_path, precision, taps):
    m = lu.Model(tmp_path, lu.sequential([lu.mamba2(conv=taps), lu.mamba2(conv=taps, heads=2, groups=1)]), seed=taps, gain=1.5)
    t = lu.tokens(m.cfg, 80, 6)
    want = m.logits(t)
    rt = m.runtime(precision)
    for least, sequence in ((1, 0), (3, 1)):
        layered.set_min_block_rows(rt, least)
        for portions in ([1], [2], [3], [1, 2, 4, 1], [taps - 1], [taps], [63, 1, 2]):
            rt.set_visible(0, sequence)
            assert lu.error(lu.feed(rt, t, portions, sequence), want) < lu.limit(precision), (least, portions)


@BOTH
def test_more_than_a_block_of_keys_and_states(tmp_path, precision):
    """Prompts past the rows of one block, rings of keys that come round, decoding past them."""
    m = lu.Model(tmp_path, lu.sequential([lu.attention(window=30), lu.mamba2(), lu.attention(kv_from=0, window=70, ff=0)]), seed=5, gain=1.5)
    t = lu.tokens(m.cfg, 1250, 2)
    want = m.logits(t)
    rt = m.runtime(precision, max_seq=1300)
    for s, portions in enumerate(([1200, 1], [511, 3, 700, 1], [600, 2])):
        assert lu.error(lu.feed(rt, t, portions, s), want) < lu.limit(precision), portions


def test_sampling_draws_from_the_models_logits(mixed):
    e = mixed.engine("f32", max_seq=80)
    prompt = lu.tokens(mixed.cfg, 12, 5)
    got, r = e.generate(prompt, 10, 0.8, {"ESPRESSO_HIP_SAMPLING_SEED": "77"})
    units, seen = eng.splitmix64_units(77, 10), list(prompt)
    for token, unit in zip(got, units):
        assert token == eng.sample_token(mixed.logits(seen)[-1], 0.8, unit)
        seen.append(token)
    assert e.runtime().generate_sampled(prompt, 10, 0.8, 77) == got


def test_command_line_and_trace_replay(mixed, tmp_path):
    prompt = lu.tokens(mixed.cfg, 12, 5)
    run = lambda *a: subprocess.run([sys.executable, "-m", "espresso_amd.run_model", mixed.dir, "--precision", "f32", "--context", "64", *a], cwd=ROOT,
                                    capture_output=True, text=True, timeout=100)
    p = run("--tokens", ",".join(map(str, prompt)), "--max-tokens", "8")
    assert p.returncode == 0, p.stderr
    assert [int(x) for x in p.stdout.strip().split(",")] == mixed.greedy(prompt, 8)
    assert run("--tokens", "1,5000").returncode == 1
    import json
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": prompt[:7], "want": [6, 1]}], "end": []}, {"step": 1, "entries": [{"id": "x", "tokens": prompt[7:9], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": prompt[9:], "want": [0, 2]}], "end": ["x"]}]
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", mixed.dir, "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "12"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
    assert p.returncode == 0 and p.stdout.splitlines() == ["done 0", "done 1", "done 2"], p.stderr
    want = mixed.logits(prompt)
    read = lambda n: np.fromfile(tmp_path / f"{n}.f32", "<f4").reshape(-1, mixed.cfg["vocab"])
    assert lu.error(read(0), want[[6, 1]]) < lu.F32_LIMIT and lu.error(read(2), want[[9, 11]]) < lu.F32_LIMIT
    assert not os.path.exists(tmp_path / "1.f32")


@pytest.mark.parametrize("cfg,brackets", [(PARALLEL, {"in": 5, "out": 5, "retention": 3, "latent": 2}), (SEQUENTIAL, {"in": 7, "out": 7, "mamba2": 3, "attention": 2, "norm": 1})])
def test_seeded_random_models_run_and_repeat(cfg, brackets):
    a, b = layered.LayeredRuntime(cfg, 64, seed=3), layered.LayeredRuntime(cfg, 64, seed=3)
    t = lu.tokens(cfg, 20)
    x = a.append(t, [19])
    assert np.all(np.isfinite(x)) and np.array_equal(x, b.append(t, [19]))
    assert layered.sequence_bytes(a) > 0 and a.weight_bytes > 0
    layered.set_kernel_timing(a, True)
    a.append([1])
    k = layered.kernel_times(a)
    assert {c: k[c]["brackets"] for c in brackets} == brackets
