"""Layered models without a GPU: reading configurations and weight files, the trace replay's bookkeeping, and the plain statement
itself (that it would notice the mistakes the GPU tests are meant to find)."""
import copy
import io
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import espresso_amd._lib as lib
import espresso_amd.engine as eng
import espresso_amd.trace_runner as tr
import layered_ref as ref
import layered_util as lu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
BASE = lu.config([lu.latent(), lu.retention(), lu.latent(kv_from=0, window=7), lu.retention(ff=0)])


SEQUENTIAL = lu.sequential([lu.mamba2(), lu.attention(factor=4.0), lu.mamba2(heads=6, vdim=20, state=40, groups=3, conv=3, norm_groups=4, kind="mamba2_2", ff=40),
                            lu.attention(kv_from=1, factor=4.0, window=7, ff=0)])


def load(tmp_path, cfg, max_seq=64):
    with open(tmp_path / "config.json", "w") as f:
        f.write(cfg if isinstance(cfg, str) else json.dumps(cfg))
    return eng.load_model_config(str(tmp_path), max_seq)


def test_registered_and_read_from_a_directory(tmp_path):
    assert "Ranavik" in eng.layered_architectures()
    c = load(tmp_path, BASE, 77)
    assert (c.architecture, c.name, c.n_layer, c.d_model, c.vocab, c.max_seq, c.hidden_dim, c.eos_token) == ("layered", "Ranavik", 4, 56, 96, 77, 48, -1)


def test_a_sequential_design_is_read_from_a_directory(tmp_path):
    assert "Forovik" in eng.layered_architectures()
    c = load(tmp_path, SEQUENTIAL, 77)
    assert (c.architecture, c.name, c.n_layer, c.d_model, c.vocab, c.max_seq, c.hidden_dim) == ("layered", "Forovik", 4, 56, 96, 77, 48)


def test_a_llama_directory_is_still_found_by_its_metadata(tmp_path):
    import espresso_amd.llama as ll
    cfg = ll.MultiModelConfig(n_layer=2, n_head=4, n_kv_head=2, d_model=64, head_dim=16, hidden_dim=96, vocab=40, max_seq=32, name="tiny")
    eng.write_metadata(cfg, str(tmp_path / "metadata.json"))
    got = eng.load_model_config(str(tmp_path), 999)
    assert (got.architecture, got.name, got.max_seq) == ("llama", "tiny", 32)


@pytest.mark.parametrize("change,message", [
    (lambda c: c.update(architecture="Other"), "unknown architecture Other"),
    (lambda c: c.pop("width"), "width is not a number"),
    (lambda c: c.update(vocab=1.5), "vocab is not a usable count"),
    (lambda c: c.update(layers=[]), "layers is not a list"),
    (lambda c: c["layers"][1].update(type="convolution"), "names no mixer"),
    (lambda c: c["layers"][1]["mixer"].update(decay=[0.5]), "one decay per head"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=18), "larger than what it rotates"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=7), "odd"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "size is not a usable count"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "scale is not a number"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=1), "without a fitting cache"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=2), "earlier layer"),
    (lambda c: c["layers"][2]["mixer"].update(kv_rank=48), "without a fitting cache"),
    (lambda c: c["layers"][0]["mlp"].update(kind="experts"), "kind is not dense"),
])
def test_configurations_that_do_not_fit_are_refused(tmp_path, change, message):
    c = copy.deepcopy(BASE)
    change(c)
    with pytest.raises(lib.EspressoError, match=message):
        load(tmp_path, c)


@pytest.mark.parametrize("change,message", [
    (lambda c: c["layers"][0].update(type="retention"), "names no mixer of this architecture: retention"),
    (lambda c: c["layers"][0]["mixer"].update(groups=3), "groups does not divide the heads"),
    (lambda c: c["layers"][0]["mixer"].update(norm_groups=5), "norm_groups does not divide"),
    (lambda c: c["layers"][0]["mixer"].pop("conv"), "conv is not a number"),
    (lambda c: c["layers"][0]["mixer"].update(state=0), "state is not a usable count"),
    (lambda c: c["layers"][1]["mixer"].update(kv_heads=3), "kv_heads does not divide"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=20), "larger than what it rotates"),
    (lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].update(factor=0), "factor is not positive"),
    (lambda c: c["layers"][1]["mixer"].pop("mask"), "mask is not an object"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=0), "without a fitting cache"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=3), "earlier layer"),
    (lambda c: c["layers"][3]["mixer"].update(dim=18), "without a fitting cache"),
    (lambda c: c["layers"][3]["mixer"]["rot"].update(base=5.0), "without a fitting cache"),
    (lambda c: c["layers"][1].update(mlp={"kind": "experts", "ff": 8}), "kind is not dense"),
])
def test_sequential_configurations_that_do_not_fit_are_refused(tmp_path, change, message):
    c = copy.deepcopy(SEQUENTIAL)
    change(c)
    with pytest.raises(lib.EspressoError, match=message):
        load(tmp_path, c)


@pytest.mark.parametrize("layer,message", [(lu.attention(dim=1040, dims=8), "1040 values per attention head exceed 1024"), (lu.mamba2(conv=300), "300 taps of a convolution exceed 256"),
                                           (lu.mamba2(state=4100), "4100 values of a state exceed 4096")])
def test_sizes_past_the_kernels_are_refused(tmp_path, layer, message):
    c = lu.sequential([layer], width=8, vocab=4)
    lu.write_model(str(tmp_path), c, lu.random_weights(c, 1))
    with pytest.raises(lib.EspressoError, match=message):
        eng.RealModelInferenceEngine(eng.load_model_config(str(tmp_path), 16), str(tmp_path))


def test_the_tensors_of_a_sequential_model():
    assert set(lu.tensor_shapes(SEQUENTIAL)) >= {"l0.mix.A_log", "l1.mix.k.norm", "l3.mix.q.norm"} and not {"head", "embed.norm", "l3.mix.k", "l0.norm2"} & set(lu.tensor_shapes(SEQUENTIAL))


def test_broken_files_are_refused(tmp_path):
    with pytest.raises(lib.EspressoError, match="config.json"):
        eng.load_model_config(str(tmp_path), 16)
    with pytest.raises(lib.EspressoError, match="not a JSON object"):
        load(tmp_path, '{"architecture": "Ranavik"')
    c = load(tmp_path, BASE)
    with pytest.raises(lib.EspressoError, match="model.safetensors"):
        eng.RealModelInferenceEngine(c, str(tmp_path))
    def file(header, data=b""):
        return len(header).to_bytes(8, "little") + header + data

    for raw, message in ((b"\x05", "too short"), ((1 << 40).to_bytes(8, "little") + b"{}", "past the end"), (file(b"[]"), "not a JSON object"),
                         (file(b'{"a": {"dtype": "BF16", "shape": [4], "data_offsets": [0, 8]}}'), "outside the file"),
                         (file(b'{"a": {"dtype": "BF16", "shape": [3], "data_offsets": [0, 8]}}', bytes(8)), "does not fit its shape"),
                         (file(b'{"a": {"dtype": "F9", "shape": [8], "data_offsets": [0, 8]}}', bytes(8)), "unknown dtype")):
        (tmp_path / "model.safetensors").write_bytes(raw)
        with pytest.raises(lib.EspressoError, match=message):
            eng.RealModelInferenceEngine(c, str(tmp_path))


def test_the_layered_part_of_the_library_is_listed_and_stands_alone():
    """Its sources exist, and none of them includes a header of the llama runtime."""
    import espresso_amd.build as build
    for s in build.COMPONENTS["layered"]:
        text = open(os.path.join(build.CSRC, s)).read()
        assert "llama_runtime.h" not in text, s
    assert build.component_path("layered") != build.LIB_PATH


# ---- trace replay ---------------------------------------------------------------------------------
class FakeModel:
    """Three sequence slots; a token's logits are (sequence-wide token count so far, token)."""

    def __init__(self):
        self.free, self.held, self.log = [0, 1, 2], {}, []

    def acquire_sequence(self):
        s = self.free.pop(0)
        self.held[s] = 0
        return s

    def release_sequence(self, s):
        del self.held[s]
        self.free.insert(0, s)

    def append(self, tokens, want, sequence):
        assert list(want) == sorted(set(want))
        start = self.held[sequence]
        self.held[sequence] += len(tokens)
        self.log.append((sequence, list(tokens)))
        return np.array([[start + w, tokens[w]] for w in want], dtype=np.float32).reshape(len(want), 2)


def test_trace_replay_orders_rows_and_returns_slots(tmp_path):
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": [5, 6, 7], "want": [2, 0]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": [1], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": [8], "want": [0]}, {"id": "b", "tokens": [2, 3], "want": [1]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "c", "tokens": [9], "want": [0]}], "end": ["b", "c"]}]
    answers, m = [], FakeModel()
    tr.run(m, io.StringIO("".join(json.dumps(s) + "\n" for s in steps)), str(tmp_path), 2, answers.append)
    assert answers == ["done 0", "done 1", "done 2", "done 3"]
    read = lambda n: np.fromfile(tmp_path / f"{n}.f32", "<f4").reshape(-1, 2).tolist()
    assert read(0) == [[2, 7], [0, 5]] and read(2) == [[3, 8], [2, 3]] and read(3) == [[0, 9]]
    assert sorted(os.listdir(tmp_path)) == ["0.f32", "2.f32", "3.f32"] and not m.held
    assert m.log[-1] == (0, [9])          # the slot of "a" serves "c"


def test_a_llama_directory_is_refused_in_float32(tmp_path):
    (tmp_path / "metadata.json").write_text("{}")
    assert tr.main(["--model", str(tmp_path), "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "4"]) == 3


def test_command_lines_explain_themselves():
    for cmd in ([os.path.join(ROOT, "bin", "trace_run"), "--help"], [sys.executable, "-m", "espresso_amd.run_model", "--help"]):
        p = subprocess.run(cmd, capture_output=True, text=True, cwd=ROOT)
        assert p.returncode == 0 and "--max-tokens" in p.stdout, p.stderr


# ---- the plain statement ---------------------------------------------------------------------------
def test_retention_recurrence_is_the_sum_over_earlier_keys():
    rng = np.random.default_rng(3)
    q, k, v = rng.normal(size=(9, 2, 4)), rng.normal(size=(9, 2, 4)), rng.normal(size=(9, 2, 3))
    o, state = ref.retention_recurrence(q, k, v, [0.5, 0.9])
    for h, g in enumerate((0.5, 0.9)):
        for t in range(9):
            want = sum(g ** (t - s) * (q[t, h] @ k[s, h]) * v[s, h] for s in range(t + 1))
            assert np.allclose(o[t, h], want)
    o2, _ = ref.retention_recurrence(q[5:], k[5:], v[5:], [0.5, 0.9], ref.retention_recurrence(q[:5], k[:5], v[:5], [0.5, 0.9])[1])
    assert np.allclose(o2, o[5:])


def test_rotation_keeps_lengths_and_depends_on_the_distance_only():
    rng = np.random.default_rng(4)
    a, b = rng.normal(size=(1, 1, 12)), rng.normal(size=(1, 1, 12))
    for interleaved in (False, True):
        rot = lu.rotary(8, 100.0)
        at = lambda x, p: ref.rotate(x, [p], rot, interleaved)[0, 0]
        assert np.isclose(at(a, 17) @ at(a, 17), a[0, 0] @ a[0, 0]) and np.array_equal(at(a, 17)[8:], a[0, 0, 8:])
        assert np.isclose(at(a, 9) @ at(b, 4), at(a, 29) @ at(b, 24)) and not np.isclose(at(a, 9) @ at(b, 4), at(a, 9) @ at(b, 5))


def test_yarn_leaves_fast_pairs_and_slows_the_others():
    f, one = ref.rotary_frequencies(lu.rotary(32, 10000.0))
    g, amp = ref.rotary_frequencies(lu.rotary(32, 10000.0, lu.YARN))
    assert one == 1.0 and np.isclose(amp, 0.1 * np.log(4.0) + 1.0)
    assert g[0] == f[0] and np.isclose(g[-1], f[-1] / 4.0) and np.all(np.diff(g / f) <= 1e-12)


def test_window_and_sink():
    w = ref.window_softmax_with_sink(np.zeros((1, 6, 6)), range(6), range(6), 3, np.array([0.0]))
    assert np.allclose(w[0, 5], [0, 0, 0, .25, .25, .25]) and np.allclose(w[0, 0], [.5, 0, 0, 0, 0, 0])


@pytest.mark.parametrize("change", [
    lambda c, w: c["layers"][0]["mixer"]["mask"].update(size=21),
    lambda c, w: c["layers"][0]["mixer"]["mask"].update(size=19),
    lambda c, w: c["layers"][2]["mixer"]["mask"].update(size=8),
    lambda c, w: w.update({"l0.mix.sink": np.full(3, -30.0)}),
    lambda c, w: c["layers"][0]["mixer"]["rot"].pop("scaling"),
    lambda c, w: c["layers"][1]["mixer"].update(decay=[0.875, 0.9374]),
    lambda c, w: c["layers"][1]["mixer"]["rot"].update(dims=14),
    lambda c, w: c["norm"].update(eps=2e-3),
    lambda c, w: c.update(logit_softcap=None),
])
def test_a_small_mistake_moves_the_logits_past_the_gpu_tests_limit(change):
    """The models of the GPU tests are sharp enough: mistakes planted here, in the statement, exceed the fp32 limit."""
    w = lu.random_weights(BASE, 7, gain=2.0)
    t = lu.tokens(BASE, 40)
    want = ref.forward(BASE, w, t)
    c, w2 = copy.deepcopy(BASE), dict(w)
    change(c, w2)
    assert lu.error(ref.forward(c, w2, t), want) > 3 * lu.F32_LIMIT


def test_selective_recurrence_is_a_weighted_sum_over_earlier_tokens():
    rng = np.random.default_rng(3)
    x, b, c, dt, rate = rng.normal(size=(9, 2, 4)), rng.normal(size=(9, 2, 3)), rng.normal(size=(9, 2, 3)), rng.uniform(0.1, 2, (9, 2)), np.array([0.3, 2.0])
    y, _ = ref.selective_recurrence(x, b, c, dt, rate)
    for h in range(2):
        for t in range(9):
            want = sum(np.exp(-rate[h] * dt[s + 1:t + 1, h].sum()) * dt[s, h] * (b[s, h] @ c[t, h]) * x[s, h] for s in range(t + 1))
            assert np.allclose(y[t, h], want)
    half = ref.selective_recurrence(x[:5], b[:5], c[:5], dt[:5], rate)[1]
    assert np.allclose(ref.selective_recurrence(x[5:], b[5:], c[5:], dt[5:], rate, half)[0], y[5:])


def test_convolution_window_norm_and_gate():
    x = np.arange(12.0).reshape(6, 2)
    y = ref.causal_convolution(x, np.array([[0., 0., 1.], [1., 0., 0.]]), np.array([0.5, 0.0]))
    assert np.allclose(y[:, 0], x[:, 0] + 0.5) and np.allclose(y[:, 1], [0, 0, 1, 3, 5, 7])
    assert np.allclose(ref.causal_convolution(x[3:], np.ones((2, 3)), np.zeros(2), x[1:3]), ref.causal_convolution(x, np.ones((2, 3)), np.zeros(2))[3:])
    w = ref.window_softmax(np.zeros((1, 5, 5)), range(5), range(5), 2)
    assert np.allclose(w[0, 4], [0, 0, 0, .5, .5]) and np.allclose(w[0, 0], [1, 0, 0, 0, 0])
    n = ref.grouped_rms_norm(np.array([[3., 4., 0., 10.]]), np.ones(4), 2, 0.0)
    assert np.allclose(n, [[3 / np.sqrt(12.5), 4 / np.sqrt(12.5), 0, np.sqrt(2)]])
    assert np.allclose(ref.gelu_tanh(np.array([-2., 0., 1.])), [-0.0454023, 0, 0.841192], atol=1e-6)
    f, one = ref.rotary_frequencies(lu.rotary(8, 100.0, {"factor": 4.0}))
    assert one == 1.0 and np.allclose(f, ref.rotary_frequencies(lu.rotary(8, 100.0))[0] / 4.0)


@pytest.mark.parametrize("change", [
    lambda c, w: c["layers"][1]["mixer"]["mask"].update(size=21),
    lambda c, w: c["layers"][1]["mixer"]["mask"].update(size=19),
    lambda c, w: c["layers"][3]["mixer"]["mask"].update(size=8),
    lambda c, w: c["layers"][1]["mixer"].update(scale=0.2501),
    lambda c, w: c["layers"][3]["mixer"].update(rot=lu.rotary(8, 10000.0, {"factor": 4.2})),
    lambda c, w: c["layers"][1]["mixer"]["rot"].update(dims=6),
    lambda c, w: c["layers"][0]["mixer"].update(norm_groups=1),
    lambda c, w: c["norm"].update(eps=2e-3),
    lambda c, w: w["l0.mix.D"].__imul__(1.01),
    lambda c, w: w["l0.mix.dt_bias"].__iadd__(0.01),
    lambda c, w: w["l0.mix.A_log"].__iadd__(0.01),
    lambda c, w: w["l2.mix.conv"][:, 0].__imul__(0.98),
    lambda c, w: w["l2.mix.conv.b"].__imul__(0.98),
    lambda c, w: w["l1.mix.k.norm"].__imul__(1.01),
])
def test_a_small_mistake_moves_a_sequential_models_logits_past_the_limit(change):
    w = lu.random_weights(SEQUENTIAL, 7, gain=2.0)
    t = lu.tokens(SEQUENTIAL, 40)
    want = ref.forward(SEQUENTIAL, w, t)
    c, w2 = copy.deepcopy(SEQUENTIAL), {k: v.copy() for k, v in w.items()}
    change(c, w2)
    assert lu.error(ref.forward(c, w2, t), want) > 3 * lu.F32_LIMIT
