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


def load(tmp_path, cfg, max_seq=64):
    with open(tmp_path / "config.json", "w") as f:
        f.write(cfg if isinstance(cfg, str) else json.dumps(cfg))
    return eng.load_model_config(str(tmp_path), max_seq)


def test_registered_and_read_from_a_directory(tmp_path):
    assert "Ranavik" in eng.layered_architectures()
    c = load(tmp_path, BASE, 77)
    assert (c.architecture, c.name, c.n_layer, c.d_model, c.vocab, c.max_seq, c.hidden_dim, c.eos_token) == ("layered", "Ranavik", 4, 56, 96, 77, 48, -1)


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
