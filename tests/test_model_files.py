"""CPU: model folders (config.json + model.safetensors) are read strictly - what is missing, misshapen
or unknown is named before anything touches the GPU -, and the plain implementations the GPU tests
compare with agree with themselves however their input is cut."""
import copy
import importlib
import json
import os
import struct

import numpy as np
import pytest

import girirax_models as GM
import girirax_oracle as GO
import lusadra_models as LM
import lusadra_oracle as O


@pytest.fixture(scope="module")
def Model():
    return importlib.import_module("cpp-tensorlib_amd.model").Model


def refused(Model, folder):
    with pytest.raises(RuntimeError) as e:
        Model.open(str(folder))
    return str(e.value)


@pytest.mark.parametrize("models,name", [(LM, "loop_of_unlike_layers"), (GM, "state_first")])
def test_good_folder_reaches_the_backend(tmp_path, Model, models, name):
    if os.path.exists("/dev/kfd"):
        pytest.skip("a GPU is present")
    cfg = models.SMALL[name]
    assert "backend unavailable" in refused(Model, LM.write(tmp_path / "m", cfg, models.weights(cfg)))


@pytest.mark.parametrize("edit,words", [
    (lambda c: c.update(architecture="Other"), "unknown architecture Other"),
    (lambda c: c.pop("architecture"), "architecture"),
    (lambda c: c.pop("width"), "width"),
    (lambda c: c.update(width=12.5), "integer"),
    (lambda c: c["layers"][0].update(type="serial"), "unknown mixer"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=3), "layer 1"),
    (lambda c: c["layers"][0]["mixer"]["left"].update(vdim=7), "vdim"),
    (lambda c: c["layers"][0]["mixer"]["left"]["mask"].update(size=0), "layer 0"),
    (lambda c: c["layers"][2]["mixer"]["right"].update(tau=0), "layer 2"),
    (lambda c: c["layers"][0]["mlp"].update(kind="experts"), "unknown feed-forward"),
    (lambda c: c["loop"].update(stop=9), "loop"),
    (lambda c: c.update(layers=[]), "no layers"),
])
def test_configurations_that_are_refused(tmp_path, Model, edit, words):
    cfg = copy.deepcopy(LM.SMALL["loop_of_unlike_layers"])
    W = LM.weights(cfg)
    edit(cfg)
    assert words in refused(Model, LM.write(tmp_path / "m", cfg, W))


@pytest.mark.parametrize("edit,words", [
    (lambda c: c.pop("residual_mult"), "residual_mult"),
    (lambda c: c.pop("embedding"), "embedding"),
    (lambda c: c["layers"][0].update(type="mamba"), "unknown mixer"),
    (lambda c: c["layers"][0]["mixer"].update(groups=4), "layer 0"),
    (lambda c: c["layers"][0]["mixer"].update(norm_groups=5), "layer 0"),
    (lambda c: c["layers"][2]["mixer"].update(conv=0), "layer 2"),
    (lambda c: c["layers"][1]["mixer"].update(rot_dim=7), "layer 1"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=4), "rot.dims"),
    (lambda c: c["layers"][3]["mixer"].pop("q_rank"), "q_rank"),
    (lambda c: c["layers"][3]["mlp"].update(kind="experts"), "unknown feed-forward"),
    (lambda c: c.update(layers=[]), "no layers"),
])
def test_girirax_configurations_that_are_refused(tmp_path, Model, edit, words):
    cfg = copy.deepcopy(GM.SMALL["state_first"])
    W = GM.weights(cfg)
    edit(cfg)
    assert words in refused(Model, LM.write(tmp_path / "m", cfg, W))


@pytest.mark.parametrize("text", ["", "{", '{"a":}', "[1,2", '{"a" 1}', '{"a":1} x', '{"a":tru}', '{"a":1,}', '"\x01"', "[1 2]", "01x"])
def test_malformed_json(tmp_path, Model, text):
    (tmp_path / "config.json").write_text(text)
    assert "JSON" in refused(Model, tmp_path)


def test_json_values(tmp_path, Model):
    """Escapes, nesting, exponents and white space are read as JSON has them."""
    (tmp_path / "config.json").write_text(
        ' { "x" : [ {} , [ ] , -1.5e-3, true , false, null, "a\\u00e9\\ud83d\\ude00\\n" ] ,\t"architecture":"\\u004cu\\tx" }\r\n')
    assert "unknown architecture Lu\tx" in refused(Model, tmp_path)


def test_malformed_safetensors(tmp_path, Model):
    cfg = LM.SMALL["no_loop"]
    good = LM.safetensors_bytes(LM.weights(cfg))
    n = struct.unpack("<Q", good[:8])[0]
    head = json.loads(good[8:8 + n])

    def with_header(h):
        b = h if isinstance(h, bytes) else json.dumps(h).encode()
        return struct.pack("<Q", len(b)) + b + good[8 + n:]

    def changed(**kw):
        h = copy.deepcopy(head)
        h["embed"].update(kw)
        return with_header(h)

    folder = LM.write(tmp_path / "m", cfg, {})
    path = os.path.join(folder, "model.safetensors")
    a, b = head["embed"]["data_offsets"]
    for data, words in [(good[:5], "too short"), (good[:8 + n // 2], "longer than the file"), (good[:-2], "bad offsets"),
                        (with_header(b"{nope"), "JSON"), (changed(data_offsets=[a, b + 2]), "bad offsets"),
                        (changed(data_offsets=[-2, b]), "bad offsets"), (changed(shape=[3, -1]), "bad shape"),
                        (changed(shape=[2 ** 40, 2 ** 40]), "bad shape"), (changed(dtype="F4"), "bad entry"),
                        (changed(data_offsets=[a]), "bad entry")]:
        with open(path, "wb") as f:
            f.write(data)
        assert words in refused(Model, folder), words
    os.unlink(path)
    assert "cannot open" in refused(Model, folder)
    assert "not found" in refused(Model, tmp_path / "nowhere")


@pytest.mark.parametrize("oracle,models,name", [(O, LM, n) for n in LM.SMALL] + [(GO, GM, n) for n in GM.SMALL])
def test_oracle_does_not_depend_on_the_cut(oracle, models, name):
    cfg = models.SMALL[name]
    o = oracle.Oracle(cfg, models.weights(cfg, 3))
    t = [int(x) for x in np.random.default_rng(4).integers(0, cfg["vocab"], 60)]
    whole = o.feed(t)
    o.reset()
    cut = np.concatenate([o.feed(t[a:b]) for a, b in ((0, 1), (1, 3), (3, 34), (34, 35), (35, 60))])
    assert np.abs(cut - whole).max() < 1e-9 * np.abs(whole).max()


def test_oracle_mechanisms_against_closed_forms():
    """Cases whose answers can be written down."""
    g = np.random.default_rng(0)
    # one visible key: its own; two equal scores apart from the distance bias
    k = g.standard_normal((6, 4))
    one = O.window_attention(g.standard_normal((6, 8)), k, 2, 1, 4, 1, 0.5, 0.0, 3)
    assert np.allclose(one, np.tile(k, (1, 2)))
    two = O.window_attention(np.zeros((2, 4)), k[:2], 1, 1, 4, 2, 1.0, 0.0, 3)
    s = np.exp(-2.0 ** -8)
    assert np.allclose(two[1], (k[1] + s * k[0]) / (1 + s))
    assert O.query_temperature(0, 0.5, 1) == 1 + 0.5 * np.log(2) and O.query_temperature(6, 0.5, 8) == 1.0
    # constant decay: the state is a geometric sum
    q, kk, v = np.ones((5, 1)), np.ones((5, 1)), np.arange(1.0, 6.0)[:, None]
    o, S = O.gated_linear_attention(q, kk, v, np.full((5, 1), 0.5), 1, 1, 1)
    want = [sum(v[s, 0] * 0.5 ** (t - s) for s in range(t + 1)) for t in range(5)]
    assert np.allclose(o[:, 0], want) and np.isclose(S[0, 0, 0], want[-1])
    assert np.allclose(O.polynorm(np.full((1, 3), 2.0), (1, 2, 3, 4), 0.0), 1 + 2 + 3 + 4)
    assert np.allclose(O.position_vector(0, 6), [0, 1, 0, 1, 0, 1])
    assert O.layer_runs({"layers": [{}] * 4, "loop": {"start": 1, "stop": 3, "times": 2}}) == \
        [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]


def test_girirax_mechanisms_against_closed_forms():
    """Cases whose answers can be written down."""
    g = np.random.default_rng(0)
    # constant inputs: the state is a geometric sum, read by C, with the skip beside it
    one = np.ones((6, 1))
    x = np.arange(1.0, 7.0)[:, None]
    a = np.exp(-2.0 * 0.3)
    y, S = GO.state_space(x, one, 3 * one, 0.3 * one, np.log([2.0]), [0.5], 1, 1, 1, 1)
    want = [3 * sum(0.3 * x[s, 0] * a ** (t - s) for s in range(t + 1)) + 0.5 * x[t, 0] for t in range(6)]
    assert np.allclose(y[:, 0], want)
    # heads of a group read its B and C: with B = 0 in group 1 only heads 0 and 1 write
    B = np.concatenate([np.ones((4, 2)), np.zeros((4, 2))], axis=1)
    y, S = GO.state_space(np.ones((4, 4)), B, B, np.ones((4, 4)), np.zeros(4), np.zeros(4), 4, 2, 2, 1)
    assert (y[:, :2] > 0).all() and not y[:, 2:].any() and S[1].any() and not S[2].any()
    y, tail = GO.causal_conv(x, np.array([[100.0, 10.0, 1.0]]), np.array([0.5]), np.zeros((2, 1)))
    assert np.allclose(y[:, 0], [1.5, 12.5, 123.5, 234.5, 345.5, 456.5]) and np.allclose(tail[:, 0], [5, 6])
    # a rotation keeps lengths, and products depend on the distance
    u, v = g.standard_normal(8), g.standard_normal(8)
    turned = [GO.rotate_half(u, p + 5, 50.0) @ GO.rotate_half(v, p, 50.0) for p in (0, 3, 1000)]
    assert np.allclose(turned, turned[0]) and np.isclose(np.linalg.norm(GO.rotate_half(u, 77, 9.0)), np.linalg.norm(u))
    assert np.allclose(GO.rotate_half(np.array([1.0, 0, 0, 0]), 1, 100.0), [np.cos(1), 0, np.sin(1), 0])
    assert np.allclose(GO.rotate_half(np.array([0, 1.0, 0, 0]), 2, 100.0), [0, np.cos(0.2), 0, np.sin(0.2)])
    # equal scores: the mean of the values
    k = g.standard_normal((5, 3))
    assert np.allclose(GO.attend(np.zeros(3), k, k, 1.0), k.mean(axis=0))
    n = GO.grouped_rms_norm(np.array([[3.0, 4.0, 0.0, 2.0]]), np.array([1.0, 1.0, 1.0, 10.0]), 2, 0.0)
    assert np.allclose(n, [[3 / np.sqrt(12.5), 4 / np.sqrt(12.5), 0, 10 * np.sqrt(2)]])
    assert np.allclose(GO.gelu_tanh(np.array([0.0, 40.0, -40.0])), [0, 40, 0]) and np.isclose(GO.gelu_tanh(1.0), 0.841192, atol=1e-6)
    assert np.allclose(GO.softplus(np.array([-800.0, 0.0, 800.0])), [0, np.log(2), 800])
