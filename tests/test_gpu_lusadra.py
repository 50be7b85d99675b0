"""Lusadra models end to end on the GPU, against the plain implementation (tests/lusadra_oracle.py):
whole prompts, portions, token by token, several sequences one after the other, far keys, long
decoding, greedy generation, and trace replay."""
import importlib
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import lusadra_models as LM
from lusadra_oracle import Oracle

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


@pytest.fixture(scope="module")
def Model():
    return importlib.import_module("cpp-tensorlib_amd.model").Model


def close(got, want, tol=1e-4):
    err = np.abs(got - want).max() / (np.abs(want).std() + 1e-9)
    assert err < tol, "largest difference over the spread: %.3g" % err


def ids(cfg, n, seed):
    return [int(t) for t in np.random.default_rng(seed).integers(0, cfg["vocab"], n)]


def make(tmp_path, Model, name, seed=1, exact=False, max_ctx=400, chunk=64, **kw):
    cfg = LM.SMALL[name]
    W = LM.weights(cfg, seed, **kw)
    return cfg, Oracle(cfg, W), Model.open(LM.write(tmp_path / name, cfg, W), max_ctx=max_ctx, chunk=chunk, exact=exact)


@pytest.mark.parametrize("exact", [False, True])
@pytest.mark.parametrize("name", list(LM.SMALL))
def test_prompt_portions_and_steps(tmp_path, Model, name, exact):
    """The logits at every position do not depend on how the tokens were cut, nor on the sequence that
    ran before in the same caches and states."""
    cfg, orc, m = make(tmp_path, Model, name, exact=exact)
    assert m.architecture == "Lusadra" and m.vocab == cfg["vocab"]
    n = 150
    t = ids(cfg, n, 2)
    want = orc.feed(t)
    close(m.feed(t, range(n)), want)                          # longer than a chunk: three of them
    for sizes in ((2,), (1,), (31, 2, 1, 1, 3), (64, 1), (7, 33)):
        m.reset()
        got, at, k = [], 0, 0
        while at < n:
            c = min(sizes[k % len(sizes)], n - at)
            got.append(m.feed(t[at:at + c], range(c)))
            at, k = at + c, k + 1
        close(np.concatenate(got), want)
    m.reset()
    orc.reset()
    u = ids(cfg, 40, 3)                                       # another sequence after those
    close(m.feed(u, [0, 1, 17, 39]), orc.feed(u)[[0, 1, 17, 39]])
    m.close()


def test_large_products_in_both_forms(Model):
    """At sizes where prompt products run over the prepared weights and the attention on the 16-bit matrix
    cores, the serving form stays within its rounding of the exact one; a chunk equals steps."""
    l = LM.layer(12, 4, 96, 160, 0.3, 50, 0.1, 8, 64, 96, 6.0, 0.9, 0.8, 3000)
    cfg = LM.config(2000, 1120, [l, l, l], loop=(1, 2, 2))
    t = ids(cfg, 700, 12)
    want = [0, 1, 100, 159, 160, 161, 511, 512, 513, 699]
    lg = {}
    for exact in (True, False):
        m = Model.random(cfg, seed=3, rank=10, max_ctx=800, exact=exact)
        lg[exact] = m.feed(t, want)
        if exact:
            m.reset()
            m.feed(t[:600])
            steps = np.concatenate([m.feed([x], [0]) for x in t[600:]])
            close(steps[-1], lg[True][-1], 1e-4)
        m.close()
    close(lg[False], lg[True], 1e-3)


def test_unfused_step_equals_fused(tmp_path, Model):
    cfg, orc, m = make(tmp_path, Model, "loop_of_unlike_layers")
    m.set_fused(False)
    t = ids(cfg, 30, 5)
    close(np.concatenate([m.feed([x], [0]) for x in t]), orc.feed(t))
    m.close()


def test_residual_after_every_layer(tmp_path, Model):
    cfg, orc, m = make(tmp_path, Model, "loop_of_unlike_layers")
    t, rows = ids(cfg, 45, 6), []
    orc.feed(t, rows)
    got = m.trace_chunk(t, cfg["width"])
    assert len(got) == len(rows) == 1 + 3 * 2 + 1
    for g, w in zip(got, rows):
        close(g, w, 3e-5)
    m.close()


def test_far_tokens_through_the_state_and_past_the_window(tmp_path, Model):
    """Slow decays: a token far outside every window still changes the logits, and by as much as the plain
    form says; with the window's edge passing over it in decoding."""
    cfg, orc, m = make(tmp_path, Model, "no_loop", decay_bias=9.0, max_ctx=700)
    t = ids(cfg, 600, 7)
    want = orc.feed(t)
    other = list(t)
    other[3] = (t[3] + 1) % cfg["vocab"]
    orc.reset()
    moved = orc.feed(other)
    assert np.abs(moved[-1] - want[-1]).max() > 3e-3 * want[-1].std()    # it shows
    for seq, lg in ((t, want), (other, moved)):
        m.reset()
        a = m.feed(seq[:280], [100, 279])
        b = np.concatenate([m.feed([x], [0]) for x in seq[280:360]])     # 300 and 40 tokens of window pass
        c = m.feed(seq[360:], [0, 100, 239])
        close(np.concatenate([a, b, c]), lg[[100, 279] + list(range(280, 360)) + [360, 460, 599]])
    m.close()


def test_long_decoding_and_many_sequences(tmp_path, Model):
    """Four hundred steps on one recorded graph, then short sequences in turn with portions, in the same
    caches: rings wrap several times, both state slots are used from either parity."""
    cfg, orc, m = make(tmp_path, Model, "loop_of_unlike_layers", chunk=16)
    t = ids(cfg, 400, 8)
    want = orc.feed(t)
    close(np.concatenate([m.feed([x], [0]) for x in t]), want)
    for k in range(4):
        orc.reset()
        m.reset()
        u = ids(cfg, 20 + 7 * k, 20 + k)
        want = orc.feed(u)
        cut = 3 + k
        close(np.concatenate([m.feed(u[:cut], range(cut)), m.feed(u[cut:cut + 1], [0]), m.feed(u[cut + 1:], range(len(u) - cut - 1))]), want)
    m.close()


@pytest.mark.parametrize("name", list(LM.SMALL))
def test_greedy_generation(tmp_path, Model, name):
    """The framework's own entry point: the token loop recorded once, run on the device."""
    cfg, orc, m = make(tmp_path, Model, name, seed=4)
    prompt = ids(cfg, 37, 9)
    got = m.generate(prompt, 60)
    lg, want = orc.feed(prompt)[-1], []
    for k in range(60):
        # where two logits are closer than rounding, either is right: go on with what the GPU took
        assert lg[got[k]] > lg.max() - 1e-3 * lg.std()
        want.append(int(np.argmax(lg)))
        lg = orc.feed([got[k]])[-1]
    assert sum(a == b for a, b in zip(got, want)) >= 59
    assert m.pos == 37 + 59
    close(m.feed([got[-1]], [0])[0], lg)                      # decoding goes on after the loop
    m.reset()
    assert m.generate(prompt, 60) == got
    m.close()


def test_refusals(tmp_path, Model):
    cfg, orc, m = make(tmp_path, Model, "no_loop", max_ctx=50, chunk=16)
    with pytest.raises(RuntimeError):
        m.feed([0] * 51)
    with pytest.raises(RuntimeError):
        m.feed([cfg["vocab"]])
    with pytest.raises(RuntimeError):
        m.feed([-1, 0, 1])
    assert m.pos == 0
    t = ids(cfg, 50, 1)
    close(m.feed(t, [49]), orc.feed(t)[[49]])
    with pytest.raises(RuntimeError):
        m.feed([1])                                           # full
    m.close()


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_replay(tmp_path, dtype):
    """bin/trace_run: portions of two requests one after the other, logits where asked."""
    cfg = LM.SMALL["loop_over_everything"]
    W = LM.weights(cfg, 11)
    folder, out = LM.write(tmp_path / "m", cfg, W), tmp_path / "out"
    out.mkdir()
    orc = Oracle(cfg, W)
    a, b = ids(cfg, 70, 1), ids(cfg, 20, 2)
    steps = [("a", a[:40], [0, 39], []), ("a", a[40:41], [], []), ("a", a[41:70], [28], ["a"]), ("b", b[:2], [1], []),
             ("b", b[2:3], [0], []), ("b", b[3:], [16], ["b"])]
    text = "".join(json.dumps({"step": n, "entries": [{"id": i, "tokens": t, "want": w}], "end": e}) + "\n"
                   for n, (i, t, w, e) in enumerate(steps))
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out", str(out),
                        "--max-tokens", "80"], input=text, capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done %d" % n for n in range(6)]
    la = orc.feed(a)
    orc.reset()
    lb = orc.feed(b)
    want = {0: la[[0, 39]], 2: la[[69]], 3: lb[[1]], 4: lb[[2]], 5: lb[[19]]}
    for n in range(6):
        f = out / ("%d.f32" % n)
        assert f.exists() == (n in want)
        if n in want:
            close(np.fromfile(f, "<f4").reshape(-1, cfg["vocab"]), want[n])


def test_qwen_through_the_same_entry_point(tmp_path, Model):
    """A GGUF file opened by the registry gives the logits of the Qwen harness's own steps: a prompt in
    portions, single tokens on the recorded step, a second sequence, generation."""
    import ggufwriter
    from test_gpu_gguf import SMALL, synth_weights
    qwen = importlib.import_module("cpp-tensorlib_amd.qwen")
    path = str(tmp_path / "model.gguf")
    ggufwriter.qwen2_file(path, SMALL, synth_weights(SMALL, seed=3))
    g = qwen.QwenGPU.from_gguf(path, fmt="bf16", max_ctx=SMALL["max_ctx"])
    m = Model.open(path, max_ctx=SMALL["max_ctx"])
    assert m.architecture == "qwen2" and m.vocab == SMALL["vocab"]
    t = [int(x) for x in np.random.default_rng(1).integers(0, SMALL["vocab"], 30)]
    want = np.stack([g.step(x, i, want_logits=True)[1] for i, x in enumerate(t)])
    for _ in range(2):
        m.reset()
        got = np.concatenate([m.feed(t[:13], range(13)), m.feed(t[13:14], [0]), m.feed(t[14:15], [0]), m.feed(t[15:], range(15))])
        close(got, want)
    m.reset()
    out = m.generate(t[:20], 12)
    g.set_cache_pos(0)
    tok = [g.step(x, i) for i, x in enumerate(t[:20])][-1]
    for k in range(12):
        assert out[k] == tok
        tok = g.step(tok, 20 + k)
    g.close()
    m.close()
