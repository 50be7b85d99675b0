"""Girirax models end to end on the GPU, against the plain implementation (tests/girirax_oracle.py):
whole prompts, portions, token by token, several sequences one after the other, far tokens through the
state and through the keys, long decoding, greedy generation, and trace replay."""
import importlib
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import girirax_models as GM
import lusadra_models as LM
from girirax_oracle import Oracle

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
# exact: every product and the latent cache; serving: the cache rounded to bf16
TOL = {True: 2e-4, False: 3e-2}


@pytest.fixture(scope="module")
def Model():
    return importlib.import_module("cpp-tensorlib_amd.model").Model


def close(got, want, tol):
    err = np.abs(got - want).max() / (np.abs(want).std() + 1e-9)
    assert err < tol, "largest difference over the spread: %.3g" % err


def ids(cfg, n, seed):
    return [int(t) for t in np.random.default_rng(seed).integers(0, cfg["vocab"], n)]


def make(tmp_path, Model, name, seed=1, exact=True, max_ctx=400, chunk=64, **kw):
    cfg = GM.SMALL[name]
    W = GM.weights(cfg, seed, **kw)
    return cfg, Oracle(cfg, W), Model.open(LM.write(tmp_path / name, cfg, W), max_ctx=max_ctx, chunk=chunk, exact=exact)


@pytest.mark.parametrize("exact", [True, False])
@pytest.mark.parametrize("name", list(GM.SMALL))
def test_prompt_portions_and_steps(tmp_path, Model, name, exact):
    """The logits at every position do not depend on how the tokens were cut, nor on the sequence that
    ran before in the same caches and states."""
    cfg, orc, m = make(tmp_path, Model, name, exact=exact)
    assert m.architecture == "Girirax" and m.vocab == cfg["vocab"]
    n = 150
    t = ids(cfg, n, 2)
    want = orc.feed(t)
    whole = m.feed(t, range(n))                               # longer than a chunk: three of them
    close(whole, want, TOL[exact])
    for sizes in ((2,), (1,), (31, 2, 1, 1, 3), (64, 1), (7, 33)):
        m.reset()
        got, at, k = [], 0, 0
        while at < n:
            c = min(sizes[k % len(sizes)], n - at)
            got.append(m.feed(t[at:at + c], range(c)))
            at, k = at + c, k + 1
        close(np.concatenate(got), want, TOL[exact])
    m.reset()
    orc.reset()
    u = ids(cfg, 40, 3)                                       # another sequence after those
    close(m.feed(u, [0, 1, 17, 39]), orc.feed(u)[[0, 1, 17, 39]], TOL[exact])
    m.close()


def test_large_products_in_both_forms(Model):
    """At sizes where prompt products run over the prepared weights, the serving form stays within its rounding of
    the exact one; a chunk equals steps."""
    cfg = GM.config(2000, 1120, [GM.ssm(24, 64, 2, 48, 4, 4, 3000), GM.latent(16, 64, 32, 96, 320, 352, 0.1, 1e4, 3000),
                                 GM.ssm(12, 96, 1, 80, 4, 3, None)], 4.0, 0.5)
    t = ids(cfg, 700, 12)
    want = [0, 1, 100, 159, 160, 161, 511, 512, 513, 699]
    lg = {}
    for exact in (True, False):
        m = Model.random(cfg, seed=3, max_ctx=800, exact=exact)
        lg[exact] = m.feed(t, want)
        m.reset()
        m.feed(t[:650])
        steps = np.concatenate([m.feed([x], [0]) for x in t[650:]])
        close(steps[-1], lg[exact][-1], 2e-4 if exact else 1e-2)
        m.close()
    close(lg[False], lg[True], 4e-2)


@pytest.mark.parametrize("name", list(GM.SMALL))
def test_unfused_step_equals_fused(tmp_path, Model, name):
    cfg, orc, m = make(tmp_path, Model, name)
    m.set_fused(False)
    t = ids(cfg, 30, 5)
    close(np.concatenate([m.feed([x], [0]) for x in t]), orc.feed(t), TOL[True])
    m.close()


@pytest.mark.parametrize("name", list(GM.SMALL))
def test_residual_after_every_layer(tmp_path, Model, name):
    cfg, orc, m = make(tmp_path, Model, name)
    t, rows = ids(cfg, 45, 6), []
    orc.feed(t, rows)
    got = m.trace_chunk(t, cfg["width"])
    assert len(got) == len(rows) == len(cfg["layers"])
    for g, w in zip(got, rows):
        close(g, w, 5e-5)
    m.close()


@pytest.mark.parametrize("exact", [True, False])
def test_far_tokens(tmp_path, Model, exact):
    """Slow decays: a token hundreds of positions back still changes the logits, and by as much as the plain form
    says, through the states and the latent keys; read in a prompt and in decoding."""
    cfg, orc, m = make(tmp_path, Model, "state_first", a_log=-7.0, dt_bias=0.0, max_ctx=700, exact=exact)
    t = ids(cfg, 600, 7)
    want = orc.feed(t)
    other = list(t)
    other[3] = (t[3] + 1) % cfg["vocab"]
    orc.reset()
    moved = orc.feed(other)
    # it shows, above the rounding
    assert np.sqrt(np.mean((moved[300:] - want[300:]) ** 2)) > 2 * TOL[True] * want[300:].std()
    assert all(np.abs(moved[k] - want[k]).max() > 2 * TOL[True] * want.std() for k in (340, 599))
    for seq, lg in ((t, want), (other, moved)):
        m.reset()
        a = m.feed(seq[:280], [100, 279])
        b = np.concatenate([m.feed([x], [0]) for x in seq[280:360]])
        c = m.feed(seq[360:], [0, 100, 239])
        close(np.concatenate([a, b, c]), lg[[100, 279] + list(range(280, 360)) + [360, 460, 599]], TOL[exact])
    m.close()


def test_long_decoding_and_many_sequences(tmp_path, Model):
    """Four hundred steps on one recorded graph, then short sequences in turn with portions, in the same
    caches: the convolution's ring wraps, both state slots are used from either parity."""
    cfg, orc, m = make(tmp_path, Model, "state_first", chunk=16)
    t = ids(cfg, 400, 8)
    want = orc.feed(t)
    close(np.concatenate([m.feed([x], [0]) for x in t]), want, TOL[True])
    for k in range(4):
        orc.reset()
        m.reset()
        u = ids(cfg, 20 + 7 * k, 20 + k)
        want = orc.feed(u)
        cut = 3 + k
        close(np.concatenate([m.feed(u[:cut], range(cut)), m.feed(u[cut:cut + 1], [0]), m.feed(u[cut + 1:], range(len(u) - cut - 1))]),
              want, TOL[True])
    m.close()


@pytest.mark.parametrize("name", list(GM.SMALL))
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
    close(m.feed([got[-1]], [0])[0], lg, TOL[True])           # decoding goes on after the loop
    m.reset()
    assert m.generate(prompt, 60) == got
    m.close()


def test_refusals(tmp_path, Model):
    cfg, orc, m = make(tmp_path, Model, "attention_first", max_ctx=50, chunk=16)
    for bad in ([0] * 51, [cfg["vocab"]], [-1, 0, 1]):
        with pytest.raises(RuntimeError):
            m.feed(bad)
    assert m.pos == 0
    t = ids(cfg, 50, 1)
    close(m.feed(t, [49]), orc.feed(t)[[49]], TOL[True])
    with pytest.raises(RuntimeError):
        m.feed([1])                                           # full
    m.close()


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_replay(tmp_path, dtype):
    """bin/trace_run: portions of two requests one after the other, logits where asked."""
    cfg = GM.SMALL["state_first"]
    W = GM.weights(cfg, 11)
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
            close(np.fromfile(f, "<f4").reshape(-1, cfg["vocab"]), want[n], TOL[dtype == "float32"])
