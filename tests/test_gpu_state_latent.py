"""State-space layers (Mamba-2), latent attention over its operand-form cache, and norms of sublayer outputs,
each mechanism alone through the C ABI against the plain implementation (tests/girirax_oracle.py)."""
import importlib

import numpy as np
import pytest

import girirax_oracle as O

pytestmark = pytest.mark.gpu


@pytest.fixture(scope="module")
def capi():
    return importlib.import_module("cpp-tensorlib_amd.capi")


def rng(seed):
    return np.random.default_rng(seed)


def bf16_bits(a):
    """f32 -> (bits, the value they hold), round to nearest even."""
    x = np.ascontiguousarray(a, np.float32).view(np.uint32)
    b = ((x + 0x7fff + ((x >> 16) & 1)) >> 16).astype(np.uint16)
    return b, (b.astype(np.uint32) << 16).view(np.float32)


def close(got, want, tol=2e-5):
    scale = np.abs(want).max() + 1e-6
    err = np.abs(got - want).max() / scale
    assert err < tol, "relative error %.3g" % err


# ---- state space ---------------------------------------------------------------------------------

class State:
    """Rows u = [pad | z | x | B | C | dt], rows y = [pad | out]."""

    def __init__(self, lib, capi, H, N, G, V, taps, seed=0, a_log=0.0, dt_bias=-1.0, spread=0.5):
        g = rng(seed)
        self.lib, self.c = lib, dict(heads=H, state=N, groups=G, vdim=V, conv=taps)
        inner, ch = H * V, H * V + 2 * G * N
        self.ch, self.inner = ch, inner
        self.w, self.b = (g.standard_normal((ch, taps)) * 1.5 / np.sqrt(taps)).astype(np.float32), (0.3 * g.standard_normal(ch)).astype(np.float32)
        self.dt_bias = (dt_bias + spread * g.standard_normal(H)).astype(np.float32)
        self.A_log = (a_log + spread * g.standard_normal(H)).astype(np.float32)
        self.D = g.standard_normal(H).astype(np.float32)
        self.W, self.ldy = 4 + inner + ch + H + 3, inner + 5
        up = lambda a: lib.to_device(np.ascontiguousarray(a, np.float32))
        self.conv = up(np.full(lib.c.tlhip_ssm_conv_bytes(H, N, G, V, taps) // 4, 9.0))
        self.state = up(np.full(lib.c.tlhip_ssm_state_bytes(H, N, V) // 4, 7.0))
        self.dev = [up(self.w.T), up(self.b), up(self.dt_bias), up(-np.exp(self.A_log.astype(np.float64)) / np.log(2)), up(self.D)]
        self.s = capi.Ssm(heads=H, state=N, groups=G, vdim=V, taps=taps, z_off=4, x_off=4 + inner, dt_off=4 + inner + ch, y_off=2,
                          conv_w=self.dev[0].ptr, conv_b=self.dev[1].ptr, dt_bias=self.dev[2].ptr, decay=self.dev[3].ptr,
                          skip=self.dev[4].ptr, conv_state=self.conv.ptr, ssm_state=self.state.ptr)

    def rows(self, T, seed):
        return rng(seed).standard_normal((T, self.W)).astype(np.float32)

    def chunk(self, u, pos0):
        T = len(u)
        du, dy = self.lib.to_device(np.ascontiguousarray(u, np.float32)), self.lib.to_device(np.zeros((T, self.ldy), np.float32))
        self.lib.ssm_chunk(du, self.W, dy, self.ldy, self.s, T, pos0)
        return dy.numpy()[:, 2:2 + self.inner]

    def step(self, u, pos, d_pos=None):
        du, dy = self.lib.to_device(np.ascontiguousarray(u, np.float32)), self.lib.to_device(np.zeros(self.ldy, np.float32))
        self.lib.ssm_step(du, dy, self.s, pos if d_pos is None else 0, d_pos)
        return dy.numpy()[2:2 + self.inner]

    def want(self, u):
        f = lambda a: a.astype(np.float64)
        return O.mamba2_core(f(u)[:, 4:], f(self.w), f(self.b), f(self.dt_bias), f(self.A_log), f(self.D), self.c, {})


STATES = [  # H, N, G, V, taps
    (6, 16, 2, 24, 4), (3, 64, 1, 64, 4), (4, 33, 4, 10, 3), (2, 128, 1, 100, 2), (5, 7, 5, 3, 1), (8, 48, 2, 32, 6), (1, 200, 1, 130, 4)]


@pytest.mark.parametrize("H,N,G,V,taps", STATES)
def test_state_space_chunks_and_steps(lib, capi, H, N, G, V, taps):
    """One prompt in one chunk, in portions, token by token, and portions and steps in turn."""
    T = 150
    s = State(lib, capi, H, N, G, V, taps, seed=N)
    u = s.rows(T, N + 1)
    want = s.want(u)
    close(s.chunk(u, 0), want)
    for size in (2, 3, 16, 33, 64, 97):                      # over what the sequence before left in the state
        close(np.concatenate([s.chunk(u[t:t + size], t) for t in range(0, T, size)]), want)
    close(np.stack([s.step(u[t], t) for t in range(T)]), want)
    got, t = [], 0
    for n in (1, 3, 1, 1, 40, 2, 1, 70, 1, 30):
        got.append(s.chunk(u[t:t + n], t) if n > 1 else s.step(u[t], t)[None])
        t += n
    close(np.concatenate(got), want)


def test_convolution_reaches_across_every_cut(lib, capi):
    """An impulse in the convolution's channels is met by each of its taps, wherever a portion ends."""
    s = State(lib, capi, 2, 16, 1, 12, 5, seed=1)
    T = 24
    u = 0.01 * s.rows(T, 2)
    u[9, 4 + s.inner:4 + s.inner + s.ch] = 30.0
    want = s.want(u)
    flat = u.copy()
    flat[9] = u[8]
    moved = np.abs(want - s.want(flat)).max(axis=1)
    assert moved[9:14].min() > 0.1 and moved[:9].max() == 0   # it shows
    for cut in range(8, 16):
        close(np.concatenate([s.chunk(u[:cut], 0), s.chunk(u[cut:cut + 2], cut), s.chunk(u[cut + 2:], cut + 2)]), want)
        close(np.concatenate([s.chunk(u[:cut], 0)] + [s.step(u[t], t)[None] for t in range(cut, T)]), want)


@pytest.mark.parametrize("dt_bias,a_log", [(-12.0, -6.0), (3.0, 3.0), (60.0, 4.0), (-40.0, 0.0), (0.0, -30.0)])
def test_state_space_under_extreme_decays(lib, capi, dt_bias, a_log):
    """Steps and decays far from one on either side: nothing overflows, tiny steps keep their relative size."""
    s = State(lib, capi, 4, 32, 2, 20, 4, seed=3, a_log=a_log, dt_bias=dt_bias)
    s.D[:] = 0                                               # the state alone
    s.dev[4].upload(s.D)
    u = s.rows(130, 4)
    want = s.want(u)
    size = np.abs(want).max()
    close(s.chunk(u, 0) / size, want / size)
    close(np.stack([s.step(u[t], t) for t in range(60)]) / size, want[:60] / size)


def test_state_space_keeps_a_far_token(lib, capi):
    """With slow decays one strong token is still read two thousand tokens later; a step can be repeated at its
    position; a new sequence starts from zero whatever the slots hold."""
    s = State(lib, capi, 2, 24, 1, 16, 4, seed=8, a_log=-9.0, dt_bias=0.0, spread=0.1)
    T = 2000
    u = 0.05 * s.rows(T, 6)
    u[5, 4 + s.inner:] = 6.0
    u[T - 1, 4 + s.inner + s.inner + 24:4 + s.inner + s.ch] = 6.0    # C of the last token
    want = s.want(u)
    lone = u.copy()
    lone[5] = u[20]
    assert np.abs(s.want(lone)[T - 1] - want[T - 1]).max() > 0.05 * np.abs(want[T - 1]).max()   # it shows
    got = np.concatenate([s.chunk(u[t:t + 499], t) for t in range(0, 1996, 499)] + [s.chunk(u[1996:T - 1], 1996)])
    close(got, want[:T - 1], 1e-4)
    d_pos = lib.to_device(np.array([T - 1], np.uint32))
    a, b, c = s.step(u[T - 1], T - 1), s.step(u[T - 1], T - 1), s.step(u[T - 1], T - 1, d_pos)
    close(a, want[T - 1], 1e-4)
    assert np.array_equal(a, b) and np.array_equal(a, c)
    v = s.rows(20, 7)
    close(np.stack([s.step(v[t], t) for t in range(20)]), s.want(v))
    close(s.chunk(v, 0), s.want(v))


# ---- latent attention ----------------------------------------------------------------------------

class Latent:
    """Rows u = [pad | latent | key part | gate], rows q, rows y = [pad | out]."""

    def __init__(self, lib, capi, H, D, R, V, L, capacity, planes=3, gate=True, scale=None, base=1e4, seed=0, eps=1e-5):
        g = rng(seed)
        self.lib, self.base, self.eps, self.gate, self.planes = lib, base, eps, gate, planes
        self.c = dict(heads=H, dim=D, rot_dim=R, vdim=V, kv_rank=L, scale=scale or (D + R) ** -0.5)
        ld = (L + 7) // 8 * 8
        up = lambda a: lib.to_device(np.ascontiguousarray(a))
        pad = lambda b: np.pad(b, ((0, 0), (0, ld - L)))
        bk, self.uk = bf16_bits(g.standard_normal((H * D, L)) / np.sqrt(L))
        bv, self.uv = bf16_bits(g.standard_normal((H * V, L)) / np.sqrt(L))
        self.norm = (1 + 0.3 * g.standard_normal(L)).astype(np.float32)
        p, i = np.arange(capacity)[:, None], np.arange(R // 2)[None]
        a = p * base ** (-2.0 * i / max(R, 1))
        tab = np.stack([np.cos(a), np.sin(a)], -1).astype(np.float32)
        kb, vb = (lib.c.tlhip_latent_cache_bytes(capacity, L, R, planes, v) for v in (0, 1))
        junk = lambda n: np.full(n // 2, 0x4120, np.uint16)  # 10.0 wherever nothing was written
        self.dev = [up(pad(bk)), up(pad(bv)), up(self.norm), up(tab) if R else lib.empty(4), up(junk(kb)), up(junk(vb))]
        self.W, self.ldy, self.ldq = 4 + L + R + H * V + 1, H * V + 3, H * (D + R) + 2
        self.a = capi.LatentAttn(heads=H, dim=D, rot_dim=R, vdim=V, kv_rank=L, kv_off=4, gate_off=4 + L + R if gate else -1, y_off=1,
                                 uk=self.dev[0].ptr, uv=self.dev[1].ptr, kv_norm=self.dev[2].ptr, angles=self.dev[3].ptr,
                                 keys=self.dev[4].ptr, values=self.dev[5].ptr, capacity=capacity, planes=planes,
                                 scale=self.c["scale"], eps=eps)

    def rows(self, T, seed, amp=1.5):
        g = rng(seed)
        return g.standard_normal((T, self.W)).astype(np.float32), (amp * g.standard_normal((T, self.ldq))).astype(np.float32)

    def run(self, u, q, pos0, d_pos=None):
        T = len(u)
        du, dq = self.lib.to_device(np.ascontiguousarray(u, np.float32)), self.lib.to_device(np.ascontiguousarray(q, np.float32))
        dy = self.lib.to_device(np.zeros((T, self.ldy), np.float32))
        self.lib.latent_attn(du, self.W, dq, self.ldq, dy, self.ldy, self.a, T, pos0 if d_pos is None else 0, d_pos)
        return dy.numpy()[:, 1:1 + self.c["heads"] * self.c["vdim"]]

    def want(self, u, q, pos0=0, st=None):
        f = lambda a: a.astype(np.float64)
        H, D, R, V, L = (self.c[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
        o = O.latent_core(f(q)[:, :H * (D + R)], f(u)[:, 4:4 + L + R], f(self.norm), f(self.uk), f(self.uv), self.c, self.base,
                          self.eps, pos0, {} if st is None else st)
        return o * O.sigmoid(f(u)[:, 4 + L + R:4 + L + R + H * V]) if self.gate else o


LATENTS = [  # H, D, R, V, L
    (4, 32, 16, 24, 96), (1, 64, 8, 64, 64), (3, 20, 6, 17, 33), (33, 8, 4, 8, 160), (5, 100, 2, 40, 7), (16, 16, 32, 16, 512),
    (2, 12, 0, 12, 40), (7, 48, 64, 130, 260)]
# three terms add up to the f32; one is a rounding of 2^-9 per cached number
PLANES = [(3, 5e-5), (1, 1.5e-2)]


@pytest.mark.parametrize("planes,tol", PLANES)
@pytest.mark.parametrize("H,D,R,V,L", LATENTS)
def test_latent_attention_chunks_and_steps(lib, capi, H, D, R, V, L, planes, tol):
    """One prompt in one chunk, in portions, token by token; the sequence before is still in the cache."""
    T = 101
    a = Latent(lib, capi, H, D, R, V, L, 128, planes, gate=L != 64, seed=L)
    u, q = a.rows(T, L + 1)
    want = a.want(u, q)
    close(a.run(u, q, 0), want, tol)
    for size in (2, 31, 32, 50):
        close(np.concatenate([a.run(u[t:t + size], q[t:t + size], t) for t in range(0, T, size)]), want, tol)
    close(np.concatenate([a.run(u[t:t + 1], q[t:t + 1], t) for t in range(T)]), want, tol)
    v, r = a.rows(40, L + 2, 3.0)                            # another sequence over the same rows
    close(np.concatenate([a.run(v[:2], r[:2], 0), a.run(v[2:3], r[2:3], 2), a.run(v[3:], r[3:], 3)]), a.want(v, r), 2 * tol)


@pytest.mark.parametrize("planes", [3, 1])
@pytest.mark.parametrize("H", [1, 3, 40])
def test_single_keys_show(lib, capi, H, planes):
    """A query that singles out ONE key by its latent: its value comes back from any distance, at and around the
    tiles' borders, for every head; the key is not seen by the token before it."""
    D, R, V, L, T = 24, 8, 16, 48, 140
    a = Latent(lib, capi, H, D, R, V, L, 160, planes, gate=False, scale=1.0, seed=5)
    u, q = a.rows(T, 6, 0.02)
    u[:, 4 + L:4 + L + R] = 0
    base = u.copy()
    base[:, 4] = 0                                           # the first latent number is the key's own
    for key in (0, 1, 31, 32, 33, 63, 64, 127, 128):
        u = base.copy()
        u[key, 4] = 30.0
        at = [t for t in (key, key + 1, 31, 32, 64, 127, 128, 139) if t >= key] + ([key - 1] if key else [])
        qk = q.copy()
        lat = O.rms_norm(u[:, 4:4 + L].astype(np.float64), a.norm, a.eps)
        for h in range(H):                                   # the query of every head points at this key only
            k = lat @ a.uk[h * D:(h + 1) * D].astype(np.float64).T
            others = np.delete(k, key, axis=0)
            d = k[key] - others.mean(axis=0)
            margin = (k[key] @ d) - (others @ d).max()
            for t in at:
                assert margin > 1
                qk[t, h * (D + R):h * (D + R) + D] = 30.0 * d / margin
        want = a.want(u, qk)
        lone = a.want(base, qk)
        for t in at:
            change = np.abs(lone[t] - want[t]).max()
            assert (change > 0.2) if t >= key else (change == 0)   # it shows, and only from its position on
        tol = 1e-4 if planes == 3 else 4e-2
        close(a.run(u, qk, 0), want, tol)
        for t in sorted(at):
            close(a.run(u[t:t + 1], qk[t:t + 1], t)[0], want[t], tol)


@pytest.mark.parametrize("planes,tol", PLANES)
def test_rotation_depends_on_the_distance(lib, capi, planes, tol):
    """Rotated parts alone: a score is a function of the distance, also deep in a context."""
    H, D, R, V, L, base = 2, 4, 16, 8, 32, 50.0
    a = Latent(lib, capi, H, D, R, V, L, 4096, planes, gate=False, scale=1.0, base=base, seed=2)
    u, q = a.rows(24, 3, 1.0)
    q.reshape(24, -1)[:, :] = 0
    for h in range(H):
        q[:, h * (D + R) + D:(h + 1) * (D + R)] = rng(9).standard_normal((24, R))
    want = a.want(u, q)
    close(a.run(u, q, 0), want, tol)
    # the same rows behind 4000 tokens whose keys are far below: only the distances are left
    T0 = 4000
    f, z = a.rows(T0, 4, 0.0)
    st = {}
    a.want(f, z, 0, st)
    deep = a.want(u, q, T0, st)
    for t in range(0, T0, 1000):
        a.run(f[t:t + 1000], z[t:t + 1000], t)
    close(a.run(u, q, T0), deep, tol)


@pytest.mark.parametrize("planes,tol", PLANES)
@pytest.mark.parametrize("H", [4, 20])
def test_long_context_in_chunks_and_steps(lib, capi, H, planes, tol):
    """Keys split over blocks: chunks and steps deep in a context; the device position gives the host position's
    bits; a step can be repeated."""
    D, R, V, L, T0, T = 24, 8, 16, 72, 1500, 77
    a = Latent(lib, capi, H, D, R, V, L, 2048, planes, seed=1)
    u, q = a.rows(T0 + T, 9)
    for t in range(0, T0, 500):
        a.run(u[t:t + 500], q[t:t + 500], t)
    got = a.run(u[T0:], q[T0:], T0)
    st = {}
    a.want(u[:T0 - 1], np.zeros_like(q[:T0 - 1]), 0, st)
    want = a.want(u[T0 - 1:], q[T0 - 1:], T0 - 1, st)[1:]
    close(got, want, tol)
    d_pos = lib.to_device(np.zeros(1, np.uint32))
    for t in (0, 1, 35, 36, 76):
        p = T0 + t
        s = a.run(u[p:p + 1], q[p:p + 1], p)
        close(s[0], want[t], tol)
        d_pos.upload(np.array([p], np.uint32))
        assert np.array_equal(a.run(u[p:p + 1], q[p:p + 1], p, d_pos), s)


# ---- norms of what a sublayer wrote, activations, token rows ---------------------------------------

@pytest.mark.parametrize("n,parts,K,N", [(96, 1, 96, 40), (60, 5, 64, 33), (105, 7, 128, 520), (2048, 8, 2048, 1000), (384, 96, 384, 16),
                                         (5000, 1, 5024, 700), (3584, 2, 3584, 4096)])
def test_product_of_a_normed_sum(lib, n, parts, K, N):
    g = rng(n)
    x, d, b = (g.standard_normal(K).astype(np.float32) for _ in range(3))
    w = np.zeros(K, np.float32)
    w[:n] = 1 + 0.3 * g.standard_normal(n)
    bits, W = bf16_bits(g.standard_normal((N, K)) / np.sqrt(K))
    dx, dd, db, dw, dW = (lib.to_device(v) for v in (x, d, b, w, bits))
    d[n:] = 5.0                                              # meets zero entries of the norm's weight
    for with_x, with_b in ((1, 1), (1, 0), (0, 0)):
        s = np.zeros(K)
        s[:n] = O.grouped_rms_norm((d + with_b * b)[None, :n].astype(np.float64), w[:n], parts, 1e-3)
        s += with_x * x
        y, out = lib.empty(N), lib.to_device(np.zeros(K, np.float32))
        lib.gemv_bf16_row_postnorm(dx if with_x else None, dd, db if with_b else None, dw, n, parts, out, dW, y, N, K, 1e-3)
        close(out.numpy(), s, 2e-6)
        close(y.numpy(), W.astype(np.float64) @ s)


@pytest.mark.parametrize("K,ff", [(64, 24), (1024, 160), (3584, 500)])
def test_gated_gelu_of_a_normed_sum(lib, K, ff):
    g = rng(K)
    x, d, b, w = (g.standard_normal(K).astype(np.float32) for _ in range(4))
    gb = (2 * g.standard_normal(2 * ff)).astype(np.float32)
    gb[:4] = (-30.0, 30.0, -9.0, 4.0)
    bits, W = bf16_bits(g.standard_normal((2 * ff, K)) / np.sqrt(K))
    s = x + O.rms_norm((d + b).astype(np.float64), w, 1e-5)
    z = W.astype(np.float64) @ s + gb
    want = O.gelu_tanh(z[:ff]) * z[ff:]
    dx, dd, db, dw, dW, dg = (lib.to_device(v) for v in (x, d, b, w, bits, gb))
    act, out = lib.empty(ff), lib.empty(K)
    lib.gemv_bf16_row_postnorm_geglu(dx, dd, db, dw, out, dW, dg, act, 2 * ff, K, 1e-5)
    close(act.numpy(), want)
    close(out.numpy(), s, 2e-6)
    rows = np.stack([z - gb, -(z - gb), np.zeros(2 * ff)]).astype(np.float32)
    o = lib.to_device(np.zeros((3, ff), np.float32))
    lib.geglu_rows(lib.to_device(rows), dg, o, ff, 3)
    zz = rows.astype(np.float64) + gb
    close(o.numpy(), O.gelu_tanh(zz[:, :ff]) * zz[:, ff:])


@pytest.mark.parametrize("n", [32, 300, 4096, 5000, 8192, 20000])
def test_normed_sums_of_rows(lib, n):
    g = rng(n)
    rows = 5
    for S, with_b in ((1, 0), (3, 1)):
        x, b, w = g.standard_normal((rows, n)).astype(np.float32), g.standard_normal(n).astype(np.float32), g.standard_normal(n).astype(np.float32)
        parts = g.standard_normal((S, rows, n)).astype(np.float32)
        want = x + O.rms_norm((parts.sum(0) + with_b * b).astype(np.float64), w, 1e-4)
        dx = lib.to_device(x)
        lib.postnorm_res_parts(dx, lib.to_device(parts), S, lib.to_device(b) if with_b else None, lib.to_device(w), dx, n, 1e-4, rows)
        close(dx.numpy(), want, 3e-6)


@pytest.mark.parametrize("n,parts,n_out", [(96, 1, 96), (60, 3, 64), (63, 7, 70), (2000, 4, 2000), (257, 1, 300)])
def test_grouped_norm_of_rows(lib, n, parts, n_out):
    g = rng(n)
    x, w = g.standard_normal((6, n + 5)).astype(np.float32), g.standard_normal(n).astype(np.float32)
    out = lib.to_device(np.full((6, n_out + 2), 3.0, np.float32))
    lib.rms_rows(lib.to_device(x), n + 5, lib.to_device(w), out, n_out + 2, n, n_out, parts, 1e-3, 6)
    got = out.numpy()
    close(got[:, :n], O.grouped_rms_norm(x[:, :n].astype(np.float64), w, parts, 1e-3), 3e-6)
    assert not got[:, n:n_out].any() and (got[:, n_out:] == 3.0).all()


def test_scaled_token_rows(lib):
    vocab, width, ldt, ld, T = 50, 37, 48, 40, 6
    bits, table = bf16_bits(rng(1).standard_normal((vocab, ldt)))
    ids = np.array([3, 49, 0, 7, 7, 21], np.int32)
    out = lib.to_device(np.full((T, ld), 9.0, np.float32))
    lib.embed_scaled(lib.to_device(bits), ldt, lib.to_device(ids), out, T, width, ld, vocab, 2.75)
    got = out.numpy()
    assert np.array_equal(got[:, :width], table[ids][:, :width] * np.float32(2.75)) and not got[:, width:].any()


def test_refusals(lib, capi):
    """Shapes outside what the kernels hold are refused before anything is launched."""
    s = State(lib, capi, 4, 16, 2, 8, 4)
    u = lib.to_device(np.zeros((8, s.W), np.float32))
    y = lib.to_device(np.zeros((8, s.ldy), np.float32))
    for field, value in (("groups", 3), ("state", 1000), ("vdim", 2000), ("taps", 65), ("ssm_state", None)):
        old = getattr(s.s, field)
        setattr(s.s, field, value)
        with pytest.raises(capi.TlHipError):
            lib.ssm_chunk(u, s.W, y, s.ldy, s.s, 4, 0)
        with pytest.raises(capi.TlHipError):
            lib.ssm_step(u, y, s.s, 0)
        setattr(s.s, field, old)
    a = Latent(lib, capi, 2, 8, 4, 8, 32, 64)
    u, q, y = (lib.to_device(np.zeros((8, w), np.float32)) for w in (a.W, a.ldq, a.ldy))
    with pytest.raises(capi.TlHipError):
        lib.latent_attn(u, a.W, q, a.ldq, y, a.ldy, a.a, 8, 60)     # past the cache's end
    for field, value in (("planes", 2), ("kv_rank", 2048), ("rot_dim", 3), ("capacity", 40), ("uk", None)):
        old = getattr(a.a, field)
        setattr(a.a, field, value)
        with pytest.raises(capi.TlHipError):
            lib.latent_attn(u, a.W, q, a.ldq, y, a.ldy, a.a, 4, 0)
        setattr(a.a, field, old)
