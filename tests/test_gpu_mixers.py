"""The mechanisms of layers with two mixers side by side, each alone through the C ABI, against the
plain implementation (tests/lusadra_oracle.py): sliding-window attention over tied keys and values,
gated linear attention, PolyNorm, token rows with sinusoidal positions, sums into the residual."""
import importlib

import numpy as np
import pytest

import lusadra_oracle as O

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


# ---- sliding-window attention --------------------------------------------------------------------

class Window:
    """One attention on the GPU: rows u = [q | k | gate], rows y = [out]."""

    def __init__(self, lib, capi, H, G, dim, window, chunk, gate=True, scale=None, coef=0.3, every=16, out_scale=1.0, exact=True):
        self.exact = exact
        self.lib, self.H, self.G, self.dim, self.window = lib, H, G, dim, window
        self.scale, self.coef, self.every = dim ** -0.5 if scale is None else scale, coef, every
        ld = lib.c.tlhip_window_ring_ld(dim)
        rows = (window - 1 + chunk + 31) // 32 * 32
        self.ring = lib.to_device(np.zeros((G, rows, ld), np.float32))
        qk = H * dim + G * dim
        self.W = (qk + (H * dim if gate else 0) + 3) // 4 * 4
        self.ldy = H * dim + 3
        self.at = capi.WindowAttn(heads=H, kv_heads=G, dim=dim, window=window, q_off=0, k_off=H * dim,
                                  gate_off=qk if gate else -1, y_off=1, ring=self.ring.ptr, ring_rows=rows, ring_ld=ld,
                                  scale=self.scale, temp_coef=coef, temp_every=every, slope_exp=8.0, out_scale=out_scale)
        self.gate, self.out_scale = gate, out_scale
        nb = lib.mix_partials_bytes(self.at)
        self.partials = lib.empty(nb // 4) if nb else None

    def chunk(self, u, pos0):
        T = len(u)
        du, dy = self.lib.to_device(np.ascontiguousarray(u, np.float32)), self.lib.to_device(np.zeros((T, self.ldy), np.float32))
        self.lib.window_attn_chunk(du, self.W, dy, self.ldy, self.at, T, pos0, self.exact)
        return dy.numpy()[:, 1:1 + self.H * self.dim]

    def step(self, u, pos, d_pos=None):
        du, dy = self.lib.to_device(np.ascontiguousarray(u, np.float32)), self.lib.to_device(np.zeros(self.ldy, np.float32))
        self.lib.mix_step(du, dy, self.at, None, None, pos if d_pos is None else 0, d_pos, self.partials)
        return dy.numpy()[1:1 + self.H * self.dim]

    def rows(self, T, seed, amp=1.0):
        u = rng(seed).standard_normal((T, self.W)).astype(np.float32)
        u[:, :self.H * self.dim] *= amp
        return u

    def want(self, u):
        H, D, G = self.H, self.dim, self.G
        a = O.window_attention(u[:, :H * D].astype(np.float64), u[:, H * D:(H + G) * D].astype(np.float64), H, G, D,
                               self.window, self.scale, self.coef, self.every)
        if self.gate:
            a = a * O.sigmoid(u[:, (H + G) * D:(H + G) * D + H * D].astype(np.float64))
        return a * self.out_scale


WINDOWS = [  # H, G, dim, window
    (3, 1, 40, 21), (6, 2, 32, 1), (4, 4, 64, 33), (7, 1, 96, 100), (2, 2, 128, 64), (5, 1, 20, 57), (4, 2, 160, 48),
    (2, 1, 256, 40), (1, 1, 30, 5)]


# the exact form of the chunk kernel, and the one whose f32 operands are two bf16 terms (2^-17 per
# product: scores of +-20 move weights by a few 1e-5)
FORMS = [(True, 2e-5), (False, 2e-4)]


@pytest.mark.parametrize("exact,tol", FORMS)
@pytest.mark.parametrize("H,G,dim,window", WINDOWS)
def test_window_attention_chunks_and_steps(lib, capi, H, G, dim, window, exact, tol):
    """One prompt in one chunk, in portions, and token by token, all against the plain form."""
    T = 2 * window + 45
    mk = lambda chunk: Window(lib, capi, H, G, dim, window, chunk=chunk, gate=dim != 64, out_scale=1.25, exact=exact)
    w = mk(T)
    u = w.rows(T, dim * 100 + window, amp=2.0)
    want = w.want(u)
    close(w.chunk(u, 0), want, tol)
    for size in (2, 31, 32, 50):
        w = mk(size)
        got = np.concatenate([w.chunk(u[t:t + size], t) for t in range(0, T, size)])
        close(got, want, tol)
    if exact:
        w = mk(1)
        close(np.stack([w.step(u[t], t) for t in range(T)]), want)


@pytest.mark.parametrize("exact", [True, False])
@pytest.mark.parametrize("H,G", [(2, 1), (9, 1), (3, 3)])
def test_window_edges_show(lib, capi, H, G, exact):
    """A query that singles out ONE key: seen at distance window - 1, gone at distance window; chunks
    and steps, keys at and around tile borders of the ring; every head, also where several share a
    block's tile or a group is spread over blocks."""
    dim, window = 32, 40
    T, far = 140, 200.0
    for key in (0, 31, 32, 63, 64, 71, 95):
        w = Window(lib, capi, H, G, dim, window, chunk=T, gate=False, coef=0.0, exact=exact)
        u = 0.1 * w.rows(T, 5)
        spike = np.zeros(dim, np.float32)
        spike[3] = 1.0
        for g in range(G):
            u[key, (H + g) * dim:(H + g + 1) * dim] = spike * far
        for t in (key + window - 1, key + window):          # just inside, just outside
            for h in range(H):
                u[t, h * dim:(h + 1) * dim] = spike * far
        want = w.want(u)
        for h in range(H):
            assert abs(want[key + window - 1, h * dim + 3]) > 100 and abs(want[key + window, h * dim + 3]) < 1   # it shows
        close(w.chunk(u, 0), want, 2e-5 if exact else 2e-4)
        if exact:
            w2 = Window(lib, capi, H, G, dim, window, chunk=1, gate=False, coef=0.0)
            close(np.stack([w2.step(u[t], t) for t in range(key + window + 2)]), want[:key + window + 2])


@pytest.mark.parametrize("H,G", [(8, 2), (7, 1), (4, 4)])
def test_window_chunks_deep_in_a_context(lib, capi, H, G):
    """Both chunk forms at positions past a long window, where the key tiles are split over blocks, in
    chunks that are no multiple of anything, against the plain form at some rows."""
    dim, window, T0, T = 64, 700, 900, 333
    outs = []
    for exact, tol in FORMS:
        w = Window(lib, capi, H, G, dim, window, chunk=T0, exact=exact)
        u = w.rows(T0 + T, 17, amp=1.5)
        w.chunk(u[:T0], 0)
        got = w.chunk(u[T0:], T0)
        k = u[:, H * dim:(H + G) * dim].astype(np.float64)
        gate = O.sigmoid(u[:, (H + G) * dim:(H + G) * dim + H * dim].astype(np.float64))
        for t in (0, 1, 31, 32, 200, 331, 332):
            i = T0 + t
            a = O.window_attention(u[i:i + 1, :H * dim].astype(np.float64), k[:i + 1], H, G, dim, window, w.scale, w.coef, w.every, pos0=i)
            close(got[t], (a * gate[i])[0], tol)
        outs.append(got)
    close(outs[1], outs[0], 2e-4)


def test_window_long_context_and_splits(lib, capi):
    """A window of several splits: decode at far positions equals the chunk kernel and the plain
    form; the device position gives the host position's bits."""
    H, G, dim, window = 8, 2, 64, 2100
    T = 2600
    w = Window(lib, capi, H, G, dim, window, chunk=T)
    assert w.partials is not None
    u = w.rows(T, 9)
    got = w.chunk(u, 0)
    rows = [0, 1, 511, 1023, 1024, 2099, 2100, 2101, 2599]
    a = O.window_attention(u[:, :H * dim].astype(np.float64)[rows[-1:]], u[:, H * dim:(H + G) * dim].astype(np.float64),
                           H, G, dim, window, w.scale, w.coef, w.every, pos0=T - 1)
    gate = O.sigmoid(u[:, (H + G) * dim:(H + G) * dim + H * dim].astype(np.float64))
    close(got[rows[-1]], (a * gate[rows[-1:]])[0])
    d_pos = lib.to_device(np.zeros(1, np.uint32))
    for t in rows:                     # the ring holds every key already: a step at t sees its own past
        s = w.step(u[t], t)
        close(s, got[t])
        d_pos.upload(np.array([t], np.uint32))
        assert np.array_equal(w.step(u[t], t, d_pos), s)


def test_window_attention_does_not_see_an_earlier_sequence(lib, capi):
    """The ring is used again without clearing: a new sequence at position 0 sees its own keys only."""
    w = Window(lib, capi, 4, 2, 48, 30, chunk=64)
    a, b = w.rows(64, 1, amp=3.0), w.rows(50, 2, amp=3.0)
    a[:, :] *= 10
    w.chunk(a, 0)
    close(w.chunk(b, 0), w.want(b))
    w.chunk(a, 0)
    close(np.stack([w.step(b[t], t) for t in range(20)]), w.want(b[:20]))


# ---- gated linear attention ----------------------------------------------------------------------

class Linear:
    """Rows u = [q | k | v | gate | low], rows y = [out]."""

    def __init__(self, lib, capi, H, dim, vdim, rank, tau, seed=0, bias=2.0, eps=1e-6, out_scale=1.0, spread=1.0):
        self.lib, self.H, self.D, self.V, self.R, self.tau, self.eps = lib, H, dim, vdim, rank, tau, eps
        g = rng(seed)
        bits, self.a2 = bf16_bits(g.standard_normal((H * dim, rank)) * spread / np.sqrt(rank))
        self.bias = (g.standard_normal(H * dim) * spread + bias).astype(np.float32)
        self.norm = (1 + 0.3 * g.standard_normal(vdim)).astype(np.float32)
        self.dev = [lib.to_device(bits), lib.to_device(self.bias), lib.to_device(self.norm)]
        self.state = lib.to_device(np.full(lib.c.tlhip_linear_state_bytes(H, dim, vdim) // 4, 7.0, np.float32))
        self.W = 2 * H * dim + 2 * H * vdim + rank
        self.W = (self.W + 3) // 4 * 4
        self.ldy, self.out_scale = H * vdim + 5, out_scale
        self.la = capi.LinearAttn(heads=H, dim=dim, vdim=vdim, rank=rank, q_off=0, k_off=H * dim, v_off=2 * H * dim,
                                  gate_off=2 * H * dim + H * vdim, low_off=2 * H * (dim + vdim), y_off=2,
                                  a2=self.dev[0].ptr, bias=self.dev[1].ptr, norm=self.dev[2].ptr, state=self.state.ptr,
                                  q_scale=dim ** -0.5, tau=tau, eps=eps, out_scale=out_scale)

    def chunk(self, u, pos0):
        T = len(u)
        du, dy = self.lib.to_device(np.ascontiguousarray(u, np.float32)), self.lib.to_device(np.zeros((T, self.ldy), np.float32))
        self.lib.linear_attn_chunk(du, self.W, dy, self.ldy, self.la, T, pos0)
        return dy.numpy()[:, 2:2 + self.H * self.V]

    def step(self, u, pos, d_pos=None):
        du, dy = self.lib.to_device(np.ascontiguousarray(u, np.float32)), self.lib.to_device(np.zeros(self.ldy, np.float32))
        self.lib.mix_step(du, dy, None, self.la, None, pos if d_pos is None else 0, d_pos)
        return dy.numpy()[2:2 + self.H * self.V]

    def rows(self, T, seed):
        return rng(seed).standard_normal((T, self.W)).astype(np.float32)

    def want(self, u):
        H, D, V = self.H, self.D, self.V
        u = u.astype(np.float64)
        cut = np.split(u, np.cumsum([H * D, H * D, H * V, H * V, self.R]), axis=1)
        alpha = O.decays(cut[4] @ self.a2.astype(np.float64).T + self.bias, self.tau)
        o, _ = O.gated_linear_attention(cut[0] * D ** -0.5, cut[1], cut[2], alpha, H, D, V)
        return O.head_norm(o, self.norm, H, V, self.eps) * cut[3] * O.sigmoid(cut[3]) * self.out_scale


LINEARS = [  # H, dim, vdim, rank, tau, bias
    (3, 24, 40, 5, 16.0, 2.0), (2, 64, 64, 16, 8.0, 0.0), (1, 16, 128, 1, 1.0, 3.0), (5, 48, 20, 12, 4.0, -1.0),
    (2, 128, 128, 16, 16.0, 4.0), (2, 200, 72, 24, 2.0, 1.0), (1, 7, 9, 3, 1.0, 0.0), (2, 32, 260, 8, 16.0, 2.0)]


@pytest.mark.parametrize("H,dim,vdim,rank,tau,bias", LINEARS)
def test_linear_attention_chunks_and_steps(lib, capi, H, dim, vdim, rank, tau, bias):
    T = 150
    mk = lambda: Linear(lib, capi, H, dim, vdim, rank, tau, seed=dim, bias=bias, out_scale=0.75)
    l = mk()
    u = l.rows(T, dim + 1)
    want = l.want(u)
    close(l.chunk(u, 0), want)
    for size in (2, 15, 16, 33, 64, 97):
        l = mk()
        close(np.concatenate([l.chunk(u[t:t + size], t) for t in range(0, T, size)]), want)
    l = mk()
    close(np.stack([l.step(u[t], t) for t in range(T)]), want)
    l = mk()                                                 # portions and steps in turn, on odd places
    got, t = [], 0
    for n in (1, 3, 1, 1, 40, 2, 1, 70, 1, 30):
        got.append(l.chunk(u[t:t + n], t) if n > 1 else l.step(u[t], t)[None])
        t += n
    assert t == T
    close(np.concatenate(got), want)


@pytest.mark.parametrize("bias", [-2.0, -12.0, -60.0, -400.0])
def test_linear_attention_under_strong_decays(lib, capi, bias):
    """tau = 1 and large negative logits: products of decays far below what one float can hold (each
    value alone must not overflow on the way), beside channels that keep everything."""
    l = Linear(lib, capi, 2, 32, 32, 4, 1.0, seed=3, bias=bias, spread=0.5)
    l.bias[::3] = 30.0                                       # every third channel forgets nothing
    l.dev[1].upload(l.bias)
    u = l.rows(130, 4)
    want = l.want(u)
    close(l.chunk(u, 0), want)
    l.step(u[0], 0)
    close(np.stack([l.step(u[t], t) for t in range(40)]), want[:40])


def test_linear_attention_keeps_a_far_token(lib, capi):
    """With decays near 1 a single strong key is still read two thousand tokens later; a step at the
    same position can be repeated; a new sequence starts from zero whatever the slots hold."""
    l = Linear(lib, capi, 2, 32, 24, 4, 16.0, seed=8, bias=14.0, spread=0.1)
    T = 2000
    u = 0.01 * l.rows(T, 6)
    u[5, 2 * 32] = 40.0                                      # k of head 0
    u[T - 1, 0] = 40.0                                       # q of head 0
    want = l.want(u)
    lone = u.copy()
    lone[5] = u[6]
    assert np.abs(l.want(lone)[T - 1, :24] - want[T - 1, :24]).max() > 0.01 * np.abs(want[T - 1, :24]).max()   # it shows
    got = np.concatenate([l.chunk(u[t:t + 499], t) for t in range(0, 1996, 499)] +
                         [l.chunk(u[1996:T - 1], 1996)])
    close(got[-1], want[T - 2])
    d_pos = lib.to_device(np.array([T - 1], np.uint32))
    a, b, c = l.step(u[T - 1], T - 1), l.step(u[T - 1], T - 1), l.step(u[T - 1], T - 1, d_pos)
    close(a[:24], want[T - 1, :24])
    assert np.array_equal(a, b) and np.array_equal(a, c)
    v = l.rows(20, 7)
    close(np.stack([l.step(v[t], t) for t in range(20)]), l.want(v))
    close(l.chunk(v, 0), l.want(v))


# ---- PolyNorm, token rows, sums ------------------------------------------------------------------

@pytest.mark.parametrize("ff", [1, 37, 512, 1024, 1025, 4096])
def test_polynorm(lib, capi, ff):
    T, W, ldy = 5, (ff + 3) // 4 * 4 + 4, ff + 9
    u = (2 * rng(ff).standard_normal((T, W))).astype(np.float32)
    pn = capi.PolyNorm(ff=ff, z_off=4, y_off=3, c1=0.7, c2=-0.4, c3=0.9, c0=0.2, eps=1e-5)
    want = O.polynorm(u[:, 4:4 + ff].astype(np.float64), (0.7, -0.4, 0.9, 0.2), 1e-5)
    dy = lib.to_device(np.zeros((T, ldy), np.float32))
    lib.polynorm_rows(lib.to_device(u), W, dy, ldy, pn, T)
    close(dy.numpy()[:, 3:3 + ff], want, 5e-6)
    for t in range(T):
        d1 = lib.to_device(np.zeros(ldy, np.float32))
        lib.mix_step(lib.to_device(u[t]), d1, None, None, pn, 0)
        close(d1.numpy()[3:3 + ff], want[t], 5e-6)


def test_all_sublayers_in_one_launch_equal_each_alone(lib, capi):
    """One launch over a row that holds everything writes the bits of three launches."""
    H, G, dim, window = 6, 2, 48, 50
    w = Window(lib, capi, H, G, dim, window, chunk=1)
    l = Linear(lib, capi, 3, 32, 40, 6, 4.0, seed=1)
    ff = 1300
    W = w.W + l.W + 1300
    for f in ("q_off", "k_off", "v_off", "gate_off", "low_off"):
        setattr(l.la, f, getattr(l.la, f) + w.W)
    l.la.y_off = w.ldy
    pn = capi.PolyNorm(ff=ff, z_off=w.W + l.W, y_off=w.ldy + l.ldy, c1=0.5, c2=0.2, c3=0.1, c0=-0.3, eps=1e-6)
    ldy = w.ldy + l.ldy + ff
    u = rng(11).standard_normal((8, W)).astype(np.float32)
    for t in range(8):
        du, one, three = lib.to_device(u[t]), lib.to_device(np.zeros(ldy, np.float32)), lib.to_device(np.zeros(ldy, np.float32))
        lib.mix_step(du, one, w.at, l.la, pn, t)
        lib.mix_step(du, three, w.at, None, None, t)
        lib.mix_step(du, three, None, l.la, None, t)
        lib.mix_step(du, three, None, None, pn, t)
        assert np.array_equal(one.numpy(), three.numpy())


def test_embed_sinusoid(lib):
    vocab, width, ld, T = 50, 37, 40, 6
    bits, table = bf16_bits(rng(1).standard_normal((vocab, width)))
    dt, ids = lib.to_device(bits), np.array([3, 49, 0, 7, 7, 21], np.int32)
    di = lib.to_device(ids)
    for pos0 in (0, 1, 4093, 100000):
        want = np.stack([table[i].astype(np.float64) + O.position_vector(pos0 + t, width) for t, i in enumerate(ids)])
        out = lib.to_device(np.full((T, ld), 9.0, np.float32))
        lib.embed_sinusoid(dt, di, out, T, width, ld, vocab, pos0)
        got = out.numpy()
        close(got[:, :width], want, 2e-6)
        assert not got[:, width:].any()
        d_pos = lib.to_device(np.array([pos0], np.uint32))
        again = lib.to_device(np.zeros((T, ld), np.float32))
        lib.embed_sinusoid(dt, di, again, T, width, ld, vocab, 0, d_pos)
        assert np.array_equal(again.numpy(), got)


def test_residual_sum_and_gather(lib):
    n, rows, S = 45, 7, 3
    g = rng(2)
    x, parts, add, vec = (g.standard_normal(s).astype(np.float32) for s in ((rows, n), (S, rows, n), (rows, n), (n,)))
    dx, dp, da, dv, out = (lib.to_device(a) for a in (x, parts, add, vec, np.zeros((rows, n), np.float32)))
    lib.residual_sum(dx, dp, S, da, dv, out, n, rows)
    close(out.numpy(), x + parts.sum(0) + add + vec, 1e-6)
    lib.residual_sum(dx, None, 0, None, dv, out, n, rows)
    assert np.array_equal(out.numpy(), x + vec)
    idx = lib.to_device(np.array([6, 0, 6, 2], np.int32))
    got = lib.to_device(np.zeros((4, n), np.float32))
    lib.gather_rows(dx, idx, got, n, 4, rows)
    assert np.array_equal(got.numpy(), x[[6, 0, 6, 2]])


def test_refusals(lib, capi):
    """Shapes outside what the kernels hold are refused before anything is launched."""
    w = Window(lib, capi, 2, 1, 32, 40, chunk=4)
    u = lib.to_device(np.zeros((200, w.W), np.float32))
    y = lib.to_device(np.zeros((200, w.ldy), np.float32))
    with pytest.raises(capi.TlHipError):                     # chunk longer than the ring can hold
        lib.window_attn_chunk(u, w.W, y, w.ldy, w.at, 120, 10)
    assert lib.c.tlhip_window_ring_ld(257) == 0
    w.at.ring_ld = 64
    with pytest.raises(capi.TlHipError):
        lib.window_attn_chunk(u, w.W, y, w.ldy, w.at, 4, 0)
    l = Linear(lib, capi, 1, 16, 16, 2, 1.0)
    l.la.dim = 600
    with pytest.raises(capi.TlHipError):
        lib.linear_attn_chunk(u, l.W, y, l.ldy, l.la, 4, 0)
