"""A plain, slow implementation of the Lusadra decoder in numpy (float64), one function per
mechanism, token by token where the mechanism is a recurrence. The GPU path is compared with it;
it shares no code with the product.

Weights are a dict name -> array (already widened); the configuration is the dict of config.json."""
import numpy as np

F = np.float64


def rms(x, eps):
    """Rows scaled to unit root mean square (last axis)."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return np.where(z >= 0, 1.0 / (1.0 + np.exp(-np.abs(z))), np.exp(-np.abs(z)) / (1.0 + np.exp(-np.abs(z))))


def position_vector(p, width):
    """Pairs of coordinates: sine and cosine of p over a wavelength that grows with the pair."""
    out = np.zeros(width, F)
    for c in range(width):
        i = c // 2
        a = p * 10000.0 ** (-2.0 * i / width)
        out[c] = np.sin(a) if c % 2 == 0 else np.cos(a)
    return out


def query_temperature(p, coef, every):
    return 1.0 + coef * np.log(np.floor((p + 1) / every) + 1.0)


def slope(h, heads):
    return 2.0 ** (-8.0 * (h + 1) / heads)


def window_attention(q, k, heads, kv_heads, dim, window, scale, coef, every, pos0=0):
    """q [T, heads*dim] for positions pos0 .. pos0+T-1, k [pos0+T, kv_heads*dim] for all positions;
    the values are the keys. A query meets itself and the window - 1 keys before it; a key loses slope
    for every position it lies back."""
    T = q.shape[0]
    out = np.zeros((T, heads * dim), F)
    for t in range(T):
        i = pos0 + t
        lo = max(0, i - window + 1)
        for h in range(heads):
            g = h // (heads // kv_heads)
            keys = k[lo:i + 1, g * dim:(g + 1) * dim]
            qv = q[t, h * dim:(h + 1) * dim] * query_temperature(i, coef, every)
            s = keys @ qv * scale - slope(h, heads) * (i - np.arange(lo, i + 1))
            w = np.exp(s - s.max())
            out[t, h * dim:(h + 1) * dim] = (w / w.sum()) @ keys
    return out


def decays(z, tau):
    """Share of a state row that outlives one token, from its logit."""
    return sigmoid(z) ** (1.0 / tau)


def gated_linear_attention(q, k, v, alpha, heads, dim, vdim, state=None):
    """Per head and token: every state row decays by its alpha and takes k_c v, then q reads the rows.
    Returns o [T, heads*vdim] and the last state [heads, dim, vdim]. q is taken as scaled already."""
    T = q.shape[0]
    S = np.zeros((heads, dim, vdim), F) if state is None else state.copy()
    o = np.zeros((T, heads * vdim), F)
    for t in range(T):
        for h in range(heads):
            kt, qt = k[t, h * dim:(h + 1) * dim], q[t, h * dim:(h + 1) * dim]
            vt = v[t, h * vdim:(h + 1) * vdim]
            S[h] = alpha[t, h * dim:(h + 1) * dim][:, None] * S[h] + np.outer(kt, vt)
            o[t, h * vdim:(h + 1) * vdim] = S[h].T @ qt
    return o, S


def head_norm(o, w, heads, vdim, eps):
    out = np.zeros_like(o)
    for h in range(heads):
        s = slice(h * vdim, (h + 1) * vdim)
        out[:, s] = rms(o[:, s], eps) * w
    return out


def polynorm(z, coef, eps):
    c1, c2, c3, c0 = coef
    return c1 * rms(z, eps) + c2 * rms(z ** 2, eps) + c3 * rms(z ** 3, eps) + c0


def left_mixer(h, W, p, c, pos0, past):
    """past: keys of the positions before pos0 [pos0, kv_heads*dim]; returns (output, all keys)."""
    q = h @ W[p + "q"].T
    k = np.concatenate([past, h @ W[p + "k"].T]) if past is not None else h @ W[p + "k"].T
    a = window_attention(q, k, c["heads"], c["kv_heads"], c["dim"], c["mask"]["size"], c["scale"],
                         c["q_temp"]["coef"], c["q_temp"]["every"], pos0)
    return (a * sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T, k


def right_mixer(h, W, p, c, eps, state):
    H, D, V = c["heads"], c["dim"], c["vdim"]
    q = h @ W[p + "q"].T * D ** -0.5
    k, v = h @ W[p + "k"].T, h @ W[p + "v"].T
    z = (h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "a2.b"]
    o, S = gated_linear_attention(q, k, v, decays(z, c["tau"]), H, D, V, state)
    o = head_norm(o, W[p + "norm"], H, V, eps)
    g = h @ W[p + "g"].T
    return (o * (g * sigmoid(g))) @ W[p + "o"].T, S


def layer(x, W, i, cfg, pos0, st):
    """One pass of layer i over rows x; st is this pass's {"k": keys so far, "S": state}."""
    c, eps, p = cfg["layers"][i], cfg["norm"]["eps"], "l%d." % i
    h = rms(x, eps) * W[p + "norm1"]
    m = c["mixer"]
    left, st["k"] = left_mixer(h, W, p + "mix.left.", m["left"], pos0, st.get("k"))
    right, st["S"] = right_mixer(h, W, p + "mix.right.", m["right"], eps, st.get("S"))
    y = m["left_scale"] * left + m["right_scale"] * right
    if c.get("mlp"):
        y = y + polynorm(h @ W[p + "mlp.up"].T, W[p + "mlp.act"], eps) @ W[p + "mlp.down"].T
    return x + y


def layer_runs(cfg):
    """[(layer, pass number or None)] in the order they run; the number is set on a pass's first layer."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    runs = [(i, None) for i in range(lp["start"])]
    for t in range(lp["times"]):
        runs += [(i, t if i == lp["start"] else None) for i in range(lp["start"], lp["stop"])]
    return runs + [(i, None) for i in range(lp["stop"], n)]


class Oracle:
    """State of one sequence; feed() takes the next tokens and returns their logits."""

    def __init__(self, cfg, weights):
        self.cfg, self.W = cfg, {k: np.asarray(v, F) for k, v in weights.items()}
        self.reset()

    def reset(self):
        self.pos = 0
        self.st = [dict() for _ in layer_runs(self.cfg)]

    def feed(self, tokens, trace=None):
        W, cfg, width = self.W, self.cfg, self.cfg["width"]
        emb = np.stack([W["embed"][t] + position_vector(self.pos + n, width) for n, t in enumerate(tokens)])
        x = emb.copy()
        for run, (i, first) in enumerate(layer_runs(cfg)):
            if first is not None:
                if first > 0:
                    x = x + emb
                x = x + W["loop.step"][first]
            x = layer(x, W, i, cfg, self.pos, self.st[run])
            if trace is not None:
                trace.append(x.copy())
        self.pos += len(tokens)
        return (rms(x, cfg["norm"]["eps"]) * W["final.norm"]) @ W["head"].T
