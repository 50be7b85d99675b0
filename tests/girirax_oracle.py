"""A plain, slow implementation of the Girirax decoder in numpy (float64), one function per mechanism,
token by token where the mechanism is a recurrence. The GPU path is compared with it; it shares no code
with the product.

Weights are a dict name -> array (already widened); the configuration is the dict of config.json."""
import numpy as np

F = np.float64


def sigmoid(z):
    e = np.exp(-np.abs(z))
    return np.where(z >= 0, 1.0, e) / (1.0 + e)


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def rms_norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def grouped_rms_norm(x, w, parts, eps):
    """Every one of `parts` equal slices of a row by its own root mean square."""
    T, n = x.shape
    y = x.reshape(T, parts, n // parts)
    y = y / np.sqrt(np.mean(y * y, axis=-1, keepdims=True) + eps)
    return y.reshape(T, n) * w


def causal_conv(x, w, b, tail):
    """x [T, channels]; w [channels, taps], its last column meets the current row; tail: the taps - 1
    rows before x (zeros at the start). Returns the sums and the new tail."""
    taps = w.shape[1]
    rows = np.concatenate([tail, x])
    y = np.stack([sum(w[:, j] * rows[t + j] for j in range(taps)) + b for t in range(len(x))])
    return y, rows[len(rows) - (taps - 1):]


def state_space(x, B, C, dt, A_log, D, heads, groups, N, vdim, S=None):
    """x [T, heads*vdim], B and C [T, groups*N], dt [T, heads] (softplus taken). Returns y and the state
    [heads, N, vdim]: a head's state shrinks by exp(-exp(A_log) dt) and takes dt B x^T; C reads it."""
    T = len(x)
    S = np.zeros((heads, N, vdim), F) if S is None else S.copy()
    y = np.zeros((T, heads * vdim), F)
    for t in range(T):
        for h in range(heads):
            g = h // (heads // groups)
            xs = x[t, h * vdim:(h + 1) * vdim]
            S[h] = np.exp(-np.exp(A_log[h]) * dt[t, h]) * S[h] + dt[t, h] * np.outer(B[t, g * N:(g + 1) * N], xs)
            y[t, h * vdim:(h + 1) * vdim] = C[t, g * N:(g + 1) * N] @ S[h] + D[h] * xs
    return y, S


def mamba2_core(u, w, b, dt_bias, A_log, D, c, st):
    """Rows u = [z | x | B | C | dt] to the gated output ahead of its norm. st: {"tail": inputs of the
    convolution, "S": state} of one sequence, updated."""
    H, N, G, V = c["heads"], c["state"], c["groups"], c["vdim"]
    inner, ch = H * V, H * V + 2 * G * N
    z, xbc, dt = u[:, :inner], u[:, inner:inner + ch], u[:, inner + ch:inner + ch + H]
    tail = st.get("tail", np.zeros((c["conv"] - 1, ch), F))
    xbc, st["tail"] = causal_conv(xbc, w, b, tail)
    xbc = silu(xbc)
    x, B, C = xbc[:, :inner], xbc[:, inner:inner + G * N], xbc[:, inner + G * N:]
    y, st["S"] = state_space(x, B, C, softplus(dt + dt_bias), A_log, D, H, G, N, V, st.get("S"))
    return y * silu(z)


def mamba2(h, W, p, c, eps, st):
    y = mamba2_core(h @ W[p + "in"].T, W[p + "conv"], W[p + "conv.b"], W[p + "dt_bias"], W[p + "A_log"], W[p + "D"], c, st)
    return grouped_rms_norm(y, W[p + "norm"], c["norm_groups"], eps) @ W[p + "o"].T


def rotate_half(x, p, base):
    """A vector of even length: coordinate i turns with coordinate i + half by p * base^(-2i / length)."""
    n = len(x) // 2
    a = p * base ** (-2.0 * np.arange(n) / (2 * n))
    u, v = x[:n], x[n:]
    return np.concatenate([u * np.cos(a) - v * np.sin(a), v * np.cos(a) + u * np.sin(a)])


def attend(q, keys, values, scale):
    s = keys @ q * scale
    w = np.exp(s - s.max())
    return (w / w.sum()) @ values


def latent_core(q, kv, kv_norm, uk, uv, c, base, eps, pos0, st):
    """Rows q (heads side by side, [dim | rot_dim], not rotated) and kv = [latent | key part], both raw, to
    the heads' outputs. Keys and values are formed from the latents head by head. st: {"c": latents, "r":
    rotated key parts} of the positions so far, updated."""
    H, D, R, V, L = c["heads"], c["dim"], c["rot_dim"], c["vdim"], c["kv_rank"]
    T = len(q)
    q = q.reshape(T, H, D + R)
    lat = rms_norm(kv[:, :L], kv_norm, eps)
    rot = np.stack([rotate_half(kv[t, L:L + R], pos0 + t, base) for t in range(T)])
    st["c"] = np.concatenate([st["c"], lat]) if "c" in st else lat
    st["r"] = np.concatenate([st["r"], rot]) if "r" in st else rot
    n = len(st["c"])
    k = (st["c"] @ uk.T).reshape(n, H, D)
    v = (st["c"] @ uv.T).reshape(n, H, V)
    out = np.zeros((T, H * V), F)
    for t in range(T):
        m = pos0 + t + 1
        for e in range(H):
            qe = np.concatenate([q[t, e, :D], rotate_half(q[t, e, D:], pos0 + t, base)])
            out[t, e * V:(e + 1) * V] = attend(qe, np.concatenate([k[:m, e], st["r"][:m]], axis=1), v[:m, e], c["scale"])
    return out


def latent_attention(h, W, p, c, eps, pos0, st):
    cq = rms_norm(h @ W[p + "dq"].T, W[p + "dq.norm"], eps)
    out = latent_core(cq @ W[p + "uq"].T, h @ W[p + "dkv"].T, W[p + "dkv.norm"], W[p + "uk"], W[p + "uv"], c,
                      c["rot"]["base"], eps, pos0, st)
    return (out * sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def gated_mlp(h, W, p):
    g = gelu_tanh(h @ W[p + "gate"].T + W[p + "gate.b"])
    return (g * (h @ W[p + "up"].T + W[p + "up.b"])) @ W[p + "down"].T + W[p + "down.b"]


def layer(x, W, i, cfg, pos0, st):
    """Sublayers read the residual itself; what they write is normed before it is added."""
    c, eps, m, p = cfg["layers"][i], cfg["norm"]["eps"], cfg["residual_mult"], "l%d." % i
    if c["type"] == "mamba2":
        y = mamba2(x, W, p + "mix.", c["mixer"], eps, st)
    else:
        y = latent_attention(x, W, p + "mix.", c["mixer"], eps, pos0, st)
    x = x + m * rms_norm(y, W[p + "norm1"], eps)
    if c.get("mlp"):
        x = x + m * rms_norm(gated_mlp(x, W, p + "mlp."), W[p + "norm2"], eps)
    return x


class Oracle:
    """State of one sequence; feed() takes the next tokens and returns their logits."""

    def __init__(self, cfg, weights):
        self.cfg, self.W = cfg, {k: np.asarray(v, F) for k, v in weights.items()}
        self.reset()

    def reset(self):
        self.pos = 0
        self.st = [dict() for _ in self.cfg["layers"]]

    def feed(self, tokens, trace=None):
        W, cfg = self.W, self.cfg
        x = W["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
        for i in range(len(cfg["layers"])):
            x = layer(x, W, i, cfg, self.pos, self.st[i])
            if trace is not None:
                trace.append(x.copy())
        self.pos += len(tokens)
        return rms_norm(x, W["final.norm"], cfg["norm"]["eps"]) @ W["embed"].T
