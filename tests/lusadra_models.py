"""Small random Lusadra models for tests: configuration, weights (bf16 values), the two files of a
model folder."""
import json
import os
import struct

import numpy as np


def to_bf16(a):
    """f32 values rounded to bf16: (bits, values)."""
    x = np.ascontiguousarray(a, np.float32).reshape(-1).view(np.uint32)
    b = ((x + 0x7fff + ((x >> 16) & 1)) >> 16).astype(np.uint16)
    return b.reshape(np.shape(a)), (b.astype(np.uint32) << 16).view(np.float32).reshape(np.shape(a))


def layer(H, G, dim, window, coef, every, scale, h2, dim2, vdim2, tau, ls, rs, ff):
    return {"type": "parallel",
            "mixer": {"left": {"heads": H, "kv_heads": G, "dim": dim, "vdim": dim, "mask": {"size": window},
                               "q_temp": {"coef": coef, "every": every}, "scale": scale},
                      "right": {"heads": h2, "dim": dim2, "vdim": vdim2, "tau": tau},
                      "left_scale": ls, "right_scale": rs},
            "mlp": {"ff": ff, "kind": "dense"} if ff else None}


def config(vocab, width, layers, loop=None, eps=1e-5):
    c = {"architecture": "Lusadra", "vocab": vocab, "width": width, "layers": layers, "norm": {"eps": eps}}
    if loop:
        c["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return c


# Sizes unlike each other: a loop over layers of different shapes, a layer without a feed-forward, one
# kv head and several, windows of one token, of a few, and longer than the sequence; widths and head
# sizes that no vector width divides.
SMALL = {
    "loop_of_unlike_layers": config(97, 72, [
        layer(3, 1, 20, 9, 0.4, 7, 0.21, 2, 12, 17, 3.0, 0.8, 1.1, 50),
        layer(4, 2, 24, 33, 0.2, 16, 0.3, 3, 16, 8, 8.0, 1.3, 0.6, None),
        layer(2, 2, 36, 1, 0.7, 5, 0.15, 1, 40, 24, 1.0, 0.5, 0.9, 131),
        layer(6, 3, 8, 64, 0.3, 11, 0.4, 2, 8, 32, 16.0, 1.0, 1.0, 64)], loop=(1, 3, 3)),
    "no_loop": config(50, 40, [
        layer(1, 1, 64, 300, 0.5, 32, 0.125, 1, 64, 64, 4.0, 1.0, 0.4, 96),
        layer(8, 1, 16, 40, 0.1, 3, 0.25, 4, 24, 12, 2.0, 0.3, 1.5, 40)]),
    "loop_over_everything": config(64, 128, [
        layer(7, 1, 128, 50, 0.6, 9, 0.09, 2, 32, 48, 5.0, 1.1, 0.7, 200)], loop=(0, 1, 2), eps=1e-6),
}


def weights(cfg, seed=0, decay_bias=2.0, gain=1.0):
    """name -> f32 values that bf16 holds exactly."""
    g = np.random.default_rng(seed)
    W = {}

    def mat(name, rows, cols, amp=1.0):
        W[name] = to_bf16(g.standard_normal((rows, cols)) * amp / np.sqrt(cols))[1]

    def vec(name, n, mean, amp):
        W[name] = to_bf16(mean + amp * g.standard_normal(n))[1]

    E = cfg["width"]
    W["embed"] = to_bf16(g.standard_normal((cfg["vocab"], E)))[1]
    for i, l in enumerate(cfg["layers"]):
        p, a, r = "l%d." % i, l["mixer"]["left"], l["mixer"]["right"]
        W[p + "norm1"] = to_bf16(np.float32(1.0 + 0.2 * g.standard_normal()))[1]
        mat(p + "mix.left.q", a["heads"] * a["dim"], E, 2.0 * gain)
        mat(p + "mix.left.k", a["kv_heads"] * a["dim"], E, gain)
        mat(p + "mix.left.g", a["heads"] * a["dim"], E)
        mat(p + "mix.left.o", E, a["heads"] * a["dim"])
        for n, rows in (("q", r["dim"]), ("k", r["dim"]), ("v", r["vdim"]), ("g", r["vdim"])):
            mat(p + "mix.right." + n, r["heads"] * rows, E)
        mat(p + "mix.right.o", E, r["heads"] * r["vdim"])
        vec(p + "mix.right.norm", r["vdim"], 1.0, 0.3)
        rank = 3 + 2 * i
        mat(p + "mix.right.a1", rank, E)
        mat(p + "mix.right.a2", r["heads"] * r["dim"], rank)
        vec(p + "mix.right.a2.b", r["heads"] * r["dim"], decay_bias, 1.0)
        if l.get("mlp"):
            ff = l["mlp"]["ff"]
            mat(p + "mlp.up", ff, E)
            mat(p + "mlp.down", E, ff)
            vec(p + "mlp.act", 4, 0.3, 0.5)
    if cfg.get("loop"):
        W["loop.step"] = to_bf16(g.standard_normal((cfg["loop"]["times"], E)))[1]
    W["final.norm"] = to_bf16(np.float32(1.3))[1]
    mat("head", cfg["vocab"], E)
    return W


def safetensors_bytes(tensors, dtype="BF16"):
    head, blobs, at = {}, [], 0
    for name, a in tensors.items():
        raw = (to_bf16(a)[0] if dtype == "BF16" else np.ascontiguousarray(a, np.float32)).tobytes()
        head[name] = {"dtype": dtype, "shape": list(np.shape(a)), "data_offsets": [at, at + len(raw)]}
        blobs.append(raw)
        at += len(raw)
    h = json.dumps(head).encode()
    h += b" " * (-len(h) % 8)
    return struct.pack("<Q", len(h)) + h + b"".join(blobs)


def write(folder, cfg, W):
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(safetensors_bytes(W))
    return str(folder)
