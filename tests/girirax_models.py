"""Small random Girirax models for tests: configuration and weights (bf16 values); the files of a model
folder are written by lusadra_models.write."""
import numpy as np

from lusadra_models import to_bf16


def ssm(heads, state, groups, vdim, conv, norm_groups, ff):
    return {"type": "mamba2",
            "mixer": {"heads": heads, "state": state, "groups": groups, "vdim": vdim, "conv": conv, "norm_groups": norm_groups},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def latent(heads, dim, rot_dim, vdim, kv_rank, q_rank, scale, base, ff):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
                      "scale": scale, "rot": {"base": base, "dims": rot_dim}},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(vocab, width, layers, embed_scale, mult, eps=1e-5):
    return {"architecture": "Girirax", "vocab": vocab, "width": width, "layers": layers, "norm": {"eps": eps},
            "embedding": {"scale": embed_scale}, "residual_mult": mult}


# Sizes unlike each other: one group and one per head, value sizes above and below the state, taps from one
# to seven, key, value and rotated sizes that differ, ranks that no vector width divides, layers without a
# feed-forward, both mixers first and last.
SMALL = {
    "state_first": config(97, 72, [
        ssm(6, 20, 3, 12, 3, 4, 50),
        latent(3, 20, 8, 28, 44, 36, 0.19, 5000.0, None),
        ssm(2, 48, 1, 36, 5, 1, None),
        latent(5, 12, 24, 8, 70, 25, 0.3, 100.0, 131)], 3.5, 0.6),
    "attention_first": config(60, 40, [
        latent(1, 64, 2, 17, 33, 64, 0.125, 1e5, 96),
        ssm(5, 16, 5, 64, 1, 5, 40),
        ssm(4, 7, 2, 9, 7, 3, 24)], 2.0, 0.7, 1e-6),
    "attention_only": config(64, 130, [latent(33, 8, 4, 8, 160, 48, 0.4, 1e4, 64)] * 2, 8.0, 0.25),
    "state_only": config(50, 96, [ssm(3, 80, 1, 70, 2, 7, 100), ssm(8, 33, 4, 16, 4, 2, None)], 1.0, 1.0),
}


def weights(cfg, seed=0, a_log=0.0, dt_bias=-1.0):
    """name -> f32 values that bf16 holds exactly. a_log, dt_bias: their mean; slow decays where both are low."""
    g = np.random.default_rng(seed)
    W = {}

    def mat(name, rows, cols, amp=1.0):
        W[name] = to_bf16(g.standard_normal((rows, cols)) * amp / np.sqrt(cols))[1]

    def vec(name, n, mean, amp):
        W[name] = to_bf16(mean + amp * g.standard_normal(n))[1]

    E = cfg["width"]
    W["embed"] = to_bf16(g.standard_normal((cfg["vocab"], E)))[1]
    for i, l in enumerate(cfg["layers"]):
        p, c = "l%d." % i, l["mixer"]
        vec(p + "norm1", E, 1.0, 0.3)
        if l["type"] == "mamba2":
            inner = c["heads"] * c["vdim"]
            ch = inner + 2 * c["groups"] * c["state"]
            mat(p + "mix.in", inner + ch + c["heads"], E, 0.6)
            mat(p + "mix.conv", ch, c["conv"], 1.5)
            vec(p + "mix.conv.b", ch, 0.0, 0.4)
            vec(p + "mix.dt_bias", c["heads"], dt_bias, 0.5)
            vec(p + "mix.A_log", c["heads"], a_log, 0.7)
            vec(p + "mix.D", c["heads"], 0.5, 0.5)
            vec(p + "mix.norm", inner, 1.0, 0.3)
            mat(p + "mix.o", E, inner)
        else:
            H, D, R, V = c["heads"], c["dim"], c["rot_dim"], c["vdim"]
            mat(p + "mix.dq", c["q_rank"], E)
            vec(p + "mix.dq.norm", c["q_rank"], 1.0, 0.3)
            mat(p + "mix.uq", H * (D + R), c["q_rank"], 1.5)
            mat(p + "mix.dkv", c["kv_rank"] + R, E, 0.4)
            vec(p + "mix.dkv.norm", c["kv_rank"], 1.0, 0.3)
            mat(p + "mix.uk", H * D, c["kv_rank"])
            mat(p + "mix.uv", H * V, c["kv_rank"])
            mat(p + "mix.g", H * V, E, 0.5)
            mat(p + "mix.o", E, H * V)
        if l.get("mlp"):
            ff = l["mlp"]["ff"]
            vec(p + "norm2", E, 1.0, 0.3)
            for n, rows, cols in (("gate", ff, E), ("up", ff, E), ("down", E, ff)):
                mat(p + "mlp." + n, rows, cols, 0.7)
                vec(p + "mlp." + n + ".b", rows, 0.1, 0.5)
    vec("final.norm", E, 1.0, 0.3)
    return W
