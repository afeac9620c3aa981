"""Small random Nubedra models for the tests: configurations, and weights that make every mechanism matter."""
import numpy as np

from util import bf16_round


def gla(heads, dim, vdim, tau=6.0, rank=5):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}, "rank": rank}


def latent(heads, dim, rot, vdim, q_rank, kv_rank, window=None, base=500.0, scaling=None, scale=None, kv_from=None):
    r = {"base": base, "dims": rot}
    if scaling:
        r["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "rot": r,
         "scale": scale or 1.1 * (dim + rot) ** -0.5}
    if window:
        m["mask"] = {"size": window}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m}


def config(layers, width, vocab, ff, mult=0.6, embed=3.0, eps=1e-5):
    """`ff`: one size a layer (None: that layer has no feed-forward).  -> (config.json's tree, rank of each layer's decay)"""
    ls = [dict({k: v for k, v in l.items() if k != "rank"}, mlp=None if f is None else {"kind": "dense", "ff": f}) for l, f in zip(layers, ff)]
    cfg = {"architecture": "Nubedra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult, "embedding": {"scale": embed},
           "layers": ls}
    return cfg, [l.get("rank") for l in layers]


YARN = (4.0, 48, 6.0, 0.5)
_ALL = {
    # every mechanism, sizes of whole vectors; a sharing layer with other heads and a wider window than the layer it reads
    "mixed": config([latent(3, 24, 8, 40, 24, 48, 9, scaling=YARN), gla(2, 16, 24, rank=8), latent(5, 32, 8, 16, 40, 48, 33, scaling=YARN, kv_from=0),
                     gla(4, 32, 16, tau=2.0, rank=16), latent(2, 16, 12, 24, 16, 32, 50, base=3000.0, scaling=(2.0, 200, 20.0, 2.0))],
                    width=80, vocab=131, ff=[96, None, 72, 64, None]),
    # nothing is a multiple of eight; a window of one token, one without an edge; no frequency scaling; layers that share at a distance
    "odd": config([gla(3, 7, 11, tau=1.0, rank=3), latent(5, 9, 6, 11, 13, 21, 1, base=60.0), latent(3, 5, 10, 7, 9, 19, base=100.0), gla(1, 18, 21, rank=1),
                   latent(4, 11, 6, 9, 6, 21, 14, base=60.0, kv_from=1), latent(2, 6, 10, 13, 11, 19, 3, base=100.0, kv_from=2)],
                  width=37, vocab=53, ff=[21, None, 45, None, 30, 13], mult=0.3, embed=2.5, eps=1e-4),
    # more heads than a tile has columns, rows and heads larger than one operand, keys of a recurrent head beyond 256 channels
    "wide": config([latent(40, 40, 24, 20, 48, 136, 70), gla(1, 260, 72, rank=24), latent(2, 250, 16, 24, 32, 264, 100, scaling=YARN), gla(2, 136, 130, rank=7)],
                   width=112, vocab=97, ff=[64, 40, 48, None]),
    # windows at the edges of tiles and splits
    "windows": config([latent(4, 16, 16, 32, 24, 40, 64), latent(4, 16, 16, 32, 24, 40, 65), latent(2, 16, 16, 16, 24, 40, 128, kv_from=0),
                       latent(2, 48, 8, 16, 24, 64, 129, scaling=(8.0, 32, 16.0, 1.0))],
                      width=64, vocab=90, ff=[72, None, None, 40]),
}
CONFIGS = {k: c for k, (c, _) in _ALL.items()}
RANKS = {k: r for k, (_, r) in _ALL.items()}


def shapes(cfg, ranks):
    d, out = cfg["width"], {}
    out["embed"], out["final.norm"] = (cfg["vocab"], d), (d,)
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.", l["mixer"]
        out[p + "norm1"] = out[p + "norm1b"] = (d,)
        H, dv = m["heads"], m["vdim"]
        if l["type"] == "gla":
            out[p + "mix.q"] = out[p + "mix.k"] = (H * m["dim"], d)
            out[p + "mix.v"] = out[p + "mix.g"] = (H * dv, d)
            out[p + "mix.norm"] = (dv,)
            out[p + "mix.a1"], out[p + "mix.a2"], out[p + "mix.a2.b"] = (ranks[i], d), (H * m["dim"], ranks[i]), (H * m["dim"],)
        else:
            out[p + "mix.dq"], out[p + "mix.dq.norm"] = (m["q_rank"], d), (m["q_rank"],)
            out[p + "mix.uq"] = (H * (m["dim"] + m["rot_dim"]), m["q_rank"])
            if m.get("kv_from") is None:
                out[p + "mix.dkv"], out[p + "mix.dkv.norm"] = (m["kv_rank"] + m["rot_dim"], d), (m["kv_rank"],)
            out[p + "mix.uk"], out[p + "mix.uv"] = (H * m["dim"], m["kv_rank"]), (H * dv, m["kv_rank"])
            out[p + "mix.sink"], out[p + "mix.g"] = (H,), (H, d)
        out[p + "mix.o"] = (d, H * dv)
        if l["mlp"]:
            f = l["mlp"]["ff"]
            out[p + "norm2"] = out[p + "norm2b"] = (d,)
            out[p + "mlp.gate"] = out[p + "mlp.up"] = (f, d)
            out[p + "mlp.down"] = (d, f)
    return out


def weights(name, seed=0):
    """float64 arrays whose values are bf16 numbers."""
    r, out = np.random.default_rng(seed), {}
    for key, sh in shapes(CONFIGS[name], RANKS[name]).items():
        leaf = key.split(".", 1)[-1]
        z = r.standard_normal(sh)
        if leaf in ("norm1", "norm1b", "norm2", "norm2b") or key == "final.norm":
            v = 0.3 * z                              # stored around zero
        elif leaf in ("mix.norm", "mix.dq.norm", "mix.dkv.norm"):
            v = 1 + 0.3 * z
        elif key == "embed":
            v = 0.4 * z
        elif leaf in ("mix.uq", "mix.uk"):
            v = z * (1.6 / np.sqrt(sh[-1]))          # scores of a few units: some keys stand out
        elif leaf == "mix.sink":
            v = 1 + z
        elif leaf == "mix.a2.b":
            v = 1 + 2 * z                            # channels that forget at once beside ones that keep
        elif leaf == "mix.a2":
            v = z * (1.5 / np.sqrt(sh[-1]))
        else:
            v = z / np.sqrt(sh[-1])
        out[key] = bf16_round(v.astype(np.float32)).astype(np.float64)
    return out
