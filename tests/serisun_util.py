"""Small random Serisun models for the tests: configurations, weights that make every mechanism matter, and the folder
(config.json, model.safetensors) a model is opened from."""
import json
import struct

import numpy as np

from util import bf16_round


def attention(heads, kv_heads, dim, vdim, every=7, coef=0.4, scale=None, temp=True):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5}
    if temp:
        m["q_temp"] = {"coef": coef, "every": every}
    return {"type": "attention", "mixer": m}


def mamba2(heads, vdim, state, groups=1, norm_groups=1, conv=4):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups,
                                        "norm_groups": norm_groups, "conv": conv}}


def config(layers, width, vocab, ff, loop=None, logit_scale=0.7, eps=1e-5):
    """`ff`: one size, or one per layer (None: that layer has no feed-forward)."""
    ff = ff if isinstance(ff, list) else [ff] * len(layers)
    ls = [dict(l, mlp=None if f is None else {"kind": "dense", "ff": f}) for l, f in zip(layers, ff)]
    c = {"architecture": "Serisun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_scale": logit_scale, "layers": ls}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


CONFIGS = {
    # every mechanism once, sizes of whole vectors
    "mixed": config([attention(4, 2, 24, 16), mamba2(4, 16, 24, 2, 2, 4), attention(6, 1, 32, 40), mamba2(6, 24, 16, 3, 4, 3)],
                    width=80, vocab=131, ff=96, loop=(1, 3, 3)),
    # nothing is a multiple of eight; a layer without a feed-forward; a mixer with one tap; a loop of one pass
    "odd": config([mamba2(3, 7, 5, 3, 7, 1), attention(6, 2, 11, 13, every=3), attention(5, 5, 9, 6, temp=False), mamba2(4, 10, 19, 1, 1, 2)],
                  width=37, vocab=53, ff=[21, None, 45, 30], loop=(0, 2, 1), logit_scale=1.3, eps=1e-4),
    # no loop, heads and states larger than one operand, more query heads per key head than a tile has columns
    "wide": config([attention(40, 1, 136, 72), mamba2(2, 80, 144, 1, 2, 5), attention(3, 3, 264, 24, every=64)],
                   width=112, vocab=97, ff=[64, 40, 48]),
    # the loop's stretch is the whole model
    "all_looped": config([mamba2(8, 8, 32, 4, 8, 4), attention(8, 4, 16, 16, every=50, coef=1.1)], width=64, vocab=90, ff=72, loop=(0, 2, 2)),
}


def shapes(cfg):
    d, out = cfg["width"], {}
    out["embed"] = out["head"] = (cfg["vocab"], d)
    out["final.norm"] = (d,)
    if cfg.get("loop"):
        out["loop.step"] = (cfg["loop"]["times"], d)
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.", l["mixer"]
        out[p + "norm1"] = out[p + "ls1"] = (d,)
        if l["type"] == "attention":
            out[p + "mix.q"] = (m["heads"] * m["dim"], d)
            out[p + "mix.k"] = (m["kv_heads"] * m["dim"], d)
            out[p + "mix.v"] = (m["kv_heads"] * m["vdim"], d)
            out[p + "mix.o"] = (d, m["heads"] * m["vdim"])
        else:
            inner, ch = m["heads"] * m["vdim"], m["heads"] * m["vdim"] + 2 * m["groups"] * m["state"]
            out[p + "mix.in"] = (inner + ch + m["heads"], d)
            out[p + "mix.conv"], out[p + "mix.conv.b"] = (ch, m["conv"]), (ch,)
            out[p + "mix.dt_bias"] = out[p + "mix.A_log"] = out[p + "mix.D"] = (m["heads"],)
            out[p + "mix.norm"], out[p + "mix.o"] = (inner,), (d, inner)
        if l["mlp"]:
            f = l["mlp"]["ff"]
            out[p + "mlp.gate"] = out[p + "mlp.up"] = (f, d)
            out[p + "mlp.down"], out[p + "ls2"] = (d, f), (d,)
    return out


def weights(cfg, seed=0):
    """float64 arrays whose values are bf16 numbers."""
    r, out = np.random.default_rng(seed), {}
    for name, sh in shapes(cfg).items():
        leaf = name.split(".", 1)[-1]
        z = r.standard_normal(sh)
        if leaf in ("norm1", "norm", "mix.norm") or name == "final.norm":
            v = 1 + 0.3 * z
        elif leaf in ("ls1", "ls2"):
            v = 0.6 + 0.4 * z
        elif name == "embed":
            v = z
        elif leaf == "step":
            v = 0.8 * z
        elif leaf in ("mix.q", "mix.k"):
            v = z * (1.5 / np.sqrt(sh[-1]))          # scores of a few units: some keys stand out
        elif leaf == "mix.dt_bias":
            v = -1.5 + z
        elif leaf == "mix.A_log":
            v = -0.5 + z
        elif leaf == "mix.D":
            v = 1 + 0.5 * z
        elif leaf in ("mix.conv", "mix.conv.b"):
            v = 0.5 * z
        elif leaf == "mix.in":
            v = z * (1.2 / np.sqrt(sh[-1]))
        else:
            v = z / np.sqrt(sh[-1])
        out[name] = bf16_round(v.astype(np.float32)).astype(np.float64)
    return out


def write(folder, cfg, w, dtypes=None):
    """config.json and model.safetensors; `dtypes`: tensor name -> "F32" / "F16" instead of BF16."""
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg))
    head, blob = {}, b""
    for name, v in w.items():
        ty = (dtypes or {}).get(name, "BF16")
        f = np.ascontiguousarray(v, np.float32)
        raw = (f.view(np.uint32) >> 16).astype("<u2").tobytes() if ty == "BF16" else f.astype("<f2" if ty == "F16" else "<f4").tobytes()
        head[name] = {"dtype": ty, "shape": list(v.shape), "data_offsets": [len(blob), len(blob) + len(raw)]}
        blob += raw
    h = json.dumps(head).encode()
    (folder / "model.safetensors").write_bytes(struct.pack("<Q", len(h)) + h + blob)
    return folder


def logit_error(got, want):
    """Root mean square difference per row, relative to the spread of all the logits (their means taken off)."""
    d = np.asarray(got, np.float64) - want
    d -= d.mean(-1, keepdims=True)
    c = want - want.mean(-1, keepdims=True)
    return np.sqrt((d * d).mean(-1)) / np.sqrt((c * c).mean())
