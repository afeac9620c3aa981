"""Prefill and decode of random-weight Nubedra models at sizes that resemble real models' layers, beside Serisun models of the same
width, depth, feed-forward, recurrent width and state, heads and context (`bench.py --nubedra`).

Rooflines and families as in serisun_bench.py.  A latent layer's attention family holds everything between its projections: the
cache rows, the products with uk and uv, the attention."""
from __future__ import annotations

from pathlib import Path

import numpy as np

from .serisun_bench import SIZES, VOCAB, flops as serisun_flops, results, serisun_config, write_random

# heads, unrotated and rotated key size, value size, ranks; three recurrent layers and a latent one in turn, as the Serisun side
LATENT = {
    "w1024": dict(heads=16, dim=64, rot_dim=32, vdim=64, kv_rank=256, q_rank=384),
    "w2048": dict(heads=16, dim=128, rot_dim=64, vdim=128, kv_rank=512, q_rank=768),
    "w4096": dict(heads=32, dim=128, rot_dim=64, vdim=128, kv_rank=512, q_rank=1536),
}
GLA_DIM, GLA_VDIM, RANK, WINDOW, CHUNK = 128, 256, 16, 4096, 64


def config(name):
    s, a = SIZES[name], LATENT[name]
    rot = {"base": 10000.0, "dims": a["rot_dim"], "scaling": {"factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}}
    lat = {"type": "latent_attention", "mixer": dict(a, scale=(a["dim"] + a["rot_dim"]) ** -0.5, mask={"size": WINDOW}, rot=rot)}
    gla = {"type": "gla", "mixer": {"heads": s["inner"] // GLA_VDIM, "dim": GLA_DIM, "vdim": GLA_VDIM, "tau": 16.0}}
    layers = [dict(lat if i % 4 == 3 else gla, mlp={"kind": "dense", "ff": s["ff"]}) for i in range(s["layers"])]
    return {"architecture": "Nubedra", "vocab": VOCAB, "width": s["width"], "norm": {"eps": 1e-6}, "residual_mult": 0.5, "embedding": {"scale": 1.0},
            "layers": layers}


def shapes(cfg):
    d, out = cfg["width"], {}
    out["embed"], out["final.norm"] = (cfg["vocab"], d), (d,)
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.", l["mixer"]
        H, dv, f = m["heads"], m["vdim"], l["mlp"]["ff"]
        for v in ("norm1", "norm1b", "norm2", "norm2b"):
            out[p + v] = (d,)
        if l["type"] == "gla":
            k = H * m["dim"]
            out.update({p + "mix.q": (k, d), p + "mix.k": (k, d), p + "mix.v": (H * dv, d), p + "mix.g": (H * dv, d), p + "mix.a1": (RANK, d),
                        p + "mix.a2": (k, RANK), p + "mix.a2.b": (k,), p + "mix.norm": (dv,)})
        else:
            r = m["kv_rank"]
            out.update({p + "mix.dq": (m["q_rank"], d), p + "mix.dq.norm": (m["q_rank"],), p + "mix.uq": (H * (m["dim"] + m["rot_dim"]), m["q_rank"]),
                        p + "mix.dkv": (r + m["rot_dim"], d), p + "mix.dkv.norm": (r,), p + "mix.uk": (H * m["dim"], r), p + "mix.uv": (H * dv, r),
                        p + "mix.sink": (H,), p + "mix.g": (H, d)})
        out.update({p + "mix.o": (d, H * dv), p + "mlp.gate": (f, d), p + "mlp.up": (f, d), p + "mlp.down": (d, f)})
    return out


def vector(name, n, r):
    v, leaf = r.standard_normal(n), name.rsplit(".", 1)[-1]
    return 1 + 0.1 * v if leaf == "norm" and name != "final.norm" else 1 + v if leaf == "b" else 0.1 * v


def flops(cfg, n):
    """Multiply-adds (two operations each) of a prefill pass of a whole prompt by family, the head left out."""
    out = {"group": 0, "residual": 0, "attend": 0, "gla": 0}
    d = cfg["width"]
    for l in cfg["layers"]:
        m, f = l["mixer"], l["mlp"]["ff"]
        H, dv = m["heads"], m["vdim"]
        out["residual"] += 2 * n * d * (H * dv + f)
        if l["type"] == "gla":
            k = H * m["dim"]
            out["group"] += 2 * n * d * (2 * k + 2 * H * dv + RANK + 2 * f)
            # causal halves of M and of M V, the read-out of the starting state, the state's own sum, the decays
            out["gla"] += n * H * (CHUNK * (m["dim"] + dv) + 4 * m["dim"] * dv) + 2 * n * k * RANK
        else:
            per = m["dim"] + m["rot_dim"]
            out["group"] += 2 * n * (d * (m["q_rank"] + m["kv_rank"] + m["rot_dim"] + H + 2 * f) + m["q_rank"] * H * per)
            out["attend"] += H * (per + dv) * n * n + 2 * n * m["kv_rank"] * H * (m["dim"] + dv)   # causal: the mean of the visible keys
    return out


def run(ih, tmp: Path, sizes, prompt_len=4096, steps=256, seed=0):
    out = []
    for name in sizes:
        prompt = np.random.default_rng(seed).integers(0, VOCAB, prompt_len).astype(np.uint32)
        ctx = prompt_len + 1024 + 8 * ((steps * 3 + 64) // 8)
        row = {"size": name, "prompt": prompt_len, "layers": SIZES[name]["layers"], "width": SIZES[name]["width"]}
        for kind in ("nubedra", "serisun"):
            if kind == "nubedra":
                cfg = config(name)
                folder, work, fp32 = write_random(tmp / f"{kind}_{name}", cfg, seed, shapes, vector), flops(cfg, prompt_len), ("gla",)
            else:
                cfg = serisun_config(SIZES[name])
                folder, work, fp32 = write_random(tmp / f"{kind}_{name}", cfg, seed), serisun_flops(cfg, prompt_len, prompt_len), ("mamba2",)
            model = ih.Model(folder)
            row[kind] = r = results(ih, model, prompt, steps, ctx, work, fp32)
            model.close()
            for f in folder.iterdir():
                f.unlink()
            print(f"# {name} {kind}: prefill {r['prefill_tok_s']} tok/s, decode {r['decode_tok_s']} tok/s", flush=True)
        out.append(row)
    return out
