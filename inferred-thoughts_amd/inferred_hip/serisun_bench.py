"""Prefill and decode of random-weight Serisun models at sizes that resemble real models' layers, beside qwen35moe models of the
same width, depth, attention, recurrent width and active feed-forward width (`bench.py --serisun`).

A family's time is the sum of HIP-event spans around its launches.  Rooflines: decode, the bytes a launch must move once over
8 TB/s; prefill, the multiply-adds of a family over the dense matrix-core peak of its operand type (bf16 / f16 2.5 PFLOP/s,
fp32 157 TFLOP/s)."""
from __future__ import annotations

import json
import struct
import time
from pathlib import Path

import numpy as np

HBM = 8e12
BF16_PEAK, FP32_PEAK = 2.5e15, 157.3e12

# width, layers (three recurrent ones and an attention layer in turn), attention heads / KV heads / head size, active
# feed-forward, recurrent inner width; the like sizes of the qwen35moe side
SIZES = {
    "w1024": dict(width=1024, layers=8, heads=16, kv=4, dim=64, ff=2816, inner=2048, groups=1,
                  q=dict(n_expert=64, n_expert_used=10, expert_ff=256, shared_ff=256, ssm_n_group=8, ssm_dt_rank=16)),
    "w2048": dict(width=2048, layers=8, heads=16, kv=2, dim=256, ff=5632, inner=4096, groups=1,
                  q=dict(n_expert=512, n_expert_used=10, expert_ff=512, shared_ff=512, ssm_n_group=16, ssm_dt_rank=32)),
    "w4096": dict(width=4096, layers=4, heads=32, kv=8, dim=128, ff=11264, inner=8192, groups=8,
                  q=dict(n_expert=64, n_expert_used=10, expert_ff=1024, shared_ff=1024, ssm_n_group=32, ssm_dt_rank=64)),
}
VOCAB, STATE, VDIM, TAPS = 32768, 128, 64, 4


def serisun_config(s):
    att = {"type": "attention", "mixer": {"heads": s["heads"], "kv_heads": s["kv"], "dim": s["dim"], "vdim": s["dim"],
                                          "scale": s["dim"] ** -0.5, "q_temp": {"coef": 0.1, "every": 4096}}}
    ssm = {"type": "mamba2", "mixer": {"heads": s["inner"] // VDIM, "vdim": VDIM, "state": STATE, "groups": s["groups"],
                                       "norm_groups": s["groups"], "conv": TAPS}}
    layers = [dict(att if i % 4 == 3 else ssm, mlp={"kind": "dense", "ff": s["ff"]}) for i in range(s["layers"])]
    return {"architecture": "Serisun", "vocab": VOCAB, "width": s["width"], "norm": {"eps": 1e-6}, "logit_scale": 1.0, "layers": layers}


def tensor_shapes(cfg):
    d, out = cfg["width"], {}
    out["embed"] = out["head"] = (cfg["vocab"], d)
    out["final.norm"] = (d,)
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.", l["mixer"]
        for v in ("norm1", "ls1", "ls2"):
            out[p + v] = (d,)
        if l["type"] == "attention":
            h, g = m["heads"], m["kv_heads"]
            out.update({p + "mix.q": (h * m["dim"], d), p + "mix.k": (g * m["dim"], d), p + "mix.v": (g * m["vdim"], d), p + "mix.o": (d, h * m["vdim"])})
        else:
            inner = m["heads"] * m["vdim"]
            ch = inner + 2 * m["groups"] * m["state"]
            out.update({p + "mix.in": (inner + ch + m["heads"], d), p + "mix.conv": (ch, m["conv"]), p + "mix.conv.b": (ch,), p + "mix.norm": (inner,),
                        p + "mix.o": (d, inner)})
            for v in ("dt_bias", "A_log", "D"):
                out[p + "mix." + v] = (m["heads"],)
        f = l["mlp"]["ff"]
        out.update({p + "mlp.gate": (f, d), p + "mlp.up": (f, d), p + "mlp.down": (d, f)})
    return out


def vector(name, n, r):
    """A vector's (or a convolution's) random values."""
    v, leaf = r.standard_normal(n), name.rsplit(".", 1)[-1]
    return 1 + 0.1 * v if leaf in ("norm1", "norm", "D") or name == "final.norm" else 0.3 + 0.02 * v if leaf in ("ls1", "ls2") else \
        -3 + v if leaf == "dt_bias" else v if leaf == "A_log" else 0.3 * v


def write_random(folder: Path, cfg, seed=0, shapes=tensor_shapes, vector=vector):
    """config.json and model.safetensors with random bf16 weights (matrices N(0, 1 / row length), cut from one random block)."""
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg))
    r = np.random.default_rng(seed)
    block = r.standard_normal(1 << 22, dtype=np.float32)

    def bits(a):
        return (np.ascontiguousarray(a, np.float32).view(np.uint32) >> 16).astype("<u2")
    head, at, parts = {}, 0, []
    for name, sh in shapes(cfg).items():
        n = int(np.prod(sh))
        head[name] = {"dtype": "BF16", "shape": list(sh), "data_offsets": [at, at + 2 * n]}
        at += 2 * n
        parts.append((name, sh, n))
    h = json.dumps(head).encode()
    h += b" " * (-len(h) % 64)
    with open(folder / "model.safetensors", "wb") as f:
        f.write(struct.pack("<Q", len(h)) + h)
        for name, sh, n in parts:
            if len(sh) == 2 and not name.endswith("conv"):
                src = bits(np.roll(block, int(r.integers(0, block.size))) * sh[1] ** -0.5)
                for lo in range(0, n, src.size):
                    src[:min(src.size, n - lo)].tofile(f)
            else:
                bits(vector(name, n, r)).tofile(f)
    return folder


def qwen_config(ih, s, seed=0):
    return ih.SynthConfig(n_layer=s["layers"], n_embd=s["width"], n_vocab=VOCAB, n_head=s["heads"], n_head_kv=s["kv"], head_dim=s["dim"],
                          n_rot=64, ssm_d_conv=4, ssm_d_state=128, full_attention_interval=4, rope_theta=1e7, rms_eps=1e-6, dense_type=ih.Q8_0,
                          expert_type=ih.NVFP4, router_type=ih.Q8_0, seed=seed, weight_std=0.02, n_threads=16, **s["q"])


def flops(cfg, n, ctx):
    """Multiply-adds (two operations each) of a prefill pass by family, the head left out."""
    out = {"group": 0, "residual": 0, "attend": 0, "mamba2": 0}
    d = cfg["width"]
    for l in cfg["layers"]:
        m, f = l["mixer"], l["mlp"]["ff"]
        if l["type"] == "attention":
            out["group"] += 2 * n * d * (m["heads"] * m["dim"] + m["kv_heads"] * (m["dim"] + m["vdim"]) + 2 * f)
            out["residual"] += 2 * n * d * (m["heads"] * m["vdim"] + f)
            out["attend"] += m["heads"] * (m["dim"] + m["vdim"]) * n * (2 * ctx - n)   # causal: the mean of the visible keys
        else:
            inner, N, L = m["heads"] * m["vdim"], m["state"], 64
            out["group"] += 2 * n * d * (2 * inner + 2 * m["groups"] * N + m["heads"] + 2 * f)
            out["residual"] += 2 * n * d * (inner + f)
            out["mamba2"] += n * (m["groups"] * L * N + inner * (L + 4 * N))   # causal halves of C B^T and M X, C S0, the state
    return out


def measure(ih, model, prompt, steps, ctx):
    be = ih.Hip()
    eng = ih.Engine(model, be, ctx, 8192)
    eng.prefill(prompt, want_logits=False)       # uploads, buffer sizes
    be.sync()
    pre = []
    for _ in range(3):
        eng.reset()
        be.sync()
        t = time.perf_counter()
        eng.prefill(prompt, want_logits=False)
        be.sync()
        pre.append(time.perf_counter() - t)
    eng.decode_greedy(8)                         # the decode graph is recorded here
    dec = []
    for _ in range(3):
        be.sync()
        t = time.perf_counter()
        eng.decode_greedy(steps)
        be.sync()
        dec.append((time.perf_counter() - t) / steps)
    be.profile_begin()
    eng.decode_greedy(16)
    d_rows = be.profile_end()
    eng.reset()
    be.profile_begin()
    eng.prefill(prompt, want_logits=False)
    p_rows = be.profile_end()
    err, graph, chain = be.take_error(), be.graph_stats(), be.chain_stats()
    eng.close()
    be.close()
    if err:
        raise SystemExit(f"device error: {err}")
    return min(pre), sorted(dec)[1], p_rows, d_rows, graph, chain


def results(ih, model, prompt, steps, ctx, work, fp32=()):
    """What measure() found, with shares of the rooflines; `work`: operations of a prefill pass by the start of a family's name, on
    the bf16 matrix cores but for the families in `fp32`."""
    pre, dec, p_rows, d_rows, graph, chain = measure(ih, model, prompt, steps, ctx)
    r = {"prefill_tok_s": round(len(prompt) / pre), "prefill_ms": round(1e3 * pre, 2), "decode_tok_s": round(1 / dec, 1),
         "decode_ms": round(1e3 * dec, 4), "decode_weight_MB": round(model.decode_weight_bytes() / 1e6, 1),
         "decode_hbm_share": round(model.decode_weight_bytes() / dec / HBM, 3), "launches_per_token": graph["graph_kernels"], "chains": chain["chains"]}
    r["decode_kernels"] = [dict(name=x["name"], per_token=x["launches"] / 16, us=round(1e3 * x["ms"] / x["launches"], 2),
                                hbm_share=round(x["bytes"] / (x["ms"] * 1e-3) / HBM, 3)) for x in d_rows]
    r["prefill_kernels"] = [dict(name=x["name"], launches=x["launches"], ms=round(x["ms"], 3)) for x in p_rows]
    for fam, fl in work.items():
        for k in r["prefill_kernels"]:
            if k["name"].startswith(fam):
                k["tflops"] = round(fl / (k["ms"] * 1e-3) / 1e12, 1)
                k["peak_share"] = round(k["tflops"] * 1e12 / (FP32_PEAK if fam in fp32 else BF16_PEAK), 3)
    return r


def run(ih, tmp: Path, sizes, prompt_len=4096, steps=256, seed=0):
    out = []
    for name in sizes:
        s = SIZES[name]
        cfg = serisun_config(s)
        prompt = np.random.default_rng(seed).integers(0, VOCAB, prompt_len).astype(np.uint32)
        ctx = prompt_len + 1024 + 8 * ((steps * 3 + 64) // 8)
        row = {"size": name, "prompt": prompt_len, "layers": s["layers"], "width": s["width"]}
        ds = write_random(tmp / f"serisun_{name}", cfg, seed)
        gguf = tmp / f"qwen_{name}.gguf"
        ih.synth_write_gguf(gguf, qwen_config(ih, s, seed))
        for kind, path in (("serisun", ds), ("qwen35moe", gguf)):
            model = ih.Model(path)
            r = results(ih, model, prompt, steps, ctx, flops(cfg, prompt_len, prompt_len) if kind == "serisun" else {}, ("mamba2",))
            row[kind] = r
            model.close()
            print(f"# {name} {kind}: prefill {r['prefill_tok_s']} tok/s, decode {r['decode_tok_s']} tok/s", flush=True)
        gguf.unlink()
        for f in ds.iterdir():
            f.unlink()
        out.append(row)
    return out
