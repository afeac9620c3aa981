"""What the tests of folder models (config.json, model.safetensors) share: a model beside its oracle, feeding it in portions, and
the limits its logits are held to."""
import numpy as np

from serisun_util import logit_error, write

MODES = {"bf16": {}, "f32": {"f32": True}, "steps": {"fuse": False}}
LIMIT = {"bf16": 2e-2, "f32": 1e-4, "steps": 2e-2}


def backend(name):
    """A backend in one of the modes, with its limit."""
    import inferred_hip as ih
    b = ih.Hip(**MODES[name])
    b.name, b.limit = name, LIMIT[name]
    return b


def done(b):
    err = b.take_error()
    b.close()
    assert err is None, err


class Case:
    """`ref`: the oracle, with forward(tokens, cfg, w)"""

    def __init__(self, ref, folder, cfg, w):
        import inferred_hip as ih
        self.ref, self.cfg, self.w = ref, cfg, w
        self.path = write(folder, cfg, w)
        self.model = ih.Model(self.path)
        self.cache = {}

    def logits(self, tokens):
        key = tuple(int(t) for t in tokens)
        if key not in self.cache:
            self.cache[key] = self.ref.forward(tokens, self.cfg, self.w)
        return self.cache[key]

    def tokens(self, n, seed=0):
        return np.random.default_rng(seed).integers(0, self.cfg["vocab"], n)


def engine(case, be, n_ctx, max_batch=512):
    import inferred_hip as ih
    return ih.Engine(case.model, be, n_ctx, max_batch)


def feed(e, tokens, sizes):
    """The logits of every token, fed in portions of the given sizes (the last one repeated)."""
    out, at, k = [], 0, 0
    while at < len(tokens):
        c = min(sizes[min(k, len(sizes) - 1)], len(tokens) - at)
        out.append(e.forward_rows(tokens[at:at + c], np.arange(c)))
        at, k = at + c, k + 1
    return np.concatenate(out)


def held(got, want, be, what=""):
    e = logit_error(got, want)
    assert np.isfinite(got).all()
    # (a norm over a few channels that are all near zero multiplies a 16-bit rounding: one token in fifty may be up to four times as far)
    assert (e > be.limit).sum() <= (max(1, len(e) // 50) if be.limit > 1e-3 else 0) and e.max() < 4 * be.limit, f"{what}: {e.max():.2e} at token {int(e.argmax())}"
