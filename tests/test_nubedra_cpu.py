"""The Nubedra oracle on its own (hand values; does every mechanism show in the logits?), and what the loader accepts and
refuses.  Runs without a GPU."""
import json

import numpy as np
import pytest

import nubedra_ref as ref
from nubedra_util import CONFIGS, weights
from serisun_util import logit_error, write

TOKENS = np.random.default_rng(5).integers(0, 53, 70)


# ---------------------------------------------------------------- hand values
def test_norm_weights_are_stored_around_zero():
    x = np.array([[3.0, -4.0]])
    assert np.allclose(ref.centred_norm(x, np.array([0.0, 1.0]), 0.0), [[3 / np.sqrt(12.5), -8 / np.sqrt(12.5)]])
    assert np.allclose(ref.centred_norm(x, np.zeros(2), 12.5), [[0.6, -0.8]])


def test_key_decay():
    assert np.allclose(ref.key_decay(np.array([0.0]), 1.0), 0.5) and np.allclose(ref.key_decay(np.array([0.0]), 2.0), np.sqrt(0.5))
    assert np.allclose(ref.key_decay(np.array([np.log(3.0)]), 4.0), 0.75 ** 0.25)
    assert np.allclose(ref.key_decay(np.array([-800.0]), 16.0), np.exp(-50.0))


def test_the_decay_acts_on_key_channels():
    q, k = np.array([[[1.0, 10.0]], [[2.0, 3.0]]]), np.array([[[5.0, 7.0]], [[1.0, -1.0]]])
    v, a = np.array([[[2.0, 0.5, 1.0]], [[1.0, 4.0, 0.0]]]), np.array([[[0.3, 0.9]], [[0.5, 0.25]]])
    o, S = ref.gated_recurrence(q, k, v, a)
    s1 = np.array([[10.0, 2.5, 5.0], [14.0, 3.5, 7.0]])                # the first token's own decay meets an empty state
    s2 = np.array([[5 + 1, 1.25 + 4, 2.5], [3.5 - 1, 0.875 - 4, 1.75]])
    assert np.allclose(o[0, 0], s1[0] + 10 * s1[1]) and np.allclose(o[1, 0], 2 * s2[0] + 3 * s2[1]) and np.allclose(S[0], s2)


def test_the_norm_of_a_head_comes_before_the_gate():
    o, z = np.array([[[3.0, 4.0], [1.0, 1.0]]]), np.array([[0.5, -1.0, 2.0, 0.1]])
    n = np.array([3 / np.sqrt(12.5) * 2, 4 / np.sqrt(12.5) * 5, 2.0, 5.0])
    assert np.allclose(ref.gated_norm(o, np.array([2.0, 5.0]), z, 0.0), n * z / (1 + np.exp(-z)))


def test_neighbouring_dimensions_turn_together():
    x = np.array([[1.0, 2.0, 3.0, 4.0, 9.0]])
    y = ref.rotate(x, [3], {"base": 100.0, "dims": 4})
    c, s, c2, s2 = np.cos(3), np.sin(3), np.cos(0.3), np.sin(0.3)
    assert np.allclose(y, [[c - 2 * s, 2 * c + s, 3 * c2 - 4 * s2, 4 * c2 + 3 * s2, 9.0]])


def test_scaled_frequencies():
    f, m = ref.rotation({"base": 16.0, "dims": 8, "scaling": {"factor": 4.0, "original": 64 * np.pi, "fast": 16.0, "slow": 1.0}})
    # 32 / turns = 16^(2 d / 8): 16 turns at dimension 1, 1 turn at dimension 5; the ramp covers pairs 1 .. 5
    ramp = np.array([0.0, 0.0, 0.25, 0.5])
    plain = 16.0 ** (-np.arange(4) / 4)
    assert np.allclose(f, plain * (1 - ramp) + plain / 4 * ramp) and np.isclose(m, 0.1 * np.log(4.0) + 1)
    f, m = ref.rotation({"base": 16.0, "dims": 8})
    assert np.allclose(f, plain) and m == 1.0


def test_a_window_counts_the_token_itself():
    assert np.array_equal(ref.visible(2, 4, 2), [[False, True, True, False], [False, False, True, True]])
    assert np.array_equal(ref.visible(3, 3, 1), np.eye(3, dtype=bool)) and np.array_equal(ref.visible(3, 3, None), np.tri(3, dtype=bool))


def test_the_sink_counts_once_and_is_not_scaled():
    s = np.log(np.array([[1.0, 2.0, 3.0]]))
    assert np.allclose(ref.sink_softmax(s, np.log(4.0)), np.array([[1, 2, 3]]) / 10.0)
    assert np.allclose(ref.sink_softmax(s + 800.0, 0.0), np.array([[1, 2, 3]]) / 6.0)
    q, c, kr = np.ones((1, 1, 2)), np.array([[np.log(2.0)], [0.0]]), np.zeros((2, 1))
    y = ref.latent_attend(q, c, kr, np.array([[2.0]]), np.array([[1.0]]), 0.5, None, np.array([np.log(3.0)]))
    assert np.allclose(y, 2 * np.log(2.0) / (2 + 1 + 3))


# ---------------------------------------------------------------- every mechanism shows
def _off(name):
    """The oracle with one mechanism wrong, and what puts it right again."""
    keep = {n: getattr(ref, n) for n in ("sink_softmax", "visible", "rotation", "rotate", "key_decay", "gated_recurrence", "gated_norm", "output_gate",
                                         "centred_norm", "relu", "silu", "latent_kv", "latent_attend")}
    k = keep
    wrong = {
        "no sink": {"sink_softmax": lambda s, sink: k["sink_softmax"](s, -1e9)},
        "a sink of one": {"sink_softmax": lambda s, sink: k["sink_softmax"](s, 0.0)},
        "a window one token wide": {"visible": lambda n, m, size: k["visible"](n, m, size and size + 1)},
        "a window one token short": {"visible": lambda n, m, size: k["visible"](n, m, size and max(1, size - 1))},
        "no window": {"visible": lambda n, m, size: k["visible"](n, m, None)},
        "no frequency scaling": {"rotation": lambda r: k["rotation"](dict(r, scaling=None))},
        "no factor of cos and sin": {"rotation": lambda r: (k["rotation"](r)[0], 1.0)},
        "halves instead of neighbours": {"rotate": lambda x, p, r: k["rotate"](x[..., np.arange(x.shape[-1]).reshape(2, -1).T.ravel()], p, r)},
        "positions one late": {"rotate": lambda x, p, r: k["rotate"](x, np.asarray(p) * (1 + (x.ndim > 2) * 0.03), r)},
        "the latent not normed": {"latent_kv": lambda h, mx, w, pre, eps: (h @ w[pre + "dkv"][:mx["kv_rank"]].T, k["latent_kv"](h, mx, w, pre, eps)[1])},
        "the key part not rotated": {"latent_kv": lambda h, mx, w, pre, eps: (k["latent_kv"](h, mx, w, pre, eps)[0], h @ w[pre + "dkv"][mx["kv_rank"]:].T)},
        "no output gate": {"output_gate": lambda z: np.ones_like(z)},
        "tau left out": {"key_decay": lambda z, tau: k["key_decay"](z, 1.0)},
        "one decay for all channels": {"key_decay": lambda z, tau: np.broadcast_to(k["key_decay"](z, tau).mean(-1, keepdims=True), z.shape)},
        "decay behind the sum": {"gated_recurrence": lambda q, kk, v, a: k["gated_recurrence"](q, kk * a, v, a)},
        "no state carried": {"gated_recurrence": lambda q, kk, v, a: k["gated_recurrence"](q, kk, v, 0 * a)},
        "gate ahead of the head's norm": {"gated_norm": lambda o, w, z, e: (ref.rms(o * k["silu"](z).reshape(o.shape), e) * w).reshape(z.shape)},
        "norm weights around one": {"centred_norm": lambda x, w, e: ref.rms(x, e) * w},
        "silu in the feed-forward": {"relu": lambda z: k["silu"](z)},
    }[name]
    return wrong, keep


@pytest.mark.parametrize("name", ["no sink", "a sink of one", "a window one token wide", "a window one token short", "no window",
                                  "no frequency scaling", "no factor of cos and sin", "halves instead of neighbours", "positions one late",
                                  "the latent not normed", "the key part not rotated", "no output gate", "tau left out", "one decay for all channels",
                                  "decay behind the sum", "no state carried", "gate ahead of the head's norm", "norm weights around one",
                                  "silu in the feed-forward"])
def test_a_mistake_shows_in_the_logits(name):
    """A mistake moves some token's logits by more than twice the 2e-2 the 16-bit kernels are held to (and by hundreds of times
    the 1e-4 of the 32-bit ones)."""
    cfg, w = CONFIGS["mixed"], weights("mixed", 1)
    good = ref.forward(TOKENS, cfg, w)
    wrong, keep = _off(name)
    try:
        for k, v in wrong.items():
            setattr(ref, k, v)
        bad = ref.forward(TOKENS, cfg, w)
    finally:
        for k, v in keep.items():
            setattr(ref, k, v)
    assert logit_error(bad, good).max() > 0.04


@pytest.mark.parametrize("change", [dict(residual_mult=0.5), dict(embedding={"scale": 2.5}), dict(norm={"eps": 0.03})])
def test_every_constant_shows_in_the_logits(change):
    cfg, w = CONFIGS["mixed"], weights("mixed", 1)
    assert logit_error(ref.forward(TOKENS, dict(cfg, **change), w), ref.forward(TOKENS, cfg, w)).max() > 0.02


def test_a_sharing_layer_reads_the_other_layers_rows():
    """The rows a sharing layer reads beyond its owner's window count too."""
    cfg, w = CONFIGS["mixed"], weights("mixed", 1)
    own = json.loads(json.dumps(cfg))
    own["layers"][2]["mixer"]["mask"]["size"] = own["layers"][0]["mixer"]["mask"]["size"]
    assert logit_error(ref.forward(TOKENS, own, w), ref.forward(TOKENS, cfg, w)).max() > 0.04


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_the_oracle_is_causal(name):
    cfg, w = CONFIGS[name], weights(name, 2)
    assert np.allclose(ref.forward(TOKENS[:20], cfg, w), ref.forward(TOKENS, cfg, w)[:20])


# ---------------------------------------------------------------- the loader
def _open(tmp_path, cfg, w):
    import inferred_hip as ih
    return ih.Model(write(tmp_path / "m", cfg, w))


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_a_folder_opens_and_knows_its_sizes(tmp_path, name):
    cfg, w = CONFIGS[name], weights(name)
    m = _open(tmp_path, cfg, w)
    assert (m.n_layer, m.n_embd, m.n_vocab) == (len(cfg["layers"]), cfg["width"], cfg["vocab"])
    mats = sum(v.size for k, v in w.items() if k.startswith("l") and v.ndim == 2)
    assert m.decode_weight_bytes() == 2 * (mats + w["embed"].size) and m.token_macs() == (mats, 0, 0)
    m.close()


@pytest.mark.parametrize("change, message", [
    (lambda c, w: w.pop("l1.mix.a2"), "missing tensor l1.mix.a2"),
    (lambda c, w: w.pop("l1.mix.a1"), "missing tensor l1.mix.a1"),
    (lambda c, w: w.pop("l4.mix.dkv"), "missing tensor l4.mix.dkv"),
    (lambda c, w: w.update({"l0.mix.sink": w["l0.mix.sink"][:-1]}), "tensor l0.mix.sink: expected"),
    (lambda c, w: w.update({"l0.mix.dkv": w["l0.mix.dkv"][:-1]}), "tensor l0.mix.dkv: expected"),
    (lambda c, w: w.update({"l0.norm2b": w["l0.norm2b"][:-1]}), "tensor l0.norm2b: expected"),
    (lambda c, w: c.pop("residual_mult"), "residual_mult"),
    (lambda c, w: c.pop("embedding"), "embedding.scale"),
    (lambda c, w: c["layers"][1]["mixer"].update(tau=0), "tau"),
    (lambda c, w: c["layers"][1]["mixer"].update(dim=600), "512 key channels"),
    (lambda c, w: c["layers"][0]["mixer"]["rot"].update(dims=7), "mixer.rot"),
    (lambda c, w: c["layers"][0]["mixer"]["rot"].update(dims=10), "mixer.rot"),
    (lambda c, w: c["layers"][0]["mixer"]["rot"]["scaling"].pop("slow"), "scaling.slow"),
    (lambda c, w: c["layers"][0]["mixer"]["rot"]["scaling"].update(factor=0), "must be positive"),
    (lambda c, w: c["layers"][0]["mixer"]["mask"].update(size=0), "mask.size"),
    (lambda c, w: c["layers"][2]["mixer"].update(kv_from=1), "kv_from does not name"),
    (lambda c, w: c["layers"][2]["mixer"].update(kv_from=4), "kv_from does not name"),
    (lambda c, w: c["layers"][4]["mixer"].update(kv_from=2), "kv_from does not name"),
    (lambda c, w: c["layers"][4]["mixer"].update(kv_from=0), "another kv_rank"),
    (lambda c, w: c["layers"][2]["mixer"]["rot"].update(base=501.0), "another kv_rank, rot_dim or rotation"),
    (lambda c, w: c["layers"][1].update(type="mamba2"), "unknown mixer 'mamba2'"),
    (lambda c, w: c["layers"][0]["mlp"].update(kind="moe"), "unknown kind"),
])
def test_a_wrong_folder_is_refused(tmp_path, change, message):
    import inferred_hip as ih
    cfg, w = json.loads(json.dumps(CONFIGS["mixed"])), weights("mixed")
    change(cfg, w)
    with pytest.raises(ih.HipError, match=message):
        _open(tmp_path, cfg, w)
