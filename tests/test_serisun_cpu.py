"""The Serisun oracle on its own (does every mechanism show in the logits?), and what the loader accepts and refuses.
Runs without a GPU."""
import json
import struct

import numpy as np
import pytest

import serisun_ref as ref
from serisun_util import CONFIGS, attention, config, logit_error, mamba2, weights, write

TOKENS = np.random.default_rng(5).integers(0, 53, 60)


# ---------------------------------------------------------------- hand values
def test_sink_softmax_adds_one_to_the_denominator():
    s = np.log(np.array([[1.0, 2.0, 3.0]]))
    assert np.allclose(ref.sink_softmax(s), np.array([[1, 2, 3]]) / 7.0)
    assert np.allclose(ref.sink_softmax(s - 800.0), 0.0) and np.allclose(ref.sink_softmax(s + 800.0), np.array([[1, 2, 3]]) / 6.0)


def test_head_slopes_and_temperature():
    assert np.allclose(ref.head_slopes(8), [2.0 ** -k for k in range(1, 9)])
    assert np.allclose(ref.head_slopes(3), [2 ** (-8 / 3), 2 ** (-16 / 3), 2 ** -8])
    t = ref.query_temperature(9, 0.5, 4)   # positions 0..2 | 3..6 | 7, 8
    assert np.allclose(t, 1 + 0.5 * np.log([1, 1, 1, 2, 2, 2, 2, 3, 3]))


def test_the_bias_grows_with_the_distance():
    q, k = np.zeros((1, 1, 2)), np.zeros((3, 1, 2))
    v = np.eye(3)[:, None, :]
    p = ref.attend(q, k, v, 1.0, np.array([np.log(2.0)]))[0, 0]
    assert np.allclose(p, np.array([0.25, 0.5, 1.0]) / 2.75)


def test_convolution_order_and_start():
    x = np.array([[1.0], [10.0], [100.0]])
    y = ref.causal_conv_silu(x, np.array([[3.0, 2.0]]), np.array([0.5]))   # last column: the current token
    raw = np.array([[2.5], [23.5], [230.5]])
    assert np.allclose(y, raw / (1 + np.exp(-raw)))


def test_state_space_by_hand():
    x, B, C = np.array([[[2.0]], [[3.0]]]), np.array([[[1.0]], [[5.0]]]), np.array([[[7.0]], [[11.0]]])
    dt = np.array([[0.5], [0.25]])
    y, S = ref.state_space(x, B, C, dt, np.array([np.log(2.0)]), np.array([0.1]))
    s1 = 0.5 * 2.0
    s2 = np.exp(-0.5) * s1 + 0.25 * 5 * 3
    assert np.allclose(y[:, 0, 0], [7 * s1 + 0.2, 11 * s2 + 0.3]) and np.allclose(S, s2)


def test_the_gate_comes_before_the_norm():
    y, z = np.array([[1.0, 2.0, 3.0, 4.0]]), np.array([[0.5, -1.0, 2.0, 0.1]])
    g = y * z / (1 + np.exp(-z))
    want = np.concatenate([g[:, :2] / np.sqrt((g[:, :2] ** 2).mean()), g[:, 2:] / np.sqrt((g[:, 2:] ** 2).mean())], 1)
    assert np.allclose(ref.gated_group_norm(y, z, np.ones(4), 2, 0.0), want)


def test_layer_order_of_a_loop():
    assert ref.layer_runs(CONFIGS["mixed"]) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (1, 2), (2, None), (3, None)]


# ---------------------------------------------------------------- every mechanism shows
def _off(name):
    """The oracle with one mechanism wrong, and what puts it right again."""
    keep = {n: getattr(ref, n) for n in ("sink_softmax", "head_slopes", "query_temperature", "causal_conv_silu", "softplus",
                                         "gated_group_norm", "state_space", "attend", "layer_runs", "rms", "silu")}
    silu = ref.silu
    wrong = {
        "no sink": {"attend": lambda q, k, v, s, b: keep["attend"](q, k, v, s, b, sink=False)},
        "no distance bias": {"head_slopes": lambda n: np.zeros(n)},
        "slopes one head off": {"head_slopes": lambda n: np.roll(keep["head_slopes"](n), 1)},
        "no temperature": {"query_temperature": lambda n, c, e: np.ones(n)},
        "temperature one position late": {"query_temperature": lambda n, c, e: np.concatenate([[1.0], keep["query_temperature"](n, c, e)[:-1]])},
        "taps reversed": {"causal_conv_silu": lambda x, t, b: keep["causal_conv_silu"](x, t[:, ::-1], b)},
        "no conv bias": {"causal_conv_silu": lambda x, t, b: keep["causal_conv_silu"](x, t, 0 * b)},
        "gate after the norm": {"gated_group_norm": lambda y, z, w, g, e: keep["gated_group_norm"](y, np.full_like(z, 1e4), w, g, e) * silu(z)},
        "norm in one part": {"gated_group_norm": lambda y, z, w, g, e: keep["gated_group_norm"](y, z, w, 1, e)},
        "no skip": {"state_space": lambda x, B, C, dt, A, D: keep["state_space"](x, B, C, dt, A, 0 * D)},
        "head to group by remainder": {"state_space": lambda x, B, C, dt, A, D: keep["state_space"](
            x, np.stack([B[:, h % B.shape[1]] for h in range(x.shape[1])], 1), np.stack([C[:, h % C.shape[1]] for h in range(x.shape[1])], 1), dt, A, D)},
        "no state carried": {"state_space": lambda x, B, C, dt, A, D: keep["state_space"](x, B, C, dt, A + 20, D)},
        "one pass too few": {"layer_runs": lambda c: keep["layer_runs"](dict(c, loop=dict(c["loop"], times=c["loop"]["times"] - 1)))},
        "the pass vector of the first pass throughout": {"layer_runs": lambda c: [(i, 0 if o is not None else None) for i, o in keep["layer_runs"](c)]},
    }[name]
    return wrong, keep


@pytest.mark.parametrize("name", ["no sink", "no distance bias", "slopes one head off", "no temperature", "temperature one position late",
                                  "taps reversed", "no conv bias", "gate after the norm", "norm in one part", "no skip",
                                  "head to group by remainder", "no state carried", "one pass too few",
                                  "the pass vector of the first pass throughout"])
def test_a_mistake_shows_in_the_logits(name):
    """A mistake moves some token's logits by more than twice the 2e-2 the 16-bit kernels are held to (and by hundreds of times
    the 1e-4 of the 32-bit ones)."""
    cfg = CONFIGS["mixed"]
    w = weights(cfg, 1)
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


def test_the_oracle_is_causal():
    cfg = CONFIGS["all_looped"]
    w = weights(cfg, 2)
    assert np.allclose(ref.forward(TOKENS[:20], cfg, w), ref.forward(TOKENS, cfg, w)[:20])


# ---------------------------------------------------------------- the loader
def _open(tmp_path, cfg, w):
    import inferred_hip as ih
    return ih.Model(write(tmp_path / "m", cfg, w))


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_a_folder_opens_and_knows_its_sizes(tmp_path, name):
    cfg = CONFIGS[name]
    w = weights(cfg, 0)
    m = _open(tmp_path, cfg, w)
    assert (m.n_layer, m.n_embd, m.n_vocab) == (len(cfg["layers"]), cfg["width"], cfg["vocab"])
    # a looped layer's matrices are read once per pass
    runs = [i for i, _ in ref.layer_runs(cfg)]
    mats = sum(v.size for i in runs for k, v in w.items() if k.startswith(f"l{i}.") and v.ndim == 2 and not k.endswith("conv"))
    assert m.decode_weight_bytes() == 2 * (mats + w["head"].size)
    assert m.token_macs() == (mats, 0, 0)
    m.close()


def test_models_are_chosen_by_the_name_their_files_give(tmp_path):
    import inferred_hip as ih
    cfg = dict(CONFIGS["odd"], architecture="Moonward")
    with pytest.raises(ih.HipError, match="unsupported architecture 'Moonward'.*Serisun"):
        _open(tmp_path, cfg, weights(CONFIGS["odd"]))
    with pytest.raises(ih.HipError, match="no such file"):
        ih.Model(tmp_path / "nothing")
    (tmp_path / "empty").mkdir()
    with pytest.raises(ih.HipError, match="config.json"):
        ih.Model(tmp_path / "empty")


@pytest.mark.parametrize("change, message", [
    (lambda c, w: w.pop("l2.mix.k"), "missing tensor l2.mix.k"),
    (lambda c, w: w.update({"l0.ls1": w["l0.ls1"][:-1]}), "tensor l0.ls1: expected"),
    (lambda c, w: w.update({"loop.step": w["loop.step"][:2]}), "tensor loop.step"),
    (lambda c, w: c.pop("logit_scale"), "logit_scale"),
    (lambda c, w: c["layers"][0]["mixer"].update(kv_heads=3), "heads do not divide"),
    (lambda c, w: c["layers"][1]["mixer"].update(norm_groups=5), "norm_groups"),
    (lambda c, w: c["layers"][1]["mixer"].update(state=2.5), "not a whole number"),
    (lambda c, w: c["layers"][1].update(type="retention"), "unknown mixer 'retention'"),
    (lambda c, w: c["layers"][1]["mlp"].update(kind="moe"), "unknown kind"),
    (lambda c, w: c["loop"].update(stop=9), "loop does not name"),
])
def test_a_wrong_folder_is_refused(tmp_path, change, message):
    import inferred_hip as ih
    cfg = json.loads(json.dumps(CONFIGS["mixed"]))
    w = weights(CONFIGS["mixed"], 0)
    change(cfg, w)
    with pytest.raises(ih.HipError, match=message):
        _open(tmp_path, cfg, w)


@pytest.mark.parametrize("blob, message", [
    (b"\x05", "too short"),
    (b"\xff" * 16, "header longer"),
    (b"\x02\0\0\0\0\0\0\0{]", "header"),
    (struct.pack("<Q", 59) + b'{"embed":{"dtype":"F32","shape":[4],"data_offsets":[0,16]}}' + b"\0" * 4, "fit its shape or the file"),
])
def test_a_broken_tensor_file_is_refused(tmp_path, blob, message):
    import inferred_hip as ih
    d = write(tmp_path / "m", CONFIGS["odd"], weights(CONFIGS["odd"]))
    (d / "model.safetensors").write_bytes(blob)
    with pytest.raises(ih.HipError, match=message):
        ih.Model(d)


@pytest.mark.parametrize("text", ['{"a": 1,}', '{"a" 1}', '{"a": 01x}', '[1, 2', '{"a": "\\q"}', '{"a": nul}', '{"a": 1} x', '{"a": 1, "a": 2}'])
def test_a_broken_configuration_is_refused(tmp_path, text):
    import inferred_hip as ih
    d = write(tmp_path / "m", CONFIGS["odd"], weights(CONFIGS["odd"]))
    (d / "config.json").write_text(text)
    with pytest.raises(ih.HipError, match="config.json"):
        ih.Model(d)
