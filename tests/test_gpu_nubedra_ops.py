"""The seam ops that Nubedra brought, each against the plain oracle (nubedra_ref.py): a normed addition ahead of a group of
products, products without a residual, gated linear attention, latent attention, windows and sinks of biased attention.  Three
backends: the default (matrix cores for batches), 32-bit mode, and one launch per operation."""
import numpy as np
import pytest

import nubedra_ref as ref
from test_gpu_float_ops import MODES, Mat, _held, f16, group_mat, read_rows, rel, res_term, tolerance
from util import rng

pytestmark = pytest.mark.gpu
TOKENS = [1, 2, 9, 16, 17, 130]


@pytest.fixture(params=sorted(MODES))
def be(request):
    import inferred_hip as ih
    b = ih.Hip(**MODES[request.param])
    b.name = request.param
    yield b
    err = b.take_error()
    b.close()
    assert err is None, err


def addition(y, w, x_new, eps, mult):
    import inferred_hip as ih
    return ih.AddNormed(y.ctypes.data, w.ctypes.data, x_new.ctypes.data, eps, mult)


# ---------------------------------------------------------------- products around norms
@pytest.mark.parametrize("n_in", [64, 37, 520, 1032])
@pytest.mark.parametrize("n", TOKENS)
def test_a_normed_addition_ahead_of_a_group(be, n, n_in):
    r = rng(n * 100 + n_in)
    f = lambda *s: r.standard_normal(s).astype(np.float32)
    x, y, yw, nw = f(n * n_in), 4 * f(n * n_in), 1 + 0.3 * f(n_in), 1 + 0.3 * f(n_in)
    x_new = np.zeros_like(x)
    mats = [Mat(r, 48, n_in), Mat(r, 7, n_in)]
    outs = [np.zeros(n * 48, np.float32), np.zeros(n * 7, np.float32)]
    be.add_norm_matmuls(x, addition(y, yw, x_new, 1e-3, 0.4), nw, n_in, 1e-4, [group_mat(m, o, scale=s) for m, o, s in zip(mats, outs, (0.5, 1.0))])
    want = x.reshape(n, -1) + 0.4 * ref.rms(y.reshape(n, -1).astype(np.float64), 1e-3) * yw
    h = ref.rms(want, 1e-4) * nw
    be.host_needs(x_new)
    assert rel(x_new.reshape(n, -1), want) < 1e-5
    for m, o, s in zip(mats, outs, (0.5, 1.0)):
        be.host_needs(o)
        assert rel(o.reshape(n, -1), h @ m.v.T * s) < tolerance(be, n)


@pytest.mark.parametrize("n_in", [40, 37, 1500, 8200])
@pytest.mark.parametrize("n", [1, 5, 40])
def test_a_normed_addition_alone(be, n, n_in):
    r = rng(n + n_in)
    x, y, w = (r.standard_normal(s).astype(np.float32) for s in (n * n_in, n * n_in, n_in))
    x_new = np.zeros_like(x)
    be.add_normed(x, n_in, addition(y, w, x_new, 1e-2, 1.7))
    be.host_needs(x_new)
    assert rel(x_new.reshape(n, -1), x.reshape(n, -1) + 1.7 * ref.rms(y.reshape(n, -1).astype(np.float64), 1e-2) * w) < 1e-5


@pytest.mark.parametrize("n_in, ff", [(64, 96), (37, 21)])
@pytest.mark.parametrize("n", TOKENS)
def test_a_pair_with_relu(be, n, n_in, ff):
    r = rng(n * 7 + ff)
    x, nw = r.standard_normal(n * n_in).astype(np.float32), np.ones(n_in, np.float32)
    gate, up, out = Mat(r, ff, n_in), Mat(r, ff, n_in), np.zeros(n * ff, np.float32)
    g = group_mat(gate, out, up=up)
    g.act = 1
    be.norm_matmuls(x, nw, n_in, 1e-5, [g])
    h = ref.rms(x.reshape(n, n_in).astype(np.float64), 1e-5)
    assert rel(read_rows(be, out, n, ff), ref.relu(h @ gate.v.T) * (h @ up.v.T)) < (3e-2 if be.name == "default" and n > 16 else 1e-2 if n > 16 and not be.f32 else 2e-5)


@pytest.mark.parametrize("nd, heads, dv", [(64, 3, 24), (37, 5, 7), (96, 1, 130), (600, 12, 64), (40, 2, 300), (24, 1, 1200)])
@pytest.mark.parametrize("gated", [True, False])
@pytest.mark.parametrize("n", TOKENS)
def test_a_product_of_normed_and_gated_heads(be, n, gated, nd, heads, dv):
    """One weight for every head's norm, the gate behind it, and nothing of what the output held."""
    r = rng(n * 31 + nd)
    o, z, w = (r.standard_normal(s).astype(np.float32) for s in (n * heads * dv, n * heads * dv, dv))
    m, out = Mat(r, nd, heads * dv), np.full(n * nd, 7.0, np.float32)
    t = res_term(m, o, norm=w, groups=heads, eps=1e-3)
    t.norm_shared = 1
    if gated:
        t.gate, t.gate_len = z.ctypes.data, z.size
    be.host_wrote(out)
    be.matmul_sum(out, [t])
    be.host_needs(out)
    v = o.reshape(n, heads, dv).astype(np.float64)
    v = ref.gated_norm(v, w, z.reshape(n, -1).astype(np.float64), 1e-3) if gated else (ref.rms(v, 1e-3) * w).reshape(n, -1)
    assert rel(out.reshape(n, nd), v @ m.v.T) < tolerance(be, n)


# ---------------------------------------------------------------- gated linear attention
class Recurrence:
    def __init__(self, r, heads, dim, vdim, rank, tau, ty="bf16", bias=None):
        self.heads, self.dim, self.vdim, self.rank, self.tau = heads, dim, vdim, rank, tau
        self.a2 = Mat(r, heads * dim, rank, ty)
        self.b = (r.standard_normal(heads * dim) * 2 + 1 if bias is None else bias).astype(np.float32)
        self.state = np.zeros(heads * vdim * dim, np.float32)

    def inputs(self, r, n):
        s = lambda *sh: r.standard_normal(sh).astype(np.float32)
        return s(n, self.heads * self.dim), s(n, self.heads * self.dim), s(n, self.heads * self.vdim), s(n, self.rank)

    def oracle(self, q, k, v, low):
        n, H = q.shape[0], self.heads
        z = low.astype(np.float64) @ self.a2.v.T + self.b
        f = lambda x: x.astype(np.float64).reshape(n, H, -1)
        o, S = ref.gated_recurrence(f(q), f(k), f(v), ref.key_decay(z, self.tau).reshape(n, H, -1))
        return o.reshape(n, -1), S.transpose(0, 2, 1)

    def run(self, be, q, k, v, low):
        import inferred_hip as ih
        a = [np.ascontiguousarray(x).reshape(-1) for x in (q, k, v, low)]
        out = np.zeros(v.size, np.float32)
        g = ih.Gla(*[x.ctypes.data for x in a], *[x.size for x in a], self.a2.w, self.b.ctypes.data, self.heads, self.dim, self.vdim, self.tau, 0)
        be.gla(g, self.state, out)
        be.host_needs(out)
        for x in a + [out]:
            be.release(x)
        return out.reshape(v.shape).copy()

    def read_state(self, be):
        be.read_state(self.state)
        return self.state.reshape(self.heads, self.vdim, self.dim).copy()


RECURRENCES = [(3, 24, 40, 8, 4.0), (2, 16, 16, 16, 1.0), (3, 7, 5, 3, 2.0), (1, 128, 80, 16, 16.0), (4, 18, 19, 1, 8.0), (2, 264, 24, 24, 16.0), (1, 500, 24, 33, 3.0),
               (5, 64, 64, 12, 16.0)]


@pytest.mark.parametrize("shape", RECURRENCES)
@pytest.mark.parametrize("pieces", [[1] * 9, [2, 3, 2, 1, 1, 2], [63], [64], [65, 1, 1], [130, 2, 64, 1], [17, 200, 3]])
def test_gla_in_pieces_against_the_whole(be, shape, pieces):
    """One call or many, alone or behind one another: the same read-outs and the same last state, from a fresh start each."""
    r = rng(sum(pieces) + shape[1])
    m = Recurrence(r, *shape)
    for turn in range(2):                         # the second sequence uses the same state again
        x = m.inputs(r, sum(pieces))
        want, S = m.oracle(*x)
        got, at = [], 0
        for c in pieces:
            got.append(m.run(be, *[a[at:at + c] for a in x]))
            at += c
        assert rel(np.concatenate(got), want) < 5e-5
        assert rel(m.read_state(be), S) < 5e-5
        m.state[:] = 0
        be.L.it_hip_zero_slab(be.h, m.state.ctypes.data)


@pytest.mark.parametrize("ty", ["f16", "f32"])
def test_gla_other_matrix_types(be, ty):
    r = rng(3)
    m = Recurrence(r, 2, 20, 12, 9, 2.0, ty)
    x = m.inputs(r, 80)
    want, S = m.oracle(*x)
    got = np.concatenate([m.run(be, *[a[lo:hi] for a in x]) for lo, hi in ((0, 70), (70, 71), (71, 80))])
    assert rel(got, want) < 5e-5 and rel(m.read_state(be), S) < 5e-5


@pytest.mark.parametrize("n", [70, 200])
def test_gla_channels_that_forget_at_once_beside_ones_that_keep_all(be, n):
    """Decays of e^-80 a token (a chunk's product far outside f32's range) beside ones of 1 - 1e-6, in the same head."""
    r = rng(n)
    bias = np.where(np.arange(4 * 32) % 3 == 0, -80.0, np.where(np.arange(4 * 32) % 3 == 1, 14.0, 0.0))
    m = Recurrence(r, 4, 32, 32, 8, 1.0, bias=bias)
    x = m.inputs(r, n)
    want, S = m.oracle(*x)
    got = m.run(be, *x)
    assert np.isfinite(got).all() and rel(got, want) < 1e-4 and rel(m.read_state(be), S) < 1e-4


@pytest.mark.parametrize("far", [0, 1, 15, 16, 31, 63, 64, 65, 127, 128])
def test_gla_one_token_far_back_is_remembered(be, far):
    """One token's key answers the last queries through a channel that keeps; every other token writes another channel."""
    r = rng(1)
    m = Recurrence(r, 1, 8, 8, 2, 1.0, bias=np.full(8, 12.0))
    n = 140
    q, k, v, low = (np.zeros_like(a) for a in m.inputs(r, n))
    q[far + 1:, 3] = 1.0
    k[:, 5], k[far] = 1.0, 0.0
    k[far, 3] = 50.0
    v[:, 0], v[:, 1] = np.arange(n) / 64.0, 1.0
    want, _ = m.oracle(q, k, v, low)
    got = np.concatenate([m.run(be, *[a[lo:hi] for a in (q, k, v, low)]) for lo, hi in ((0, 137), (137, 138), (138, 140))])
    assert np.allclose(want[-1, 0], 50 * far / 64.0, rtol=1e-2) and np.allclose(got, want, rtol=1e-4, atol=1e-4)


def test_gla_over_more_chunks_than_are_taken_at_once(be):
    """A state so large that the chunked form takes eight chunks at a time: one call of ten against two calls of fewer."""
    r = rng(2)
    m = Recurrence(r, 32, 512, 320, 4, 16.0)
    x = m.inputs(r, 600)
    runs = []
    for pieces in ((600,), (300, 300)):
        at, out = 0, []
        for c in pieces:
            out.append(m.run(be, *[a[at:at + c] for a in x]))
            at += c
        runs.append((np.concatenate(out), m.read_state(be)))
        m.state[:] = 0
        be.L.it_hip_zero_slab(be.h, m.state.ctypes.data)
    assert rel(runs[0][0], runs[1][0]) < 1e-4 and rel(runs[0][1], runs[1][1]) < 1e-4 and np.abs(runs[0][1]).max() > 0.1


# ---------------------------------------------------------------- latent attention
class LatentLayer:
    def __init__(self, r, heads, dim, rot, vdim, rank, window, cap, f32, n_rot=None, scaling=None, ty="bf16", sink=True, gate=True):
        self.heads, self.dim, self.rot, self.vdim, self.rank, self.window, self.cap = heads, dim, rot, vdim, rank, window, cap
        self.n_rot, self.scaling = rot if n_rot is None else n_rot, scaling
        self.uk, self.uv = Mat(r, heads * dim, rank, ty), Mat(r, heads * vdim, rank, ty)
        self.norm = (1 + 0.3 * r.standard_normal(rank)).astype(np.float32)
        self.sink = r.standard_normal(heads).astype(np.float32) if sink else None
        self.gated, self.scale, self.eps = gate, 1.5 * (dim + rot) ** -0.5, 1e-4
        self.row = (rank + rot + 7) // 8 * 8
        self.slab = np.zeros(cap * self.row, np.float32 if f32 else np.float16)

    def inputs(self, r, n):
        s = lambda *sh: r.standard_normal(sh).astype(np.float32)
        return s(n, self.heads * (self.dim + self.rot)), s(n, self.rank + self.rot), s(n, self.heads)

    def rotation(self):
        return {"base": 40.0, "dims": self.n_rot, "scaling": dict(zip(("factor", "original", "fast", "slow"), self.scaling)) if self.scaling else None}

    def oracle(self, q, kv, z, window=None):
        n, H = q.shape[0], self.heads
        q, kv, z = (a.astype(np.float64) for a in (q, kv, z))
        pos = np.arange(n)
        c = ref.rms(kv[:, :self.rank], self.eps) * self.norm
        kr = ref.rotate(kv[:, self.rank:], pos, self.rotation())
        q = q.reshape(n, H, -1)
        q = np.concatenate([q[..., :self.dim], ref.rotate(q[..., self.dim:], pos, self.rotation())], -1)
        sink = self.sink.astype(np.float64) if self.sink is not None else np.full(H, -1e9)
        y = ref.latent_attend(q, c, kr, self.uk.v, self.uv.v, self.scale, window or self.window, sink)
        return (y * ref.output_gate(z)[:, :, None] if self.gated else y).reshape(n, -1)

    def run(self, be, q, kv, z, pos, slab=None, window=None):
        """kv None: the rows are in the slab"""
        import inferred_hip as ih
        n = q.shape[0]
        q, z = np.ascontiguousarray(q).reshape(-1).copy(), np.ascontiguousarray(z).reshape(-1)
        kv = None if kv is None else np.ascontiguousarray(kv).reshape(-1)
        out = np.zeros(n * self.heads * self.vdim, np.float32)
        slab = self.slab if slab is None else slab
        sc = self.scaling or (0.0, 0.0, 0.0, 0.0)
        a = ih.AttnLatent(q=q.ctypes.data, q_len=q.size, slab=slab.ctypes.data, slab_len=slab.size, uk=self.uk.w, uv=self.uv.w, heads=self.heads,
                          dim=self.dim, rot_dim=self.rot, vdim=self.vdim, rank=self.rank, pos=pos, window=window or self.window or 0, scale=self.scale,
                          eps=self.eps, rope=ih.Rope(40.0, self.n_rot, *sc))
        if kv is not None:
            a.kv, a.kv_len, a.kv_norm = kv.ctypes.data, kv.size, self.norm.ctypes.data
        if self.sink is not None:
            a.sinks = self.sink.ctypes.data
        if self.gated:
            a.gate, a.gate_len = z.ctypes.data, z.size
        be.attend_latent(a, out)
        _held.append((q, kv, z, out, self))
        if n > 16 and be.name == "default":
            got = read_rows(be, out, n, self.heads * self.vdim)
        else:
            be.host_needs(out)
            got = out.reshape(n, -1)
        got = got.copy()
        for b in (q, z, out) + (() if kv is None else (kv,)):
            be.release(b)
        return got

    def pieces(self, be, x, sizes, **kw):
        at, got = 0, []
        for s in sizes:
            got.append(self.run(be, *[a[at:at + s] for a in x], at, **kw))
            at += s
        return np.concatenate(got)


LATENTS = [(3, 24, 8, 40, 48, None), (6, 40, 16, 24, 96, 70), (2, 9, 6, 11, 21, 5), (40, 16, 24, 8, 136, 33), (2, 250, 16, 24, 264, 40), (4, 128, 64, 96, 512, 100),
           (3, 16, 8, 264, 40, 64), (1, 8, 32, 16, 700, None), (33, 8, 2, 8, 8, 1)]


def near(be):
    return 2e-5 if be.f32 else 1e-2 if be.name == "steps" else 2.5e-2   # (16-bit cache rows; 16-bit operands)


@pytest.mark.parametrize("shape", LATENTS)
@pytest.mark.parametrize("sizes", [[1, 1, 2], [16, 1, 3], [17], [130, 1, 2, 17, 40], [64, 65, 1], [200]])
def test_latent_attention_in_pieces(be, shape, sizes):
    r = rng(shape[0] * 100 + sum(sizes))
    m = LatentLayer(r, *shape, sum(sizes) + 3, be.f32)
    x = m.inputs(r, sum(sizes))
    assert rel(m.pieces(be, x, sizes), m.oracle(*x)) < near(be)
    be.release(m.slab)


@pytest.mark.parametrize("kw", [dict(n_rot=4), dict(scaling=(4.0, 30, 8.0, 0.5)), dict(scaling=(2.0, 4000, 1.0, 0.9)), dict(sink=False), dict(gate=False), dict(ty="f32"),
                                dict(ty="f16"), dict(n_rot=0)])
def test_each_part_of_latent_attention_alone(be, kw):
    r = rng(17)
    m = LatentLayer(r, 3, 16, 12, 24, 40, 50, 100, be.f32, **kw)
    x = m.inputs(r, 90)
    assert rel(m.pieces(be, x, [30, 1, 5, 54]), m.oracle(*x)) < near(be)
    be.release(m.slab)


@pytest.mark.parametrize("sizes", [[40, 1, 2, 30, 7], [80]])
def test_rows_of_another_layer(be, sizes):
    """A second layer over the first one's rows, with matrices and a wider window of its own; the rows stay as they are."""
    r = rng(4)
    a, b = LatentLayer(r, 3, 16, 8, 24, 40, 6, 90, be.f32), LatentLayer(r, 5, 8, 8, 16, 40, 31, 90, be.f32)
    x, (q, _, z) = a.inputs(r, 80), b.inputs(r, 80)
    b.norm = a.norm
    at, first, second = 0, [], []
    for s in sizes:
        first.append(a.run(be, *[v[at:at + s] for v in x], at))
        second.append(b.run(be, q[at:at + s], None, z[at:at + s], at, slab=a.slab))
        at += s
    assert rel(np.concatenate(first), a.oracle(*x)) < near(be)
    assert rel(np.concatenate(second), b.oracle(q, x[1], z)) < near(be)
    be.release(a.slab)


@pytest.mark.parametrize("window", [1, 2, 16, 63, 64, 65, 128, 200])
@pytest.mark.parametrize("n", [1, 7, 33])
def test_a_key_just_inside_and_just_outside_the_window(be, window, n):
    """One key whose score stands out, its value another than all others': seen up to window - 1 tokens back, and not a token
    further.  The last n of 300 tokens ask, so some see it and some do not."""
    r = rng(window)
    m = LatentLayer(r, 2, 8, 4, 8, 16, window, 300, be.f32, sink=False, gate=False)
    m.norm[:] = 1.0
    for w in (m.uk, m.uv):
        w.raw[:], w.v[:] = 0, 0.0
    for h in range(2):                            # unrotated key channel 0 reads latent channel 3, value 2 and 5 read channels 6 and 3
        for w, j, k, v in ((m.uk, h * 8, 3, 1.0), (m.uv, h * 8 + 2, 6, 1.0), (m.uv, h * 8 + 5, 3, 1.0)):
            w.raw[j, k], w.v[j, k] = np.float32(v).view(np.uint32) >> 16, v
    m.scale = 4.0
    q, kv, z = (np.zeros_like(a) for a in m.inputs(r, 300))
    q.reshape(300, 2, 12)[:, :, 0] = 4.0
    kv[:, 6] = 1.0
    for far in {max(0, 300 - window - n // 2), 300 - window, max(0, 300 - window - 1), max(0, 301 - window - n)}:
        if far >= 300:
            continue
        k2 = kv.copy()
        k2[far], k2[far, 3] = 0.0, 1.0
        want = m.oracle(q, k2, z)[-n:]
        got = m.pieces(be, (q, k2, z), [300 - n, n])[-n:]
        i = np.arange(300 - n, 300)
        inside = (i - far >= 0) & (i - far < window)
        assert (want[inside][:, 5] > 3.9).all() and (want[~inside][:, 5] == 0).all()      # (4: one of sixteen channels, normed)
        assert np.allclose(got, want, rtol=1e-2, atol=1e-2)
    be.release(m.slab)


@pytest.mark.parametrize("n", [1, 18])
@pytest.mark.parametrize("level", [-20.0, -6.0, 0.0, 30.0])
def test_a_sink_per_head_against_scores_below_and_above_it(be, n, level):
    """Equal keys: head h's output is m e^level / (e^sink_h + m e^level) of the value, to relative precision also where it is tiny."""
    r = rng(3)
    m = LatentLayer(r, 3, 8, 2, 8, 16, None, 70, be.f32, gate=False)
    m.sink[:] = [-9.0, 0.0, 11.0]
    q, kv, z = m.inputs(r, 70)
    kv[:] = np.abs(kv[0])
    kv[:, 16:] = 0
    q[:] = 0
    key = (ref.rms(kv[:1, :16].astype(np.float64), m.eps) * m.norm) @ m.uk.v.T
    for h in range(3):
        k0 = key[0, h * 8:h * 8 + 8]
        q.reshape(70, 3, 10)[:, h, :8] = level / m.scale * k0 / (k0 @ k0)
    want = m.oracle(q, kv, z)[-n:]
    got = m.pieces(be, (q, kv, z), [70 - n, n])[-n:]
    share = 70 * np.exp(level) / (np.exp(m.sink.astype(np.float64)) + 70 * np.exp(level))
    assert np.allclose(want[-1].reshape(3, 8)[:, 0] / m.oracle(q, kv, z)[-1].reshape(3, 8)[:, 0], 1)
    v = ((ref.rms(kv[:1, :16].astype(np.float64), m.eps) * m.norm) @ m.uv.v.T).reshape(3, 8)
    assert np.allclose(want[-1].reshape(3, 8), v * share[:, None], rtol=1e-6)
    assert np.allclose(got, want, rtol=2e-4 if be.f32 else 4e-2, atol=(1e-6 if be.f32 else 4e-3) * np.abs(want).max())
    be.release(m.slab)


def test_latent_operands_that_do_not_fit_are_refused():
    import inferred_hip as ih
    b = ih.Hip()
    b.name = "default"
    r = rng(0)
    m = LatentLayer(r, 2, 8, 4, 8, 16, None, 10, False)
    x = m.inputs(r, 5)
    for change, text in [(lambda: m.run(b, *x, 6), "past the end of the slab"), (lambda: m.run(b, x[0], x[1][:4], x[2], 0), "kv.len()"),
                         (lambda: m.run(b, x[0], x[1], x[2][:4], 0), "gate.len()"), (lambda: setattr(m, "n_rot", 3) or m.run(b, *x, 0), "must be even")]:
        change()
        assert text in (b.take_error() or "")
    g = Recurrence(r, 1, 8, 8, 2, 1.0)
    q, k, v, low = g.inputs(r, 3)
    for args, text in [((q, k[:2], v, low), "another size"), ((q, k, v, low[:1]), "another size")]:
        g.run(b, *args)
        assert text in (b.take_error() or "")
    y = np.zeros(8, np.float32)
    b.add_normed(y, 8, addition(np.zeros(8, np.float32), y, y, 0.0, 1.0))
    assert "in place" in (b.take_error() or "")
    b.close()


# ---------------------------------------------------------------- windows and sinks of biased attention
@pytest.mark.parametrize("window", [1, 5, 64, 65, 200])
@pytest.mark.parametrize("n, m", [(1, 64), (1, 300), (9, 130), (17, 17), (70, 200), (130, 300)])
def test_biased_attention_with_a_window_and_sinks(be, window, n, m):
    import inferred_hip as ih
    r = rng(window + n * m)
    H, G, d, dv = 6, 2, 24, 40
    q, k, v = (f16(r.standard_normal(s)) for s in ((n, H, d), (m, G, d), (m, G, dv)))
    sinks, slopes = r.standard_normal(H).astype(np.float32), np.array([0.3, 0.01, 0.1, 0.02, 0.0, 0.5], np.float32)
    ty = np.float32 if be.f32 else np.float16
    ks, vs = np.full((m + 9, G, d), np.nan, ty), np.full((m + 9, G, dv), np.nan, ty)
    ks[:m], vs[:m] = k, v
    qs, out = np.ascontiguousarray(q, np.float32), np.zeros(n * H * dv, np.float32)
    a = ih.AttnBias(q=qs.ctypes.data, q_len=qs.size, k=ks.ctypes.data, v=vs.ctypes.data, k_len=ks.size, v_len=vs.size, n_pos=m, k_dim=d, v_dim=dv, k_stride=d,
                    v_stride=dv, n_head=H, n_head_kv=G, scale=0.25, sink=1, slopes=slopes.ctypes.data, temp_coef=0.0, temp_every=1,
                    sinks=sinks.ctypes.data, window=window)
    _held.append((qs, ks, vs, sinks, slopes, out))
    be.attend_bias(a, out)
    got = read_rows(be, out, n, H * dv) if n > 16 and be.name == "default" else None
    if got is None:
        be.host_needs(out)
        got = out
    dist = np.arange(m - n, m)[:, None] - np.arange(m)[None, :]
    want = np.zeros((n, H, dv))
    for h in range(H):
        s = q[:, h] @ k[:, h // 3].T * 0.25 - slopes[h] * dist
        want[:, h] = ref.sink_softmax(np.where(ref.visible(n, m, window), s, -np.inf), float(sinks[h])) @ v[:, h // 3]
    assert rel(got.reshape(n, H, dv), want) < (1e-5 if be.name != "default" else 1e-2)
    for b in (qs, ks, vs, out):
        be.release(b)
