"""The seam ops of models with unquantized matrices, each against the plain oracle (serisun_ref.py): groups of products
behind a norm, residual sums, biased attention with a sink, the Mamba-2 mixer.  Three backends: the default (bf16 matrix
cores for batches), 32-bit mode, and one launch per operation."""
import ctypes as C

import numpy as np
import pytest

import serisun_ref as ref
from util import bf16_round, rng

pytestmark = pytest.mark.gpu

MODES = {"default": {}, "f32": {"f32": True}, "steps": {"fuse": False}}


@pytest.fixture(params=sorted(MODES))
def be(request):
    import inferred_hip as ih
    b = ih.Hip(**MODES[request.param])
    b.name = request.param
    yield b
    err = b.take_error()
    b.close()
    assert err is None, err


class Mat:
    """A matrix in one of the stored types, with its values as float64."""

    def __init__(self, r, n_out, n_in, ty="bf16", scale=None):
        import inferred_hip as ih
        v = (r.standard_normal((n_out, n_in)) * (scale or n_in ** -0.5)).astype(np.float32)
        if ty == "bf16":
            v = bf16_round(v)
            self.raw, code = np.ascontiguousarray(v.view(np.uint32) >> 16, np.uint32).astype(np.uint16), ih.BF16
        elif ty == "f16":
            self.raw, code = v.astype(np.float16), ih.F16
            v = self.raw.astype(np.float32)
        else:
            self.raw, code = v, ih.F32
        self.v = v.astype(np.float64)
        self.w = ih.weights(self.raw, code, n_in, n_out)


def group_mat(m, out=None, up=None, scale=1.0, slab=None, slab_elems=0, row=0, head_dim=0, stride=0):
    import inferred_hip as ih
    g = ih.GroupMat(w=m.w, scale=scale)
    if up is not None:
        g.up = up.w
    if slab is not None:
        g.slab, g.slab_len, g.slab_row, g.head_dim, g.head_stride = slab.ctypes.data, slab_elems, row, head_dim, stride
    else:
        g.out, g.out_len = out.ctypes.data, out.size
    return g


def res_term(m, inp, scale=None, norm=None, groups=1, eps=1e-5):
    import inferred_hip as ih
    t = ih.ResTerm(w=m.w, inp=inp.ctypes.data, in_len=inp.size, norm_groups=groups, eps=eps)
    if scale is not None:
        t.scale = scale.ctypes.data
    if norm is not None:
        t.norm_w = norm.ctypes.data
    return t


_held = []


def read_rows(be, buf, n, width):
    """The rows an op left in `buf`, through a product with the identity: it reads the bf16 form where a batch op left one."""
    r = rng(0)
    eye = Mat(r, width, width)
    eye.raw = np.ascontiguousarray((np.eye(width, dtype=np.float32).view(np.uint32) >> 16).astype(np.uint16))
    import inferred_hip as ih
    eye.w = ih.weights(eye.raw, ih.BF16, width, width)
    x = np.zeros(n * width, np.float32)
    _held.append((eye, x))   # device copies are keyed on these addresses
    be.host_wrote(x)
    be.matmul_residual(x, [res_term(eye, buf)])
    be.host_needs(x)
    return x.reshape(n, width)


def rel(a, b):
    """Largest error relative to the value itself plus the root mean square of all of them."""
    b = np.asarray(b, np.float64)
    return float((np.abs(np.asarray(a, np.float64) - b) / (np.abs(b) + np.sqrt((b * b).mean()))).max())


def tolerance(be, n):
    return 2.5e-2 if be.name == "default" and n > 16 else 2e-5   # bf16 operands: the largest error of many outputs


TOKENS = [1, 2, 5, 9, 16, 17, 63, 130, 257]


@pytest.mark.parametrize("n_in, n_outs", [(64, (48, 130, 7)), (37, (21, 5)), (200, (129, 64, 1)), (520, (300,)), (1032, (96, 40))])
@pytest.mark.parametrize("n", TOKENS)
def test_group_of_products_behind_a_norm(be, n, n_in, n_outs):
    r = rng(n * 1000 + n_in)
    x, nw = r.standard_normal(n * n_in).astype(np.float32), (1 + 0.3 * r.standard_normal(n_in)).astype(np.float32)
    mats = [Mat(r, o, n_in) for o in n_outs]
    outs = [np.zeros(n * o, np.float32) for o in n_outs]
    scales = [1.0, 0.25, 3.0][:len(mats)]
    be.norm_matmuls(x, nw, n_in, 1e-4, [group_mat(m, o, scale=s) for m, o, s in zip(mats, outs, scales)])
    h = ref.rms(x.reshape(n, n_in).astype(np.float64), 1e-4) * nw
    for m, o, s in zip(mats, outs, scales):
        be.host_needs(o)
        assert rel(o.reshape(n, -1), h @ m.v.T * s) < tolerance(be, n)


@pytest.mark.parametrize("ty", ["f16", "f32"])
@pytest.mark.parametrize("n, n_in", [(1, 96), (1, 41), (4, 96), (40, 96), (40, 41)])
def test_other_matrix_types_stay_32_bit(be, ty, n, n_in):
    r = rng(n + n_in)
    x = r.standard_normal(n * n_in).astype(np.float32)
    m, o = Mat(r, 50, n_in, ty), np.zeros(n * 50, np.float32)
    be.norm_matmuls(x, None, n_in, 0.0, [group_mat(m, o)])
    be.host_needs(o)
    assert rel(o.reshape(n, -1), x.reshape(n, n_in) @ m.v.T) < 2e-5


@pytest.mark.parametrize("n_in, ff", [(64, 96), (37, 21), (136, 130)])
@pytest.mark.parametrize("n", TOKENS)
def test_gated_pair_and_slab_rows(be, n, n_in, ff):
    """silu(gate) * up beside a matrix whose rows go to a cache slab, some rows in, heads padded apart."""
    r = rng(n * 7 + ff)
    x, nw = r.standard_normal(n * n_in).astype(np.float32), np.ones(n_in, np.float32)
    gate, up, kv = Mat(r, ff, n_in), Mat(r, ff, n_in), Mat(r, 3 * 10, n_in)
    out = np.zeros(n * ff, np.float32)
    row, start, cap = 3 * 16, 5, n + 9
    slab = np.full(cap * row, 7.0, np.float32 if be.f32 else np.float16)
    be.norm_matmuls(x, nw, n_in, 1e-5, [group_mat(kv, slab=slab, slab_elems=slab.size, row=start, head_dim=10, stride=16), group_mat(gate, out, up=up)])
    h = ref.rms(x.reshape(n, n_in).astype(np.float64), 1e-5)
    assert rel(read_rows(be, out, n, ff), ref.silu(h @ gate.v.T) * (h @ up.v.T)) < (3e-2 if be.name == "default" and n > 16 else 1e-2 if n > 16 and not be.f32 else 2e-5)
    words = slab.view(np.uint16)
    be.L.it_hip_read_kv(be.h, words.ctypes.data, words.size)
    got = slab.reshape(cap, 3, 16).astype(np.float64)
    assert rel(got[start:start + n, :, :10].reshape(n, 30), h @ kv.v.T) < (2.5e-2 if be.name == "default" and n > 16 else 2e-3 if not be.f32 else 2e-5)
    assert (got[:start] == 7).all() and (got[start + n:] == 7).all() and (got[start:start + n, :, 10:] == 7).all()


@pytest.mark.parametrize("nd, ins, groups", [(64, (48, 96), 3), (37, (21, 14), 7), (130, (520, 64), 1), (96, (200,), 4)])
@pytest.mark.parametrize("n", TOKENS)
def test_residual_sum_with_a_group_norm(be, n, nd, ins, groups):
    r = rng(n * 31 + nd)
    x = r.standard_normal(n * nd).astype(np.float32)
    want = x.reshape(n, nd).astype(np.float64)
    terms, keep = [], []
    for k, w in enumerate(ins):
        m, a, s = Mat(r, nd, w), r.standard_normal(n * w).astype(np.float32), r.standard_normal(nd).astype(np.float32)
        g = (1 + 0.3 * r.standard_normal(w)).astype(np.float32) if k == 0 else None
        keep.append((m, a, s, g))
        terms.append(res_term(m, a, s, g, groups, 1e-3))
        v = a.reshape(n, w).astype(np.float64)
        if g is not None:
            v = ref.rms(v.reshape(n, groups, w // groups), 1e-3).reshape(n, w) * g
        want = want + (v @ m.v.T) * s
    be.host_wrote(x)
    be.matmul_residual(x, terms)
    be.host_needs(x)
    assert rel(x.reshape(n, nd), want) < tolerance(be, n)


# ---------------------------------------------------------------- attention
def run_attention(be, q, k, v, scale, slopes, sink, coef, every, cap):
    """q [n, H, d], k [m, G, d], v [m, G, dv] through slabs of `cap` rows; -> [n, H, dv]"""
    import inferred_hip as ih
    n, H, d = q.shape
    m, G, dv = v.shape
    ks, vs = (d + 7) // 8 * 8, (dv + 7) // 8 * 8
    ty = np.float32 if be.f32 else np.float16
    kslab, vslab = np.zeros((cap, G, ks), ty), np.zeros((cap, G, vs), ty)
    kslab[:m, :, :d], vslab[:m, :, :dv] = k, v
    kslab[m:], vslab[m:] = np.nan, np.nan          # rows past the context must not reach any result
    q = np.ascontiguousarray(q, np.float32)
    sl = None if slopes is None else np.ascontiguousarray(slopes, np.float32)
    out = np.zeros(n * H * dv, np.float32)
    _held.append((q, kslab, vslab, sl, out))
    a = ih.AttnBias(q=q.ctypes.data, q_len=q.size, k=kslab.ctypes.data, v=vslab.ctypes.data, k_len=kslab.size, v_len=vslab.size, n_pos=m,
                    k_dim=d, v_dim=dv, k_stride=ks, v_stride=vs, n_head=H, n_head_kv=G, scale=scale, sink=sink,
                    slopes=None if sl is None else sl.ctypes.data, temp_coef=coef, temp_every=every)
    be.attend_bias(a, out)
    got = read_rows(be, out, n, H * dv) if n > 16 and be.name == "default" else None
    if got is None:
        be.host_needs(out)
        got = out
    got = got.reshape(n, H, dv).copy()
    for b in (q, kslab, vslab, out):
        be.release(b)
    return got


def f16(a):
    return a.astype(np.float16).astype(np.float64)


def expected_attention(q, k, v, scale, slopes, sink, coef, every):
    n, m = q.shape[0], k.shape[0]
    t = ref.query_temperature(m, coef, every)[m - n:] if coef else np.ones(n)
    return ref.attend(q * t[:, None, None], k, v, scale, np.zeros(q.shape[1]) if slopes is None else slopes, sink=bool(sink))


HEADS = [(10, 1, 96, 88), (6, 2, 24, 40), (4, 4, 11, 13), (3, 1, 136, 72), (40, 1, 64, 32), (5, 5, 264, 24), (12, 4, 192, 200)]


@pytest.mark.parametrize("H, G, d, dv", HEADS)
@pytest.mark.parametrize("n, m", [(1, 1), (1, 63), (1, 64), (1, 65), (1, 300), (2, 2), (3, 130), (16, 200), (17, 17), (65, 128), (40, 300), (129, 129)])
def test_biased_attention(be, H, G, d, dv, n, m):
    r = rng(H * 1000 + n * m)
    q, k, v = (f16(r.standard_normal(s) * c) for s, c in (((n, H, d), 2.0), ((m, G, d), 1.0), ((m, G, dv), 1.0)))
    slopes = ref.head_slopes(H)
    got = run_attention(be, q, k, v, d ** -0.5, slopes, 1, 0.3, 50, m + 70)
    want = expected_attention(q, k, v, d ** -0.5, slopes, 1, 0.3, 50)
    assert rel(got, want) < (1e-5 if be.name != "default" else 1e-2 if n > 16 else 1e-5 if max(d, dv) > 256 else 6e-3)


@pytest.mark.parametrize("n, m", [(1, 200), (20, 200)])
@pytest.mark.parametrize("slopes, sink, coef", [(None, 0, 0.0), (None, 1, 0.0), ("some", 0, 0.0), (None, 0, 0.7)])
def test_each_term_of_the_attention_alone(be, n, m, slopes, sink, coef):
    r = rng(9)
    H, G, d, dv = 4, 2, 32, 24
    q, k, v = f16(r.standard_normal((n, H, d))), f16(r.standard_normal((m, G, d))), f16(r.standard_normal((m, G, dv)))
    sl = np.array([0.5, 0.03, 0.2, 0.001]) if slopes else None
    got = run_attention(be, q, k, v, 0.3, sl, sink, coef, 13, m)
    assert rel(got, expected_attention(q, k, v, 0.3, sl, sink, coef, 13)) < (1e-5 if be.name != "default" else 2e-2)


@pytest.mark.parametrize("far", [0, 1, 63, 64, 65, 127, 128, 255, 256, 399])
@pytest.mark.parametrize("n", [1, 33])
def test_one_key_far_away_stands_out(be, n, far):
    """Every key is orthogonal to the queries but one, whose score beats its distance: the output is that key's value, at
    every tile's and split's edge; a key one position off would be another value altogether."""
    H, G, d, dv, m = 8, 2, 16, 16, 400
    q, k = np.zeros((n, H, d)), np.zeros((m, G, d))
    q[:, :, 3] = 8.0
    k[:, :, 5] = 1.0
    v = np.zeros((m, G, dv))
    v[:, :, 0] = np.arange(m)[:, None] / 64.0
    v[:, :, 1] = 1.0
    k[far, :, 3] = 32.0
    slopes = ref.head_slopes(H)
    got = run_attention(be, q, k, v, 1.0, slopes, 1, 0.0, 1, m + 3)
    want = expected_attention(q, k, v, 1.0, slopes, 1, 0.0, 1)
    i = np.arange(m - n, m)
    seen = i >= far
    assert np.allclose(want[seen][:, :, 0], far / 64.0, atol=1e-6)   # (256 less at most 200: it stands out at any distance)
    assert np.allclose(got, want, rtol=5e-3, atol=1e-3)
    if not seen.all():   # a future key is not seen at all
        assert np.abs(got[~seen][:, :, 0] - far / 64.0).min() > 1e-2 or far == m - 1


@pytest.mark.parametrize("n", [1, 18])
@pytest.mark.parametrize("level", [-30.0, -12.0, 0.0, 9.0, 40.0])
def test_the_sink_against_scores_far_below_and_above_it(be, n, level):
    """All scores equal: the output is m e^level / (1 + m e^level) of the mean value, to relative precision also where it is tiny."""
    H, G, d, dv, m = 2, 1, 8, 8, 70
    r = rng(3)
    q, k, v = np.zeros((n, H, d)), np.zeros((m, G, d)), f16(1 + 0.1 * r.standard_normal((m, G, dv)))
    q[:, :, 0], k[:, :, 0] = level, 1.0
    got = run_attention(be, q, k, v, 1.0, None, 1, 0.0, 1, m)
    want = expected_attention(q, k, v, 1.0, None, 1, 0.0, 1)
    assert np.allclose(got, want, rtol=5e-3 if be.name == "default" else 2e-5, atol=0)


def test_the_temperature_steps_at_its_edges(be):
    """Positions just below and at a multiple of `every`."""
    H, d = 1, 8
    for every in (1, 4, 64):
        for m in (every - 1, every, every + 1, 3 * every - 1, 3 * every):
            if m < 1:
                continue
            q, k, v = np.zeros((1, H, d)), np.zeros((m, 1, d)), np.zeros((m, 1, d))
            q[..., 0], k[..., 0], v[..., 0] = 1.0, 1.0, 1.0
            got = run_attention(be, q, k, v, -3.0, None, 1, 0.5, every, m)
            assert np.allclose(got, expected_attention(q, k, v, -3.0, None, 1, 0.5, every), rtol=3e-3, atol=0)


# ---------------------------------------------------------------- Mamba-2
class Mixer:
    def __init__(self, r, heads, vdim, n, groups, taps, fast_decay=False):
        self.heads, self.vdim, self.n, self.groups, self.taps = heads, vdim, n, groups, taps
        self.inner = heads * vdim
        self.ch = self.inner + 2 * groups * n
        self.ud = self.inner + self.ch + heads
        f = lambda *s: r.standard_normal(s).astype(np.float32)
        self.conv_w, self.conv_b = 0.6 * f(self.ch, taps), 0.3 * f(self.ch)
        self.dt_bias, self.a_log, self.d = f(heads) - (0 if fast_decay else 2), f(heads) + (2.5 if fast_decay else -0.5), f(heads)
        for name in ("conv_w", "conv_b", "dt_bias", "a_log", "d"):
            setattr(self, name, np.ascontiguousarray(getattr(self, name), np.float32))
        self.fresh()

    def fresh(self):
        self.ring, self.state = np.zeros(self.taps * self.ch, np.float32), np.zeros(self.inner * self.n, np.float32)

    def oracle(self, u):
        n = u.shape[0]
        u = u.astype(np.float64)
        z, raw, dt = u[:, :self.inner], u[:, self.inner:self.inner + self.ch], u[:, self.inner + self.ch:]
        c = ref.causal_conv_silu(raw, self.conv_w.astype(np.float64), self.conv_b)
        x = c[:, :self.inner].reshape(n, self.heads, self.vdim)
        B = c[:, self.inner:self.inner + self.groups * self.n].reshape(n, self.groups, self.n)
        Cc = c[:, self.inner + self.groups * self.n:].reshape(n, self.groups, self.n)
        y, S = ref.state_space(x, B, Cc, ref.softplus(dt + self.dt_bias), self.a_log.astype(np.float64), self.d)
        return y.reshape(n, self.inner) * ref.silu(z), S.transpose(0, 2, 1)

    def run(self, be, u, pos):
        import inferred_hip as ih
        u = np.ascontiguousarray(u, np.float32)
        out = np.zeros(u.shape[0] * self.inner, np.float32)
        a = ih.Mamba2(self.conv_w.ctypes.data, self.conv_b.ctypes.data, self.dt_bias.ctypes.data, self.a_log.ctypes.data, self.d.ctypes.data,
                      self.heads, self.vdim, self.n, self.groups, self.taps, pos)
        be.mamba2(a, u.reshape(-1), self.ring, self.state, out)
        be.host_needs(out)
        be.release(u)
        be.release(out)
        return out.reshape(-1, self.inner).copy()

    def read_state(self, be):
        be.read_state(self.state)
        return self.state.reshape(self.heads, self.vdim, self.n).copy()


MIXERS = [(5, 24, 40, 1, 3), (4, 16, 24, 2, 4), (3, 7, 5, 3, 1), (2, 80, 144, 1, 5), (4, 10, 19, 1, 2), (2, 64, 128, 2, 4), (1, 24, 300, 1, 16)]


@pytest.mark.parametrize("shape", MIXERS)
@pytest.mark.parametrize("pieces", [[1] * 9, [2, 3, 2, 1, 1, 2], [63], [64], [65, 1, 1], [130, 2, 64, 1], [17, 200, 3]])
def test_mamba2_in_pieces_against_the_whole(be, shape, pieces):
    """One call or many, alone or behind one another: the same read-outs and the same last state, from a fresh start each."""
    r = rng(sum(pieces) + shape[0])
    m = Mixer(r, *shape)
    for turn in range(2):                         # the second sequence uses the same ring and state again
        u = r.standard_normal((sum(pieces), m.ud)).astype(np.float32)
        want, S = m.oracle(u)
        got, at = [], 0
        for c in pieces:
            got.append(m.run(be, u[at:at + c], at))
            at += c
        tol = 2e-5 if be.name != "default" else 1e-4
        assert rel(np.concatenate(got), want) < tol
        assert rel(m.read_state(be), S) < tol
        m.ring[:], m.state[:] = 0, 0
        for b in (m.ring, m.state):
            be.L.it_hip_zero_slab(be.h, b.ctypes.data)


@pytest.mark.parametrize("n", [70, 200])
def test_mamba2_where_tokens_forget_almost_everything(be, n):
    """Decays down to e^-hundreds beside ones near 1 in the same chunk."""
    r = rng(n)
    m = Mixer(r, 8, 16, 16, 2, 4, fast_decay=True)
    u = r.standard_normal((n, m.ud)).astype(np.float32)
    u[:, -m.heads:] *= 6.0                        # step sizes from 0 to about 20
    want, S = m.oracle(u)
    assert rel(m.run(be, u, 0), want) < 1e-4 and rel(m.read_state(be), S) < 1e-4


def test_mamba2_over_more_chunks_than_are_taken_at_once(be):
    """A state so large that the chunked form takes eight chunks at a time: one call of ten against two calls of fewer."""
    r = rng(2)
    m = Mixer(r, 128, 64, 512, 1, 2)
    u = 0.5 * r.standard_normal((600, m.ud)).astype(np.float32)
    runs = []
    for pieces in ((600,), (300, 300)):
        at, out = 0, []
        for c in pieces:
            out.append(m.run(be, u[at:at + c], at))
            at += c
        runs.append((np.concatenate(out), m.read_state(be)))
        for b in (m.ring, m.state):
            b[:] = 0
            be.L.it_hip_zero_slab(be.h, b.ctypes.data)
    assert rel(runs[0][0], runs[1][0]) < 1e-4 and rel(runs[0][1], runs[1][1]) < 1e-4 and np.abs(runs[0][1]).max() > 0.1


# ---------------------------------------------------------------- the small ones
@pytest.mark.parametrize("ff", [24, 21])
def test_rows_left_in_bf16_are_read_as_f32_where_an_op_needs_them(be, ff):
    """A batch's gated pair, read by the host and by a product of another matrix type."""
    r = rng(ff)
    n, n_in = 40, 32
    x, gate, up = r.standard_normal(n * n_in).astype(np.float32), Mat(r, ff, n_in), Mat(r, ff, n_in)
    down, out, y = Mat(r, 16, ff, "f32"), np.zeros(n * ff, np.float32), np.zeros(n * 16, np.float32)
    be.norm_matmuls(x, None, n_in, 0.0, [group_mat(gate, out, up=up)])
    be.matmul_residual(y, [res_term(down, out)])
    be.host_needs(out)
    be.host_needs(y)
    h = x.reshape(n, n_in).astype(np.float64)
    g = ref.silu(h @ gate.v.T) * (h @ up.v.T)
    assert rel(out.reshape(n, ff), g) < tolerance(be, n) and rel(y.reshape(n, 16), g @ down.v.T) < tolerance(be, n)


def test_add_rows_and_gather_rows(be):
    r = rng(1)
    x, rows, vec = (r.standard_normal(s).astype(np.float32) for s in (5 * 33, 5 * 33, 33))
    want = (x + rows).reshape(5, 33) + vec
    be.add_rows(x, rows, vec)
    be.host_needs(x)
    assert np.allclose(x.reshape(5, 33), want, rtol=1e-6, atol=1e-6)
    be.add_rows(x, None, vec)
    out = np.zeros(3 * 33, np.float32)
    be.gather_rows(x, 33, [4, 0, 2], out)
    be.host_needs(out)
    assert np.allclose(out.reshape(3, 33), (want + vec)[[4, 0, 2]], rtol=1e-6, atol=1e-6)


def test_operands_that_do_not_fit_are_refused():
    import inferred_hip as ih
    b = ih.Hip()
    r = rng(0)
    m, x, o = Mat(r, 8, 16), np.zeros(32, np.float32), np.zeros(16, np.float32)
    slab = np.zeros(64, np.float16)
    for call, text in [
        (lambda: b.norm_matmuls(x, None, 16, 0.0, [group_mat(m, o[:8])]), "out.len"),
        (lambda: b.norm_matmuls(x, None, 32, 0.0, [group_mat(m, o)]), "row length"),
        (lambda: b.norm_matmuls(x, None, 16, 0.0, [group_mat(m, slab=slab, slab_elems=64, row=7, head_dim=4, stride=4)]), "past the end of the slab"),
        (lambda: b.matmul_residual(o, [res_term(m, x[:16])]), "in.len"),
        (lambda: b.attend_bias(ih.AttnBias(q=x.ctypes.data, q_len=32, k=slab.ctypes.data, v=slab.ctypes.data, k_len=64, v_len=64, n_pos=9, k_dim=8, v_dim=8,
                                           k_stride=8, v_stride=8, n_head=1, n_head_kv=1, scale=1.0), np.zeros(32, np.float32)), "outside the slabs"),
        (lambda: b.mamba2(ih.Mamba2(*[x.ctypes.data] * 5, 1, 2, 600, 1, 2, 0), np.zeros(2 + 2 + 1200 + 1, np.float32), np.zeros(2 * 1202, np.float32),
                          np.zeros(1200, np.float32), np.zeros(2, np.float32)), "at most 512 columns"),
    ]:
        call()
        assert text in (b.take_error() or "")
    b.close()
