"""Rows of parallel blocks, grouped-head attention with one or two maps, the gated delta rule and mixture of experts (include/bitnet_hip.h
section 5), one at a time through the C ABI, against the plain restatement in oracle/stack_oracle.py or f64 numpy."""
import numpy as np
import pytest

from oracle import stack_oracle as so
from tests import stack_util as u

pytestmark = pytest.mark.gpu
F32_TOL, BF_TOL = 3e-6, 6e-3


def rng(*seed):
    return np.random.default_rng(list(seed))


def pos_dev(p):
    return u.dev(np.array([p], np.int32))


# ---- rows and vectors of a block ---------------------------------------------------------------------------------------
@pytest.mark.parametrize("n", [80, 90, 1001, 2560, 4096, 5000])
def test_gemv_layer_norm_of_a_plain_residual(hip, pkg, n):
    g = rng(n)
    rows, ld, cols, eps, mult = 90, u.up_to(n, 64), u.up_to(n, 8), 1e-3, 0.37
    w = u.rounded(g.standard_normal((rows, n)) / np.sqrt(n))
    x, y, nw, nb = (g.standard_normal(n).astype(np.float32) for _ in range(4))
    x += 1.5
    out, xo, ho = u.zeros_f32(rows), u.zeros_f32(n), u.zeros_f32(n)
    hip.dense_gemv_dev(u.dev_f32(x), u.dev_bf16(u.padded(w, ld)), rows, cols, ld, out, kind=pkg.IN_RESIDUAL_NORM, eps=eps, weight=u.dev_f32(nw), norm_bias=u.dev_f32(nb),
                       center=True, res=u.dev_f32(y), mult=mult, x_out=xo, h_out=ho, n=n)
    x2 = x.astype(np.float64) + mult * y
    h = so.layer_norm(x2, nw, nb, eps)
    assert u.rms_error(u.host(xo), x2) < F32_TOL and u.rms_error(u.host(ho), h) < F32_TOL
    assert u.rms_error(u.host(out), w @ h) < F32_TOL


@pytest.mark.parametrize("n", [88, 90, 256, 2560, 4500])
def test_gemv_of_two_halves(hip, pkg, n):
    g = rng(n, 1)
    rows, cols, ld = 70, u.up_to(2 * n, 8), u.up_to(2 * n, 64)
    w = u.rounded(g.standard_normal((rows, 2 * n)) / np.sqrt(n))
    x, y, x2 = (g.standard_normal(n).astype(np.float32) for _ in range(3))
    wd = u.dev_bf16(u.padded(w, ld))
    for res in (None, u.dev_f32(y)):
        out = u.zeros_f32(rows)
        hip.dense_gemv_dev(u.dev_f32(x), wd, rows, cols, ld, out, kind=pkg.IN_CONCAT, res=res, mult=-0.6, x2=u.dev_f32(x2), n=n)
        first = x.astype(np.float64) - (0.6 * y if res is not None else 0.0)
        assert u.rms_error(u.host(out), w @ np.concatenate([first, x2])) < F32_TOL


@pytest.mark.parametrize("width", [96, 90, 1000, 2560, 4096, 5000])
@pytest.mark.parametrize("f32", [True, False])
def test_sum_norm_rows(hip, pkg, width, f32):
    g = rng(width, 2)
    m, top, ldh, eps, mult = 5, 3, u.up_to(2 * width, 64), 1e-2, 0.7
    lde = u.up_to(width, 64)
    x, y, x2 = (g.standard_normal((m, width)).astype(np.float32) for _ in range(3))
    e = g.standard_normal((m * top, width)).astype(np.float32)
    e = e if f32 else u.rounded(e)
    slots, sw = g.permutation(m * top).astype(np.int32).reshape(m, top), g.random((m, top)).astype(np.float32)
    nw, nb = g.standard_normal(width).astype(np.float32), g.standard_normal(width).astype(np.float32)
    put = u.dev_f32 if f32 else u.dev_bf16
    keep = [u.dev_f32(y), put(u.padded(e, lde)), u.dev(slots), u.dev_f32(sw), u.dev_f32(nw), u.dev_f32(nb), u.dev_f32(x2)]
    p = [k.data_ptr() for k in keep]
    want = x.astype(np.float64) + mult * (y + np.einsum("mk,mkw->mw", sw.astype(np.float64), e[slots].astype(np.float64)))
    tol = F32_TOL if f32 else BF_TOL
    new = u.zeros_f32 if f32 else u.zeros_bf16

    def run(**kw):
        xd, h = u.dev_f32(x), new(m, ldh) + 3
        r = pkg.SumRows(x=xd.data_ptr(), m=m, width=width, mult=mult, eps=eps, h_f32=f32, h=h.data_ptr(), ldh=ldh, **kw)
        hip.sum_norm_rows_dev(r)
        return u.host(xd), u.host(h)

    experts = dict(y=p[0], ldy=width, expert_rows=p[1], ld_expert=lde, top=top, slots=p[2], slot_weights=p[3])
    xs, h = run(center=1, weight=p[4], bias=p[5], **experts)
    assert u.rms_error(xs, want) < F32_TOL
    assert u.rms_error(h[:, :width], so.layer_norm(want, nw, nb, eps)) < tol and not h[:, width:].any()
    xs, h = run(weight=p[4], weight_offset=1.0, y=p[0], ldy=width)
    assert u.rms_error(h[:, :width], so.norm_around_zero(x + mult * y.astype(np.float64), nw, eps)) < tol
    xs, h = run(x2=p[6], **experts)
    assert u.rms_error(h[:, :2 * width], np.concatenate([want, x2], axis=1)) < tol and not h[:, 2 * width:].any()
    xs, h = run(center=1, weight=p[4], bias=p[5])
    assert np.array_equal(xs, x) and u.rms_error(h[:, :width], so.layer_norm(x.astype(np.float64), nw, nb, eps)) < tol


@pytest.mark.parametrize("width", [96, 90, 2560, 5000])
@pytest.mark.parametrize("f32", [True, False])
def test_sum_norm_rows_behind_experts(hip, pkg, width, f32):
    """the experts' rows and the input of identity experts, normed together ahead of the stream; the next input is the stream itself or its norm,
    and may take the place of the input that the identities hand through"""
    g = rng(width, 3)
    m, top, ldh, eps = 6, 4, u.up_to(width, 64), 1e-2
    x, y = (g.standard_normal((m, width)).astype(np.float32) for _ in range(2))
    e, inp = g.standard_normal((m * top, width)).astype(np.float32), g.standard_normal((m, width)).astype(np.float32)
    put, new, tol = (u.dev_f32, u.zeros_f32, F32_TOL) if f32 else (u.dev_bf16, u.zeros_bf16, BF_TOL)
    if not f32:
        e, inp = u.rounded(e), u.rounded(inp)
    slots, sw = g.permutation(m * top).astype(np.int32).reshape(m, top), g.random((m, top)).astype(np.float32)
    slots[0, 1], slots[1], slots[4, 2:] = -1, -1, -1
    pw, sc, nw = ((1.0 + 0.3 * g.standard_normal(width)).astype(np.float32) for _ in range(3))
    keep = [put(u.padded(e, ldh)), u.dev(slots), u.dev_f32(sw), u.dev_f32(pw), u.dev_f32(sc), u.dev_f32(nw), u.dev_f32(y)]
    p = [k.data_ptr() for k in keep]
    f64 = np.float64

    def summed(through, start):
        out = np.array(start, f64)
        for i in range(m):
            for k in range(top):
                out[i] += f64(sw[i, k]) * (e[slots[i, k]] if slots[i, k] >= 0 else through[i])
        return out

    def run(h, **kw):
        xd = u.dev_f32(x)
        r = pkg.SumRows(x=xd.data_ptr(), m=m, width=width, eps=eps, h_f32=f32, h=h.data_ptr(), ldh=ldh, expert_rows=p[0], ld_expert=ldh, top=top, slots=p[1],
                        slot_weights=p[2], identity=1, **kw)
        hip.sum_norm_rows_dev(r)
        return u.host(xd), u.host(h)

    want = x + so.norm_plain(summed(x, np.zeros((m, width))), pw, eps)
    xs, h = run(new(m, ldh) + 3, post_weight=p[3])
    assert u.rms_error(xs, want) < F32_TOL and u.rms_error(h[:, :width], want) < tol and not h[:, width:].any()
    want = x + sc * so.norm_plain(summed(inp, y), pw, eps)
    h = put(u.padded(inp, ldh))
    xs, h = run(h, post_weight=p[3], scale=p[4], y=p[6], ldy=width, weight=p[5], input=h.data_ptr(), ld_input=ldh)
    assert u.rms_error(xs, want) < F32_TOL and u.rms_error(h[:, :width], so.norm_plain(want, nw, eps)) < tol
    xs, h = run(new(m, ldh), mult=0.6)
    assert u.rms_error(xs, x + 0.6 * summed(x, np.zeros((m, width)))) < F32_TOL


@pytest.mark.parametrize("width", [40, 77, 2560, 4500])
def test_norm_behind_the_embedding(hip, width):
    g = rng(width, 4)
    ld, tokens = u.up_to(width, 64), np.array([5, 0, 11, 11], np.int32)
    table, w = u.rounded(g.standard_normal((12, width))), g.standard_normal(width).astype(np.float32)
    out = u.zeros_f32(3, width)
    hip.embed_norm_bf16_dev(u.dev_bf16(u.padded(table, ld)), ld, u.dev(tokens), u.dev_f32(w), 1e-2, out, 3, width, 12, offset=pos_dev(1), scale=0.3)
    assert u.rms_error(u.host(out), so.norm_plain(0.3 * table[tokens[1:]].astype(np.float64), w, 1e-2)) < F32_TOL


@pytest.mark.parametrize("n", [40, 77, 256, 2560, 4500])
def test_gemv_reads_the_stream_itself(hip, pkg, n):
    g = rng(n, 5)
    rows, ld, cols, eps = 70, u.up_to(n, 64), u.up_to(n, 8), 1e-2
    w = u.rounded(g.standard_normal((rows, n)) / np.sqrt(n))
    x, y, pw = (g.standard_normal(n).astype(np.float32) for _ in range(3))
    wd = u.dev_bf16(u.padded(w, ld))
    out, xo = u.zeros_f32(rows), u.zeros_f32(n)
    hip.dense_gemv_dev(u.dev_f32(x), wd, rows, cols, ld, out, kind=pkg.IN_RESIDUAL, eps=eps, res=u.dev_f32(y), post_weight=u.dev_f32(pw), x_out=xo, n=n)
    want = x + so.norm_plain(y.astype(np.float64), pw, eps)
    assert u.rms_error(u.host(xo), want) < F32_TOL and u.rms_error(u.host(out), w @ want) < F32_TOL
    hip.dense_gemv_dev(u.dev_f32(x), wd, rows, cols, ld, out, kind=pkg.IN_RESIDUAL, n=n)
    assert u.rms_error(u.host(out), w @ x.astype(np.float64)) < F32_TOL


ACTS = {"ACT_GELU_TANH": so.gelu_tanh, "ACT_SILU": so.silu, "ACT_RELU2": so.relu_squared}


@pytest.mark.parametrize("act", list(ACTS))
@pytest.mark.parametrize("rows,cols", [(1, 40), (7, 64), (33, 200), (300, 2560), (3000, 520), (9000, 2048)])
def test_gemv_of_gated_pairs(hip, pkg, rows, cols, act):
    g = rng(rows, cols)
    ld = u.up_to(cols, 64)
    w = u.rounded(2.0 * g.standard_normal((2 * rows, cols)) / np.sqrt(cols))
    x, bias = g.standard_normal(cols).astype(np.float32), g.standard_normal(2 * rows).astype(np.float32)
    out = u.zeros_f32(rows + 1) + 7
    hip.dense_gemv_dev(u.dev_f32(x), u.dev_bf16(u.padded(w, ld)), 2 * rows, cols, ld, out, bias=u.dev_f32(bias), act0=getattr(pkg, act) | pkg.ACT_GATED)
    z, got = w @ x.astype(np.float64) + bias, u.host(out)
    assert u.rms_error(got[:rows], ACTS[act](z[0::2]) * z[1::2]) < F32_TOL and got[rows] == 7


@pytest.mark.parametrize("act", list(ACTS))
@pytest.mark.parametrize("m,n,k", [(1, 1, 64), (5, 35, 128), (70, 64, 192), (130, 333, 64), (2100, 1100, 1088), (4096, 2816, 1152), (300, 9000, 2048)])
@pytest.mark.parametrize("f32", [True, False])
def test_matmul_of_gated_pairs(hip, pkg, m, n, k, f32, act):
    """every tile form (64, 128, 256 columns), ragged ends; the padding behind a row of the output stays"""
    if f32 and m * n * k > 1 << 28:
        m = 150
    g = rng(m, n, k)
    w = u.rounded(2.0 * g.standard_normal((2 * n, k), np.float32) / np.sqrt(k))
    x = g.standard_normal((m, k), np.float32)
    x = x if f32 else u.rounded(x)
    ldc = u.up_to(n + 1, 64)
    out = (u.zeros_f32 if f32 else u.zeros_bf16)(m, ldc)
    out[:, n:] = 3
    hip.dense_matmul_dev((u.dev_f32 if f32 else u.dev_bf16)(x), k, f32, u.dev_bf16(w), k, m, 2 * n, k, out, ldc, f32, act0=getattr(pkg, act) | pkg.ACT_GATED)
    some = np.unique(np.r_[0, m // 3, m // 2, m - 1, g.integers(0, m, 60)])
    z = x[some].astype(np.float64) @ w.T.astype(np.float64)
    assert u.rms_error(u.host(out)[some, :n], ACTS[act](z[:, 0::2]) * z[:, 1::2]) < (F32_TOL if f32 else 4e-3)
    assert bool((out[:, n:] == 3).all())


@pytest.mark.parametrize("f32", [True, False])
def test_matmul_gelu(hip, pkg, f32):
    g = rng(6)
    x, w = u.rounded(g.standard_normal((90, 128))), u.rounded(3.0 * g.standard_normal((70, 128)) / np.sqrt(128))
    z = x.astype(np.float64) @ w.T
    out = u.zeros_f32(90, 70)
    for split in (0, 33):
        hip.dense_matmul_dev((u.dev_f32 if f32 else u.dev_bf16)(x), 128, f32, u.dev_bf16(w), 128, 90, 70, 128, out, 70, True, act0=pkg.ACT_GELU_TANH, act1=pkg.ACT_NONE, act_split=split)
        want = np.where(np.arange(70) < (split or 70), so.gelu_tanh(z), z)
        assert u.rms_error(u.host(out), want) < (F32_TOL if f32 else 2e-5)


# ---- attention ---------------------------------------------------------------------------------------------------------
class Attention:
    """random projections of n tokens in the library's layout, and the attention's output by definition"""

    def __init__(self, pkg, n, heads, kv, dim, vdim, maps, f32, seed=0):
        g = rng(n, heads, dim, seed)
        self.n, self.heads, self.f32 = n, heads, f32
        self.dimp, self.vdim, self.vdimp, self.cap = u.up_to(dim, 32), vdim, u.up_to(vdim, 32), u.up_to(n, 128)
        store = (lambda a: a.astype(np.float32)) if f32 else u.rounded
        q, k = store(g.standard_normal((n, heads, maps, dim))), store(g.standard_normal((n, kv, maps, dim)))
        v = store(g.standard_normal((n, kv, vdim)))
        self.rows = np.concatenate([u.padded(q, self.dimp).reshape(n, -1), u.padded(k, self.dimp).reshape(n, -1), u.padded(v, self.vdimp).reshape(n, -1)], axis=1)
        self.ld = u.up_to(self.rows.shape[1], 64)
        self.rows = u.padded(self.rows, self.ld)
        qw, kw = (1.0 + 0.3 * g.standard_normal(dim)).astype(np.float32), (1.0 + 0.3 * g.standard_normal(dim)).astype(np.float32)
        factor = (0.6 / np.sqrt(dim) * (1.0 + g.random(self.cap))).astype(np.float32)
        eps, lam, diff = 1e-3, 0.45, 0.35
        f64 = np.float64
        self.q = so.norm_plain(q.astype(f64), qw, eps) * factor[:n, None, None, None]
        self.k, self.v = so.norm_plain(k.astype(f64), kw, eps), v.astype(f64)
        a = so.softmax_maps(self.q, self.k, self.v)
        self.want = so.difference(a, lam, diff, eps) if maps == 2 else a[:, :, 0]
        new = u.zeros_f32 if f32 else u.zeros_bf16
        self.keep = [u.dev_f32(qw), u.dev_f32(kw), u.dev_f32(factor), new(kv, maps, self.cap, self.dimp), new(kv, self.vdimp, self.cap)]
        p = [t.data_ptr() for t in self.keep]
        self.attn = pkg.Gqa(heads, kv, maps, dim, self.dimp, vdim, self.vdimp, self.cap, eps, lam, 1.0 - diff, *p)

    def put(self, a):
        return u.dev_f32(a) if self.f32 else u.dev_bf16(a)

    def new(self, *shape):
        return u.zeros_f32(*shape) if self.f32 else u.zeros_bf16(*shape)

    def fill(self, hip, n0, n1):
        """norms and appends of tokens n0 .. n1 - 1; their prepared rows"""
        rows = self.put(self.rows[n0:n1])
        hip.gqa_rows_dev(self.attn, rows, self.ld, self.f32, self.f32, pos_dev(n0), n1 - n0)
        return rows

    def check(self, got, n0, tol):
        got = u.host(got).reshape(-1, self.heads, self.vdimp)
        assert u.rms_error(got[:, :, :self.vdim], self.want[n0:n0 + len(got)]) < tol
        assert not got[:, :, self.vdim:].any()


SHAPES = [(4, 2, 24, 40, 2), (6, 6, 128, 128, 2), (20, 1, 64, 100, 2), (8, 2, 96, 64, 1), (2, 1, 200, 256, 2), (5, 1, 40, 16, 1), (34, 2, 16, 24, 2)]


class ChunkAttention:
    """as above for heads of one map with everything optional on: rotation, unit norms, chunks, a sink, keys as values and a gate behind them"""

    def __init__(self, pkg, n, heads, kv, dim, rot, chunk, f32, seed=0, own_values=False):
        g = rng(n, heads, dim, chunk, seed)
        self.n, self.heads, self.f32, self.dim = n, heads, f32, dim
        self.dimp = self.vdimp = u.up_to(dim, 32)
        self.vdim, self.cap = dim, u.up_to(n, 128)
        store = (lambda a: a.astype(np.float32)) if f32 else u.rounded
        q, k = store(g.standard_normal((n, heads, dim))), store(g.standard_normal((n, kv, dim)))
        v = store(g.standard_normal((n, kv, dim))) if own_values else k
        gate = store(2.0 * g.standard_normal((n, heads)))
        parts = [u.padded(a, self.dimp).reshape(n, -1) for a in ((q, k, v) if own_values else (q, k))]
        self.gate_at = sum(a.shape[1] for a in parts)
        self.rows = np.concatenate(parts + [gate], axis=1)
        self.ld = u.up_to(self.rows.shape[1], 64)
        self.rows = u.padded(self.rows, self.ld)
        eps, f64 = 1e-3, np.float64
        self.scale = 1.3 / np.sqrt(dim)
        spec = {"dims": rot, "base": 50.0, "scaling": dict(u.BANDS, original=30)}
        self.q, self.k = (so.rms_divide(so.rotate_neighbours(a.astype(f64), spec), eps) for a in (q, k))
        sink = g.standard_normal(heads).astype(np.float32)
        self.want = np.zeros((n, heads, dim))
        for a in range(heads):
            for i in range(n):
                first = i // chunk * chunk if chunk else 0
                s = np.exp(self.k[first:i + 1, a // (heads // kv)] @ self.q[i, a] * self.scale)
                self.want[i, a] = s @ v[first:i + 1, a // (heads // kv)].astype(f64) / (s.sum() + np.exp(f64(sink[a]))) * so.sigmoid(f64(gate[i, a]))
        f = so.banded_frequencies(spec)
        angle = np.arange(self.cap)[:, None] * f
        new = u.zeros_f32 if f32 else u.zeros_bf16
        factor = np.full(self.cap, self.scale, np.float32)
        self.keep = [u.dev_f32(factor), new(kv, self.cap, self.dimp), new(kv, self.vdimp, self.cap), u.dev_f32(np.cos(angle)), u.dev_f32(np.sin(angle)), u.dev_f32(sink)]
        p = [t.data_ptr() for t in self.keep]
        self.attn = pkg.Gqa(heads, kv, 1, dim, self.dimp, dim, self.vdimp, self.cap, eps, 0.0, 1.0, 0, 0, p[0], p[1], p[2], 1, 0 if own_values else 1, rot, chunk, p[3], p[4], p[5])

    put, new, fill, check = Attention.put, Attention.new, Attention.fill, Attention.check

    def gated(self, rows, first=0):
        """the gates are read from these rows"""
        self.attn.gate = rows.data_ptr() + (first * self.ld + self.gate_at) * (4 if rows.element_size() == 4 else 2)
        self.attn.ldgate, self.attn.gate_f32 = self.ld, rows.element_size() == 4


CHUNKED = [(4, 2, 24, 16, 37), (6, 6, 128, 128, 64), (20, 1, 64, 2, 1), (5, 1, 40, 0, 100), (34, 2, 16, 16, 129), (2, 1, 200, 64, 300), (8, 2, 96, 32, 0)]


@pytest.mark.parametrize("own_values", [False, True])
@pytest.mark.parametrize("f32", [True, False])
def test_chunk_attention_rows(hip, pkg, f32, own_values):
    t = ChunkAttention(pkg, 200, 4, 2, 24, 16, 37, f32, own_values=own_values)
    tol = F32_TOL if f32 else BF_TOL
    for n0, n1 in ((0, 3), (3, 130), (130, 200)):
        rows = u.host(t.fill(hip, n0, n1))
        got = rows[:, :4 * t.dimp].reshape(-1, 4, t.dimp)
        assert u.rms_error(got[..., :24], t.q[n0:n1] * t.scale) < tol and not got[..., 24:].any()
        assert np.array_equal(rows[:, 4 * t.dimp:], t.rows[n0:n1, 4 * t.dimp:])  # what lies behind the queries stays
    k, v = u.host(t.keep[1]), u.host(t.keep[2])
    at = (4 + (2 if own_values else 0)) * t.dimp
    assert u.rms_error(k[:, :200, :24], t.k.transpose(1, 0, 2)) < tol and not k[..., 24:].any() and not k[:, 200:].any()
    assert np.array_equal(v[:, :, :200], t.rows[:, at:at + 2 * t.dimp].reshape(200, 2, t.dimp).transpose(1, 2, 0))


@pytest.mark.parametrize("own_values", [False, True])
@pytest.mark.parametrize("n,nq", [(1, 1), (2, 2), (65, 65), (128, 128), (129, 2), (300, 37), (300, 300)])
@pytest.mark.parametrize("shape", CHUNKED)
def test_chunk_attention_portion(hip, pkg, shape, n, nq, own_values):
    t = ChunkAttention(pkg, n, *shape, False, own_values=own_values)
    t.fill(hip, 0, n)
    rows = t.put(t.rows[n - nq:])
    hip.gqa_rows_dev(t.attn, rows, t.ld, False, False, pos_dev(n - nq), nq)
    t.gated(rows)
    out = t.new(nq, t.heads * t.vdimp)
    hip.gqa_prefill_dev(t.attn, rows, t.ld, n, nq, out, t.heads * t.vdimp)
    t.check(out, n - nq, 2e-2)


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("n,nq", [(1, 1), (130, 130), (300, 2)])
@pytest.mark.parametrize("shape", CHUNKED + [(2, 1, 300, 210, 70)])
def test_chunk_attention_of_any_size(hip, pkg, shape, n, nq, f32):
    t = ChunkAttention(pkg, n, *shape, f32)
    rows = t.fill(hip, 0, n)
    t.gated(rows, n - nq)
    scratch = u.zeros_f32(hip.gqa_scratch_bytes(t.heads, 1, t.vdimp, nq) // 4)
    out = u.zeros_f32(nq, t.heads * t.vdimp)
    hip.gqa_any_dev(t.attn, rows[n - nq:].contiguous(), t.ld, f32, f32, pos_dev(n - nq), 0, nq, scratch)
    hip.gqa_merge_dev(t.attn, pos_dev(n - nq), 0, nq, scratch, out, t.heads * t.vdimp, False)
    t.check(out, n - nq, 1e-5 if f32 else 2e-2)


@pytest.mark.parametrize("n", [1, 2, 32, 33, 64, 65, 128, 129, 257, 700])
@pytest.mark.parametrize("shape", CHUNKED)
def test_chunk_attention_step(hip, pkg, shape, n):
    t = ChunkAttention(pkg, n, *shape, False)
    if n > 1:
        t.fill(hip, 0, n - 1)
    scratch = u.zeros_f32(hip.gqa_scratch_bytes(t.heads, 1, t.vdimp, 1) // 4)
    out, row = u.zeros_f32(1, t.heads * t.vdimp), u.dev_f32(t.rows[n - 1])
    t.gated(row)
    hip.gqa_step_dev(t.attn, row, pos_dev(n - 1), scratch)
    hip.gqa_merge_dev(t.attn, pos_dev(n - 1), 0, 1, scratch, out, t.heads * t.vdimp, False)
    t.check(out, n - 1, 1e-2)
    k, v = u.host(t.keep[1]), u.host(t.keep[2])
    assert u.rms_error(k[:, n - 1, :t.dim], t.k[n - 1]) < BF_TOL and not k[:, n:].any()
    at = t.heads * t.dimp
    assert np.array_equal(v[:, :, n - 1], t.rows[n - 1, at:at + len(v) * t.dimp].reshape(len(v), t.dimp)) and not v[:, :, n:].any()


@pytest.mark.parametrize("f32", [True, False])
def test_attention_rows(hip, pkg, f32):
    heads, kv, dim, vdim, maps = 4, 2, 24, 40, 2
    t = Attention(pkg, 200, heads, kv, dim, vdim, maps, f32)
    tol = F32_TOL if f32 else BF_TOL
    for n0, n1 in ((0, 3), (3, 130), (130, 200)):
        rows = u.host(t.fill(hip, n0, n1))
        got = rows[:, :heads * maps * t.dimp].reshape(-1, heads, maps, t.dimp)
        assert u.rms_error(got[..., :dim], t.q[n0:n1]) < tol and not got[..., dim:].any()
    k, v = u.host(t.keep[3]), u.host(t.keep[4])
    assert u.rms_error(k[:, :, :200, :dim], t.k.transpose(1, 2, 0, 3)) < tol and not k[:, :, 200:].any() and not k[..., dim:].any()
    assert np.array_equal(v[:, :vdim, :200], t.v.transpose(1, 2, 0).astype(np.float32)) and not v[:, vdim:].any() and not v[:, :, 200:].any()


@pytest.mark.parametrize("n,nq", [(1, 1), (2, 2), (65, 65), (128, 128), (129, 2), (300, 37), (300, 300)])
@pytest.mark.parametrize("shape", SHAPES)
def test_attention_portion(hip, pkg, shape, n, nq):
    t = Attention(pkg, n, *shape, False)
    t.fill(hip, 0, n)
    rows = t.put(t.rows[n - nq:])
    hip.gqa_rows_dev(t.attn, rows, t.ld, False, False, pos_dev(n - nq), nq)
    out = t.new(nq, t.heads * t.vdimp)
    hip.gqa_prefill_dev(t.attn, rows, t.ld, n, nq, out, t.heads * t.vdimp)
    t.check(out, n - nq, 2e-2)


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("n,nq", [(1, 1), (130, 130), (300, 2)])
@pytest.mark.parametrize("shape", SHAPES + [(2, 1, 300, 270, 2)])
def test_attention_of_any_size(hip, pkg, shape, n, nq, f32):
    t = Attention(pkg, n, *shape, f32)
    rows = t.fill(hip, 0, n)
    scratch = u.zeros_f32(hip.gqa_scratch_bytes(t.heads, shape[4], t.vdimp, nq) // 4)
    out = u.zeros_f32(nq, t.heads * t.vdimp)
    hip.gqa_any_dev(t.attn, rows[n - nq:].contiguous(), t.ld, f32, f32, pos_dev(n - nq), 0, nq, scratch)
    hip.gqa_merge_dev(t.attn, pos_dev(n - nq), 0, nq, scratch, out, t.heads * t.vdimp, False)
    t.check(out, n - nq, 1e-5 if f32 else 2e-2)


@pytest.mark.parametrize("n", [1, 2, 32, 33, 128, 129, 257, 700])
@pytest.mark.parametrize("shape", SHAPES)
def test_attention_step(hip, pkg, shape, n):
    """the raw f32 row of the last token: normed, appended and attended in one launch"""
    t = Attention(pkg, n, *shape, False)
    if n > 1:
        t.fill(hip, 0, n - 1)
    scratch = u.zeros_f32(hip.gqa_scratch_bytes(t.heads, shape[4], t.vdimp, 1) // 4)
    out = u.zeros_f32(1, t.heads * t.vdimp)
    hip.gqa_step_dev(t.attn, u.dev_f32(t.rows[n - 1]), pos_dev(n - 1), scratch)
    hip.gqa_merge_dev(t.attn, pos_dev(n - 1), 0, 1, scratch, out, t.heads * t.vdimp, False)
    t.check(out, n - 1, 1e-2)
    k, v = u.host(t.keep[3]), u.host(t.keep[4])
    assert u.rms_error(k[:, :, n - 1, :shape[2]], t.k[n - 1]) < BF_TOL and not k[:, :, n:].any()
    assert np.array_equal(v[:, :shape[3], n - 1], t.v[n - 1].astype(np.float32)) and not v[:, :, n:].any()


def test_attention_step_with_more_tiles_than_records(hip, pkg):
    n = 128 * 128 + 200
    t = Attention(pkg, 300, 4, 2, 32, 32, 2, False)  # (weights and layout)
    g = rng(77)
    cap = u.up_to(n, 128)
    k, v = u.rounded(g.standard_normal((2, 2, cap, 32))), u.rounded(g.standard_normal((2, 32, cap)))
    q = g.standard_normal((4, 2, 32)).astype(np.float32)
    row = np.concatenate([q.reshape(-1), g.standard_normal(2 * 2 * 32), g.standard_normal(2 * 32)]).astype(np.float32)
    one, factor = np.ones(32, np.float32), np.full(cap, 0.3, np.float32)
    keep = [u.dev_f32(one), u.dev_f32(one), u.dev_f32(factor), u.dev_bf16(k), u.dev_bf16(v)]
    attn = pkg.Gqa(4, 2, 2, 32, 32, 32, 32, cap, 1e-5, 0.4, 0.7, *[x.data_ptr() for x in keep])
    scratch, out = u.zeros_f32(hip.gqa_scratch_bytes(4, 2, 32, 1) // 4), u.zeros_f32(4, 32)
    hip.gqa_step_dev(attn, u.dev_f32(row), pos_dev(n - 1), scratch)
    hip.gqa_merge_dev(attn, pos_dev(n - 1), 0, 1, scratch, out, 128, False)
    k, v = u.host(keep[3]).astype(np.float64)[:, :, :n], u.host(keep[4]).astype(np.float64)[:, :, :n]  # (with the new position)
    qn = so.norm_plain(q.astype(np.float64), one, 1e-5) * 0.3
    maps = np.zeros((4, 2, 32))
    for h in range(4):
        for j in range(2):
            s = k[h // 2, j] @ qn[h, j]
            e = np.exp(s - s.max())
            maps[h, j] = v[h // 2] @ (e / e.sum())
    assert u.rms_error(u.host(out), so.difference(maps, 0.4, 0.3, 1e-5)) < 2e-3
    assert t.n == 300


# ---- gated delta rule --------------------------------------------------------------------------------------------------
class DeltaCase:
    """random projections of n tokens in the library's layout, the layer's output and last state by definition"""

    def __init__(self, pkg, n, heads, kv, dim, vdim, taps, f32, seed=0):
        g = rng(n, heads, dim, taps, seed)
        self.pkg, self.n, self.heads, self.kv, self.vdim, self.f32 = pkg, n, heads, kv, vdim, f32
        self.dim, self.dimp, self.vdimp, self.taps = dim, u.up_to(dim, 32), u.up_to(vdim, 32), taps
        store = (lambda a: a.astype(np.float32)) if f32 else u.rounded
        q, k = store(g.standard_normal((n, kv, dim))), store(g.standard_normal((n, kv, dim)))
        v, gate = store(g.standard_normal((n, heads, vdim))), store(g.standard_normal((n, heads, vdim)))
        self.ba = g.standard_normal((n, 2 * heads)).astype(np.float32)
        cq, ck, cv = (0.5 * g.standard_normal((c, d, taps)).astype(np.float32) for c, d in ((kv, dim), (kv, dim), (heads, vdim)))
        rate = np.exp(g.standard_normal(heads) - 1.0).astype(np.float32)
        rate[0] = 1e-3
        dt, norm = g.standard_normal(heads).astype(np.float32), (1.0 + 0.3 * g.standard_normal(vdim)).astype(np.float32)
        pd, pv = lambda a: u.padded(a, self.dimp).reshape(n, -1), lambda a: u.padded(a, self.vdimp).reshape(n, -1)
        self.rows = np.concatenate([pd(q), pd(k), pv(v), pv(gate)], axis=1)
        self.ld = u.up_to(self.rows.shape[1], 64)
        self.rows = u.padded(self.rows, self.ld)

        def channels(w, to):  # [c, d, taps] -> [taps, c * to]
            return u.padded(w.transpose(2, 0, 1), to).reshape(taps, -1)

        conv = np.concatenate([channels(cq, self.dimp), channels(ck, self.dimp), channels(cv, self.vdimp)], axis=1)
        eps = 1e-3
        f64 = np.float64

        def convolved(a, w):
            return so.silu(so.short_convolution(a.reshape(n, -1).astype(f64), w.reshape(-1, taps).astype(f64))).reshape(a.shape)

        self.q, self.k, self.v = so.unit(convolved(q, cq)) * dim ** -0.5, so.unit(convolved(k, ck)), convolved(v, cv)
        self.beta = so.sigmoid(self.ba[:, :heads].astype(f64))
        self.logg = -rate * so.softplus(self.ba[:, heads:].astype(f64) + dt)
        S0 = 0.3 * g.standard_normal((heads, dim, vdim))
        state = np.zeros((heads, self.dimp, self.vdimp), np.float32)
        state[:, :dim, :vdim] = S0
        self.want, self.S = np.zeros((n, heads, vdim)), np.zeros_like(S0)
        for h in range(heads):
            j = h // (heads // kv)
            o, self.S[h] = so.delta_rule(self.q[:, j], self.k[:, j], self.v[:, h], np.exp(self.logg[:, h]), self.beta[:, h], state[h, :dim, :vdim].astype(f64))
            self.want[:, h] = so.norm_plain(o, norm, eps) * so.silu(gate[:, h].astype(f64))
        self.state0, self.C = state, conv.shape[1]
        self.keep = [u.dev_f32(conv), u.dev_f32(rate), u.dev_f32(dt), u.dev_f32(u.padded(norm, self.vdimp)), u.dev_f32(state), u.zeros_f32(taps, self.C)]
        p = [t.data_ptr() for t in self.keep]
        self.d = pkg.Delta(heads, kv, dim, self.dimp, vdim, self.vdimp, taps, *p[:4], dim ** -0.5, 1e-6, eps, *p[4:])

    def put(self, a):
        return u.dev_f32(a) if self.f32 else u.dev_bf16(a)

    def portion(self, hip, n0, n1, chunked):
        n, no = n1 - n0, self.heads * self.vdimp
        rows, ba, pos = self.put(self.rows[n0:n1]), u.dev_f32(self.ba[n0:n1]), pos_dev(n0)
        new = u.zeros_f32 if self.f32 else u.zeros_bf16
        qk, v, gates, out = u.zeros_f32(n, 2 * self.kv * self.dimp), new(n, no), u.zeros_f32(n, 2 * self.heads), new(n, no)
        hip.delta_rows_dev(self.d, rows, self.ld, self.f32, ba, 2 * self.heads, pos, n, qk, v, gates)
        hip.delta_keep_dev(self.d, rows, self.ld, self.f32, pos, n)
        if chunked:
            nb = hip.delta_workspace_bytes(n, self.heads, self.dimp, self.vdimp)
            hip.delta_chunked_dev(self.d, qk, v, gates, rows, self.ld, n, out, no, u.zeros_f32(nb // 4), nb)
        else:
            hip.delta_recurrent_dev(self.d, qk, v, gates, rows, self.ld, self.f32, n, out, no)
        self.prepared = u.host(qk), u.host(v), u.host(gates)
        return u.host(out)

    def step(self, hip, i):
        out = u.zeros_f32(1, self.heads * self.vdimp)
        hip.delta_step_dev(self.d, u.dev_f32(self.rows[i]), u.dev_f32(self.ba[i]), pos_dev(i), out)
        return u.host(out)

    def check(self, got, tol, state_tol):
        got = got.reshape(self.n, self.heads, self.vdimp)
        for h in range(self.heads):
            assert u.rms_error(got[:, h, :self.vdim], self.want[:, h]) < tol, h
        assert not got[:, :, self.vdim:].any()
        S = u.host(self.keep[4])
        assert u.rms_error(S[:, :self.dim, :self.vdim], self.S) < state_tol
        assert not S[:, self.dim:].any() and not S[:, :, self.vdim:].any()


DELTA = [(1, 2, 1, 24, 40, 4), (5, 4, 2, 32, 32, 2), (64, 3, 3, 64, 48, 3), (65, 2, 2, 40, 96, 1), (130, 6, 2, 128, 128, 4), (200, 2, 1, 96, 200, 3), (77, 1, 1, 8, 8, 7)]


@pytest.mark.parametrize("n,heads,kv,dim,vdim,taps", DELTA + [(20, 2, 1, 200, 250, 4)])
def test_delta_token_by_token(hip, pkg, n, heads, kv, dim, vdim, taps):
    t = DeltaCase(pkg, n, heads, kv, dim, vdim, taps, True)
    t.check(np.concatenate([t.step(hip, i) for i in range(n)]), 1e-5, 1e-5)
    t = DeltaCase(pkg, n, heads, kv, dim, vdim, taps, True)
    t.check(t.portion(hip, 0, n, False), 1e-5, 1e-5)
    qk, v, gates = t.prepared
    qk = qk.reshape(n, 2, kv, t.dimp)
    assert u.rms_error(qk[:, 0, :, :dim], t.q) < F32_TOL and u.rms_error(qk[:, 1, :, :dim], t.k) < F32_TOL and not qk[..., dim:].any()
    assert u.rms_error(v.reshape(n, heads, -1)[..., :vdim], t.v) < F32_TOL
    assert u.rms_error(gates[:, :heads], t.logg) < F32_TOL and u.rms_error(gates[:, heads:], t.beta) < F32_TOL


@pytest.mark.parametrize("n,heads,kv,dim,vdim,taps", DELTA)
def test_delta_in_chunks(hip, pkg, n, heads, kv, dim, vdim, taps):
    t = DeltaCase(pkg, n, heads, kv, dim, vdim, taps, False)
    t.check(t.portion(hip, 0, n, True), 8e-3, 4e-3)  # (bf16: the convolved values and the outputs are rounded)


def test_delta_chunks_hold_32_bits(hip, pkg):
    """the recurrence itself, apart from the rounded values and outputs: the chunked state against the one token by token on the same rows"""
    a, b = (DeltaCase(pkg, 400, 4, 2, 64, 64, 3, False) for _ in range(2))
    a.portion(hip, 0, 400, True)
    b.portion(hip, 0, 400, False)
    assert u.rms_error(u.host(a.keep[4]), u.host(b.keep[4])) < 1e-4


def test_delta_more_than_one_segment(hip, pkg):
    a, b = (DeltaCase(pkg, 700, 64, 32, 16, 16, 4, False) for _ in range(2))  # (eight chunks of 64 heads per pass)
    x, y = a.portion(hip, 0, a.n, True), b.portion(hip, 0, b.n, False)
    assert u.rms_error(x, y) < 8e-3 and u.rms_error(u.host(a.keep[4]), u.host(b.keep[4])) < 1e-4


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("taps", [1, 2, 4, 9])
def test_delta_portions_hand_over(hip, pkg, f32, taps):
    """portions of every size and single steps between them: state and the convolution's inputs carry"""
    t = DeltaCase(pkg, 300, 4, 2, 32, 40, taps, f32)
    got, at = [], 0
    for size in (2, 1, 3, 1, 1, 64, 2, 1, 65, 63, 1, 96):
        got.append(t.step(hip, at) if size == 1 else t.portion(hip, at, at + size, not f32))
        at += size
    assert at == 300
    t.check(np.concatenate(got), 1e-5 if f32 else 8e-3, 1e-5 if f32 else 4e-3)


# ---- experts -----------------------------------------------------------------------------------------------------------
def routing(m, experts, top, seed):
    z = 2.0 * rng(m, experts, seed).standard_normal((m, experts)).astype(np.float32)
    if m > 3:
        z[3] = z[3, 0]  # all alike: the lowest indices
    s = np.exp(z.astype(np.float64))
    s /= s.sum(axis=1, keepdims=True)
    ids = np.argsort(-z, axis=1, kind="stable")[:, :top]
    w = np.take_along_axis(s, ids, 1)
    return z, ids, w / (w.sum(axis=1, keepdims=True) + 1e-20)


@pytest.mark.parametrize("m,experts,top,tile", [(1, 4, 1, 64), (2, 16, 16, 64), (70, 6, 3, 64), (300, 64, 8, 64), (257, 100, 5, 128), (500, 3, 2, 128), (64, 1024, 32, 64)])
def test_route(hip, pkg, m, experts, top, tile):
    z, ids, w = routing(m, experts, top, 0)
    nb = hip.experts_plan_bytes(m, experts, top)
    ws = u.dev(np.zeros(nb // 4 + 4, np.int32))
    for _ in range(2):  # (a plan leaves its workspace ready for the next one)
        plan = hip.experts_plan_make(ws, nb, m, experts, top, tile)
        hip.experts_route_dev(u.dev_f32(z), experts, pkg.Router(experts, 0, top, 1.7), plan)
        raw, base = u.host(ws), ws.data_ptr()

        def at(p, n):
            return raw[(p - base) // 4:(p - base) // 4 + n]

        assert np.array_equal(at(plan.ids, m * top).reshape(m, top), ids)
        got = at(plan.weights, m * top).view(np.float32).reshape(m, top)
        assert u.rms_error(got, 1.7 * w) < F32_TOL
        slots, tokens = at(plan.slots, m * top), at(plan.tokens, m * top)
        assert sorted(slots) == list(range(m * top)) and np.array_equal(tokens[slots], np.repeat(np.arange(m), top))
        tiles = at(plan.tiles, 4 * int(at(plan.n_tiles, 1)[0])).reshape(-1, 4)
        expert_of = np.full(m * top, -1)
        for e, first, count, _ in tiles:
            assert 0 < count <= tile and (expert_of[first:first + count] == -1).all()
            expert_of[first:first + count] = e
        assert np.array_equal(expert_of[slots], ids.reshape(-1))


@pytest.mark.parametrize("m,experts,top,tile", [(1, 4, 2, 64), (2, 6, 3, 64), (130, 5, 2, 64), (300, 6, 4, 128), (90, 40, 3, 128)])
@pytest.mark.parametrize("width,ff", [(112, 24), (256, 136)])
@pytest.mark.parametrize("f32", [True, False])
def test_experts_of_a_portion(hip, pkg, m, experts, top, tile, width, ff, f32):
    if f32 and tile == 128:
        tile = 64
    g = rng(m, experts, width)
    z, ids, w = routing(m, experts, top, 1)
    ldw, ldf = u.up_to(width, 64), u.up_to(ff, 64)
    up, down = u.rounded(g.standard_normal((experts, ff, width)) / np.sqrt(width)), u.rounded(g.standard_normal((experts, width, ff)) / np.sqrt(ff))
    x = g.standard_normal((m, width)).astype(np.float32) if f32 else u.rounded(g.standard_normal((m, width)))
    nb = hip.experts_plan_bytes(m, experts, top)
    ws = u.dev(np.zeros(nb // 4 + 4, np.int32))
    plan = hip.experts_plan_make(ws, nb, m, experts, top, tile)
    hip.experts_route_dev(u.dev_f32(z), experts, pkg.Router(experts, 0, top, 1.0), plan)
    put, new = (u.dev_f32, u.zeros_f32) if f32 else (u.dev_bf16, u.zeros_bf16)
    act, rows = new(m * top, ldf), new(m * top, ldw)
    hip.experts_matmul_dev(plan, True, put(u.padded(x, ldw)), ldw, f32, u.dev_bf16(u.padded(up, ldw)), ff, ldw, ldw, pkg.ACT_RELU2, act, ldf, f32)
    hip.experts_matmul_dev(plan, False, act, ldf, f32, u.dev_bf16(u.padded(down, ldf)), width, ldf, ldf, pkg.ACT_NONE, rows, ldw, f32)
    slots = u.host(ws)[(plan.slots - ws.data_ptr()) // 4:][:m * top].reshape(m, top)
    got = u.host(rows)[slots][:, :, :width]
    want = np.stack([[down[e].astype(np.float64) @ so.relu_squared(up[e].astype(np.float64) @ x[i]) for e in ids[i]] for i in range(m)])
    assert u.rms_error(got, want) < (F32_TOL if f32 else 8e-3)


@pytest.mark.parametrize("experts,top,width,ff,cols0", [(4, 1, 64, 24, 8), (6, 6, 112, 40, 200), (12, 3, 320, 72, 160), (64, 8, 1000, 520, 1032), (128, 4, 2560, 768, 3328), (9, 3, 90, 16, 64)])
def test_experts_of_one_token(hip, pkg, experts, top, width, ff, cols0):
    g = rng(experts, width, ff)
    z, ids, w = routing(1, experts, top, 2)
    ldw, ldf, ld0, cols, colf = u.up_to(width, 64), u.up_to(ff, 64), u.up_to(cols0, 64), u.up_to(width, 8), u.up_to(ff, 8)
    up, down = u.rounded(g.standard_normal((experts, ff, width)) / np.sqrt(width)), u.rounded(g.standard_normal((experts, width, ff)) / np.sqrt(ff))
    w0, bias = u.rounded(g.standard_normal((width, cols0)) / np.sqrt(cols0)), g.standard_normal(width).astype(np.float32)
    x, x0 = g.standard_normal(width).astype(np.float32), g.standard_normal(cols0).astype(np.float32)
    act, idd, y = u.zeros_f32(top, ldf), u.dev(np.zeros(64, np.int32)), u.zeros_f32(width)
    hip.experts_up_dev(u.dev_f32(z[0]), pkg.Router(experts, 0, top, 2.5), u.dev_f32(u.padded(x, cols)), u.dev_bf16(u.padded(up, ldw)), ff, cols, ldw, pkg.ACT_RELU2, act, ldf, idd)
    assert np.array_equal(u.host(idd)[:top], ids[0])
    want = 2.5 * w[0][:, None] * np.stack([so.relu_squared(up[e].astype(np.float64) @ x) for e in ids[0]])
    assert u.rms_error(u.host(act)[:, :ff], want) < F32_TOL
    hip.experts_out_dev(u.dev_f32(x0), u.dev_bf16(u.padded(w0, ld0)), cols0, ld0, u.dev_f32(bias), act, ldf, u.dev_bf16(u.padded(down, ldf)), colf, ldf, idd, top, width, y)
    want = w0.astype(np.float64) @ x0 + bias + sum(down[e].astype(np.float64) @ want[k] for k, e in enumerate(ids[0]))
    assert u.rms_error(u.host(y), want) < F32_TOL


# experts that hand their input through, choice by corrected scores, weights as the scores are, gated pairs
def corrected(m, experts, identity, top, seed):
    n = experts + identity
    g = rng(m, n, top, seed, 9)
    z, c = 1.5 * g.standard_normal((m, n)).astype(np.float32), g.uniform(-0.3, 0.3, n).astype(np.float32)
    if m > 3:
        z[3] = 30.0 * (np.arange(n) < 1)  # one takes all; the others by their corrections
    s = np.exp(z.astype(np.float64) - z.max(axis=1, keepdims=True))
    s /= s.sum(axis=1, keepdims=True)
    order = np.argsort(-(s + c), axis=1, kind="stable")
    return z, c, order[:, :top], np.take_along_axis(s, order[:, :top], 1)


def same_choice(got, z, c, ids):
    """the oracle's choice, up to choice scores that lie within rounding of each other"""
    s = np.exp(z.astype(np.float64) - z.max(axis=1, keepdims=True))
    choice = s / s.sum(axis=1, keepdims=True) + c
    return np.abs(np.take_along_axis(choice, np.asarray(got, np.int64), 1) - np.take_along_axis(choice, ids, 1)).max() < 1e-6


CORRECTED = [(1, 4, 2, 1, 64), (2, 16, 1, 17, 64), (70, 6, 3, 3, 64), (300, 56, 8, 8, 64), (257, 100, 30, 5, 128), (500, 3, 9, 2, 128), (64, 1000, 24, 32, 64), (90, 1, 5, 4, 64)]


@pytest.mark.parametrize("m,experts,identity,top,tile", CORRECTED)
def test_corrected_route(hip, pkg, m, experts, identity, top, tile):
    z, c, ids, w = corrected(m, experts, identity, top, 0)
    nb, ldz = hip.experts_plan_bytes(m, experts, top), experts + identity + 3
    ws, cd = u.dev(np.zeros(nb // 4 + 4, np.int32)), u.dev_f32(c)
    for raw_weights in (1, 0):
        plan = hip.experts_plan_make(ws, nb, m, experts, top, tile)
        hip.experts_route_dev(u.dev_f32(u.padded(z, ldz)), ldz, pkg.Router(experts, identity, top, 0.8, raw_weights, cd.data_ptr()), plan)
        raw, base = u.host(ws), ws.data_ptr()

        def at(p, n):
            return raw[(p - base) // 4:(p - base) // 4 + n]

        got = at(plan.ids, m * top).reshape(m, top)
        assert same_choice(got, z, c, ids)
        s = np.exp(z.astype(np.float64) - z.max(axis=1, keepdims=True))
        want = np.take_along_axis(s / s.sum(axis=1, keepdims=True), got.astype(np.int64), 1)
        want = want if raw_weights else want / want.sum(axis=1, keepdims=True)
        assert u.rms_error(at(plan.weights, m * top).view(np.float32).reshape(m, top), 0.8 * want) < F32_TOL
        slots, real = at(plan.slots, m * top).reshape(m, top), got < experts
        assert (slots[~real] == -1).all() and sorted(slots[real]) == list(range(real.sum()))
        assert np.array_equal(at(plan.tokens, m * top)[slots[real]], np.repeat(np.arange(m), top).reshape(m, top)[real])
        tiles = at(plan.tiles, 4 * int(at(plan.n_tiles, 1)[0])).reshape(-1, 4)
        expert_of = np.full(m * top, -1)
        for e, first, count, _ in tiles:
            assert 0 < count <= tile and (expert_of[first:first + count] == -1).all()
            expert_of[first:first + count] = e
        assert np.array_equal(expert_of[slots[real]], got[real]) and (expert_of[real.sum():] == -1).all()


@pytest.mark.parametrize("m,experts,identity,top,tile", [(2, 6, 2, 3, 64), (130, 5, 1, 2, 64), (300, 6, 4, 4, 128), (90, 1, 5, 4, 64)])
@pytest.mark.parametrize("width,ff", [(112, 24), (256, 135), (192, 300)])
@pytest.mark.parametrize("f32", [True, False])
def test_gated_experts_of_a_portion(hip, pkg, m, experts, identity, top, tile, width, ff, f32):
    if f32 and tile == 128:
        tile = 64
    g = rng(m, experts, width, 8)
    z, c, ids, _ = corrected(m, experts, identity, top, 1)
    ldw, ldf = u.up_to(width, 64), u.up_to(ff, 64)
    up, down = u.rounded(2.0 * g.standard_normal((experts, 2 * ff, width)) / np.sqrt(width)), u.rounded(g.standard_normal((experts, width, ff)) / np.sqrt(ff))
    x = g.standard_normal((m, width)).astype(np.float32) if f32 else u.rounded(g.standard_normal((m, width)))
    nb, cd = hip.experts_plan_bytes(m, experts, top), u.dev_f32(c)
    ws = u.dev(np.zeros(nb // 4 + 4, np.int32))
    plan = hip.experts_plan_make(ws, nb, m, experts, top, tile)
    hip.experts_route_dev(u.dev_f32(z), experts + identity, pkg.Router(experts, identity, top, 1.0, 1, cd.data_ptr()), plan)
    put, new = (u.dev_f32, u.zeros_f32) if f32 else (u.dev_bf16, u.zeros_bf16)
    act, rows = new(m * top, ldf), new(m * top, ldw)
    hip.experts_matmul_dev(plan, True, put(u.padded(x, ldw)), ldw, f32, u.dev_bf16(u.padded(up, ldw)), 2 * ff, ldw, ldw, pkg.ACT_SILU | pkg.ACT_GATED, act, ldf, f32)
    hip.experts_matmul_dev(plan, False, act, ldf, f32, u.dev_bf16(u.padded(down, ldf)), width, ldf, ldf, pkg.ACT_NONE, rows, ldw, f32)
    raw = u.host(ws)
    slots, got_ids = (raw[(q - ws.data_ptr()) // 4:][:m * top].reshape(m, top) for q in (plan.slots, plan.ids))
    got, want = [], []
    for i in range(m):
        for k in range(top):
            e = got_ids[i, k]
            if e >= experts:
                continue
            h = up[e].astype(np.float64) @ x[i]
            want.append(down[e].astype(np.float64) @ (so.silu(h[0::2]) * h[1::2]))
            got.append(u.host(rows[slots[i, k]])[:width])
    if want:
        assert u.rms_error(got, want) < (F32_TOL if f32 else 8e-3)


@pytest.mark.parametrize("experts,identity,top,width,ff,cols0", [(4, 2, 1, 64, 24, 0), (6, 2, 8, 112, 40, 200), (12, 5, 3, 320, 72, 0), (64, 8, 8, 1000, 519, 0), (64, 8, 8, 2560, 576, 0),
                                                                 (2, 60, 9, 90, 16, 64), (1, 9, 3, 200, 130, 0)])
@pytest.mark.parametrize("seed", [2, 3, 4])
def test_gated_experts_of_one_token(hip, pkg, experts, identity, top, width, ff, cols0, seed):
    """also with none but identities among the chosen (few experts, many identities)"""
    g = rng(experts, width, ff, 8)
    z, c, ids, w = corrected(1, experts, identity, top, seed)
    ldw, ldf, ld0, cols, colf = u.up_to(width, 64), u.up_to(ff, 64), u.up_to(cols0, 64), u.up_to(width, 8), u.up_to(ff, 8)
    up, down = u.rounded(2.0 * g.standard_normal((experts, 2 * ff, width)) / np.sqrt(width)), u.rounded(g.standard_normal((experts, width, ff)) / np.sqrt(ff))
    w0, bias = u.rounded(g.standard_normal((width, cols0)) / np.sqrt(max(cols0, 1))), g.standard_normal(width).astype(np.float32)
    x, x0 = g.standard_normal(width).astype(np.float32), g.standard_normal(cols0).astype(np.float32)
    act, idd, y, through, cd = u.zeros_f32(top, ldf), u.dev(np.full(64, 77, np.int32)), u.zeros_f32(width), u.zeros_f32(1), u.dev_f32(c)
    xd = u.dev_f32(u.padded(x, cols))
    hip.experts_up_dev(u.dev_f32(z[0]), pkg.Router(experts, identity, top, 2.5, 1, cd.data_ptr()), xd, u.dev_bf16(u.padded(up, ldw)), 2 * ff, cols, ldw, pkg.ACT_SILU | pkg.ACT_GATED,
                       act, ldf, idd, through)
    real = ids[0] < experts
    n = int(real.sum())
    got = u.host(idd)
    assert np.array_equal(got[:n], ids[0][real]) and (got[n:top] == -1).all() and (got[top:] == 77).all()
    assert abs(u.host(through)[0] - 2.5 * w[0][~real].sum()) < 1e-5
    want = np.zeros((n, ff))
    for k, (e, s) in enumerate(zip(ids[0][real], w[0][real])):
        h = up[e].astype(np.float64) @ x
        want[k] = 2.5 * s * so.silu(h[0::2]) * h[1::2]
    if n:
        assert u.rms_error(u.host(act)[:n, :ff], want) < F32_TOL
    first = (u.dev_f32(x0), u.dev_bf16(u.padded(w0, ld0))) if cols0 else (None, None)
    hip.experts_out_dev(*first, cols0, ld0, u.dev_f32(bias), act, ldf, u.dev_bf16(u.padded(down, ldf)), colf, ldf, idd, top, width, y, identity=through, input=xd)
    want = w0.astype(np.float64) @ x0 + bias + 2.5 * w[0][~real].sum() * x.astype(np.float64) + sum(down[e].astype(np.float64) @ want[k] for k, e in enumerate(ids[0][real]))
    assert u.rms_error(u.host(y), want) < F32_TOL
