"""What a product does besides multiplying (pairs and plain rows, convolutions, table factors, xIELU), gated rows of the residual, windowed attention with
distance penalties and convolutions ahead of it, grouped routing, token pairs and latent attention without a sink (include/bitnet_hip.h section 5), one at a
time through the C ABI, against the plain restatement in oracle/stack_oracle.py or f64 numpy."""
import numpy as np
import pytest

from oracle import stack_oracle as so
from tests import stack_util as u

pytestmark = pytest.mark.gpu
F32_TOL, BF_TOL = 3e-6, 6e-3
f64 = np.float64


def rng(*seed):
    return np.random.default_rng(list(seed))


def pos_dev(p):
    return u.dev(np.array([p], np.int32))


def ptr(t, offset=0):
    return t.data_ptr() + offset


# ---- products ----------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("pairs,rows,cols", [(4, 3, 40), (64, 65, 200), (128, 200, 2560), (1792, 2625, 2560), (8, 9000, 1288), (6000, 30, 64)])
def test_gemv_of_pairs_and_plain_rows(hip, pkg, pairs, rows, cols):
    """pairs, then rows of two kinds of activation: the layout of a block with a gated shared expert"""
    g = rng(pairs, rows, cols)
    ld, n, sig = u.up_to(cols, 64), pairs + rows, rows * 2 // 3
    w, x, b = u.rounded(2.0 * g.standard_normal((n, cols)) / np.sqrt(cols)), g.standard_normal(cols).astype(np.float32), g.standard_normal(n).astype(np.float32)
    out = u.zeros_f32(pairs // 2 + rows + 1) + 7
    hip.dense_gemv_dev(u.dev_f32(x), u.dev_bf16(u.padded(w, ld)), n, cols, ld, out, bias=u.dev_f32(b), act0=pkg.ACT_SILU | pkg.ACT_GATED, act1=pkg.ACT_SIGMOID, act_split=pairs,
                       more=pkg.Epilogue(pairs=pairs, act2_from=pairs + sig, act2=pkg.ACT_NONE))
    z = w @ x.astype(f64) + b
    plain = z[pairs:].copy()
    plain[:sig] = so.sigmoid(plain[:sig])
    got = u.host(out)
    assert u.rms_error(got[:-1], np.concatenate([so.silu(z[0:pairs:2]) * z[1:pairs:2], plain])) < F32_TOL and got[-1] == 7


@pytest.mark.parametrize("taps", [1, 2, 3, 4, 9, 64])
@pytest.mark.parametrize("ahead,channels,behind,cols", [(0, 5, 0, 40), (64, 96, 33, 200), (3, 1000, 500, 520), (128, 3000, 0, 2560)])
def test_gemv_convolves_its_rows(hip, pkg, taps, ahead, channels, behind, cols):
    """one token after the other, from the first on: the ring holds the last taps of them"""
    g = rng(taps, channels, cols)
    ld, n, steps = u.up_to(cols, 64), ahead + channels + behind, min(2 * taps + 3, 70)
    w, b = u.rounded(g.standard_normal((n, cols)) / np.sqrt(cols)), g.standard_normal(n).astype(np.float32)
    xs, f = g.standard_normal((steps, cols)).astype(np.float32), g.standard_normal((channels, taps)).astype(np.float32)
    wd, bd, fd, ring = u.dev_bf16(u.padded(w, ld)), u.dev_f32(b), u.dev_f32(f.T), u.zeros_f32(taps, channels) + 99
    z = xs.astype(f64) @ w.T.astype(f64) + b
    want = z.copy()
    want[:, ahead:ahead + channels] = so.short_convolution(z[:, ahead:ahead + channels], f.astype(f64))
    want[:, :ahead] = so.sigmoid(want[:, :ahead])
    for i in range(steps):
        out, pos = u.zeros_f32(n), pos_dev(i)
        more = pkg.Epilogue(conv_from=ahead, channels=channels, taps=taps, conv=ptr(fd), ring=ptr(ring), pos=ptr(pos))
        hip.dense_gemv_dev(u.dev_f32(xs[i]), wd, n, cols, ld, out, bias=bd, act0=pkg.ACT_SIGMOID if ahead else 0, act1=0, act_split=ahead, more=more)
        assert u.rms_error(u.host(out), want[i]) < F32_TOL, i
    kept = u.host(ring)
    for i in range(max(0, steps - taps), steps):
        assert u.rms_error(kept[i % taps], z[i, ahead:ahead + channels]) < F32_TOL


XIELU = (0.9, 1.3)  # the constants behind the softplus


def xielu(z):
    inverse = [np.log(np.expm1(v)) for v in (XIELU[0], XIELU[1] - 0.5)]
    return so.xielu(z, *inverse)


@pytest.mark.parametrize("rows,cols", [(3, 8), (200, 136), (7000, 2560)])
def test_gemv_xielu(hip, pkg, rows, cols):
    g = rng(rows, 1)
    ld = u.up_to(cols, 64)
    w, x = u.rounded(3.0 * g.standard_normal((rows, cols)) / np.sqrt(cols)), g.standard_normal(cols).astype(np.float32)
    out = u.zeros_f32(rows)
    hip.dense_gemv_dev(u.dev_f32(x), u.dev_bf16(u.padded(w, ld)), rows, cols, ld, out, act0=pkg.ACT_XIELU, more=pkg.Epilogue(act_a=XIELU[0], act_b=XIELU[1]))
    assert u.rms_error(u.host(out), xielu(w @ x.astype(f64))) < F32_TOL


@pytest.mark.parametrize("m,n,k", [(1, 5, 64), (70, 130, 128), (300, 417, 320), (2050, 1100, 1152)])
@pytest.mark.parametrize("f32", [True, False])
def test_matmul_xielu_ahead_of_gates(hip, pkg, m, n, k, f32):
    """alone, and with sigmoids from a column in the middle of a tile on"""
    g = rng(m, n, k, 1)
    x, w = g.standard_normal((m, k)), u.rounded(3.0 * g.standard_normal((n, k)) / np.sqrt(k))
    x = x.astype(np.float32) if f32 else u.rounded(x)
    z = x.astype(f64) @ w.T.astype(f64)
    more = pkg.Epilogue(act_a=XIELU[0], act_b=XIELU[1])
    for split in (0, n // 3 + 1):
        out = (u.zeros_f32 if f32 else u.zeros_bf16)(m, n)
        hip.dense_matmul_dev((u.dev_f32 if f32 else u.dev_bf16)(x), k, f32, u.dev_bf16(w), k, m, n, k, out, n, f32, act0=pkg.ACT_XIELU, act1=pkg.ACT_SIGMOID, act_split=split, more=more)
        want = np.where(np.arange(n) < (split or n), xielu(z), so.sigmoid(z))
        assert u.rms_error(u.host(out), want) < (F32_TOL if f32 else 4e-3)


@pytest.mark.parametrize("n", [1, 12, 64, 70, 256])
@pytest.mark.parametrize("f32", [True, False])
def test_products_weighed_by_the_tokens(hip, pkg, n, f32):
    """gelu of the product times a part of the row of each token's table: a portion, and its tokens one by one"""
    g = rng(n, 2)
    m, k, vocab, layers, first = 150, 192, 30, 3, 7
    x, w = g.standard_normal((m, k)), u.rounded(2.0 * g.standard_normal((n, k)) / np.sqrt(k))
    x = x.astype(np.float32) if f32 else u.rounded(x)
    table, tokens = u.rounded(g.standard_normal((vocab, layers * n))), g.integers(0, vocab, first + m).astype(np.int32)
    ld, ldc = u.up_to(layers * n, 64), u.up_to(n + 1, 64)
    td, tok, pos, wd = u.dev_bf16(u.padded(table, ld)), u.dev(tokens), pos_dev(first), u.dev_bf16(w)
    put, new = (u.dev_f32, u.zeros_f32) if f32 else (u.dev_bf16, u.zeros_bf16)
    want = so.gelu_tanh(x.astype(f64) @ w.T.astype(f64)) * table[tokens[first:], n:2 * n]
    more = pkg.Epilogue(mul=ptr(td, 2 * n), ld_mul=ld, mul_rows=vocab, mul_tokens=ptr(tok), mul_at=ptr(pos))
    out = new(m, ldc)
    out[:, n:] = 3
    hip.dense_matmul_dev(put(x), k, f32, wd, k, m, n, k, out, ldc, f32, act0=pkg.ACT_GELU_TANH, more=more)
    assert u.rms_error(u.host(out)[:, :n], want) < (F32_TOL if f32 else 4e-3) and bool((out[:, n:] == 3).all())
    for i in (0, 1, m - 1):
        pos = pos_dev(first + i)
        more.mul_at = ptr(pos)
        y = u.zeros_f32(n)
        hip.dense_gemv_dev(u.dev_f32(x[i]), wd, n, k, k, y, act0=pkg.ACT_GELU_TANH, more=more)
        assert u.rms_error(u.host(y), want[i]) < F32_TOL


# ---- rows and vectors of the residual stream -----------------------------------------------------------------------------
@pytest.mark.parametrize("n", [80, 90, 1001, 2560, 4096, 5000])
def test_gemv_adds_a_gated_sublayer(hip, pkg, n):
    g = rng(n, 3)
    rows, ld, cols, eps, mult = 70, u.up_to(n, 64), u.up_to(n, 8), 1e-3, 0.8
    w = u.rounded(g.standard_normal((rows, n)) / np.sqrt(n))
    x, y, nw, nb, pw = (g.standard_normal(n).astype(np.float32) for _ in range(5))
    gate = g.random(n).astype(np.float32)
    wd = u.dev_bf16(u.padded(w, ld))
    for post in (None, pw):
        out, xo = u.zeros_f32(rows), u.zeros_f32(n)
        hip.dense_gemv_dev(u.dev_f32(x), wd, rows, cols, ld, out, kind=pkg.IN_RESIDUAL_NORM, eps=eps, weight=u.dev_f32(nw), norm_bias=u.dev_f32(nb), center=True, res=u.dev_f32(y),
                           mult=mult, post_weight=None if post is None else u.dev_f32(post), y_gate=u.dev_f32(gate), x_out=xo, n=n)
        added = mult * y.astype(f64) if post is None else so.norm_plain(y.astype(f64), post, eps)
        x2 = x + added * gate
        assert u.rms_error(u.host(xo), x2) < F32_TOL and u.rms_error(u.host(out), w @ so.layer_norm(x2, nw, nb, eps)) < F32_TOL


@pytest.mark.parametrize("width", [96, 90, 1000, 2560, 4096, 5000])
@pytest.mark.parametrize("f32", [True, False])
def test_rows_add_a_gated_sublayer(hip, pkg, width, f32):
    """a number per row on y (a column of another matrix), the experts' rows, a gate per column; also behind a norm"""
    g = rng(width, 4)
    m, top, eps, mult, ld = 6, 3, 1e-2, 0.7, u.up_to(width, 64)
    ldg = ld + 64
    x, y = (g.standard_normal((m, width)).astype(np.float32) for _ in range(2))
    e, gate, numbers = g.standard_normal((m * top, width)), g.random((m, width)), g.random((m, 5)).astype(np.float32)
    store = (lambda a: a.astype(np.float32)) if f32 else u.rounded
    e, gate = store(e), store(gate)
    slots, sw = g.permutation(m * top).astype(np.int32).reshape(m, top), g.random((m, top)).astype(np.float32)
    nw, nb, pw = (g.standard_normal(width).astype(np.float32) for _ in range(3))
    put, new, tol = (u.dev_f32, u.zeros_f32, F32_TOL) if f32 else (u.dev_bf16, u.zeros_bf16, BF_TOL)
    keep = [u.dev_f32(y), put(u.padded(e, ld)), u.dev(slots), u.dev_f32(sw), u.dev_f32(nw), u.dev_f32(nb), put(u.padded(gate, ldg)), u.dev_f32(numbers), u.dev_f32(pw)]
    p = [k.data_ptr() for k in keep]
    t = numbers[:, 2:3].astype(f64) * y + np.einsum("mk,mkw->mw", sw.astype(f64), e[slots].astype(f64))
    for post in (0, p[8]):
        xd, h = u.dev_f32(x), new(m, ld) + 3
        hip.sum_norm_rows_dev(pkg.SumRows(x=xd.data_ptr(), m=m, width=width, mult=mult, eps=eps, h_f32=f32, h=h.data_ptr(), ldh=ld, y=p[0], ldy=width, expert_rows=p[1], ld_expert=ld,
                                          top=top, slots=p[2], slot_weights=p[3], center=1, weight=p[4], bias=p[5], gate=p[6], ld_gate=ldg, y_scale=p[7] + 8, ld_y_scale=5, post_weight=post))
        want = x + gate.astype(f64) * (so.norm_plain(t, pw, eps) if post else mult * t)
        assert u.rms_error(u.host(xd), want) < F32_TOL
        assert u.rms_error(u.host(h)[:, :width], so.layer_norm(want, nw, nb, eps)) < tol and not u.host(h)[:, width:].any()


@pytest.mark.parametrize("width", [40, 77, 2560, 4500])
@pytest.mark.parametrize("buckets,prev,cur", [(1, 0, 0), (13, 5, 3), (499, 113, 29), (97, 2000000011, 1999999973)])
def test_embedding_of_token_pairs(hip, width, buckets, prev, cur):
    g = rng(width, buckets)
    ld, tokens = u.up_to(width, 64), np.array([5, 0, 11, 11, 3, 7], np.int32)
    table, pairs = u.rounded(g.standard_normal((12, width))), u.rounded(g.standard_normal((buckets + 1, width)))
    rows = so.bigram_rows(tokens, {"buckets": buckets, "mul_prev": prev, "mul_cur": cur})
    want = 0.3 * table[tokens].astype(f64) + pairs[rows]
    td, pd, tok = u.dev_bf16(u.padded(table, ld)), u.dev_bf16(u.padded(pairs, ld)), u.dev(tokens)
    for first, n in ((0, 6), (0, 1), (1, 1), (2, 4), (5, 1)):
        out = u.zeros_f32(n, width)
        hip.embed_pairs_bf16_dev(td, ld, pd, ld, buckets, prev, cur, tok, out, n, width, 12, offset=pos_dev(first), scale=0.3)
        assert u.rms_error(u.host(out), want[first:first + n]) < F32_TOL


# ---- attention -----------------------------------------------------------------------------------------------------------
class WindowAttention:
    """random projections of n tokens in the library's layout, and by definition what becomes of them: convolutions, a window, a penalty of the distance, a gate
    per column.  far: one head that loses little with the distance."""

    def __init__(self, pkg, n, heads, kv, dim, vdim, window, taps, f32, seed=0):
        g = rng(n, heads, dim, window, taps, seed)
        self.pkg, self.n, self.heads, self.kv, self.f32, self.dim, self.vdim, self.taps = pkg, n, heads, kv, f32, dim, vdim, taps
        self.dimp, self.vdimp, self.cap = u.up_to(dim, 32), u.up_to(vdim, 32), u.up_to(n, 128)
        store = (lambda a: a.astype(np.float32)) if f32 else u.rounded
        q, k, v = store(g.standard_normal((n, heads, dim))), store(g.standard_normal((n, kv, dim))), store(g.standard_normal((n, kv, vdim)))
        gate = store(2.0 * g.standard_normal((n, heads, vdim)))
        parts = [u.padded(a, to).reshape(n, -1) for a, to in ((q, self.dimp), (k, self.dimp), (v, self.vdimp), (gate, self.vdimp))]
        self.channels = sum(a.shape[1] for a in parts[:3])
        self.rows = np.concatenate(parts, axis=1)
        self.ld = u.up_to(self.rows.shape[1], 64)
        self.rows = u.padded(self.rows, self.ld)
        self.scale = 1.7 / np.sqrt(dim)
        conv = []
        for i, (a, to) in enumerate(((q, self.dimp), (k, self.dimp), (v, self.vdimp))):
            w = g.standard_normal((a.shape[1], a.shape[2], max(taps, 1))).astype(np.float32) / np.sqrt(max(taps, 1))
            conv.append(u.padded(w.transpose(2, 0, 1), to).reshape(max(taps, 1), -1))
            a = a.astype(f64).reshape(n, -1)
            done = so.short_convolution(a, w.reshape(a.shape[1], -1).astype(f64)) if taps else a
            setattr(self, "qkv"[i], done.reshape(n, w.shape[0], w.shape[1]))
        self.r1, self.r2 = g.uniform(0.1, 1.2, heads).astype(np.float32), g.uniform(0.01, 2.0, heads).astype(np.float32)
        self.r1[0] = 0.02
        as_kept = (lambda a: a) if f32 else (lambda a: u.rounded(a).astype(f64))  # (what the caches hold)
        o = so.window_softmax(self.q, as_kept(self.k), as_kept(self.v), self.scale, window or n, self.r1.astype(f64), self.r2.astype(f64))
        self.want = o * so.sigmoid(gate.astype(f64))
        new = u.zeros_f32 if f32 else u.zeros_bf16
        self.keep = [u.dev_f32(np.full(self.cap, self.scale)), new(kv, self.cap, self.dimp), new(kv, self.vdimp, self.cap), u.dev_f32(self.r1), u.dev_f32(self.r2),
                     u.dev_f32(np.concatenate(conv, axis=1)), u.zeros_f32(max(taps, 1), self.channels) + 99]
        p = [t.data_ptr() for t in self.keep]
        self.attn = pkg.Gqa(heads, kv, 1, dim, self.dimp, vdim, self.vdimp, self.cap, 1e-3, 0.0, 1.0, 0, 0, p[0], p[1], p[2], gate_columns=1, window=window, far_weight=p[3], far_rate=p[4])
        if taps:
            self.attn.taps, self.attn.conv, self.attn.ring = taps, p[5], p[6]

    def put(self, a):
        return u.dev_f32(a) if self.f32 else u.dev_bf16(a)

    def new(self, *shape):
        return u.zeros_f32(*shape) if self.f32 else u.zeros_bf16(*shape)

    def gated(self, rows):
        self.attn.gate = rows.data_ptr() + self.channels * (4 if rows.element_size() == 4 else 2)
        self.attn.ldgate, self.attn.gate_f32 = self.ld, rows.element_size() == 4

    def fill(self, hip, n0, n1):
        """convolutions and appends of tokens n0 .. n1 - 1; (raw rows, queries, leading dimension of those)"""
        rows, pos = self.put(self.rows[n0:n1]), pos_dev(n0)
        self.gated(rows)
        if not self.taps:
            hip.gqa_rows_dev(self.attn, rows, self.ld, self.f32, self.f32, pos, n1 - n0)
            return rows, rows, self.ld
        ldq = self.heads * self.dimp
        q = self.new(n1 - n0, ldq)
        hip.gqa_rows_dev(self.attn, rows, self.ld, self.f32, self.f32, pos, n1 - n0, q, ldq)
        hip.conv_keep_dev(rows, self.ld, self.f32, self.channels, self.taps, self.keep[6], pos, n1 - n0)
        return rows, q, ldq

    def check(self, got, n0, tol):
        got = u.host(got).reshape(-1, self.heads, self.vdimp)
        want = self.want[n0:n0 + len(got)]
        for h in range(self.heads):
            assert u.rms_error(got[:, h, :self.vdim], want[:, h]) < tol, h
        assert not got[:, :, self.vdim:].any()

    def portion(self, hip, n0, n1):
        rows, q, ldq = self.fill(hip, n0, n1)
        n, no = n1 - n0, self.heads * self.vdimp
        out = self.new(n, no)
        if not self.f32 and hip.c.bitnet_hip_gqa_supported(self.dimp, self.vdimp):
            hip.gqa_prefill_dev(self.attn, q, ldq, n1, n, out, no)
        else:
            scratch, pos = u.zeros_f32(hip.gqa_scratch_bytes(self.heads, 1, self.vdimp, n) // 4), pos_dev(n0)
            hip.gqa_any_dev(self.attn, q, ldq, self.f32, self.f32, pos, 0, n, scratch)
            hip.gqa_merge_dev(self.attn, pos, 0, n, scratch, out, no, not self.f32)
        return out

    def step(self, hip, i, queries_only=False):
        """the last token from its convolved row, as the product ahead of it leaves it"""
        row = self.rows[i].copy()
        parts = [u.padded(a[i], to).reshape(-1) for a, to in ((self.q, self.dimp), (self.k, self.dimp), (self.v, self.vdimp))]
        row[:self.channels] = np.concatenate(parts)
        row = u.dev_f32(row)
        self.gated(row)
        taps, self.attn.taps, self.attn.queries_only = self.attn.taps, 0, queries_only
        scratch, out, pos = u.zeros_f32(hip.gqa_scratch_bytes(self.heads, 1, self.vdimp, 1) // 4), u.zeros_f32(1, self.heads * self.vdimp), pos_dev(i)
        hip.gqa_step_dev(self.attn, row, pos, scratch)
        hip.gqa_merge_dev(self.attn, pos, 0, 1, scratch, out, self.heads * self.vdimp, False)
        self.attn.taps, self.attn.queries_only = taps, 0
        return out


# heads, kv heads, dim, vdim, window, taps
WINDOWED = [(4, 2, 24, 40, 37, 3), (6, 6, 128, 128, 64, 2), (20, 1, 64, 100, 1, 4), (5, 1, 40, 16, 100, 1), (34, 2, 16, 24, 129, 3), (2, 1, 200, 256, 300, 5), (8, 2, 96, 64, 0, 0),
            (8, 4, 128, 64, 200, 0)]


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("shape", WINDOWED + [(2, 1, 300, 270, 50, 3), (2, 2, 24, 40, 30, 64)])
def test_convolved_rows(hip, pkg, shape, f32):
    """queries, keys and values across every cut, raw rows left as they are, the ring as the last tokens leave it"""
    n = 200
    t = WindowAttention(pkg, n, *shape, f32)
    heads, kv, dim, vdim, _, taps = shape
    tol = F32_TOL if f32 else BF_TOL
    for n0, n1 in ((0, 1), (1, 3), (3, 5), (5, 130), (130, 200)):
        rows, q, ldq = t.fill(hip, n0, n1)
        got = u.host(q)[:, :heads * t.dimp].reshape(-1, heads, t.dimp)
        assert u.rms_error(got[..., :dim], t.q[n0:n1] * t.scale) < tol and not got[..., dim:].any()
        if taps:
            assert np.array_equal(u.host(rows), t.rows[n0:n1])
    k, v = u.host(t.keep[1]), u.host(t.keep[2])
    assert u.rms_error(k[:, :n, :dim], t.k.transpose(1, 0, 2)) < tol and not k[..., dim:].any() and not k[:, n:].any()
    assert u.rms_error(v[:, :vdim, :n], t.v.transpose(1, 2, 0)) < tol and not v[:, vdim:].any() and not v[:, :, n:].any()
    ring = u.host(t.keep[6])
    for i in range(n - taps + 1, n) if taps else ():
        assert np.array_equal(ring[i % taps], t.rows[i, :t.channels])


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("cuts", [[1], [2], [65], [128], [129, 2], [300], [263, 37], [3, 1, 60, 2, 1, 64, 65, 100]])
@pytest.mark.parametrize("shape", WINDOWED)
def test_window_attention_portions(hip, pkg, shape, cuts, f32):
    t = WindowAttention(pkg, sum(cuts), *shape, f32)
    at = 0
    for n in cuts:
        out = t.portion(hip, at, at + n)
        t.check(out, at, 1e-5 if f32 else 2e-2)
        at += n


@pytest.mark.parametrize("f32", [True, False])
def test_window_attention_of_huge_heads(hip, pkg, f32):
    t = WindowAttention(pkg, 130, 2, 1, 300, 270, 50, 3, f32)
    for n0, n1 in ((0, 70), (70, 130)):
        t.check(t.portion(hip, n0, n1), n0, 1e-5 if f32 else 2e-2)


@pytest.mark.parametrize("n", [1, 2, 32, 33, 64, 65, 128, 129, 257, 700])
@pytest.mark.parametrize("shape", WINDOWED)
def test_window_attention_step(hip, pkg, shape, n):
    """one token with keys of its own, and -- the row of projections has only queries then -- on keys that another layer has put there already"""
    t = WindowAttention(pkg, n, *shape, False)
    if n > 1:
        t.fill(hip, 0, n - 1)
    t.check(t.step(hip, n - 1), n - 1, 1e-2)
    k, v = u.host(t.keep[1]), u.host(t.keep[2])
    assert u.rms_error(k[:, n - 1, :t.dim], t.k[n - 1]) < BF_TOL and not k[:, n:].any()
    assert u.rms_error(v[:, :t.vdim, n - 1], t.v[n - 1]) < BF_TOL and not v[:, :, n:].any()
    t.check(t.step(hip, n - 1, queries_only=True), n - 1, 1e-2)
    assert np.array_equal(u.host(t.keep[1]), k) and np.array_equal(u.host(t.keep[2]), v)


@pytest.mark.parametrize("f32", [True, False])
def test_queries_of_another_layers_keys(hip, pkg, f32):
    """rows without keys and values: the caches stay, the queries pass their convolution"""
    t = WindowAttention(pkg, 150, 6, 2, 40, 24, 33, 3, f32)
    t.fill(hip, 0, 150)
    before = [u.host(t.keep[i]) for i in (1, 2)]
    nq, heads = t.heads * t.dimp, t.heads
    rows = np.concatenate([t.rows[:, :nq], t.rows[:, t.channels:t.channels + heads * t.vdimp]], axis=1)
    ld = u.up_to(rows.shape[1], 64)
    conv, ring = u.dev_f32(u.host(t.keep[5])[:, :nq]), u.zeros_f32(3, nq) + 99
    t.attn.queries_only, t.attn.conv, t.attn.ring = 1, ptr(conv), ptr(ring)
    at = 0
    for n in (2, 1, 64, 83):
        rd, pos, q = t.put(u.padded(rows[at:at + n], ld)), pos_dev(at), t.new(n, nq)
        t.attn.gate, t.attn.ldgate, t.attn.gate_f32 = rd.data_ptr() + nq * (4 if f32 else 2), ld, f32
        hip.gqa_rows_dev(t.attn, rd, ld, f32, f32, pos, n, q, nq)
        hip.conv_keep_dev(rd, ld, f32, nq, 3, ring, pos, n)
        out, no = t.new(n, heads * t.vdimp), heads * t.vdimp
        if f32:
            scratch = u.zeros_f32(hip.gqa_scratch_bytes(heads, 1, t.vdimp, n) // 4)
            hip.gqa_any_dev(t.attn, q, nq, True, True, pos, 0, n, scratch)
            hip.gqa_merge_dev(t.attn, pos, 0, n, scratch, out, no, False)
        else:
            hip.gqa_prefill_dev(t.attn, q, nq, at + n, n, out, no)
        t.check(out, at, 1e-5 if f32 else 2e-2)
        at += n
    assert all(np.array_equal(u.host(t.keep[i]), b) for i, b in zip((1, 2), before))


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("nq", [1, 70])
def test_latent_attention_without_a_sink(hip, pkg, f32, nq):
    """queries out of wider rows, no sink: decode records and the prompt's form"""
    g = rng(nq, 6)
    L, heads, dim, rot, vdim, rank, scale = 150, 3, 24, 12, 40, 72, 0.3
    dimp, rotp, vdimp, ldc, cap = 32, 32, 64, 128, 192
    qd, ldq = dimp + rotp, 3 * 64 + 128
    store = (lambda a: a.astype(np.float32)) if f32 else u.rounded
    q, c, kr = store(g.standard_normal((nq, heads, dim + rot))), store(g.standard_normal((L, rank))), store(g.standard_normal((L, rot)))
    uk, uv = u.rounded(g.standard_normal((heads, dim, rank)) / np.sqrt(rank)), u.rounded(g.standard_normal((heads, vdim, rank)) / np.sqrt(rank))
    spec = {"dims": rot, "base": 500.0}
    f, _ = so.rotary_frequencies(spec)
    angle = np.arange(cap)[:, None] * f
    cos, sin = u.dev_f32(np.cos(angle)), u.dev_f32(np.sin(angle))
    qr = np.stack([so.rotate(q[i:i + 1, :, dim:].astype(f64), [L - nq + i], spec)[0] for i in range(nq)])
    s = (np.einsum("nhd,hdr,lr->nhl", q[..., :dim].astype(f64), uk.astype(f64), c.astype(f64)) + np.einsum("nhd,ld->nhl", qr, kr.astype(f64))) * scale
    for i in range(nq):
        s[i, :, L - nq + i + 1:] = -np.inf
    e = np.exp(s - s.max(axis=2, keepdims=True))
    want = np.einsum("nhl,lr,hvr->nhv", e / e.sum(axis=2, keepdims=True), c.astype(f64), uv.astype(f64))
    rows = np.zeros((nq, ldq), np.float32)
    for h in range(heads):
        rows[:, h * qd:h * qd + dim], rows[:, h * qd + dimp:h * qd + dimp + rot] = q[:, h, :dim], q[:, h, dim:]
    put, new = (u.dev_f32, u.zeros_f32) if f32 else (u.dev_bf16, u.zeros_bf16)
    cc, cr = np.zeros((cap, ldc), np.float32), np.zeros((cap, rotp), np.float32)
    cc[:L, :rank], cr[:L, :rot] = c, kr
    cd, rd = put(cc), put(cr)
    uvp = np.zeros((heads, vdimp, ldc), np.float32)
    uvp[:, :vdim, :rank] = uv
    attn = pkg.LatentAttention(heads, dimp, qd, vdimp, rank, rot, scale, 0, ptr(cd), ptr(rd), ldc, rotp, cap, ptr(cos), ptr(sin), ldq)
    qabs = np.zeros((nq, heads, ldc), np.float32)
    qabs[..., :rank] = np.einsum("nhd,hdr->nhr", q[..., :dim].astype(f64), uk.astype(f64))
    scratch, out, pos = u.zeros_f32(hip.latent_scratch_bytes(heads, ldc, nq) // 4), u.zeros_f32(nq, heads * vdimp), pos_dev(L - nq)
    hip.latent_decode_dev(attn, u.dev_f32(rows), u.dev_f32(qabs), pos, 0, nq, f32, scratch)
    hip.latent_merge_dev(attn, u.dev_bf16(uvp), pos, 0, nq, scratch, out, heads * vdimp, False)
    assert u.rms_error(u.host(out).reshape(nq, heads, vdimp)[..., :vdim], want) < (1e-5 if f32 else 1e-2)
    if f32:
        return
    k, vt = np.zeros((cap, heads, dimp), np.float32), np.zeros((heads, vdimp, cap), np.float32)
    k[:L, :, :dim] = np.einsum("lr,hdr->lhd", c.astype(f64), uk.astype(f64))
    vt[:, :vdim, :L] = np.einsum("lr,hvr->hvl", c.astype(f64), uv.astype(f64))
    out = new(nq, heads * vdimp)
    hip.latent_prefill_dev(attn, put(rows), put(k), put(vt), cap, L, nq, out, heads * vdimp)
    assert u.rms_error(u.host(out).reshape(nq, heads, vdimp)[..., :vdim], want) < 2e-2


# ---- experts ---------------------------------------------------------------------------------------------------------------
# experts, groups, keep, top
GROUPED = [(4, 2, 1, 2), (6, 2, 1, 2), (8, 8, 3, 3), (9, 3, 2, 5), (16, 4, 2, 8), (24, 3, 1, 8), (60, 12, 5, 7), (64, 8, 4, 8), (64, 1, 1, 6), (72, 8, 3, 9), (96, 6, 3, 12), (128, 8, 4, 8),
           (160, 8, 3, 6), (256, 8, 4, 8), (320, 10, 4, 20), (1000, 40, 6, 32), (5, 0, 0, 2), (64, 0, 0, 8)]


def grouped(m, experts, groups, keep, top, seed, bias):
    g = rng(m, experts, groups, top, seed, 5)
    z, c = 1.5 * g.standard_normal((m, experts)).astype(np.float32), (bias + g.uniform(-0.3, 0.3, experts)).astype(np.float32)
    if m > 3 and not groups:
        z[3] = 0.25
    return z, c, so.route_in_groups(z.astype(f64), np.eye(experts), c.astype(f64), top, {"count": groups, "keep": keep} if groups else None)


def as_good(got, z, c, groups, keep, top):
    """every token's choice is the restatement's, or one that lies within rounding of it"""
    choice = so.sigmoid(z.astype(f64)) + c
    spec = {"count": groups, "keep": keep} if groups else None
    want, _ = so.route_in_groups(z.astype(f64), np.eye(z.shape[1]), c.astype(f64), top, spec)
    return all(np.array_equal(a, b) or u.group_margins(row, top, spec) < 1e-6 or np.abs(row[a] - row[b]).max() < 1e-6 for a, b, row in zip(got, want, choice))


@pytest.mark.parametrize("bias", [0.0, -3.0])
@pytest.mark.parametrize("experts,groups,keep,top", GROUPED)
def test_grouped_route(hip, pkg, experts, groups, keep, top, bias):
    """also with corrections that make every choice score negative"""
    m = 150
    z, c, (ids, w) = grouped(m, experts, groups, keep, top, 0, bias)
    nb, ldz = hip.experts_plan_bytes(m, experts, top), experts + 2
    ws, cd = u.dev(np.zeros(nb // 4 + 4, np.int32)), u.dev_f32(c)
    plan = hip.experts_plan_make(ws, nb, m, experts, top, 64)
    hip.experts_route_dev(u.dev_f32(u.padded(z, ldz)), ldz, pkg.Router(experts, 0, top, 1.0, 1, cd.data_ptr(), 1, groups, keep), plan)
    raw, base = u.host(ws), ws.data_ptr()
    got = raw[(plan.ids - base) // 4:][:m * top].reshape(m, top)
    assert as_good(got, z, c, groups, keep, top)
    weights = raw[(plan.weights - base) // 4:][:m * top].view(np.float32).reshape(m, top)
    assert u.rms_error(weights, so.sigmoid(np.take_along_axis(z, got.astype(np.int64), 1).astype(f64))) < F32_TOL


def test_equal_groups_and_experts_take_the_lower_index(hip, pkg):
    m, experts, top = 4, 16, 4
    z = np.zeros((m, experts), np.float32)
    z[1, 9], z[2, 4:8], z[3, 15] = 1.0, 0.5, -1.0
    for groups, span in ((4, 4), (8, 2)):
        nb = hip.experts_plan_bytes(m, experts, top)
        ws = u.dev(np.zeros(nb // 4 + 4, np.int32))
        plan = hip.experts_plan_make(ws, nb, m, experts, top, 64)
        hip.experts_route_dev(u.dev_f32(z), experts, pkg.Router(experts, 0, top, 1.0, 1, None, 1, groups, 2), plan)
        got = u.host(ws)[(plan.ids - ws.data_ptr()) // 4:][:m * top].reshape(m, top)
        want, _ = so.route_in_groups(z.astype(f64), np.eye(experts), np.zeros(experts), top, {"count": groups, "keep": 2})
        assert np.array_equal(got, want), span


@pytest.mark.parametrize("experts,groups,keep,top,width,ff,cols0", [(8, 4, 2, 3, 64, 24, 8), (9, 3, 2, 5, 112, 40, 200), (64, 8, 4, 8, 1000, 520, 1032), (64, 8, 4, 8, 2560, 448, 896),
                                                                    (160, 8, 3, 6, 320, 72, 160)])
def test_grouped_experts_of_one_token(hip, pkg, experts, groups, keep, top, width, ff, cols0):
    """choice, gated experts, and a first product whose input is multiplied by a number"""
    g = rng(experts, width, ff, 7)
    z, c, (ids, w) = grouped(1, experts, groups, keep, top, 3, 0.0)
    ldw, ldf, ld0, cols, colf = u.up_to(width, 64), u.up_to(ff, 64), u.up_to(cols0, 64), u.up_to(width, 8), u.up_to(ff, 8)
    up, down = u.rounded(2.0 * g.standard_normal((experts, 2 * ff, width)) / np.sqrt(width)), u.rounded(g.standard_normal((experts, width, ff)) / np.sqrt(ff))
    w0, x, x0 = u.rounded(g.standard_normal((width, cols0)) / np.sqrt(cols0)), g.standard_normal(width).astype(np.float32), g.standard_normal(cols0).astype(np.float32)
    act, idd, y, cd, number = u.zeros_f32(top, ldf), u.dev(np.zeros(64, np.int32)), u.zeros_f32(width), u.dev_f32(c), u.dev_f32([0.37])
    hip.experts_up_dev(u.dev_f32(z[0]), pkg.Router(experts, 0, top, 1.0, 1, cd.data_ptr(), 1, groups, keep), u.dev_f32(u.padded(x, cols)), u.dev_bf16(u.padded(up, ldw)), 2 * ff, cols,
                       ldw, pkg.ACT_SILU | pkg.ACT_GATED, act, ldf, idd)
    assert np.array_equal(u.host(idd)[:top], ids[0])
    want = np.zeros((top, ff))
    for k, e in enumerate(ids[0]):
        h = up[e].astype(f64) @ x
        want[k] = w[0, k] * so.silu(h[0::2]) * h[1::2]
    assert u.rms_error(u.host(act)[:, :ff], want) < F32_TOL
    hip.experts_out_dev(u.dev_f32(x0), u.dev_bf16(u.padded(w0, ld0)), cols0, ld0, None, act, ldf, u.dev_bf16(u.padded(down, ldf)), colf, ldf, idd, top, width, y, x0_scale=number)
    want = 0.37 * (w0.astype(f64) @ x0) + sum(down[e].astype(f64) @ want[k] for k, e in enumerate(ids[0]))
    assert u.rms_error(u.host(y), want) < 2 * F32_TOL
