"""The bf16-weight operators and sequence mixers (include/bitnet_hip.h section 5), one at a time through the C ABI, against the
plain restatement in oracle/stack_oracle.py or f64 numpy."""
import numpy as np
import pytest

from oracle import stack_oracle as so
from tests import stack_util as u

pytestmark = pytest.mark.gpu
F32_TOL, BF_TOL = 3e-6, 6e-3


def rng(*seed):
    return np.random.default_rng(list(seed))


@pytest.mark.parametrize("rows,cols", [(5, 8), (33, 32), (100, 80), (64, 200), (300, 264), (1000, 512), (70, 1000), (2500, 2560), (9000, 1288), (40, 6912), (3, 17000)])
def test_gemv_plain(hip, pkg, rows, cols):
    g = rng(rows, cols)
    ld = u.up_to(cols, 64)
    w, x, b = u.rounded(g.standard_normal((rows, cols))), g.standard_normal(cols).astype(np.float32), g.standard_normal(rows).astype(np.float32)
    y = u.zeros_f32(rows)
    hip.dense_gemv_dev(u.dev_f32(x), u.dev_bf16(u.padded(w, ld)), rows, cols, ld, y, bias=u.dev_f32(b), act0=pkg.ACT_NONE, act1=pkg.ACT_RELU2, act_split=rows // 2)
    want = w.astype(np.float64) @ x + b
    want[rows // 2:] = so.relu_squared(want[rows // 2:])
    assert u.rms_error(u.host(y), want) < F32_TOL


@pytest.mark.parametrize("n", [80, 96, 384, 1001, 2560, 4096, 5000])
@pytest.mark.parametrize("kind", ["norm", "gated", "residual", "first"])
def test_gemv_input_transforms(hip, pkg, n, kind):
    g = rng(n, len(kind))
    rows, ld, cols, eps = 90, u.up_to(n, 64), u.up_to(n, 8), 1e-3
    w = u.rounded(g.standard_normal((rows, n)) / np.sqrt(n))
    x, y, nw, pw, ls, gate = (g.standard_normal(n).astype(np.float32) for _ in range(6))
    out, xo = u.zeros_f32(rows), u.zeros_f32(n)
    wd, xd = u.dev_bf16(u.padded(w, ld)), u.dev_f32(x)
    x64 = x.astype(np.float64)
    if kind == "norm":
        hip.dense_gemv_dev(xd, wd, rows, cols, ld, out, kind=pkg.IN_NORM, eps=eps, weight=u.dev_f32(nw), n=n, act0=pkg.ACT_SILU)
        want = so.silu(w @ so.norm_plain(x64, nw, eps))
    elif kind == "gated":
        hip.dense_gemv_dev(xd, wd, rows, cols, ld, out, kind=pkg.IN_NORM, eps=eps, weight=u.dev_f32(nw), gate=u.dev_f32(gate), n=n, mean_n=n - 7, act0=pkg.ACT_SIGMOID)
        want = so.sigmoid(w @ (x64 / np.sqrt((x64 ** 2).sum() / (n - 7) + eps) * nw * gate))
    elif kind == "first":
        hip.dense_gemv_dev(xd, wd, rows, cols, ld, out, kind=pkg.IN_RESIDUAL_NORM, eps=eps, weight_offset=1.0, weight=u.dev_f32(nw), n=n)
        want = w @ so.norm_around_zero(x64, nw, eps)
    else:
        hip.dense_gemv_dev(xd, wd, rows, cols, ld, out, kind=pkg.IN_RESIDUAL_NORM, eps=eps, weight_offset=1.0, weight=u.dev_f32(nw), res=u.dev_f32(y),
                           post_weight=u.dev_f32(pw), scale=u.dev_f32(ls), x_out=xo, n=n)
        x2 = x64 + ls * so.norm_around_zero(y.astype(np.float64), pw, eps)
        want = w @ so.norm_around_zero(x2, nw, eps)
        assert u.rms_error(u.host(xo), x2) < F32_TOL
    assert u.rms_error(u.host(out), want) < F32_TOL


@pytest.mark.parametrize("heads,rows,cols", [(3, 64, 32), (5, 128, 96), (2, 512, 128)])
def test_gemv_batched(hip, heads, rows, cols):
    g = rng(heads, rows)
    ld, step = u.up_to(cols, 64), cols + 32
    w, x = u.rounded(g.standard_normal((heads, rows, cols))), g.standard_normal((heads, step)).astype(np.float32)
    y = u.zeros_f32(heads, rows)
    hip.dense_gemv_dev(u.dev_f32(x), u.dev_bf16(u.padded(w, ld)), rows, cols, ld, y, batch=heads, w_batch=rows * ld, x_batch=step, y_batch=rows)
    assert u.rms_error(u.host(y), np.einsum("hrc,hc->hr", w.astype(np.float64), x[:, :cols])) < F32_TOL


@pytest.mark.parametrize("m,n,k", [(1, 5, 64), (2, 130, 128), (127, 128, 64), (128, 129, 192), (300, 417, 320), (257, 1000, 512), (1030, 258, 2560)])
@pytest.mark.parametrize("f32", [False, True])
def test_matmul(hip, pkg, m, n, k, f32):
    g = rng(m, n, k)
    a, w, b = u.rounded(g.standard_normal((m, k))), u.rounded(g.standard_normal((n, k)) / np.sqrt(k)), g.standard_normal(n).astype(np.float32)
    if f32:
        a = g.standard_normal((m, k)).astype(np.float32)
    ad, wd = (u.dev_f32(a) if f32 else u.dev_bf16(a)), u.dev_bf16(w)
    want = a.astype(np.float64) @ w.T.astype(np.float64) + b
    want[:, n // 3:] = so.silu(want[:, n // 3:])
    for c_f32 in (True, False):
        ldc = n + 3
        c = u.zeros_f32(m, ldc) if c_f32 else u.zeros_bf16(m, ldc)
        hip.dense_matmul_dev(ad, k, f32, wd, k, m, n, k, c, ldc, c_f32, bias=u.dev_f32(b), act0=pkg.ACT_NONE, act1=pkg.ACT_SILU, act_split=n // 3)
        got = u.host(c)
        assert u.rms_error(got[:, :n], want) < (F32_TOL if c_f32 else 3e-3)
        assert not got[:, n:].any()


def test_matmul_batched_f32(hip):
    g = rng(9)
    heads, m, n, k, step = 3, 70, 64, 64, 96
    a, w = g.standard_normal((m, heads * step)).astype(np.float32), u.rounded(g.standard_normal((heads, n, k)))
    c = u.zeros_f32(m, heads * n)
    hip.dense_matmul_dev(u.dev_f32(a), heads * step, True, u.dev_bf16(w), k, m, n, k, c, heads * n, True, batch=heads, a_batch=step, w_batch=n * k, c_batch=n)
    want = np.concatenate([a[:, h * step:h * step + k].astype(np.float64) @ w[h].T for h in range(heads)], axis=1)
    assert u.rms_error(u.host(c), want) < F32_TOL


@pytest.mark.parametrize("width", [96, 1000, 2560, 4096, 5000])
def test_residual_norm_rows(hip, width):
    g = rng(width)
    m, ldh, eps = 5, u.up_to(width, 64), 1e-2
    x, y = (g.standard_normal((m, width)).astype(np.float32) for _ in range(2))
    pw, ls, nw = (g.standard_normal(width).astype(np.float32) for _ in range(3))
    xd, h = u.dev_f32(x), u.zeros_f32(m, ldh)
    hip.residual_norm_rows_dev(xd, m, width, eps, 1.0, y=u.dev_f32(y), ldy=width, post_weight=u.dev_f32(pw), scale=u.dev_f32(ls), next_weight=u.dev_f32(nw), h=h, ldh=ldh)
    want = x + ls * so.norm_around_zero(y.astype(np.float64), pw, eps)
    assert u.rms_error(u.host(xd), want) < F32_TOL
    assert u.rms_error(u.host(h)[:, :width], so.norm_around_zero(want, nw, eps)) < F32_TOL
    hb = u.zeros_bf16(m, ldh) + 7
    hip.residual_norm_rows_dev(xd, m, width, eps, 1.0, next_weight=u.dev_f32(nw), h=hb, ldh=ldh, h_f32=False)
    assert u.rms_error(u.host(hb)[:, :width], so.norm_around_zero(want, nw, eps)) < BF_TOL
    assert not u.host(hb)[:, width:].any()


# ---- latent attention --------------------------------------------------------------------------------------------------
class Latent:
    """random queries, cache and weights of one latent attention, in the library's layouts, and its output by definition"""

    def __init__(self, pkg, L, nq, heads, dim, rot, vdim, rank, f32, seed=0, spike=None):
        g = rng(L, nq, heads, dim, seed)
        self.L, self.nq, self.heads, self.f32 = L, nq, heads, f32
        store = (lambda a: a.astype(np.float32)) if f32 else u.rounded
        self.dimp, self.rotp, self.vdimp, self.ldc, self.cap = u.up_to(dim, 32), u.up_to(rot, 32), u.up_to(vdim, 32), u.up_to(rank, 64), u.up_to(L, 64)
        self.qd = self.dimp + self.rotp
        q = store(g.standard_normal((nq, heads, dim + rot)))
        c, kr = store(g.standard_normal((L, rank))), store(g.standard_normal((L, rot)))
        uk, uv = u.rounded(g.standard_normal((heads, dim, rank)) / np.sqrt(rank)), u.rounded(g.standard_normal((heads, vdim, rank)) / np.sqrt(rank))
        sink = g.standard_normal(heads).astype(np.float32)
        spec = {"dims": rot, "base": 5000.0, "scaling": {"factor": 4.0, "original": 64, "fast": 16.0, "slow": 1.0}}
        f, mult = so.rotary_frequencies(spec)
        ang = np.arange(self.cap)[:, None] * f
        self.cos, self.sin = u.dev_f32(np.cos(ang) * mult), u.dev_f32(np.sin(ang) * mult)
        scale = 0.2
        if spike is not None:  # one key whose score stands far above the others for every query and head
            c[spike] = store(c[spike] * 0)
            qr = np.stack([so.rotate(q[i:i + 1, :, dim:], [L - nq + i], spec)[0] for i in range(nq)])
            v = qr.mean(axis=(0, 1))
            kr[spike] = store(v / np.linalg.norm(v) * 6)
            q[:, :, dim:] = q[:1, :1, dim:]
            qr = np.stack([so.rotate(q[i:i + 1, :, dim:], [L - nq + i], spec)[0] for i in range(nq)])
            kr[spike] = store(qr[0, 0] / np.linalg.norm(qr[0, 0]) * 30)
        q64 = q.astype(np.float64)
        qr = np.stack([so.rotate(q64[i:i + 1, :, dim:], [L - nq + i], spec)[0] for i in range(nq)])
        out = np.zeros((nq, heads, vdim))
        for h in range(heads):
            k, v = c.astype(np.float64) @ uk[h].T, c.astype(np.float64) @ uv[h].T
            s = (q64[:, h, :dim] @ k.T + qr[:, h] @ kr.T.astype(np.float64)) * scale
            for i in range(nq):
                n = L - nq + i + 1
                top = max(s[i, :n].max(), sink[h])
                e = np.exp(s[i, :n] - top)
                out[i, h] = e @ v[:n] / (e.sum() + np.exp(sink[h] - top))
        self.want = out
        dq = np.zeros((nq, heads, self.qd), np.float32)
        dq[:, :, :dim], dq[:, :, self.dimp:self.dimp + rot] = q[:, :, :dim], q[:, :, dim:]
        self.q = dq
        put = u.dev_f32 if f32 else u.dev_bf16
        cache = np.zeros((self.cap, self.ldc), np.float32)
        cache[:L, :rank] = c
        rc = np.zeros((self.cap, self.rotp), np.float32)
        rc[:L, :rot] = kr
        self.c_host, self.cache, self.rcache, self.sink = cache, put(cache), put(rc), u.dev_f32(sink)
        self.uv_host = np.zeros((heads, self.vdimp, self.ldc), np.float32)
        self.uv_host[:, :vdim, :rank] = uv
        self.uk_host = np.zeros((heads, self.dimp, self.ldc), np.float32)
        self.uk_host[:, :dim, :rank] = uk
        self.vdim = vdim
        self.attn = pkg.LatentAttention(heads, self.dimp, self.qd, self.vdimp, rank, rot, scale, self.sink.data_ptr(), self.cache.data_ptr(), self.rcache.data_ptr(),
                                        self.ldc, self.rotp, self.cap, self.cos.data_ptr(), self.sin.data_ptr())

    def decode(self, hip):
        qabs = np.einsum("nhd,hdc->nhc", self.q[:, :, :self.dimp].astype(np.float64), self.uk_host)
        scratch = u.zeros_f32(hip.latent_scratch_bytes(self.heads, self.ldc, self.nq) // 4)
        pos, out = u.dev(np.array([self.L - self.nq], np.int32)), u.zeros_f32(self.nq, self.heads, self.vdimp)
        hip.latent_decode_dev(self.attn, u.dev_f32(self.q), u.dev_f32(qabs), pos, 0, self.nq, self.f32, scratch)
        hip.latent_merge_dev(self.attn, u.dev_bf16(self.uv_host), pos, 0, self.nq, scratch, out, self.heads * self.vdimp, False)
        return u.host(out)

    def prefill(self, hip):
        k = np.einsum("lc,hdc->lhd", self.c_host, self.uk_host)
        vt = np.einsum("lc,hvc->hvl", self.c_host, self.uv_host)
        out = u.zeros_bf16(self.nq, self.heads, self.vdimp)
        hip.latent_prefill_dev(self.attn, u.dev_bf16(self.q), u.dev_bf16(k), u.dev_bf16(vt), self.cap, self.L, self.nq, out, self.heads * self.vdimp)
        return u.host(out)

    def check(self, got, tol):
        assert u.rms_error(got[:, :, :self.vdim], self.want) < tol
        assert not got[:, :, self.vdim:].any()


SHAPES = [(4, 32, 32, 32, 64), (3, 24, 16, 40, 72), (17, 128, 64, 128, 512), (20, 64, 32, 100, 320), (2, 180, 40, 256, 200)]


@pytest.mark.parametrize("L", [1, 2, 63, 64, 65, 700])
@pytest.mark.parametrize("shape", SHAPES)
@pytest.mark.parametrize("f32", [True, False])
def test_latent_decode(hip, pkg, shape, L, f32):
    t = Latent(pkg, L, 1, *shape, f32)
    t.check(t.decode(hip), 1e-5 if f32 else 1e-4)  # (bf16 cache values are exact inputs here: only the query's split is rounded)


@pytest.mark.parametrize("f32", [True, False])
def test_latent_decode_long_and_several_queries(hip, pkg, f32):
    t = Latent(pkg, 8500, 2, 5, 32, 32, 32, 64, f32)  # more tiles than records
    t.check(t.decode(hip), 1e-5 if f32 else 1e-4)
    t = Latent(pkg, 130, 70, *SHAPES[1], f32)
    t.check(t.decode(hip), 1e-5 if f32 else 1e-4)


def test_latent_decode_large_latent_in_bf16(hip, pkg):
    t = Latent(pkg, 150, 2, 3, 64, 64, 32, 900, False)  # beyond the matrix-core form's latent
    t.check(t.decode(hip), 1e-4)


@pytest.mark.parametrize("L,nq", [(1, 1), (2, 2), (64, 64), (65, 2), (129, 129), (300, 37), (700, 700)])
@pytest.mark.parametrize("shape", SHAPES + [(9, 96, 96, 64, 128), (1, 160, 96, 16, 64)])
def test_latent_prefill(hip, pkg, shape, L, nq):
    t = Latent(pkg, L, nq, *shape, False)
    t.check(t.prefill(hip), 1.5e-2 if L > 1 else 4e-2)  # (one key: its rounded score decides its share against the sink)


@pytest.mark.parametrize("spike", [0, 1, 63, 64, 127, 128, 500, 639])
def test_latent_attention_finds_one_key(hip, pkg, spike):
    """one key takes nearly all of the weight, wherever it lies"""
    t = Latent(pkg, 640, 1, *SHAPES[0], False, seed=spike, spike=spike)
    v = np.abs(t.want).max()
    assert v < 0.2  # (its value vector is zero: a kernel that misses it returns an average of the others)
    assert np.abs(t.decode(hip)[:, :, :t.vdim] - t.want).max() < 1e-3
    assert np.abs(t.prefill(hip)[:, :, :t.vdim] - t.want).max() < 5e-3


@pytest.mark.parametrize("f32", [True, False])
def test_latent_rows(hip, pkg, f32):
    g = rng(5)
    m, qr, kr, rot, pos0, eps = 7, 56, 72, 16, 61, 1e-2
    ldq, ldc, ldr, cap = 64, 128, 32, 128
    z, qw, kw = g.standard_normal((m, qr + kr + rot)).astype(np.float32), g.standard_normal(qr).astype(np.float32), g.standard_normal(kr).astype(np.float32)
    spec = {"dims": rot, "base": 300.0}
    f, _ = so.rotary_frequencies(spec)
    ang = np.arange(cap)[:, None] * f
    new = u.zeros_f32 if f32 else u.zeros_bf16
    cq, c, r = new(m, ldq), new(cap, ldc), new(cap, ldr)
    keep = [u.dev_f32(v) for v in (z, qw, kw, np.cos(ang), np.sin(ang))] + [u.dev(np.array([pos0], np.int32))]
    a = [t.data_ptr() for t in keep]
    rows = pkg.LatentRows(a[0], z.shape[1], qr, kr, rot, a[1], a[2], eps, cq.data_ptr(), ldq, c.data_ptr(), r.data_ptr(), ldc, ldr, a[3], a[4], a[5])
    hip.latent_rows_dev(rows, m, f32)
    z64, tol = z.astype(np.float64), F32_TOL if f32 else BF_TOL
    assert u.rms_error(u.host(cq)[:, :qr], so.norm_plain(z64[:, :qr], qw, eps)) < tol and not u.host(cq)[:, qr:].any()
    assert u.rms_error(u.host(c)[pos0:pos0 + m, :kr], so.norm_plain(z64[:, qr:qr + kr], kw, eps)) < tol
    assert u.rms_error(u.host(r)[pos0:pos0 + m, :rot], so.rotate(z64[:, qr + kr:], range(pos0, pos0 + m), spec)) < tol
    got = u.host(c)
    assert not got[:pos0].any() and not got[pos0 + m:].any() and not got[:, kr:].any()


# ---- linear attention --------------------------------------------------------------------------------------------------
def linear_case(n, heads, dim, vdim, decay, seed=0):
    g = rng(n, heads, dim, seed)
    dimp, vdimp = u.up_to(dim, 32), u.up_to(vdim, 32)
    q, k, v = u.rounded(g.standard_normal((n, heads, dim))), u.rounded(g.standard_normal((n, heads, dim))), u.rounded(g.standard_normal((n, heads, vdim)))
    S = g.standard_normal((heads, dim, vdim))
    state = np.zeros((heads, vdimp, dimp), np.float32)
    state[:, :vdim, :dim] = S.transpose(0, 2, 1)
    S = state[:, :vdim, :dim].transpose(0, 2, 1).astype(np.float64)
    out = np.zeros((n, heads, vdim))
    for t in range(n):
        S = np.array(decay)[:, None, None] * S + k[t].astype(np.float64)[:, :, None] * v[t].astype(np.float64)[:, None, :]
        out[t] = np.einsum("hdv,hd->hv", S, q[t].astype(np.float64))
    qkv = np.concatenate([u.padded(q, dimp).reshape(n, -1), u.padded(k, dimp).reshape(n, -1), u.padded(v, vdimp).reshape(n, -1)], axis=1)
    pw = np.array([[d ** i for i in range(129)] for d in decay], np.float32)
    return dimp, vdimp, qkv, state, pw, out, S


LINEAR = [(1, 3, 40, 24), (2, 2, 64, 64), (127, 2, 32, 96), (128, 6, 64, 64), (129, 2, 128, 128), (300, 1, 200, 160), (521, 2, 96, 32)]


@pytest.mark.parametrize("n,heads,dim,vdim", LINEAR)
@pytest.mark.parametrize("form", ["recurrent", "chunked"])
def test_linear_attention(hip, form, n, heads, dim, vdim):
    decay = [0.5, 0.999, 1.0, 0.0, 0.9, 0.97][:heads]
    dimp, vdimp, qkv, state, pw, want, S = linear_case(n, heads, dim, vdim, decay)
    st, out, pd = u.dev_f32(state), u.zeros_f32(n, heads, vdimp), u.dev_f32(pw)
    if form == "recurrent":
        hip.linear_recurrent_dev(u.dev_f32(qkv), qkv.shape[1], n, heads, dimp, vdimp, pd, st, out, heads * vdimp)
    else:
        nb = hip.linear_workspace_bytes(n, heads, dimp, vdimp)
        hip.linear_chunked_dev(u.dev_bf16(qkv), qkv.shape[1], n, heads, dimp, vdimp, pd, st, out, heads * vdimp, u.zeros_f32(nb // 4), nb)
    got, gs = u.host(out), u.host(st)
    tol = 1e-5 if form == "recurrent" else 1e-4
    for h in range(heads):
        assert u.rms_error(got[:, h, :vdim], want[:, h]) < tol, (h, decay[h])
        assert u.rms_error(gs[h, :vdim, :dim].T, S[h]) < tol, (h, decay[h])
    assert not got[:, :, vdim:].any()


def test_linear_attention_forms_hand_the_state_over(hip):
    """portions of every size through both forms: the state carries"""
    heads, dim, vdim, n = 2, 64, 32, 400
    dimp, vdimp, qkv, state, pw, want, _ = linear_case(n, heads, dim, vdim, [0.95, 0.999])
    st, pd, got, at = u.dev_f32(state), u.dev_f32(pw), [], 0
    for size in (2, 1, 130, 3, 128, 1, 127, 8):
        out, part = u.zeros_f32(size, heads, vdimp), qkv[at:at + size]
        if size == 1:
            hip.linear_recurrent_dev(u.dev_f32(part), qkv.shape[1], size, heads, dimp, vdimp, pd, st, out, heads * vdimp)
        else:
            nb = hip.linear_workspace_bytes(size, heads, dimp, vdimp)
            hip.linear_chunked_dev(u.dev_bf16(part), qkv.shape[1], size, heads, dimp, vdimp, pd, st, out, heads * vdimp, u.zeros_f32(nb // 4), nb)
        got.append(u.host(out))
        at += size
    assert at == n and u.rms_error(np.concatenate(got)[:, :, :vdim], want) < 1e-4


def test_gated_norm_rows(hip):
    g = rng(3)
    m, n, mean_n, ldh, eps = 4, 96, 80, 128, 1e-2
    o, w, gate = g.standard_normal((m, n)).astype(np.float32), g.standard_normal(n).astype(np.float32), g.standard_normal((m, 200)).astype(np.float32)
    h = u.zeros_f32(m, ldh) + 1
    hip.gated_norm_rows_dev(u.dev_f32(o), n, u.dev_f32(w), u.dev_f32(gate), 200, eps, True, m, n, mean_n, h, ldh, True)
    o64 = o.astype(np.float64)
    want = o64 / np.sqrt((o64 ** 2).sum(1, keepdims=True) / mean_n + eps) * w * gate[:, :n]
    assert u.rms_error(u.host(h)[:, :n], want) < F32_TOL and not u.host(h)[:, n:].any()
