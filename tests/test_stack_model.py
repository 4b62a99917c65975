"""Whole mixer-stack models through the framework's own entry points (open by path, prompt portions, captured single-token steps,
greedy generation), against oracle/stack_oracle.py on small random models."""
import numpy as np
import pytest

from oracle import stack_oracle as so
from tests import stack_util as u

pytestmark = pytest.mark.gpu

YARN = {"factor": 6.0, "original": 48, "fast": 8.0, "slow": 1.0}
# small models that differ in everything a configuration can say; none of the sizes is a multiple the kernels would like
MODELS = {
    "latent_only": u.lasapel([u.latent_layer(ff=70)], width=96, vocab=130),
    "latent_without_ff": u.lasapel([u.latent_layer(heads=1, dim=8, rot_dim=2, vdim=8, q_rank=8, kv_rank=8, base=50.0)], width=40, vocab=33, eps=1e-3),
    "lightning_only": u.lasapel([u.lightning_layer()], width=72, vocab=90),
    "lightning_with_ff": u.lasapel([u.lightning_layer(heads=3, dim=24, vdim=72, decay=[1.0, 0.5, 0.0], ff=88)], width=136, vocab=101),
    "mixed": u.lasapel([u.lightning_layer(heads=5, dim=16, vdim=16, ff=48), u.latent_layer(heads=5, scaling=YARN, ff=200), u.lightning_layer(),
                        u.latent_layer(heads=2, dim=48, vdim=24, q_rank=24, kv_from=1, scaling=YARN), u.latent_layer(kv_rank=24, scale=0.3, ff=64)],
                       width=152, vocab=190),
    "wide_heads": u.lasapel([u.latent_layer(heads=2, dim=100, rot_dim=60, vdim=140, q_rank=120, kv_rank=200, scaling=dict(YARN, factor=1.5, slow=2.0), ff=33),
                             u.lightning_layer(heads=1, dim=200, vdim=136)], width=200, vocab=64),
    "huge_heads": u.lasapel([u.latent_layer(heads=1, dim=230, rot_dim=40, vdim=270, q_rank=40, kv_rank=600), u.lightning_layer(heads=1, dim=290, vdim=48)],
                            width=88, vocab=70),
    # layers side by side with experts, a loop around two kinds of mixer, a layer without feed-forward
    "mimolix": u.mimolix([u.delta_layer(mlp=u.expert_mlp()), u.attention_layer(mlp=u.expert_mlp(experts=5, top=1, ff=40, scale=0.8)),
                          u.delta_layer(heads=3, kv_heads=3, dim=40, vdim=24, conv=2), u.attention_layer(heads=2, kv_heads=1, dim=36, vdim=12, every=50, mlp=u.expert_mlp())],
                         width=120, vocab=170, loop=(1, 3, 2)),
    "mimolix_delta": u.mimolix([u.delta_layer(heads=6, kv_heads=1, dim=8, vdim=64, conv=1, mlp=u.expert_mlp(experts=9, top=9, ff=16, shared=0))], width=90, vocab=101, mult=1.0,
                               embed=1.0, loop=(0, 1, 3)),
    "mimolix_attention": u.mimolix([u.attention_layer(heads=5, kv_heads=5, dim=64, vdim=8, coef=0.0, mlp=u.expert_mlp(experts=70, top=5, ff=8, shared=72))], width=200, vocab=64,
                                   eps=1e-3),
    "mimolix_wide": u.mimolix([u.attention_layer(heads=20, kv_heads=1, dim=150, vdim=200, scale=0.1), u.delta_layer(heads=2, kv_heads=1, dim=130, vdim=230, conv=3),
                               u.delta_layer(heads=2, kv_heads=2, dim=100, vdim=160, mlp=u.expert_mlp(experts=4, top=2, ff=100, shared=130))], width=136, vocab=77),
    "mimolix_huge": u.mimolix([u.attention_layer(heads=2, kv_heads=2, dim=300, vdim=270, scale=0.05), u.attention_layer(heads=4, kv_heads=2, dim=8, vdim=300)], width=64, vocab=50),
    # chunks of several sizes, banded and plain rotation, all kinds of feed-forward and none
    "lurepel": u.lurepel([u.chunk_layer(mlp=u.gated_mlp(), scaling=u.BANDS), u.chunk_layer(heads=4, kv_heads=1, dim=36, dims=36, chunk=64, mlp=u.corrected_mlp()),
                          u.chunk_layer(chunk=150, scaling=dict(u.BANDS, factor=2.0, original=40)),
                          u.chunk_layer(heads=5, kv_heads=5, dim=16, dims=2, chunk=100, mlp=u.corrected_mlp(experts=5, identity=1, top=4, ff=72))], width=120, vocab=170),
    "lurepel_identities": u.lurepel([u.chunk_layer(heads=3, kv_heads=1, dim=64, dims=32, chunk=1, mlp=u.corrected_mlp(experts=2, identity=6, top=5, ff=16)),
                                     u.chunk_layer(chunk=7, mlp=u.corrected_mlp(experts=1, identity=9, top=1, ff=130))], width=90, vocab=101, eps=1e-3),
    "lurepel_dense": u.lurepel([u.chunk_layer(heads=2, kv_heads=2, dim=128, dims=128, chunk=1000, mlp=u.gated_mlp(71)), u.chunk_layer(dims=0, mlp=u.gated_mlp(8))], width=77, vocab=64),
    "lurepel_wide": u.lurepel([u.chunk_layer(heads=20, kv_heads=1, dim=150, dims=64, chunk=40, scale=0.1, mlp=u.corrected_mlp(experts=70, identity=30, top=20, ff=8))],
                              width=200, vocab=77),
    "lurepel_huge": u.lurepel([u.chunk_layer(heads=4, kv_heads=2, dim=300, dims=210, chunk=33, scale=0.05, scaling=u.BANDS, mlp=u.corrected_mlp(experts=4, identity=0, top=4, ff=100))],
                              width=64, vocab=50),
    # windows of several sizes and none, convolutions of one to five taps, another layer's keys under another window, every kind of feed-forward and none
    "sipelorn": u.sipelorn([u.window_layer(mlp=u.xielu_mlp()), u.direct_latent_layer(scaling=u.YARN, mlp=u.grouped_mlp()),
                            u.window_layer(kv_from=0, window=100, taps=2, scale=0.4, mlp=u.grouped_mlp(experts=6, groups=(2, 1), top=2, ff=72, shared=24)),
                            u.window_layer(heads=5, kv_heads=1, dim=36, vdim=16, window=0, taps=4), u.direct_latent_layer(heads=2, rot_dim=2, kv_rank=24),
                            u.window_layer(heads=10, kv_heads=1, dim=36, vdim=16, window=64, taps=5, kv_from=3, mlp=u.xielu_mlp(9))], vocab=170),
    "sipelorn_narrow": u.sipelorn([u.window_layer(heads=1, kv_heads=1, dim=8, vdim=8, window=1, taps=1, mlp=u.grouped_mlp(experts=9, groups=(3, 3), top=9, ff=16, shared=0)),
                                   u.direct_latent_layer(heads=1, dim=8, rot_dim=2, vdim=8, kv_rank=8, base=50.0, mlp=u.grouped_mlp(experts=4, groups=None, top=1, ff=130, shared=8))],
                                  width=77, vocab=60, eps=1e-3, embed=1.0, pairs=(1, 0, 1), side=1),
    "sipelorn_attention": u.sipelorn([u.window_layer(heads=2, kv_heads=2, dim=128, vdim=64, window=128, taps=2, scale=0.1, mlp=u.xielu_mlp(71)),
                                      u.window_layer(heads=4, kv_heads=4, dim=64, vdim=128, window=65, mlp=u.grouped_mlp(experts=20, groups=(5, 4), top=4, ff=8, shared=16))],
                                     width=90, vocab=64, embed=0.7, pairs=(97, 3, 1), side=70),
    "sipelorn_wide": u.sipelorn([u.window_layer(heads=20, kv_heads=1, dim=150, vdim=200, window=50, taps=3, scale=0.08),
                                 u.direct_latent_layer(heads=2, dim=100, rot_dim=60, vdim=140, kv_rank=200, scaling=dict(u.YARN, factor=1.5), mlp=u.xielu_mlp(100))],
                                width=136, vocab=77, side=8),
    "sipelorn_huge": u.sipelorn([u.window_layer(heads=4, kv_heads=2, dim=300, vdim=270, window=33, taps=4, scale=0.05, mlp=u.xielu_mlp(33)),
                                 u.direct_latent_layer(heads=2, dim=230, rot_dim=40, vdim=270, kv_rank=600, scale=0.07), u.window_layer(heads=6, kv_heads=2, dim=300, vdim=270, window=0,
                                                                                                                                        taps=20, scale=0.05, kv_from=0)], width=64, vocab=50),
    "many_heads": u.lasapel([u.latent_layer(heads=19, dim=16, rot_dim=8, vdim=16, q_rank=40, kv_rank=136, ff=16)], width=64, vocab=500),
}
SEQUENCES = ["mixed", "mimolix", "lurepel", "sipelorn"]  # the models of the tests about sequences
LIMIT = {"float32": 2e-5, "bfloat16": 6e-2}


class Case:
    def __init__(self, pkg, root, name):
        self.config = MODELS[name]
        self.tensors = u.random_tensors(self.config, sum(map(ord, name)))
        self.path = u.save_model(str(root / name), self.config, self.tensors)
        self.pkg, self.models, self.truth = pkg, {}, {}

    def model(self, dtype, max_pos=400):
        if dtype not in self.models:
            self.models[dtype] = self.pkg.open_model(self.path, dtype, max_pos)
        m = self.models[dtype]
        m.reset()
        return m

    def oracle(self, tokens):
        key = bytes(np.asarray(tokens, np.int32))
        if key not in self.truth:
            self.truth[key] = so.forward(self.config, self.tensors, tokens)
        return self.truth[key]


@pytest.fixture(scope="module")
def cases(pkg, hip, tmp_path_factory):
    root, made = tmp_path_factory.mktemp("stack"), {}

    def get(name):
        if name not in made:
            made[name] = Case(pkg, root, name)
        return made[name]

    yield get
    for c in made.values():
        for m in c.models.values():
            m.close()


def tokens_of(config, n, seed=0):
    return np.random.default_rng([n, seed]).integers(0, config["vocab"], n).astype(np.int32)


def error(got, want) -> float:
    """per position: rms of the difference (means taken off) over the rms of all logits; the worst"""
    d = np.asarray(got, np.float64) - want
    d -= d.mean(axis=1, keepdims=True)
    w = want - want.mean(axis=1, keepdims=True)
    return float(np.sqrt((d ** 2).mean(axis=1)).max() / np.sqrt((w ** 2).mean()))


def in_portions(m, tokens, sizes):
    out, at, i = [], 0, 0
    while at < len(tokens):
        n = min(sizes[i % len(sizes)], len(tokens) - at)
        out.append(m.forward(tokens[at:at + n], range(n)))
        at, i = at + n, i + 1
    return np.concatenate(out)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(MODELS))
def test_prompt_and_decoding(cases, name, dtype):
    """the whole prompt at once, and token by token through the cache: every position"""
    c = cases(name)
    t = tokens_of(c.config, 75)
    want = c.oracle(t)[0]
    assert error(c.model(dtype).forward(t, range(len(t))), want) < LIMIT[dtype]
    assert error(in_portions(c.model(dtype), t, [1]), want) < LIMIT[dtype]


@pytest.mark.parametrize("name", SEQUENCES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", [[2], [3, 1, 2], [64, 1], [63, 2, 65], [127, 2, 1, 130], [129], [40, 100, 2, 1, 1]])
def test_portions(cases, dtype, sizes, name):
    c = cases(name)
    t = tokens_of(c.config, 290)
    want = c.oracle(t)[0]
    assert error(in_portions(c.model(dtype), t, sizes), want) < LIMIT[dtype]


@pytest.mark.parametrize("name", SEQUENCES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_first_tokens(cases, dtype, name):
    """sequences of one, two and three tokens: the sink weighs most there, states are empty"""
    c = cases(name)
    for n in (1, 2, 3):
        t = tokens_of(c.config, n, 5)
        want = c.oracle(t)[0]
        assert error(c.model(dtype).forward(t, range(n)), want) < LIMIT[dtype]
        assert error(in_portions(c.model(dtype), t, [1]), want) < LIMIT[dtype]


@pytest.mark.parametrize("name", SEQUENCES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_residual_stream_after_each_layer(cases, pkg, tmp_path, dtype, name):
    """the model cut after each of its layers: the stream ahead of the final norm, from the prompt and from a step"""
    c = cases(name)
    t = tokens_of(c.config, 21)
    for k in range(1, len(c.config["layers"]) + 1):
        config, tensors = dict(c.config, layers=c.config["layers"][:k]), c.tensors
        if config.get("token_side"):
            tensors = dict(tensors, **{"side.embed": tensors["side.embed"][:, :k * config["token_side"]["dim"]]})
        loop = config.pop("loop", None)
        if loop and loop["start"] < k:
            config["loop"] = dict(loop, stop=min(loop["stop"], k))
        after = so.forward(config, tensors, t)[1]
        m = pkg.open_model(u.save_model(str(tmp_path / str(k)), config, tensors), dtype, 64)
        m.feed(t)
        m.prefill(20, with_logits=False)
        assert u.rms_error(m.last_hidden(), after[-1, 19]) < LIMIT[dtype]
        m.run(1)
        assert u.rms_error(m.last_hidden(), after[-1, 20]) < LIMIT[dtype]
        m.close()


@pytest.mark.parametrize("name", SEQUENCES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(cases, dtype, name):
    """300 steps behind a short prompt: several cache tiles, states carried all the way"""
    c = cases(name)
    t = tokens_of(c.config, 310, 3)
    want = c.oracle(t)[0]
    m = c.model(dtype)
    got = [m.forward(t[:10], range(10))] + [m.forward(t[i:i + 1], [0]) for i in range(10, 310)]
    assert error(np.concatenate(got), want) < LIMIT[dtype]


@pytest.mark.parametrize("name", SEQUENCES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_requests_follow_one_another(cases, dtype, name):
    """a slot used again: nothing of the longer sequence before shows in the next one, and a repeat is bit for bit the same"""
    c = cases(name)
    long, short = tokens_of(c.config, 200, 1), tokens_of(c.config, 30, 2)
    m = c.model(dtype)
    first = m.forward(short, range(30))
    for before in (long, long[:65]):
        m.reset()
        m.forward(before, [])
        m.forward(before[:1], [0])
        m.reset()
        assert np.array_equal(m.forward(short, range(30)), first)
    assert error(first, c.oracle(short)[0]) < LIMIT[dtype]


@pytest.mark.parametrize("name", SEQUENCES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_graph_replays_match_eager_steps(cases, dtype, name):
    c = cases(name)
    t = tokens_of(c.config, 40, 4)
    out = []
    for use_graph in (True, False):
        m = c.model(dtype)
        m.feed(t)
        m.prefill(20, with_logits=False)
        rows = []
        for _ in range(20):
            m.run(1, use_graph=use_graph)
            rows.append(m.last_logits())
        out.append(np.stack(rows))
    assert np.array_equal(out[0], out[1])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["mixed", "lightning_only", "many_heads", "mimolix", "mimolix_delta", "lurepel", "lurepel_identities", "sipelorn", "sipelorn_narrow"])
def test_greedy_generation(cases, name, dtype):
    """generate(): each token is the argmax of the oracle's logits over what was generated so far (or as good as it)"""
    c = cases(name)
    p = tokens_of(c.config, 12, 6)
    m = c.model(dtype)
    new = m.generate(p, 16)
    want = c.oracle(np.concatenate([p, new]))[0]
    spread = np.sqrt(((want - want.mean(axis=1, keepdims=True)) ** 2).mean())
    for i, tok in enumerate(new):
        row = want[len(p) - 1 + i]
        assert row.max() - row[tok] <= 2 * LIMIT[dtype] * spread, (i, tok)
    assert np.array_equal(m.generate(p, 16, use_graph=False), new)
    if dtype == "float32":
        assert sum(want[len(p) - 1 + i].argmax() == tok for i, tok in enumerate(new)) >= 15


def one_key_model(cases_root, pkg, far):
    """One latent layer in which the query of a marked token scores one other marked token far above all others: the value it
    carries must come through however far back it lies."""
    W, V = 32, 40
    layer = u.latent_layer(heads=1, dim=8, rot_dim=2, vdim=8, q_rank=8, kv_rank=8, scale=1.0, base=1e6)
    config = u.lasapel([layer], width=W, vocab=V, eps=1e-6)
    t = u.random_tensors(config, 11)
    t["embed"] = u.rounded(np.random.default_rng(8).standard_normal((V, W)) * 0.05)
    t["embed"][:, 0] = 1.0   # every token
    t["embed"][1, 1] = 6.0   # the token looked for
    t["embed"][2, 2] = 6.0   # the token that looks
    for k in ("dq", "dkv", "uq", "uk"):
        t["l0.mix." + k] *= 0.02
    t["l0.mix.dq"][0, 2] = t["l0.mix.dkv"][0, 1] = 1.0
    t["l0.mix.dq"][1, 0] = t["l0.mix.dkv"][1, 0] = 0.5
    t["l0.mix.dq.norm"][:], t["l0.mix.dkv.norm"][:] = 1.0, 1.0
    t["l0.norm1"][:] = 0.0
    t["l0.mix.uq"][0, 0], t["l0.mix.uk"][0, 0] = 3.0, 3.0
    t = {k: u.rounded(v) for k, v in t.items()}
    return config, t, u.save_model(str(cases_root / f"far{far}"), config, t)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("far", [0, 1, 62, 63, 64, 127, 128, 300, 398])
def test_one_far_key(pkg, hip, tmp_path, dtype, far):
    """with and without the looked-for token: the last position's logits differ as the oracle's do, in a prompt and decoded"""
    config, t, path = one_key_model(tmp_path, pkg, far)
    n = 400
    base = np.random.default_rng(far).integers(3, 40, n).astype(np.int32)
    base[-1] = 2
    marked = base.copy()
    marked[far] = 1
    m = pkg.open_model(path, dtype, n + 8)
    for tokens in (base, marked):
        want = so.forward(config, t, tokens)[0][-1:]
        m.reset()
        assert error(m.forward(tokens, [n - 1]), want) < LIMIT[dtype]
        m.reset()
        m.forward(tokens[:-1], [])
        assert error(m.forward(tokens[-1:], [0]), want) < LIMIT[dtype]
    a, b = so.forward(config, t, base)[0][-1], so.forward(config, t, marked)[0][-1]
    assert u.rms_error(a - a.mean(), b - b.mean()) > 0.2  # the key shows
    m.close()


def one_key_differential(root, far):
    """One differential layer in which a marked token's first map scores one other marked token far above all others; the second map sees them
    all alike."""
    W, V, D = 32, 40, 8
    config = u.mimolix([u.attention_layer(heads=2, kv_heads=1, dim=D, vdim=24, scale=3.0, diff=0.3, every=64)], width=W, vocab=V, eps=1e-6, embed=1.0, mult=1.0)
    t = u.random_tensors(config, 12)
    t["embed"] = u.rounded(np.random.default_rng(9).standard_normal((V, W)) * 0.3)
    t["embed"][:, :3] = 0.0
    t["embed"][1, 1] = 8.0   # the token looked for
    t["embed"][2, 2] = 8.0   # the token that looks
    t["l0.norm1"][:], t["l0.norm1.b"][:] = 1.0, 0.0
    t["l0.norm1.b"][0] = 1.0  # every token
    for k in ("q", "k"):
        t["l0.mix." + k] *= 0.02
        t["l0.mix." + k + ".norm"][:] = 1.0
    for head in range(2):  # map 1 of both heads; keys of other tokens point elsewhere
        t["l0.mix.q"][head * 2 * D, 2] = 4.0
    t["l0.mix.k"][0, 1], t["l0.mix.k"][1, 0] = 4.0, 2.0
    t = {k: u.rounded(v) for k, v in t.items()}
    return config, t, u.save_model(str(root / f"diff{far}"), config, t)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("far", [0, 1, 31, 32, 63, 64, 126, 127, 128, 129, 255, 256, 300, 398])
def test_one_far_key_of_one_map(pkg, hip, tmp_path, dtype, far):
    config, t, path = one_key_differential(tmp_path, far)
    n = 400
    base = np.random.default_rng(far).integers(3, 40, n).astype(np.int32)
    base[-1] = 2
    marked = base.copy()
    marked[far] = 1
    m = pkg.open_model(path, dtype, n + 8)
    for tokens in (base, marked):
        want = so.forward(config, t, tokens)[0][-1:]
        m.reset()
        assert error(m.forward(tokens, [n - 1]), want) < LIMIT[dtype]
        m.reset()
        m.forward(tokens[:-1], [])
        assert error(m.forward(tokens[-1:], [0]), want) < LIMIT[dtype]
    a, b = so.forward(config, t, base)[0][-1], so.forward(config, t, marked)[0][-1]
    assert u.rms_error(a - a.mean(), b - b.mean()) > 0.2  # the key shows
    m.close()


def one_key_chunked(root, chunk):
    """One layer in which a marked token's query scores one other marked token far above all others; queries and keys of unit length point where
    a column says: every token's own way, or the mark's."""
    W, V, D = 32, 40, 8
    config = u.lurepel([u.chunk_layer(heads=2, kv_heads=1, dim=D, scale=1.5, chunk=chunk, dims=2, base=1e6)], width=W, vocab=V, eps=1e-6)
    t = u.random_tensors(config, 13)
    t["embed"] = u.rounded(np.random.default_rng(10).standard_normal((V, W)) * 0.3)
    t["embed"][:, :3] = 0.0
    t["embed"][:, 0] = 2.0   # every token
    t["embed"][1, 1] = 8.0   # the token looked for
    t["embed"][2, 2] = 8.0   # the token that looks
    for k in ("q", "k"):
        t["l0.mix." + k] *= 0.02
    for head in range(2):
        t["l0.mix.q"][head * D + 4, 2] = 4.0
    t["l0.mix.k"][4, 1], t["l0.mix.k"][5, 0] = 4.0, 2.0
    t = {k: u.rounded(v) for k, v in t.items()}
    return config, t, u.save_model(str(root), config, t)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("chunk", [1, 2, 31, 64, 96, 100, 128, 130, 257, 399, 400, 5000])
def test_keys_at_the_edge_of_a_chunk(pkg, hip, tmp_path, dtype, chunk):
    """a marked key at the chunk's first position, beside it and near its query shows; one position ahead of the chunk and far ahead of it, it changes
    no bit -- in whole prompts, at the end of portions and decoded"""
    config, t, path = one_key_chunked(tmp_path, chunk)
    n, p = 400, 399
    first = p // chunk * chunk
    base = np.random.default_rng(chunk).integers(3, 40, n).astype(np.int32)
    base[-1] = 2
    m = pkg.open_model(path, dtype, n + 8)

    def last(tokens):
        rows = []
        for cut in (0, n - 1, n - 2, max(first - 1, 1), min(first + 1, n - 1)):
            m.reset()
            if cut:
                m.forward(tokens[:cut], [])
            rows.append(m.forward(tokens[cut:], [n - cut - 1])[0])
        return np.stack(rows)

    plain = last(base)
    want = so.forward(config, t, base)[0][-1]
    assert error(plain, np.broadcast_to(want, plain.shape)) < LIMIT[dtype]
    for far in {0, first - 2, first - 1, first, first + 1, p - 1}:
        if not 0 <= far < p:
            continue
        marked = base.copy()
        marked[far] = 1
        got, truth = last(marked), so.forward(config, t, marked)[0][-1]
        assert error(got, np.broadcast_to(truth, got.shape)) < LIMIT[dtype]
        if far < first:
            assert np.array_equal(got, plain)
        else:
            assert u.rms_error(truth - truth.mean(), want - want.mean()) > 0.2
    m.close()


def one_key_windowed(root, windows, sharpen):
    """Attention layers in which a marked token's query scores one other marked token far above all others, in the first or only in the last of them (which
    reads the first one's keys); the convolutions pass the current token on unchanged.  sharpen: what the marked score is multiplied by."""
    W, V, D = 32, 40, 8
    layers = [u.window_layer(heads=2, kv_heads=1, dim=D, vdim=24, scale=1.0, window=windows[0], taps=3)]
    if len(windows) > 1:
        layers.append(u.window_layer(heads=2, kv_heads=1, dim=D, vdim=24, scale=1.0, window=windows[1], taps=2, kv_from=0))
    config = u.sipelorn(layers, width=W, vocab=V, eps=1e-6, embed=1.0, side=4)
    t = u.random_tensors(config, 14)
    t["embed"] = u.rounded(np.random.default_rng(11).standard_normal((V, W)) * 0.3)
    t["bigram"] *= 0.1
    t["embed"][:, :2] = 0.0
    t["embed"][1, 0] = 8.0   # the token looked for
    t["embed"][2, 1] = 8.0   # the token that looks
    looks = len(windows) - 1
    for i in range(len(windows)):
        for name in ("l%d.norm1" % i,):
            t[name][:], t[name + ".b"][:] = 1.0, 0.0
        for k in ("q", "k") if i == 0 else ("q",):
            t[f"l{i}.mix.{k}"] *= 0.02
            t[f"l{i}.mix.{k}.b"] *= 0.02
            t[f"l{i}.mix.{k}.conv"][:, :-1] *= 0.05
            t[f"l{i}.mix.{k}.conv"][:, -1] = 1.0
    t["l0.mix.o"] *= 1.0 if looks == 0 else 0.02
    t["l0.side.norm"] *= 1.0 if looks == 0 else 0.02
    for head in range(2):
        t[f"l{looks}.mix.q"][head * D + 4, 1] = sharpen
    t["l0.mix.k"][4, 0] = 1.0
    t = {k: u.rounded(v) for k, v in t.items()}
    return config, t, u.save_model(str(root), config, t)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("windows", [(1,), (2,), (31,), (64,), (100,), (128,), (130,), (257,), (399,), (400,), (5000,), (0,), (9, 150), (200, 64), (3, 0)])
def test_keys_at_the_edge_of_a_window(pkg, hip, tmp_path, dtype, windows):
    """a marked key just inside the window, beside it and near its query shows; just outside it and far outside it changes nothing of what the query sees -- in
    whole prompts, at the end of portions and decoded, also where the keys are another layer's that has a window of its own"""
    config, t, path = one_key_windowed(tmp_path, windows, 6.0)
    n, p = 400, 399
    first = max(0, p - windows[-1] + 1) if windows[-1] else 0
    base = np.random.default_rng(windows[-1]).integers(3, 40, n).astype(np.int32)
    base[-1] = 2
    m = pkg.open_model(path, dtype, n + 8)

    def last(tokens):
        rows = []
        for cut in (0, n - 1, n - 2, max(first - 1, 1), min(first + 1, n - 1)):
            m.reset()
            if cut:
                m.forward(tokens[:cut], [])
            rows.append(m.forward(tokens[cut:], [n - cut - 1])[0])
        return np.stack(rows)

    plain = last(base)
    want = so.forward(config, t, base)[0][-1]
    assert error(plain, np.broadcast_to(want, plain.shape)) < LIMIT[dtype]
    for far in {0, first - 5, first - 4, first - 1, first, first + 1, p - 4}:
        if not 0 <= far < p - 3:  # (the convolution's taps and the pair table bring the neighbours of a token along)
            continue
        marked = base.copy()
        marked[far] = 1
        got, truth = last(marked), so.forward(config, t, marked)[0][-1]
        assert error(got, np.broadcast_to(truth, got.shape)) < LIMIT[dtype]
        shift = u.rms_error(truth - truth.mean(), want - want.mean())
        if far >= first:
            assert shift > 0.1, far
        elif far + 3 < first and len(windows) == 1:
            assert (got == plain).all() and shift < 1e-12
    m.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_penalty_of_the_distance(pkg, hip, tmp_path, dtype):
    """two marked keys of equal scores, one near and one far: the far one's share is what the penalty leaves of it"""
    config, t, path = one_key_windowed(tmp_path, (0,), 3.0)
    t["l0.mix.r1"], t["l0.mix.r2"] = u.rounded(np.array([1.5, 0.4])), u.rounded(np.array([0.05, 2.0]))
    path = u.save_model(str(tmp_path / "p"), config, t)
    n = 400
    m = pkg.open_model(path, dtype, n + 8)
    base = np.random.default_rng(5).integers(3, 40, n).astype(np.int32)
    base[-1] = 2
    for far in (390, 300, 128, 63, 0):
        tokens = base.copy()
        tokens[far] = tokens[395] = 1
        want = so.forward(config, t, tokens)[0][-1:]
        m.reset()
        assert error(m.forward(tokens, [n - 1]), want) < LIMIT[dtype]
        m.reset()
        m.forward(tokens[:-1], [])
        assert error(m.forward(tokens[-1:], [0]), want) < LIMIT[dtype]
    m.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_decoding_across_windows(pkg, hip, tmp_path, dtype):
    """single tokens until the windows have passed over prompt and decoded tokens; portions that end at, ahead of and behind their size; the taps of every
    convolution across each cut"""
    config = u.sipelorn([u.window_layer(window=48, taps=4), u.window_layer(window=65, heads=3, taps=2, kv_from=0, mlp=u.xielu_mlp()), u.direct_latent_layer(scaling=u.YARN)],
                        width=72, vocab=60)
    t = u.random_tensors(config, 42)
    m = pkg.open_model(u.save_model(str(tmp_path), config, t), dtype, 260)
    tokens = tokens_of(config, 250, 12)
    want = so.forward(config, t, tokens)[0]
    for sizes in ([1], [2], [3, 1], [47, 1, 1], [48], [49, 2], [65, 63, 2], [130, 1, 119], [200, 50]):
        m.reset()
        assert error(in_portions(m, tokens, sizes), want) < LIMIT[dtype], sizes
    m.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_pairs_of_tokens(pkg, hip, tmp_path, dtype):
    """a pair table that outweighs the embedding, factors whose products leave 32 bits: the previous token across every cut, the first token's own row"""
    config = u.sipelorn([u.window_layer(window=1, taps=1)], width=40, vocab=90, embed=0.25, pairs=(83, 99999989, 87654321))
    t = u.random_tensors(config, 43)
    t["bigram"] = u.rounded(4.0 * t["bigram"])
    m = pkg.open_model(u.save_model(str(tmp_path), config, t), dtype, 80)
    tokens = tokens_of(config, 60, 13)
    want = so.forward(config, t, tokens)[0]
    for sizes in ([60], [1], [2], [3, 1, 5]):
        m.reset()
        assert error(in_portions(m, tokens, sizes), want) < LIMIT[dtype], sizes
    m.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_decoding_across_chunks(pkg, hip, tmp_path, dtype):
    """single tokens through several chunks, each compared; portions that end inside, at and behind an edge"""
    config = u.lurepel([u.chunk_layer(chunk=48, scaling=u.BANDS), u.chunk_layer(chunk=65, heads=4, kv_heads=2, mlp=u.gated_mlp())], width=72, vocab=60)
    t = u.random_tensors(config, 41)
    m = pkg.open_model(u.save_model(str(tmp_path), config, t), dtype, 260)
    tokens = tokens_of(config, 250, 12)
    want = so.forward(config, t, tokens)[0]
    for sizes in ([1], [47, 1, 1], [48], [49, 2], [65, 63, 2], [130, 1, 119], [200, 50]):
        m.reset()
        assert error(in_portions(m, tokens, sizes), want) < LIMIT[dtype], sizes
    m.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_query_temperature_steps(pkg, hip, tmp_path, dtype):
    """a temperature that changes much from step to step: the positions around every step, prompt and decoded"""
    config = u.mimolix([u.attention_layer(heads=2, kv_heads=1, dim=16, vdim=16, coef=3.0, every=7, scale=0.4)], width=48, vocab=60)
    t = u.random_tensors(config, 21)
    m = pkg.open_model(u.save_model(str(tmp_path), config, t), dtype, 80)
    tokens = tokens_of(config, 64, 11)
    want = so.forward(config, t, tokens)[0]
    assert error(m.forward(tokens, range(64)), want) < LIMIT[dtype]
    m.reset()
    assert error(in_portions(m, tokens, [6, 1, 1]), want) < LIMIT[dtype]
    m.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_slow_decay_carries_the_first_tokens(pkg, hip, tmp_path, dtype):
    """a state that forgets next to nothing over several chunks: the first token still shows in the last logits, in a prompt and decoded"""
    config = u.mimolix([u.delta_layer(heads=2, kv_heads=1, dim=32, vdim=16, conv=3)], width=48, vocab=60, mult=1.0)
    t = u.random_tensors(config, 31)
    t["l0.mix.A_log"][:], t["l0.mix.dt_bias"][:] = -8.0, -2.0
    t["l0.mix.b"][:] = 0.0
    t["l0.mix.b"][:, 0] = u.rounded(np.array([-3.0, -2.0]))  # step sizes well below one, except after a marked token
    t["embed"][:, 0] = 1.0
    t["embed"][1, 0] = -2.0
    t = {k: u.rounded(v) for k, v in t.items()}
    n = 200
    m = pkg.open_model(u.save_model(str(tmp_path), config, t), dtype, n + 8)
    base = np.random.default_rng(1).integers(2, 60, n).astype(np.int32)
    marked = base.copy()
    marked[0] = 1
    rows = []
    for tokens in (base, marked):
        want = so.forward(config, t, tokens)[0]
        rows.append(want[-1] - want[-1].mean())
        m.reset()
        assert error(m.forward(tokens, range(n)), want) < LIMIT[dtype]
        m.reset()
        assert error(in_portions(m, tokens, [70, 1, 2, 64, 1]), want) < LIMIT[dtype]
    assert u.rms_error(rows[0], rows[1]) > 3 * LIMIT[dtype]
    m.close()


def test_errors_leave_a_usable_model(cases, pkg):
    c = cases("lightning_only")
    m = c.model("bfloat16")
    with pytest.raises(pkg.BitNetHipError, match="out of range"):
        m.forward([c.config["vocab"]], [0])
    with pytest.raises(pkg.BitNetHipError, match="wanted place"):
        m.forward([1, 2], [2])
    with pytest.raises(pkg.BitNetHipError, match="overflow"):
        m.forward(np.zeros(401, np.int32), [])
    m.reset()
    t = tokens_of(c.config, 9)
    assert error(m.forward(t, range(9)), c.oracle(t)[0]) < LIMIT["bfloat16"]


def test_command_line_generates(cases, capsys):
    import importlib

    cli = importlib.import_module("bitnet-rs_amd.cli")
    c = cases("mixed")
    p = tokens_of(c.config, 9, 7)
    assert cli.main(["--model", c.path, "--tokens", ",".join(map(str, p)), "--new", "6"]) == 0
    assert capsys.readouterr().out.strip() == ",".join(map(str, c.model("bfloat16").generate(p, 6)))


@pytest.mark.parametrize("name", SEQUENCES)
def test_trace_runner_matches_the_library(cases, pkg, tmp_path, name):
    """the program's logits are those of the same portions through the library, bit for bit"""
    import json
    import subprocess

    c = cases(name)
    prog = pkg._load_build_module().build_program("trace_run")
    a, b = tokens_of(c.config, 20, 8), tokens_of(c.config, 7, 9)
    steps = [("a", a[:12], [0, 11], []), ("a", a[12:13], [], []), ("a", a[13:], [6, 1], ["a"]), ("b", b, [6], ["b"])]
    text = "".join(json.dumps({"step": i, "entries": [{"id": n, "tokens": t.tolist(), "want": w}], "end": e}) + "\n" for i, (n, t, w, e) in enumerate(steps))
    p = subprocess.run([prog, "--model", c.path, "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "64"], input=text, capture_output=True, text=True, timeout=60)
    assert p.returncode == 0 and p.stdout.split("\n")[:4] == [f"done {i}" for i in range(4)], p.stderr
    m = c.model("float32")
    for i, (request, t, w, _) in enumerate(steps):
        if request == "b":
            m.reset()
        want = m.forward(t, w)
        if w:
            assert np.array_equal(np.fromfile(str(tmp_path / f"{i}.f32"), np.float32).reshape(want.shape), want)
    assert not (tmp_path / "1.f32").exists()
