"""Host side of the mixer-stack models without a GPU: registry, configuration and tensor checks, and known values of the plain
restatement the GPU tests compare with."""
import copy
import math
import os
import struct

import numpy as np
import pytest

from oracle import stack_oracle as so
from tests import stack_util as u


@pytest.fixture(scope="module")
def built(pkg):
    pkg._load_build_module().build()
    return pkg


BASE = u.lasapel([u.latent_layer(ff=24), u.lightning_layer()], width=40, vocab=20)


def test_registry_names(built):
    names = built.registered_models()
    assert {"Lasapel", "Mimolix", "Lurepel", "Sipelorn"} <= set(names) and ".gguf" in names


PARALLEL = u.mimolix([u.delta_layer(mlp=u.expert_mlp()), u.attention_layer()], width=40, vocab=20, loop=(0, 1, 2))


@pytest.mark.parametrize("change,message", [
    (lambda c: c.pop("residual_mult"), "residual_mult: missing"),
    (lambda c: c["embedding"].pop("scale"), "embedding.scale: missing"),
    (lambda c: c["loop"].update(stop=3), "loop's range"),
    (lambda c: c["loop"].update(times=0), "loop.times: not an integer"),
    (lambda c: c["layers"][0].update(type="latent_attention"), r"layers\[0\].type: unknown mixer"),
    (lambda c: c["layers"][0]["mixer"].pop("conv"), r"layers\[0\].mixer.conv: missing"),
    (lambda c: c["layers"][0]["mixer"].update(dim=300), "layer 0: delta"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), r"layers\[0\].mlp.kind: unknown"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=7), "layer 0: experts"),
    (lambda c: c["layers"][1]["mixer"].update(kv_heads=4), "layer 1: attention"),
    (lambda c: c["layers"][1]["mixer"]["q_temp"].pop("every"), r"layers\[1\].mixer.q_temp.every: missing"),
    (lambda c: c["layers"][1]["mixer"].pop("diff"), r"layers\[1\].mixer.diff: missing"),
])
def test_bad_parallel_configurations_say_why(built, tmp_path, change, message):
    c = copy.deepcopy(PARALLEL)
    change(c)
    path = u.save_model(str(tmp_path), c, u.random_tensors(PARALLEL, 1))
    with pytest.raises(built.BitNetHipError, match=message):
        built.open_model(path)


CHUNKED = u.lurepel([u.chunk_layer(mlp=u.gated_mlp(), scaling=u.BANDS), u.chunk_layer(mlp=u.corrected_mlp()), u.chunk_layer()], width=40, vocab=20)


@pytest.mark.parametrize("change,message", [
    (lambda c: c["norm"].pop("eps"), "norm.eps: missing"),
    (lambda c: c["layers"][0].update(type="delta"), r"layers\[0\].type: unknown mixer"),
    (lambda c: c["layers"][0]["mixer"].pop("kv_heads"), r"layers\[0\].mixer.kv_heads: missing"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=4), "layer 0: attention: query heads in whole groups"),
    (lambda c: c["layers"][0]["mixer"].update(vdim=24), "layer 0: attention: keys that are the values"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), r"layers\[0\].mixer.mask.size: not an integer"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=22), "layer 0: attention: an even number of rotated columns"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), "layer 0: attention: an even number of rotated columns"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("high"), r"layers\[0\].mixer.rot.scaling.high: missing"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(high=1.5), "bands in order"),
    (lambda c: c["layers"][0]["mlp"].update(kind="sparse"), r"layers\[0\].mlp.kind: unknown"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=9), "layer 1: experts"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(identity=-1), r"layers\[1\].mlp.router.identity: not an integer"),
])
def test_bad_chunked_configurations_say_why(built, tmp_path, change, message):
    c = copy.deepcopy(CHUNKED)
    change(c)
    path = u.save_model(str(tmp_path), c, u.random_tensors(CHUNKED, 1))
    with pytest.raises(built.BitNetHipError, match=message):
        built.open_model(path)


WINDOWED = u.sipelorn([u.window_layer(mlp=u.xielu_mlp()), u.direct_latent_layer(scaling=u.YARN, mlp=u.grouped_mlp()), u.window_layer(kv_from=0)], width=40, vocab=20)


@pytest.mark.parametrize("change,message", [
    (lambda c: c["norm"].pop("eps"), "norm.eps: missing"),
    (lambda c: c["embedding"].pop("scale"), "embedding.scale: missing"),
    (lambda c: c["embedding"]["bigram"].update(buckets=0), "embedding.bigram.buckets: not an integer"),
    (lambda c: c["embedding"]["bigram"].pop("mul_prev"), "embedding.bigram.mul_prev: missing"),
    (lambda c: c["token_side"].update(dim=0), "token_side.dim: not an integer"),
    (lambda c: c["layers"][0].update(type="delta"), r"layers\[0\].type: unknown mixer"),
    (lambda c: c["layers"][0]["mixer"].pop("conv"), r"layers\[0\].mixer.conv: missing"),
    (lambda c: c["layers"][0]["mixer"].update(conv=65), "layer 0: attention: at most 64 taps"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=4), "layer 0: attention: query heads in whole groups"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), r"layers\[0\].mixer.mask.size: not an integer"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=1), "layer 2 reads the cache of layer 1"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=2), "layer 2 reads the cache of layer 2"),
    (lambda c: c["layers"][2]["mixer"].update(dim=24), "layer 2 reads the cache of layer 0"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=10), "rotated part must be even"),
    (lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].pop("fast"), r"layers\[1\].mixer.rot.scaling.fast: missing"),
    (lambda c: c["layers"][0]["mlp"].update(kind="sparse"), r"layers\[0\].mlp.kind: unknown"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=5), "layer 1: experts: equal groups"),
    (lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(count=3), "layer 1: experts: equal groups"),
    (lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(keep=5), "layer 1: experts: equal groups"),
])
def test_bad_windowed_configurations_say_why(built, tmp_path, change, message):
    c = copy.deepcopy(WINDOWED)
    change(c)
    path = u.save_model(str(tmp_path), c, u.random_tensors(WINDOWED, 1))
    with pytest.raises(built.BitNetHipError, match=message):
        built.open_model(path)


def broken(change):
    c = copy.deepcopy(BASE)
    change(c)
    return c


@pytest.mark.parametrize("change,message", [
    (lambda c: c.pop("width"), "width: missing"),
    (lambda c: c.update(width=0), "width: not an integer"),
    (lambda c: c.update(layers=[]), "layers: missing"),
    (lambda c: c["norm"].pop("eps"), "norm.eps: missing"),
    (lambda c: c["layers"][0].update(type="other"), r"layers\[0\].type: unknown mixer"),
    (lambda c: c["layers"][0]["mixer"].pop("kv_rank"), r"layers\[0\].mixer.kv_rank: missing"),
    (lambda c: c["layers"][0]["mixer"]["rot"].pop("base"), r"layers\[0\].mixer.rot.base: missing"),
    (lambda c: c["layers"][0]["mlp"].update(kind="sparse"), r"layers\[0\].mlp.kind: unknown"),
    (lambda c: c["layers"][1]["mixer"].update(decay=["a"]), r"layers\[1\].mixer.decay: not an array of numbers"),
    (lambda c: c.update(architecture="Nothing"), "'Nothing' is not registered"),
])
def test_bad_configurations_say_why(built, tmp_path, change, message):
    path = u.save_model(str(tmp_path), broken(change), u.random_tensors(BASE, 1))
    with pytest.raises(built.BitNetHipError, match=message):
        built.open_model(path)


def test_bad_files_say_why(built, tmp_path):
    with pytest.raises(built.BitNetHipError, match="neither a known file format"):
        built.open_model(str(tmp_path / "nothing"))
    path = u.save_model(str(tmp_path / "m"), BASE, u.random_tensors(BASE, 1))
    with open(os.path.join(path, "config.json"), "w") as f:
        f.write('{"architecture": ')
    with pytest.raises(built.BitNetHipError, match="JSON"):
        built.open_model(path)
    path = u.save_model(str(tmp_path / "n"), BASE, u.random_tensors(BASE, 1))
    st = os.path.join(path, "model.safetensors")
    data = open(st, "rb").read()
    for raw, message in ((data[:4], "cannot be read"), (struct.pack("<Q", 1 << 40) + data[8:], "header longer"), (data[:-2], "bad byte range")):
        open(st, "wb").write(raw)
        with pytest.raises(built.BitNetHipError, match=message):
            built.open_model(path)


def test_no_gpu_is_an_error(built, tmp_path):
    import torch

    if torch.cuda.is_available():
        pytest.skip("GPU present")
    with pytest.raises(built.BitNetHipError, match="no HIP device"):
        built.open_model(u.save_model(str(tmp_path), BASE, u.random_tensors(BASE, 1)))


def test_entry_points_check_shapes_before_any_launch(built):
    hip = built.load()
    bad = [
        (lambda: hip.dense_matmul_dev(8, 96, False, 8, 96, 4, 4, 96, 8, 4, True), "multiple of 64"),
        (lambda: hip.dense_matmul_dev(8, 64, False, 8, 64, 4, 8, 64, 8, 4, True), "dense_matmul"),
        (lambda: hip.dense_gemv_dev(8, 8, 4, 12, 64, 8), "bad shape"),
        (lambda: hip.dense_gemv_dev(8, 8, 4, 64, 64, 8, kind=built.IN_RESIDUAL_NORM, weight=8, res=8, post_weight=8, x_out=8, n=64), "buffer of its own"),
        (lambda: hip.linear_recurrent_dev(8, 96, 1, 1, 32, 24, 8, 8, 8, 32), "bad shape"),
        (lambda: hip.linear_chunked_dev(8, 96, 1, 1, 32, 32, 8, 8, 8, 32, 8, 16), "workspace"),
        (lambda: hip.gqa_step_dev(built.Gqa(6, 4, 2, 16, 32, 16, 32, 128, 1e-5, 0.1, 0.9, 8, 8, 8, 8, 8), 8, 8, 8), "gqa: bad shape"),
        (lambda: hip.gqa_any_dev(built.Gqa(4, 4, 2, 16, 32, 16, 32, 128, 1e-5, 0.1, 0.9, 8, 8, 8, 8, 8), 8, 128, True, True, 8, 0, 1, 8), "gqa_any"),
        (lambda: hip.delta_step_dev(built.Delta(4, 2, 16, 32, 16, 48, 4, 8, 8, 8, 8, 1.0, 1e-6, 1e-5, 8, 8), 8, 8, 8, 8), "delta: bad shape"),
        (lambda: hip.delta_chunked_dev(built.Delta(4, 2, 16, 32, 16, 32, 4, 8, 8, 8, 8, 1.0, 1e-6, 1e-5, 8, 8), 8, 8, 8, 8, 512, 9, 8, 128, 8, 64), "workspace"),
        (lambda: hip.experts_plan_make(16, 1 << 20, 4, 8, 33, 64), "experts_plan"),
        (lambda: hip.gqa_step_dev(built.Gqa(4, 2, 2, 16, 32, 16, 32, 128, 1e-5, 0.1, 0.9, 8, 8, 8, 8, 8, sink=8), 8, 8, 8), "gqa: bad chunk, sink"),
        (lambda: hip.gqa_step_dev(built.Gqa(4, 2, 1, 16, 32, 24, 32, 128, 1e-5, 0.1, 0.9, 8, 8, 8, 8, 8, values_are_keys=1), 8, 8, 8), "gqa: bad chunk, sink"),
        (lambda: hip.gqa_step_dev(built.Gqa(4, 2, 1, 16, 32, 16, 32, 128, 1e-5, 0.1, 0.9, 8, 8, 8, 8, 8, rot_dims=18, rope_cos=8, rope_sin=8), 8, 8, 8), "gqa: bad rotation"),
        (lambda: hip.dense_matmul_dev(8, 64, False, 8, 64, 4, 7, 64, 8, 8, False, act0=built.ACT_GATED), "gated"),
        (lambda: hip.experts_up_dev(8, built.Router(8, 4, 13, 1.0), 8, 8, 16, 8, 64, 0, 8, 16, 8), "bad router"),
        (lambda: hip.experts_up_dev(8, built.Router(8, 4, 2, 1.0), 8, 8, 16, 8, 64, 0, 8, 16, 8), "experts_up"),
        (lambda: hip.experts_up_dev(8, built.Router(8, 0, 2, 1.0), 8, 8, 16, 12, 64, 0, 8, 16, 8), "experts_up"),
        (lambda: hip.experts_out_dev(8, 8, 64, 64, None, 8, 8, 8, 16, 64, 8, 2, 16, 8), "experts_out"),
        (lambda: hip.sum_norm_rows_dev(built.SumRows(x=8, m=1, width=8, h=8, ldh=7)), "sum_norm_rows"),
        (lambda: hip.sum_norm_rows_dev(built.SumRows(x=8, m=1, width=8, h=8, ldh=8, gate=8, ld_gate=7)), "sum_norm_rows: bad gate"),
        (lambda: hip.gqa_step_dev(built.Gqa(4, 2, 2, 16, 32, 16, 32, 128, 1e-5, 0.1, 0.9, 8, 8, 8, 8, 8, far_weight=8, far_rate=8), 8, 8, 8), "gqa: bad window"),
        (lambda: hip.gqa_step_dev(built.Gqa(4, 2, 1, 16, 32, 16, 32, 128, 1e-5, 0.1, 0.9, 8, 8, 8, 8, 8, far_weight=8), 8, 8, 8), "gqa: bad window"),
        (lambda: hip.gqa_step_dev(built.Gqa(4, 2, 1, 16, 32, 16, 32, 128, 1e-5, 0.1, 0.9, 8, 8, 8, 8, 8, gate=8, ldgate=127, gate_columns=1), 8, 8, 8), "gqa: bad chunk"),
        (lambda: hip.gqa_rows_dev(built.Gqa(4, 2, 1, 16, 32, 16, 32, 128, 1e-5, 0.1, 0.9, 8, 8, 8, 8, 8, taps=3, conv=8, ring=8), 16, 256, True, True, 8, 2), "place of the queries"),
        (lambda: hip.gqa_rows_dev(built.Gqa(4, 2, 1, 16, 32, 16, 32, 128, 1e-5, 0.1, 0.9, 8, 8, 8, 8, 8, taps=3), 16, 256, True, True, 8, 2, 8, 128), "gqa: bad window"),
        (lambda: hip.conv_keep_dev(8, 64, True, 65, 3, 8, 8, 2), "conv_keep"),
        (lambda: hip.experts_up_dev(8, built.Router(8, 0, 4, 1.0, groups=4, keep=1), 8, 8, 16, 8, 64, 0, 8, 16, 8), "bad groups"),
        (lambda: hip.experts_up_dev(8, built.Router(8, 0, 2, 1.0, groups=3, keep=1), 8, 8, 16, 8, 64, 0, 8, 16, 8), "bad groups"),
        (lambda: hip.dense_gemv_dev(8, 8, 16, 64, 64, 8, act0=built.ACT_GATED, more=built.Epilogue(pairs=8)), "gated rows come in pairs"),
        (lambda: hip.dense_gemv_dev(8, 8, 16, 64, 64, 8, more=built.Epilogue(conv=8, ring=8, pos=8, taps=3, channels=9, conv_from=8)), "bad convolution"),
        (lambda: hip.dense_gemv_dev(8, 8, 16, 64, 64, 8, more=built.Epilogue(mul=8, mul_tokens=8, mul_at=8, mul_rows=4, ld_mul=15)), "bad table"),
        (lambda: hip.dense_matmul_dev(8, 64, False, 8, 64, 4, 16, 64, 8, 16, True, more=built.Epilogue(mul=8, mul_tokens=8, mul_at=8, mul_rows=4, ld_mul=16)), "dense_matmul: what"),
        (lambda: hip.embed_pairs_bf16_dev(8, 64, 8, 32, 5, 1, 1, 8, 8, 1, 64, 9), "embed_pairs"),
        (lambda: hip.latent_decode_dev(built.LatentAttention(1, 20, 52, 16, 64, 16, 1.0, 8, 8, 8, 64, 32, 64, 8, 8), 8, 8, 8, 0, 1, True, 8), "bad shape"),
    ]
    for call, message in bad:
        with pytest.raises(built.BitNetHipError, match=message):
            call()


# ---- the oracle itself -------------------------------------------------------------------------------------------------
def test_oracle_rotation_and_yarn():
    f, mult = so.rotary_frequencies({"dims": 8, "base": 10000.0})
    assert mult == 1.0 and np.allclose(f, [1, 0.1, 0.01, 0.001])
    x = np.arange(8.0)[None]
    y = so.rotate(x, [3], {"dims": 8, "base": 10000.0})[0]
    assert np.isclose(y[1], 1 * math.cos(0.3) - 5 * math.sin(0.3)) and np.isclose(y[5], 5 * math.cos(0.3) + 1 * math.sin(0.3))
    s = {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0}
    f2, mult = so.rotary_frequencies({"dims": 16, "base": 100.0, "scaling": s})
    f1, _ = so.rotary_frequencies({"dims": 16, "base": 100.0})
    assert np.isclose(mult, 0.1 * math.log(4) + 1)
    # lo = floor(16 ln(64 / 16 pi) / (2 ln 100)) = 0, hi = ceil(16 ln(64 / 2 pi) / (2 ln 100)) = 5
    for i in range(8):
        ramp = min(i / 5, 1.0)
        assert np.isclose(f2[i], f1[i] * (1 - ramp) + f1[i] / 4 * ramp)


def test_oracle_linear_attention_by_powers():
    """the recurrence against the sum over all earlier tokens with explicit powers of the decay"""
    g = np.random.default_rng(0)
    m, W, n = {"heads": 2, "dim": 3, "vdim": 4, "decay": [0.7, 1.0]}, 6, 5
    t = {k: g.standard_normal((2 * (3 if k in "qk" else 4), W)) for k in "qkvg"}
    t.update(o=np.eye(8), norm=np.ones(8))
    h = g.standard_normal((n, W))
    got = so.lightning(h, t, "", m, 1e-6)
    q, k, v = (so.silu(h @ t[x].T).reshape(n, 2, -1) for x in "qkv")
    o = np.zeros((n, 2, 4))
    for i in range(n):
        for j in range(i + 1):
            for a in range(2):
                o[i, a] += m["decay"][a] ** (i - j) * (q[i, a] @ k[j, a]) * v[j, a]
    assert np.allclose(got, so.norm_plain(o.reshape(n, 8), 1.0, 1e-6) * so.sigmoid(h @ t["g"].T))


def test_oracle_sink_takes_a_share():
    """one token: the weight of its only key is exp(s) / (exp(s) + exp(sink))"""
    config = u.lasapel([u.latent_layer(heads=1, dim=4, rot_dim=2, vdim=4, q_rank=4, kv_rank=4)], width=8, vocab=5)
    t = {k: np.asarray(v, np.float64) for k, v in u.random_tensors(config, 3).items()}
    h, m, p = np.random.default_rng(1).standard_normal((1, 8)), config["layers"][0]["mixer"], "l0.mix."
    t[p + "o"] = np.eye(8, 4)
    outs = {}
    for sink in (-50.0, 0.3):
        t[p + "sink"] = np.array([sink])
        outs[sink], (c, kr) = so.latent_attention(h, t, p, m, 1e-6)
    q = so.norm_plain(h @ t[p + "dq"].T, t[p + "dq.norm"], 1e-6) @ t[p + "uq"].T
    s = (q[0, :4] @ (t[p + "uk"] @ c[0]) + q[0, 4:] @ kr[0]) * m["scale"]
    assert np.allclose(outs[0.3], outs[-50.0] * np.exp(s) / (np.exp(s) + np.exp(0.3)))


def test_oracle_delta_rule_by_hand():
    """two tokens, keys alike: the second write replaces what the first one left, as far as its step size goes"""
    k, v = np.array([[1.0, 0.0], [1.0, 0.0]]), np.array([[2.0], [6.0]])
    o, S = so.delta_rule(k, k, v, np.array([1.0, 0.5]), np.array([1.0, 0.25]), np.zeros((2, 1)))
    assert np.allclose(o[:, 0], [2.0, 1.0 + 0.25 * (6.0 - 1.0)]) and np.allclose(S[:, 0], [2.25, 0.0])


def test_oracle_chunks_and_sink():
    """scores of zero: the mean over what a chunk shows so far and the sink's nothing"""
    v = np.arange(1.0, 6.0).reshape(5, 1, 1)
    o = so.chunk_softmax(np.ones((5, 2, 3)), np.zeros((5, 1, 3)), v, 1.0, 3)
    assert np.allclose(o[:, :, 0].T, [1.0 / 2, 3.0 / 3, 6.0 / 4, 4.0 / 2, 9.0 / 3])
    o = so.chunk_softmax(np.ones((1, 1, 2)), np.ones((1, 1, 2)), np.ones((1, 1, 1)), 0.5, 9)
    assert np.isclose(o[0, 0, 0], math.e / (1.0 + math.e))


def test_oracle_neighbours_turn_and_bands():
    rot = {"dims": 4, "base": 10.0}
    v = np.arange(12.0).reshape(2, 1, 6)
    o = so.rotate_neighbours(v, rot)
    assert np.array_equal(o[0], v[0]) and np.array_equal(o[1, :, 4:], v[1, :, 4:])
    for i, f in enumerate((1.0, 10.0 ** -0.5)):
        assert np.isclose(complex(*o[1, 0, 2 * i:2 * i + 2]), complex(*v[1, 0, 2 * i:2 * i + 2]) * np.exp(1j * f))
    plain = so.banded_frequencies({"dims": 40, "base": 1000.0})
    bands = so.banded_frequencies({"dims": 40, "base": 1000.0, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 200}})
    turns = 200 * plain / (2 * math.pi)
    assert np.array_equal(bands[turns > 4], plain[turns > 4]) and np.allclose(bands[turns < 1], plain[turns < 1] / 8) and (turns > 4).any() and (turns < 1).any()
    between = (turns > 1) & (turns < 4)
    assert between.any() and np.allclose(bands[between], plain[between] * ((turns[between] - 1) / 3 * 7 / 8 + 1 / 8))


def test_oracle_corrected_choice():
    z = np.log(np.array([[0.1, 0.2, 0.3, 0.4]]))
    ids, w = so.route_corrected(np.ones((1, 1)), z.T, np.array([0.35, 0.0, 0.0, -0.15]), 2)
    assert ids.tolist() == [[0, 2]] and np.allclose(w, [[0.1, 0.3]])
    assert np.allclose(so.gelu_tanh(np.array([-50.0, 0.0, 50.0])), [0.0, 0.0, 50.0]) and np.isclose(so.gelu_tanh(1.0), 0.841192, atol=1e-6)


def test_oracle_window_and_penalty():
    """scores of zero: the mean over the window; a penalty of r1 ln(1 + r2 d) leaves (1 + r2 d)^-r1 of a weight"""
    v = np.arange(1.0, 6.0).reshape(5, 1, 1)
    o = so.window_softmax(np.ones((5, 2, 3)), np.zeros((5, 1, 3)), v, 1.0, 3, np.zeros(2), np.ones(2))
    assert np.allclose(o[:, :, 0].T, [1.0, 1.5, 2.0, 3.0, 4.0])
    o = so.window_softmax(np.ones((3, 1, 3)), np.zeros((3, 1, 3)), v[:3], 1.0, 9, np.full(1, 2.0), np.full(1, 3.0))
    w = np.array([7.0, 4.0, 1.0]) ** -2.0
    assert np.isclose(o[2, 0, 0], (w @ [1.0, 2.0, 3.0]) / w.sum())


def test_oracle_groups():
    score = np.array([[0.9, 0.1, 0.1, 0.6, 0.6, 0.2, 0.8, 0.1, 0.05]])
    z = np.log(score / (1 - score))
    ids, w = so.route_in_groups(np.ones((1, 1)), z.T, np.zeros(9), 2, {"count": 3, "keep": 1})
    assert ids.tolist() == [[3, 4]] and np.allclose(w, 0.6)  # the group of the two best together, not of the best one
    ids, w = so.route_in_groups(np.ones((1, 1)), z.T, np.array([0.0] * 5 + [0.0, 0.0, 0.45, 0.0]), 2, {"count": 3, "keep": 1})
    assert ids.tolist() == [[6, 7]] and np.allclose(w, [[0.8, 0.1]])
    ids, _ = so.route_in_groups(np.ones((1, 1)), z.T, np.full(9, -2.0), 3, {"count": 3, "keep": 2})
    assert ids.tolist() == [[0, 3, 4]]  # corrected scores below zero are still above what cannot be chosen


def test_oracle_pairs_xielu_and_neighbours():
    assert so.bigram_rows([4, 2, 7], {"buckets": 10, "mul_prev": 3, "mul_cur": 5}) == [10, (12 + 10) % 10, (6 + 35) % 10]
    z = np.array([-30.0, -1e-4, 0.0, 1e-4, 3.0])
    p, q = 0.4, -0.7
    a, b = math.log(1 + math.exp(p)), 0.5 + math.log(1 + math.exp(q))
    assert np.allclose(so.xielu(z, p, q), [b * 29.0 - 15.0, -0.5e-4 + b * 0.5e-8, 0.0, 0.5e-4 + a * 1e-8, 9 * a + 1.5], rtol=1e-5)
    rot = {"dims": 6, "base": 30.0, "scaling": {"factor": 4.0, "original": 64, "fast": 16.0, "slow": 1.0}}
    f, mult = so.rotary_frequencies(rot)
    v = np.random.default_rng(1).standard_normal((1, 2, 6))
    turned = so.rotate_pairs(v, [5], rot)
    for i in range(3):
        for h in range(2):
            assert np.isclose(complex(*turned[0, h, 2 * i:2 * i + 2]), complex(*v[0, h, 2 * i:2 * i + 2]) * np.exp(5j * f[i]) * mult)
    halves = so.rotate(np.concatenate([v[..., 0::2], v[..., 1::2]], axis=-1), [5], rot)
    assert np.allclose(halves, np.concatenate([turned[..., 0::2], turned[..., 1::2]], axis=-1))


def test_oracle_token_side_input():
    x, t = np.array([[1.0, 2.0]]), {"gate": np.array([[1.0, -1.0]]), "proj": np.array([[3.0], [4.0]]), "norm": np.array([1.0, 2.0])}
    y = so.token_side_input(x, np.array([[-2.0]]), t, "", 0.0)
    assert np.allclose(y, np.array([[3.0, 8.0]]) / math.sqrt(12.5))  # (gelu(-1) < 0, times -2: positive)


def test_oracle_convolution_and_routing():
    x = np.array([[1.0], [2.0], [3.0]])
    assert np.allclose(so.short_convolution(x, np.array([[10.0, 1.0]]))[:, 0], [1.0, 12.0, 23.0])
    ids, w = so.route(np.eye(3)[:1], np.array([[0.0, 0, 0], [2.0, 0, 0], [1.0, 0, 0], [2.0, 0, 0]]), 3, 2.0)
    assert ids.tolist() == [[1, 3, 2]] and np.isclose(w.sum(), 2.0) and np.isclose(w[0, 0] / w[0, 2], math.e)
    assert [so.query_temperature(p, {"q_temp": {"coef": 1.0, "every": 4}}) for p in (2, 3, 6, 7)] == [1.0, 1.0 + math.log(2), 1.0 + math.log(2), 1.0 + math.log(3)]


def test_oracle_difference_of_maps():
    """one token: both maps give its own value, whatever the scores"""
    v = np.array([[[3.0, -4.0]]])
    a = so.softmax_maps(np.ones((1, 2, 2, 3)), np.ones((1, 1, 2, 3)), v)
    assert np.allclose(a, np.broadcast_to(v[0], (1, 2, 2, 2)))
    assert np.allclose(so.difference(a, 0.25, 0.5, 0.0)[0, 0], 0.5 * v[0, 0] / math.sqrt(12.5))


def test_oracle_loop_order():
    c = u.mimolix([u.delta_layer()] * 4, loop=(1, 3, 2))
    assert so.layer_runs(c) == [(0, False), (1, True), (2, False), (1, True), (2, False), (3, False)]


def test_trace_runner_refuses_bad_use(built):
    import subprocess

    build = built._load_build_module()
    prog = build.build_program("trace_run")
    for args in ([], ["--model", "x", "--dtype", "float16", "--out", "y", "--max-tokens", "5"], ["--nonsense", "1"]):
        p = subprocess.run([prog, *args], capture_output=True, text=True, stdin=subprocess.DEVNULL, timeout=60)
        assert p.returncode == 1 and "trace_run" in p.stderr


def test_command_line_arguments(built, capsys):
    import importlib

    cli = importlib.import_module("bitnet-rs_amd.cli")
    a = cli.parse(["--model", "m", "--tokens", "3,1,4", "--new", "5"])
    assert a.tokens == [3, 1, 4] and a.max_pos == 10 and a.dtype == "bfloat16"
    for bad in (["--model", "m", "--tokens", "x"], ["--model", "m", "--tokens", "1", "--new", "0"], ["--tokens", "1"]):
        with pytest.raises(SystemExit):
            cli.parse(bad)
    assert cli.main(["--model", "/nothing", "--tokens", "1"]) == 1
    assert "neither a known file format" in capsys.readouterr().err
