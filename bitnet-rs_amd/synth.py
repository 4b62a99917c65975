"""Synthetic bitnet-b1.58 weights and prompts (there is no model file in the build
environment; SURVEY.md 8d fixes the recipe).  Data only: no arithmetic of the path.

  * I2_S codes: uniform 2-bit codes from a counter-based PRNG, seed 42, one stream per
    tensor (crates/bitnet-models/tests/qk256_avx2_correctness.rs:72-88 uses uniform codes);
  * norm gammas ~ U(0.5, 1.5) / (w_rms * sqrt(hidden)), w_rms = the format's weight rms
    (1.58 for unscaled {-2,-1,+1,+2}, 0.181 for ternary x block scales), so that projections
    of a normalised vector stay O(1) and greedy tokens vary;
  * tied embedding table f16 ~ N(0, 1);
  * prompt ids (1000 + 37 i) mod vocab with BOS first.
"""
from __future__ import annotations

from dataclasses import dataclass, asdict

import json
import os
import struct

import numpy as np

BITNET_2B_4T = dict(hidden=2560, n_layers=30, n_heads=20, n_kv_heads=5, head_dim=128, ffn=6912, vocab=128256, max_pos=4096, eps=1e-5, rope_theta=10000.0)
# crates/bitnet-models/src/qk256_utils.rs:95-104 (shape), T:957 (eps default), crates/bitnet-rope/src/lib.rs:11 (theta default)

PROJ = ("q", "k", "v", "o", "gate", "up", "down")


@dataclass
class ModelConfig:
    hidden: int = 2560
    n_layers: int = 30
    n_heads: int = 20
    n_kv_heads: int = 5
    head_dim: int = 128
    ffn: int = 6912
    vocab: int = 128256
    max_pos: int = 4096
    eps: float = 1e-5
    rope_theta: float = 10000.0

    def shapes(self):
        """[rows=out, cols=in] per projection (crates/bitnet-models/src/qk256_utils.rs:19-55)."""
        qd, kd = self.n_heads * self.head_dim, self.n_kv_heads * self.head_dim
        return {"q": (qd, self.hidden), "k": (kd, self.hidden), "v": (kd, self.hidden), "o": (self.hidden, qd),
                "gate": (self.ffn, self.hidden), "up": (self.ffn, self.hidden), "down": (self.hidden, self.ffn)}

    def asdict(self):
        return asdict(self)


def _stream(seed: int, *ids: int) -> np.random.Generator:
    return np.random.Generator(np.random.Philox(key=seed, counter=[*ids, 0, 0, 0][:4]))


def qk256_codes(rows: int, cols: int, seed: int, layer: int, proj: int) -> np.ndarray:
    stride = -(-cols // 256) * 64
    return _stream(seed, layer, proj).integers(0, 256, rows * stride, dtype=np.uint8)


def ternary_weights(rows: int, cols: int, block: int, seed: int, layer: int, proj: int):
    """Codes from {0,1,3} with P(0)=.5, P(+1)=P(-1)=.25 and scales 1/((i%100)+1)
    (crates/bitnet-quantization/benches/qk256_gemv.rs:41-43), scaled to keep O(1) outputs."""
    rng = _stream(seed, layer, proj, 1)
    assert cols % 4 == 0
    # per 2-bit field: low bit ~ Bernoulli(.5) (code is odd: +-1), high bit = low & Bernoulli(.5)
    # (code 3 = -1)  ->  P(0)=.5, P(1)=.25, P(3)=.25, never 2
    a = rng.integers(0, 256, rows * cols // 4, dtype=np.uint8)
    b = rng.integers(0, 256, rows * cols // 4, dtype=np.uint8)
    packed = (a & 0x55) | (((a & b) & 0x55) << 1)
    nblk = -(-cols // block)
    # BitNet32-F16 stores one f16 scale per 32 weights: the synthetic scales are f16 values (held as f32)
    scales = (2.0 / ((np.arange(rows * nblk) % 100) + 1)).astype(np.float16).astype(np.float32)
    return packed.reshape(-1), scales


# rms of one weight: QK256 codes uniform over {-2,-1,+1,+2} -> sqrt(2.5) = 1.58; ternary {0,+-1} with P(+-1) = .5 times the
# scales 2/((i%100)+1) -> sqrt(.5 * mean(s^2)) = sqrt(.5 * 4 * 0.01635) = 0.181
W_RMS = {"qk256": 1.58, "i2s": 0.181}


def make_layer(cfg: ModelConfig, layer: int, seed: int = 42, fmt: str = "qk256", block: int = 32) -> dict:
    g = _stream(seed, layer, 100)
    # gammas sized for the format's weight rms, so that the projections of a normalised vector are O(1) in BOTH formats
    # (round 1 used the QK256 figure for the ternary format too: projections ~0.1, the residual stream stayed the token's own
    # embedding and the tied logits returned the input token forever)
    norm_scale = 1.0 / (W_RMS["qk256" if fmt == "qk256" else "i2s"] * np.sqrt(cfg.hidden))
    out = {
        "attn_norm": (g.uniform(0.5, 1.5, cfg.hidden) * norm_scale).astype(np.float32),
        "ffn_norm": (g.uniform(0.5, 1.5, cfg.hidden) * norm_scale).astype(np.float32),
    }
    for i, name in enumerate(PROJ):
        rows, cols = cfg.shapes()[name]
        if fmt == "qk256":
            out[name] = qk256_codes(rows, cols, seed, layer, i)
        else:
            out[name], out[name + "_scales"] = ternary_weights(rows, cols, block, seed, layer, i)
    return out


def make_globals(cfg: ModelConfig, seed: int = 42) -> dict:
    g = _stream(seed, 1 << 20)
    emb = g.standard_normal((cfg.vocab, cfg.hidden), dtype=np.float32).astype(np.float16)
    return {"embed_f16": emb.view(np.uint16).reshape(-1), "final_norm": g.uniform(0.5, 1.5, cfg.hidden).astype(np.float32)}


def prompt(n: int, vocab: int, bos: int = 128000) -> np.ndarray:
    ids = (1000 + 37 * np.arange(n)) % vocab
    ids[0] = bos % vocab
    return ids.astype(np.int32)


# ---- random models of the mixer-stack designs, at sizes that resemble a real model's layers -------------------------
STACK_SIZES = {  # width, ff, heads, kv heads of the BitNet model of equal size, q_rank, vocab
    "1b": dict(width=1536, ff=4096, heads=12, n_kv=3, q_rank=768, vocab=32768),
    "2b": dict(width=2560, ff=6912, heads=20, n_kv=5, q_rank=1536, vocab=128256),
    "3b": dict(width=3072, ff=8192, heads=24, n_kv=6, q_rank=1536, vocab=32768),
}


def lasapel_config(size: str, n_layers: int) -> dict:
    """latent attention (heads of 128 + 64 rotated / 128, latent 512) and linear attention (heads of 128 / 128) in turn, every layer
    with a feed-forward; the fifth layer reads the first one's cache."""
    s = STACK_SIZES[size]
    layers = []
    for i in range(n_layers):
        if i % 2 == 0:
            m = {"heads": s["heads"], "dim": 128, "rot_dim": 64, "vdim": 128, "q_rank": s["q_rank"], "kv_rank": 512, "scale": 0.0722,
                 "rot": {"base": 500000.0, "dims": 64, "scaling": {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}
            if i == 4:
                m["kv_from"] = 0
            layers.append({"type": "latent_attention", "mixer": m, "mlp": {"kind": "dense", "ff": s["ff"]}})
        else:
            decay = [float(np.exp(-(2.0 ** (-8.0 * (h + 1) / s["heads"])))) for h in range(s["heads"])]
            layers.append({"type": "lightning", "mixer": {"heads": s["heads"], "dim": 128, "vdim": 128, "decay": decay}, "mlp": {"kind": "dense", "ff": s["ff"]}})
    return {"architecture": "Lasapel", "vocab": s["vocab"], "width": s["width"], "norm": {"eps": 1e-6}, "layers": layers}


MIMOLIX_EXPERTS = {"1b": (448, 512), "2b": (768, 768), "3b": (896, 1024)}  # columns of one of 64 experts, of the shared one: 8 and 1 make up the size's ff


def mimolix_config(size: str, runs: int) -> dict:
    """delta rule (heads of 128 / 128, two on one q / k head) and differential attention (heads of 2 x 64 / 128, kv heads of the size) in turn,
    64 experts of which a token takes 8, one shared; `runs` layer runs, four of them two layers run twice."""
    s = STACK_SIZES[size]
    ff, shared = MIMOLIX_EXPERTS[size]
    mlp = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": 64, "scale": 2.5, "top": 8}, "shared": {"ff": shared}}
    delta = {"type": "delta", "mixer": {"heads": s["heads"], "kv_heads": s["heads"] // 2, "dim": 128, "vdim": 128, "conv": 4}, "mlp": mlp}
    attention = {"type": "attention", "mixer": {"heads": s["heads"], "kv_heads": s["n_kv"], "dim": 64, "vdim": 128, "scale": 0.125, "diff": 0.5,
                                                "q_temp": {"coef": 0.1, "every": 2048}}, "mlp": mlp}
    return {"architecture": "Mimolix", "vocab": s["vocab"], "width": s["width"], "norm": {"eps": 1e-6}, "residual_mult": 0.5, "embedding": {"scale": 4.0},
            "loop": {"start": 0, "stop": 2, "times": 2}, "layers": [delta, attention] * ((runs - 2) // 2)}


def mimolix_shapes(config: dict) -> dict:
    W = config["width"]
    shapes = {"embed": (config["vocab"], W), "head": (config["vocab"], W), "final.norm": (W,), "final.norm.b": (W,), "loop.in": (W, 2 * W)}
    for i, layer in enumerate(config["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        q, H, G, D, V = p + "mix.", m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        shapes.update({p + "norm1": (W,), p + "norm1.b": (W,), q + "o": (W, H * V)})
        if layer["type"] == "attention":
            shapes.update({q + "q": (H * 2 * D, W), q + "k": (G * 2 * D, W), q + "v": (G * V, W)})
            shapes.update({q + n: (D,) for n in ("q.norm", "k.norm", "lq1", "lk1", "lq2", "lk2")})
        else:
            for n, c in (("q", G * D), ("k", G * D), ("v", H * V)):
                shapes.update({q + n: (c, W), q + n + ".conv": (c, m["conv"])})
            shapes.update({q + "b": (H, W), q + "a": (H, W), q + "g": (H * V, W), q + "A_log": (H,), q + "dt_bias": (H,), q + "norm": (V,)})
        for e in [f"e{k}" for k in range(f["router"]["experts"])] + ["shared"]:
            ff = (f["shared"] if e == "shared" else f["expert"])["ff"]
            shapes.update({f"{p}mlp.{e}.up": (ff, W), f"{p}mlp.{e}.down": (W, ff)})
        shapes[p + "mlp.router"] = (f["router"]["experts"], W)
    return shapes


def write_mimolix(folder: str, config: dict, seed: int = 42) -> str:
    ones = ("norm1", "q.norm", "k.norm", "mix.norm", "final.norm")
    return write_random(folder, config, mimolix_shapes(config), seed, lambda name: 1.0 if name.endswith(ones) else -1.0 if name.endswith(("A_log", "dt_bias")) else 0.0)


LUREPEL_FF = {"1b": 2688, "2b": 4608, "3b": 5440}  # three gated matrices of about the bytes of the size's two; 8 experts of an eighth each
LUREPEL_CHUNK = 8192


def lurepel_config(size: str, n_layers: int, chunk: int = LUREPEL_CHUNK) -> dict:
    """attention within chunks (heads of 128, half of it rotated, kv heads of the size), dense gated feed-forwards and mixtures of 64 experts and 8
    identity experts, of which a token takes 8, in turn."""
    s, ff = STACK_SIZES[size], LUREPEL_FF[size]
    mixer = {"heads": s["heads"], "kv_heads": s["n_kv"], "dim": 128, "vdim": 128, "scale": 0.0884, "mask": {"size": chunk},
             "rot": {"base": 500000.0, "dims": 64, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 4096}}}
    dense = {"kind": "dense", "ff": ff}
    moe = {"kind": "moe", "expert": {"ff": ff // 8}, "router": {"experts": 64, "identity": 8, "top": 8}}
    return {"architecture": "Lurepel", "vocab": s["vocab"], "width": s["width"], "norm": {"eps": 1e-6},
            "layers": [{"type": "attention", "mixer": mixer, "mlp": moe if i % 2 else dense} for i in range(n_layers)]}


def write_lurepel(folder: str, config: dict, seed: int = 42) -> str:
    W = config["width"]
    shapes = {"embed": (config["vocab"], W), "embed.norm": (W,), "head": (config["vocab"], W), "final.norm": (W,)}
    for i, layer in enumerate(config["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        H, G, D = m["heads"], m["kv_heads"], m["dim"]
        shapes.update({p + "norm1": (W,), p + "norm2": (W,), p + "mix.q": (H * D, W), p + "mix.k": (G * D, W), p + "mix.g": (H, W), p + "mix.o": (W, H * D)})
        parts = {"": f["ff"]} if f["kind"] == "dense" else {f"e{e}.": f["expert"]["ff"] for e in range(f["router"]["experts"])}
        for e, ff in parts.items():
            shapes.update({f"{p}mlp.{e}gate": (ff, W), f"{p}mlp.{e}up": (ff, W), f"{p}mlp.{e}down": (W, ff)})
        if f["kind"] == "moe":
            n = f["router"]["experts"] + f["router"]["identity"]
            shapes.update({p + "mlp.router": (n, W), p + "mlp.correction": (n,)})
    return write_random(folder, config, shapes, seed, lambda name: 0.0 if name.endswith("correction") else 1.0)


SIPELORN_SIDE = 256     # columns of a token's input per layer
SIPELORN_WINDOW = 8192  # positions


def sipelorn_config(size: str, n_layers: int, window: int = SIPELORN_WINDOW) -> dict:
    """attention within a window (heads of 128, kv heads of the size, three taps) with latent attention (heads of 128 + 64 rotated / 128, latent 512) in every
    fourth layer, the sixth layer on the fifth one's keys; a dense feed-forward of the size in every fourth layer, in the others 64 experts in 8 groups, of which
    a token takes 8 from 4 groups, and a shared one of the size of two."""
    s, ff = STACK_SIZES[size], LUREPEL_FF[size]
    attention = {"heads": s["heads"], "kv_heads": s["n_kv"], "dim": 128, "vdim": 128, "scale": 0.0884, "conv": 3, "mask": {"size": window}}
    latent = {"heads": s["heads"], "dim": 128, "rot_dim": 64, "vdim": 128, "kv_rank": 512, "scale": 0.0722,
              "rot": {"base": 500000.0, "dims": 64, "scaling": {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}
    expert = ff // 640 * 64  # (ten of them at work: about the active feed-forward of the size)
    moe = {"kind": "moe", "expert": {"ff": expert}, "router": {"experts": 64, "top": 8, "groups": {"count": 8, "keep": 4}}, "shared": {"ff": 2 * expert}}
    layers = [{"type": "latent_attention", "mixer": latent, "mlp": moe} if i % 4 == 1 else
              {"type": "attention", "mixer": dict(attention, kv_from=4) if i == 6 else attention, "mlp": moe if i % 4 else {"kind": "dense", "ff": s["ff"]}}
              for i in range(n_layers)]
    return {"architecture": "Sipelorn", "vocab": s["vocab"], "width": s["width"], "norm": {"eps": 1e-6},
            "embedding": {"scale": 1.0, "bigram": {"buckets": 65521, "mul_prev": 8191, "mul_cur": 127}}, "token_side": {"dim": SIPELORN_SIDE}, "layers": layers}


def write_sipelorn(folder: str, config: dict, seed: int = 42) -> str:
    W, V, side, n = config["width"], config["vocab"], config["token_side"]["dim"], len(config["layers"])
    shapes = {"embed": (V, W), "bigram": (config["embedding"]["bigram"]["buckets"] + 1, W), "side.embed": (V, n * side), "head": (V, W), "final.norm": (W,), "final.norm.b": (W,)}
    for i, layer in enumerate(config["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        q, H, D, VD = p + "mix.", m["heads"], m["dim"], m["vdim"]
        for k in "12":
            shapes.update({p + "norm" + k: (W,), p + f"norm{k}.b": (W,), p + "rg" + k: (W, W), p + f"rg{k}.b": (W,)})
        shapes.update({p + "side.gate": (side, W), p + "side.proj": (W, side), p + "side.norm": (W,), q + "o": (W, H * VD)})
        if layer["type"] == "attention":
            G = m["kv_heads"]
            for name, rows in (("q", H * D),) + (() if "kv_from" in m else (("k", G * D), ("v", G * VD))):
                shapes.update({q + name: (rows, W), q + name + ".b": (rows,), q + name + ".conv": (rows, m["conv"])})
            shapes.update({q + "g": (H * VD, W), q + "r1": (H,), q + "r2": (H,)})
        else:
            R, C = m["rot_dim"], m["kv_rank"]
            shapes.update({q + "q": (H * (D + R), W), q + "dkv": (C + R, W), q + "dkv.norm": (C,), q + "uk": (H * D, C), q + "uv": (H * VD, C)})
        if f["kind"] == "dense":
            shapes.update({p + "mlp.up": (f["ff"], W), p + "mlp.down": (W, f["ff"]), p + "mlp.act": (2,)})
        else:
            parts = {f"e{e}": f["expert"]["ff"] for e in range(f["router"]["experts"])}
            for e, ff in {**parts, "shared": f["shared"]["ff"]}.items():
                shapes.update({f"{p}mlp.{e}.gate": (ff, W), f"{p}mlp.{e}.up": (ff, W), f"{p}mlp.{e}.down": (W, ff)})
            shapes.update({p + "mlp.router": (f["router"]["experts"], W), p + "mlp.correction": (f["router"]["experts"],), p + "mlp.shared.sg": (1, W)})
    ones = ("norm", "norm1", "norm2", "r1", "r2")
    return write_random(folder, config, shapes, seed, lambda name: 1.0 if name.endswith(ones) else 0.0)


def write_lasapel(folder: str, config: dict, seed: int = 42) -> str:
    shapes = {"embed": (config["vocab"], config["width"]), "head": (config["vocab"], config["width"]), "final.norm": (config["width"],)}
    W = config["width"]
    for i, layer in enumerate(config["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        q, H = p + "mix.", m["heads"]
        shapes.update({p + n: (W,) for n in ("norm1", "norm1b", "norm2", "norm2b", "ls1", "ls2")})
        if layer["type"] == "latent_attention":
            shapes.update({q + "dq": (m["q_rank"], W), q + "dq.norm": (m["q_rank"],), q + "uq": (H * (m["dim"] + m["rot_dim"]), m["q_rank"]),
                           q + "uk": (H * m["dim"], m["kv_rank"]), q + "uv": (H * m["vdim"], m["kv_rank"]), q + "sink": (H,), q + "o": (W, H * m["vdim"])})
            if "kv_from" not in m:
                shapes.update({q + "dkv": (m["kv_rank"] + m["rot_dim"], W), q + "dkv.norm": (m["kv_rank"],)})
        else:
            shapes.update({q + n: (H * d, W) for n, d in (("q", m["dim"]), ("k", m["dim"]), ("v", m["vdim"]), ("g", m["vdim"]))})
            shapes.update({q + "norm": (H * m["vdim"],), q + "o": (W, H * m["vdim"])})
        f = layer["mlp"]["ff"]
        shapes.update({p + "mlp.up": (f, W), p + "mlp.up.b": (f,), p + "mlp.down": (W, f), p + "mlp.down.b": (W,)})
    return write_random(folder, config, shapes, seed,
                        lambda name: 1.0 if name.endswith("q.norm") or name.endswith("v.norm") or name.endswith("mix.norm") else 0.5 if ".ls" in name else 0.0)


def write_random(folder: str, config: dict, shapes: dict, seed: int, centre) -> str:
    """config.json + model.safetensors with random bf16 weights: slices of one random block, matrices scaled to unit gain, vectors around
    centre(name) (a router's correction: next to nothing, so that its experts carry like loads)."""
    block = _stream(seed, 7).standard_normal(1 << 22, dtype=np.float32)
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as fh:
        json.dump(config, fh)
    head, at = {}, 0
    for name, shape in shapes.items():
        n = 2 * int(np.prod(shape))
        head[name] = {"dtype": "BF16", "shape": list(shape), "data_offsets": [at, at + n]}
        at += n
    h = json.dumps(head).encode()
    with open(os.path.join(folder, "model.safetensors"), "wb") as fh:
        fh.write(struct.pack("<Q", len(h)) + h)
        made = {}
        for k, (name, shape) in enumerate(shapes.items()):
            n = int(np.prod(shape))
            gain, mid = ((1.0 if name == "embed" else 1.0 / np.sqrt(shape[1])), 0.0) if len(shape) == 2 else (0.001 if name.endswith("correction") else 0.1, centre(name))
            if (gain, mid) not in made:
                made[gain, mid] = np.tile(((block * np.float32(gain) + np.float32(mid)).view(np.uint32) >> 16).astype(np.uint16), 2)
            bits, start = made[gain, mid], (k * 9973) % block.size
            for a in range(0, n, block.size):
                fh.write(bits[start: start + min(block.size, n - a)].data)
    return folder
