"""Helpers of the mixer-stack tests: bf16 arrays, a safetensors writer, small random models (names, shapes and configurations of
the designs the host library registers) and device buffers."""
import json
import os
import struct

import numpy as np


def bf16_bits(a) -> np.ndarray:
    """float32 -> bf16 bit patterns, round to nearest even"""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def bf16_value(bits) -> np.ndarray:
    return (np.asarray(bits, np.uint16).astype(np.uint32) << 16).view(np.float32)


def rounded(a) -> np.ndarray:
    return bf16_value(bf16_bits(a))


def up_to(v: int, a: int) -> int:
    return -(-v // a) * a


def padded(a, ld: int) -> np.ndarray:
    """last axis zero-padded to ld"""
    a = np.asarray(a)
    out = np.zeros(a.shape[:-1] + (ld,), a.dtype)
    out[..., :a.shape[-1]] = a
    return out


def save_model(folder: str, config: dict, tensors: dict) -> str:
    """config.json + model.safetensors (tensors: float arrays, stored as bf16)"""
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(config, f)
    head, at, parts = {}, 0, []
    for name, t in tensors.items():
        raw = bf16_bits(t).tobytes()
        head[name] = {"dtype": "BF16", "shape": list(np.shape(t)), "data_offsets": [at, at + len(raw)]}
        at += len(raw)
        parts.append(raw)
    h = json.dumps(head).encode()
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(h)) + h + b"".join(parts))
    return folder


def latent_layer(heads=3, dim=24, rot_dim=16, vdim=40, q_rank=56, kv_rank=72, scale=0.17, base=10000.0, scaling=None, kv_from=None, ff=None) -> dict:
    rot = {"base": base, "dims": rot_dim}
    if scaling:
        rot["scaling"] = scaling
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale, "rot": rot}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def lightning_layer(heads=2, dim=40, vdim=24, decay=None, ff=None) -> dict:
    decay = decay if decay is not None else [float(np.exp(-2.0 ** -(1 + 3 * h))) for h in range(heads)]
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def lasapel(layers, width=112, vocab=150, eps=1e-5) -> dict:
    return {"architecture": "Lasapel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


def expert_mlp(experts=6, top=3, ff=24, scale=1.7, shared=40) -> dict:
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "scale": scale, "top": top}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def attention_layer(heads=6, kv_heads=3, dim=20, vdim=28, scale=0.31, diff=0.2, coef=0.4, every=8, mlp=None) -> dict:
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "diff": diff,
                                           "q_temp": {"coef": coef, "every": every}}, "mlp": mlp}


def delta_layer(heads=4, kv_heads=2, dim=24, vdim=40, conv=4, mlp=None) -> dict:
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}, "mlp": mlp}


def mimolix(layers, width=112, vocab=150, eps=1e-5, mult=0.4, embed=3.0, loop=None) -> dict:
    c = {"architecture": "Mimolix", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult, "embedding": {"scale": embed}, "layers": layers}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


def random_mimolix(config: dict, seed: int) -> dict:
    """bf16-representable weights, everything away from its neutral value.  A router's choice must not hang on the last bit of its input: the
    first columns of an embedding row say which experts the token takes (well apart from each other and from the rest), nothing is added to these
    columns behind the embedding, and the router reads them (and a little of the rest)."""
    g = np.random.default_rng(seed)
    W, V = config["width"], config["vocab"]
    codes = max([layer["mlp"]["router"]["experts"] for layer in config["layers"] if layer["mlp"]], default=0)
    tops = max([layer["mlp"]["router"]["top"] for layer in config["layers"] if layer["mlp"]], default=0)
    t = {}

    def mat(name, rows, cols, gain=1.0):
        t[name] = rounded(g.standard_normal((rows, cols)) * gain / np.sqrt(cols))

    def back(name, cols):  # a matrix back to the residual stream
        mat(name, W, cols)
        t[name][:codes] = 0.0

    def around(name, n, centre, spread):
        t[name] = rounded(centre + spread * g.standard_normal(n))

    def norm(name):
        around(name, W, 1.0, 0.2)
        around(name + ".b", W, 0.0, 0.2)
        t[name][:codes], t[name + ".b"][:codes] = 1.0, 0.0

    t["embed"] = g.standard_normal((V, W)) / config["embedding"]["scale"]
    for i in range(V):
        order = g.permutation(codes)
        t["embed"][i, order] = (-0.5 - g.random(codes)) / config["embedding"]["scale"]
        first = order[:tops + 1]
        t["embed"][i, first] = (2.5 - 0.7 * np.arange(len(first))) / config["embedding"]["scale"]
    t["embed"] = rounded(t["embed"])
    for i, layer in enumerate(config["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        H, G, D, VD, q = m["heads"], m["kv_heads"], m["dim"], m["vdim"], f"l{i}.mix."
        norm(p + "norm1")
        if layer["type"] == "attention":
            for name, rows in (("q", H * 2 * D), ("k", G * 2 * D), ("v", G * VD)):
                mat(q + name, rows, W)
            around(q + "q.norm", D, 1.2, 0.3)
            around(q + "k.norm", D, 1.2, 0.3)
            for name in ("lq1", "lk1", "lq2", "lk2"):
                around(q + name, D, 0.0, 0.15)
        else:
            for name, rows in (("q", G * D), ("k", G * D), ("v", H * VD)):
                mat(q + name, rows, W)
                t[q + name + ".conv"] = rounded(0.5 * g.standard_normal((rows, m["conv"])))
            for name, rows in (("b", H), ("a", H), ("g", H * VD)):
                mat(q + name, rows, W)
            around(q + "A_log", H, -0.5, 0.7)
            t[q + "A_log"][0] = -5.0  # one head that forgets slowly
            around(q + "dt_bias", H, -1.0, 0.7)
            around(q + "norm", VD, 1.0, 0.3)
        back(q + "o", H * VD)
        if layer["mlp"]:
            f, r = p + "mlp.", layer["mlp"]["router"]
            t[f + "router"] = rounded(np.concatenate([2.0 * np.eye(r["experts"], codes), 0.02 * g.standard_normal((r["experts"], W - codes))], axis=1))
            parts = {f"e{e}.": layer["mlp"]["expert"]["ff"] for e in range(r["experts"])}
            if "shared" in layer["mlp"]:
                parts["shared."] = layer["mlp"]["shared"]["ff"]
            for name, ff in parts.items():
                mat(f + name + "up", ff, W)
                back(f + name + "down", ff)
    if config.get("loop"):
        t["loop.in"] = g.standard_normal((W, 2 * W)) * 0.6 / np.sqrt(W)
        t["loop.in"][:codes] = 0.0
        t["loop.in"][:codes, :codes] = t["loop.in"][:codes, W:W + codes] = 0.5 * np.eye(codes)
        t["loop.in"] = rounded(t["loop.in"])
    norm("final.norm")
    mat("head", V, W)
    return t


BANDS = {"factor": 5.0, "low": 1.5, "high": 6.0, "original": 96}


def chunk_layer(heads=6, kv_heads=3, dim=20, scale=0.27, chunk=37, dims=12, base=300.0, scaling=None, mlp=None) -> dict:
    rot = {"base": base, "dims": dims}
    if scaling:
        rot["scaling"] = scaling
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale, "mask": {"size": chunk}, "rot": rot}, "mlp": mlp}


def gated_mlp(ff=40) -> dict:
    return {"kind": "dense", "ff": ff}


def corrected_mlp(experts=6, identity=2, top=3, ff=24) -> dict:
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "identity": identity, "top": top}}


def lurepel(layers, width=112, vocab=150, eps=1e-5) -> dict:
    return {"architecture": "Lurepel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


def random_lurepel(config: dict, seed: int) -> dict:
    """bf16-representable weights, everything away from its neutral value.  As with the parallel design, the first columns of an embedding row say
    which experts its token takes and no sublayer adds to them; rows are drawn again until, in every layer, what is chosen and what is not lie well
    apart."""
    g = np.random.default_rng(seed)
    W, V, eps = config["width"], config["vocab"], config["norm"]["eps"]
    routers = {i: layer["mlp"]["router"] for i, layer in enumerate(config["layers"]) if layer["mlp"] and layer["mlp"]["kind"] == "moe"}
    codes = max([r["experts"] + r["identity"] for r in routers.values()], default=0)
    t = {}

    def mat(name, rows, cols, gain=1.0):
        t[name] = rounded(g.standard_normal((rows, cols)) * gain / np.sqrt(cols))

    def norm(name, keep):
        t[name] = rounded(1.0 + 0.25 * g.standard_normal(W))
        t[name][:codes] = keep

    norm("embed.norm", 1.0)
    for i, r in routers.items():
        n = r["experts"] + r["identity"]
        t[f"l{i}.mlp.router"] = rounded(np.concatenate([1.2 * np.eye(n)[g.permutation(n)], np.zeros((n, codes - n)), 0.0003 * g.standard_normal((n, W - codes))], axis=1))
        t[f"l{i}.mlp.correction"] = rounded(g.uniform(-0.25, 0.25, n))

    def apart(row):
        x = row / np.sqrt(np.mean(row ** 2) + eps) * t["embed.norm"]
        for i, r in routers.items():
            z = t[f"l{i}.mlp.router"].astype(np.float64) @ x
            s = np.exp(z - z.max())
            choice = np.sort(s / s.sum() + t[f"l{i}.mlp.correction"])[::-1]
            if r["top"] < len(choice) and choice[r["top"] - 1] - choice[r["top"]] < 0.02:
                return False
        return True

    t["embed"] = np.zeros((V, W), np.float32)
    for k in range(V):
        while True:
            row = rounded(np.concatenate([g.uniform(-1.0, 2.0, codes), 0.8 * g.standard_normal(W - codes)]))
            if apart(row.astype(np.float64)):
                break
        t["embed"][k] = row
    for i, layer in enumerate(config["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        H, G, D = m["heads"], m["kv_heads"], m["dim"]
        norm(p + "norm1", 0.0)
        mat(p + "mix.q", H * D, W)
        mat(p + "mix.k", G * D, W)
        mat(p + "mix.g", H, W, 1.5)
        mat(p + "mix.o", W, H * D)
        if not f:
            continue
        norm(p + "norm2", 0.0)
        parts = {"": f["ff"]} if f["kind"] == "dense" else {f"e{e}.": f["expert"]["ff"] for e in range(f["router"]["experts"])}
        for e, ff in parts.items():
            mat(f"{p}mlp.{e}gate", ff, W)
            mat(f"{p}mlp.{e}up", ff, W)
            mat(f"{p}mlp.{e}down", W, ff)
    norm("final.norm", 1.0)
    mat("head", V, W)
    return t


YARN = {"factor": 5.0, "original": 60, "fast": 9.0, "slow": 1.5}


def window_layer(heads=6, kv_heads=3, dim=20, vdim=28, scale=0.24, window=37, taps=3, kv_from=None, mlp=None) -> dict:
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "conv": taps}
    if window:
        m["mask"] = {"size": window}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m, "mlp": mlp}


def direct_latent_layer(heads=3, dim=24, rot_dim=12, vdim=40, kv_rank=72, scale=0.19, base=700.0, scaling=None, mlp=None) -> dict:
    rot = {"base": base, "dims": rot_dim}
    if scaling:
        rot["scaling"] = scaling
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale, "rot": rot}, "mlp": mlp}


def xielu_mlp(ff=44) -> dict:
    return {"kind": "dense", "ff": ff}


def grouped_mlp(experts=8, groups=(4, 2), top=3, ff=24, shared=40) -> dict:
    f = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if groups:
        f["router"]["groups"] = dict(zip(("count", "keep"), groups))
    if shared:
        f["shared"] = {"ff": shared}
    return f


def sipelorn(layers, width=120, vocab=150, eps=1e-5, embed=2.5, pairs=(61, 13, 5), side=20) -> dict:
    return {"architecture": "Sipelorn", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"scale": embed, "bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), pairs))}, "token_side": {"dim": side}, "layers": layers}


def group_margins(choice, top, groups):
    """how far the choice among these scores is from another one"""
    margins = []
    if groups:
        part = choice.reshape(groups["count"], -1)
        worth = np.sort(part, axis=1)[:, -2:].sum(axis=1)
        order = np.argsort(-worth, kind="stable")
        if groups["keep"] < groups["count"]:
            margins.append(worth[order[groups["keep"] - 1]] - worth[order[groups["keep"]]])
        choice = part[order[:groups["keep"]]].reshape(-1)
    ranked = np.sort(choice)[::-1]
    if top < len(ranked):
        margins.append(ranked[top - 1] - ranked[top])
    return min(margins, default=1.0)


def random_sipelorn(config: dict, seed: int) -> dict:
    """bf16-representable weights, everything away from its neutral value.  No choice of experts may hang on the last bit of the router's input: its first
    columns are large, come from the token's embedding alone (nothing is added to them, and they make up most of the stream's variance), and embedding rows are
    drawn until what is chosen and what is not lie apart in every layer, whatever the other columns' variance."""
    g = np.random.default_rng(seed)
    W, V, side = config["width"], config["vocab"], config["token_side"]["dim"]
    routers = {i: layer["mlp"]["router"] for i, layer in enumerate(config["layers"]) if layer["mlp"] and layer["mlp"]["kind"] == "moe"}
    codes = max([r["experts"] for r in routers.values()], default=0)
    t = {}

    def mat(name, rows, cols, gain=1.0):
        t[name] = rounded(g.standard_normal((rows, cols)) * gain / np.sqrt(cols))

    def back(name, cols):  # a matrix back to the residual stream
        mat(name, W, cols)
        t[name][:codes] = 0.0

    def around(name, n, centre, spread):
        t[name] = rounded(centre + spread * g.standard_normal(n))

    def norm(name):
        around(name, W, 1.0, 0.2)
        around(name + ".b", W, 0.0, 0.2)
        t[name][:codes], t[name + ".b"][:codes] = 1.0, 0.0

    for i, r in routers.items():
        n = r["experts"]
        t[f"l{i}.mlp.router"] = rounded(np.concatenate([1.5 * np.eye(n)[g.permutation(n)], np.zeros((n, codes - n)), 0.0003 * g.standard_normal((n, W - codes))], axis=1))
        t[f"l{i}.mlp.correction"] = rounded(g.uniform(-0.2, 0.2, n))

    def apart(code):
        for i, r in routers.items():
            w, c = t[f"l{i}.mlp.router"][:, :codes].astype(np.float64), t[f"l{i}.mlp.correction"].astype(np.float64)
            for rest in (0.3, 0.7, 1.2, 2.0, 3.5, 6.0):  # variance of the columns that are added to
                for shift in (-0.15, 0.0, 0.15):
                    mean = code.sum() / W + shift
                    h = (code - mean) / np.sqrt(((code - mean) ** 2).sum() / W + rest * (W - codes) / W)
                    if group_margins(1.0 / (1.0 + np.exp(-(w @ h))) + c, r["top"], r.get("groups")) < 0.012:
                        return False
        return True

    scale = config["embedding"]["scale"]
    t["embed"] = np.zeros((V, W), np.float32)
    for k in range(V):
        while True:
            row = rounded(np.concatenate([g.uniform(-4.0, 4.0, codes), 0.8 * g.standard_normal(W - codes)]) / scale)
            if apart(row[:codes].astype(np.float64) * scale):
                break
        t["embed"][k] = row
    t["bigram"] = rounded(0.7 * g.standard_normal((config["embedding"]["bigram"]["buckets"] + 1, W)))
    t["bigram"][:, :codes] = 0.0
    t["side.embed"] = rounded(g.standard_normal((V, side * len(config["layers"]))))
    for i, layer in enumerate(config["layers"]):
        p, q, m, f = f"l{i}.", f"l{i}.mix.", layer["mixer"], layer["mlp"]
        H, D, VD = m["heads"], m["dim"], m["vdim"]
        for k in "12" if f else "1":
            norm(p + "norm" + k)
            mat(p + "rg" + k, W, W)
            around(p + f"rg{k}.b", W, 0.0, 0.5)
        if layer["type"] == "attention":
            G = m["kv_heads"]
            for name, rows in (("q", H * D),) + (() if "kv_from" in m else (("k", G * D), ("v", G * VD))):
                mat(q + name, rows, W)
                around(q + name + ".b", rows, 0.0, 0.4)
                t[q + name + ".conv"] = rounded(0.2 + 0.6 * g.standard_normal((rows, m["conv"])))
            t[q + "r1"], t[q + "r2"] = rounded(g.uniform(0.1, 0.9, H)), rounded(g.uniform(0.02, 1.5, H))
            mat(q + "g", H * VD, W, 1.5)
        else:
            R, C = m["rot_dim"], m["kv_rank"]
            mat(q + "q", H * (D + R), W, 1.5)
            mat(q + "dkv", C + R, W)
            around(q + "dkv.norm", C, 1.0, 0.3)
            mat(q + "uk", H * D, C, 1.5)
            mat(q + "uv", H * VD, C)
        back(q + "o", H * VD)
        if f and f["kind"] == "dense":
            mat(p + "mlp.up", f["ff"], W)
            back(p + "mlp.down", f["ff"])
            around(p + "mlp.act", 2, 0.3, 0.5)
        elif f:
            parts = {f"e{e}.": f["expert"]["ff"] for e in range(f["router"]["experts"])}
            if f.get("shared"):
                parts["shared."] = f["shared"]["ff"]
                mat(p + "mlp.shared.sg", 1, W, 1.5)
            for e, ff in parts.items():
                mat(p + f"mlp.{e}gate", ff, W)
                mat(p + f"mlp.{e}up", ff, W)
                back(p + f"mlp.{e}down", ff)
        mat(p + "side.gate", side, W)
        back(p + "side.proj", side)
        around(p + "side.norm", W, 0.6, 0.2)
        t[p + "side.norm"][:codes] = 0.0
    norm("final.norm")
    mat("head", V, W)
    return t


def random_tensors(config: dict, seed: int) -> dict:
    return {"Lasapel": random_lasapel, "Mimolix": random_mimolix, "Lurepel": random_lurepel, "Sipelorn": random_sipelorn}[config["architecture"]](config, seed)


def random_lasapel(config: dict, seed: int) -> dict:
    """bf16-representable weights; every norm, scale, bias and sink away from its neutral value"""
    g = np.random.default_rng(seed)
    W, V = config["width"], config["vocab"]
    t = {}

    def mat(name, rows, cols, gain=1.0):
        t[name] = rounded(g.standard_normal((rows, cols)) * gain / np.sqrt(cols))

    def around(name, n, centre, spread):
        t[name] = rounded(centre + spread * g.standard_normal(n))

    t["embed"] = rounded(g.standard_normal((V, W)))
    for i, layer in enumerate(config["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        H = m["heads"]
        for name in ("norm1", "norm1b") + (("norm2", "norm2b") if layer["mlp"] else ()):
            around(p + name, W, 0.0, 0.3)
        around(p + "ls1", W, 0.7, 0.2)
        q = p + "mix."
        if layer["type"] == "latent_attention":
            mat(q + "dq", m["q_rank"], W)
            around(q + "dq.norm", m["q_rank"], 1.0, 0.3)
            mat(q + "uq", H * (m["dim"] + m["rot_dim"]), m["q_rank"], 1.5)
            if "kv_from" not in m:
                mat(q + "dkv", m["kv_rank"] + m["rot_dim"], W)
                around(q + "dkv.norm", m["kv_rank"], 1.0, 0.3)
            mat(q + "uk", H * m["dim"], m["kv_rank"], 1.5)
            mat(q + "uv", H * m["vdim"], m["kv_rank"])
            around(q + "sink", H, 0.5, 1.0)
            mat(q + "o", W, H * m["vdim"])
        else:
            for k, n in (("q", m["dim"]), ("k", m["dim"]), ("v", m["vdim"]), ("g", m["vdim"])):
                mat(q + k, H * n, W)
            around(q + "norm", H * m["vdim"], 1.0, 0.3)
            mat(q + "o", W, H * m["vdim"])
        if layer["mlp"]:
            around(p + "ls2", W, 0.7, 0.2)
            F = layer["mlp"]["ff"]
            mat(p + "mlp.up", F, W)
            around(p + "mlp.up.b", F, 0.1, 0.2)
            mat(p + "mlp.down", W, F)
            around(p + "mlp.down.b", W, 0.0, 0.2)
    around("final.norm", W, 0.0, 0.3)
    mat("head", V, W)
    return t


# ---- device buffers ----------------------------------------------------------------------------------------------------
def dev(a, dtype=None):
    import torch

    t = torch.from_numpy(np.ascontiguousarray(a))
    return (t if dtype is None else t.to(dtype)).cuda()


def dev_f32(a):
    return dev(np.asarray(a, np.float32))


def dev_bf16(a):
    """bf16 bit patterns on the device (as int16)"""
    return dev(bf16_bits(a).view(np.int16))


def zeros_f32(*shape):
    import torch

    return torch.zeros(shape, dtype=torch.float32, device="cuda")


def zeros_bf16(*shape):
    import torch

    return torch.zeros(shape, dtype=torch.int16, device="cuda")


def host(t) -> np.ndarray:
    import torch

    torch.cuda.synchronize()
    a = t.cpu().numpy()
    return bf16_value(a.view(np.uint16)) if a.dtype == np.int16 else a


def rms_error(got, want) -> float:
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    return float(np.sqrt(np.mean((got - want) ** 2)) / max(np.sqrt(np.mean(want ** 2)), 1e-30))
