"""Plain restatement of the mixer-stack designs (TEST INFRASTRUCTURE, float64 numpy): one function per mechanism,
whole sequences only, no cache, no state carried between calls.  It shares no code with the product path (which has no
Python arithmetic at all) and is written for clarity: a token at a time where that is the plainest form.

    logits, layers = forward(config, tensors, tokens)

config is the parsed config.json, tensors maps names to arrays.
"""
from __future__ import annotations

import math

import numpy as np

F = np.float64


# ---- norms -----------------------------------------------------------------------------------------------------------
def rms_divide(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def norm_plain(x, w, eps):
    return rms_divide(x, eps) * w


def norm_around_zero(x, w, eps):
    return rms_divide(x, eps) * (1.0 + w)


def layer_norm(x, w, b, eps):
    d = x - np.mean(x, axis=-1, keepdims=True)
    return d / np.sqrt(np.mean(d * d, axis=-1, keepdims=True) + eps) * w + b


# ---- activations -----------------------------------------------------------------------------------------------------
def silu(z):
    return z / (1.0 + np.exp(-z))


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def relu_squared(z):
    return np.maximum(z, 0.0) ** 2


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def xielu(z, p, q):
    """a parabola for positive arguments, an exponential for the others; the two numbers pass a softplus"""
    up = softplus(p) * z * z + 0.5 * z
    down = (0.5 + softplus(q)) * (np.expm1(np.minimum(z, 0.0)) - z) + 0.5 * z
    return np.where(z > 0.0, up, down)


# ---- rotary positions ------------------------------------------------------------------------------------------------
def rotary_frequencies(rot):
    """(frequency per pair, factor on cos and sin)"""
    dims, base = rot["dims"], float(rot["base"])
    f = np.array([base ** (-2.0 * i / dims) for i in range(dims // 2)], F)
    s = rot.get("scaling")
    if not s:
        return f, 1.0

    def dim_of(turns):
        return dims * math.log(s["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo, hi = max(math.floor(dim_of(s["fast"])), 0), min(math.ceil(dim_of(s["slow"])), dims - 1)
    for i in range(dims // 2):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        f[i] = f[i] / s["factor"] * ramp + f[i] * (1.0 - ramp)
    return f, 0.1 * math.log(s["factor"]) + 1.0


def rotate(v, positions, rot):
    """v [tokens, ..., dims]: element i turns with element i + dims / 2"""
    f, mult = rotary_frequencies(rot)
    half = rot["dims"] // 2
    out = np.array(v, F)
    for t, p in enumerate(positions):
        a = p * f
        c, s = np.cos(a) * mult, np.sin(a) * mult
        u, w = v[t][..., :half], v[t][..., half:2 * half]
        out[t][..., :half] = u * c - w * s
        out[t][..., half:2 * half] = w * c + u * s
    return out


def rotate_pairs(v, positions, rot):
    """v [tokens, ..., dims]: elements 2i and 2i + 1 turn together, by the frequencies and the factor of rotary_frequencies"""
    f, mult = rotary_frequencies(rot)
    out = np.array(v, F)
    for t, p in enumerate(positions):
        c, s = np.cos(p * f) * mult, np.sin(p * f) * mult
        a, b = v[t][..., 0::2], v[t][..., 1::2]
        out[t][..., 0::2], out[t][..., 1::2] = a * c - b * s, b * c + a * s
    return out


def banded_frequencies(rot):
    """frequency per pair: slow pairs (long wavelengths) divided by the factor, fast ones kept, a line between the two bands"""
    out, s = [], rot.get("scaling")
    for i in range(rot["dims"] // 2):
        f = float(rot["base"]) ** (-2.0 * i / rot["dims"])
        if s:
            turns = s["original"] * f / (2.0 * math.pi)  # within the original length
            if turns < s["low"]:
                f = f / s["factor"]
            elif turns <= s["high"]:
                keep = (turns - s["low"]) / (s["high"] - s["low"])
                f = (1.0 - keep) * f / s["factor"] + keep * f
        out.append(f)
    return np.array(out, F)


def rotate_neighbours(v, rot):
    """v [tokens, heads, dim]: elements 2i and 2i + 1 turn together, elements from rot["dims"] on stay"""
    out, f = np.array(v, F), banded_frequencies(rot)
    for p in range(len(v)):
        for i, fi in enumerate(f):
            c, s = math.cos(p * fi), math.sin(p * fi)
            a, b = v[p, :, 2 * i], v[p, :, 2 * i + 1]
            out[p, :, 2 * i], out[p, :, 2 * i + 1] = a * c - b * s, b * c + a * s
    return out


# ---- mixers ----------------------------------------------------------------------------------------------------------
def latent_of(h, t, p, m, eps):
    """the pair a layer with its own down-projection leaves behind: (normed latent, rotated shared key part)"""
    z = h @ t[p + "dkv"].T
    c = norm_plain(z[:, :m["kv_rank"]], t[p + "dkv.norm"], eps)
    return c, rotate(z[:, m["kv_rank"]:], range(len(h)), m["rot"])


def latent_attention(h, t, p, m, eps, shared=None):
    n, H, D, R, V = len(h), m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, kr = latent_of(h, t, p, m, eps) if shared is None else shared
    q = norm_plain(h @ t[p + "dq"].T, t[p + "dq.norm"], eps) @ t[p + "uq"].T
    q = q.reshape(n, H, D + R)
    qr = rotate(q[:, :, D:], range(n), m["rot"])
    k = (c @ t[p + "uk"].T).reshape(n, H, D)
    v = (c @ t[p + "uv"].T).reshape(n, H, V)
    out = np.zeros((n, H, V), F)
    for a in range(H):
        s = (q[:, a, :D] @ k[:, a].T + qr[:, a] @ kr.T) * m["scale"]
        s[np.triu_indices(n, 1)] = -np.inf
        top = np.maximum(s.max(axis=1), t[p + "sink"][a])
        e = np.exp(s - top[:, None])
        den = e.sum(axis=1) + np.exp(t[p + "sink"][a] - top)
        out[:, a] = (e / den[:, None]) @ v[:, a]
    return out.reshape(n, H * V) @ t[p + "o"].T, (c, kr)


def lightning(h, t, p, m, eps):
    n, H, D, V = len(h), m["heads"], m["dim"], m["vdim"]
    q = silu(h @ t[p + "q"].T).reshape(n, H, D)
    k = silu(h @ t[p + "k"].T).reshape(n, H, D)
    v = silu(h @ t[p + "v"].T).reshape(n, H, V)
    o = np.zeros((n, H, V), F)
    for a in range(H):
        S = np.zeros((D, V), F)
        for i in range(n):
            S = m["decay"][a] * S + np.outer(k[i, a], v[i, a])
            o[i, a] = S.T @ q[i, a]
    y = norm_plain(o.reshape(n, H * V), t[p + "norm"], eps) * sigmoid(h @ t[p + "g"].T)
    return y @ t[p + "o"].T


def query_temperature(p, m):
    s = m["q_temp"]
    return 1.0 + s["coef"] * math.log(math.floor((p + 1) / s["every"]) + 1.0)


def softmax_maps(q, k, v):
    """q [n, heads, maps, dim], k [n, kv heads, maps, dim], v [n, kv heads, vdim]: causal softmax of q.k over the values, per head and map"""
    n, H, M, _ = q.shape
    out = np.zeros((n, H, M, v.shape[2]), F)
    for a in range(H):
        g = a // (H // k.shape[1])
        for j in range(M):
            s = q[:, a, j] @ k[:, g, j].T
            s[np.triu_indices(n, 1)] = -np.inf
            e = np.exp(s - s.max(axis=1, keepdims=True))
            out[:, a, j] = e / e.sum(axis=1, keepdims=True) @ v[:, g]
    return out


def difference(maps, lam, diff, eps):
    """[..., 2, vdim] -> [..., vdim]"""
    return rms_divide(maps[..., 0, :] - lam * maps[..., 1, :], eps) * (1.0 - diff)


def differential_attention(h, t, p, m, eps):
    """two softmax maps per head over the same values; the second, weighted, is taken from the first"""
    n, H, G, D, V = len(h), m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = norm_plain((h @ t[p + "q"].T).reshape(n, H, 2, D), t[p + "q.norm"], eps)
    k = norm_plain((h @ t[p + "k"].T).reshape(n, G, 2, D), t[p + "k.norm"], eps)
    v = (h @ t[p + "v"].T).reshape(n, G, V)
    lam = math.exp(t[p + "lq1"] @ t[p + "lk1"]) - math.exp(t[p + "lq2"] @ t[p + "lk2"]) + m["diff"]
    factor = np.array([query_temperature(i, m) * m["scale"] for i in range(n)])
    out = difference(softmax_maps(q * factor[:, None, None, None], k, v), lam, m["diff"], eps)
    return out.reshape(n, H * V) @ t[p + "o"].T


def chunk_softmax(q, k, v, scale, chunk):
    """q [n, heads, dim], k [n, kv heads, dim], v [n, kv heads, vdim]: a token sees what lies ahead of it in its own chunk of positions; the
    softmax's denominator holds one more"""
    n, H, _ = q.shape
    out = np.zeros((n, H, v.shape[2]), F)
    for a in range(H):
        g = a // (H // k.shape[1])
        for i in range(n):
            first = i // chunk * chunk
            s = k[first:i + 1, g] @ q[i, a] * scale
            top = max(s.max(), 0.0)
            e = np.exp(s - top)
            out[i, a] = e @ v[first:i + 1, g] / (math.exp(-top) + e.sum())
    return out


def chunk_attention(h, t, p, m, eps):
    n, H, G, D = len(h), m["heads"], m["kv_heads"], m["dim"]
    q, k = (h @ t[p + "q"].T).reshape(n, H, D), (h @ t[p + "k"].T).reshape(n, G, D)
    qr, kr = (rms_divide(rotate_neighbours(x, m["rot"]), eps) for x in (q, k))
    o = chunk_softmax(qr, kr, k, m["scale"], m["mask"]["size"])
    o = o * sigmoid(h @ t[p + "g"].T)[:, :, None]
    return o.reshape(n, H * D) @ t[p + "o"].T


def short_convolution(x, w):
    """x [tokens, channels], w [channels, taps]: the last tap meets the current token, zeros stand ahead of the first"""
    taps = w.shape[1]
    out = np.zeros_like(x)
    for i in range(len(x)):
        for j in range(taps):
            if i - (taps - 1 - j) >= 0:
                out[i] += w[:, j] * x[i - (taps - 1 - j)]
    return out


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def delta_rule(q, k, v, decay, beta, S):
    """one head: q, k [n, dim], v [n, vdim], S [dim, vdim] -> outputs, S behind the last token"""
    o = np.zeros_like(v)
    for i in range(len(q)):
        S = decay[i] * S
        S = S + np.outer(k[i], beta[i] * (v[i] - S.T @ k[i]))
        o[i] = S.T @ q[i]
    return o, S


def gated_delta(h, t, p, m, eps):
    n, H, G, D, V = len(h), m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(short_convolution(h @ t[p + x].T, t[p + x + ".conv"])) for x in "qkv")
    q, k, v = unit(q.reshape(n, G, D)) * D ** -0.5, unit(k.reshape(n, G, D)), v.reshape(n, H, V)
    beta = sigmoid(h @ t[p + "b"].T)
    decay = np.exp(-np.exp(t[p + "A_log"]) * softplus(h @ t[p + "a"].T + t[p + "dt_bias"]))
    o = np.zeros((n, H, V), F)
    for a in range(H):
        g = a // (H // G)
        o[:, a], _ = delta_rule(q[:, g], k[:, g], v[:, a], decay[:, a], beta[:, a], np.zeros((D, V), F))
    y = norm_plain(o, t[p + "norm"], eps).reshape(n, H * V) * silu(h @ t[p + "g"].T)
    return y @ t[p + "o"].T


def latent_attention_direct(h, t, p, m, eps):
    """queries straight from the input, pairs of neighbouring elements turn, no sink"""
    n, H, D, R, V = len(h), m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    z = h @ t[p + "dkv"].T
    c = norm_plain(z[:, :m["kv_rank"]], t[p + "dkv.norm"], eps)
    kr = rotate_pairs(z[:, m["kv_rank"]:], range(n), m["rot"])
    q = (h @ t[p + "q"].T).reshape(n, H, D + R)
    qr = rotate_pairs(q[:, :, D:], range(n), m["rot"])
    k, v = (c @ t[p + "uk"].T).reshape(n, H, D), (c @ t[p + "uv"].T).reshape(n, H, V)
    out = np.zeros((n, H, V), F)
    for a in range(H):
        s = (q[:, a, :D] @ k[:, a].T + qr[:, a] @ kr.T) * m["scale"]
        s[np.triu_indices(n, 1)] = -np.inf
        e = np.exp(s - s.max(axis=1, keepdims=True))
        out[:, a] = e / e.sum(axis=1, keepdims=True) @ v[:, a]
    return out.reshape(n, H * V) @ t[p + "o"].T


def distance_penalty(i, j, r1, r2):
    return r1 * np.log(1.0 + r2 * (i - j))


def window_softmax(q, k, v, scale, size, r1, r2):
    """q [n, heads, dim], k [n, kv heads, dim], v [n, kv heads, vdim]: a token sees itself and the size - 1 tokens ahead of it, far ones with a
    penalty that grows with the logarithm of the distance"""
    n, H, _ = q.shape
    out = np.zeros((n, H, v.shape[2]), F)
    for a in range(H):
        g = a // (H // k.shape[1])
        for i in range(n):
            j = np.arange(max(0, i - size + 1), i + 1)
            s = k[j, g] @ q[i, a] * scale - distance_penalty(i, j, r1[a], r2[a])
            e = np.exp(s - s.max())
            out[i, a] = e @ v[j, g] / e.sum()
    return out


def convolved(h, t, name):
    return short_convolution(h @ t[name].T + t[name + ".b"], t[name + ".conv"])


def window_attention(h, t, p, m, shared=None):
    """(output, (keys, values)); shared: the keys and values of another layer"""
    n, H, G, D, V = len(h), m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = convolved(h, t, p + "q").reshape(n, H, D)
    k, v = shared or (convolved(h, t, p + "k").reshape(n, G, D), convolved(h, t, p + "v").reshape(n, G, V))
    size = m["mask"]["size"] if m.get("mask") else n
    o = window_softmax(q, k, v, m["scale"], size, t[p + "r1"], t[p + "r2"]).reshape(n, H * V)
    return (o * sigmoid(h @ t[p + "g"].T)) @ t[p + "o"].T, (k, v)


# ---- feed-forward ----------------------------------------------------------------------------------------------------
def dense_mlp(h, t, p):
    z = relu_squared(h @ t[p + "up"].T + t[p + "up.b"])
    return z @ t[p + "down"].T + t[p + "down.b"]


def expert(h, t, p):
    return relu_squared(h @ t[p + "up"].T) @ t[p + "down"].T


def route(h, router, top, scale):
    """per token: the chosen experts (largest score first) and their weights"""
    z = h @ router.T
    s = np.exp(z - z.max(axis=1, keepdims=True))
    s /= s.sum(axis=1, keepdims=True)
    ids = np.argsort(-s, axis=1, kind="stable")[:, :top]
    w = np.take_along_axis(s, ids, 1)
    return ids, w / (w.sum(axis=1, keepdims=True) + 1e-20) * scale


def expert_mlp(h, t, p, f):
    r = f["router"]
    ids, w = route(h, t[p + "router"], r["top"], r["scale"])
    out = expert(h, t, p + "shared.") if f.get("shared") else np.zeros_like(h)
    for i in range(len(h)):
        for e, x in zip(ids[i], w[i]):
            out[i] += x * expert(h[i:i + 1], t, p + f"e{e}.")[0]
    return out


def gated_mlp(h, t, p, act):
    return (act(h @ t[p + "gate"].T) * (h @ t[p + "up"].T)) @ t[p + "down"].T


def route_corrected(h, router, correction, top):
    """per token: the experts with the largest corrected scores, and their uncorrected scores"""
    z = h @ router.T
    s = np.exp(z - z.max(axis=1, keepdims=True))
    s /= s.sum(axis=1, keepdims=True)
    ids = np.argsort(-(s + correction), axis=1, kind="stable")[:, :top]
    return ids, np.take_along_axis(s, ids, 1)


def expert_or_identity_mlp(h, t, p, f):
    """experts behind the last one with tensors hand their input through"""
    r = f["router"]
    ids, w = route_corrected(h, t[p + "router"], t[p + "correction"], r["top"])
    out = np.zeros_like(h)
    for i in range(len(h)):
        for e, x in zip(ids[i], w[i]):
            out[i] += x * (gated_mlp(h[i:i + 1], t, p + f"e{e}.", silu)[0] if e < r["experts"] else h[i])
    return out


def xielu_mlp(h, t, p):
    return xielu(h @ t[p + "up"].T, *t[p + "act"]) @ t[p + "down"].T


def route_in_groups(h, router, correction, top, groups=None):
    """per token: the experts with the largest corrected scores among the best groups of neighbours, and their uncorrected scores"""
    score = sigmoid(h @ router.T)
    ids = np.zeros((len(h), top), int)
    for i in range(len(h)):
        choice = score[i] + correction
        if groups:
            part = choice.reshape(groups["count"], -1)
            worth = np.sort(part, axis=1)[:, -2:].sum(axis=1)
            keep = np.argsort(-worth, kind="stable")[:groups["keep"]]
            masked = np.full_like(part, -np.inf)
            masked[keep] = part[keep]
            choice = masked.reshape(-1)
        ids[i] = np.argsort(-choice, kind="stable")[:top]
    return ids, np.take_along_axis(score, ids, 1)


def grouped_expert_mlp(h, t, p, f):
    r = f["router"]
    ids, w = route_in_groups(h, t[p + "router"], t[p + "correction"], r["top"], r.get("groups"))
    out = np.zeros_like(h)
    if f.get("shared"):
        out += gated_mlp(h, t, p + "shared.", silu) * sigmoid(h @ t[p + "shared.sg"].T)
    for i in range(len(h)):
        for e, x in zip(ids[i], w[i]):
            out[i] += x * gated_mlp(h[i:i + 1], t, p + f"e{e}.", silu)[0]
    return out


# ---- what a token brings along ----
def bigram_rows(tokens, b):
    """row of the pair table per token: the first token of a sequence has a row of its own"""
    return [b["buckets"] if i == 0 else (int(tokens[i - 1]) * b["mul_prev"] + int(tokens[i]) * b["mul_cur"]) % b["buckets"] for i in range(len(tokens))]


def token_side_input(x, e, t, p, eps):
    g = gelu_tanh(x @ t[p + "gate"].T) * e
    return norm_plain(g @ t[p + "proj"].T, t[p + "norm"], eps)


# ---- the stack -------------------------------------------------------------------------------------------------------
def forward(config, tensors, tokens):
    """(logits [n, vocab], residual stream after every layer run [runs, n, width])"""
    t = {k: np.asarray(v, F) for k, v in tensors.items()}
    return {"Lasapel": forward_lasapel, "Mimolix": forward_mimolix, "Lurepel": forward_lurepel, "Sipelorn": forward_sipelorn}[config["architecture"]](config, t, tokens)


def layer_runs(config):
    """(layer, first of a pass) in the order they run"""
    n, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    body = [(i, i == loop["start"]) for i in range(loop["start"], loop["stop"])]
    return [(i, False) for i in range(loop["start"])] + body * loop["times"] + [(i, False) for i in range(loop["stop"], n)]


def forward_mimolix(config, t, tokens):
    eps, mult = config["norm"]["eps"], config["residual_mult"]
    x0 = t["embed"][np.asarray(tokens)] * config["embedding"]["scale"]
    x, after = x0, []
    for i, enters in layer_runs(config):
        p, layer = f"l{i}.", config["layers"][i]
        if enters:
            x = np.concatenate([x, x0], axis=1) @ t["loop.in"].T
        h = layer_norm(x, t[p + "norm1"], t[p + "norm1.b"], eps)
        y = {"attention": differential_attention, "delta": gated_delta}[layer["type"]](h, t, p + "mix.", layer["mixer"], eps)
        if layer.get("mlp"):
            y = y + expert_mlp(h, t, p + "mlp.", layer["mlp"])
        x = x + mult * y
        after.append(x)
    return layer_norm(x, t["final.norm"], t["final.norm.b"], eps) @ t["head"].T, np.stack(after)


def forward_lasapel(config, t, tokens):
    eps = config["norm"]["eps"]
    x = t["embed"][np.asarray(tokens)]
    after, latents = [], {}
    for i, layer in enumerate(config["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = norm_around_zero(x, t[p + "norm1"], eps)
        if layer["type"] == "latent_attention":
            y, latents[i] = latent_attention(h, t, p + "mix.", m, eps, latents[m["kv_from"]] if "kv_from" in m else None)
        elif layer["type"] == "lightning":
            y = lightning(h, t, p + "mix.", m, eps)
        else:
            raise ValueError(layer["type"])
        x = x + norm_around_zero(y, t[p + "norm1b"], eps) * t[p + "ls1"]
        if layer.get("mlp"):
            y = dense_mlp(norm_around_zero(x, t[p + "norm2"], eps), t, p + "mlp.")
            x = x + norm_around_zero(y, t[p + "norm2b"], eps) * t[p + "ls2"]
        after.append(x)
    return norm_around_zero(x, t["final.norm"], eps) @ t["head"].T, np.stack(after)


def forward_lurepel(config, t, tokens):
    eps = config["norm"]["eps"]
    x = norm_plain(t["embed"][np.asarray(tokens)], t["embed.norm"], eps)
    after = []
    for i, layer in enumerate(config["layers"]):
        p, f = f"l{i}.", layer.get("mlp")
        x = x + norm_plain(chunk_attention(x, t, p + "mix.", layer["mixer"], eps), t[p + "norm1"], eps)
        if f:
            y = gated_mlp(x, t, p + "mlp.", gelu_tanh) if f["kind"] == "dense" else expert_or_identity_mlp(x, t, p + "mlp.", f)
            x = x + norm_plain(y, t[p + "norm2"], eps)
        after.append(x)
    return norm_plain(x, t["final.norm"], eps) @ t["head"].T, np.stack(after)


def forward_sipelorn(config, t, tokens):
    eps, tokens = config["norm"]["eps"], np.asarray(tokens)
    x = t["embed"][tokens] * config["embedding"]["scale"]
    if config["embedding"].get("bigram"):
        x = x + t["bigram"][bigram_rows(tokens, config["embedding"]["bigram"])]
    side = config["token_side"]["dim"] if config.get("token_side") else 0
    after, shared = [], {}

    def gated(y, h, name):
        return y * sigmoid(h @ t[name].T + t[name + ".b"])

    for i, layer in enumerate(config["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer.get("mlp")
        h = layer_norm(x, t[p + "norm1"], t[p + "norm1.b"], eps)
        if layer["type"] == "attention":
            y, shared[i] = window_attention(h, t, p + "mix.", m, shared[m["kv_from"]] if m.get("kv_from") is not None else None)
        else:
            y = latent_attention_direct(h, t, p + "mix.", m, eps)
        x = x + gated(y, h, p + "rg1")
        if f:
            h = layer_norm(x, t[p + "norm2"], t[p + "norm2.b"], eps)
            y = xielu_mlp(h, t, p + "mlp.") if f["kind"] == "dense" else grouped_expert_mlp(h, t, p + "mlp.", f)
            x = x + gated(y, h, p + "rg2")
        if side:
            x = x + token_side_input(x, t["side.embed"][tokens][:, i * side:(i + 1) * side], t, p + "side.", eps)
        after.append(x)
    return layer_norm(x, t["final.norm"], t["final.norm.b"], eps) @ t["head"].T, np.stack(after)
