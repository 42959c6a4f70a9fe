"""Plain, slow restatement of the Letevik design in numpy (float64), one function per mechanism, token by token: the oracle the engine's kernels are held to.
It shares no code with the product path (file reading and bfloat16 rounding come from the other oracle of this folder, which is test infrastructure too).

A model is {"config": <the config.json dictionary>, "tensors": {name: float64 array}}.

Notation.  R(y) = y / sqrt(mean(y^2) + eps), one eps for the whole model.
Embedding:   x = E[token] + P[(prev * mul_prev + token * mul_cur) mod buckets], prev the token before it; a sequence's first token takes P's last row (number `buckets`).
Layer:       x += mixer(R(x) * norm1);  x += ff(R(x) * norm2).
Runs:        layers [start, stop) of `loop` run `times` times in a row with the same tensors and a cache and state per pass; x += loop.step[t] ahead of pass t.
attention    q, k, v = W h, every channel through a causal convolution of `conv` taps (zeros ahead of the sequence);  a query / key head is two maps of `dim` values, each turned in
             pairs (2i, 2i + 1);  token i sees j <= i with i - j < size or j < keep_first;  a1, a2: the maps' soft-max outputs over the same values;
             o = R(a1 - lam a2) (1 - diff) per head, lam = e^(lq1 . lk1) - e^(lq2 . lk2) + diff;  W_o o.
latent_attention   c_q = R(W_dq h) * norm, q = W_uq c_q, per head [dim plain | rot_dim turned];  W_dkv h = [c | r]: c <- R(c) * norm, r turned (one for all heads);
             k = [W_uk c | r], v = W_uv c per head;  all tokens up to i;  soft-max of q . k * scale with one more term e^(sink) in the denominator;  all heads' outputs * sigmoid(W_g h);  W_o.
             Turned here: pairs (i, i + rot_dim / 2).
Feed-forward g = min(W_gate h, limit), u = clip(W_up h, +-limit);  W_down (g sigmoid(1.702 g) (u + 1)).
Output:      E (R(x) * final.norm).
"""
import math

import numpy as np

from tests.fasovik_oracle import bf16_round, read_model, write_model  # noqa: F401  (files and rounding: shared test infrastructure)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-np.asarray(z, np.float64)))


def unit_rms(y, eps):
    return y / np.sqrt((y * y).mean(-1, keepdims=True) + eps)


def softmax(s, sink=None):
    m = s.max() if sink is None else max(s.max(), sink)
    e = np.exp(s - m)
    return e / (e.sum() + (0.0 if sink is None else math.exp(sink - m)))


# ---- embedding -------------------------------------------------------------------------------------------------------------------------
def pair_row(b, prev, token):
    return b["buckets"] if prev is None else (prev * b["mul_prev"] + token * b["mul_cur"]) % b["buckets"]


def embedding(model, prev, token):
    c, T = model["config"], model["tensors"]
    b = (c.get("embedding") or {}).get("bigram")
    return T["embed"][token] + (T["bigram"][pair_row(b, prev, token)] if b else 0.0)


# ---- rotation --------------------------------------------------------------------------------------------------------------------------
def turn(vec, pos, rot, neighbours):
    """the first rot.dims values of `vec` turned by the position; pairs (2i, 2i + 1) or (i, i + dims / 2)"""
    out = np.array(vec, np.float64)
    if not rot:
        return out
    dims = rot["dims"]
    for i in range(dims // 2):
        a = pos * rot["base"] ** (-2.0 * i / dims)
        p, q = (2 * i, 2 * i + 1) if neighbours else (i, i + dims // 2)
        u, v = vec[p], vec[q]
        out[p], out[q] = u * math.cos(a) - v * math.sin(a), v * math.cos(a) + u * math.sin(a)
    return out


# ---- attention -------------------------------------------------------------------------------------------------------------------------
def short_conv(w, past, u):
    """past: the channel inputs of the tokens before this one (may be fewer than the taps need); w [channels][taps], the last tap weighs the token itself"""
    taps = w.shape[1]
    y = w[:, taps - 1] * u
    for back in range(1, taps):
        if back <= len(past):
            y = y + w[:, taps - 1 - back] * past[-back]
    return y


def seen(pos, mask):
    """the positions a token looks at: the last `size` ones and the first `keep_first`"""
    if not mask:
        return list(range(pos + 1))
    return [j for j in range(pos + 1) if pos - j < mask["size"] or j < mask.get("keep_first", 0)]


def lam_of(T, p, c):
    return math.exp(float(T[p + "lq1"] @ T[p + "lk1"])) - math.exp(float(T[p + "lq2"] @ T[p + "lk2"])) + c["diff"]


def combine_maps(a1, a2, lam, diff, eps):
    return unit_rms(a1 - lam * a2, eps) * (1.0 - diff)


def attention_step(T, p, c, eps, h, pos, st):
    H, G, D, V = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    x = {}
    for n in "qkv":
        u = T[p + n] @ h
        if c.get("conv"):
            past = st.setdefault("in_" + n, [])
            x[n] = short_conv(T[p + n + ".conv"], past, u)
            past.append(u)
            del past[:max(0, len(past) - (c["conv"] - 1))]
        else:
            x[n] = u
    q, k = x["q"].reshape(H, 2, D), x["k"].reshape(G, 2, D)
    rot = c.get("rot")
    st.setdefault("k", []).append(np.array([[turn(k[g, m], pos, rot, True) for m in range(2)] for g in range(G)]))
    st.setdefault("v", []).append(x["v"].reshape(G, V))
    toks = seen(pos, c.get("mask"))
    K, Vs = np.stack([st["k"][j] for j in toks]), np.stack([st["v"][j] for j in toks])          # [tokens][G][2][D], [tokens][G][V]
    lam = lam_of(T, p, c)
    out = np.zeros((H, V))
    for a in range(H):
        g = a // (H // G)
        maps = [softmax(K[:, g, m] @ turn(q[a, m], pos, rot, True) * c["scale"]) @ Vs[:, g] for m in range(2)]
        out[a] = combine_maps(maps[0], maps[1], lam, c["diff"], eps)
    return T[p + "o"] @ out.reshape(-1)


# ---- latent attention ------------------------------------------------------------------------------------------------------------------
def latent_attention_step(T, p, c, eps, h, pos, st):
    H, D, R, V, rank = c["heads"], c["dim"], c["rot_dim"], c["vdim"], c["kv_rank"]
    q = (T[p + "uq"] @ (unit_rms(T[p + "dq"] @ h, eps) * T[p + "dq.norm"])).reshape(H, D + R)
    low = T[p + "dkv"] @ h
    rot = c.get("rot")
    st.setdefault("c", []).append(unit_rms(low[:rank], eps) * T[p + "dkv.norm"])
    st.setdefault("r", []).append(turn(low[rank:], pos, rot, False))
    C, Rk = np.stack(st["c"]), np.stack(st["r"])
    uk, uv = T[p + "uk"].reshape(H, D, rank), T[p + "uv"].reshape(H, V, rank)
    out = np.zeros((H, V))
    for a in range(H):
        s = (C @ uk[a].T) @ q[a, :D] + Rk @ turn(q[a, D:], pos, rot, False)
        out[a] = softmax(s * c["scale"], float(T[p + "sink"][a])) @ (C @ uv[a].T)
    return T[p + "o"] @ (out.reshape(-1) * sigmoid(T[p + "g"] @ h))


def feed_forward(T, p, c, h):
    g, u = T[p + "gate"] @ h, T[p + "up"] @ h
    if c.get("limit") is not None:
        g, u = np.minimum(g, c["limit"]), np.clip(u, -c["limit"], c["limit"])
    return T[p + "down"] @ (g * sigmoid(1.702 * g) * (u + 1.0))


# ---- the model -------------------------------------------------------------------------------------------------------------------------
def run_order(c):
    """[(layer, the pass it opens or None)] in the order the layers run"""
    n, loop = len(c["layers"]), c.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    return [(i, None) for i in range(a)] + [(i, t if i == a else None) for t in range(loop["times"]) for i in range(a, b)] + [(i, None) for i in range(b, n)]


def new_state():
    return {"pos": 0, "prev": None, "runs": {}}


def step(model, state, token, layers_out=None):
    """one token of one sequence through the model; returns the logits.  layers_out (a list) receives the stream after every layer run"""
    c, T = model["config"], model["tensors"]
    eps, pos = c["norm"]["eps"], state["pos"]
    x = embedding(model, state["prev"], token)
    for r, (i, opens) in enumerate(run_order(c)):
        L, p = c["layers"][i], "l%d." % i
        if opens is not None:
            x = x + T["loop.step"][opens]
        st = state["runs"].setdefault(r, {})
        h = unit_rms(x, eps) * T[p + "norm1"]
        if L["type"] == "attention":
            x = x + attention_step(T, p + "mix.", L["mixer"], eps, h, pos, st)
        elif L["type"] == "latent_attention":
            x = x + latent_attention_step(T, p + "mix.", L["mixer"], eps, h, pos, st)
        else:
            raise ValueError(L["type"])
        if L.get("mlp"):
            x = x + feed_forward(T, p + "mlp.", L["mlp"], unit_rms(x, eps) * T[p + "norm2"])
        if layers_out is not None:
            layers_out.append(x)
    state["pos"], state["prev"] = pos + 1, token
    return T["embed"] @ (unit_rms(x, eps) * T["final.norm"])


def run(model, tokens, state=None, layers=None):
    """logits [len(tokens)][vocab] of a sequence (continued from `state`); layers (a list) receives [layer runs][width] per token"""
    state = new_state() if state is None else state
    out = []
    for t in tokens:
        lo = [] if layers is not None else None
        out.append(step(model, state, int(t), lo))
        if layers is not None:
            layers.append(np.stack(lo))
    return np.stack(out)


def greedy(model, prompt, n):
    state = new_state()
    lg = run(model, prompt, state)[-1]
    out = []
    for _ in range(n):
        out.append(int(np.argmax(lg)))
        lg = step(model, state, out[-1])
    return out


# ---- random models for the tests -------------------------------------------------------------------------------------------------------
def dense(ff, limit=1.2):
    return {"kind": "dense", "ff": ff, "limit": limit} if ff else None


def attention_layer(heads=4, kv_heads=2, dim=10, vdim=6, conv=3, size=9, keep_first=2, rot_dims=6, base=300.0, scale=0.9, diff=0.3, ff=None, limit=1.2):
    mx = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "diff": diff}
    if conv:
        mx["conv"] = conv
    if size:
        mx["mask"] = {"size": size, "keep_first": keep_first}
    if rot_dims:
        mx["rot"] = {"dims": rot_dims, "base": base}
    return {"type": "attention", "mixer": mx, "mlp": dense(ff, limit)}


def latent_layer(heads=3, dim=7, rot_dim=6, vdim=5, q_rank=11, kv_rank=12, base=300.0, scale=0.6, ff=None, limit=1.2):
    mx = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale}
    if rot_dim:
        mx["rot"] = {"dims": rot_dim, "base": base}
    return {"type": "latent_attention", "mixer": mx, "mlp": dense(ff, limit)}


def random_model(rng, vocab, width, layers, loop=None, buckets=37, mul_prev=11, mul_cur=5, eps=1e-5):
    """weights rounded to bfloat16 (what the file holds), sized so that every mechanism matters in the logits"""
    def rb(a):
        return bf16_round(np.asarray(a, np.float32)).astype(np.float64)

    def w(*shape, s=None):
        return rb(rng.standard_normal(shape) * (s if s is not None else 1.0 / np.sqrt(shape[-1])))

    def near_one(n):
        return rb(1.0 + 0.3 * rng.standard_normal(n))

    T = {"embed": w(vocab, width, s=0.8), "final.norm": near_one(width)}
    if buckets:
        T["bigram"] = w(buckets + 1, width, s=0.6)
    if loop:
        T["loop.step"] = w(loop["times"], width, s=0.7)
    for i, L in enumerate(layers):
        p, mx, m = "l%d." % i, L["mixer"], "l%d.mix." % i
        T[p + "norm1"] = near_one(width)
        H, D, V = mx["heads"], mx["dim"], mx["vdim"]
        if L["type"] == "attention":
            G = mx["kv_heads"]
            for n, rows in (("q", 2 * H * D), ("k", 2 * G * D), ("v", G * V)):
                T[m + n] = w(rows, width)
                if mx.get("conv"):
                    T[m + n + ".conv"] = rb(0.5 * rng.standard_normal((rows, mx["conv"])) + np.eye(mx["conv"])[-1])
            for n in ("lq1", "lk1", "lq2", "lk2"):
                T[m + n] = w(D, s=0.6 / np.sqrt(D))
        else:
            R, rank, qr = mx["rot_dim"], mx["kv_rank"], mx["q_rank"]
            T[m + "dq"], T[m + "dq.norm"], T[m + "uq"] = w(qr, width), near_one(qr), w(H * (D + R), qr)
            T[m + "dkv"], T[m + "dkv.norm"] = w(rank + R, width), near_one(rank)
            T[m + "uk"], T[m + "uv"] = w(H * D, rank), w(H * V, rank)
            T[m + "sink"], T[m + "g"] = rb(1.0 + rng.standard_normal(H)), w(H * V, width, s=2.0 / np.sqrt(width))
        T[m + "o"] = w(width, H * V)
        if L.get("mlp"):
            ff = L["mlp"]["ff"]
            T[p + "norm2"] = near_one(width)
            T[p + "mlp.gate"], T[p + "mlp.up"], T[p + "mlp.down"] = w(ff, width, s=1.5 / np.sqrt(width)), w(ff, width, s=1.5 / np.sqrt(width)), w(width, ff)
    config = {"architecture": "Letevik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": [dict(L) for L in layers]}
    if buckets:
        config["embedding"] = {"bigram": {"buckets": buckets, "mul_prev": mul_prev, "mul_cur": mul_cur}}
    if loop:
        config["loop"] = dict(loop)
    return {"config": config, "tensors": T}
