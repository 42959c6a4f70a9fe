"""Plain, slow restatement of the Rerizen design in numpy (float64), one function per mechanism, token by token: the oracle the engine's kernels are held to.
It shares no code with the product path (file reading and bfloat16 rounding come from the other oracle of this folder, which is test infrastructure too).

A model is {"config": <the config.json dictionary>, "tensors": {name: float64 array}}.

Notation.  R(y) = y / sqrt(mean(y^2) + eps), one eps for the whole model.
Streams:     the residual is X [streams][width], every row the embedding row at first.  A sublayer (mixer: hc1, feed-forward: hc2) reads u = in . X, h = R(u) * norm, and
             with y = sublayer(h):  X'[t] = sum_s mix[s][t] X[s] + out[t] y.  Behind the last layer x = sum_s X[s].
mlstm        q, k [heads][dim], v [heads][vdim], g = W h;  i = cap tanh((W_i h + b_i) / cap), f = log sigmoid(cap tanh((W_f h + b_f) / cap)) per head;
             m' = max(f + m, i);  S' = e^(f + m - m') S + e^(i - m') k v^T,  n' likewise with k;  o = S'^T q' / (max(|n' . q'|, e^(-m')) + 1e-6), q' = q / sqrt(dim);
             all of S, n, m start at zero;  y = W_o (R(o) per head * norm * sigmoid(g)).
attention    q [heads][dim], k, v [kv_heads] = W h + b;  q, k <- R(.) per head;  q <- q (1 + coef ln(floor((pos + 1) / every) + 1));  causal soft-max of q . k * scale;  W_o.
             kv_from: the layer computes q only and reads the keys and values of that layer.
latent_attention   c_q = R(W_dq h) * norm, q = W_uq c_q, per head [dim plain | rot_dim turned];  W_dkv h = [c | r]: c <- R(c) * norm, r turned (one for all heads);
             k = [W_uk c | r], v = W_uv c per head;  tokens 0 <= i - j < size;  soft-max of q . k * scale;  head h's output * sigmoid(W_g h)_h;  W_o.
             Turned: pairs (2i, 2i + 1) by pos * f_i; long wavelengths slowed down along a ramp over the pair index, cos and sin stretched.
Feed-forward W_down (silu(W_gate h) * W_up h).
Output:      head @ (R(x) * final.norm) * logit_scale.
"""
import math

import numpy as np

from tests.fasovik_oracle import bf16_round, read_model, write_model  # noqa: F401  (files and rounding: shared test infrastructure)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-np.asarray(z, np.float64)))


def log_sigmoid(z):
    return -np.logaddexp(0.0, -np.asarray(z, np.float64))


def silu(z):
    return z * sigmoid(z)


def unit_rms(y, eps):
    return y / np.sqrt((y * y).mean(-1, keepdims=True) + eps)


def softmax(s):
    e = np.exp(s - s.max())
    return e / e.sum()


# ---- the residual streams --------------------------------------------------------------------------------------------------------------
def streams_read(T, p, X):
    return T[p + "in"] @ X


def streams_write(T, p, X, y):
    n = X.shape[0]
    return np.stack([sum(T[p + "mix"][s, t] * X[s] for s in range(n)) + T[p + "out"][t] * y for t in range(n)])


# ---- mlstm -----------------------------------------------------------------------------------------------------------------------------
def capped(z, cap):
    return cap * np.tanh(z / cap)


def memory_gates(T, p, cap, h, m):
    """log gates and the running maximum: (forget factor, input factor, new maximum) per head"""
    i = capped(T[p + "i"] @ h + T[p + "i.b"], cap)
    f = log_sigmoid(capped(T[p + "f"] @ h + T[p + "f.b"], cap))
    new = np.maximum(f + m, i)
    return np.exp(f + m - new), np.exp(i - new), new


def memory_step(S, n, forget, put, k, v):
    return forget * S + put * np.outer(k, v), forget * n + put * k


def memory_read(S, n, q, m):
    return S.T @ q / (max(abs(float(n @ q)), math.exp(-m)) + 1e-6)


def mlstm_step(T, p, c, eps, h, st):
    H, D, V = c["heads"], c["dim"], c["vdim"]
    q, k, v = (T[p + "q"] @ h).reshape(H, D) / math.sqrt(D), (T[p + "k"] @ h).reshape(H, D), (T[p + "v"] @ h).reshape(H, V)
    S, n, m = st.get("S", np.zeros((H, D, V))), st.get("n", np.zeros((H, D))), st.get("m", np.zeros(H))
    forget, put, m = memory_gates(T, p, c["gate_cap"], h, m)
    out = np.zeros((H, V))
    S, n = S.copy(), n.copy()
    for a in range(H):
        S[a], n[a] = memory_step(S[a], n[a], forget[a], put[a], k[a], v[a])
        out[a] = unit_rms(memory_read(S[a], n[a], q[a], m[a]), eps)
    st["S"], st["n"], st["m"] = S, n, m
    return T[p + "o"] @ (out.reshape(-1) * T[p + "norm"] * sigmoid(T[p + "g"] @ h))


# ---- attention -------------------------------------------------------------------------------------------------------------------------
def temperature(c, pos):
    qt = c.get("q_temp")
    return 1.0 + qt["coef"] * math.log((pos + 1) // qt["every"] + 1) if qt else 1.0


def attention_step(T, p, c, eps, h, pos, st, shared=None):
    """shared: the state of the layer whose keys and values this one reads (it has taken this token already)"""
    H, G, D, V = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q = unit_rms((T[p + "q"] @ h + T[p + "q.b"]).reshape(H, D), eps) * temperature(c, pos)
    if shared is None:
        st.setdefault("k", []).append(unit_rms((T[p + "k"] @ h + T[p + "k.b"]).reshape(G, D), eps))
        st.setdefault("v", []).append((T[p + "v"] @ h + T[p + "v.b"]).reshape(G, V))
        shared = st
    K, Vs = np.stack(shared["k"]), np.stack(shared["v"])               # [tokens][G][.]
    out = np.zeros((H, V))
    for a in range(H):
        g = a // (H // G)
        out[a] = softmax(K[:, g] @ q[a] * c["scale"]) @ Vs[:, g]
    return T[p + "o"] @ out.reshape(-1)


# ---- latent attention ------------------------------------------------------------------------------------------------------------------
def turn_steps(rot):
    """(angle per position of every pair, factor on cos and sin)"""
    dims, base = rot["dims"], rot["base"]
    f = np.array([base ** (-2.0 * i / dims) for i in range(dims // 2)])
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0

    def index_of(turns):                                              # the (fractional) pair index whose wavelength makes `turns` turns over the original length
        return dims * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(index_of(sc["fast"])), 0), min(math.ceil(index_of(sc["slow"])), dims - 1)
    ramp = np.clip((np.arange(dims // 2) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / sc["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(sc["factor"]) + 1.0


def turn(vec, pos, rot):
    out = np.array(vec, np.float64)
    f, amp = turn_steps(rot)
    for i, fi in enumerate(f):
        c, s = amp * math.cos(pos * fi), amp * math.sin(pos * fi)
        u, v = vec[2 * i], vec[2 * i + 1]
        out[2 * i], out[2 * i + 1] = u * c - v * s, v * c + u * s
    return out


def seen(pos, size):
    return range(max(0, pos - size + 1) if size else 0, pos + 1)


def latent_attention_step(T, p, c, eps, h, pos, st):
    H, D, R, V, rank = c["heads"], c["dim"], c["rot_dim"], c["vdim"], c["kv_rank"]
    q = (T[p + "uq"] @ (unit_rms(T[p + "dq"] @ h, eps) * T[p + "dq.norm"])).reshape(H, D + R)
    low = T[p + "dkv"] @ h
    st.setdefault("c", []).append(unit_rms(low[:rank], eps) * T[p + "dkv.norm"])
    st.setdefault("r", []).append(turn(low[rank:], pos, c["rot"]))
    toks = list(seen(pos, (c.get("mask") or {}).get("size")))
    C, Rk = np.stack([st["c"][j] for j in toks]), np.stack([st["r"][j] for j in toks])
    gate = sigmoid(T[p + "g"] @ h)
    uk, uv = T[p + "uk"].reshape(H, D, rank), T[p + "uv"].reshape(H, V, rank)
    out = np.zeros((H, V))
    for a in range(H):
        s = (C @ uk[a].T) @ q[a, :D] + Rk @ turn(q[a, D:], pos, c["rot"])
        out[a] = gate[a] * (softmax(s * c["scale"]) @ (C @ uv[a].T))
    return T[p + "o"] @ out.reshape(-1)


def feed_forward(T, p, h):
    return T[p + "down"] @ (silu(T[p + "gate"] @ h) * (T[p + "up"] @ h))


# ---- the model -------------------------------------------------------------------------------------------------------------------------
def new_state():
    return {"pos": 0, "layers": {}}


def step(model, state, token, layers_out=None):
    """one token of one sequence through the model; returns the logits.  layers_out (a list) receives the sum of the streams after every layer"""
    c, T = model["config"], model["tensors"]
    eps, pos = c["norm"]["eps"], state["pos"]
    X = np.repeat(T["embed"][token][None], c["streams"], axis=0)
    for i, L in enumerate(c["layers"]):
        p, mx = "l%d." % i, L["mixer"]
        st = state["layers"].setdefault(i, {})
        h = unit_rms(streams_read(T, p + "hc1.", X), eps) * T[p + "norm1"]
        if L["type"] == "mlstm":
            y = mlstm_step(T, p + "mix.", mx, eps, h, st)
        elif L["type"] == "attention":
            y = attention_step(T, p + "mix.", mx, eps, h, pos, st, state["layers"][mx["kv_from"]] if mx.get("kv_from") is not None else None)
        elif L["type"] == "latent_attention":
            y = latent_attention_step(T, p + "mix.", mx, eps, h, pos, st)
        else:
            raise ValueError(L["type"])
        X = streams_write(T, p + "hc1.", X, y)
        if L.get("mlp"):
            h = unit_rms(streams_read(T, p + "hc2.", X), eps) * T[p + "norm2"]
            X = streams_write(T, p + "hc2.", X, feed_forward(T, p + "mlp.", h))
        if layers_out is not None:
            layers_out.append(X.sum(0))
    state["pos"] = pos + 1
    return T["head"] @ (unit_rms(X.sum(0), eps) * T["final.norm"]) * c["logit_scale"]


def run(model, tokens, state=None, layers=None):
    """logits [len(tokens)][vocab] of a sequence (continued from `state`); layers (a list) receives [layers][width] per token"""
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
def mlstm_layer(heads=3, dim=8, vdim=6, cap=5.0, ff=None):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}, "mlp": dense(ff)}


def attention_layer(heads=4, kv_heads=2, dim=10, vdim=6, coef=0.4, every=5, scale=0.9, kv_from=None, ff=None):
    mx = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if coef is not None:
        mx["q_temp"] = {"coef": coef, "every": every}
    if kv_from is not None:
        mx["kv_from"] = kv_from
    return {"type": "attention", "mixer": mx, "mlp": dense(ff)}


def latent_layer(heads=3, dim=7, rot_dim=6, vdim=5, q_rank=11, kv_rank=12, size=9, base=300.0, scaling=(4.0, 8.0, 1.0, 48), scale=0.6, ff=None):
    mx = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale, "rot": {"dims": rot_dim, "base": base}}
    if scaling:
        mx["rot"]["scaling"] = dict(zip(("factor", "fast", "slow", "original"), scaling))
    if size:
        mx["mask"] = {"size": size}
    return {"type": "latent_attention", "mixer": mx, "mlp": dense(ff)}


def dense(ff):
    return {"kind": "dense", "ff": ff} if ff else None


def random_model(rng, vocab, width, layers, streams=3, eps=1e-5, logit_scale=0.7):
    """weights rounded to bfloat16 (what the file holds), sized so that every mechanism matters in the logits"""
    def rb(a):
        return bf16_round(np.asarray(a, np.float32)).astype(np.float64)

    def w(*shape, s=None):
        return rb(rng.standard_normal(shape) * (s if s is not None else 1.0 / np.sqrt(shape[-1])))

    def near_one(n):
        return rb(1.0 + 0.3 * rng.standard_normal(n))

    def connections(p):
        T[p + "in"], T[p + "out"] = rb(1.0 / streams + 0.4 * rng.standard_normal(streams)), rb(1.0 + 0.5 * rng.standard_normal(streams))
        T[p + "mix"] = rb(0.8 * np.eye(streams) + 0.25 * rng.standard_normal((streams, streams)))

    T = {"embed": w(vocab, width, s=0.8), "final.norm": near_one(width), "head": w(vocab, width)}
    for i, L in enumerate(layers):
        p, mx, m = "l%d." % i, L["mixer"], "l%d.mix." % i
        T[p + "norm1"] = near_one(width)
        connections(p + "hc1.")
        H, D, V = mx["heads"], mx["dim"], mx["vdim"]
        if L["type"] == "mlstm":
            T[m + "q"], T[m + "k"], T[m + "v"], T[m + "g"], T[m + "o"] = w(H * D, width), w(H * D, width), w(H * V, width), w(H * V, width), w(width, H * V)
            T[m + "norm"] = near_one(H * V)
            T[m + "i"], T[m + "i.b"] = w(H, width, s=2.5 / np.sqrt(width)), rb(rng.standard_normal(H) - 0.5)
            T[m + "f"], T[m + "f.b"] = w(H, width, s=2.0 / np.sqrt(width)), rb(rng.standard_normal(H) + 2.0)
        elif L["type"] == "attention":
            G = mx["kv_heads"]
            names = [("q", H * D)] + ([] if mx.get("kv_from") is not None else [("k", G * D), ("v", G * V)])
            for n, rows in names:
                T[m + n], T[m + n + ".b"] = w(rows, width), w(rows, s=0.4)
            T[m + "o"] = w(width, H * V)
        else:
            R, rank, qr = mx["rot_dim"], mx["kv_rank"], mx["q_rank"]
            T[m + "dq"], T[m + "dq.norm"], T[m + "uq"] = w(qr, width), near_one(qr), w(H * (D + R), qr)
            T[m + "dkv"], T[m + "dkv.norm"] = w(rank + R, width), near_one(rank)
            T[m + "uk"], T[m + "uv"] = w(H * D, rank), w(H * V, rank)
            T[m + "g"], T[m + "o"] = w(H, width, s=2.0 / np.sqrt(width)), w(width, H * V)
        if L.get("mlp"):
            T[p + "norm2"] = near_one(width)
            connections(p + "hc2.")
            ff = L["mlp"]["ff"]
            T[p + "mlp.gate"], T[p + "mlp.up"], T[p + "mlp.down"] = w(ff, width), w(ff, width), w(width, ff)
    config = {"architecture": "Rerizen", "vocab": vocab, "width": width, "streams": streams, "logit_scale": logit_scale, "norm": {"eps": eps}, "layers": [dict(L) for L in layers]}
    return {"config": config, "tensors": T}
