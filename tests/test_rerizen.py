"""The Rerizen design (residual streams mixed around every sublayer; a normalised matrix memory with exponential gates, attention with a query temperature over keys of its own or of another
layer, windowed latent attention behind a query latent with a rotated part and a head gate; a gated dense feed-forward) on the engine, held to the plain numpy restatement in
tests/rerizen_oracle.py: every mechanism alone through its operator, then whole models through llama_decode — prompts against token-by-token decoding, portions down to two tokens, batches of
unequal requests, cells and state slots freed and used again, keys far away and at the borders of windows, long decoding, greedy generation, the trace runner.  Models are small, random and
made here; sizes are chosen so that nothing that could be mixed up is equal."""
import ctypes as C
import json
import math
import os

import numpy as np
import pytest

from pipeinfer_amd import lib as L, llama as LL
from tests import rerizen_oracle as O

BF16 = 30
F = 1 << 30                                    # "this sequence starts from nothing" on the first token of a run (slot words)
NONE, SILU, SIGMOID = 0, 1, 2
SOFTMAX, WINDOW = 1, 1
NORM_LAST, NORM_FIRST = 0, 1
NEIGHBOURS = 1


def rel_rms(got, want):
    d = np.asarray(got, np.float64) - np.asarray(want, np.float64)
    return float(np.sqrt((d * d).mean()) / (np.sqrt((np.asarray(want, np.float64) ** 2).mean()) + 1e-30))


def logit_err(got, want):
    d = np.asarray(got, np.float64) - want
    d = d - d.mean(-1, keepdims=True)
    return np.sqrt((d * d).mean(-1)) / (want - want.mean(-1, keepdims=True)).std()


TOL = {True: 3e-4, False: 6e-2}          # exact (fp32) / serving precision (bfloat16 matrix inputs)


def within(err, exact, tol=None):
    """fp32: every position within the tolerance.  Serving precision is held to the float64 restatement too, whose distance is the rounding of bfloat16 matrix inputs: nine positions in ten; the
    fp32 runs of the same tests are the sharp ones"""
    tol = tol if tol is not None else TOL[exact]
    return err.max() < tol if exact else np.quantile(err, 0.9) < tol


VOCAB = 79
# layer mixes and stream counts: the default one, the values another model may make equal or one, wide heads, one kind of layer only, keys shared over a distance and twice
VARIANTS = {
    "mixed": (None, 3),
    "edges": ([O.mlstm_layer(heads=1, dim=1, vdim=1, cap=2.0, ff=1), O.latent_layer(heads=1, dim=1, rot_dim=2, vdim=1, q_rank=1, kv_rank=2, size=1, ff=None),
               O.attention_layer(heads=1, kv_heads=1, dim=2, vdim=2, every=1, ff=3), O.latent_layer(heads=2, dim=4, rot_dim=4, vdim=4, q_rank=4, kv_rank=4, size=None, scaling=None, ff=4),
               O.attention_layer(heads=3, kv_heads=1, dim=2, vdim=2, coef=None, kv_from=2, ff=None)], 1),
    "wide_heads": ([O.latent_layer(heads=4, dim=70, rot_dim=66, vdim=40, q_rank=72, kv_rank=136, size=23, base=5000.0, scaling=(8.0, 32.0, 1.0, 96), scale=0.1, ff=96),
                    O.mlstm_layer(heads=2, dim=72, vdim=130, cap=15.0, ff=40), O.attention_layer(heads=6, kv_heads=2, dim=136, vdim=66, scale=0.3, every=7, ff=None)], 2),
    "only_memory": ([O.mlstm_layer(), O.mlstm_layer(heads=5, dim=3, vdim=11, cap=8.0, ff=12)], 4),
    "only_attention": ([O.attention_layer(ff=8), O.attention_layer(heads=6, kv_from=0), O.attention_layer(heads=2, kv_heads=1, dim=4, vdim=8, coef=-0.2, every=3), O.attention_layer(heads=2, coef=0.1, every=40, kv_from=0, ff=5)], 2),
    "only_latent": ([O.latent_layer(ff=9), O.latent_layer(heads=2, dim=3, rot_dim=8, vdim=9, q_rank=5, kv_rank=6, size=4, base=40.0, scaling=(2.0, 4.0, 2.0, 64)), O.latent_layer(heads=5, size=4)], 5),
    "many_streams": ([O.attention_layer(), O.mlstm_layer(ff=6), O.latent_layer()], 9),
}


def default_layers():
    return [O.mlstm_layer(ff=24), O.attention_layer(ff=20), O.latent_layer(ff=18), O.attention_layer(heads=2, coef=0.25, every=11, scale=0.7, kv_from=1, ff=None),
            O.mlstm_layer(heads=2, dim=5, vdim=9, cap=9.0, ff=None), O.latent_layer(heads=4, dim=3, rot_dim=4, vdim=8, q_rank=9, kv_rank=7, size=14, base=90.0, scaling=(3.0, 6.0, 1.0, 30), ff=22)]


def small_model(seed=0, width=40, vocab=VOCAB, layers=None, streams=3, **kw):
    return O.random_model(np.random.default_rng(seed), vocab, width, layers or default_layers(), streams=streams, **kw)


def variant_model(name, seed=11):
    layers, streams = VARIANTS[name]
    return small_model(seed=seed, layers=layers, streams=streams, width={"wide_heads": 64, "edges": 18, "only_latent": 37}.get(name, 40))


def write(folder, m):
    O.write_model(folder, m["config"], {k: v.astype(np.float32) for k, v in m["tensors"].items()})


class Engine:
    def __init__(self, tmp_path, model, n_ctx=256, n_batch=64, exact=True, slots=4, name="m"):
        folder = os.path.join(str(tmp_path), name)
        write(folder, model)
        self.model = LL.Model(folder)
        self.ctx = LL.Context(self.model, n_ctx=n_ctx, n_batch=n_batch)
        self.ctx.set_state_slots(slots)
        self.ctx.set_precision(exact)

    def close(self):
        self.ctx.free()
        self.model.free()


# ---- without a GPU ---------------------------------------------------------------------------------------------------------------
def test_model_folder_is_read_and_described(tmp_path):
    for name in VARIANTS:                                            # also without a window, a temperature, stretched steps, a feed-forward, with shared keys
        folder = str(tmp_path / name)
        write(folder, variant_model(name, seed=1))
        mod = LL.Model(folder)
        assert mod.n_vocab == VOCAB
        buf = C.create_string_buffer(64)
        mod.lib.llama_model_desc.argtypes = [C.c_void_p, C.c_char_p, C.c_size_t]
        mod.lib.llama_model_desc(mod.h, buf, 64)
        assert buf.value.lower().startswith(b"rerizen")
        mod.free()


@pytest.mark.parametrize("breakage", ["type", "kv_heads", "rot", "rot_dims", "kind", "streams", "kv_later", "kv_type", "kv_sizes", "kv_chain", "cap", "scaling", "every", "logit_scale"])
def test_a_wrong_description_is_refused(tmp_path, breakage):
    m = small_model()
    cfg = json.loads(json.dumps(m["config"]))
    mx = [l["mixer"] for l in cfg["layers"]]
    if breakage == "type":
        cfg["layers"][0]["type"] = "slstm"
    elif breakage == "kv_heads":
        mx[1]["kv_heads"] = 3
    elif breakage == "rot":
        mx[2]["rot"]["base"] = 0
    elif breakage == "rot_dims":
        mx[2]["rot"]["dims"] = 4
    elif breakage == "kind":
        cfg["layers"][0]["mlp"]["kind"] = "moe"
    elif breakage == "streams":
        cfg["streams"] = 0
    elif breakage == "kv_later":
        mx[3]["kv_from"] = 3
    elif breakage == "kv_type":
        mx[3]["kv_from"] = 2
    elif breakage == "kv_sizes":
        mx[3]["dim"] = 8
    elif breakage == "kv_chain":
        cfg["layers"].append(json.loads(json.dumps(cfg["layers"][3])))
        cfg["layers"][-1]["mixer"]["kv_from"] = 3
    elif breakage == "cap":
        mx[0]["gate_cap"] = 0
    elif breakage == "scaling":
        del mx[2]["rot"]["scaling"]["slow"]
    elif breakage == "every":
        mx[1]["q_temp"]["every"] = 0
    elif breakage == "logit_scale":
        del cfg["logit_scale"]
    folder = str(tmp_path / "bad")
    O.write_model(folder, cfg, {k: v.astype(np.float32) for k, v in m["tensors"].items()})
    with pytest.raises(L.PipeInferError):
        LL.Model(folder)


@pytest.mark.gpu
@pytest.mark.parametrize("breakage", ["missing", "shape", "mix"])
def test_a_wrong_tensor_is_refused_when_the_weights_load(tmp_path, breakage):
    m = small_model()
    tensors = dict(m["tensors"])
    if breakage == "missing":
        del tensors["l1.mix.v.b"]
    elif breakage == "shape":
        tensors["l2.mix.dkv"] = tensors["l2.mix.dkv"][:-1]
    else:
        tensors["l0.hc2.mix"] = tensors["l0.hc2.mix"][:, :-1]
    folder = str(tmp_path / "bad")
    O.write_model(folder, m["config"], {k: v.astype(np.float32) for k, v in tensors.items()})
    mod = LL.Model(folder)
    ctx = LL.Context(mod, n_ctx=32, n_batch=8)
    with pytest.raises(L.PipeInferError):
        ctx.decode([1], [0], [[0]])
    ctx.free()
    mod.free()


def test_oracle_mechanisms_behave_as_stated():
    """the restatement itself: streams mixed [from][to], the memory independent of where its running maximum starts (but for the normaliser's floor), temperatures constant inside a block of
    positions, rotations that depend on the distance only, the ramp's ends, windows"""
    T = {"a.mix": np.array([[1.0, 2.0], [3.0, 4.0]]), "a.out": np.array([10.0, 100.0]), "a.in": np.array([1.0, -1.0])}
    X = np.array([[1.0, 0.0], [0.0, 1.0]])
    assert np.allclose(O.streams_write(T, "a.", X, np.array([1.0, 1.0])), [[1 + 10, 3 + 10], [2 + 100, 4 + 100]]) and np.allclose(O.streams_read(T, "a.", X), [1.0, -1.0])
    rng = np.random.default_rng(1)
    # the memory, un-normalised: S_t = sum_j exp(i_j + sum f) k v^T, whatever the maximum subtracted on the way
    H, D, V, n = 1, 3, 2, 6
    G = {"i": rng.standard_normal((H, 4)), "i.b": np.array([-1.0]), "f": rng.standard_normal((H, 4)), "f.b": np.array([1.0])}
    hs, ks, vs, q = rng.standard_normal((n, 4)), rng.standard_normal((n, D)), rng.standard_normal((n, V)), rng.standard_normal(D)
    S, nn, m = np.zeros((D, V)), np.zeros(D), np.zeros(H)
    logs = []
    for t in range(n):
        a, b, m = O.memory_gates(G, "", 4.0, hs[t], m)
        S, nn = O.memory_step(S, nn, a[0], b[0], ks[t], vs[t])
        logs.append((O.capped(G["i"] @ hs[t] + G["i.b"], 4.0)[0], O.log_sigmoid(O.capped(G["f"] @ hs[t] + G["f.b"], 4.0))[0]))
    w = [math.exp(logs[j][0] + sum(f for _, f in logs[j + 1:])) for j in range(n)]
    S_true = sum(w[j] * np.outer(ks[j], vs[j]) for j in range(n))
    n_true = sum(w[j] * ks[j] for j in range(n))
    assert np.allclose(S * math.exp(m[0]), S_true) and np.allclose(nn * math.exp(m[0]), n_true)
    assert np.allclose(O.memory_read(S, nn, q, m[0]), S_true.T @ q / max(abs(n_true @ q), 1.0), rtol=1e-4)      # the floor e^-m is 1 on the un-normalised scale
    c = {"q_temp": {"coef": 0.5, "every": 4}}
    assert O.temperature(c, 0) == O.temperature(c, 2) == 1.0 and O.temperature(c, 3) == O.temperature(c, 6) == 1.0 + 0.5 * math.log(2.0) and O.temperature({}, 99) == 1.0
    rot = {"dims": 6, "base": 100.0, "scaling": {"factor": 4.0, "fast": 8.0, "slow": 1.0, "original": 64}}
    a, b = rng.standard_normal(6), rng.standard_normal(6)
    assert np.isclose(O.turn(a, 9, rot) @ O.turn(b, 5, rot), O.turn(a, 104, rot) @ O.turn(b, 100, rot))
    assert np.isclose(np.linalg.norm(O.turn(a, 7, rot)), np.linalg.norm(a) * (0.1 * math.log(4.0) + 1.0))
    f, _ = O.turn_steps({"dims": 32, "base": 10000.0, "scaling": {"factor": 4.0, "fast": 32.0, "slow": 1.0, "original": 4096}})
    plain = 10000.0 ** (-np.arange(16) / 16.0)
    assert f[0] == plain[0] and np.isclose(f[15], plain[15] / 4.0) and (np.diff(f) < 0).all() and plain[9] / 4 < f[9] < plain[9]
    assert list(O.seen(5, 3)) == [3, 4, 5] and list(O.seen(1, 3)) == [0, 1] and list(O.seen(4, None)) == [0, 1, 2, 3, 4] and list(O.seen(4, 1)) == [4]


def test_oracle_is_sensitive_to_every_constant():
    """each constant of the description and each small tensor changes the logits by far more than the tolerances of this file, so that a wrong one would show"""
    m = small_model(seed=3)
    toks = [int(t) for t in np.random.default_rng(4).integers(0, VOCAB, 26)]
    want = O.run(m, toks)

    def off(edit):
        cfg, T = json.loads(json.dumps(m["config"])), dict(m["tensors"])
        edit(cfg, T)
        return logit_err(O.run({"config": cfg, "tensors": T}, toks), want).max()

    def mixer(i, **kw):
        return lambda c, T: c["layers"][i]["mixer"].update(kw)

    def zero(name):
        return lambda c, T: T.update({name: np.zeros_like(T[name])})
    edits = [mixer(0, gate_cap=6.0), mixer(1, scale=1.0), mixer(1, q_temp={"coef": 0.4, "every": 6}), mixer(1, q_temp={"coef": 0.5, "every": 5}), mixer(2, mask={"size": 8}), mixer(2, mask={"size": 10}),
             mixer(2, scale=0.7), mixer(3, q_temp={"coef": 0.25, "every": 12}), lambda c, T: c["layers"][2]["mixer"]["rot"].update(base=400.0), lambda c, T: c["layers"][2]["mixer"]["rot"]["scaling"].update(factor=5.0),
             lambda c, T: c["layers"][5]["mixer"]["rot"]["scaling"].update(original=60), lambda c, T: T.update({"l1.hc1.mix": T["l1.hc1.mix"].T}), lambda c, T: T.update({"l2.hc2.out": T["l2.hc2.out"][::-1]}),
             zero("l0.mix.i.b"), zero("l0.mix.f.b"), zero("l1.mix.k.b"), zero("l1.mix.q.b"), zero("l1.mix.v.b"), zero("l3.mix.q.b"), zero("l2.mix.g"), zero("l0.mix.g")]
    for k, e in enumerate(edits):
        assert off(e) > 10 * TOL[True], k


# ---- operators alone ---------------------------------------------------------------------------------------------------------------
def gpu():
    from tests import gpu_util as U
    return U, U.init()


def upload_bf16(lib, w):
    u = (np.ascontiguousarray(w, np.float32).view(np.uint32) >> 16).astype(np.uint16)
    h = lib.pi_weight_upload(BF16, w.shape[1], w.shape[0], u.ctypes.data_as(C.c_void_p), None)
    assert h, lib.pi_last_error()
    return h


def pack_mask(vis, n_kv):
    m = np.zeros((vis.shape[0], (n_kv + 31) // 32), np.uint32)
    for t, j in zip(*np.nonzero(vis)):
        m[t, j >> 5] |= np.uint32(1 << (j & 31))
    return m


def unpack_mask(m, n_kv):
    return np.array([[(row[j >> 5] >> (j & 31)) & 1 for j in range(n_kv)] for row in m]).astype(bool)


@pytest.mark.gpu
@pytest.mark.parametrize("K,N,T", [(24, 11, 5), (64, 70, 1), (520, 9, 3), (64, 130, 40), (128, 131, 200), (7, 5, 2)])
@pytest.mark.parametrize("exact", [1, 0])
def test_dense_with_bias(K, N, T, exact):
    """every kernel a width can reach (mat-vec of one, few and many tokens, both matrix-core kernels, odd sizes): the bias is added ahead of the activation"""
    U, lib = gpu()
    rng = np.random.default_rng(K + N)
    W, x, b = O.bf16_round((rng.standard_normal((N, K)) / np.sqrt(K)).astype(np.float32)), O.bf16_round(rng.standard_normal((T, K)).astype(np.float32)), rng.standard_normal(N).astype(np.float32)
    w, xd, bd, od = upload_bf16(lib, W), U.Dev(x), U.Dev(b), U.Dev(nbytes=4 * T * (N + 1))
    split = N // 2
    L.check(lib.pi_op_dense_bias(w, bd.ptr, xd.ptr, K, T, od.ptr, N + 1, SILU, split, NONE, exact, None))
    z = x.astype(np.float64) @ W.T.astype(np.float64) + b
    z[:, :split] = O.silu(z[:, :split])
    assert rel_rms(od.get(np.float32, (T, N + 1))[:, :N], z) < 3e-6
    lib.pi_weight_free(w)


@pytest.mark.gpu
@pytest.mark.parametrize("streams,n,T", [(1, 40, 3), (2, 37, 2), (3, 256, 5), (4, 4096, 2), (5, 1030, 2), (8, 64, 7), (16, 100, 1), (2, 5000, 2), (3, 6000, 1), (2, 4099, 1)])
def test_streams_step(streams, n, T):
    """the step from the old streams, all at once and in place; the next input and its norm; the start (every stream the same row) and the end (the plain sum)"""
    U, lib = gpu()
    rng = np.random.default_rng(streams * 1000 + n)
    X, y, w = (rng.standard_normal(s).astype(np.float32) for s in ((T, streams, n), (T, n), (n,)))
    mix, out, inn = (rng.standard_normal(s).astype(np.float32) for s in ((streams, streams), (streams,), (streams,)))
    eps = 1e-3
    xd, yd, wd, md, od, idv = (U.Dev(a) for a in (X, y, w, mix, out, inn))
    hd = U.Dev(nbytes=4 * T * n)
    L.check(lib.pi_op_hyper_step(xd.ptr, streams * n, n, streams, yd.ptr, n, md.ptr, od.ptr, idv.ptr, wd.ptr, eps, n, T, xd.ptr, hd.ptr, n, None))
    Tn = {"mix": mix.astype(np.float64), "out": out.astype(np.float64), "in": inn.astype(np.float64)}
    want = np.stack([O.streams_write(Tn, "", X[t].astype(np.float64), y[t].astype(np.float64)) for t in range(T)])
    h = np.stack([O.unit_rms(O.streams_read(Tn, "", want[t]), eps) * w for t in range(T)])
    assert rel_rms(xd.get(np.float32, X.shape), want) < 2e-6 and rel_rms(hd.get(np.float32, (T, n)), h) < 5e-6
    L.check(lib.pi_op_hyper_step(xd.ptr, streams * n, n, streams, yd.ptr, n, md.ptr, od.ptr, None, wd.ptr, eps, n, T, None, hd.ptr, n, None))        # the end: nothing stored, the sum of the streams normed
    last = np.stack([O.streams_write(Tn, "", want[t], y[t].astype(np.float64)).sum(0) for t in range(T)])
    assert rel_rms(hd.get(np.float32, (T, n)), O.unit_rms(last, eps) * w) < 1e-5 and rel_rms(xd.get(np.float32, X.shape), want) < 2e-6
    L.check(lib.pi_op_hyper_step(yd.ptr, n, 0, streams, None, 0, None, None, idv.ptr, wd.ptr, eps, n, T, xd.ptr, hd.ptr, n, None))                   # the start
    assert np.array_equal(xd.get(np.float32, X.shape), np.repeat(y[:, None], streams, 1))
    assert rel_rms(hd.get(np.float32, (T, n)), O.unit_rms(y.astype(np.float64) * inn.astype(np.float64).sum(), eps) * w) < 2e-5


def gate_runs(rng, H, steps, cap, slots, scale=3.0):
    """raw gates of passes [(slot, tokens, fresh), ..] and the oracle's factors"""
    bi, bf = rng.standard_normal(H).astype(np.float32), (rng.standard_normal(H) + 1.0).astype(np.float32)
    m = {}
    for step in steps:
        T = sum(c for _, c, _ in step)
        ri, rf = (rng.standard_normal((T, H)) * scale).astype(np.float32), (rng.standard_normal((T, H)) * scale).astype(np.float32)
        rec, want, at = [], np.zeros((3, T, H)), 0
        for slot, count, fresh in step:
            if fresh:
                m[slot] = np.zeros(H)
            for i in range(count):
                rec.append(slot | (F if fresh and i == 0 else 0))
                Tn = {"i": np.diag(ri[at].astype(np.float64)), "f": np.diag(rf[at].astype(np.float64)), "i.b": bi, "f.b": bf}
                a, b, m[slot] = O.memory_gates(Tn, "", cap, np.ones(H), m[slot])
                want[:, at] = a, b, np.exp(-m[slot])
                at += 1
        yield ri, rf, bi, bf, np.array(rec, np.int32), want, {s: v.copy() for s, v in m.items()}


STEPS = [[(0, 1200, True), (1, 5, True)], [(1, 2, True)], [(1, 1, False), (0, 4, True)], [(0, 150, False), (1, 3, False)], [(2, 64, True), (1, 65, False)], [(1, 1, False)], [(0, 63, True), (2, 1, False), (1, 70, True)]]


@pytest.mark.gpu
@pytest.mark.parametrize("H,cap", [(1, 5.0), (7, 12.5), (3, 0.5)])
def test_memory_gates(H, cap):
    """running maxima of sequences that start, continue, share a pass, and cross the 64 tokens a wave and the 1024 a workgroup takes at once"""
    U, lib = gpu()
    rng = np.random.default_rng(H)
    md = U.Dev((rng.standard_normal((3, H)) * 50).astype(np.float32))         # what an earlier owner left
    for ri, rf, bi, bf, rec, want, m in gate_runs(rng, H, STEPS, cap, 3):
        T = len(rec)
        raw = np.concatenate([ri, rf, np.zeros((T, 1), np.float32)], 1)
        rd, bid, bfd, recd, out = U.Dev(raw), U.Dev(bi), U.Dev(bf), U.Dev(rec), [U.Dev(nbytes=4 * T * H) for _ in range(3)]
        L.check(lib.pi_op_memory_gates(rd.ptr, rd.ptr + 4 * H, 2 * H + 1, bid.ptr, bfd.ptr, cap, H, md.ptr, recd.ptr, T, out[0].ptr, out[1].ptr, out[2].ptr, None))
        for k in range(3):
            got = out[k].get(np.float32, (T, H))
            assert np.abs(got / want[k] - 1.0).max() < 3e-5, k
        state = md.get(np.float32, (3, H))
        for s, v in m.items():
            assert np.abs(state[s] - v).max() < 2e-5


@pytest.mark.gpu
@pytest.mark.parametrize("H,D,V", [(3, 8, 6), (1, 1, 1), (2, 33, 70), (2, 128, 64), (1, 64, 257)])
def test_memory_recurrence_and_its_normaliser(H, D, V):
    """the linear recurrence with the keys' sum as one more column, in one launch and in pieces, then division, head norm, weight and gate"""
    U, lib = gpu()
    rng = np.random.default_rng(D + V)
    slots, cap, eps, mult = 3, 6.0, 1e-4, D ** -0.5
    S = {s: [np.zeros((H, D, V)), np.zeros((H, D))] for s in range(slots)}
    st = U.Dev((rng.standard_normal((slots, H, D, V + 1)) * 9).astype(np.float32))
    md = U.Dev(np.zeros((slots, H), np.float32))
    w = (1.0 + 0.3 * rng.standard_normal(H * V)).astype(np.float32)
    wd = U.Dev(w)
    for ri, rf, bi, bf, rec, want_g, m in gate_runs(rng, H, STEPS, cap, slots):
        T, ps = len(rec), H * (2 * D + 2 * V) + 3
        P = rng.standard_normal((T, ps)).astype(np.float32)
        pd, fd, ud, ld, recd = U.Dev(P), U.Dev(want_g[0].astype(np.float32)), U.Dev(want_g[1].astype(np.float32)), U.Dev(want_g[2].astype(np.float32)), U.Dev(rec)
        n_scr = lib.pi_op_linear_attention_scratch_floats(H, D, V + 1, T, slots)
        scr, zd, od = U.Dev(nbytes=4 * max(n_scr, 4)), U.Dev(nbytes=4 * T * H * (V + 1)), U.Dev(nbytes=4 * T * H * V)
        L.check(lib.pi_op_linear_attention_keysum(pd.ptr, pd.ptr + 4 * H * D, pd.ptr + 8 * H * D, ps, H, H, D, V, 1, None, fd.ptr, ud.ptr, H, None, st.ptr, recd.ptr, T, slots, scr.ptr, n_scr, zd.ptr, H * (V + 1), None))
        L.check(lib.pi_op_memory_norm(zd.ptr, H * (V + 1), ld.ptr, mult, 1e-6, H, V, eps, wd.ptr, pd.ptr + 4 * H * (2 * D + V), ps, SIGMOID, T, od.ptr, H * V, None))
        z, o = np.zeros((T, H, V + 1)), np.zeros((T, H * V))
        for t in range(T):
            s = int(rec[t]) & ~F
            if rec[t] & F:
                S[s] = [np.zeros((H, D, V)), np.zeros((H, D))]
            q, k, v, g = (a.astype(np.float64) for a in np.split(P[t, :H * (2 * D + 2 * V)], [H * D, 2 * H * D, H * (2 * D + V)]))
            out = np.zeros((H, V))
            for h in range(H):
                kk, qq = k[h * D:(h + 1) * D], q[h * D:(h + 1) * D]
                S[s][0][h], S[s][1][h] = O.memory_step(S[s][0][h], S[s][1][h], want_g[0, t, h], want_g[1, t, h], kk, v[h * V:(h + 1) * V])
                z[t, h, :V], z[t, h, V] = S[s][0][h].T @ qq, S[s][1][h] @ qq
                out[h] = O.unit_rms(O.memory_read(S[s][0][h], S[s][1][h], qq * mult, -math.log(want_g[2, t, h])), eps)
            o[t] = out.reshape(-1) * w * O.sigmoid(g)
        assert rel_rms(zd.get(np.float32, (T, H, V + 1)), z) < 1e-5 and rel_rms(od.get(np.float32, (T, H * V)), o) < 2e-4
        got = st.get(np.float32, (slots, H, D, V + 1))
        for s in set(int(r) & ~F for r in rec):
            assert rel_rms(got[s, ..., :V], S[s][0]) < 1e-5 and rel_rms(got[s, ..., V], S[s][1]) < 1e-5
    assert lib.pi_op_memory_norm(zd.ptr, H * V, ld.ptr, mult, 1e-6, H, V, eps, wd.ptr, None, 0, NONE, 1, od.ptr, H * V, None) != 0      # rows too short for the normaliser's column


@pytest.mark.gpu
@pytest.mark.parametrize("H,G,D,V,coef,every", [(4, 2, 10, 6, 0.4, 5), (3, 3, 64, 64, -0.1, 1), (6, 1, 130, 3, 0.35, 100), (2, 1, 7, 9, 0.0, 0)])
@pytest.mark.parametrize("own", [True, False])
def test_queries_with_a_temperature(H, G, D, V, coef, every, own):
    """unit-RMS queries and keys without a rotation, the temperature at block borders and far positions; without keys of its own a pass writes no cell"""
    U, lib = gpu()
    rng = np.random.default_rng(H + D)
    pos = np.array([0, 1, every - 2, every - 1, every, 3 * every - 1, 5000, 99999], np.int32).clip(0)
    T, n_cells, eps = len(pos), 20, 1e-2
    stride = H * D + G * (D + V) + 1
    P = rng.standard_normal((T, stride)).astype(np.float32)
    cells = rng.permutation(n_cells)[:T].astype(np.int32)
    dyn = np.concatenate([[0, n_cells, T, 1], cells, np.full(T, n_cells)]).astype(np.int32)
    pd, posd, dd, qd = U.Dev(P), U.Dev(pos), U.Dev(dyn), U.Dev(nbytes=4 * T * H * D)
    kd, vd, cd = U.Dev(np.full((n_cells, G, D), 7.0, np.float32)), U.Dev(np.full((n_cells, G, V), 7.0, np.float32)), U.Dev(np.full(n_cells, -5, np.int32))
    rot = lib.pi_rotary_table_create(32, 0, 10000.0)
    L.check(lib.pi_op_qkv_prepare_temp(pd.ptr, pd.ptr + 4 * H * D if own else None, pd.ptr + 4 * (H + G) * D if own else None, stride, None, None, eps, H, G, D, V, rot, NORM_LAST, NEIGHBOURS, 0, coef, every, posd.ptr, T,
                                       qd.ptr, H * D, kd.ptr, vd.ptr, cd.ptr, dd.ptr, None))
    q = O.unit_rms(P[:, :H * D].reshape(T, H, D).astype(np.float64), eps)
    if every:
        q = q * np.array([O.temperature({"q_temp": {"coef": coef, "every": every}}, int(p)) for p in pos])[:, None, None]
    assert rel_rms(qd.get(np.float32, (T, H, D)), q) < 2e-6
    kw, vw, cw = np.full((n_cells, G, D), 7.0), np.full((n_cells, G, V), 7.0), np.full(n_cells, -5)
    if own:
        kw[cells] = O.unit_rms(P[:, H * D:(H + G) * D].reshape(T, G, D).astype(np.float64), eps)
        vw[cells] = P[:, (H + G) * D:(H + G) * D + G * V].reshape(T, G, V)
        cw[cells] = pos
    assert rel_rms(kd.get(np.float32, kw.shape), kw) < 2e-6 and np.array_equal(vd.get(np.float32, vw.shape), vw.astype(np.float32)) and np.array_equal(cd.get(np.int32, (n_cells,)), cw)
    lib.pi_rotary_table_free(rot)


@pytest.mark.gpu
@pytest.mark.parametrize("size,n_kv,T", [(1, 40, 5), (7, 300, 9), (1000, 70, 3), (32, 9000, 2)])
def test_window_mask(size, n_kv, T):
    """cells in any order, several sequences in the mask, positions of the pass's own cells learned in the same launch"""
    U, lib = gpu()
    rng = np.random.default_rng(size)
    cpos = rng.integers(0, n_kv, n_kv).astype(np.int32)
    vis = rng.random((T, n_kv)) < 0.6
    cells, pos = rng.permutation(n_kv)[:T].astype(np.int32), rng.integers(0, n_kv, T).astype(np.int32)
    stale = cpos.copy()
    stale[cells] = -9
    cpos[cells] = pos
    vis[np.arange(T), cells] = True
    dyn = np.concatenate([[0, n_kv, T, 1], cells, np.full(T, n_kv)]).astype(np.int32)
    words = (n_kv + 31) // 32
    md, pd, cd, dd, od = U.Dev(pack_mask(vis, n_kv)), U.Dev(pos), U.Dev(stale), U.Dev(dyn), U.Dev(np.full((T, words), 0xFFFFFFFF, np.uint32))
    L.check(lib.pi_op_window_mask(md.ptr, pd.ptr, cd.ptr, size, T, n_kv, od.ptr, dd.ptr, None))
    want = vis & (cpos[None, :] > pos[:, None] - size)
    assert np.array_equal(od.get(np.uint32, (T, words)), pack_mask(want, n_kv)) and np.array_equal(cd.get(np.int32, (n_kv,)), cpos)


ROTS = [None, (4.0, 8.0, 1.0, 48), (16.0, 24.0, 1.5, 1024), (2.0, 1.0, 1.0, 16), (1.0, 4.0, 2.0, 64)]


def rot_of(dims, base, scaling):
    return {"dims": dims, "base": base, **({"scaling": dict(zip(("factor", "fast", "slow", "original"), scaling))} if scaling else {})}


def rot_table(lib, n_pos, rot):
    sc = rot.get("scaling")
    t = lib.pi_rotary_table_create_ramp(n_pos, rot["dims"], rot["base"], sc["factor"], sc["original"], sc["fast"], sc["slow"]) if sc else lib.pi_rotary_table_create(n_pos, rot["dims"], rot["base"])
    assert t, lib.pi_last_error()
    return t


@pytest.mark.gpu
@pytest.mark.parametrize("q_rank,rank,rdim,base", [(11, 12, 6, 300.0), (96, 256, 64, 10000.0), (1, 2, 2, 50.0), (300, 70, 130, 2e5)])
@pytest.mark.parametrize("scaling", ROTS)
def test_both_latents(q_rank, rank, rdim, base, scaling):
    U, lib = gpu()
    rng = np.random.default_rng(q_rank)
    pos = np.array([0, 1, 2, 17, 63, 512, 2999], np.int32)
    T, n_cells, eps = len(pos), 11, 1e-3
    rot = rot_of(rdim, base, scaling)
    t = rot_table(lib, 3000, rot)
    P = rng.standard_normal((T, q_rank + rank + rdim + 3)).astype(np.float32)
    qw, kw = rng.standard_normal(q_rank).astype(np.float32), rng.standard_normal(rank).astype(np.float32)
    cells = rng.permutation(n_cells)[:T].astype(np.int32)
    dyn = np.concatenate([[0, n_cells, T, 1], cells, np.full(T, n_cells)]).astype(np.int32)
    ds = [U.Dev(a) for a in (P, qw, kw, pos, dyn)]
    cq, cache = U.Dev(nbytes=4 * T * (q_rank + 2)), U.Dev(np.zeros((n_cells, rank + rdim), np.float32))
    L.check(lib.pi_op_latent_prepare(ds[0].ptr, P.shape[1], q_rank, ds[1].ptr, rank, ds[2].ptr, rdim, t, eps, ds[3].ptr, T, cq.ptr, q_rank + 2, cache.ptr, ds[4].ptr, None))
    P64 = P.astype(np.float64)
    assert rel_rms(cq.get(np.float32, (T, q_rank + 2))[:, :q_rank], O.unit_rms(P64[:, :q_rank], eps) * qw) < 2e-6
    got = cache.get(np.float32, (n_cells, rank + rdim))
    want = np.zeros((n_cells, rank + rdim))
    for i in range(T):
        want[cells[i], :rank] = O.unit_rms(P64[i, q_rank:q_rank + rank], eps) * kw
        want[cells[i], rank:] = O.turn(P64[i, q_rank + rank:q_rank + rank + rdim], int(pos[i]), rot)
    assert rel_rms(got[:, :rank], want[:, :rank]) < 2e-6 and rel_rms(got[:, rank:], want[:, rank:]) < 2e-6
    lib.pi_rotary_table_free(t)


def latent_case(U, lib, rng, H, D, R, V, rank, n_kv, pos, vis, rot, gate, sink, scale, cache=None, q=None):
    """the operator's output and the plain one: cells carry no positions here, visibility is the mask's alone"""
    T = len(pos)
    t = rot_table(lib, int(max(pos)) + 2, rot) if R else None
    Wuk, Wuv = O.bf16_round((rng.standard_normal((H * D, rank)) / np.sqrt(rank)).astype(np.float32)), O.bf16_round((rng.standard_normal((H * V, rank)) / np.sqrt(rank)).astype(np.float32))
    q = q if q is not None else rng.standard_normal((T, H, D + R)).astype(np.float32)
    cache = cache if cache is not None else rng.standard_normal((n_kv, rank + R)).astype(np.float32)
    g, s = rng.standard_normal((T, H)).astype(np.float32), rng.standard_normal(H).astype(np.float32)
    uk, uv = upload_bf16(lib, Wuk), upload_bf16(lib, Wuv)
    dyn = np.array([0, n_kv, T, 0], np.int32)
    qd, cd, md, gd, sd, pd, dd = (U.Dev(a) for a in (q, cache, pack_mask(vis, n_kv), g, s, np.asarray(pos, np.int32), dyn))
    n_scr = lib.pi_op_latent_attention_rot_scratch_floats(H, rank, R, T, n_kv)
    scr, od = U.Dev(np.full(n_scr, np.nan, np.float32)), U.Dev(nbytes=4 * T * H * V)        # (what no split has written is not read)
    L.check(lib.pi_op_latent_attention_rot(qd.ptr, H * (D + R), cd.ptr, md.ptr, uk, uv, sd.ptr if sink else None, gd.ptr if gate else None, H, SIGMOID, scale, H, D, R, V, rank, t, pd.ptr, T, n_kv, scr.ptr, n_scr,
                                           od.ptr, H * V, dd.ptr, None))
    want = np.zeros((T, H, V))
    Wk, Wv, C64 = Wuk.reshape(H, D, rank).astype(np.float64), Wuv.reshape(H, V, rank).astype(np.float64), cache.astype(np.float64)
    for i in range(T):
        js = np.nonzero(vis[i])[0]
        for h in range(H):
            sc = (C64[js, :rank] @ Wk[h].T) @ q[i, h, :D].astype(np.float64)
            if R:
                sc = sc + C64[js, rank:] @ O.turn(q[i, h, D:].astype(np.float64), int(pos[i]), rot)
            e = np.exp(sc * scale - (sc * scale).max())
            den = e.sum() + (math.exp(s[h] - (sc * scale).max()) if sink else 0.0)
            want[i, h] = (e / den) @ (C64[js, :rank] @ Wv[h].T) * (O.sigmoid(g[i, h]) if gate else 1.0)
    lib.pi_weight_free(uk)
    lib.pi_weight_free(uv)
    if t:
        lib.pi_rotary_table_free(t)
    return od.get(np.float32, (T, H, V)), want


@pytest.mark.gpu
@pytest.mark.parametrize("H,D,R,V,rank", [(3, 7, 6, 5, 12), (1, 1, 2, 1, 2), (16, 32, 16, 24, 64), (5, 70, 66, 40, 136), (4, 8, 64, 8, 512), (2, 6, 0, 7, 20), (20, 16, 8, 8, 300)])
@pytest.mark.parametrize("T,n_kv", [(1, 33), (1, 700), (5, 90), (70, 70), (33, 400)])
def test_latent_attention_with_a_rotated_part(H, D, R, V, rank, T, n_kv):
    """few and many tokens (splits of the cells, score rows in LDS), windows that leave whole splits empty, with and without gate and sink"""
    U, lib = gpu()
    rng = np.random.default_rng(H * 100 + T)
    pos = np.arange(n_kv - T, n_kv)
    rot = rot_of(R, 500.0, ROTS[1])
    cells = np.arange(n_kv)
    for window, gate, sink in ((None, True, False), (20, True, False), (1, False, False), (90, False, True)):
        vis = cells[None, :] <= pos[:, None]
        if window:
            vis &= cells[None, :] > pos[:, None] - window
        got, want = latent_case(U, lib, rng, H, D, R, V, rank, n_kv, pos, vis, rot, gate, sink, (D + R) ** -0.5)
        assert rel_rms(got, want) < 1e-5, (window, gate, sink)


@pytest.mark.gpu
@pytest.mark.parametrize("T", [1, 40])
def test_a_loud_key_at_the_windows_edge(T):
    """one rotated key far louder than every other: just inside the window it takes the mass, one position earlier it is not seen; among hundreds of plain causal keys it is always heard"""
    U, lib = gpu()
    H, D, R, V, rank, n_kv, size = 2, 4, 4, 6, 16, 600, 37
    rot = rot_of(R, 100.0, None)
    pos, cells = np.arange(n_kv - T, n_kv), np.arange(n_kv)
    for window in (size, None):
        for back in (0, size - 1, size, 300):
            rng = np.random.default_rng(back + T)
            cache = (rng.standard_normal((n_kv, rank + R)) * 0.3).astype(np.float32)
            q = np.zeros((T, H, D + R), np.float32)
            loud = n_kv - 1 - back
            q[-1, :, D:] = [1.0, 0.0, 1.0, 0.0]
            cache[loud, rank:] = O.turn(np.array([1.0, 0.0, 1.0, 0.0]), n_kv - 1, rot) * 40.0
            vis = cells[None, :] <= pos[:, None]
            if window:
                vis &= cells[None, :] > pos[:, None] - window
            got, want = latent_case(U, lib, np.random.default_rng(5), H, D, R, V, rank, n_kv, pos, vis, rot, False, False, 1.0, cache=cache, q=q)
            assert rel_rms(got, want) < 1e-5
            heard = window is None or back < size
            Wuv = np.random.default_rng(5)
            Wuv.standard_normal((H * D, rank))
            Wuv = O.bf16_round((Wuv.standard_normal((H * V, rank)) / np.sqrt(rank)).astype(np.float32)).astype(np.float64)
            assert (rel_rms(got[-1].reshape(-1), Wuv @ cache[loud, :rank]) < 1e-4) == heard, (window, back)


@pytest.mark.gpu
def test_a_far_key_of_the_attention_is_heard():
    """unit-norm keys and a sharp scale: of 900 keys the one that equals the query carries the output, from the first cell to the last, also where the cells' order is not the positions'"""
    U, lib = gpu()
    rng = np.random.default_rng(8)
    H, G, D, V, n_kv = 4, 2, 16, 5, 900
    k = O.unit_rms(rng.standard_normal((n_kv, G, D)), 1e-6).astype(np.float32)
    v = rng.standard_normal((n_kv, G, V)).astype(np.float32)
    cpos = rng.permutation(n_kv).astype(np.int32)
    kd, vd, cd, pd, dd = U.Dev(k), U.Dev(v), U.Dev(cpos), U.Dev(np.array([n_kv - 1], np.int32)), U.Dev(np.array([0, n_kv, 1, 0], np.int32))
    md = U.Dev(pack_mask(np.ones((1, n_kv), bool), n_kv))
    n_scr = lib.pi_op_window_attention_scratch_floats(H, V, 1)
    scr, od = U.Dev(nbytes=4 * n_scr), U.Dev(nbytes=4 * H * V)
    for cell in (0, 31, 32, 255, 256, 500, n_kv - 1):
        q = np.repeat(k[cell], H // G, axis=0)[None]
        qd = U.Dev(q)
        L.check(lib.pi_op_window_attention(qd.ptr, H * D, kd.ptr, vd.ptr, cd.ptr, md.ptr, pd.ptr, None, None, None, 0, NONE, 6.0, 1.0, SOFTMAX, 0.0, WINDOW, 0, 0, 0, 0, H, G, D, V, 1, n_kv, scr.ptr, n_scr, od.ptr, H * V,
                                           dd.ptr, None))
        assert np.allclose(od.get(np.float32, (H, V)), np.repeat(v[cell], H // G, axis=0), atol=2e-3), cell


# ---- whole models through llama_decode ---------------------------------------------------------------------------------------------------
@pytest.mark.gpu
@pytest.mark.parametrize("variant", list(VARIANTS))
@pytest.mark.parametrize("exact", [True, False])
def test_prompt_portions_and_decoding_agree_with_the_oracle(tmp_path, variant, exact):
    m = variant_model(variant)
    rng = np.random.default_rng(5)
    toks = [int(t) for t in rng.integers(0, VOCAB, 75)]
    want = O.run(m, toks)
    e = Engine(tmp_path, m, n_ctx=96, n_batch=48, exact=exact)
    tol = TOL[exact] * (3 if variant in ("wide_heads", "edges") or (variant == "mixed" and not exact) else 1)       # (the six-layer mix is 0.11 away from itself at nine positions in ten when its matrix inputs are rounded to bfloat16)
    whole = np.concatenate([e.ctx.feed(toks[:48], 0, 0), e.ctx.feed(toks[48:], 48, 0)])
    assert within(logit_err(whole, want), exact, tol)
    e.ctx.seq_rm(0, -1, -1)
    parts, at = [], 0
    for n in [2, 3, 31, 2, 1, 1, 7, 2, 5, 1, 1, 1, 2, 16]:                 # portions down to two tokens and single tokens, cut inside windows and temperature blocks
        parts.append(e.ctx.feed(toks[at:at + n], at, 1))
        at += n
    assert at == 75 and within(logit_err(np.concatenate(parts), want), exact, tol)
    e.ctx.seq_rm(1, -1, -1)
    single = np.concatenate([e.ctx.feed(toks[i:i + 1], i, 2) for i in range(40)])
    assert within(logit_err(single, want[:40]), exact, tol)
    e.close()


@pytest.mark.gpu
@pytest.mark.parametrize("exact", [True, False])
def test_a_wider_model_with_long_passes(tmp_path, exact):
    """widths and passes that reach the matrix-core products: 300 tokens in passes of 128 (longer than the window), then single tokens"""
    layers = [O.attention_layer(heads=8, kv_heads=2, dim=24, vdim=48, scale=0.5, coef=0.2, every=64, ff=160), O.mlstm_layer(heads=4, dim=40, vdim=72, cap=10.0, ff=192),
              O.latent_layer(heads=6, dim=24, rot_dim=16, vdim=40, q_rank=64, kv_rank=80, size=70, base=10000.0, scaling=(8.0, 32.0, 1.0, 128), scale=0.2, ff=256),
              O.attention_layer(heads=4, kv_heads=2, dim=24, vdim=48, scale=0.4, coef=0.3, every=100, kv_from=0, ff=None)]
    m = small_model(seed=13, layers=layers, width=128, vocab=200, streams=2)
    rng = np.random.default_rng(6)
    toks = [int(t) for t in rng.integers(0, 200, 320)]
    want = O.run(m, toks)
    e = Engine(tmp_path, m, n_ctx=330, n_batch=128, exact=exact)
    got = np.concatenate([e.ctx.feed(toks[:300], 0, 0)] + [e.ctx.feed(toks[i:i + 1], i, 0) for i in range(300, 320)])
    assert within(logit_err(got, want), exact, TOL[exact] * 2)
    e.close()


@pytest.mark.gpu
def test_residual_streams_layer_by_layer(tmp_path):
    """models cut after 1, 2, ... layers give the oracle's logits, so the first wrong layer would be named"""
    full = small_model(seed=4)
    toks = [5, 17, 3, 78, 0, 41, 41, 7, 9, 9, 30, 2, 2, 61, 8, 8, 8, 12, 70, 3, 3, 44]
    for n in range(1, 7):
        m = {"config": dict(full["config"], layers=full["config"]["layers"][:n]), "tensors": full["tensors"]}
        e = Engine(tmp_path, m, n_ctx=32, n_batch=8, name="cut%d" % n)
        assert logit_err(e.ctx.feed(toks, 0, 0), O.run(m, toks)).max() < TOL[True], n
        e.close()


@pytest.mark.gpu
def test_first_tokens_of_a_sequence(tmp_path):
    """a sequence's first tokens see no memory, no running maximum and no key of whoever held the slot and the cells before"""
    m = small_model(seed=17)
    e = Engine(tmp_path, m, n_ctx=64, n_batch=8, slots=1)
    for toks in ([7], [7, 7], [78, 7, 3], [3, 78, 7, 7, 2, 2, 2, 9, 1, 4, 4]):
        got = np.concatenate([e.ctx.feed(toks[i:i + 3], i, 0) for i in range(0, len(toks), 3)])
        assert logit_err(got, O.run(m, toks)).max() < TOL[True], toks
        e.ctx.seq_rm(0, -1, -1)
    e.close()


@pytest.mark.gpu
@pytest.mark.parametrize("exact", [True, False])
def test_batches_of_unequal_requests_equal_each_alone(tmp_path, exact):
    """three requests of unequal length share passes, one starts in the middle: every row equals the same request fed alone through the engine, and in fp32 the oracle"""
    m = small_model(seed=21)
    rng = np.random.default_rng(8)
    reqs = [[int(t) for t in rng.integers(0, VOCAB, n)] for n in (23, 5, 14)]
    extra = [int(t) for t in rng.integers(0, VOCAB, 6)]
    e = Engine(tmp_path, m, n_ctx=128, n_batch=64, exact=exact, slots=5)
    alone = []
    for r in reqs + [extra]:
        alone.append(e.ctx.feed(r, 0, 4))
        e.ctx.seq_rm(4, -1, -1)
    first = [9, 2, 14]
    toks = sum((r[:n] for r, n in zip(reqs, first)), [])
    pos = sum((list(range(n)) for n in first), [])
    seqs = sum(([[s]] * n for s, n in enumerate(first)), [])
    lg = e.ctx.decode(toks, pos, seqs)
    at, got = 0, [[], [], [], []]
    for s, n in enumerate(first):
        got[s].append(lg[at:at + n])
        at += n
    toks = reqs[1][2:] + extra + reqs[0][9:]
    pos = list(range(2, 5)) + list(range(6)) + list(range(9, 23))
    seqs = [[1]] * 3 + [[3]] * 6 + [[0]] * 14
    lg = e.ctx.decode(toks, pos, seqs)
    got[1].append(lg[:3]); got[3].append(lg[3:9]); got[0].append(lg[9:])
    for s, toks in enumerate(reqs + [extra]):
        mine = np.concatenate(got[s])
        assert np.quantile(logit_err(mine, alone[s].astype(np.float64)), 1.0 if exact else 0.9) < (1e-5 if exact else 2e-2), s
        if exact:
            assert logit_err(mine, O.run(m, toks)).max() < TOL[True], s
    e.close()


@pytest.mark.gpu
def test_freed_cells_and_slots_are_used_again(tmp_path):
    """more requests than slots and cells, one after the other and interleaved: a finished request gives back what it held, the next one starts from nothing; a copied sequence continues like
    the original"""
    m = small_model(seed=31)
    rng = np.random.default_rng(9)
    e = Engine(tmp_path, m, n_ctx=48, n_batch=16, slots=2)
    for round_ in range(5):
        a = [int(t) for t in rng.integers(0, VOCAB, 20 + round_)]
        b = [int(t) for t in rng.integers(0, VOCAB, 11)]
        la = e.ctx.feed(a[:7], 0, 0)
        lb = e.ctx.feed(b, 0, 1)
        la = np.concatenate([la, e.ctx.feed(a[7:], 7, 0)])
        assert e.ctx.state_slots_used() == 2
        with pytest.raises(L.PipeInferError):
            e.ctx.decode([1], [0], [[2]])
        e.ctx.seq_rm(1, -1, -1)
        lc = e.ctx.feed(b[:5], 0, 2)
        for got, toks in ((la, a), (lb, b), (lc, b[:5])):
            assert logit_err(got, O.run(m, toks)).max() < TOL[True], round_
        e.ctx.seq_rm(0, -1, -1)
        e.ctx.seq_rm(2, -1, -1)
        assert e.ctx.state_slots_used() == 0
    a = [int(t) for t in rng.integers(0, VOCAB, 12)]
    e.ctx.feed(a[:8], 0, 0)
    e.ctx.seq_cp(0, 1, -1, -1)
    assert logit_err(e.ctx.feed(a[8:] + [50, 51], 8, 1), O.run(m, a + [50, 51])[8:]).max() < TOL[True]
    assert logit_err(e.ctx.feed(a[8:] + [60], 8, 0), O.run(m, a + [60])[8:]).max() < TOL[True]
    e.close()


@pytest.mark.gpu
@pytest.mark.parametrize("exact", [True, False])
def test_window_and_temperature_borders_show_in_prompts_and_in_decoding(tmp_path, exact):
    """sharp attention over several hundred tokens, windows and temperature blocks that divide neither each other nor the pass width: a key wrongly seen or lost at a window's edge or a
    temperature one token early shows far above rounding — the same model with a window or a block one position longer is far away"""
    layers = [O.latent_layer(heads=2, dim=4, rot_dim=8, vdim=8, q_rank=16, kv_rank=12, size=50, base=200.0, scale=2.0, ff=None),
              O.attention_layer(heads=2, kv_heads=1, dim=8, vdim=6, coef=1.5, every=37, scale=1.2, ff=16), O.mlstm_layer(heads=2, dim=6, vdim=5, cap=4.0, ff=None),
              O.latent_layer(heads=3, dim=6, rot_dim=2, vdim=4, q_rank=8, kv_rank=10, size=21, base=50.0, scaling=None, scale=1.5, ff=12)]
    m = small_model(seed=41, layers=layers, width=32, streams=2)
    rng = np.random.default_rng(12)
    toks = [int(t) for t in rng.integers(0, VOCAB, 330)]
    want = O.run(m, toks)
    e = Engine(tmp_path, m, n_ctx=340, n_batch=128, exact=exact)
    got = np.concatenate([e.ctx.feed(toks[:290], 0, 0)] + [e.ctx.feed(toks[i:i + 1], i, 0) for i in range(290, 330)])       # every decoded token moves both windows; a temperature block ends at 296
    assert within(logit_err(got, want), exact)
    if exact:                                                         # (at serving precision one key more or less among fifty is not far enough from rounding to tell)
        for where, edit in ((0, {"mask": {"size": 51}}), (0, {"mask": {"size": 49}}), (3, {"mask": {"size": 22}}), (1, {"q_temp": {"coef": 1.5, "every": 36}})):
            other = json.loads(json.dumps(m["config"]))
            other["layers"][where]["mixer"].update(edit)
            off = logit_err(got, O.run({"config": other, "tensors": m["tensors"]}, toks))
            assert off[100:290].max() > 30 * TOL[exact] and off[290:].max() > 30 * TOL[exact], (where, edit)
    e.close()


@pytest.mark.gpu
def test_long_decoding_token_by_token(tmp_path):
    m = small_model(seed=45)
    rng = np.random.default_rng(13)
    toks = [int(t) for t in rng.integers(0, VOCAB, 200)]
    want = O.run(m, toks)
    e = Engine(tmp_path, m, n_ctx=224, n_batch=8, exact=True)
    got = np.concatenate([e.ctx.feed(toks[:3], 0, 0)] + [e.ctx.feed(toks[i:i + 1], i, 0) for i in range(3, 200)])
    assert logit_err(got, want).max() < TOL[True]
    e.close()


@pytest.mark.gpu
def test_greedy_generation_through_the_engine(tmp_path):
    m = small_model(seed=51)
    prompt = [3, 14, 15, 72, 65, 35]
    e = Engine(tmp_path, m, n_ctx=160, n_batch=16, exact=True)
    got = e.ctx.generate(prompt, 100)
    want = O.greedy(m, prompt, 100)
    k = next((i for i, (a, b) in enumerate(zip(got, want)) if a != b), len(want))
    if k < len(want):                                               # (an arg-max between two nearly equal logits may fall either way in fp32 against float64: it must be a near tie)
        lg = O.run(m, prompt + want[:k])[-1]
        assert abs(lg[got[k]] - lg[want[k]]) < 1e-3 * np.abs(lg).max()
    assert k >= 20
    e.close()


@pytest.mark.gpu
def test_graph_replays_equal_eager_launches(tmp_path):
    m = small_model(seed=61)
    rng = np.random.default_rng(3)
    toks = [int(t) for t in rng.integers(0, VOCAB, 60)]
    outs = []
    for graphs in (True, False):
        e = Engine(tmp_path, m, n_ctx=64, n_batch=16, exact=False, name="g%d" % graphs)
        e.ctx.set_graphs(graphs)
        lg = []
        for rep in range(3):
            lg.append(np.concatenate([e.ctx.feed(toks[:37], 0, rep % 2), e.ctx.feed(toks[37:38], 37, rep % 2), e.ctx.feed(toks[38:], 38, rep % 2)]))
            e.ctx.seq_rm(rep % 2, -1, -1)
        assert all(np.array_equal(lg[0], x) for x in lg[1:])
        outs.append(lg[0])
        e.close()
    assert np.array_equal(outs[0], outs[1])


@pytest.mark.gpu
def test_a_second_longer_context_of_the_same_model(tmp_path):
    """rotation tables grow with the longest context; the shorter one goes on"""
    m = small_model(seed=67, layers=[O.latent_layer(size=12, ff=None), O.mlstm_layer()])
    folder = str(tmp_path / "m")
    write(folder, m)
    mod = LL.Model(folder)
    toks = [int(t) for t in np.random.default_rng(2).integers(0, VOCAB, 90)]
    want = O.run(m, toks)
    short = LL.Context(mod, n_ctx=40, n_batch=16)
    short.set_precision(True)
    a = short.feed(toks[:20], 0, 0)
    longer = LL.Context(mod, n_ctx=96, n_batch=32)
    longer.set_precision(True)
    b = longer.feed(toks, 0, 0)
    a = np.concatenate([a, short.feed(toks[20:32], 20, 0)])
    assert logit_err(a, want[:32]).max() < TOL[True] and logit_err(b, want).max() < TOL[True]
    short.free(); longer.free(); mod.free()


@pytest.mark.gpu
def test_generate_command_line(tmp_path, capsys):
    from pipeinfer_amd.tools import generate as G
    m = small_model(seed=71)
    folder = str(tmp_path / "g")
    write(folder, m)
    assert G.main(["--model", folder, "--prompt-ids", "5,6,7", "--n-predict", "12", "--float32"]) == 0
    greedy = [int(t) for t in capsys.readouterr().out.strip().split(",")]
    want = O.greedy(m, [5, 6, 7], 12)
    k = next((i for i, (a, b) in enumerate(zip(greedy, want)) if a != b), 12)
    assert k >= 6


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_runner_replays_steps_and_writes_the_wanted_rows(tmp_path, dtype):
    import subprocess
    import sys
    m = variant_model("mixed", seed=81)
    folder, out = str(tmp_path / "model"), str(tmp_path / "out")
    write(folder, m)
    rng = np.random.default_rng(5)
    a, b = [int(t) for t in rng.integers(0, VOCAB, 41)], [int(t) for t in rng.integers(0, VOCAB, 9)]
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:3], "want": [0, 2]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[3:33], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[33:40], "want": [6, 1]}], "end": []},
             {"step": 3, "entries": [{"id": "a", "tokens": a[40:], "want": [0]}], "end": ["a"]},
             {"step": 4, "entries": [{"id": "b", "tokens": b, "want": [8]}], "end": ["b"]}]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out", out, "--max-tokens", "48", "--n-batch", "16"],
                       input="".join(json.dumps(x) + "\n" for x in steps), capture_output=True, text=True, timeout=600)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done %d" % i for i in range(5)]
    la, lb = O.run(m, a), O.run(m, b)
    want = {0: la[[0, 2]], 2: la[[39, 34]], 3: la[[40]], 4: lb[[8]]}
    assert sorted(os.listdir(out)) == sorted("%d.f32" % k for k in want)
    for k, w in want.items():
        got = np.fromfile(os.path.join(out, "%d.f32" % k), "<f4").reshape(-1, VOCAB)
        assert got.shape == w.shape and (logit_err(got, w).max() < TOL[True] if dtype == "float32" else np.median(logit_err(got, w)) < TOL[False]), k
