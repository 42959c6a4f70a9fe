"""The Letevik design (plain pre-norm blocks, a hashed pair embedding, a run of layers repeated behind a learned vector per pass; differential attention in windows with kept first tokens behind short
convolutions, latent attention with a sink and a gate per output value; a clipped gated feed-forward) on the engine, held to the plain numpy restatement in tests/letevik_oracle.py: every mechanism
alone through its operator, then whole models through llama_decode — prompts against token-by-token decoding, portions down to two tokens, batches of unequal requests, cells and state slots freed and
used again, keys far away and at the borders of windows and of the kept tokens, long decoding, greedy generation, the trace runner.  Models are small, random and made here; sizes are chosen so that
nothing that could be mixed up is equal."""
import ctypes as C
import json
import math
import os

import numpy as np
import pytest

from pipeinfer_amd import lib as L, llama as LL
from tests import letevik_oracle as O

BF16 = 30
F = 1 << 30                                    # "this sequence starts from nothing" on the first token of a run (slot words)
NONE, SIGMOID = 0, 2
HALVES, NEIGHBOURS = 0, 1
GLU_CLIPPED = 2


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


VOCAB = 83
LOOP = {"start": 1, "stop": 3, "times": 3}
# (layers, repeated run, pair buckets): the default mix, the values another model may make equal or one, wide heads, one kind of layer only, absent optional parts, runs at the ends of the list
VARIANTS = {
    "mixed": (None, LOOP, 37),
    "edges": ([O.attention_layer(heads=1, kv_heads=1, dim=2, vdim=2, conv=1, size=1, keep_first=0, rot_dims=2, diff=0.0, ff=1, limit=0.5),
               O.latent_layer(heads=1, dim=1, rot_dim=2, vdim=1, q_rank=1, kv_rank=2, ff=None), O.attention_layer(heads=3, kv_heads=1, dim=2, vdim=2, conv=2, size=2, keep_first=1, rot_dims=2, diff=0.9, ff=2),
               O.latent_layer(heads=2, dim=4, rot_dim=4, vdim=4, q_rank=4, kv_rank=4, base=1.5, ff=4)], {"start": 0, "stop": 4, "times": 1}, 1),
    "wide_heads": ([O.latent_layer(heads=4, dim=70, rot_dim=66, vdim=40, q_rank=72, kv_rank=136, base=5000.0, scale=0.1, ff=96, limit=0.8),
                    O.attention_layer(heads=6, kv_heads=2, dim=72, vdim=130, conv=9, size=23, keep_first=5, rot_dims=40, scale=0.12, ff=40)], {"start": 1, "stop": 2, "times": 2}, 101),
    "only_attention": ([O.attention_layer(ff=8), O.attention_layer(heads=6, kv_heads=3, dim=4, vdim=9, size=4, keep_first=30, rot_dims=4), O.attention_layer(heads=2, kv_heads=2, dim=6, vdim=5, conv=4, size=30, keep_first=0)],
                       {"start": 0, "stop": 2, "times": 2}, 11),
    "only_latent": ([O.latent_layer(ff=9), O.latent_layer(heads=2, dim=3, rot_dim=8, vdim=9, q_rank=5, kv_rank=6, base=40.0), O.latent_layer(heads=5, ff=7, limit=3.0)], {"start": 2, "stop": 3, "times": 4}, 53),
    "no_options": ([O.attention_layer(conv=None, size=None, rot_dims=0, ff=6), O.latent_layer(rot_dim=0)], None, None),
    "no_pairs": ([O.attention_layer(), O.latent_layer(ff=5)], {"start": 0, "stop": 1, "times": 2}, None),
}


def default_layers():
    return [O.latent_layer(ff=24), O.attention_layer(ff=20), O.latent_layer(heads=4, dim=3, rot_dim=4, vdim=8, q_rank=9, kv_rank=7, base=90.0, ff=22, limit=0.7),
            O.attention_layer(heads=3, kv_heads=3, dim=6, vdim=7, conv=5, size=14, keep_first=4, rot_dims=6, base=50.0, scale=0.7, diff=0.6, ff=None), O.latent_layer(heads=2, ff=None)]


def small_model(seed=0, width=40, vocab=VOCAB, layers=None, loop=LOOP, **kw):
    return O.random_model(np.random.default_rng(seed), vocab, width, layers or default_layers(), loop=loop, **kw)


def variant_model(name, seed=11):
    layers, loop, buckets = VARIANTS[name]
    return small_model(seed=seed, layers=layers, loop=loop, buckets=buckets, width={"wide_heads": 64, "edges": 18, "only_latent": 37}.get(name, 40))


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
    for name in VARIANTS:                                            # also without pairs, a repeated run, a window, a convolution, a rotation, a feed-forward
        folder = str(tmp_path / name)
        write(folder, variant_model(name, seed=1))
        mod = LL.Model(folder)
        assert mod.n_vocab == VOCAB
        buf = C.create_string_buffer(64)
        mod.lib.llama_model_desc.argtypes = [C.c_void_p, C.c_char_p, C.c_size_t]
        mod.lib.llama_model_desc(mod.h, buf, 64)
        assert buf.value.lower().startswith(b"letevik")
        mod.free()


@pytest.mark.parametrize("breakage", ["type", "kv_heads", "rot", "rot_dims", "rot_odd", "kind", "limit", "loop", "loop_times", "buckets", "diff", "conv", "window", "keep", "scale", "q_rank", "eps"])
def test_a_wrong_description_is_refused(tmp_path, breakage):
    m = small_model()
    cfg = json.loads(json.dumps(m["config"]))
    mx = [l["mixer"] for l in cfg["layers"]]
    if breakage == "type":
        cfg["layers"][0]["type"] = "mlstm"
    elif breakage == "kv_heads":
        mx[1]["kv_heads"] = 3
    elif breakage == "rot":
        mx[2]["rot"]["base"] = 0
    elif breakage == "rot_dims":
        mx[2]["rot"]["dims"] = 2
    elif breakage == "rot_odd":
        mx[1]["rot"]["dims"] = 5
    elif breakage == "kind":
        cfg["layers"][0]["mlp"]["kind"] = "moe"
    elif breakage == "limit":
        cfg["layers"][0]["mlp"]["limit"] = 0
    elif breakage == "loop":
        cfg["loop"]["stop"] = 6
    elif breakage == "loop_times":
        del cfg["loop"]["times"]
    elif breakage == "buckets":
        cfg["embedding"]["bigram"]["buckets"] = 0
    elif breakage == "diff":
        del mx[1]["diff"]
    elif breakage == "conv":
        mx[1]["conv"] = 0
    elif breakage == "window":
        mx[1]["mask"]["size"] = 0
    elif breakage == "keep":
        mx[1]["mask"]["keep_first"] = -1
    elif breakage == "scale":
        del mx[0]["scale"]
    elif breakage == "q_rank":
        del mx[0]["q_rank"]
    elif breakage == "eps":
        del cfg["norm"]
    folder = str(tmp_path / "bad")
    O.write_model(folder, cfg, {k: v.astype(np.float32) for k, v in m["tensors"].items()})
    with pytest.raises(L.PipeInferError):
        LL.Model(folder)


@pytest.mark.gpu
@pytest.mark.parametrize("name,cut", [("l1.mix.v.conv", None), ("l2.mix.g", slice(0, -1)), ("loop.step", slice(0, -1)), ("bigram", slice(0, -1)), ("l0.mix.sink", None), ("l3.mix.lk2", slice(0, -1)), ("l1.norm2", None)])
def test_a_wrong_tensor_is_refused_when_the_weights_load(tmp_path, name, cut):
    m = small_model()
    tensors = dict(m["tensors"])
    if cut is None:
        del tensors[name]
    else:
        tensors[name] = tensors[name][cut]
    folder = str(tmp_path / "bad")
    O.write_model(folder, m["config"], {k: v.astype(np.float32) for k, v in tensors.items()})
    mod = LL.Model(folder)
    ctx = LL.Context(mod, n_ctx=32, n_batch=8)
    with pytest.raises(L.PipeInferError):
        ctx.decode([1], [0], [[0]])
    ctx.free()
    mod.free()


def test_oracle_mechanisms_behave_as_stated():
    """the restatement itself: window and kept tokens, the convolution's order, rotations in both pairings that depend on the distance only, the order of the layer runs, pair rows, the difference of maps"""
    assert O.seen(5, {"size": 3, "keep_first": 1}) == [0, 3, 4, 5] and O.seen(1, {"size": 3, "keep_first": 9}) == [0, 1] and O.seen(4, None) == [0, 1, 2, 3, 4] and O.seen(4, {"size": 1, "keep_first": 0}) == [4]
    assert O.seen(4, {"size": 2, "keep_first": 3}) == [0, 1, 2, 3, 4] and O.seen(5, {"size": 2, "keep_first": 3}) == [0, 1, 2, 4, 5]
    w = np.array([[1.0, 10.0, 100.0]])
    assert O.short_conv(w, [], np.array([2.0]))[0] == 200.0 and O.short_conv(w, [np.array([5.0]), np.array([3.0])], np.array([2.0]))[0] == 235.0 and O.short_conv(w, [np.array([3.0])], np.array([2.0]))[0] == 230.0
    rng = np.random.default_rng(1)
    rot = {"dims": 6, "base": 100.0}
    a, b = rng.standard_normal(8), rng.standard_normal(8)
    for nb in (True, False):
        assert np.isclose(O.turn(a, 9, rot, nb) @ O.turn(b, 5, rot, nb), O.turn(a, 104, rot, nb) @ O.turn(b, 100, rot, nb)) and np.array_equal(O.turn(a, 7, rot, nb)[6:], a[6:])
        i, j = (0, 1) if nb else (0, 3)
        assert np.isclose(O.turn(a, 1, rot, nb)[i], a[i] * math.cos(1.0) - a[j] * math.sin(1.0)) and np.isclose(O.turn(a, 1, rot, nb)[j], a[j] * math.cos(1.0) + a[i] * math.sin(1.0))
    assert [i for i, _ in O.run_order({"layers": [0] * 4, "loop": {"start": 1, "stop": 3, "times": 2}})] == [0, 1, 2, 1, 2, 3]
    assert [t for _, t in O.run_order({"layers": [0] * 4, "loop": {"start": 1, "stop": 3, "times": 2}})] == [None, 0, None, 1, None, None]
    bg = {"buckets": 10, "mul_prev": 3, "mul_cur": 7}
    assert O.pair_row(bg, None, 4) == 10 and O.pair_row(bg, 0, 4) == 8 and O.pair_row(bg, 4, 0) == 2
    o = O.combine_maps(np.array([3.0, 1.0]), np.array([1.0, 2.0]), 0.5, 0.25, 0.0)
    assert np.allclose(o, np.array([2.5, 0.0]) / math.sqrt(2.5 ** 2 / 2) * 0.75)
    e = np.exp([1.0, 2.0])
    assert np.allclose(O.softmax(np.array([1.0, 2.0]), 0.5), e / (e.sum() + math.exp(0.5))) and np.allclose(O.softmax(np.array([1.0, 2.0]), 50.0).sum(), 0.0)


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
    edits = [mixer(1, scale=1.0), mixer(1, diff=0.35), mixer(1, mask={"size": 8, "keep_first": 2}), mixer(1, mask={"size": 10, "keep_first": 2}), mixer(1, mask={"size": 9, "keep_first": 1}),
             mixer(1, mask={"size": 9, "keep_first": 3}), mixer(3, mask={"size": 14, "keep_first": 0}), mixer(1, rot={"dims": 4, "base": 300.0}), mixer(1, rot={"dims": 6, "base": 400.0}), mixer(2, scale=0.7),
             mixer(0, rot={"dims": 6, "base": 400.0}), lambda c, T: c["layers"][2]["mlp"].update(limit=0.8), lambda c, T: c["layers"][1]["mlp"].pop("limit"), lambda c, T: c["embedding"]["bigram"].update(mul_prev=12),
             lambda c, T: c["embedding"]["bigram"].update(mul_cur=6), lambda c, T: c["loop"].update(times=2), lambda c, T: c["loop"].update(stop=2), lambda c, T: T.update({"loop.step": T["loop.step"][::-1]}), lambda c, T: T.update({"l1.mix.v.conv": T["l1.mix.v.conv"][:, ::-1]}),
             lambda c, T: T.update({"l1.mix.k": np.roll(T["l1.mix.k"], 10, 0)}), zero("l1.mix.lq1"), zero("l3.mix.lk2"), zero("l0.mix.sink"), zero("l2.mix.g"),
             lambda c, T: T.update({"bigram": np.concatenate([T["bigram"][:-1], T["bigram"][:1]])})]
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


@pytest.mark.gpu
@pytest.mark.parametrize("n,T", [(40, 3), (37, 2), (1, 2), (256, 5), (4096, 2), (1030, 2), (4099, 1), (6000, 3)])
def test_residual_step(n, T):
    """the sum, in place and elsewhere, with and without the fixed vector and the sublayer's result; the norm of what came out"""
    U, lib = gpu()
    rng = np.random.default_rng(n)
    x, y, w, shift = (rng.standard_normal(s).astype(np.float32) for s in ((T, n), (T, n + 3), (n,), (n,)))
    eps = 1e-3
    for use_y in (True, False):
        for use_s in (True, False):
            for in_place in (True, False):
                xd, yd, wd, sd, hd = U.Dev(x), U.Dev(y), U.Dev(w), U.Dev(shift), U.Dev(nbytes=4 * T * (n + 1))
                od = xd if in_place else U.Dev(nbytes=4 * T * n)
                L.check(lib.pi_op_residual_norm(xd.ptr, yd.ptr if use_y else None, n + 3, sd.ptr if use_s else None, wd.ptr, eps, n, T, od.ptr, hd.ptr, n + 1, None))
                want = x.astype(np.float64) + (y[:, :n] if use_y else 0.0) + (shift if use_s else 0.0)
                assert rel_rms(od.get(np.float32, (T, n)), want) < 1e-6 and rel_rms(hd.get(np.float32, (T, n + 1))[:, :n], O.unit_rms(want, eps) * w) < 3e-6, (use_y, use_s, in_place)


@pytest.mark.gpu
@pytest.mark.parametrize("H,G,D,V,R", [(3, 1, 8, 6, 4), (4, 2, 10, 7, 10), (2, 2, 33, 130, 32), (6, 3, 70, 66, 0), (1, 1, 2, 1, 2)])
@pytest.mark.parametrize("pairing", [NEIGHBOURS, HALVES])
def test_queries_and_keys_of_two_maps(H, G, D, V, R, pairing):
    """every map is turned by itself, values go to their cell as they are; a pass's cells learn their positions, no other cell is touched"""
    U, lib = gpu()
    rng = np.random.default_rng(H * 100 + D)
    pos = np.array([0, 1, 2, 63, 64, 511, 2999], np.int32)
    T, n_cells, rot = len(pos), 20, {"dims": R, "base": 500.0} if R else None
    qw, kw, vw = 2 * H * D, 2 * G * D, G * V
    P = rng.standard_normal((T, qw + kw + vw + 1)).astype(np.float32)
    cells = rng.permutation(n_cells)[:T].astype(np.int32)
    dyn = np.concatenate([[0, n_cells, T, 1], cells, np.full(T, n_cells)]).astype(np.int32)
    pd, posd, dd, qd = U.Dev(P), U.Dev(pos), U.Dev(dyn), U.Dev(nbytes=4 * T * qw)
    kd, vd, cd = U.Dev(np.full((n_cells, kw), 7.0, np.float32)), U.Dev(np.full((n_cells, vw), 7.0, np.float32)), U.Dev(np.full(n_cells, -5, np.int32))
    t = lib.pi_rotary_table_create(3000, R, 500.0)
    L.check(lib.pi_op_qkv_prepare_maps(pd.ptr, pd.ptr + 4 * qw, pd.ptr + 4 * (qw + kw), P.shape[1], H, G, 2, D, V, t, pairing, posd.ptr, T, qd.ptr, qw, kd.ptr, vd.ptr, cd.ptr, dd.ptr, None))

    def turned(rows, i):
        return np.concatenate([O.turn(r, int(pos[i]), rot, pairing == NEIGHBOURS) for r in rows.reshape(-1, D).astype(np.float64)])
    want_q = np.stack([turned(P[i, :qw], i) for i in range(T)])
    want_k, want_v, want_c = np.full((n_cells, kw), 7.0), np.full((n_cells, vw), 7.0), np.full(n_cells, -5)
    for i in range(T):
        want_k[cells[i]], want_v[cells[i]], want_c[cells[i]] = turned(P[i, qw:qw + kw], i), P[i, qw + kw:qw + kw + vw], pos[i]
    assert rel_rms(qd.get(np.float32, (T, qw)), want_q) < 2e-6 and rel_rms(kd.get(np.float32, want_k.shape), want_k) < 2e-6
    assert np.array_equal(vd.get(np.float32, want_v.shape), want_v.astype(np.float32)) and np.array_equal(cd.get(np.int32, (n_cells,)), want_c)
    assert lib.pi_op_qkv_prepare_maps(pd.ptr, None, None, P.shape[1], H, G, 2, D, V, t, pairing, posd.ptr, T, qd.ptr, qw, kd.ptr, vd.ptr, cd.ptr, dd.ptr, None) != 0
    lib.pi_rotary_table_free(t)


def diff_attention_ref(q, kc, vc, cpos, vis, pos, scale, size, keep, maps, lam, mult, eps, H, G):
    """explicit sums over the cells that mask, window and kept positions show"""
    T, V = len(pos), vc.shape[-1]
    out = np.zeros((T, H, V))
    for t in range(T):
        ok = vis[t] & ((cpos < keep) | (pos[t] - cpos < size) if size else True)
        js = np.nonzero(ok)[0]
        for h in range(H):
            g = h // (H // G)
            a = [O.softmax(kc[js, g, m].astype(np.float64) @ q[t, h, m].astype(np.float64) * scale) @ vc[js, g].astype(np.float64) for m in range(maps)]
            out[t, h] = O.unit_rms(a[0] - lam * a[1], eps) * mult if maps == 2 else a[0] * mult
    return out


def run_diff(U, lib, q, kc, vc, cpos, vis, pos, scale, size, keep, maps, lam, mult, eps, H, G, splits):
    T, n_kv, D, V = len(pos), vis.shape[1], q.shape[-1], vc.shape[-1]
    ds = [U.Dev(a) for a in (q, kc, vc, cpos, pack_mask(vis, n_kv), np.asarray(pos, np.int32), np.array([0, n_kv, T, 0], np.int32))]
    od = U.Dev(nbytes=4 * T * H * V)
    n_scr = lib.pi_op_window_attention_scratch_floats(H * maps, V, T) if splits else 0
    scr = U.Dev(np.full(max(n_scr, 1), np.nan, np.float32))
    L.check(lib.pi_op_diff_attention(ds[0].ptr, H * maps * D, ds[1].ptr, ds[2].ptr, ds[3].ptr, ds[4].ptr, ds[5].ptr, scale, size, keep, maps, lam, mult, eps, H, G, D, V, T, n_kv, scr.ptr if splits else None, n_scr,
                                     od.ptr, H * V, ds[6].ptr, None))
    return od.get(np.float32, (T, H, V))


@pytest.mark.gpu
@pytest.mark.parametrize("H,G,D,V,size,keep,n_kv,T", [(1, 1, 4, 6, 3, 2, 20, 2), (3, 1, 8, 6, 7, 0, 70, 5), (8, 2, 40, 72, 48, 6, 700, 9), (4, 4, 33, 130, 100, 300, 320, 4), (12, 2, 16, 24, 0, 0, 520, 3),
                                                       (2, 2, 64, 64, 300, 1, 1100, 2), (4, 2, 96, 64, 9, 33, 400, 70), (32, 1, 64, 128, 60, 4, 300, 3), (2, 1, 1, 1, 1, 1, 40, 1)])
@pytest.mark.parametrize("maps", [2, 1])
@pytest.mark.parametrize("splits", [False, True])
def test_differential_attention_against_explicit_sums(H, G, D, V, size, keep, n_kv, T, maps, splits):
    """cells in any order, garbage behind the live cells, large scores (the running maxima of the two maps go their own ways), query heads split over workgroups; in one launch, and with the cell range cut
    into splits that a second launch merges; the plain soft-max over the same mask (one map) too"""
    U, lib = gpu()
    rng = np.random.default_rng(H + D + n_kv)
    kc, vc = (rng.standard_normal((n_kv + 13, G, maps, D)) * 1.5).astype(np.float32), rng.standard_normal((n_kv + 13, G, V)).astype(np.float32)
    kc[n_kv:], vc[n_kv:] = np.nan, np.nan
    cpos = rng.permutation(n_kv + 13).astype(np.int32)
    pos = np.sort(rng.integers(n_kv // 2, n_kv, T)).astype(np.int32)
    vis = (cpos[None, :n_kv] <= pos[:, None]) & (rng.random((T, n_kv)) < 0.8)
    for t in range(T):                                               # (the mask never shows a later position; a token sees at least itself)
        if size:
            near = np.nonzero(cpos[:n_kv] <= pos[t])[0]
            near = near[np.argmax(cpos[near])]
            vis[t, near] = True
            pos[t] = cpos[near]
    vis &= cpos[None, :n_kv] <= pos[:, None]
    q = (rng.standard_normal((T, H, maps, D)) * 2).astype(np.float32)
    args = (q, kc, vc, cpos, vis, pos, 0.6 * D ** -0.25, size, keep, maps, 0.45, 0.7, 1e-3, H, G)
    want = diff_attention_ref(*(a[:n_kv] if a is kc or a is vc or a is cpos else a for a in args))
    assert rel_rms(run_diff(U, lib, *args, splits), want) < 1e-5


@pytest.mark.gpu
@pytest.mark.parametrize("size,keep,p", [(8, 3, 23), (64, 6, 200), (5, 1, 11), (300, 40, 700), (1, 2, 6), (16, 0, 90)])
@pytest.mark.parametrize("T", [1, 70])
def test_edges_of_the_window_and_of_the_kept_tokens(size, keep, p, T):
    """one key far louder than every other in map 1 (or 2): just inside the window and on the last kept position it takes that map, one position further it is not seen — for a token alone and for the
    last of a pass"""
    U, lib = gpu()
    T = min(T, p + 1)
    rng = np.random.default_rng(size + p)
    D, V, n_kv, lam, eps = 8, 5, p + 1, 0.4, 1e-5
    kc, vc = (rng.standard_normal((n_kv, 1, 2, D)) * 0.1).astype(np.float32), rng.standard_normal((n_kv, 1, V)).astype(np.float32)
    cpos = rng.permutation(n_kv).astype(np.int32)
    cell = np.argsort(cpos)
    pos = np.arange(p - T + 1, p + 1)
    vis = cpos[None, :] <= pos[:, None]
    q = np.zeros((T, 1, 2, D), np.float32)
    q[..., 0] = 1.0
    edge = p - size + 1
    for m in (0, 1):
        for at in {edge, edge - 1, keep - 1, keep, 0, p}:
            if not 0 <= at <= p:
                continue
            k2 = kc.copy()
            k2[cell[at], 0, m, 0] = 80.0
            got = run_diff(U, lib, q, k2, vc, cpos, vis, pos, 1.0, size, keep, 2, lam, 0.8, eps, 1, 1, True)
            assert rel_rms(got, diff_attention_ref(q, k2, vc, cpos, vis, pos, 1.0, size, keep, 2, lam, 0.8, eps, 1, 1)) < 1e-4
            quiet = diff_attention_ref(q, kc, vc, cpos, vis, pos, 1.0, size, keep, 2, lam, 0.8, eps, 1, 1)
            seen = at >= edge or at < keep
            alone = size == 1 and keep == 0                          # (a single visible key carries both maps whatever it scores)
            assert alone or (rel_rms(got[-1], quiet[-1]) > 1e-2) == seen, (m, at)


@pytest.mark.gpu
def test_attention_over_maps_refuses_what_it_does_not_serve():
    U, lib = gpu()
    d = U.Dev(nbytes=4096)
    for maps, qs, keep, H, G in ((3, 64, 0, 2, 1), (2, 7, 0, 2, 1), (2, 64, -1, 2, 1), (2, 64, 0, 3, 2)):
        assert lib.pi_op_diff_attention(d.ptr, qs, d.ptr, d.ptr, d.ptr, d.ptr, d.ptr, 1.0, 4, keep, maps, 0.5, 1.0, 1e-5, H, G, 4, 4, 1, 8, None, 0, d.ptr, 64, d.ptr, None) != 0
    assert lib.pi_op_latent_attention_gated(d.ptr, 64, d.ptr, d.ptr, None, None, None, d.ptr, 64, SIGMOID, 3, 1.0, 2, 4, 2, 4, 8, None, 0, d.ptr, 1, 8, d.ptr, 1024, d.ptr, 64, d.ptr, None) != 0


@pytest.mark.gpu
@pytest.mark.parametrize("q_rank,rank,rdim,base", [(11, 12, 6, 300.0), (96, 256, 64, 10000.0), (1, 2, 2, 50.0), (300, 70, 130, 2e5), (5, 9, 0, 10.0)])
@pytest.mark.parametrize("pairing", [HALVES, NEIGHBOURS])
def test_both_latents_in_both_pairings(q_rank, rank, rdim, base, pairing):
    U, lib = gpu()
    rng = np.random.default_rng(q_rank)
    pos = np.array([0, 1, 2, 17, 63, 512, 2999], np.int32)
    T, n_cells, eps, rot = len(pos), 11, 1e-3, {"dims": rdim, "base": base}
    t = lib.pi_rotary_table_create(3000, rdim, base)
    P = rng.standard_normal((T, q_rank + rank + rdim + 3)).astype(np.float32)
    qw, kw = rng.standard_normal(q_rank).astype(np.float32), rng.standard_normal(rank).astype(np.float32)
    cells = rng.permutation(n_cells)[:T].astype(np.int32)
    dyn = np.concatenate([[0, n_cells, T, 1], cells, np.full(T, n_cells)]).astype(np.int32)
    ds = [U.Dev(a) for a in (P, qw, kw, pos, dyn)]
    cq, cache = U.Dev(nbytes=4 * T * (q_rank + 2)), U.Dev(np.zeros((n_cells, rank + rdim), np.float32))
    L.check(lib.pi_op_latent_prepare_ex(ds[0].ptr, P.shape[1], q_rank, ds[1].ptr, rank, ds[2].ptr, rdim, t, pairing, eps, ds[3].ptr, T, cq.ptr, q_rank + 2, cache.ptr, ds[4].ptr, None))
    P64 = P.astype(np.float64)
    assert rel_rms(cq.get(np.float32, (T, q_rank + 2))[:, :q_rank], O.unit_rms(P64[:, :q_rank], eps) * qw) < 2e-6
    want = np.zeros((n_cells, rank + rdim))
    for i in range(T):
        want[cells[i], :rank] = O.unit_rms(P64[i, q_rank:q_rank + rank], eps) * kw
        want[cells[i], rank:] = O.turn(P64[i, q_rank + rank:q_rank + rank + rdim], int(pos[i]), rot, pairing == NEIGHBOURS)
    got = cache.get(np.float32, (n_cells, rank + rdim))
    assert rel_rms(got[:, :rank], want[:, :rank]) < 2e-6 and (rdim == 0 or rel_rms(got[:, rank:], want[:, rank:]) < 2e-6)
    lib.pi_rotary_table_free(t)


def latent_case(U, lib, rng, H, D, R, V, rank, n_kv, pos, base, pairing, gate_width, sink, scale, cache=None, q=None):
    """the operator's output and the plain one; causal, cells in position order"""
    T = len(pos)
    rot = {"dims": R, "base": base}
    vis = np.arange(n_kv)[None, :] <= np.asarray(pos)[:, None]
    t = lib.pi_rotary_table_create(int(max(pos)) + 2, R, base) if R else None
    Wuk, Wuv = (O.bf16_round((rng.standard_normal((H * s, rank)) / np.sqrt(rank)).astype(np.float32)) for s in (D, V))
    q = q if q is not None else rng.standard_normal((T, H, D + R)).astype(np.float32)
    cache = cache if cache is not None else rng.standard_normal((n_kv, rank + R)).astype(np.float32)
    g = rng.standard_normal((T, H * max(gate_width, 1) + 1)).astype(np.float32)
    uk, uv = upload_bf16(lib, Wuk), upload_bf16(lib, Wuv)
    s = np.zeros(H, np.float32) if sink is None else np.asarray(sink, np.float32)
    qd, cd, md, gd, sd, pd, dd = (U.Dev(a) for a in (q, cache, pack_mask(vis, n_kv), g, s, np.asarray(pos, np.int32), np.array([0, n_kv, T, 0], np.int32)))
    n_scr = lib.pi_op_latent_attention_rot_scratch_floats(H, rank, R, T, n_kv)
    scr, od = U.Dev(np.full(n_scr, np.nan, np.float32)), U.Dev(nbytes=4 * T * H * V)        # (what no split has written is not read)
    L.check(lib.pi_op_latent_attention_gated(qd.ptr, H * (D + R), cd.ptr, md.ptr, uk, uv, sd.ptr if sink is not None else None, gd.ptr if gate_width else None, g.shape[1], SIGMOID, max(gate_width, 1), scale, H, D, R, V, rank, t,
                                             pairing, pd.ptr, T, n_kv, scr.ptr, n_scr, od.ptr, H * V, dd.ptr, None))
    want = np.zeros((T, H, V))
    Wk, Wv, C64 = Wuk.reshape(H, D, rank).astype(np.float64), Wuv.reshape(H, V, rank).astype(np.float64), cache.astype(np.float64)
    for i in range(T):
        js = np.nonzero(vis[i])[0]
        for h in range(H):
            sc = (C64[js, :rank] @ Wk[h].T) @ q[i, h, :D].astype(np.float64)
            if R:
                sc = sc + C64[js, rank:] @ O.turn(q[i, h, D:].astype(np.float64), int(pos[i]), rot, pairing == NEIGHBOURS)
            gate = O.sigmoid(g[i, h * gate_width:(h + 1) * gate_width]) if gate_width else 1.0
            want[i, h] = O.softmax(sc * scale, None if sink is None else float(s[h])) @ (C64[js, :rank] @ Wv[h].T) * gate
    lib.pi_weight_free(uk)
    lib.pi_weight_free(uv)
    if t:
        lib.pi_rotary_table_free(t)
    return od.get(np.float32, (T, H, V)), want


@pytest.mark.gpu
@pytest.mark.parametrize("H,D,R,V,rank", [(3, 7, 6, 5, 12), (1, 1, 2, 1, 2), (16, 32, 16, 24, 64), (5, 70, 66, 40, 136), (4, 8, 64, 8, 512), (2, 6, 0, 7, 20), (20, 16, 8, 18, 300)])
@pytest.mark.parametrize("T,n_kv", [(1, 33), (1, 700), (5, 90), (70, 70), (33, 400)])
def test_latent_attention_with_a_sink_and_a_gate_per_value(H, D, R, V, rank, T, n_kv):
    """few and many tokens (splits of the cells, score rows in LDS), both pairings, a gate per value, per head and none, with and without a sink"""
    U, lib = gpu()
    rng = np.random.default_rng(H * 100 + T)
    pos = np.arange(n_kv - T, n_kv)
    for pairing, width, sink in ((HALVES, V, True), (NEIGHBOURS, V, False), (HALVES, 1, True), (HALVES, 0, False)):
        got, want = latent_case(U, lib, rng, H, D, R, V, rank, n_kv, pos, 500.0, pairing, width, rng.standard_normal(H) * 2 if sink else None, (D + R) ** -0.5)
        assert rel_rms(got, want) < 1e-5, (pairing, width, sink)


@pytest.mark.gpu
@pytest.mark.parametrize("T", [1, 40])
def test_a_loud_far_key_and_a_loud_sink(T):
    """of 600 keys one rotated key far louder than every other takes the mass, near or far; a sink of its height takes half of it, a higher one everything (the sink is not scaled)"""
    U, lib = gpu()
    H, D, R, V, rank, n_kv, scale = 2, 4, 4, 6, 16, 600, 0.5
    pos = np.arange(n_kv - T, n_kv)
    for back in (0, 1, 63, 64, 300, n_kv - 1):
        cache = (np.random.default_rng(back).standard_normal((n_kv, rank + R)) * 0.3).astype(np.float32)
        q = np.zeros((T, H, D + R), np.float32)
        loud, e = n_kv - 1 - back, np.array([1.0, 1.0, 0.0, 0.0])
        q[-1, :, D:] = e
        cache[loud, rank:] = O.turn(e, n_kv - 1, {"dims": R, "base": 100.0}, False) * 60.0                # the last token's score on it: 120 * scale
        alone = None
        for sink, part in ((None, 1.0), (60.0, 0.5), (120.0, 0.0)):
            got, want = latent_case(U, lib, np.random.default_rng(5), H, D, R, V, rank, n_kv, pos, 100.0, HALVES, 0, None if sink is None else [sink] * H, scale, cache=cache, q=q)
            assert np.abs(got - want).max() < 1e-4
            alone = got[-1] if alone is None else alone
            assert np.allclose(got[-1], part * alone, atol=2e-4), (back, sink)


@pytest.mark.gpu
@pytest.mark.parametrize("taps", [1, 2, 4, 9])
@pytest.mark.parametrize("ch", [37, 300])
def test_convolution_ahead_of_the_attention(taps, ch):
    """q | k | v channels side by side over input rows that are wider; sequences that start over an earlier owner's state, continue with fewer tokens than taps, share passes, and passes above 32 tokens"""
    U, lib = gpu()
    rng = np.random.default_rng(taps)
    slots = 2
    w = rng.standard_normal((ch, taps)).astype(np.float32)
    wd, state, past = U.Dev(w), U.Dev((rng.standard_normal((slots, max(taps - 1, 1), ch)) * 30).astype(np.float32)), {}
    for step in ([(1, 2, True)], [(1, 1, False), (0, 4, True)], [(0, 45, False), (1, 3, False)], [(1, 1, False)], [(1, 1, True)], [(1, 1, False), (0, 2, True)]):
        T = sum(c for _, c, _ in step)
        x = rng.standard_normal((T, ch + 3)).astype(np.float32)
        rec, want, at = [], np.zeros((T, ch)), 0
        for slot, count, fresh in step:
            if fresh:
                past[slot] = []
            for i in range(count):
                rec.append(slot | (F if fresh and i == 0 else 0))
                u = x[at, :ch].astype(np.float64)
                want[at] = O.short_conv(w.astype(np.float64), past[slot], u)
                past[slot].append(u)
                at += 1
        od, xd, rd = U.Dev(nbytes=4 * T * (ch + 1)), U.Dev(x), U.Dev(np.array(rec, np.int32))
        L.check(lib.pi_op_causal_conv(xd.ptr, ch + 3, ch, taps, wd.ptr, None, state.ptr, rd.ptr, T, NONE, od.ptr, ch + 1, None))
        assert rel_rms(od.get(np.float32, (T, ch + 1))[:, :ch], want) < 2e-6, step


@pytest.mark.gpu
@pytest.mark.parametrize("ff,limit,big", [(7, 0.75, 2.0), (300, None, 2.0), (64, 7.0, 30.0)])
def test_clipped_hidden_layer(ff, limit, big):
    """values on both sides of the bounds and on them; without a bound too"""
    U, lib = gpu()
    rng = np.random.default_rng(ff)
    T = 6
    x = (rng.standard_normal((T, 2 * ff)) * big).astype(np.float32)
    if limit:
        x[0, :3] = x[0, ff:ff + 3] = [limit, -limit, 0.0]
    xd, od = U.Dev(x), U.Dev(nbytes=4 * T * ff)
    L.check(lib.pi_op_glu_mul_ex(xd.ptr, 2 * ff, ff, GLU_CLIPPED, limit or 0.0, -1, T, od.ptr, ff, None))
    eye = {"gate": np.eye(2 * ff)[:ff], "up": np.eye(2 * ff)[ff:], "down": np.eye(ff)}
    assert rel_rms(od.get(np.float32, (T, ff)), np.stack([O.feed_forward(eye, "", {"limit": limit}, r.astype(np.float64)) for r in x])) < 3e-6


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
    tol = TOL[exact] * (3 if variant in ("wide_heads", "edges") else 1)
    whole = np.concatenate([e.ctx.feed(toks[:48], 0, 0), e.ctx.feed(toks[48:], 48, 0)])
    assert within(logit_err(whole, want), exact, tol)
    e.ctx.seq_rm(0, -1, -1)
    parts, at = [], 0
    for n in [2, 3, 31, 2, 1, 1, 7, 2, 5, 1, 1, 1, 2, 16]:                 # portions down to two tokens and single tokens, cut inside windows and convolutions
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
    layers = [O.attention_layer(heads=8, kv_heads=2, dim=24, vdim=48, conv=4, size=70, keep_first=5, rot_dims=16, base=1000.0, scale=0.25, diff=0.4, ff=160),
              O.latent_layer(heads=6, dim=24, rot_dim=16, vdim=40, q_rank=64, kv_rank=80, base=10000.0, scale=0.2, ff=256)]
    m = small_model(seed=13, layers=layers, width=128, vocab=200, loop={"start": 0, "stop": 2, "times": 2}, buckets=311)
    rng = np.random.default_rng(6)
    toks = [int(t) for t in rng.integers(0, 200, 320)]
    want = O.run(m, toks)
    e = Engine(tmp_path, m, n_ctx=330, n_batch=128, exact=exact)
    got = np.concatenate([e.ctx.feed(toks[:300], 0, 0)] + [e.ctx.feed(toks[i:i + 1], i, 0) for i in range(300, 320)])
    assert within(logit_err(got, want), exact, TOL[exact] * 2)
    e.close()


@pytest.mark.gpu
def test_residual_stream_run_by_run(tmp_path):
    """models cut after 1, 2, ... layers, with and without a repeated run, give the oracle's logits, so the first wrong layer would be named"""
    full = small_model(seed=4)
    toks = [5, 17, 3, 80, 0, 41, 41, 7, 9, 9, 30, 2, 2, 61, 8, 8, 8, 12, 70, 3, 3, 44]
    for n in range(1, 6):
        for loop in (None, {"start": 0, "stop": n, "times": 2}, {"start": n - 1, "stop": n, "times": 3}):
            cfg, T = dict(full["config"], layers=full["config"]["layers"][:n]), dict(full["tensors"])
            cfg.pop("loop", None)
            if loop:
                cfg["loop"] = loop
                T["loop.step"] = T["loop.step"][:loop["times"]]
            m = {"config": cfg, "tensors": T}
            e = Engine(tmp_path, m, n_ctx=32, n_batch=8, name="cut%d_%s" % (n, loop and loop["times"]))
            assert logit_err(e.ctx.feed(toks, 0, 0), O.run(m, toks)).max() < TOL[True], (n, loop)
            e.close()


@pytest.mark.gpu
def test_first_tokens_of_a_sequence(tmp_path):
    """a sequence's first tokens see no previous token, no convolution input and no key of whoever held the slot and the cells before"""
    m = small_model(seed=17)
    e = Engine(tmp_path, m, n_ctx=64, n_batch=8, slots=1)
    for toks in ([7], [7, 7], [78, 7, 3], [3, 78, 7, 7, 2, 2, 2, 9, 1, 4, 4]):
        got = np.concatenate([e.ctx.feed(toks[i:i + 3], i, 0) for i in range(0, len(toks), 3)])
        assert logit_err(got, O.run(m, toks)).max() < TOL[True], toks
        e.ctx.seq_rm(0, -1, -1)
    e.close()


@pytest.mark.gpu
def test_pair_rows_with_large_multipliers(tmp_path):
    """products of token and multiplier far beyond 32 bits, across the border between two passes too"""
    m = small_model(seed=19, layers=[O.latent_layer(ff=None)], loop=None, buckets=59, mul_prev=2654435761, mul_cur=4294967311)
    toks = [82, 81, 0, 0, 82, 7, 40, 41, 3]
    e = Engine(tmp_path, m, n_ctx=32, n_batch=4)
    assert logit_err(np.concatenate([e.ctx.feed(toks[:5], 0, 0), e.ctx.feed(toks[5:], 5, 0)]), O.run(m, toks)).max() < TOL[True]
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
        assert np.quantile(logit_err(mine, alone[s].astype(np.float64)), 1.0 if exact else 0.9) < (2e-5 if exact else 3e-2), s
        if exact:
            assert logit_err(mine, O.run(m, toks)).max() < TOL[True], s
    e.close()


@pytest.mark.gpu
def test_freed_cells_and_slots_are_used_again(tmp_path):
    """more requests than slots and cells, one after the other and interleaved: a finished request gives back what it held, the next one starts from nothing; a copied sequence continues like
    the original (previous token and convolution inputs included)"""
    m = small_model(seed=31)
    rng = np.random.default_rng(9)
    e = Engine(tmp_path, m, n_ctx=48, n_batch=16, slots=2)
    for again in range(5):
        a = [int(t) for t in rng.integers(0, VOCAB, 20 + again)]
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
            assert logit_err(got, O.run(m, toks)).max() < TOL[True], again
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
def test_window_borders_and_kept_tokens_show_in_prompts_and_in_decoding(tmp_path, exact):
    """sharp attention over several hundred tokens, windows that do not divide the pass width: a key wrongly seen or lost at a window's edge, or one kept token too many or too few, shows far above
    rounding — the same model with a window or a number of kept tokens that is one off is far away"""
    layers = [O.attention_layer(heads=2, kv_heads=1, dim=8, vdim=6, conv=3, size=50, keep_first=6, rot_dims=4, base=200.0, scale=1.0, diff=0.2, ff=16),
              O.latent_layer(heads=2, dim=4, rot_dim=8, vdim=8, q_rank=16, kv_rank=12, base=200.0, scale=1.0, ff=None),
              O.attention_layer(heads=3, kv_heads=3, dim=6, vdim=4, conv=2, size=21, keep_first=3, rot_dims=2, base=50.0, scale=1.2, diff=0.5, ff=12)]
    m = small_model(seed=41, layers=layers, width=32, loop=None)
    rng = np.random.default_rng(12)
    toks = [int(t) for t in rng.integers(0, VOCAB, 330)]
    want = O.run(m, toks)
    e = Engine(tmp_path, m, n_ctx=340, n_batch=128, exact=exact)
    got = np.concatenate([e.ctx.feed(toks[:290], 0, 0)] + [e.ctx.feed(toks[i:i + 1], i, 0) for i in range(290, 330)])       # every decoded token moves both windows
    assert within(logit_err(got, want), exact)
    if exact:                                                         # (at serving precision one key more or less among fifty is not far enough from rounding to tell)
        for where, mask in ((0, (51, 6)), (0, (49, 6)), (0, (50, 5)), (0, (50, 7)), (2, (22, 3)), (2, (21, 2)), (2, (21, 4))):
            other = json.loads(json.dumps(m["config"]))
            other["layers"][where]["mixer"]["mask"] = {"size": mask[0], "keep_first": mask[1]}
            off = logit_err(got, O.run({"config": other, "tensors": m["tensors"]}, toks))
            assert off[100:290].max() > 30 * TOL[exact] and off[290:].max() > 30 * TOL[exact], (where, mask)
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
    m = small_model(seed=67, layers=[O.latent_layer(ff=None), O.attention_layer()], loop={"start": 0, "stop": 2, "times": 2})
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
