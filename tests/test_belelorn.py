"""The Belelorn design in the engine against the plain implementation of tests/plain_belelorn.py.

The configurations and weights are made here.  The CPU tests cover the configuration reader, the plan, the random
checkpoint and the plain implementation's own consistency on cases worked by hand; the GPU tests run the engine's step
function, cache, scheduler and kernels: each mixer and feed-forward alone, loops over layers, whole prompts against
token-by-token decoding, prompts in portions, unequal batches, slots, pages and states used again, keys that stand out
at the edges of the window, among the first keys, at page borders and far back (in prompts and in decoding), memories
that last, long decoding through recorded graphs, odd sizes, configurations drawn from seeds, and greedy generation
through the server."""
import json
import math

import numpy as np
import pytest
import torch

import plain_belelorn as P
from helpers import rel_err

TOL = {"float32": 2e-5, "bfloat16": 8e-2}


class Rows:
    """Collects rows of logits beside what they should be.  float32: every row within the tolerance.  bfloat16: a
    rounding can tip a router's choice between two experts whose scores are close, which changes that token's row by
    far more than roundings do and is no fault, so nine rows in ten must be within the tolerance, and every row finite."""

    def __init__(self, dtype):
        self.dtype, self.errs = dtype, []

    def add(self, got, want, note=None):
        got, want = np.atleast_2d(np.asarray(got, dtype=np.float64)), np.atleast_2d(want)
        assert got.shape == want.shape and np.isfinite(got).all(), note
        scale = max(1e-30, np.abs(want).max())
        self.errs += [(float(np.abs(g - x).max() / scale), note) for g, x in zip(got, want)]

    def check(self):
        tol = TOL[self.dtype]
        bad = [e for e in self.errs if e[0] > tol]
        if self.dtype == "float32":
            assert not bad, bad[:5]
        else:
            assert len(bad) * 10 <= len(self.errs), (len(bad), len(self.errs), bad[:5])


# ---- configurations and weights of the tests --------------------------------------------------
def moe(experts=5, top=2, ff=24, limit=1.2, shared=16, shared_limit=0.7):
    f = dict(kind="moe", expert=dict(ff=ff, limit=limit), router=dict(experts=experts, top=top))
    if shared:
        f["shared"] = dict(ff=shared, limit=shared_limit)
    return f


def dense(ff=56):
    return dict(kind="dense", ff=ff)


def pair(heads=4, kv_heads=2, dim=16, scale=0.4, softcap=20.0, size=40, keep=3, r_heads=3, r_dim=12, r_vdim=20,
         decay=(0.5, 0.9, 1.0), mlp="default"):
    left = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, scale=scale, softcap=softcap)
    if size:
        left["mask"] = dict(size=size, keep_first=keep)
    right = dict(heads=r_heads, dim=r_dim, vdim=r_vdim, decay=list(decay))
    return dict(type="parallel", mixer=dict(left=left, right=right), mlp=dense() if mlp == "default" else mlp)


def memory(heads=3, dim=16, vdim=24, cap=8.0, mlp="default"):
    return dict(type="mlstm", mixer=dict(heads=heads, dim=dim, vdim=vdim, gate_cap=cap), mlp=moe() if mlp == "default" else mlp)


def config(layers, width=48, vocab=101, eps=1e-5, logit_scale=0.7, loop=None):
    cfg = dict(architecture="Belelorn", layers=layers, norm=dict(eps=eps), vocab=vocab, width=width, logit_scale=logit_scale)
    if loop:
        cfg["loop"] = dict(start=loop[0], stop=loop[1], times=loop[2])
    return cfg


# layers that differ from each other in every size, both mixers and every feed-forward inside and outside the loop, which
# starts behind a layer and ends before one and runs three times
MIXED = config([memory(heads=2, dim=8, vdim=40, mlp=dense(40)),
                pair(),
                memory(mlp=None),
                pair(heads=6, kv_heads=1, dim=8, size=70, keep=66, r_heads=2, r_dim=16, r_vdim=8, decay=(0.97, 0.3), scale=0.9,
                     mlp=moe(experts=4, top=1, shared=0)),
                memory(heads=1, dim=48, vdim=16, cap=15.0),
                pair(heads=2, kv_heads=2, dim=32, size=1, keep=0, r_heads=1, r_dim=24, r_vdim=40, decay=(0.999,), mlp=moe(experts=1, top=1))],
               loop=(1, 4, 3))
# sizes that are no multiples of eight, no window, no cap, a logit scale of one, one value lane more than a block's
# columns, every expert chosen, a loop of one pass over everything
ODD = config([pair(heads=3, kv_heads=3, dim=10, size=0, softcap=None, r_heads=3, r_dim=10, r_vdim=14, decay=(0.2, 0.8, 0.95),
                   mlp=moe(experts=3, top=3, ff=12, shared=5)),
              memory(heads=3, dim=9, vdim=65, mlp=dense(13)),
              memory(heads=5, dim=70, vdim=6, cap=3.0, mlp=moe(experts=7, top=2, ff=5, limit=0.5, shared=7)),
              pair(heads=5, kv_heads=1, dim=6, size=7, keep=1, r_heads=1, r_dim=5, r_vdim=65, decay=(1.0,), mlp=None)],
             width=36, vocab=53, eps=1e-6, logit_scale=1.0, loop=(0, 4, 1))


def make_weights(cfg, seed, lasting=False):
    """float64 arrays that are exact in bfloat16.  Sublayers join the residual with a gain of about 0.4: with one of one, a
    chain of a dozen random layers multiplies a rounding so much that bfloat16 rows have little in common with exact ones.
    lasting: forget gates of the matrix memories near one."""
    g = np.random.default_rng(seed)
    D = cfg["width"]
    bf = lambda a: torch.from_numpy(np.asarray(a, dtype=np.float32)).bfloat16().double().numpy()
    mat = lambda o, i, s=1.0: bf(g.standard_normal((o, i)) * s / math.sqrt(i))
    near = lambda n, c: bf(c + 0.15 * g.standard_normal(n))
    w = {"embed": bf(g.standard_normal((cfg["vocab"], D))), "final.norm": near(D, 0), "head": mat(cfg["vocab"], D)}
    if cfg.get("loop"):
        w["loop.in"], w["loop.step"] = mat(D, 2 * D), bf(0.5 * g.standard_normal((cfg["loop"]["times"], D)))
    for i, L in enumerate(cfg["layers"]):
        l, m, f = f"l{i}.", L["mixer"], L["mlp"]
        w[l + "norm1"], w[l + "norm1b"] = near(D, 0), near(D, -0.6)
        p = l + "mix."
        if L["type"] == "mlstm":
            H, dk, dv = m["heads"], m["dim"], m["vdim"]
            for r, n in (("q", H * dk), ("k", H * dk), ("v", H * dv), ("g", H * dv), ("i", H), ("f", H)):
                w[p + r] = mat(n, D)
            w[p + "i.b"], w[p + "f.b"] = bf(g.standard_normal(H)), bf(g.uniform(5.0, 8.0, H) if lasting else g.uniform(-1.0, 5.0, H))
            w[p + "norm"], w[p + "o"] = near(H * dv, 1), mat(D, H * dv)
        else:
            a, b = m["left"], m["right"]
            H, G, d = a["heads"], a["kv_heads"], a["dim"]
            w[p + "left.q"], w[p + "left.k"], w[p + "left.o"] = mat(H * d, D), mat(G * d, D), mat(D, H * d)
            w[p + "left.q.b"], w[p + "left.k.b"] = bf(0.5 * g.standard_normal(H * d)), bf(0.5 * g.standard_normal(G * d))
            H, dk, dv = b["heads"], b["dim"], b["vdim"]
            for r, n in (("q", H * dk), ("k", H * dk), ("v", H * dv), ("g", H * dv)):
                w[p + "right." + r] = mat(n, D)
            w[p + "right.norm"], w[p + "right.o"] = near(H * dv, 1), mat(D, H * dv)
            w[p + "left.out"], w[p + "right.out"] = near(D, 1), near(D, 1)
        if f is None:
            continue
        w[l + "norm2"], w[l + "norm2b"] = near(D, 0), near(D, -0.6)
        p = l + "mlp."
        if f["kind"] == "dense":
            w[p + "up"], w[p + "down"] = mat(f["ff"], D), mat(D, f["ff"])
            continue
        w[p + "router"] = mat(f["router"]["experts"], D, 2.0)
        for e, n in [(f"e{e}.", f["expert"]["ff"]) for e in range(f["router"]["experts"])] + \
                ([("shared.", f["shared"]["ff"])] if f.get("shared") else []):
            w[p + e + "gate"], w[p + e + "up"], w[p + e + "down"] = mat(n, D, 2.0), mat(n, D, 2.0), mat(D, n)
    return w


def write_folder(path, cfg, w):
    from burn_lm_amd.weights import safetensors_io as st
    with open(path / "config.json", "w") as f:
        json.dump(cfg, f)
    st.write_file(str(path / "model.safetensors"), ((k, torch.from_numpy(v).bfloat16()) for k, v in w.items()))
    return str(path)


def tokens_of(cfg, seed, n):
    return [int(x) for x in np.random.default_rng(seed).integers(0, cfg["vocab"], n)]


# ---- CPU: configuration, plan, random checkpoint, plain implementation ----------------------------
def test_config_is_read_and_refused_by_key():
    from burn_lm_amd import registry
    from burn_lm_amd.errors import ConfigError
    import burn_lm_amd.models  # noqa: F401
    arch = registry.architecture_of(MIXED)
    assert arch.name == "Belelorn"
    cfg = arch.read_config(MIXED)
    assert cfg.layers[2].mlp is None and cfg.layers[3].mlp.shared_ff == 0 and cfg.layers[0].mixer.gate_cap == 8.0
    assert cfg.layers[3].mixer.left.keep_first == 66 and cfg.layers[5].mixer.left.window == 1 and cfg.loop.times == 3
    odd = arch.read_config(ODD)
    assert odd.layers[0].mixer.left.window == 0 and odd.layers[0].mixer.left.softcap == 0.0 and odd.logit_scale == 1.0
    for path, value, word in ((("layers", 1, "mixer", "left", "vdim"), None, "vdim"), (("width",), "48", "width"),
                              (("layers", 0, "type"), "serial", "type"), (("norm",), {}, "eps"), (("logit_scale",), None, "logit_scale"),
                              (("layers", 1, "mixer", "left", "kv_heads"), 3, "kv_heads"),
                              (("layers", 1, "mixer", "left", "vdim"), 8, "keys"),
                              (("layers", 1, "mixer", "left", "mask"), dict(size=0, keep_first=1), "size"),
                              (("layers", 1, "mixer", "left", "mask"), dict(size=4, keep_first=-1), "keep_first"),
                              (("layers", 1, "mixer", "left", "softcap"), -1.0, "softcap"),
                              (("layers", 1, "mixer", "right", "decay"), [0.5, 0.5], "decay"),
                              (("layers", 1, "mixer", "right", "decay"), [0.5, 0.5, 1.5], "decay"),
                              (("layers", 0, "mixer", "gate_cap"), 0.0, "gate_cap"),
                              (("layers", 3, "mlp", "router", "top"), 5, "top"),
                              (("layers", 4, "mlp", "shared", "limit"), None, "limit"),
                              (("layers", 1, "mlp", "kind"), "glu", "kind"),
                              (("loop",), dict(start=1, stop=7, times=2), "loop"), (("loop",), dict(start=2, stop=2, times=2), "loop"),
                              (("loop",), dict(start=0, stop=2), "times")):
        bad = json.loads(json.dumps(MIXED))
        at = bad
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = value
        with pytest.raises(ConfigError, match=word):
            arch.read_config(bad)
    one = json.loads(json.dumps(MIXED))
    one["layers"][1]["mixer"]["right"]["decay"] = 0.75      # one number stands for every head
    assert arch.read_config(one).layers[1].mixer.right.decay == (0.75,) * 3


def test_plan_asks_for_the_checkpoints_tensors():
    from burn_lm_amd import registry
    import burn_lm_amd.parts  # noqa: F401
    from burn_lm_amd.engine.model import Model
    from burn_lm_amd.parts.base import KVNeed, StateNeed
    for cfg_dict in (MIXED, ODD):
        w = make_weights(cfg_dict, 0)
        arch = registry.architecture_of(cfg_dict)
        cfg = arch.read_config(cfg_dict)
        model = Model(arch.plan(cfg, {k: v.shape for k, v in w.items()}))
        assert {k: tuple(s.shape) for k, s in model.tensor_specs().items()} == {k: tuple(v.shape) for k, v in w.items()}
        assert {k: tuple(v[0]) for k, v in arch.checkpoint_tensors(cfg).items()} == {k: tuple(v.shape) for k, v in w.items()}
        # the places of the layer order are the runs of the plain implementation
        assert [(p.layer, p.turn is not None) for p in model.plan.order] == [(i, first) for i, _, first in P.runs(cfg_dict)]
        assert [p.turn for p in model.plan.order if p.turn is not None] == list(range(cfg_dict["loop"]["times"]))
        assert all(part.graph_safe for part in model.all_parts())
    needs = model.cache_needs()
    assert needs[0] == (KVNeed(3, 10, 0, value_dim=10), StateNeed((3, 10, 14)))
    assert needs[1] == (StateNeed((3, 9, 65)), StateNeed((3, 9)), StateNeed((3,)))
    assert needs[3][0] == KVNeed(1, 6, 7, value_dim=6, keep_first=1)
    # without a loop: no entry, every layer once
    plain = dict(MIXED, loop=None)
    plan = arch.plan(arch.read_config(plain))
    assert plan.entry is None and [p.layer for p in plan.order] == list(range(6))


def test_a_pass_needs_an_entry():
    from burn_lm_amd import registry
    import burn_lm_amd.models  # noqa: F401
    from burn_lm_amd.engine.model import Model
    arch = registry.architecture("Belelorn")
    plan = arch.plan(arch.read_config(MIXED))
    plan.entry = None
    with pytest.raises(ValueError, match="entry"):
        Model(plan)


def test_random_folder_loads_into_the_plain_implementation(tmp_path):
    import burn_lm_amd
    from burn_lm_amd.weights import safetensors_io as st
    folder = burn_lm_amd.write_random_model(str(tmp_path), ODD, seed=5)
    w = {n: f.tensor(n).double().numpy() for n, f in st.open_folder(folder).items()}
    assert w["l0.mlp.router"].shape == (3, 36) and "l3.norm2" not in w and w["l3.mix.right.norm"].shape == (65,)
    logits = P.forward(w, ODD, tokens_of(ODD, 0, 9))
    assert logits.shape == (9, 53) and np.isfinite(logits).all() and logits.std() > 0.05


def test_plain_mechanisms_on_cases_worked_by_hand():
    # position vectors: sine and cosine in turn, the second pair slower by base^(-2/4)
    v = P.position_vectors([0, 3], 4)
    assert np.allclose(v, [[0, 1, 0, 1], [math.sin(3), math.cos(3), math.sin(0.03), math.cos(0.03)]], atol=1e-12)
    # equal scores: a query averages the keys it sees (the values are the keys as projected); a window of two beside
    # which the first token stays
    m = dict(heads=1, kv_heads=1, dim=2, vdim=2, scale=1.0, softcap=None, mask=dict(size=2, keep_first=1))
    W = {"a.q": np.zeros((2, 1)), "a.q.b": np.zeros(2), "a.k": np.array([[1.0], [0.0]]), "a.k.b": np.array([0.0, 5.0]), "a.o": np.eye(2)}
    h = np.array([[2.0], [4.0], [6.0], [8.0]])
    assert np.allclose(P.softmax_attention(W, "a.", m, h, 1e-12), [[2, 5], [3, 5], [4, 5], [(2 + 6 + 8) / 3, 5]])
    m["mask"]["keep_first"] = 0
    assert np.allclose(P.softmax_attention(W, "a.", m, h, 1e-12)[3], [7, 5])
    assert [P.visible(5, j, 3, 2) for j in range(7)] == [True, True, False, True, True, True, False]
    # unit-norm queries and keys: the score is scale * dim * cosine; capped scores keep their order and stay below the cap
    m = dict(heads=1, kv_heads=1, dim=2, vdim=2, scale=3.0, softcap=1.0, mask=None)
    W.update({"a.q": np.array([[1.0], [0.0]]), "a.k": np.array([[1.0], [0.0]]), "a.k.b": np.array([0.0, 0.0])})
    got = P.softmax_attention(W, "a.", m, np.array([[-7.0], [0.5]]), 0.0)
    e = math.exp(math.tanh(6.0)) / math.exp(math.tanh(-6.0))
    assert np.allclose(got[1, 0], (0.5 * e - 7.0) / (e + 1.0))
    # matrix memory: against the same recurrence without stabiliser, whose numbers here are small
    g = np.random.default_rng(1)
    q, k, v = g.standard_normal((9, 2, 3)), g.standard_normal((9, 2, 3)), g.standard_normal((9, 2, 4))
    li, lf = g.standard_normal((9, 2)), P.log_sigmoid(g.standard_normal((9, 2)))
    o, (S, n, top) = P.matrix_memory(q, k, v, li, lf)
    A, b = np.zeros((2, 3, 4)), np.zeros((2, 3))
    for t in range(9):
        for hd in range(2):
            A[hd] = math.exp(lf[t, hd]) * A[hd] + math.exp(li[t, hd]) * np.outer(k[t, hd], v[t, hd])
            b[hd] = math.exp(lf[t, hd]) * b[hd] + math.exp(li[t, hd]) * k[t, hd]
    for hd in range(2):
        s = math.exp(top[hd])
        assert np.allclose(S[hd] * s, A[hd]) and np.allclose(n[hd] * s, b[hd]) and top[hd] >= li[8, hd]
        assert np.allclose(o[8, hd], (A[hd].T @ q[8, hd]) / (max(abs(b[hd] @ q[8, hd]), 1.0) + 1e-6 * s))
    # the stabiliser starts at zero: a first input gate far below it counts for what it is
    o, (_, _, top) = P.matrix_memory(np.ones((1, 1, 1)), np.ones((1, 1, 1)), np.full((1, 1, 1), 5.0), np.full((1, 1), -3.0), np.full((1, 1), -1.0))
    assert top[0] == -1.0 and np.allclose(o, 5 * math.exp(-2) / (math.exp(1.0) + 1e-6))
    # experts: the weight is the score itself and sits on the input, where it meets the limits
    f = dict(kind="moe", expert=dict(ff=1, limit=2.0), router=dict(experts=3, top=1), shared=dict(ff=1, limit=0.5))
    W = {"m.router": np.array([[0.0], [2.0], [-1.0]]), "m.shared.gate": np.array([[1.0]]), "m.shared.up": np.array([[-9.0]]), "m.shared.down": np.array([[1.0]])}
    for e in range(3):
        W[f"m.e{e}.gate"], W[f"m.e{e}.up"], W[f"m.e{e}.down"] = np.array([[1.0]]), np.array([[3.0]]), np.array([[10.0 ** e]])
    w = P.sigmoid(2.0)
    want = 10 * (w * P.sigmoid(1.702 * w) * (min(3 * w, 2.0) + 1)) + 0.5 * P.sigmoid(0.851) * (-0.5 + 1)
    assert np.allclose(P.experts(W, "m.", f, np.array([[1.0]])), want)
    assert np.allclose(P.dense({"d.up": np.array([[1.0], [-1.0]]), "d.down": np.array([[1.0, 7.0]])}, "d.", None, np.array([[3.0]])), 9.0)
    # the order of a loop: layer 0, then layers 1 and 2 twice, then layer 3
    order = P.runs(dict(layers=[0] * 4, loop=dict(start=1, stop=3, times=2)))
    assert order == [(0, None, False), (1, 0, True), (2, 0, False), (1, 1, True), (2, 1, False), (3, None, False)]


# ---- GPU ----------------------------------------------------------------------------------------
def engine_for(tmp_path, cfg, w, dtype, **kw):
    from burn_lm_amd.engine.loading import load_engine
    kw.setdefault("max_tokens", 1024)
    return load_engine(write_folder(tmp_path, cfg, w), dtype=dtype, **kw)


def whole(eng, toks):
    s = eng.open()
    out = eng.step([(s, toks, list(range(len(toks))))]).double().cpu().numpy()
    eng.close(s)
    return out


ALONE = {
    "pair": config([pair(mlp=None)]),
    "pair_ungrouped_no_window": config([pair(heads=6, kv_heads=6, dim=8, size=0, mlp=None)]),
    "pair_one_kv_head_no_cap": config([pair(heads=8, kv_heads=1, dim=32, softcap=None, size=65, keep=64, mlp=None)]),
    "pair_wide_heads": config([pair(heads=2, kv_heads=1, dim=96, scale=0.1, size=30, keep=70, mlp=None)]),
    "memory": config([memory(mlp=None)]),
    "memory_one_wide_head": config([memory(heads=1, dim=70, vdim=150, cap=2.0, mlp=None)]),
    "dense": config([memory(mlp=dense(80))]),
    "experts": config([memory(mlp=moe())]),
    "experts_top1_unshared": config([memory(mlp=moe(experts=3, top=1, shared=0))]),
    "experts_all": config([memory(mlp=moe(experts=4, top=4, limit=0.3, shared=40, shared_limit=3.0))]),
    "loop_of_one_layer": config([memory(mlp=dense())], loop=(0, 1, 3)),
    "loop_in_the_middle": config([memory(mlp=None), pair(mlp=None), memory(heads=1, mlp=None)], loop=(1, 2, 2)),
    "loop_of_one_pass": config([memory(mlp=None), pair(mlp=None)], loop=(1, 2, 1)),
    "loop_over_everything": config([pair(mlp=None), memory(mlp=None)], loop=(0, 2, 4)),
}


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(ALONE))
def test_every_mechanism_alone(tmp_path, name, dtype):
    cfg = ALONE[name]
    w = make_weights(cfg, 3)
    eng = engine_for(tmp_path, cfg, w, dtype, graphs=False)
    toks = tokens_of(cfg, 4, 150)       # three pages
    want = P.forward(w, cfg, toks)
    rows = Rows(dtype)
    rows.add(whole(eng, toks), want, "whole")
    # one token at a time from the first one on: the first tokens of a sequence, then a page border
    s = eng.open()
    rows.add(np.stack([eng.step([(s, [t], [0])])[0].double().cpu().numpy() for t in toks[:70]]), want[:70], "one by one")
    eng.close(s)
    rows.check()


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_portions_batches_and_slots_used_again(tmp_path, dtype):
    cfg = MIXED
    w = make_weights(cfg, 5)
    eng = engine_for(tmp_path, cfg, w, dtype, max_tokens=1536, max_seqs=6)
    reqs = [tokens_of(cfg, 10 + i, n) for i, n in enumerate((200, 7, 66, 129, 1))]
    want = [P.forward(w, cfg, r) for r in reqs]
    rows = Rows(dtype)
    for r, x in zip(reqs, want):
        rows.add(whole(eng, r), x, "whole")
    # a prompt in portions of several sizes, down to two tokens and one
    for sizes in ((2, 5, 57, 64, 3, 69), (63, 2, 1, 1, 133), (128, 72), (1, 1, 1, 2, 195)):
        s, at = eng.open(), 0
        for n in sizes:
            rows.add(eng.step([(s, reqs[0][at:at + n], list(range(n)))]).double().cpu().numpy(), want[0][at:at + n], sizes)
            at += n
        eng.close(s)
        assert at == 200
    # unequal batches: prompts in one step, then one token each; shorter requests end earlier; the second round
    # finds slots, pages and states that the first one used
    for round_ in range(2):
        order = [0, 1, 2, 3, 4] if round_ == 0 else [3, 4, 0, 2, 1]
        slots = {i: eng.open() for i in order}
        cut = {i: max(1, len(reqs[i]) - 6) for i in order}
        got = eng.step([(slots[i], reqs[i][:cut[i]], list(range(cut[i]))) for i in order]).double().cpu().numpy()
        o = 0
        for i in order:
            rows.add(got[o:o + cut[i]], want[i][:cut[i]], (round_, i))
            o += cut[i]
            if cut[i] == len(reqs[i]):
                eng.close(slots[i])
        for k in range(6):
            live = [i for i in order if cut[i] + k < len(reqs[i])]
            got = eng.step([(slots[i], [reqs[i][cut[i] + k]], [0]) for i in live]).double().cpu().numpy()
            for row, i in enumerate(live):
                rows.add(got[row], want[i][cut[i] + k], (round_, i, k))
            for i in order:
                if cut[i] + k + 1 == len(reqs[i]):
                    eng.close(slots[i])
    rows.check()
    assert eng.cache.pages_in_use() == 0 and eng.cache.free_slots == 6


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_through_recorded_steps(tmp_path, dtype):
    cfg = MIXED
    w = make_weights(cfg, 6, lasting=True)
    eng = engine_for(tmp_path, cfg, w, dtype)
    a, b = tokens_of(cfg, 20, 200), tokens_of(cfg, 21, 150)
    wa, wb = P.forward(w, cfg, a), P.forward(w, cfg, b)
    sa, sb = eng.open(), eng.open()
    rows = Rows(dtype)
    got = eng.step([(sa, a[:30], [29]), (sb, b[:3], [2])]).double().cpu().numpy()
    rows.add(got, np.stack([wa[29], wb[2]]), "prompts")
    for k in range(140):          # across two page borders; one shape, recorded and replayed
        got = eng.step([(sa, [a[30 + k]], [0]), (sb, [b[3 + k]], [0])]).double().cpu().numpy()
        rows.add(got, np.stack([wa[30 + k], wb[3 + k]]), k)
    rows.check()
    assert eng.graphs.replays >= 100


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_prompts_through_recorded_steps(tmp_path, dtype):
    """The same prompt shape several times: recorded, then replayed at a padded size, between steps that change states and
    pages in the meantime."""
    cfg = MIXED
    w = make_weights(cfg, 12)
    eng = engine_for(tmp_path, cfg, w, dtype)
    rows = Rows(dtype)
    for i, n in enumerate((100, 90, 101, 128, 97)):
        toks = tokens_of(cfg, 50 + i, n + 3)
        want = P.forward(w, cfg, toks)
        s = eng.open()
        rows.add(eng.step([(s, toks[:n], [n - 1])]).double().cpu().numpy(), want[n - 1:n], ("prompt", i))
        for k in range(3):
            rows.add(eng.step([(s, [toks[n + k]], [0])]).double().cpu().numpy(), want[n + k:n + k + 1], ("next", i, k))
        eng.close(s)
    rows.check()
    assert eng.graphs.replays >= 3


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_sizes_that_are_no_multiples_of_eight(tmp_path, dtype):
    cfg = ODD
    w = make_weights(cfg, 7)
    eng = engine_for(tmp_path, cfg, w, dtype)
    reqs = [tokens_of(cfg, 30 + i, n) for i, n in enumerate((90, 31))]
    want = [P.forward(w, cfg, r) for r in reqs]
    slots = [eng.open(), eng.open()]
    rows = Rows(dtype)
    got = eng.step([(slots[0], reqs[0][:80], list(range(80))), (slots[1], reqs[1][:21], list(range(21)))]).double().cpu().numpy()
    rows.add(got[:80], want[0][:80], "prompt 0")
    rows.add(got[80:], want[1][:21], "prompt 1")
    for k in range(10):
        got = eng.step([(slots[0], [reqs[0][80 + k]], [0]), (slots[1], [reqs[1][21 + k]], [0])]).double().cpu().numpy()
        rows.add(got, np.stack([want[0][80 + k], want[1][21 + k]]), k)
    rows.check()


@pytest.mark.gpu
def test_a_lasting_memory_and_pages_that_leave_the_window(tmp_path):
    """Two sequences that differ in their first token alone, compared hundreds of tokens later, when that token has long
    left every window without kept tokens: what is left of it are the memories.  The window's pages go back meanwhile,
    those of the first keys stay."""
    cfg = config([memory(heads=2, dim=16, vdim=16, cap=30.0, mlp=None), pair(size=20, keep=0, decay=(1.0, 0.999, 0.99), mlp=None),
                  pair(size=33, keep=70, r_heads=1, decay=(0.5,), mlp=None)])
    w = make_weights(cfg, 12, lasting=True)
    eng = engine_for(tmp_path, cfg, w, "float32", max_tokens=1024)
    a = tokens_of(cfg, 60, 420)
    b = [(a[0] + 1) % cfg["vocab"]] + a[1:]
    wa, wb = P.forward(w, cfg, a), P.forward(w, cfg, b)
    assert np.abs(wa[-1] - wb[-1]).max() > 1e-3 * np.abs(wa).max()      # far above the tolerance
    rows = Rows("float32")
    for toks, want in ((a, wa), (b, wb)):
        s, at = eng.open(), 0
        for n in (250, 64, 70):
            rows.add(eng.step([(s, toks[at:at + n], list(range(n)))]).double().cpu().numpy(), want[at:at + n], n)
            at += n
        for k in range(at, 420):
            rows.add(eng.step([(s, [toks[k]], [0])]).double().cpu().numpy(), want[k:k + 1], k)
        held = {g.need.keep_first: [i for i, p in enumerate(g.tables[s]) if p >= 0] for g in eng.cache.groups}
        assert held == {0: [6], 70: [0, 1, 6]}
        eng.close(s)
    rows.check()
    assert eng.cache.pages_in_use() == 0


def drawn_config(seed):
    """A configuration drawn from the seed: one to four layers of both types, head counts and sizes that are and are not
    multiples of eight, any grouping of the queries, windows shorter and longer than a page, first keys kept or not,
    feed-forwards of every kind or none, a loop anywhere or none."""
    rng = np.random.default_rng(seed)
    pick = lambda *a: a[int(rng.integers(0, len(a)))]
    layers = []
    for _ in range(int(rng.integers(1, 5))):
        kind = rng.random()
        if kind < 0.2:
            mlp = None
        elif kind < 0.5:
            mlp = dense(pick(16, 48, 37, 128))
        else:
            n = int(rng.integers(1, 9))
            mlp = moe(experts=n, top=int(rng.integers(1, n + 1)), ff=pick(8, 16, 40, 6), limit=pick(0.5, 1.0, 4.0),
                      shared=pick(0, 8, 24, 9), shared_limit=pick(0.5, 2.0))
        if rng.random() < 0.4:
            layers.append(memory(heads=int(rng.integers(1, 5)), dim=pick(8, 16, 24, 48, 5, 64, 128, 100), vdim=pick(8, 16, 32, 20, 3, 64, 130, 256),
                                 cap=pick(2.0, 10.0, 15.0), mlp=mlp))
        else:
            G, rh = int(rng.integers(1, 4)), int(rng.integers(1, 5))
            layers.append(pair(heads=G * int(rng.integers(1, 5)), kv_heads=G, dim=pick(8, 16, 32, 48, 64, 12, 6, 80, 96, 112, 128),
                               scale=pick(0.05, 0.2, 0.5), softcap=pick(None, 5.0, 30.0), size=pick(0, 1, 5, 32, 64, 65, 130),
                               keep=pick(0, 1, 4, 64, 65), r_heads=rh, r_dim=pick(8, 16, 24, 48, 5, 64, 128),
                               r_vdim=pick(8, 16, 32, 20, 3, 64, 128),
                               decay=[pick(0.3, 0.8, 0.95, 0.99, 0.999, 1.0) for _ in range(rh)], mlp=mlp))
    loop = None
    if rng.random() < 0.7:
        start = int(rng.integers(0, len(layers)))
        loop = (start, int(rng.integers(start + 1, len(layers) + 1)), int(rng.integers(1, 4)))
    return config(layers, width=pick(40, 64, 96, 128, 72), vocab=pick(50, 101, 257), eps=pick(1e-5, 1e-6), logit_scale=pick(0.3, 1.0, 2.0), loop=loop)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", [11, 12, 13, 14, 15, 16, 17, 18])
def test_drawn_configurations(tmp_path, seed, dtype):
    """Unequal prompts in one step, then 32 tokens one by one, for configurations nobody chose by hand."""
    cfg = drawn_config(seed)
    w = make_weights(cfg, 100 + seed)
    eng = engine_for(tmp_path, cfg, w, dtype, max_tokens=2048)
    reqs = [tokens_of(cfg, 7 + seed + i, n) for i, n in enumerate((230, 9, 140))]
    want = [P.forward(w, cfg, r) for r in reqs]
    rows = Rows(dtype)
    slots = [eng.open() for _ in reqs]
    cut = [max(1, len(r) - 32) for r in reqs]
    got = eng.step([(s, r[:c], list(range(c))) for s, r, c in zip(slots, reqs, cut)]).double().cpu().numpy()
    o = 0
    for i, c in enumerate(cut):
        rows.add(got[o:o + c], want[i][:c], ("prompt", i))
        o += c
    for k in range(32):
        live = [i for i in range(len(reqs)) if cut[i] + k < len(reqs[i])]
        got = eng.step([(slots[i], [reqs[i][cut[i] + k]], [0]) for i in live]).double().cpu().numpy()
        rows.add(got, np.stack([want[i][cut[i] + k] for i in live]), k)
    rows.check()


@pytest.mark.gpu
def test_a_middle_sized_model_in_bfloat16(tmp_path):
    """Sizes at which products run on the matrix cores in every form: a prompt of more than 512 tokens (the loop's entry as
    partial planes, routers and gates in groups of K), decode steps of one, 20 and 70 sequences."""
    cfg = config([pair(heads=8, kv_heads=2, dim=64, scale=0.125, size=200, keep=5, r_heads=4, r_dim=64, r_vdim=96, decay=(0.5, 0.9, 0.99, 1.0),
                       mlp=dense(1024)),
                  memory(heads=4, dim=64, vdim=128, mlp=moe(experts=8, top=2, ff=64, shared=128))], width=768, vocab=512, loop=(0, 2, 2))
    w = make_weights(cfg, 14)
    eng = engine_for(tmp_path, cfg, w, "bfloat16", max_tokens=8192, max_seqs=72)
    long = tokens_of(cfg, 70, 603)
    want = P.forward(w, cfg, long)
    rows = Rows("bfloat16")
    s = eng.open()
    rows.add(eng.step([(s, long[:600], list(range(600)))]).double().cpu().numpy(), want[:600], "prompt")
    for k in range(600, 603):
        rows.add(eng.step([(s, [long[k]], [0])]).double().cpu().numpy(), want[k:k + 1], k)
    eng.close(s)
    short = [tokens_of(cfg, 80 + i, 12) for i in range(4)]
    wants = [P.forward(w, cfg, t) for t in short]
    for n in (20, 70):
        slots = [eng.open() for _ in range(n)]
        got = eng.step([(s, short[i % 4][:9], [8]) for i, s in enumerate(slots)]).double().cpu().numpy()
        rows.add(got, np.stack([wants[i % 4][8] for i in range(n)]), n)
        for k in (9, 10, 11):
            got = eng.step([(s, [short[i % 4][k]], [0]) for i, s in enumerate(slots)]).double().cpu().numpy()
            rows.add(got, np.stack([wants[i % 4][k] for i in range(n)]), (n, k))
        for s in slots:
            eng.close(s)
    rows.check()


@pytest.mark.gpu
def test_narrow_float_products_in_groups():
    from burn_lm_amd.engine.runtime import Runtime
    rt = Runtime()
    g = torch.Generator().manual_seed(0)
    for M, N, K in ((300, 16, 2048), (65, 8, 512), (130, 64, 1536), (2000, 48, 768), (300, 72, 2048)):
        x, w = (torch.randn(n, K, generator=g).to("cuda", torch.bfloat16) for n in (M, N))
        assert (rt.narrow_groups(M, N, K) > 1) == (N <= 64)
        want = (x.double() @ w.double().t()).cpu().numpy()
        assert rel_err(rt.linear(x, rt.weight(w), out_dtype=torch.float32).double().cpu().numpy(), want) < 1e-5, (M, N, K)


class _Step:
    """The index arrays that the kernels read, for sequences laid out by hand; `padding` tokens of no sequence behind."""

    def __init__(self, news, pasts, slots, dev, padding=0):
        i32 = lambda a: torch.tensor(a, dtype=torch.int32, device=dev)
        self.n_tokens, self.n_seqs = sum(news) + padding, len(news)
        self.positions = i32([p + t for n, p in zip(news, pasts) for t in range(n)] + [0] * padding)
        self.token_seq = i32([b for b, n in enumerate(news) for _ in range(n)] + [-1] * padding)
        self.cu_seqlens = i32([sum(news[:b]) for b in range(len(news) + 1)])
        self.seq_slots = i32(slots)
        self.lens_after = i32([p + n for n, p in zip(news, pasts)])
        self.max_position = max(p + n for n, p in zip(news, pasts)) - 1
        self.max_new, self.max_len_after = max(news), self.max_position + 1
        self.token_source = None


def _attend(form, q, out, step, table, kc, vc, ps, H, G, d, scale, window, keep, cap):
    """The generic kernel, or the matrix-core ones (16 or 32 queries per wavefront in prompts, key ranges whole or cut in
    decoding)."""
    from burn_lm_amd.csrc import ops
    if form == "generic":
        return ops.sink_attn(q, out, None, None, step, table, kc, vc, ps, H, G, d, d, scale, window, keep_first=keep, softcap=cap)
    if step.max_new == 1:
        return ops.attn_decode(q, q.stride(0), out, step.positions, step.token_seq, table, kc, vc, ps, H, G, d, scale, window,
                               n_splits=3 if form == "matrix_2" else 1, keep_first=keep, softcap=cap)
    return ops.attn_prefill_mfma(q, q.stride(0), out, step.positions, step.cu_seqlens, table, kc, vc, ps, step.n_seqs, step.max_new,
                                 H, G, d, scale, window, queries=32 if form == "matrix_2" else 16, keep_first=keep, softcap=cap)


@pytest.mark.gpu
@pytest.mark.parametrize("form,dtype", [("generic", torch.float32), ("generic", torch.bfloat16), ("matrix_1", torch.bfloat16), ("matrix_2", torch.bfloat16)],
                         ids=["generic-float32", "generic-bfloat16", "matrix_1", "matrix_2"])
@pytest.mark.parametrize("decode", [False, True], ids=["prompt", "decoding"])
@pytest.mark.parametrize("window,keep", [(100, 4), (64, 64), (65, 70), (1, 1), (37, 0), (0, 0), (300, 129)])
def test_keys_that_stand_out_at_every_edge(form, dtype, decode, window, keep):
    """One key's capped score towers over all others: where it is visible, the result is that key's value, and where it
    is not, the others' (zero).  Keys at both edges of the window, at the last of the first keys and the next one, at page
    borders and far back among hundreds; a sequence's pages lie scattered, and pages that no visible key lies in hold
    keys that would win if they were read."""
    dev = "cuda"
    H, G, d, ps, n = 4, 2, 32, 64, 420
    pages = [7, 2, 9, 0, 8, 3, 5]
    table = torch.tensor([pages + [-1] * 2], dtype=torch.int32, device=dev)
    p = n - 1
    edges = {p, p - 1, max(0, p - window + 1), max(0, p - window), keep - 1, keep, 0, 1, 63, 64, 127, 128, 191, 192, p // 2}
    for j in sorted(e for e in edges if 0 <= e <= p):
        g = torch.Generator().manual_seed(j)
        kc = torch.randn(10, G, ps, d, generator=g) * 0.02
        vc = torch.zeros(10, G, d, ps)
        kc[[1, 4, 6]] = 50.0            # of no sequence
        vc[[1, 4, 6]] = 1e3
        at = n                           # what lies behind the sequence in its last page
        kc[pages[at // ps], :, at % ps:] = 50.0
        vc[pages[at // ps], :, :, at % ps:] = 1e3
        kc[pages[j // ps], :, j % ps, :] = 1.0
        vc[pages[j // ps], :, :, j % ps] = 3.0
        kd, vd = kc.to(dev, dtype).contiguous(), vc.to(dev, dtype).contiguous()
        step = _Step([1], [p], [0], dev) if decode else _Step([n], [0], [0], dev)
        q = torch.full((step.n_tokens, H * d), 2.0, device=dev, dtype=dtype)
        out = torch.empty(step.n_tokens, H * d, dtype=dtype, device=dev)
        _attend(form, q, out, step, table, kd, vd, ps, H, G, d, 0.5, window, keep, 25.0)      # 32 before the cap, 21 behind it
        out = out.float().cpu().view(step.n_tokens, H, d)
        want = torch.tensor([3.0 if P.visible(pos, j, window, keep) else 0.0 for pos in ([p] if decode else range(n))])
        wrong = (out - want.view(-1, 1, 1)).abs().amax((1, 2)) > 2e-3
        assert not wrong.any(), (j, wrong.nonzero().view(-1).tolist()[:5])


@pytest.mark.gpu
@pytest.mark.parametrize("form,dtype", [("generic", torch.float32), ("matrix_1", torch.bfloat16), ("matrix_2", torch.bfloat16)],
                         ids=["generic", "matrix_1", "matrix_2"])
@pytest.mark.parametrize("d", [16, 32, 48, 64, 80, 96, 112, 128])
@pytest.mark.parametrize("window,keep,cap", [(50, 5, 8.0), (0, 0, 3.0), (90, 70, 0.0)])
def test_attention_kernels_against_plain_softmax(form, dtype, d, window, keep, cap):
    """Random keys and queries of two sequences, one of them with a past, prompts and single tokens."""
    if form == "matrix_2" and d % 32:
        pytest.skip("no form with 32 queries for this head size")
    dev = "cuda"
    H, G, ps = 6, 2, 64
    rng = np.random.default_rng(d)
    bf = lambda a: torch.from_numpy(a).to(dtype)
    tables = torch.tensor([[3, 0, 6, 7], [5, 1, 4, 2]], dtype=torch.int32, device=dev)
    K, V = bf(rng.standard_normal((8, G, ps, d))), bf(rng.standard_normal((8, G, d, ps)))
    for news, pasts in (([150, 33], [0, 190]), ([1, 1], [149, 222])):
        step = _Step(news, pasts, [0, 1], dev)
        q = bf(rng.standard_normal((sum(news), H * d)))
        out = torch.empty(sum(news), H * d, dtype=dtype, device=dev)
        _attend(form, q.to(dev), out, step, tables, K.to(dev), V.to(dev), ps, H, G, d, 0.9 / math.sqrt(d), window, keep, cap)
        got, row = out.double().cpu().numpy().reshape(-1, H, d), 0
        for b, (n, past) in enumerate(zip(news, pasts)):
            pg = tables[b].cpu().tolist()
            ks = np.concatenate([K[x].double().numpy() for x in pg], axis=1)                       # [G, keys, d]
            vs = np.concatenate([V[x].double().numpy() for x in pg], axis=2)                       # [G, d, keys]
            for t in range(n):
                pos = past + t
                see = [j for j in range(pos + 1) if P.visible(pos, j, window, keep)]
                for hd in range(H):
                    s = ks[hd // (H // G)][see] @ q[row, hd * d:(hd + 1) * d].double().numpy() * (0.9 / math.sqrt(d))
                    s = cap * np.tanh(s / cap) if cap else s
                    e = np.exp(s - s.max())
                    want = vs[hd // (H // G)][:, see] @ e / e.sum()
                    assert np.abs(got[row, hd] - want).max() < (1e-5 if dtype == torch.float32 else 3e-2), (b, t, hd)
                row += 1


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["float32", "bfloat16"])
def test_queries_and_keys_are_normed_with_their_biases_and_values_are_not(dtype):
    from burn_lm_amd.csrc import ops
    dev = "cuda"
    H, G, dk, ps, eps = 3, 2, 70, 64, 0.1                        # an eps that shows
    rng = np.random.default_rng(3)
    news, pasts, slots = [3, 1], [62, 130], [0, 1]               # one sequence crosses a page border
    step = _Step(news, pasts, slots, dev, padding=2)
    T = step.n_tokens
    rows = torch.from_numpy(rng.standard_normal((T, (H + G) * dk + 6))).to(dtype)     # six columns nobody may touch
    tables = torch.tensor([[4, 1, -1], [0, 5, 2]], dtype=torch.int32, device=dev)
    bias = rng.standard_normal((H + G) * dk).astype(np.float32)
    kc = torch.zeros(6, G, ps, dk, dtype=dtype, device=dev)
    vc = torch.zeros(6, G, dk, ps, dtype=dtype, device=dev)
    qkv = rows.to(dev).clone()
    ops.qkv_prepare(qkv, torch.from_numpy(bias).to(dev), None, 0, step, tables, kc, vc, ps, H, G, dk, dk, values_are_keys=True,
                    unit_norm_eps=eps)
    x = rows.double().numpy()
    x[:, :(H + G) * dk] += bias
    q, k = x[:, :H * dk].reshape(T, H, dk), x[:, H * dk:(H + G) * dk].reshape(T, G, dk)
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    assert np.abs(qkv[:4, :H * dk].double().cpu().numpy().reshape(4, H, dk) - P.unit_rms(q, eps)[:4]).max() < tol
    assert torch.equal(qkv[:, H * dk:].cpu(), rows[:, H * dk:]) and torch.equal(qkv[4:].cpu(), rows[4:])
    for t, (b, p) in enumerate([(0, 62), (0, 63), (0, 64), (1, 130)]):
        page = int(tables[b, p // ps])
        assert np.abs(kc[page, :, p % ps].double().cpu().numpy() - P.unit_rms(k, eps)[t]).max() < tol
        assert np.abs(vc[page, :, :, p % ps].double().cpu().numpy() - k[t]).max() < tol
    assert float(kc[[0, 3, 5]].float().abs().sum()) == 0 and float(vc[[0, 3, 5]].float().abs().sum()) == 0


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["float32", "bfloat16"])
@pytest.mark.parametrize("H,dk,dv", [(3, 12, 20), (2, 128, 256), (3, 70, 33), (1, 64, 129), (1, 136, 40), (1, 5, 3)],
                         ids=["small", "wide", "odd", "one_column_more", "more_than_128_keys", "tiny"])
@pytest.mark.parametrize("form", ["step", "chunks"])
@pytest.mark.parametrize("news,slots", [([300, 40, 1], [2, 0, 3]), ([64, 65, 63, 128, 129, 1, 8, 2], [5, 0, 3, 8, 2, 7, 4, 6])],
                         ids=["long", "chunk_edges"])
def test_matrix_memory_kernels_against_the_plain_function(dtype, H, dk, dv, form, news, slots):
    """Sequences of several lengths in one step, from zero states and from others; heads whose gates forget at once,
    slowly and hardly; a state slot that is not in the step stays as it was; padding rows become zero."""
    from burn_lm_amd.csrc import ops
    dev = "cuda"
    ops.matrix_memory_init(dev)
    if form == "chunks" and not ops.matrix_memory_chunks_supported(dk, dv, dtype):
        pytest.skip("heads of this size are not run in chunks")
    if form == "step":
        news = [min(n, 70) for n in news]
    rng = np.random.default_rng(4)
    bf = lambda a: torch.from_numpy(np.asarray(a, dtype=np.float32)).to(dtype).double().numpy()
    f32 = lambda a: torch.tensor(np.asarray(a), dtype=torch.float32, device=dev)
    norm_w, cap = rng.uniform(0.5, 1.5, H * dv), 9.0
    n_slots = max(slots) + 1
    S0, n0, m0 = rng.standard_normal((n_slots, H, dk, dv)), rng.standard_normal((n_slots, H, dk)), rng.uniform(-2, 4, (n_slots, H))
    S0[slots[0]], n0[slots[0]], m0[slots[0]] = 0.0, 0.0, 0.0
    pad = 3
    T = sum(news) + pad
    proj = bf(rng.standard_normal((T, 2 * H * dk + 2 * H * dv + 5)))
    z = rng.standard_normal((T, 2 * H + 3)) * 3
    bi, bfg = rng.standard_normal(H), np.array(([-6.0, 3.0, 9.0] * 3)[:H])
    z, bi32, bf32 = f32(z), f32(bi), f32(bfg)
    zd = z.double().cpu().numpy()
    li = cap * np.tanh((zd[:, :H] + bi32.double().cpu().numpy()) / cap)
    lf = P.log_sigmoid(cap * np.tanh((zd[:, H:2 * H] + bf32.double().cpu().numpy()) / cap))
    want, at = [], 0
    for n, slot in zip(news, slots):
        q, k, v, gl, _ = np.split(proj[at:at + n], [H * dk, 2 * H * dk, 2 * H * dk + H * dv, 2 * H * (dk + dv)], axis=1)
        o, st = P.matrix_memory(q.reshape(n, H, dk) * dk ** -0.5, k.reshape(n, H, dk), v.reshape(n, H, dv), li[at:at + n], lf[at:at + n],
                                (S0[slot], n0[slot], m0[slot]))
        want.append((P.unit_rms(o, 1e-5).reshape(n, H * dv) * norm_w * P.sigmoid(gl), st))
        at += n
    step = _Step(news, [0, 77, 500, 3, 64, 640, 1, 0][:len(news)], slots, dev, padding=pad)
    state = (f32(S0), f32(n0), f32(m0))
    rows = torch.from_numpy(proj).to(dev, dtype)
    if form == "step" and dtype == torch.bfloat16 and len(news) == 3:
        rows = rows.float()      # what a step of few tokens hands over
    out = torch.full((T, H * dv), 7.0, dtype=dtype, device=dev)
    ops.matrix_memory(rows, z, bi32, bf32, cap, dk ** -0.5, f32(norm_w), 1e-5, state, out, step, H, dk, dv, form == "chunks")
    # (a head of three lanes whose numerator nearly cancels is brought back to unit size with its roundings)
    tol, at = ((2e-5 if dv > 3 else 1e-4) if dtype == torch.float32 else 2e-2), 0
    for (o, st), n, slot in zip(want, news, slots):
        assert rel_err(out[at:at + n].double().cpu().numpy(), o) < tol, slot
        for got, x in zip(state, st):
            assert rel_err(got[slot].double().cpu().numpy(), x) < 2e-5, slot
        at += n
    assert float(out[at:].float().abs().sum()) == 0
    for got, x in zip(state, (S0, n0, m0)):
        assert torch.equal(got[1].cpu(), f32(x)[1].cpu())
    assert int(ops.arrival_counters(torch.device("cuda:0")).abs().sum()) == 0


@pytest.mark.gpu
@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16], ids=["float32", "bfloat16"])
@pytest.mark.parametrize("D", [24, 18, 1000, 2048, 4100, 9000])
def test_joining_kernel_against_the_plain_norms(act, D):
    """Results with and without norms of their own, a norm behind their sum, a residual that grows or starts anew, a vector,
    partial planes, listed rows, outputs inside wider rows and outputs that are not normed."""
    from burn_lm_amd.csrc import ops
    dev, T = "cuda", 5
    rng = np.random.default_rng(D)
    f32 = lambda a: torch.tensor(np.asarray(a), dtype=torch.float32, device=dev)
    dbl = lambda t: t.double().cpu().numpy()
    h0, a, b = rng.standard_normal((T, D)) * 3, rng.standard_normal((3, T, D)), f32(rng.standard_normal((T, D))).to(act)
    ga, gb, gp, go, vec = (f32(rng.uniform(0.5, 1.5, D)) for _ in range(5))
    tol = 2e-5 if act == torch.float32 else 1e-2
    two = 0.5 * P.unit_rms(a.sum(0), 1e-2) * dbl(ga) + 0.25 * P.unit_rms(dbl(b), 1e-3) * dbl(gb)
    terms2 = [(f32(a), 0.5, ga, 1e-2), (b, 0.25, gb, 1e-3)]
    cases = [(terms2, two), ([(f32(a), 2.0, None, 0.0)], 2 * a.sum(0)), ([(b, 1.0, None, 0.0)], dbl(b)),
             ([(f32(a[:1]), 1.0, ga, 1e-2), (b, -1.0, None, 0.0)], P.unit_rms(a[0], 1e-2) * dbl(ga) - dbl(b))]
    for terms, y in cases:
        for post in (None, (gp, 1e-4)):
            for fresh, v in ((False, None), (True, vec)):
                yy = y if post is None else P.unit_rms(y, 1e-4) * dbl(gp)
                want = (0.0 if fresh else dbl(f32(h0))) + (0.0 if v is None else dbl(v)) + yy
                h = f32(h0)
                wide = torch.full((T, 2 * D), 5.0, dtype=act, device=dev)
                ops.post_norm(h, terms, post=post, fresh=fresh, vec=v, gamma=go, eps=1e-5, out=wide[:, D:])
                assert rel_err(dbl(h), want) < 1e-5
                assert rel_err(dbl(wide[:, D:]), P.unit_rms(want, 1e-5) * dbl(go)) < tol and float((wide[:, :D] - 5.0).abs().sum()) == 0
                h = f32(h0)                               # listed rows, nothing written back
                rows = torch.tensor([3, 0, 3], dtype=torch.int32, device=dev)
                out = torch.empty(3, D, dtype=act, device=dev)
                ops.post_norm(h, terms, post=post, fresh=fresh, vec=v, write_h=False, gamma=go, eps=1e-5, out=out, rows=rows)
                assert torch.equal(h, f32(h0)) and rel_err(dbl(out), (P.unit_rms(want, 1e-5) * dbl(go))[[3, 0, 3]]) < tol
                out = torch.empty(T, D, dtype=act, device=dev)      # the rows as they are
                ops.post_norm(h, terms, post=post, fresh=fresh, vec=v, write_h=False, out=out)
                assert torch.equal(h, f32(h0)) and rel_err(dbl(out), want) < tol
                ops.post_norm(h, terms, post=post, fresh=fresh, vec=v)   # the residual alone
                assert rel_err(dbl(h), want) < 1e-5


@pytest.mark.gpu
def test_routing_gating_and_embedding_kernels_against_the_plain_functions():
    from burn_lm_amd.csrc import ops
    dev = "cuda"
    rng = np.random.default_rng(2)
    f32 = lambda a: torch.tensor(np.asarray(a), dtype=torch.float32, device=dev)
    for E, top in ((5, 2), (1, 1), (12, 1), (7, 7), (100, 9)):
        T = 257
        logits = rng.standard_normal((T, E + 3)) * 2              # three columns of padding behind the logits
        chosen, wts = P.route({"m.router": np.eye(E)}, "m.", dict(router=dict(top=top)), logits[:, :E].astype(np.float32).astype(np.float64))
        want = np.zeros((T, E + 1))
        np.put_along_axis(want, chosen, wts, axis=1)
        got = ops.moe_route_grouped(f32(logits), None, E, 0, 1, 1, top, torch.empty(T, E + 1, dtype=torch.float32, device=dev),
                                    score="sigmoid", renormalize=False)
        assert np.abs(got.double().cpu().numpy() - want).max() < 1e-5, (E, top)
    # the weight on the input meets the limits; a shared expert with its own limit behind the others or none; inner sizes
    # that are and are not multiples of eight
    for dtype in (torch.float32, torch.bfloat16):
        for E, ff, s in ((3, 16, 8), (3, 16, 0), (2, 5, 7), (1, 8, 24)):
            T, I = 9, E * ff + s
            gu = torch.from_numpy(rng.standard_normal((T, 2 * I)) * 3).to(dev, dtype)
            w = f32(rng.uniform(0, 1, (T, E + 1)) * (rng.random((T, E + 1)) < 0.6))
            got = ops.moe_gate_clamped(gu, w, torch.empty(T, I, dtype=dtype, device=dev), E, ff, 1.1, 1.702, 0.4 if s else None)
            x, wd = gu.double().cpu().numpy(), w.double().cpu().numpy()
            ws = np.concatenate([np.repeat(wd[:, :E], ff, axis=1), np.ones((T, s))], axis=1)
            lim = np.concatenate([np.full(E * ff, 1.1), np.full(s, 0.4)])
            g, u = np.minimum(ws * x[:, :I], lim), np.clip(ws * x[:, I:], -lim, lim)
            assert rel_err(got.double().cpu().numpy(), g * P.sigmoid(1.702 * g) * (u + 1)) < (1e-5 if dtype == torch.float32 else 1e-2)
        for n in (64, 37):
            z = torch.from_numpy(rng.standard_normal((3, n))).to(dev, dtype)
            want = np.maximum(z.double().cpu().numpy(), 0) ** 2
            assert rel_err(ops.relu2(z, z).double().cpu().numpy(), want) < (1e-6 if dtype == torch.float32 else 1e-2)
    # position vectors at the first positions and a million tokens on (a 32-bit angle would be off by a tenth there), an
    # odd width, rows copied into wider ones, tokens that only the device knows
    for D in (48, 37):
        table = torch.from_numpy(rng.standard_normal((20, D))).to(dev, torch.bfloat16)
        ids, positions = [3, 19, 0, 7, 7], [0, 1, 77, 4096, 1000003]
        turns = (10000.0 ** (torch.arange((D + 1) // 2, dtype=torch.float64) * (-2.0 / D)) / (2 * math.pi)).to(dev)
        i32 = lambda a: torch.tensor(a, dtype=torch.int32, device=dev)
        want = table.double().cpu().numpy()[ids] + P.position_vectors(positions, D)
        h, wide = torch.empty(5, D, dtype=torch.float32, device=dev), torch.zeros(5, 2 * D, dtype=torch.bfloat16, device=dev)
        picked = i32([9, 7])
        cell = torch.tensor([picked.data_ptr()], dtype=torch.int64, device=dev)
        ops.embed_positions(table, i32([3, 19, 0, 0, 0]), i32(positions), turns, h, copy=wide[:, D:], source=(i32([-1, -1, -1, 1, 1]), cell))
        assert np.abs(h.double().cpu().numpy() - want).max() < 1e-6
        assert torch.equal(wide[:, D:], h.bfloat16()) and float(wide[:, :D].abs().sum()) == 0
        ops.embed_positions(table, i32(ids), i32(positions), None, h)
        assert torch.equal(h, table[i32(ids).long()].float())


@pytest.mark.gpu
def test_greedy_generation_through_the_server(tmp_path):
    from burn_lm_amd.server import InferenceServer
    cfg = MIXED
    w = make_weights(cfg, 8)
    folder = write_folder(tmp_path, cfg, w)
    prompts = [tokens_of(cfg, 40 + i, n) for i, n in enumerate((5, 11, 2, 70))]

    def plain_greedy(p, n):
        toks = list(p)
        for _ in range(n):
            toks.append(int(np.argmax(P.forward(w, cfg, toks)[-1])))
        return toks[len(p):]

    want = [plain_greedy(p, 6) for p in prompts]
    server = InferenceServer(folder, dtype="float32", batch_size=3)       # two batches: slots are used again
    server.config.update(max_seq_len=256, sample_len=6, temperature=0.0)
    results, _ = server.generate(prompts, stop_ids=[])
    assert [r.tokens for r in results] == want
    server.unload()
