"""The Netanex design in the engine against the plain implementation of tests/plain_netanex.py.

The configurations and weights are made here.  The CPU tests cover the configuration reader, the plan, the random
checkpoint and the plain implementation's own consistency on cases worked by hand; the GPU tests run the engine's step
function, cache, scheduler and kernels: each mixer and the feed-forward alone, layers that share tensors, whole prompts
against token-by-token decoding, prompts in portions, unequal batches, slots and pages used again, keys that stand out at
the edges of the window, at page borders, among the first tokens and far back (in prompts and in decoding), sinks that
matter, long decoding through recorded graphs, odd sizes, configurations drawn from seeds, and greedy generation through
the server."""
import json
import math

import numpy as np
import pytest
import torch

import plain_netanex as P
from helpers import rel_err

TOL = {"float32": 2e-5, "bfloat16": 6e-2}


class Rows:
    """Collects rows of logits beside what they should be; every row within the tolerance."""

    def __init__(self, dtype):
        self.dtype, self.errs = dtype, []

    def add(self, got, want, note=None):
        got, want = np.atleast_2d(np.asarray(got, dtype=np.float64)), np.atleast_2d(want)
        assert got.shape == want.shape and np.isfinite(got).all(), note
        scale = max(1e-30, np.abs(want).max())
        self.errs += [(float(np.abs(g - x).max() / scale), note) for g, x in zip(got, want)]

    def check(self):
        bad = [e for e in self.errs if e[0] > TOL[self.dtype]]
        assert not bad, (len(bad), len(self.errs), sorted(bad, key=lambda e: -e[0])[:5])


# ---- configurations and weights of the tests --------------------------------------------------
def moe(experts=5, top=2, ff=24):
    return dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top))


def pick_mlp(mlp):
    return moe() if mlp == "default" else mlp


def maps(heads=4, kv_heads=2, dim=16, vdim=32, scale=0.3, diff=0.4, temp=(0.5, 10), mlp="default"):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, diff=diff)
    if temp:
        m["q_temp"] = dict(coef=temp[0], every=temp[1])
    return dict(type="attention", mixer=m, mlp=pick_mlp(mlp))


def latent(heads=4, dim=24, rot_dim=16, vdim=20, kv_rank=64, scale=0.2, size=40, base=1000.0, yarn=(4.0, 64, 8.0, 1.0), mlp="default"):
    m = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, scale=scale,
             rot=dict(base=base, dims=rot_dim, scaling=dict(zip(("factor", "original", "fast", "slow"), yarn)) if yarn else None))
    if size:
        m["mask"] = dict(size=size)
    return dict(type="latent_attention", mixer=m, mlp=pick_mlp(mlp))


def gated(heads=4, kv_heads=2, dim=32, vdim=32, scale=0.25, mlp="default"):
    return dict(type="attention_2", mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale), mlp=pick_mlp(mlp))


def again(layers, j):
    return dict(layers[j], weights_of=j)


def config(layers, width=48, vocab=101, eps=1e-5):
    return dict(architecture="Netanex", layers=layers, norm=dict(eps=eps), vocab=vocab, width=width)


# layers that differ from each other in every size, sizes for every kernel (values of the keys' size and others, latents
# with and without a matrix-core form), layers without a feed-forward, layers that take others' tensors, in another order
_MIXED = [latent(size=50),
          gated(),
          maps(mlp=moe(experts=4, top=1, ff=40)),
          gated(heads=6, kv_heads=1, dim=24, vdim=40, scale=0.4, mlp=None),
          latent(heads=3, dim=16, rot_dim=8, vdim=32, kv_rank=40, size=0, yarn=None, mlp=moe(experts=7, top=3, ff=16)),
          maps(heads=3, kv_heads=3, dim=24, vdim=16, diff=0.8, temp=None, mlp=None)]
MIXED = config(_MIXED + [again(_MIXED, 2), again(_MIXED, 0), again(_MIXED, 1), again(_MIXED, 5)])
# sizes that are no multiples of eight, one head, a window of one, every expert chosen, a single expert, a temperature that
# grows with every token
_ODD = [maps(heads=3, kv_heads=1, dim=5, vdim=7, scale=0.7, temp=(0.1, 1), mlp=moe(experts=3, top=3, ff=5)),
        latent(heads=1, dim=9, rot_dim=2, vdim=11, kv_rank=13, size=1, yarn=(2.0, 16, 4.0, 2.0), mlp=moe(experts=1, top=1, ff=12)),
        gated(heads=5, kv_heads=5, dim=6, vdim=9, mlp=moe(experts=7, top=4, ff=3)),
        latent(heads=5, dim=6, rot_dim=6, vdim=3, kv_rank=21, size=7, mlp=None)]
ODD = config(_ODD + [again(_ODD, 3), again(_ODD, 0)], width=36, vocab=53, eps=1e-6)


def make_weights(cfg, seed):
    """float64 arrays that are exact in bfloat16.  Sublayers join the residual with a gain of about 0.4: with one of one, a
    chain of a dozen random layers multiplies a rounding so much that bfloat16 rows have little in common with exact ones."""
    g = np.random.default_rng(seed)
    D = cfg["width"]
    bf = lambda a: torch.from_numpy(np.asarray(a, dtype=np.float32)).bfloat16().double().numpy()
    mat = lambda o, i, s=1.0: bf(g.standard_normal((o, i)) * s / math.sqrt(i))
    near = lambda n, c: bf(c + 0.15 * g.standard_normal(n))
    w = {"embed": bf(g.standard_normal((cfg["vocab"], D))), "embed.norm": near(D, 0), "final.norm": near(D, 0)}
    for i, L in enumerate(cfg["layers"]):
        if L.get("weights_of") is not None:
            continue
        l, m, f = f"l{i}.", L["mixer"], L["mlp"]
        w[l + "norm1"], w[l + "norm1b"] = near(D, 0), near(D, -0.6)
        p, H, d, dv = l + "mix.", m["heads"], m["dim"], m["vdim"]
        w[p + "o"] = mat(D, H * dv)
        if L["type"] == "latent_attention":
            R, dr = m["kv_rank"], m["rot_dim"]
            w.update({p + "q": mat(H * (d + dr), D, 1.5), p + "dkv": mat(R + dr, D), p + "dkv.norm": near(R, 1), p + "uk": mat(H * d, R),
                      p + "uv": mat(H * dv, R), p + "sink": bf(1.5 * g.standard_normal(H)), p + "g": mat(H * dv, D)})
        else:
            n = 2 if L["type"] == "attention" else 1
            for r, rows in (("q", H * n * d), ("k", m["kv_heads"] * n * d), ("v", m["kv_heads"] * dv)):
                w[p + r], w[p + r + ".b"] = mat(rows, D), bf(0.5 * g.standard_normal(rows))
            if n == 2:
                w[p + "q.norm"], w[p + "k.norm"], w[p + "o.b"] = near(d, 1), near(d, 1), bf(0.3 * g.standard_normal(D))
                w.update({p + r: bf(0.7 * d ** -0.25 * g.standard_normal(d)) for r in ("lq1", "lk1", "lq2", "lk2")})
            else:
                w[p + "q.norm"], w[p + "k.norm"], w[p + "g"] = near(H * d, 1), near(m["kv_heads"] * d, 1), mat(H, D)
        if f is None:
            continue
        w[l + "norm2"], w[l + "norm2b"] = near(D, 0), near(D, -0.6)
        p, E, top, ff = l + "mlp.", f["router"]["experts"], f["router"]["top"], f["expert"]["ff"]
        w[p + "table"] = np.stack([g.permutation(E)[:top] for _ in range(cfg["vocab"])]).astype(np.int32)
        for e in range(E):
            e = f"{p}e{e}."
            w[e + "gate"], w[e + "up"], w[e + "down"] = mat(ff, D), mat(ff, D), mat(D, ff)
    return w


def write_folder(path, cfg, w):
    from burn_lm_amd.weights import safetensors_io as st
    with open(path / "config.json", "w") as f:
        json.dump(cfg, f)
    kept = lambda v: torch.from_numpy(v) if v.dtype == np.int32 else torch.from_numpy(v).bfloat16()
    st.write_file(str(path / "model.safetensors"), ((k, kept(v)) for k, v in w.items()))
    return str(path)


def tokens_of(cfg, seed, n):
    return [int(x) for x in np.random.default_rng(seed).integers(0, cfg["vocab"], n)]


# ---- CPU: configuration, plan, random checkpoint, plain implementation ----------------------------
def test_config_is_read_and_refused_by_key():
    from burn_lm_amd import registry
    from burn_lm_amd.errors import ConfigError
    import burn_lm_amd.models  # noqa: F401
    arch = registry.architecture_of(MIXED)
    assert arch.name == "Netanex"
    cfg = arch.read_config(MIXED)
    assert cfg.layers[3].mlp is None and cfg.layers[4].mixer.window == 0 and cfg.layers[4].mixer.yarn is None
    assert cfg.layers[0].mixer.yarn == (4.0, 64.0, 8.0, 1.0) and cfg.layers[2].mixer.growth == (0.5, 10) and cfg.layers[5].mixer.growth is None
    assert [layer.owner for layer in cfg.layers] == [0, 1, 2, 3, 4, 5, 2, 0, 1, 5]
    for path, value, word in ((("layers", 1, "mixer", "vdim"), None, "vdim"), (("width",), "48", "width"),
                              (("layers", 0, "type"), "attention_3", "type"), (("norm",), {}, "eps"),
                              (("layers", 1, "mixer", "kv_heads"), 3, "kv_heads"), (("layers", 5, "mixer", "diff"), None, "diff"),
                              (("layers", 0, "mixer", "mask"), dict(size=0), "size"), (("layers", 0, "mixer", "rot", "dims"), 8, "dims"),
                              (("layers", 4, "mixer", "rot", "base"), -1.0, "base"),
                              (("layers", 4, "mixer", "rot", "scaling"), dict(factor=2.0), "original"),
                              (("layers", 5, "mixer", "q_temp"), dict(coef=0.5), "every"),
                              (("layers", 3, "mlp"), dict(kind="dense", ff=4), "kind"),
                              (("layers", 4, "mlp", "router", "top"), 8, "top"),
                              (("layers", 6, "weights_of"), 6, "weights_of"), (("layers", 6, "weights_of"), 1, "weights_of"),
                              (("layers", 6, "mixer", "scale"), 0.9, "differs")):
        bad = json.loads(json.dumps(MIXED))
        at = bad
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = value
        with pytest.raises(ConfigError, match=word):
            arch.read_config(bad)
    # a layer may take the tensors of one that takes another's
    chain = json.loads(json.dumps(MIXED))
    chain["layers"].append(dict(chain["layers"][6], weights_of=6))
    assert arch.read_config(chain).layers[-1].owner == 2 and P.owner(chain, 10) == 2


def test_plan_asks_for_the_checkpoints_tensors():
    from burn_lm_amd import registry
    import burn_lm_amd.parts  # noqa: F401
    from burn_lm_amd.engine.model import Model
    from burn_lm_amd.parts.base import KVNeed
    for cfg_dict in (MIXED, ODD):
        w = make_weights(cfg_dict, 0)
        arch = registry.architecture_of(cfg_dict)
        cfg = arch.read_config(cfg_dict)
        model = Model(arch.plan(cfg, {k: v.shape for k, v in w.items()}))
        assert {k: tuple(s.shape) for k, s in model.tensor_specs().items()} == {k: tuple(v.shape) for k, v in w.items()}
        assert {k: tuple(v[0]) for k, v in arch.checkpoint_tensors(cfg).items()} == {k: tuple(v.shape) for k, v in w.items()}
        assert len(model.plan.layers) == sum(1 for L in cfg_dict["layers"] if L.get("weights_of") is None)
        assert len(model.plan.order) == len(cfg_dict["layers"]) and all(p.reads_cache_of is None for p in model.plan.order)
        assert all(part.graph_safe for part in model.all_parts())
    needs = model.cache_needs()
    assert needs[0] == needs[5] == KVNeed(1, 10, 0, value_dim=7)
    assert needs[1] == KVNeed(1, 15, 1, no_values=True) and needs[3] == KVNeed(1, 27, 7, no_values=True)


def test_random_folder_loads_into_the_plain_implementation(tmp_path):
    import burn_lm_amd
    from burn_lm_amd.weights import safetensors_io as st
    folder = burn_lm_amd.write_random_model(str(tmp_path), ODD, seed=5)
    w = {n: f.tensor(n) for n, f in st.open_folder(folder).items()}
    w = {n: t.numpy() if t.dtype == torch.int32 else t.double().numpy() for n, t in w.items()}
    for i, (E, top) in {0: (3, 3), 1: (1, 1), 2: (7, 4)}.items():
        table = w[f"l{i}.mlp.table"]
        assert table.shape == (53, top) and table.min() >= 0 and table.max() < E and all(len(set(r)) == top for r in table.tolist())
    assert len({tuple(r) for r in w["l2.mlp.table"].tolist()}) > 20
    logits = P.forward(w, ODD, tokens_of(ODD, 0, 9))
    assert logits.shape == (9, 53) and np.isfinite(logits).all() and logits.std() > 0.05


def test_plain_mechanisms_on_cases_worked_by_hand():
    # a sink and one added to the denominator take their share and give nothing
    assert np.allclose(P.weights_over(np.array([0.0, math.log(2.0)]), math.log(3.0)), [1 / 6, 2 / 6])
    assert np.allclose(P.weights_over(np.array([700.0, -700.0]), 0.0), [1.0, 0.0]) and np.allclose(P.weights_over(np.zeros(3), 0.0), 0.25)
    # queries grow by steps of the logarithm
    assert [P.query_factor(p, 2.0, 3) for p in (0, 1, 2, 4, 5)] == [1.0, 1.0, 1 + 2 * math.log(2), 1 + 2 * math.log(2), 1 + 2 * math.log(3)]
    # equal scores: both maps average, so the difference is (1 - lambda) times the mean, brought to unit size by the norm
    W = {"a.q": np.zeros((4, 1)), "a.q.b": np.zeros(4), "a.k": np.zeros((4, 1)), "a.k.b": np.ones(4), "a.v": np.array([[1.0], [0.0]]),
         "a.v.b": np.array([0.0, 1.0]), "a.q.norm": np.ones(2), "a.k.norm": np.ones(2), "a.o": np.eye(2), "a.o.b": np.array([0.0, 10.0]),
         "a.lq1": np.array([1.0, 0.0]), "a.lk1": np.array([math.log(2.0), 5.0]), "a.lq2": np.zeros(2), "a.lk2": np.ones(2)}
    assert math.isclose(P.two_map_lambda(W, "a.", 0.5), 2.0 - 1.0 + 0.5)
    m = dict(heads=1, kv_heads=1, dim=2, vdim=2, scale=1.0, diff=0.5)
    got = P.differential_attention(W, "a.", m, np.array([[2.0], [4.0]]), 1e-12)
    u = np.array([3.0, 1.0])
    assert np.allclose(got[1], -u / math.sqrt(5.0) * 0.5 + [0, 10])
    # one map that picks a key, subtracted from one that averages
    W.update({"a.q.b": np.array([0.0, 0.0, 30.0, 0.0]), "a.k": np.array([[0.0], [0.0], [1.0], [0.0]]), "a.k.b": np.array([1.0, 1.0, -3.0, 0.0])})
    m["scale"] = 30.0
    got = P.differential_attention(W, "a.", m, np.array([[2.0], [4.0]]), 1e-12)
    u = u - 1.5 * np.array([4.0, 1.0])
    assert np.allclose(got[1], u / math.sqrt((u * u).mean()) * 0.5 + [0, 10], atol=1e-6)
    # rotation: fast pairs stay, slow ones are divided, both are lengthened
    rot = dict(dims=8, base=10000.0, scaling=dict(factor=4.0, original=1000, fast=20.0, slow=1.0))
    f, a = P.turning(rot)
    assert math.isclose(a, 1 + 0.1 * math.log(4.0)) and math.isclose(f[0], 1.0) and math.isclose(f[3], 0.001 / 4)
    assert f[1] < 0.1 and f[1] > 0.1 / 4                     # pairs 0.9 .. 2.2 of the ramp (0 to 3)
    x = P.turn(np.tile(np.arange(1.0, 9.0), (3, 1)), rot)
    assert math.isclose(x[2, 0], a * (math.cos(2) - 5 * math.sin(2))) and math.isclose(x[2, 4], a * (5 * math.cos(2) + math.sin(2)))
    assert [P.visible(5, j, 3) for j in range(7)] == [False, False, False, True, True, True, False] and P.visible(5, 0, 0)
    # experts: the table's rows, equally weighted
    W = {"m.table": np.array([[1, 0], [2, 1]], dtype=np.int32)}
    for e in range(3):
        W[f"m.e{e}.gate"], W[f"m.e{e}.up"], W[f"m.e{e}.down"] = np.array([[1.0]]), np.array([[2.0]]), np.array([[10.0 ** e]])
    z = P.silu(3.0) * 6.0
    assert np.allclose(P.table_experts(W, "m.", np.array([[3.0], [3.0]]), [0, 1]), [[5.5 * z], [55 * z]])


def test_entry_points_take_what_their_signatures_say():
    """Number and kind of every argument in the library's sources against what is passed to it: a pointer that goes through as
    a 32-bit integer would be cut short."""
    import ctypes
    import glob
    import os
    import re
    from burn_lm_amd.csrc import ops
    folder = os.path.dirname(ops.__file__)
    text = "".join(open(f).read() for f in sorted(glob.glob(os.path.join(folder, "*.hip"))))

    def kind(arg):
        if "*" in arg or "hipStream_t" in arg:
            return ctypes.c_void_p
        return ctypes.c_longlong if "long long" in arg else {"float": ctypes.c_float, "double": ctypes.c_double, "int": ctypes.c_int}[arg.split()[0]]

    for name, given in ops._SIGNATURES.items():
        found = re.search(r'extern "C" (?:int|long long) %s\(([^)]*)\)' % name, text)
        assert found, name
        assert [kind(a.strip()) for a in found.group(1).split(",") if a.strip() not in ("", "void")] == list(given), name


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


_PLAIN = maps(mlp=None)
ALONE = {
    "maps": config([_PLAIN]),
    "maps_values_of_another_size": config([maps(heads=6, kv_heads=2, dim=16, vdim=24, mlp=None)]),
    "maps_ungrouped_no_growth": config([maps(heads=3, kv_heads=3, dim=32, vdim=64, temp=None, mlp=None)]),
    "maps_one_kv_head_wide": config([maps(heads=8, kv_heads=1, dim=64, vdim=128, scale=0.125, diff=0.1, mlp=None)]),
    "maps_wide_values": config([maps(heads=2, kv_heads=1, dim=100, vdim=200, scale=0.1, mlp=None)]),
    "latent": config([latent(mlp=None)]),
    "latent_no_window": config([latent(heads=5, size=0, mlp=None)]),
    "latent_one_head_no_scaling": config([latent(heads=1, size=64, yarn=None, mlp=None)]),
    "latent_generic_form": config([latent(heads=4, kv_rank=56, rot_dim=12, size=65, mlp=None)]),
    "latent_ramp_of_one_pair": config([latent(yarn=(8.0, 100, 2.0, 2.0), rot_dim=32, kv_rank=96, size=33, mlp=None)]),
    "gated": config([gated(mlp=None)]),
    "gated_ungrouped": config([gated(heads=3, kv_heads=3, dim=16, vdim=16, mlp=None)]),
    "gated_values_of_another_size": config([gated(heads=8, kv_heads=2, dim=40, vdim=24, mlp=None)]),
    "gated_wide": config([gated(heads=4, kv_heads=1, dim=128, vdim=128, scale=0.1, mlp=None)]),
    "experts": config([gated(mlp=moe())]),
    "experts_top1": config([gated(mlp=moe(experts=3, top=1, ff=40))]),
    "experts_all": config([gated(mlp=moe(experts=4, top=4, ff=8))]),
    "a_layer_twice": config([_PLAIN, dict(_PLAIN, weights_of=0)]),
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
    for sizes in ((2, 5, 57, 64, 3, 69), (63, 2, 1, 1, 133), (128, 72), (1, 1, 1, 2, 195), (50, 51, 99)):
        s, at = eng.open(), 0
        for n in sizes:
            rows.add(eng.step([(s, reqs[0][at:at + n], list(range(n)))]).double().cpu().numpy(), want[0][at:at + n], sizes)
            at += n
        eng.close(s)
        assert at == 200
    # unequal batches: prompts in one step, then one token each; shorter requests end earlier; the second round finds slots
    # and pages that the first one used
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
    # prompts' portions beside tokens of sequences that are already decoding
    a, b = eng.open(), eng.open()
    rows.add(eng.step([(a, reqs[0][:150], [149])]).double().cpu().numpy(), want[0][149:150], "before")
    at = 0
    for k, n in enumerate((40, 2, 70)):
        got = eng.step([(a, [reqs[0][150 + k]], [0]), (b, reqs[3][at:at + n], list(range(n)))]).double().cpu().numpy()
        rows.add(got, np.concatenate([want[0][150 + k:151 + k], want[3][at:at + n]]), ("mixed", k))
        at += n
    eng.close(a)
    eng.close(b)
    rows.check()
    assert eng.cache.pages_in_use() == 0 and eng.cache.free_slots == 6


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_through_recorded_steps(tmp_path, dtype):
    cfg = MIXED
    w = make_weights(cfg, 6)
    eng = engine_for(tmp_path, cfg, w, dtype)
    a, b = tokens_of(cfg, 20, 200), tokens_of(cfg, 21, 150)
    wa, wb = P.forward(w, cfg, a), P.forward(w, cfg, b)
    sa, sb = eng.open(), eng.open()
    rows = Rows(dtype)
    got = eng.step([(sa, a[:30], [29]), (sb, b[:3], [2])]).double().cpu().numpy()
    rows.add(got, np.stack([wa[29], wb[2]]), "prompts")
    for k in range(140):          # across two page borders and the window's length; one shape, recorded and replayed
        got = eng.step([(sa, [a[30 + k]], [0]), (sb, [b[3 + k]], [0])]).double().cpu().numpy()
        rows.add(got, np.stack([wa[30 + k], wb[3 + k]]), k)
    rows.check()
    assert eng.graphs.replays >= 100


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_prompts_through_recorded_steps(tmp_path, dtype):
    """The same prompt shape several times: recorded, then replayed at a padded size, with other steps in the meantime."""
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
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", ["maps", "gated", "latent"])
def test_a_far_token_that_towers_over_hundreds(tmp_path, kind, dtype):
    """Queries and keys read one lane of the embedding's that a single marked token has, so that its score stands out: where
    it is visible it decides the result, and two sequences that differ in that token alone differ until it leaves the window."""
    L = dict(maps=maps(heads=2, kv_heads=1, dim=16, vdim=32, scale=1.0, mlp=None), gated=gated(heads=2, kv_heads=1, dim=16, vdim=16, scale=1.0, mlp=None),
             latent=latent(heads=2, kv_rank=32, rot_dim=8, dim=16, vdim=16, scale=1.0, size=130, mlp=None))[kind]
    cfg = config([L])
    w = make_weights(cfg, 9)
    mark, p = 7, "l0.mix."
    w["embed"][:, 0] = 0.0
    w["embed"][mark, 0] = 6.0                    # nobody else has the lane
    bf = lambda a: torch.from_numpy(a).bfloat16().double().numpy()
    if kind == "latent":
        w[p + "dkv"][0] *= 0.0
        w[p + "dkv"][0, 0] = 4.0                  # the latent's first lane is the mark
        w[p + "uk"][:, 0] = bf(1.5 * np.sign(w[p + "uk"][:, 0]))
        w[p + "q"] = bf(2.0 * w[p + "q"])
        w[p + "sink"][:] = 0.0
    else:
        signs = np.sign(w[p + "k"][:, 0])
        w[p + "k"][:, 0] = 2.0 * signs
        w[p + "q.b"] = np.tile(3.0 * signs, 2)    # both heads look for the mark
        if kind == "maps":
            w[p + "q.b"].reshape(2, 2, 16)[:, 1] = 0.0        # with their first map alone
    eng = engine_for(tmp_path, cfg, w, dtype, max_tokens=1024)
    n = 300
    other = [t if t != mark else 8 for t in tokens_of(cfg, 33, n)]
    rows = Rows(dtype)
    for at in (0, 1, 63, 64, 127, 128, 170):
        toks = other[:at] + [mark] + other[at + 1:]
        want = P.forward(w, cfg, toks)
        if at == 64:
            plain = P.forward(w, cfg, other)
            far = np.abs(want - plain).max(axis=1) / np.median(np.abs(want).max(axis=1))
            seen = slice(at + 1, at + 130) if kind == "latent" else slice(at + 1, n)
            assert np.median(far[seen]) > 0.1, "the mark does not show"
            assert kind != "latent" or far[at + 130:].max() < 1e-12
        rows.add(whole(eng, toks), want, at)
        s = eng.open()
        eng.step([(s, toks[:at + 100], [])])
        for k in range(at + 100, min(n, at + 135)):     # in decoding across the window's edge
            rows.add(eng.step([(s, [toks[k]], [0])]).double().cpu().numpy(), want[k:k + 1], (at, k))
        eng.close(s)
    rows.check()


@pytest.mark.gpu
def test_pages_that_leave_the_window_go_back(tmp_path):
    cfg = config([latent(size=70, mlp=None), gated(mlp=None), latent(heads=2, kv_rank=40, size=20, mlp=None)])
    w = make_weights(cfg, 12)
    eng = engine_for(tmp_path, cfg, w, "float32", max_tokens=1024)
    a = tokens_of(cfg, 60, 420)
    want = P.forward(w, cfg, a)
    rows = Rows("float32")
    s, at = eng.open(), 0
    for n in (250, 64, 70):
        rows.add(eng.step([(s, a[at:at + n], list(range(n)))]).double().cpu().numpy(), want[at:at + n], n)
        at += n
    for k in range(at, 420):
        rows.add(eng.step([(s, [a[k]], [0])]).double().cpu().numpy(), want[k:k + 1], k)
    held = {g.need.window: [i for i, p in enumerate(g.tables[s]) if p >= 0] for g in eng.cache.groups}
    assert held == {70: [5, 6], 0: list(range(7)), 20: [6]}
    eng.close(s)
    rows.check()
    assert eng.cache.pages_in_use() == 0


def drawn_config(seed):
    """A configuration drawn from the seed: one to five layers of all types, head counts and sizes that are and are not
    multiples of eight, any grouping of the queries, windows shorter and longer than a page or none, scaled rotations or
    not, experts or none, layers that take others' tensors."""
    rng = np.random.default_rng(seed)
    pick = lambda *a: a[int(rng.integers(0, len(a)))]
    layers = []
    for i in range(int(rng.integers(1, 6))):
        if i and rng.random() < 0.25:
            j = int(rng.integers(0, i))
            layers.append(dict(layers[j], weights_of=j))
            continue
        n = int(rng.integers(1, 9))
        mlp = None if rng.random() < 0.2 else moe(experts=n, top=int(rng.integers(1, n + 1)), ff=pick(8, 16, 40, 6))
        G, kind = int(rng.integers(1, 4)), rng.random()
        if kind < 0.35:
            d = pick(8, 16, 32, 48, 6, 20, 64)
            layers.append(maps(heads=G * int(rng.integers(1, 5)), kv_heads=G, dim=d, vdim=pick(2 * d, 2 * d, 16, 48, 10, 128), scale=pick(0.1, 0.3, 0.6),
                               diff=pick(0.2, 0.5, 0.8), temp=pick(None, (0.2, 7), (0.5, 64), (1.0, 1)), mlp=mlp))
        elif kind < 0.7:
            r, dr = pick((64, 16), (96, 32), (128, 64), (32, 8), (40, 10), (72, 24))
            layers.append(latent(heads=int(rng.integers(1, 7)), dim=pick(8, 16, 24, 64, 10), rot_dim=dr, vdim=pick(8, 16, 64, 12), kv_rank=r,
                                 scale=pick(0.1, 0.2, 0.4), size=pick(0, 1, 5, 32, 64, 65, 130), base=pick(100.0, 10000.0),
                                 yarn=pick(None, (2.0, 100, 8.0, 1.0), (16.0, 4096, 32.0, 1.0)), mlp=mlp))
        else:
            d = pick(8, 16, 32, 48, 6, 20, 64, 128)
            layers.append(gated(heads=G * int(rng.integers(1, 5)), kv_heads=G, dim=d, vdim=pick(d, d, 16, 40, 10), scale=pick(0.1, 0.3, 0.6), mlp=mlp))
    return config(layers, width=pick(40, 64, 96, 128, 72), vocab=pick(50, 101, 257), eps=pick(1e-5, 1e-6))


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", [11, 12, 13, 14, 15, 16, 17, 18, 19, 20])
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
    """Sizes at which products run on the matrix cores in every form: a prompt of more than 512 tokens, decode steps of one,
    20 and 70 sequences."""
    L = [maps(heads=8, kv_heads=2, dim=32, vdim=64, scale=0.2, temp=(0.2, 100), mlp=moe(experts=8, top=2, ff=128)),
         latent(heads=8, dim=64, rot_dim=32, vdim=64, kv_rank=128, scale=0.1, size=200, mlp=moe(experts=6, top=3, ff=192)),
         gated(heads=8, kv_heads=4, dim=64, vdim=64, scale=0.15, mlp=moe(experts=16, top=1, ff=64))]
    cfg = config(L + [dict(L[0], weights_of=0)], width=768, vocab=512)
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


class _Step:
    """The index arrays that the kernels read, for sequences laid out by hand; `padding` tokens of no sequence behind."""

    def __init__(self, news, pasts, dev, padding=0):
        i32 = lambda a: torch.tensor(a, dtype=torch.int32, device=dev)
        self.n_tokens, self.n_seqs = sum(news) + padding, len(news)
        self.positions = i32([p + t for n, p in zip(news, pasts) for t in range(n)] + [0] * padding)
        self.token_seq = i32([b for b, n in enumerate(news) for _ in range(n)] + [-1] * padding)
        self.cu_seqlens = i32([sum(news[:b]) for b in range(len(news) + 1)])
        self.lens_after = i32([p + n for n, p in zip(news, pasts)])
        self.max_position = max(p + n for n, p in zip(news, pasts)) - 1
        self.max_new, self.max_len_after = max(news), self.max_position + 1
        self.token_source = None


@pytest.mark.gpu
@pytest.mark.parametrize("form,dtype", [("generic", torch.float32), ("generic", torch.bfloat16), ("matrix", torch.bfloat16)],
                         ids=["generic-float32", "generic-bfloat16", "matrix"])
@pytest.mark.parametrize("decode", [False, True], ids=["prompt", "decoding"])
@pytest.mark.parametrize("window", [0, 1, 64, 65, 100, 300])
def test_latent_rows_that_stand_out_at_every_edge(form, dtype, decode, window):
    """One row's score towers over all others: where it is visible, the result is that row's latent, and where it is not,
    the others' (zero).  Rows at both edges of the window, at page borders, the first and far back among hundreds; a
    sequence's pages lie scattered, and pages and places that no visible row lies in would win if they were read."""
    from burn_lm_amd.csrc import ops
    dev = "cuda"
    ops.latent_attn_init(dev)
    H, R, Dr, ps, n = 3, 64, 16, 64, 420
    pages = [7, 2, 9, 0, 8, 3, 5]
    table = torch.tensor([pages + [-1] * 2], dtype=torch.int32, device=dev)
    p = n - 1
    edges = {p, p - 1, max(0, p - window + 1), max(0, p - window), 0, 1, 63, 64, 127, 128, 191, 192, p // 2}
    W = R + Dr
    for j in sorted(e for e in edges if 0 <= e <= p):
        g = torch.Generator().manual_seed(j)
        rows = torch.zeros(10, 1, ps, W)
        rows[..., R:] = torch.randn(10, 1, ps, Dr, generator=g) * 0.02
        rows[[1, 4, 6]] = 50.0                          # of no sequence
        rows[pages[n // ps], :, n % ps:] = 50.0         # what lies behind the sequence in its last page
        rows[pages[j // ps], 0, j % ps, :R] = 3.0
        rows[pages[j // ps], 0, j % ps, R:] = 1.0
        kc = rows.to(dev, dtype).contiguous()
        vc = rows[..., :R].transpose(2, 3).contiguous().to(dev, dtype)
        step = _Step([1], [p], dev) if decode else _Step([n], [0], dev)
        q = torch.zeros(step.n_tokens, H, W)
        q[..., R:] = 2.0
        olat = torch.empty(step.n_tokens, H, R, dtype=torch.float32, device=dev)
        for splits in ((1, 3, 7, 14, 20) if decode else (1,)):
            if form == "matrix":
                ops.latent_attn_mfma(q.to(dev, dtype), olat, kc, vc, step, table, ps, H, R, Dr, 0.5, splits, window=window)
            else:
                ops.latent_attn(q.to(dev), olat, kc, step, table, ps, H, R, Dr, 0.5, splits, window=window)
            want = torch.tensor([3.0 if P.visible(pos, j, window) else 0.0 for pos in ([p] if decode else range(n))])
            wrong = (olat.cpu() - want.view(-1, 1, 1)).abs().amax((1, 2)) > 5e-3
            assert not wrong.any(), (j, splits, wrong.nonzero().view(-1).tolist()[:5])


@pytest.mark.gpu
@pytest.mark.parametrize("in_dtype,out_dtype", [(torch.bfloat16, torch.bfloat16), (torch.float32, torch.bfloat16), (torch.bfloat16, torch.float32)])
@pytest.mark.parametrize("T", [1, 7, 16, 33, 128, 129, 300])
@pytest.mark.parametrize("N,K,gap", [(64, 96, 32), (130, 128, 0), (16, 40, 8), (12, 24, 8), (96, 512, 64), (10, 18, 3)])
def test_products_per_head(in_dtype, out_dtype, T, N, K, gap):
    """Every head's product at row counts on both sides of each form's limits, K with and without a piece of less than 32,
    columns that fill no tile, heads with lanes in between; what lies beside the results stays as it was."""
    from burn_lm_amd.csrc import ops
    dev, H, ld_head = "cuda", 3, N + 6
    g = torch.Generator().manual_seed(T * 1000 + N + K)
    x = torch.randn(T, H * (K + gap) + 8, generator=g).to(in_dtype)
    w = (torch.randn(H, N, K, generator=g) * K ** -0.5).bfloat16()
    out = torch.full((T, H * ld_head), 7.0, dtype=out_dtype, device=dev)
    ops.head_project(x.to(dev), K + gap, w.to(dev), out, ld_head, K=K)
    got = out.view(T, H, ld_head).double().cpu()
    want = torch.stack([x[:, h * (K + gap):h * (K + gap) + K].bfloat16().double() @ w[h].double().T for h in range(H)], 1)
    off = 2e-2 if out_dtype == torch.bfloat16 or in_dtype == torch.float32 else 1e-4
    assert (got[..., :N] - want).abs().max() < off * (1 + want.abs().max())
    assert (got[..., N:] == 7.0).all()


@pytest.mark.gpu
@pytest.mark.parametrize("form", ["generic", "matrix"])
@pytest.mark.parametrize("R,Dr", [(64, 16), (96, 32), (512, 64), (32, 8)])
@pytest.mark.parametrize("window,sinks", [(50, True), (0, True), (70, False), (1, True)])
def test_latent_kernels_against_plain_softmax(form, R, Dr, window, sinks):
    """Random rows and queries of two sequences, one of them with a past, prompts and single tokens, whole and in pieces; sinks
    from far below every score to far above."""
    from burn_lm_amd.csrc import ops
    dev = "cuda"
    ops.latent_attn_init(dev)
    dtype = torch.float32 if form == "generic" else torch.bfloat16
    H, ps, W, scale = 5, 64, R + Dr, 0.9 / math.sqrt(R + Dr)
    rng = np.random.default_rng(R + window)
    rt = lambda a: torch.from_numpy(a).to(dtype)
    tables = torch.tensor([[3, 0, 6, 7], [5, 1, 4, 2]], dtype=torch.int32, device=dev)
    K = rt(rng.standard_normal((8, 1, ps, W)))
    V = K[..., :R].transpose(2, 3).contiguous()
    sink = np.array([-30.0, -1.0, 0.0, 2.0, 30.0])
    s32 = torch.tensor(sink, dtype=torch.float32, device=dev) if sinks else None
    for news, pasts in (([100, 33], [0, 190]), ([1, 1], [149, 222])):
        step = _Step(news, pasts, dev)
        q = rt(rng.standard_normal((sum(news), H, W)))
        for splits in ((1, 3, 7, 19) if step.max_new == 1 else (1,)):
            olat = torch.empty(sum(news), H, R, dtype=torch.float32, device=dev)
            if form == "matrix":
                ops.latent_attn_mfma(q.to(dev), olat, K.to(dev), V.to(dev), step, tables, ps, H, R, Dr, scale, splits, window=window, sinks=s32)
            else:
                ops.latent_attn(q.to(dev), olat, K.to(dev), step, tables, ps, H, R, Dr, scale, splits, window=window, sinks=s32)
            got, row = olat.double().cpu().numpy(), 0
            for b, (n, past) in enumerate(zip(news, pasts)):
                ks = np.concatenate([K[x, 0].double().numpy() for x in tables[b].cpu().tolist()])
                for t in range(n):
                    pos = past + t
                    see = [j for j in range(pos + 1) if P.visible(pos, j, window)]
                    for h in range(H):
                        wts = P.weights_over((ks[see] @ q[row, h].double().numpy()) * scale, sink[h] if sinks else None)
                        assert np.abs(got[row, h] - wts @ ks[see, :R]).max() < (1e-5 if form == "generic" else 3e-2), (b, t, h, splits)
                    row += 1


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["float32", "bfloat16"])
@pytest.mark.parametrize("mode", ["heads", "rows", "maps"])
def test_norms_growth_and_page_writes(dtype, mode):
    """Biases enter ahead of the norm, values are not normed, queries grow with their position, two maps lie side by side in
    the pages and apart in the queries; columns behind the rows and pages of others stay as they were."""
    from burn_lm_amd.csrc import ops
    dev = "cuda"
    H, G, dk, dv, ps, eps = 4, 2, 35, 23, 64, 0.1                # an eps that shows
    rng = np.random.default_rng(3)
    step = _Step([3, 1], [62, 130], dev, padding=2)              # one sequence crosses a page border
    T, need = step.n_tokens, (H + G) * dk + (G // 2 if mode == "maps" else G) * dv
    Gv = G // 2 if mode == "maps" else G
    rows = torch.from_numpy(rng.standard_normal((T, need + 6))).to(dtype)     # six columns nobody may touch
    tables = torch.tensor([[4, 1, -1], [0, 5, 2]], dtype=torch.int32, device=dev)
    f32 = lambda a: torch.tensor(np.asarray(a), dtype=torch.float32, device=dev)
    bias = f32(rng.standard_normal(need))
    qw, kw = (f32(rng.uniform(0.5, 1.5, n * dk if mode == "rows" else dk)) for n in (H, G))
    kc = torch.zeros(6, Gv, ps, dk * (G // Gv), dtype=dtype, device=dev)
    vc = torch.zeros(6, Gv, dv, ps, dtype=dtype, device=dev)
    qkv = rows.to(dev).clone()
    q_out = torch.full((T, 2 * H * dk), 9.0, dtype=dtype, device=dev) if mode == "maps" else None
    ops.qkv_norm(qkv, bias, qw, kw, eps, step, tables, kc, vc, ps, H, G, dk, dv, whole_rows=mode == "rows", growth=(0.7, 20), q_out=q_out)
    x = rows.double().numpy()
    x[:, :need] += bias.double().cpu().numpy()
    q, k, v = x[:, :H * dk], x[:, H * dk:(H + G) * dk], x[:, (H + G) * dk:need].reshape(T, Gv, dv)
    if mode == "rows":
        q, k = P.unit_rms(q, eps) * qw.double().cpu().numpy(), P.unit_rms(k, eps) * kw.double().cpu().numpy()
        q, k = q.reshape(T, H, dk), k.reshape(T, G, dk)
    else:
        q, k = P.unit_rms(q.reshape(T, H, dk), eps) * qw.double().cpu().numpy(), P.unit_rms(k.reshape(T, G, dk), eps) * kw.double().cpu().numpy()
    at = [(0, 62), (0, 63), (0, 64), (1, 130)]
    q = q[:4] * np.array([P.query_factor(p, 0.7, 20) for _, p in at])[:, None, None]
    tol = 1e-5 if dtype == torch.float32 else 3e-2
    if mode == "maps":
        wide = np.zeros((4, H, 2, dk))
        for h in range(H):
            wide[:, h, h % 2] = q[:, h]
        assert np.abs(q_out[:4].double().cpu().numpy() - wide.reshape(4, -1)).max() < tol
        k = k.reshape(T, G // 2, 2 * dk)
        assert torch.equal(qkv.cpu(), rows)
    else:
        assert np.abs(qkv[:4, :H * dk].double().cpu().numpy().reshape(4, H, dk) - q).max() < tol
        assert torch.equal(qkv[:, H * dk:].cpu(), rows[:, H * dk:]) and torch.equal(qkv[4:].cpu(), rows[4:])
    for t, (b, p) in enumerate(at):
        page = int(tables[b, p // ps])
        assert np.abs(kc[page, :, p % ps].double().cpu().numpy() - k[t]).max() < tol
        assert np.abs(vc[page, :, :, p % ps].double().cpu().numpy() - v[t]).max() < tol
    assert float(kc[[0, 3, 5]].float().abs().sum()) == 0 and float(vc[[0, 3, 5]].float().abs().sum()) == 0


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["float32", "bfloat16"])
def test_gates_differences_tables_and_biases(dtype):
    from burn_lm_amd.csrc import ops
    dev = "cuda"
    rng = np.random.default_rng(2)
    f32 = lambda a: torch.tensor(np.asarray(a), dtype=torch.float32, device=dev)
    i32 = lambda a: torch.tensor(a, dtype=torch.int32, device=dev)
    dbl = lambda t: t.double().cpu().numpy()
    tol = 1e-5 if dtype == torch.float32 else 1e-2
    # one gate per head, its columns inside wider rows
    for H, dv in ((3, 40), (1, 7), (8, 128)):
        x, wide = (torch.from_numpy(rng.standard_normal((5, n))).to(dev, dtype) for n in (H * dv, H + 6))
        want = dbl(x).reshape(5, H, dv) * P.sigmoid(dbl(wide)[:, 2:2 + H])[:, :, None]
        assert rel_err(dbl(ops.head_gate(x, wide[:, 2:2 + H], dv)), want.reshape(5, -1)) < tol
    # two maps to one result; rows of no sequence become zero whatever they held
    for H, dv in ((3, 40), (1, 7), (2, 200)):
        step = _Step([2, 1], [5, 9], dev, padding=2)
        a = f32(rng.standard_normal((5, 2 * H, dv)))
        a[4] = float("nan")
        out = torch.full((5, H * dv), 3.0, dtype=dtype, device=dev)
        ops.map_difference(a, out, step, H, dv, 0.83, 0.02, 0.4)
        u = dbl(a)[:3, 0::2] - 0.83 * dbl(a)[:3, 1::2]
        assert rel_err(dbl(out)[:3], (P.unit_rms(u, 0.02) * 0.4).reshape(3, -1)) < tol and float(out[3:].float().abs().sum()) == 0
    # experts by table: ids from the host and ids that only the device knows
    for E, top in ((5, 2), (1, 1), (7, 7), (100, 9)):
        table = np.stack([rng.permutation(E)[:top] for _ in range(30)]).astype(np.int32)
        ids = [int(t) for t in rng.integers(0, 30, 9)]
        want = np.zeros((9, E + 1))
        for t, i in enumerate(ids):
            want[t, table[i]] = 1.0 / top
        want[:, E] = 1.0
        picked = i32(ids[::-1])
        cell = torch.tensor([picked.data_ptr()], dtype=torch.int64, device=dev)
        given = [i if t % 2 else 0 for t, i in enumerate(ids)]
        source = (i32([-1 if t % 2 else 8 - t for t in range(9)]), cell)
        for got in (ops.moe_table(i32(table), i32(ids), torch.empty(9, E + 1, dtype=torch.float32, device=dev), E),
                    ops.moe_table(i32(table), i32(given), torch.empty(9, E + 1, dtype=torch.float32, device=dev), E, source)):
            assert np.abs(dbl(got) - want).max() < 1e-7
    # a last projection's bias ahead of the norm behind it
    for D in (24, 18, 2048, 9000):
        h0, y, z = rng.standard_normal((4, D)), f32(rng.standard_normal((2, 4, D))), f32(rng.standard_normal((4, D))).to(dtype)
        ga, gp, go, b1, b2 = (f32(rng.uniform(0.5, 1.5, D)) for _ in range(5))
        for terms, want in (([(y, 1.0, None, 0.0, b1)], dbl(y).sum(0) + dbl(b1)), ([(z, 1.0, None, 0.0, b2)], dbl(z) + dbl(b2)),
                            ([(y, 0.5, ga, 1e-3, b1), (z, 2.0, None, 0.0, b2)],
                             0.5 * P.unit_rms(dbl(y).sum(0) + dbl(b1), 1e-3) * dbl(ga) + 2 * (dbl(z) + dbl(b2)))):
            h, out = f32(h0), torch.empty(4, D, dtype=dtype, device=dev)
            ops.post_norm(h, terms, post=(gp, 1e-4), gamma=go, eps=1e-5, out=out)
            want = dbl(f32(h0)) + P.unit_rms(want, 1e-4) * dbl(gp)
            assert rel_err(dbl(h), want) < 1e-5 and rel_err(dbl(out), P.unit_rms(want, 1e-5) * dbl(go)) < tol


@pytest.mark.gpu
@pytest.mark.parametrize("form", ["matrix_16", "matrix_32", "sink", "generic"])
@pytest.mark.parametrize("decode", [False, True], ids=["prompt", "decoding"])
def test_attention_kernels_hand_float_results_on(form, decode):
    """The same kernels with a float32 output: the values that the bfloat16 output rounds."""
    from burn_lm_amd.csrc import ops
    dev = "cuda"
    ops.latent_attn_init(dev)
    H, G, d, ps = 8, 2, 64, 64
    rng = np.random.default_rng(5)
    bf = lambda *s: torch.from_numpy(rng.standard_normal(s)).to(dev, torch.bfloat16)
    tables = torch.tensor([[3, 0, 6, 7], [5, 1, 4, 2]], dtype=torch.int32, device=dev)
    K, V = bf(8, G, ps, d), bf(8, G, d, ps)
    step = _Step([1, 1], [149, 222], dev) if decode else _Step([150, 33], [0, 190], dev)
    q = bf(step.n_tokens, H * d)
    outs = []
    for dtype in (torch.float32, torch.bfloat16):
        out = torch.empty(step.n_tokens, H * d, dtype=dtype, device=dev)
        if form == "generic":
            ops.sink_attn(q, out, None, None, step, tables, K, V, ps, H, G, d, d, 0.1, 0)
        elif form == "sink":
            ops.sink_attn_mfma(q, out, None, None, step, tables, K, V, ps, H, G, d, d, 0.1, 0, n_splits=2 if decode else 1)
        elif decode:
            ops.attn_decode(q, q.stride(0), out, step.positions, step.token_seq, tables, K, V, ps, H, G, d, 0.1, 0, n_splits=3 if form == "matrix_32" else 1)
        else:
            ops.attn_prefill_mfma(q, q.stride(0), out, step.positions, step.cu_seqlens, tables, K, V, ps, 2, 150, H, G, d, 0.1, 0, queries=int(form[-2:]))
        outs.append(out)
    assert torch.equal(outs[0].bfloat16(), outs[1]) and not torch.equal(outs[0], outs[1].float())


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
