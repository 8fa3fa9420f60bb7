"""The Belelorn design as a plan of parts.

A decoder with sinusoidal position vectors on its embedding and a norm before and behind every sublayer, of which a run
of layers runs several times with the same weights: each pass starts from a projection of the residual beside the
embedding's output, plus a vector of its own, and keeps its own cache and state.  A layer's mixer is a matrix memory
with an exponential input gate (mLSTM), or a pair: softmax attention (grouped queries, biases, unit-norm queries and
keys, capped scores, a sliding window beside which the first tokens stay visible, values that are the keys as projected)
beside lightning attention, each result normed on its own and half of each added.  The feed-forward is dense with a
squared ReLU, or a mixture of clamped experts chosen by sigmoid scores that weight the experts' inputs, beside a shared
expert; a layer may have none.  Output: norm, a head matrix of its own, a logit scale.

Checkpoint tensor names: ``embed``, ``head``, ``final.norm``, ``loop.in``, ``loop.step``; per layer i ``l<i>.norm1``,
``l<i>.norm1b``, ``l<i>.norm2``, ``l<i>.norm2b``; ``l<i>.mix.left.q|q.b|k|k.b|o|out``, ``l<i>.mix.right.q|k|v|g|norm|o|out``
or ``l<i>.mix.q|k|v|g|i|i.b|f|f.b|norm|o``; ``l<i>.mlp.up|down`` or ``l<i>.mlp.router|e<j>.gate|up|down|shared.gate|up|down``."""
from __future__ import annotations

from ..config.belelorn import MAX_POSITIONS, BelelornConfig
from ..parts.base import PartSpec
from ..registry import Architecture, register_architecture
from ..weights.random_init import Normal, Ones, Uniform
from .plan import LayerPlan, ModelPlan, Place

POSITION_BASE = 10000.0
EXPERT_ALPHA = 1.702


def _mixer(cfg, i):
    m, p, D = cfg.layers[i].mixer, f"l{i}.mix.", cfg.width
    if m.kind == "mlstm":
        names = {r: p + r for r in ("q", "k", "v", "g", "i", "f", "norm", "o")}
        return PartSpec("mlstm", dict(width=D, heads=m.heads, dim=m.dim, vdim=m.vdim, gate_cap=m.gate_cap, eps=cfg.eps),
                        dict(names, i_bias=p + "i.b", f_bias=p + "f.b"))
    a, b = m.left, m.right
    left = PartSpec("sink_attention",
                    dict(width=D, heads=a.heads, kv_heads=a.kv_heads, dim=a.dim, vdim=a.vdim, scale=a.scale, window=a.window,
                         keep_first=a.keep_first, softcap=a.softcap, rot_dims=0, sink=False, talk=False, bias=True,
                         output_bias=False, values="keys", unit_norm_eps=cfg.eps),
                    {"q": p + "left.q", "q_bias": p + "left.q.b", "k": p + "left.k", "k_bias": p + "left.k.b", "o": p + "left.o"})
    right = PartSpec("lightning_attention", dict(width=D, heads=b.heads, dim=b.dim, vdim=b.vdim, decay=b.decay, eps=cfg.eps),
                     {r: f"{p}right.{r}" for r in ("q", "k", "v", "g", "norm", "o")})
    return PartSpec("mixer_pair", dict(width=D, left=left, right=right, left_scale=0.5, right_scale=0.5, norm_eps=cfg.eps),
                    dict(left_norm=p + "left.out", right_norm=p + "right.out"))


def _feed_forward(cfg, i):
    f, p = cfg.layers[i].mlp, f"l{i}.mlp."
    if f.kind == "dense":
        return PartSpec("dense_relu2", dict(width=cfg.width, inner=f.ff), dict(up=p + "up", down=p + "down"))
    names = dict(router=p + "router")
    for e in [f"e{e}" for e in range(f.experts)] + (["shared"] if f.shared_ff else []):
        names.update({f"{e}.{r}": f"{p}{e}.{r}" for r in ("gate", "up", "down")})
    return PartSpec("grouped_experts",
                    dict(width=cfg.width, experts=f.experts, top=f.top, expert_inner=f.ff, correction=False, score="sigmoid",
                         renormalize=False, form="clamped", limit=f.limit, alpha=EXPERT_ALPHA, shared_inner=f.shared_ff,
                         shared_limit=f.shared_limit), names)


def _order(cfg):
    n, loop = len(cfg.layers), cfg.loop
    if loop is None:
        return [Place(i) for i in range(n)]
    places = [Place(i) for i in range(loop.start)]
    for t in range(loop.times):
        places += [Place(i, turn=t if i == loop.start else None) for i in range(loop.start, loop.stop)]
    return places + [Place(i) for i in range(loop.stop, n)]


def plan(cfg: BelelornConfig, checkpoint=None) -> ModelPlan:
    D = cfg.width
    norm = lambda name, scale=1.0: PartSpec("rmsnorm", dict(width=D, eps=cfg.eps, offset=1.0, scale=scale), dict(weight=name))
    layers = []
    for i, layer in enumerate(cfg.layers):
        l = f"l{i}."
        parts = dict(mixer_norm=norm(l + "norm1"), mixer=_mixer(cfg, i), mixer_post=norm(l + "norm1b"))
        if layer.mlp is None:
            layers.append(LayerPlan("post_norm_mixer_only", parts))
        else:
            parts.update(ffn_norm=norm(l + "norm2"), feed_forward=_feed_forward(cfg, i), ffn_post=norm(l + "norm2b"))
            layers.append(LayerPlan("post_norm", parts))
    ignorable = [rf"^l{i}\.norm2b?$" for i, layer in enumerate(cfg.layers) if layer.mlp is None]
    if cfg.loop is None:
        ignorable.append(r"^loop\.(in|step)$")
    entry = None if cfg.loop is None else PartSpec("loop_entry", dict(width=D, times=cfg.loop.times),
                                                   dict(proj="loop.in", step="loop.step"))
    return ModelPlan(
        vocab_size=cfg.vocab, width=D, max_positions=MAX_POSITIONS,
        embedding=PartSpec("table", dict(vocab=cfg.vocab, width=D, position_base=POSITION_BASE), dict(weight="embed")),
        layers=layers, order=_order(cfg), entry=entry,
        final_norm=norm("final.norm", cfg.logit_scale),      # the logits are linear in the norm's weight
        head=PartSpec("linear", dict(vocab=cfg.vocab, width=D), dict(weight="head")),
        stop_ids=(), ignorable_tensors=tuple(ignorable))


def checkpoint_tensors(cfg: BelelornConfig):
    """Name -> (shape, initialiser) of a fresh checkpoint: matrices N(0, 1/sqrt(fan-in)), weights of norms near one (those
    stored as the distance from one near zero), gate biases under which memories last."""
    D = cfg.width
    lin = lambda n_out, n_in: ((n_out, n_in), Normal(n_in ** -0.5))
    near_zero = ((D,), Normal(0.1))
    out = {"embed": ((cfg.vocab, D), Normal(1.0, layout="table")), "head": lin(cfg.vocab, D), "final.norm": near_zero}
    if cfg.loop is not None:
        out["loop.in"], out["loop.step"] = lin(D, 2 * D), ((cfg.loop.times, D), Normal(0.3))
    for i, layer in enumerate(cfg.layers):
        l, m, f = f"l{i}.", layer.mixer, layer.mlp
        out[l + "norm1"], out[l + "norm1b"] = near_zero, near_zero
        p = l + "mix."
        if m.kind == "mlstm":
            HK, HV = m.heads * m.dim, m.heads * m.vdim
            out.update({p + "q": lin(HK, D), p + "k": lin(HK, D), p + "v": lin(HV, D), p + "g": lin(HV, D), p + "o": lin(D, HV),
                        p + "norm": ((HV,), Ones(0.1)), p + "i": lin(m.heads, D), p + "i.b": ((m.heads,), Normal(1.0)),
                        p + "f": lin(m.heads, D), p + "f.b": ((m.heads,), Uniform(2.0, 6.0))})
        else:
            a, b = m.left, m.right
            out.update({p + "left.q": lin(a.heads * a.dim, D), p + "left.q.b": ((a.heads * a.dim,), Normal(0.3)),
                        p + "left.k": lin(a.kv_heads * a.dim, D), p + "left.k.b": ((a.kv_heads * a.dim,), Normal(0.3)),
                        p + "left.o": lin(D, a.heads * a.vdim), p + "left.out": ((D,), Ones(0.1))})
            HK, HV = b.heads * b.dim, b.heads * b.vdim
            out.update({p + "right.q": lin(HK, D), p + "right.k": lin(HK, D), p + "right.v": lin(HV, D), p + "right.g": lin(HV, D),
                        p + "right.norm": ((HV,), Ones(0.1)), p + "right.o": lin(D, HV), p + "right.out": ((D,), Ones(0.1))})
        if f is None:
            continue
        out[l + "norm2"], out[l + "norm2b"] = near_zero, near_zero
        p = l + "mlp."
        if f.kind == "dense":
            out[p + "up"], out[p + "down"] = lin(f.ff, D), lin(D, f.ff)
            continue
        out[p + "router"] = lin(f.experts, D)
        for e, ff in [(f"e{e}.", f.ff) for e in range(f.experts)] + ([("shared.", f.shared_ff)] if f.shared_ff else []):
            out[p + e + "gate"], out[p + e + "up"], out[p + e + "down"] = lin(ff, D), lin(ff, D), lin(D, ff)
    return out


BELELORN = Architecture(name="Belelorn", read_config=BelelornConfig.from_dict, plan=plan,
                        checkpoint_tensors=checkpoint_tensors, display_name="Belelorn", created_by="")
register_architecture(BELELORN, "belelorn")
