"""The Netanex design as a plan of parts.

A decoder with a norm on its embedding and norms before and behind every sublayer.  A layer's mixer is differential
attention (two maps per head over the same values, the second one subtracted; queries and keys normed per head and map;
queries that grow with the logarithm of their position; biases), latent attention (low-rank keys and values, YaRN-scaled
rotation, a sliding window, a learned sink, an elementwise output gate), or grouped-query attention whose queries and keys
are normed over their whole rows, with one added to the softmax's denominator and an output gate per head; only the latent
attention turns anything by position.  The feed-forward is a mixture of experts that a table of the token ids chooses; a
layer may have none.  A layer may use another layer's tensors, with a cache of its own.  The embedding is also the head.

Checkpoint tensor names: ``embed``, ``embed.norm``, ``final.norm``; per layer i with tensors of its own ``l<i>.norm1``,
``l<i>.norm1b``, ``l<i>.norm2``, ``l<i>.norm2b``; ``l<i>.mix.q|q.b|k|k.b|v|v.b|q.norm|k.norm|lq1|lk1|lq2|lk2|o|o.b``,
``l<i>.mix.q|dkv|dkv.norm|uk|uv|sink|g|o`` or ``l<i>.mix.q|q.b|k|k.b|v|v.b|q.norm|k.norm|g|o``;
``l<i>.mlp.table|e<j>.gate|up|down``."""
from __future__ import annotations

from ..config.netanex import MAX_POSITIONS, NetanexConfig
from ..parts.base import PartSpec
from ..registry import Architecture, register_architecture
from ..weights.random_init import DistinctRows, Normal, Ones
from .plan import LayerPlan, ModelPlan, Place

_QKV = {"q": "q", "q_bias": "q.b", "k": "k", "k_bias": "k.b", "v": "v", "v_bias": "v.b", "q_norm": "q.norm", "k_norm": "k.norm", "o": "o"}


def _position(m):
    """Key of the rotary table a latent layer turns with: one table for all layers of equal rotations."""
    return (m.rot_dims, m.rot_base, m.yarn) if m.kind == "latent_attention" else None


def _mixer(cfg, i):
    m, p, D = cfg.layers[i].mixer, f"l{i}.mix.", cfg.width
    if m.kind == "latent_attention":
        names = dict({r: p + r for r in ("q", "uk", "uv", "o", "dkv", "sink", "g")}, dkv_norm=p + "dkv.norm")
        return PartSpec("latent_attention", dict(width=D, heads=m.heads, dim=m.dim, rot_dim=m.rot_dim, vdim=m.vdim, kv_rank=m.kv_rank,
                                                 scale=m.scale, rot_dims=m.rot_dims, eps=cfg.eps, window=m.window, sink=True, gate=True),
                        names)
    params = dict(width=D, heads=m.heads, kv_heads=m.kv_heads, dim=m.dim, vdim=m.vdim, scale=m.scale, window=0, rot_dims=0,
                  talk=False, bias=True, norm_eps=cfg.eps)
    names = {r: p + n for r, n in _QKV.items()}
    if m.kind == "attention":
        names.update({r: p + r for r in ("lq1", "lk1", "lq2", "lk2")}, o_bias=p + "o.b")
        return PartSpec("differential_attention", dict(params, qk_norm="heads", sink=False, growth=m.growth, diff=m.diff), names)
    return PartSpec("sink_attention", dict(params, qk_norm="rows", sink="one", gate="heads", output_bias=False), dict(names, g=p + "g"))


def _feed_forward(cfg, i):
    f, p = cfg.layers[i].mlp, f"l{i}.mlp."
    names = {"table": p + "table"}
    for e in range(f.experts):
        names.update({f"e{e}.{r}": f"{p}e{e}.{r}" for r in ("gate", "up", "down")})
    return PartSpec("table_experts", dict(width=cfg.width, vocab=cfg.vocab, experts=f.experts, top=f.top, expert_inner=f.ff), names)


def plan(cfg: NetanexConfig, checkpoint=None) -> ModelPlan:
    D = cfg.width
    norm = lambda name: PartSpec("rmsnorm", dict(width=D, eps=cfg.eps, offset=1.0), dict(weight=name))
    owners = [i for i, layer in enumerate(cfg.layers) if layer.owner == i]
    tables = {}
    for i in owners:
        key = _position(cfg.layers[i].mixer)
        if key is not None and key not in tables:
            tables[key] = f"rot{len(tables)}"
    layers = []
    for i in owners:
        l, layer = f"l{i}.", cfg.layers[i]
        parts = dict(mixer_norm=norm(l + "norm1"), mixer=_mixer(cfg, i), mixer_post=norm(l + "norm1b"))
        if layer.mlp is not None:
            parts.update(ffn_norm=norm(l + "norm2"), feed_forward=_feed_forward(cfg, i), ffn_post=norm(l + "norm2b"))
        layers.append(LayerPlan("post_norm" if layer.mlp is not None else "post_norm_mixer_only", parts,
                                position=tables.get(_position(layer.mixer))))
    return ModelPlan(
        vocab_size=cfg.vocab, width=D, max_positions=MAX_POSITIONS,
        embedding=PartSpec("table", dict(vocab=cfg.vocab, width=D, norm_eps=cfg.eps, norm_offset=1.0),
                           dict(weight="embed", norm="embed.norm")),
        layers=layers, order=[Place(owners.index(layer.owner)) for layer in cfg.layers],
        final_norm=norm("final.norm"), head=PartSpec("linear", dict(vocab=cfg.vocab, width=D), dict(weight="embed")),
        positions={name: PartSpec("rope", dict(head_dim=key[0], theta=key[1], scaling=None, pairing="half", yarn=key[2]))
                   for key, name in tables.items()},
        stop_ids=(), ignorable_tensors=tuple(rf"^l{i}\.norm2b?$" for i in owners if cfg.layers[i].mlp is None))


def checkpoint_tensors(cfg: NetanexConfig):
    """Name -> (shape, initialiser) of a fresh checkpoint: matrices N(0, 1/sqrt(fan-in)), weights of norms near one (those
    stored as the distance from one near zero), tables of different experts."""
    D = cfg.width
    lin = lambda n_out, n_in: ((n_out, n_in), Normal(n_in ** -0.5))
    near_zero = ((D,), Normal(0.1))
    out = {"embed": ((cfg.vocab, D), Normal(D ** -0.5, layout="table")), "embed.norm": near_zero, "final.norm": near_zero}
    for i, layer in enumerate(cfg.layers):
        if layer.owner != i:
            continue
        l, m, f = f"l{i}.", layer.mixer, layer.mlp
        out[l + "norm1"], out[l + "norm1b"] = near_zero, near_zero
        p, H = l + "mix.", m.heads
        if m.kind == "latent_attention":
            out.update({p + "q": lin(H * (m.dim + m.rot_dim), D), p + "dkv": lin(m.kv_rank + m.rot_dim, D),
                        p + "dkv.norm": ((m.kv_rank,), Ones(0.1)), p + "uk": lin(H * m.dim, m.kv_rank),
                        p + "uv": lin(H * m.vdim, m.kv_rank), p + "sink": ((H,), Normal(1.0)), p + "g": lin(H * m.vdim, D),
                        p + "o": lin(D, H * m.vdim)})
        else:
            maps = 2 if m.kind == "attention" else 1
            q, k, v = H * maps * m.dim, m.kv_heads * maps * m.dim, m.kv_heads * m.vdim
            for r, n in (("q", q), ("k", k), ("v", v)):
                out[p + r], out[p + r + ".b"] = lin(n, D), ((n,), Normal(0.3))
            out[p + "o"] = lin(D, H * m.vdim)
            if m.kind == "attention":
                out.update({p + "q.norm": ((m.dim,), Ones(0.1)), p + "k.norm": ((m.dim,), Ones(0.1)), p + "o.b": ((D,), Normal(0.3))})
                out.update({p + r: ((m.dim,), Normal(0.3 * m.dim ** -0.25)) for r in ("lq1", "lk1", "lq2", "lk2")})
            else:
                out.update({p + "q.norm": ((q,), Ones(0.1)), p + "k.norm": ((k,), Ones(0.1)), p + "g": lin(H, D)})
        if f is None:
            continue
        out[l + "norm2"], out[l + "norm2b"] = near_zero, near_zero
        p = l + "mlp."
        out[p + "table"] = ((cfg.vocab, f.top), DistinctRows(f.experts))
        for e in range(f.experts):
            e = f"{p}e{e}."
            out[e + "gate"], out[e + "up"], out[e + "down"] = lin(f.ff, D), lin(f.ff, D), lin(D, f.ff)
    return out


NETANEX = Architecture(name="Netanex", read_config=NetanexConfig.from_dict, plan=plan, checkpoint_tensors=checkpoint_tensors,
                       display_name="Netanex", created_by="")
register_architecture(NETANEX, "netanex")
