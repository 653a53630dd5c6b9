"""The Nidasun decoder as a model spec.

A list of layers over a residual of several streams that mix (hyper-connections, ``parts/block.py``, ``streams``): every
sublayer, mixer and feed-forward, reads a weighted sum of the streams through an RMS norm, and its result joins all of
them while they are mixed.  A run of layers (``loop``) is repeated with the same weights: its blocks stand several times
in the run order, every time with a cache entry and states of its own; nothing stands between the passes.

* mixer ``attention`` (``parts/attention.py``): grouped-query attention with biases on all four products, rotate-half
  rotation of the first ``rot.dims`` numbers, keys of the position's own chunk only, a sink whose score is a number of
  the head's own;
* mixer ``lightning`` (``parts/linear_attention.py``): linear attention with a constant decay a head on activated
  queries, keys and values, its heads normed together and gated;
* mixer ``parallel`` (``side_by_side``): attention whose queries and keys are normed over the whole projection, over a
  window of keys, with every frequency divided by a factor, beside a gated linear recurrence behind a short convolution
  (``parts/recurrent.py``, ``gated_lru``); the two results are added with a multiplier each;
* feed-forward ``dense``: W_down max(W_up h, 0)^2 (``parts/ffn.py``); ``moe``: gated silu experts chosen by corrected
  sigmoid scores within the best groups (``parts/moe.py``);
* logits: the model's norm of the streams' sum, the head's own matrix.

Tensor names: ``embed``, ``head``, ``final.norm``, and per layer i ``l<i>.norm1``, ``l<i>.norm2``, ``l<i>.hc1.<in|out|mix>``,
``l<i>.hc2.<in|out|mix>``, ``l<i>.mix.<role>`` (``l<i>.mix.left.<role>``, ``l<i>.mix.right.<role>``), ``l<i>.mlp.<role>``.
"""
from __future__ import annotations

from ..config.nidasun import AttentionConfig, LightningConfig, MoEFFConfig, NidasunConfig
from ..config.registry import register_architecture
from ..parts.attention import ROW_NORM, attention_spec
from ..parts.block import streams_block_spec
from ..parts.embedding import head_spec, streams_embedding_spec
from ..parts.ffn import dense_ffn_spec
from ..parts.linear_attention import lightning_spec, side_by_side_spec
from ..parts.moe import moe_ffn_spec
from ..parts.norm import rmsnorm_spec, streams_norm_spec
from ..parts.position import rope_spec, stretched_frequencies
from ..parts.recurrent import gated_lru_spec
from ..parts.spec import ModelSpec, OrderEntry, PartSpec

ATTENTION_NAMES = {"q_weight": "q", "k_weight": "k", "v_weight": "v", "o_weight": "o", "q_bias": "q.b", "k_bias": "k.b",
                   "v_bias": "v.b", "o_bias": "o.b", "q_norm": "q.norm", "k_norm": "k.norm", "sink": "sink"}


def _rotation(rot, dim: int) -> PartSpec:
    if not rot.dims:
        return PartSpec("position", "none")
    frequencies = stretched_frequencies(rot.dims, rot.base, "linear" if rot.factor else None, rot.factor or 1.0)[0]
    return rope_spec(dim, rot.base, rot_dims=rot.dims, frequencies=frequencies)


def build_spec(cfg: NidasunConfig) -> ModelSpec:
    d, eps, S = cfg.width, cfg.norm_eps, cfg.streams
    blocks, keeps, ignorable = [], [], []
    for i, layer in enumerate(cfg.layers):
        p, m = f"l{i}.", layer.mixer
        mp = p + "mix."
        keeps.append(not isinstance(m, LightningConfig))
        if isinstance(m, AttentionConfig):
            mixer = attention_spec(mp, d, m.heads, m.kv_heads, m.dim, _rotation(m.rot, m.dim), scale=m.scale, qkv_bias=True, out_bias=True,
                                   v_dim=m.vdim, sink=True, sink_scores=True, chunk=m.mask, names=ATTENTION_NAMES)
        elif isinstance(m, LightningConfig):
            mixer = lightning_spec(mp, d, m.heads, m.dim, m.vdim, m.decay, eps)
        else:
            a, b = m.left, m.right
            mixer = side_by_side_spec(
                attention_spec(mp + "left.", d, a.heads, a.kv_heads, a.dim, _rotation(a.rot, a.dim), window=a.mask, scale=a.scale,
                               qkv_bias=False, v_dim=a.vdim, qk_norm=ROW_NORM, qk_norm_eps=eps, names=ATTENTION_NAMES, given_input=True),
                gated_lru_spec(mp + "right.", d, b.width, b.blocks, b.conv, given_input=True),
                d, weight=(m.left_scale, m.right_scale))
        ffn = None
        f = layer.mlp
        if isinstance(f, MoEFFConfig):
            ffn = moe_ffn_spec(p + "mlp.", d, f.experts, f.top, f.ff, 0.0, activation="silu", router_score="sigmoid_corrected",
                               router_scale=f.scale, groups=f.groups, keep_groups=f.keep)
        elif f is not None:
            ffn = dense_ffn_spec(p + "mlp.up", p + "mlp.down", d, f.ff, "relu_sq")
        numbers = [{role: f"{p}hc{q}.{role}" for role in ("in", "out", "mix")} for q in (1, 2)]
        if ffn is None:
            ignorable += [p + "norm2", *numbers[1].values()]
        blocks.append(streams_block_spec(S, rmsnorm_spec(p + "norm1", d, eps), mixer, numbers[0],
                                         None if ffn is None else rmsnorm_spec(p + "norm2", d, eps), ffn, numbers[1]))
    n, loop = len(blocks), cfg.loop
    runs = list(range(n))
    if loop is not None:
        runs = list(range(loop.start)) + list(range(loop.start, loop.stop)) * loop.times + list(range(loop.stop, n))
    order = [OrderEntry(block=i, cache=k if keeps[i] else None) for k, i in enumerate(runs)]
    spec = ModelSpec(
        architecture=cfg.architecture, width=d, vocab=cfg.vocab,
        embedding=streams_embedding_spec("embed", cfg.vocab, d, S),
        blocks=blocks, order=order,
        final_norm=streams_norm_spec("final.norm", d, S, eps),
        head=head_spec("head", cfg.vocab, d),
        max_positions=0,
        stop_tokens=tuple(cfg.eos_token_ids),
        ignorable_tensors=tuple(ignorable),
    )
    spec.validate()
    return spec


register_architecture("Nidasun", NidasunConfig, build_spec)
