"""The Dudatar decoder as a model spec.

A list of layers with one norm each, whose mixer and feed-forward read that norm's result side by side:

    h = layernorm(x);  x += mixer(h) + ff(h)        (layers without a feed-forward: the mixer's branch alone)

* a run of layers (``loop``) is repeated with the same weights: its blocks stand several times in the run order,
  every time with a cache entry and states of its own, and every pass begins with a junction,
  x <- W [x; x0] + step[pass] (``parts/junction.py``);
* mixer ``parallel`` (``parts/linear_attention.py``, ``side_by_side``): grouped-query attention whose queries and keys
  are rotated, then divided by their root mean square a head, with a sigmoid output gate of one number a head
  (``parts/attention.py``), beside retention, linear attention with a constant decay a head; the two results are
  RMS-normed over the width and averaged;
* mixer ``gla``: gated linear attention, a decay per head and key channel;
* norms: layer norm with a weight and no bias (``parts/norm.py``);
* feed-forward: gated by the hyperbolic-tangent form of GELU (``parts/ffn.py``);
* logits: the model's norm, the head's own matrix, then cap * tanh(logits / cap).

Tensor names: ``embed``, ``head``, ``final.norm``, ``loop.in``, ``loop.step``, and per layer i ``l<i>.norm1``,
``l<i>.mix.<role>`` (``l<i>.mix.left.<role>``, ``l<i>.mix.right.<role>``), ``l<i>.mlp.<role>``.
"""
from __future__ import annotations

from ..config.dudatar import DudatarConfig, ParallelConfig
from ..config.registry import register_architecture
from ..parts.attention import HEAD_GATE, attention_spec
from ..parts.block import parallel_block_spec
from ..parts.embedding import head_spec, positional_embedding_spec
from ..parts.ffn import gated_ffn_spec
from ..parts.junction import mix_embedding_spec
from ..parts.linear_attention import gated_linear_attention_spec, retention_spec, side_by_side_spec
from ..parts.norm import layernorm_spec
from ..parts.position import rope_spec, stretched_frequencies
from ..parts.spec import ModelSpec, OrderEntry, PartSpec

ATTENTION_NAMES = {"q_weight": "q", "k_weight": "k", "v_weight": "v", "o_weight": "o", "g_weight": "g"}


def _rotation(rot, dim: int) -> PartSpec:
    if not rot.dims:
        return PartSpec("position", "none")
    return rope_spec(dim, rot.base, rot_dims=rot.dims, frequencies=stretched_frequencies(rot.dims, rot.base)[0])


def build_spec(cfg: DudatarConfig) -> ModelSpec:
    d, eps = cfg.width, cfg.norm_eps
    blocks, keeps = [], []
    for i, layer in enumerate(cfg.layers):
        p, mx = f"l{i}.", layer.mixer
        keeps.append(isinstance(mx, ParallelConfig))
        if isinstance(mx, ParallelConfig):
            a, b, mp = mx.left, mx.right, p + "mix."
            mixer = side_by_side_spec(
                attention_spec(mp + "left.", d, a.heads, a.kv_heads, a.dim, _rotation(a.rot, a.dim), scale=a.scale, qkv_bias=False,
                               v_dim=a.vdim, qk_norm=True, qk_norm_eps=eps, qk_norm_weight=False, out_gate=HEAD_GATE,
                               names=ATTENTION_NAMES, given_input=True),
                retention_spec(mp + "right.", d, b.heads, b.dim, b.vdim, b.decay, eps, _rotation(b.rot, b.dim), given_input=True),
                d, eps, mp + "left.out", mp + "right.out")
        else:
            mixer = gated_linear_attention_spec(p + "mix.", d, mx.heads, mx.dim, mx.vdim, mx.tau, eps, rank=mx.rank)
        ffn = None
        if layer.mlp is not None:
            ffn = gated_ffn_spec(p + "mlp.", d, layer.mlp.ff, "gelu_tanh", names=("gate", "up", "down"))
        blocks.append(parallel_block_spec(layernorm_spec(p + "norm1", d, eps), mixer, None, ffn))
    # the run order: (layer, the pass it begins)
    n, loop, junctions = len(blocks), cfg.loop, []
    runs = [(i, None) for i in range(n)]
    if loop is not None:
        junctions.append(mix_embedding_spec("loop.in", "loop.step", d, loop.times))
        runs = [(i, None) for i in range(loop.start)]
        for turn in range(loop.times):
            runs += [(i, turn if i == loop.start else None) for i in range(loop.start, loop.stop)]
        runs += [(i, None) for i in range(loop.stop, n)]
    order = [OrderEntry(block=i, cache=k if keeps[i] else None, junction=None if turn is None else 0, turn=turn or 0)
             for k, (i, turn) in enumerate(runs)]
    spec = ModelSpec(
        architecture=cfg.architecture, width=d, vocab=cfg.vocab,
        embedding=positional_embedding_spec("embed", cfg.vocab, d),
        blocks=blocks, order=order, junctions=junctions,
        final_norm=layernorm_spec("final.norm", d, eps),
        head=head_spec("head", cfg.vocab, d, softcap=cfg.logit_softcap),
        max_positions=0,
        stop_tokens=tuple(cfg.eos_token_ids),
    )
    spec.validate()
    return spec


register_architecture("Dudatar", DudatarConfig, build_spec)
