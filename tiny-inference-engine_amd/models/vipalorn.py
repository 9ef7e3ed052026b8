"""Vipalorn as a ModelSpec.

A decoder whose config.json lists its layers one by one. ``x = norm(embed[token])``; a layer norms the stream once,
both its sub-layers read those rows, and ``x += residual_mult * (mixer(h) + ff(h))`` (``parallel_residual``). Norms are
layer norms with a weight and no bias. A layer's mixer is

* ``latent_attention``: attention whose keys and values are made from one cached latent per token and whose rotated
  key part is shared by all heads; rotate-half pairs, every earlier key visible, one sigmoid gate a head
  (``latent_attention`` with ``gate_per`` head);
* ``delta``: a gated delta rule with one decay a head, short convolutions on q, k and v, and a silu gate on the normed
  heads' outputs (``gated_delta_rule`` with ``decay`` head and one-step projections).

The feed-forward is a routed mixture of gated experts whose gate and up sums are cut off at a limit,
``g sigmoid(1.702 g) (u + 1)``; the experts with the largest logits (with a bias) are chosen and weighted by the softmax
over the chosen logits (``routed_experts``). The head norms the wanted rows, multiplies by the embedding table and
scales the logits.

Tensor names: ``embed``, ``embed.norm``, ``final.norm``; ``l<i>.norm1``; latent attention
``l<i>.mix.{q,dkv,dkv.norm,uk,uv,g,o}``; delta ``l<i>.mix.{q,k,v,b,a,g,o,A_log,dt_bias,norm}`` with
``.{q,k,v}.conv``; ``l<i>.mlp.router{,.b}``, ``l<i>.mlp.e<j>.{gate,up,down}``.
"""

from __future__ import annotations

from ..config.registry import register_architecture
from ..config.vipalorn import VipalornConfig
from .spec import LayerCall, LayerSpec, ModelSpec, PartSpec

NAME = "Vipalorn"
GATE_SLOPE = 1.702         # an expert's gate is g sigmoid(GATE_SLOPE g)
UP_SHIFT = 1.0             # ... and meets u + UP_SHIFT


def build_vipalorn_spec(config: VipalornConfig) -> ModelSpec:
    width, eps = config.width, config.norm_eps

    def norm(name: str) -> PartSpec:
        return PartSpec("layer_norm", {"dim": width, "eps": eps, "weight": name})

    layers = []
    for i, layer in enumerate(config.layers):
        p = f"l{i}.mix."
        m = layer.mixer
        if layer.kind == "latent_attention":
            position = PartSpec("rope_yarn", {"head_dim": m.rot_dim, "theta": m.rotation.base, "scaling": None,
                                              "rotary_dim": m.rotation.dims, "pairing": "rotate_half"})
            mixer = PartSpec("latent_attention", {
                "hidden": width, "num_heads": m.heads, "head_dim": m.dim, "rope_dim": m.rot_dim, "value_dim": m.vdim,
                "kv_rank": m.kv_rank, "scale": m.scale, "window": None, "eps": eps, "position": position,
                "gate_per": "head",
                "names": {"q": p + "q", "dkv": p + "dkv", "dkv_norm": p + "dkv.norm", "uk": p + "uk", "uv": p + "uv",
                          "g": p + "g", "o": p + "o"},
            })
        else:
            mixer = PartSpec("gated_delta_rule", {
                "hidden": width, "heads": m.heads, "kv_heads": m.kv_heads, "key_dim": m.dim, "value_dim": m.vdim,
                "conv": m.conv, "eps": eps, "decay": "head", "gate_activation": "silu",
                "names": {**{k: p + k for k in ("q", "k", "v", "b", "a", "g", "o", "A_log", "dt_bias", "norm")},
                          "q_conv": p + "q.conv", "k_conv": p + "k.conv", "v_conv": p + "v.conv"},
            })
        feed_forward = None
        if layer.mlp is not None:
            f, r = f"l{i}.mlp.", layer.mlp
            feed_forward = PartSpec("routed_experts", {
                "hidden": width, "expert_intermediate": r.ff, "experts": r.experts, "top": r.top,
                "scoring": "softmax_chosen", "expert_activation": "clipped_gate",
                "activation_params": {"limit": r.limit, "slope": GATE_SLOPE, "shift": UP_SHIFT},
                "names": {"router": f + "router", "router_bias": f + "router.b", "correction": None,
                          **{k: [f"{f}e{e}.{k}" for e in range(r.experts)] for k in ("gate", "up", "down")}},
            })
        layers.append(LayerSpec(block=PartSpec("parallel_residual", {"hidden": width, "scale": config.residual_mult}),
                                mixer=mixer, feed_forward=feed_forward, norms={"pre": norm(f"l{i}.norm1")}))
    return ModelSpec(
        architecture=NAME,
        vocab_size=config.vocab,
        hidden_size=width,
        max_positions=config.max_positions,
        embedding=PartSpec("token_embedding", {"vocab": config.vocab, "hidden": width, "weight": "embed",
                                               "norm": norm("embed.norm")}),
        layers=tuple(layers),
        order=tuple(LayerCall(i) for i in range(len(layers))),
        head=PartSpec("lm_head", {"vocab": config.vocab, "hidden": width, "norm": norm("final.norm"),
                                  "weight": None, "tied_to": "embed", "logit_scale": config.logit_scale}),
    )


register_architecture(NAME, VipalornConfig.from_json, build_vipalorn_spec)
