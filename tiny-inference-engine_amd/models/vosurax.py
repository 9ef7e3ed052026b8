"""Vosurax as a ModelSpec.

A decoder whose config.json lists its layers one by one, some of which run several times in a row with the same weights
(each run with a cache or state of its own); before every such pass a vector of the pass's own is added to the stream
(``add_vector`` before the pass's first layer). Every layer is the ``pre_norm`` arrangement with RMS norms whose weights
are stored around zero. A layer's mixer is

* ``parallel``: two mixers on the same rows, ``y = (N_l(left(h)) + N_r(right(h))) / 2`` with an RMS norm of its own behind
  each (``parallel`` with ``output_norms``). Left: grouped-query softmax attention in causal chunks without any position
  encoding, biased q, k and v, a per-head RMS norm on q and k, the heads' outputs multiplied by ``sigmoid(Wg h)``
  (``paged_attention`` with ``chunk`` and ``gate``). Right: a matrix memory with exponential gates (``matrix_memory``);
* ``retention``: linear attention with a fixed decay per head, rotated q and k, every head's output normed by itself and
  gated with ``silu(Wg h)`` (``decay_attention`` with ``position`` and ``norm_per`` head).

The feed-forward is ``down(gelu_tanh(up(h)))`` (``mlp``) or a routed mixture of SiLU-gated experts whose sigmoid scores
multiply the experts' input, beside an expert every token uses (``routed_experts`` with ``weight_on`` input). The head norms
the wanted rows and multiplies by a matrix of its own.

Tensor names: ``embed``, ``head``, ``final.norm``, ``loop.step``; ``l<i>.norm1``, ``l<i>.norm2``; parallel
``l<i>.mix.left.{q,k,v}{,.b}``, ``l<i>.mix.left.{g,o,q.norm,k.norm,out}``,
``l<i>.mix.right.{q,k,v,g,o,norm,i,i.b,f,f.b,out}``; retention ``l<i>.mix.{q,k,v,g,o}``; ``l<i>.mlp.{up,down}`` or
``l<i>.mlp.router``, ``l<i>.mlp.{e<j>,shared}.{gate,up,down}``.
"""

from __future__ import annotations

from ..config.registry import register_architecture
from ..config.vosurax import DenseFfConfig, VosuraxConfig
from .spec import LayerCall, LayerSpec, ModelSpec, PartSpec

NAME = "Vosurax"
BRANCH_SHARE = 0.5         # of each of the two mixers that run side by side


def _parallel(m, p: str, width: int, eps: float) -> PartSpec:
    left, right, lp, rp = m.left, m.right, p + "left.", p + "right."
    attention = PartSpec("paged_attention", {
        "hidden": width, "num_heads": left.heads, "num_kv_heads": left.kv_heads, "head_dim": left.dim,
        "value_dim": left.vdim, "scale": left.scale, "window": None, "chunk": left.chunk, "gate": lp + "g",
        "qk_norm": {"eps": eps, "q_weight": lp + "q.norm", "k_weight": lp + "k.norm"},
        "position": PartSpec("none"),
        "names": {k: lp + k for k in ("q", "k", "v", "o")},
        "bias": {k: f"{lp}{k}.b" for k in ("q", "k", "v")},
    })
    memory = PartSpec("matrix_memory", {
        "hidden": width, "heads": right.heads, "key_dim": right.dim, "value_dim": right.vdim, "gate_cap": right.gate_cap,
        "eps": eps,
        "names": {**{k: rp + k for k in ("q", "k", "v", "g", "o", "norm", "i", "f")}, "i_bias": rp + "i.b",
                  "f_bias": rp + "f.b"},
    })
    return PartSpec("parallel", {
        "hidden": width, "branches": [(attention, BRANCH_SHARE), (memory, BRANCH_SHARE)],
        "output_norms": {"eps": eps, "weights": [lp + "out", rp + "out"]}})


def _retention(m, p: str, width: int, eps: float) -> PartSpec:
    return PartSpec("decay_attention", {
        "hidden": width, "heads": m.heads, "key_dim": m.dim, "value_dim": m.vdim, "decay": list(m.decay),
        "activation": "none", "key_scale": m.dim ** -0.5, "eps": eps, "norm_per": "head", "gate_activation": "silu",
        "position": PartSpec("rope_yarn", {"head_dim": m.dim, "theta": m.rotation.base, "rotary_dim": m.rotation.dims,
                                           "pairing": "rotate_half", "scaling": None}),
        "names": {**{k: p + k for k in ("q", "k", "v", "g", "o")}, "norm": None},
    })


def _feed_forward(r, f: str, width: int) -> PartSpec:
    if isinstance(r, DenseFfConfig):
        return PartSpec("mlp", {"hidden": width, "intermediate": r.ff, "activation": "gelu_tanh",
                                "names": {"up": f + "up", "down": f + "down"}})
    parts = ("gate", "up", "down")
    shared = None if r.shared_ff is None else {"intermediate": r.shared_ff, "gate_logit": None,
                                               **{k: f"{f}shared.{k}" for k in parts}}
    return PartSpec("routed_experts", {
        "hidden": width, "expert_intermediate": r.ff, "experts": r.experts, "top": r.top, "scoring": "sigmoid",
        "weight_on": "input", "shared": shared,
        "names": {"router": f + "router", "correction": None,
                  **{k: [f"{f}e{e}.{k}" for e in range(r.experts)] for k in parts}}})


def build_vosurax_spec(config: VosuraxConfig) -> ModelSpec:
    width, eps = config.width, config.norm_eps

    def norm(name: str) -> PartSpec:
        return PartSpec("rms_norm", {"dim": width, "eps": eps, "weight": name, "one_plus": True})

    layers = []
    for i, layer in enumerate(config.layers):
        mixer = (_parallel if layer.kind == "parallel" else _retention)(layer.mixer, f"l{i}.mix.", width, eps)
        norms = {"pre_mixer": norm(f"l{i}.norm1")}
        feed_forward = None
        if layer.mlp is not None:
            feed_forward = _feed_forward(layer.mlp, f"l{i}.mlp.", width)
            norms["pre_feed_forward"] = norm(f"l{i}.norm2")
        layers.append(LayerSpec(block=PartSpec("pre_norm"), mixer=mixer, feed_forward=feed_forward, norms=norms))
    order = [LayerCall(i) for i in range(len(layers))]
    if config.loop is not None:
        loop, passes = config.loop, []
        for t in range(loop.times):
            step = PartSpec("add_vector", {"hidden": width, "table": "loop.step", "rows": loop.times, "row": t})
            passes += [LayerCall(i, before=step if i == loop.start else None) for i in range(loop.start, loop.stop)]
        order[loop.start:loop.stop] = passes
    return ModelSpec(
        architecture=NAME,
        vocab_size=config.vocab,
        hidden_size=width,
        max_positions=config.max_positions,
        embedding=PartSpec("token_embedding", {"vocab": config.vocab, "hidden": width, "weight": "embed"}),
        layers=tuple(layers),
        order=tuple(order),
        head=PartSpec("lm_head", {"vocab": config.vocab, "hidden": width, "norm": norm("final.norm"),
                                  "weight": "head", "tied_to": None}),
    )


register_architecture(NAME, VosuraxConfig.from_json, build_vosurax_spec)
