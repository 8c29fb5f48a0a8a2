"""Benolix as a ``ModelSpec``.

The embedding's rows times a constant start a float32 stream that is normed after every sum: a layer is
``x <- norm1(alpha x + mixer(x))``, then ``x <- norm2(alpha x + ff(x))`` where it has a feed-forward, with RMS norms
whose weight the checkpoint stores as its distance from one.  The mixer is attention over cached latents within a
window: queries are projected up from a normed latent of their own, a head's rotated part turns in neighbouring pairs,
and every entry of the concatenated heads is gated by a sigmoid.  A layer that names ``kv_from`` projects no latents: its
run reads the rows that layer's run cached, with queries, up-projections, window and gate of its own.  The feed-forward
is SiLU-gated and dense, or routed experts: scores are a softmax over experts and identity experts together, a correction
enters the choice only, the chosen scores are divided by their sum and scaled; an expert's gate and up rows are clamped.
A final norm of the same kind and an untied head.

Checkpoint names: ``embed``, ``l<i>.norm1`` / ``.norm2``, ``l<i>.mix.{dq,dq.norm,uq,dkv,dkv.norm,uk,uv,g,o}``,
``l<i>.mlp.{gate,up,down}`` or ``l<i>.mlp.{router,correction,e<n>.*}``, ``final.norm``, ``head``; matrices carry no
``.weight`` suffix.
"""

from __future__ import annotations

from ..config.model_config import BenolixConfig
from ..parts.base import PartChoice
from .model import LayerRun, ModelSpec

EXPERT_SLOPE = 1.702      # an expert's gate is g * sigmoid(1.702 g) ...
EXPERT_SHIFT = 1.0        # ... times its up row plus one
WEIGHT_EPS = 1e-20        # added to the sum that the chosen experts' scores are divided by


def _mixer(cfg: BenolixConfig, layer: dict) -> PartChoice:
    m = layer["mixer"]
    rope = PartChoice("scaled_rotary", {"dims": m["rot"]["dims"], "base": m["rot"]["base"]})
    return PartChoice("latent_attention", {
        "hidden_size": cfg.hidden_size, "num_heads": m["heads"], "head_dim": m["dim"], "rot_dim": m["rot_dim"],
        "value_dim": m["vdim"], "kv_rank": m["kv_rank"], "query_rank": m["q_rank"], "scale": m["scale"],
        "norm_eps": cfg.norm_eps, "position_encoding": rope, "gate": "entry",
        "window": (m.get("mask") or {}).get("size"), "own_keys": m.get("kv_from") is None})


def _feed_forward(cfg: BenolixConfig, layer: dict) -> PartChoice | None:
    mlp = layer.get("mlp")
    if mlp is None:
        return None
    if mlp["kind"] == "dense":
        return PartChoice("gated_mlp", {"hidden_size": cfg.hidden_size, "intermediate_size": mlp["ff"],
                                        "activation": "silu", "weight_suffix": "",
                                        "names": {"gate": "gate", "up": "up", "down": "down"}})
    router, expert = mlp["router"], mlp["expert"]
    scale = router.get("scale")
    return PartChoice("routed_experts", {
        "hidden_size": cfg.hidden_size, "expert_size": expert["ff"], "num_experts": router["experts"],
        "identity": router.get("identity") or 0, "top": router["top"], "activation": "silu", "limit": expert["limit"],
        "slope": EXPERT_SLOPE, "shift": EXPERT_SHIFT, "correction": True, "score": "softmax", "renormalize": True,
        "weight_eps": WEIGHT_EPS, "weight_scale": 1.0 if scale is None else scale})


def benolix_spec(cfg: BenolixConfig) -> ModelSpec:
    norm = PartChoice("rmsnorm", {"size": cfg.hidden_size, "eps": cfg.norm_eps, "weight_name": "", "one_plus": True})
    blocks = [PartChoice("normed_sum", {"mixer": _mixer(cfg, layer), "feed_forward": _feed_forward(cfg, layer),
                                        "norm": norm, "alpha": cfg.postln_alpha}) for layer in cfg.layers]
    return ModelSpec(
        vocab_size=cfg.vocab_size, hidden_size=cfg.hidden_size, blocks=blocks, final_norm=norm,
        tie_word_embeddings=False,
        embedding=PartChoice("scaled_f32_embedding", {"scale": cfg.embedding_scale, "weight_name": ""}),
        head=PartChoice("lm_head", {"weight_name": ""}),
        order=[LayerRun(i, reads_run=layer["mixer"].get("kv_from")) for i, layer in enumerate(cfg.layers)],
        max_positions=0, embedding_prefix="embed", layer_prefix="l{}", final_norm_prefix="final.norm", head_prefix="head")
