"""Typed configuration of the Pekarax decoder, read from config.json.

Keys: ``architecture`` ("Pekarax"), ``vocab``, ``width``, ``norm.eps``, ``postln_alpha`` and ``layers``: a list whose entries
give ``type`` ("channel_delta", "gla" or "parallel"), ``mixer`` (the sizes and constants of that mixer) and ``mlp``: null or
{kind: "moe", router{experts, top, groups{count, keep} or absent, identity or absent, scale}, expert{ff, limit}}.  Mixers:
"channel_delta" {heads, kv_heads, dim, vdim, conv}; "gla" {heads, dim, vdim, tau}; "parallel" {left{heads, kv_heads, dim, vdim,
conv, rot{dims, base}, scale}, left_scale, right{heads, dim, vdim, gate_cap}, right_scale}.  Tensor names: ``embed``,
``final.norm``, ``head`` and per layer i ``l<i>.norm1`` / ``norm2``, ``l<i>.mix.*`` (``mix.left.*`` and ``mix.right.*``),
``l<i>.mlp.router`` / ``correction`` / ``e<j>.gate`` / ``.up`` / ``.down``.  The inner sizes of the low-rank products
(``a1``, ``g1``) are the tensors' own.

The design, layer by layer (x the float32 residual stream, r(z) = z / sqrt(mean(z^2) + eps)):
  x_0 = E[token]
  x <- r(alpha x + mixer(x)) (1 + w_1);   x <- r(alpha x + ff(x)) (1 + w_2)       (alpha: ``postln_alpha``)
  logits = W_head (r(x) (1 + w_final))
"channel_delta" is the delta rule with a decay per key channel, "gla" linear attention with one, "parallel" softmax attention
over convolved, rotated, normed keys beside a matrix memory with exponential gates (``parts/matrix_memory.py``,
``parts/span_attention.py``, ``parts/parallel.py``).  The routed feed-forward is ``parts/routed_experts.py``.
"""
from dataclasses import dataclass, field
from typing import List, Optional

from .registry import ConfigError, register_architecture
from .spec import LayerSpec, ModelSpec, PartSpec, default_schedule

DEFAULT_CONTEXT = 65536        # the design has no limit of its own; a serving cap (max_tokens) replaces this
EXPERT_SLOPE = 1.702           # the sigmoid's slope in the experts' bounded unit: fixed by the design
MIXERS = ("channel_delta", "gla", "parallel")


def _need(d, key: str, where: str):
    if not isinstance(d, dict) or d.get(key) is None:
        raise ConfigError("config.json lacks %s%s" % (where, key))
    return d[key]


@dataclass
class PekaraxLayer:
    kind: str
    mixer: dict                  # the mixer's sizes and constants as config.json gives them
    mlp: Optional[dict]          # None: the layer has no feed-forward


@dataclass
class PekaraxConfig:
    vocab_size: int
    hidden_size: int
    norm_eps: float
    residual_alpha: float
    layers: List[PekaraxLayer]
    context_cap: Optional[int] = None
    eos_token_id: List[int] = field(default_factory=list)
    bos_token_id: Optional[int] = None
    model_type: str = "Pekarax"

    @classmethod
    def from_dict(cls, cfg: dict, max_tokens: Optional[int] = None) -> "PekaraxConfig":
        raw_layers = _need(cfg, "layers", "")
        if not isinstance(raw_layers, list) or not raw_layers:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        layers = []
        for i, l in enumerate(raw_layers):
            where = "layers[%d]." % i
            kind = _need(l, "type", where)
            if kind not in MIXERS:
                raise ConfigError("%stype %r: this design has the mixers %s" % (where, kind, ", ".join(MIXERS)))
            m = _need(l, "mixer", where)
            if not isinstance(m, dict):
                raise ConfigError("%smixer must be an object" % where)
            mlp = l.get("mlp")
            if mlp is not None and not isinstance(mlp, dict):
                raise ConfigError("%smlp must be an object or null" % where)
            layers.append(PekaraxLayer(kind, dict(m), dict(mlp) if mlp else None))
        eos = cfg.get("eos_token_id", [])
        eos = [] if eos is None else ([eos] if isinstance(eos, int) else list(eos))
        out = cls(vocab_size=int(_need(cfg, "vocab", "")), hidden_size=int(_need(cfg, "width", "")),
                  norm_eps=float(_need(_need(cfg, "norm", ""), "eps", "norm.")), residual_alpha=float(_need(cfg, "postln_alpha", "")),
                  layers=layers, context_cap=int(max_tokens) if max_tokens is not None else None,
                  eos_token_id=[int(e) for e in eos], bos_token_id=cfg.get("bos_token_id"))
        out.validate()
        return out

    def validate(self) -> None:
        if self.vocab_size <= 0 or self.hidden_size <= 0:
            raise ConfigError("vocab and width must be positive")
        if not self.norm_eps > 0:
            raise ConfigError("norm.eps must be positive")
        if self.context_cap is not None and self.context_cap <= 0:
            raise ConfigError("max_tokens (the cap on the context) must be positive")
        for i, l in enumerate(self.layers):
            self._mixer_spec(i, l)          # names what is missing
            self._ffn_spec(i, l)

    @property
    def max_positions(self) -> int:
        return self.context_cap if self.context_cap is not None else DEFAULT_CONTEXT

    context_is_open = True      # positions are bounded by the serving cap or the cache pool only

    @property
    def default_dtype(self) -> str:
        return "bfloat16"

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    def to_dict(self) -> dict:
        return {"architecture": "Pekarax", "vocab": self.vocab_size, "width": self.hidden_size, "norm": {"eps": self.norm_eps},
                "postln_alpha": self.residual_alpha,
                "layers": [{"type": l.kind, "mixer": dict(l.mixer), "mlp": dict(l.mlp) if l.mlp else None} for l in self.layers]}

    def _mixer_spec(self, i: int, l: PekaraxLayer) -> PartSpec:
        d, eps, name, where = self.hidden_size, self.norm_eps, "l%d.mix." % i, "layers[%d].mixer." % i

        def sizes(m, where, *keys):
            out = {k: int(_need(m, k, where)) for k in keys}
            for k, v in out.items():
                if v <= 0:
                    raise ConfigError("%s%s must be positive (got %d)" % (where, k, v))
            return out

        def kv_heads(m, heads, where):
            g = int(m.get("kv_heads") or heads)
            if g <= 0 or heads % g:
                raise ConfigError("%sheads (%d) must be a multiple of kv_heads (%d)" % (where, heads, g))
            return g
        if l.kind == "channel_delta":
            s = sizes(l.mixer, where, "heads", "dim", "vdim", "conv")
            return PartSpec("gated_delta", name, {
                "hidden_size": d, "heads": s["heads"], "kv_heads": kv_heads(l.mixer, s["heads"], where), "key_dim": s["dim"],
                "value_dim": s["vdim"], "conv_taps": s["conv"], "norm_eps": eps})
        if l.kind == "gla":
            s = sizes(l.mixer, where, "heads", "dim", "vdim")
            return PartSpec("gated_linear_attention", name, {
                "hidden_size": d, "heads": s["heads"], "key_dim": s["dim"], "value_dim": s["vdim"],
                "tau": float(_need(l.mixer, "tau", where)), "norm_eps": eps})
        left, right = _need(l.mixer, "left", where), _need(l.mixer, "right", where)
        s, rot = sizes(left, where + "left.", "heads", "dim"), left.get("rot") or {}
        dims = int(rot.get("dims") or 0)
        attention = PartSpec("span_attention", name + "left.", {
            "hidden_size": d, "num_heads": s["heads"], "num_kv_heads": kv_heads(left, s["heads"], where + "left."), "key_dim": s["dim"],
            "value_dim": int(left.get("vdim") or s["dim"]), "softmax_scale": float(_need(left, "scale", where + "left.")),
            "qk_norm": "head", "qk_norm_weight": False, "qk_norm_eps": eps, "conv_taps": int(left.get("conv") or 0),
            "rot_dims": dims, "rot_base": float(_need(rot, "base", where + "left.rot.")) if dims else None})
        s = sizes(right, where + "right.", "heads", "dim", "vdim")
        memory = PartSpec("exponential_memory", name + "right.", {
            "hidden_size": d, "heads": s["heads"], "key_dim": s["dim"], "value_dim": s["vdim"],
            "gate_cap": float(_need(right, "gate_cap", where + "right.")), "norm_eps": eps})
        return PartSpec("parallel", name, {"branches": [(attention, float(_need(l.mixer, "left_scale", where))),
                                                        (memory, float(_need(l.mixer, "right_scale", where)))]})

    def _ffn_spec(self, i: int, l: PekaraxLayer) -> Optional[PartSpec]:
        if l.mlp is None:
            return None
        where = "layers[%d].mlp." % i
        kind = l.mlp.get("kind", "moe")
        if kind != "moe":
            raise ConfigError("%skind %r: this design's feed-forward is moe" % (where, kind))
        router, expert = _need(l.mlp, "router", where), _need(l.mlp, "expert", where)
        experts, top = int(_need(router, "experts", where + "router.")), int(_need(router, "top", where + "router."))
        identity = int(router.get("identity") or 0)
        groups = router.get("groups") or {"count": 1, "keep": 1}
        count, keep = int(_need(groups, "count", where + "router.groups.")), int(_need(groups, "keep", where + "router.groups."))
        ff, limit = int(_need(expert, "ff", where + "expert.")), float(_need(expert, "limit", where + "expert."))
        total = experts + identity
        if not (0 < top <= total) or experts <= 0 or identity < 0 or ff <= 0 or not limit > 0:
            raise ConfigError("%s: positive experts, 0 < top <= experts + identity, positive expert.ff and expert.limit" % where)
        if count <= 0 or total % count or not 0 < keep <= count or keep * (total // count) < top:
            raise ConfigError("%srouter.groups: %d router outputs in %d groups of which %d stay, %d chosen" % (where, total, count, keep, top))
        return PartSpec("routed_experts", "l%d.mlp." % i, {
            "hidden_size": self.hidden_size, "experts": experts, "top": top, "expert_size": ff, "scores": "softmax",
            "renormalize": True, "weight_on": "output", "correction": True, "groups": count, "group_keep": keep,
            "identity": identity, "scale": float(router.get("scale", 1.0)), "unit": "clamped", "limit": limit, "slope": EXPERT_SLOPE})

    def model_spec(self) -> ModelSpec:
        d, eps = self.hidden_size, self.norm_eps
        norm = lambda tensor: PartSpec("rmsnorm", "", {"size": d, "eps": eps, "tensor": tensor, "weight_offset": 1.0})
        layers = []
        for i, l in enumerate(self.layers):
            p = "l%d." % i
            ffn = self._ffn_spec(i, l)
            layers.append(LayerSpec(block=PartSpec("sum_norm_residual", p, {"alpha": self.residual_alpha}), mixer=self._mixer_spec(i, l),
                                    mixer_norm=norm(p + "norm1"), feed_forward=ffn,
                                    feed_forward_norm=None if ffn is None else norm(p + "norm2")))
        return ModelSpec(
            architecture=self.model_type, vocab_size=self.vocab_size, hidden_size=d, max_positions=self.max_positions,
            embedding=PartSpec("embedding", "embed.", {"vocab_size": self.vocab_size, "hidden_size": d, "tensor": "embed"}),
            layers=layers, schedule=default_schedule(len(layers)), final_norm=norm("final.norm"),
            head=PartSpec("lm_head", "head.", {"vocab_size": self.vocab_size, "hidden_size": d, "tensor": "head"}),
            eos_token_ids=list(self.eos_token_id), bos_token_id=self.bos_token_id)


register_architecture(["Pekarax", "pekarax"], PekaraxConfig)
