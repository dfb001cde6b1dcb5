"""Typed configuration of the Fokinex decoder, read from config.json.

Keys: ``architecture`` ("Fokinex"), ``vocab``, ``width``, ``norm.eps``, ``embedding.scale`` and ``layers``: a list whose entries give
``type`` ("latent_attention" or "parallel"), ``mixer`` (the sizes and constants of that mixer) and ``mlp``: null or {kind: "dense",
ff}.  Mixers: "latent_attention" {heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, mask{size}, rot{base, dims, scaling{factor,
original, fast, slow}}, kv_from}; "parallel" {left{heads, kv_heads, dim, vdim, scale, softcap, mask{size}}, left_scale, right{heads,
kv_heads, dim, vdim, conv}, right_scale}.  ``kv_from``, ``mask``, ``rot.scaling``, ``softcap`` and ``embedding`` may be absent, and ``q_rank`` (the
tensors then decide it).  Tensor
names: ``embed``, ``final.norm``, ``head`` and per layer i ``l<i>.norm1``, ``l<i>.mix.*`` (``mix.left.*`` and ``mix.right.*``),
``l<i>.mlp.gate`` / ``.up`` / ``.down``.

The design, layer by layer (x the float32 residual stream, r(z) = z / sqrt(mean(z^2) + eps)):
  x_0 = scale E[token]
  h = r(x) w;   x <- x + mixer(h) + W_down (silu(W_gate h) * (W_up h))        (one norm; the last term only with an ``mlp``)
  logits = W_head (r(x) w_final)
"latent_attention" is softmax attention through a latent with a window, a learned sink per head and stretched rotary wavelengths; with
``kv_from`` j the layer caches nothing and reads the rows of layer j (``parts/latent_attention.py``).  "parallel" is attention whose
values are its projected keys, with norms over whole rows, capped scores, a distance bias and an output gate, beside the delta
rule with one decay per head (``parts/span_attention.py``, ``parts/matrix_memory.py``, ``parts/parallel.py``).
"""
from dataclasses import dataclass, field
from typing import List, Optional

from .registry import ConfigError, register_architecture
from .spec import ExecEntry, LayerSpec, ModelSpec, PartSpec

DEFAULT_CONTEXT = 65536        # the design has no limit of its own; a serving cap (max_tokens) replaces this
SLOPE_EXPONENT = 8.0           # head h of H takes off 2^(-8 (h + 1) / H) per token of distance: fixed by the design
MIXERS = ("latent_attention", "parallel")


def _need(d, key: str, where: str):
    if not isinstance(d, dict) or d.get(key) is None:
        raise ConfigError("config.json lacks %s%s" % (where, key))
    return d[key]


def _sizes(m, where: str, *keys):
    out = {k: int(_need(m, k, where)) for k in keys}
    for k, v in out.items():
        if v <= 0:
            raise ConfigError("%s%s must be positive (got %d)" % (where, k, v))
    return out


def _kv_heads(m, heads: int, where: str) -> int:
    g = int(m.get("kv_heads") or heads)
    if g <= 0 or heads % g:
        raise ConfigError("%sheads (%d) must be a multiple of kv_heads (%d)" % (where, heads, g))
    return g


def _window(m, where: str) -> Optional[int]:
    size = (m.get("mask") or {}).get("size")
    if size is not None and int(size) <= 0:
        raise ConfigError("%smask.size must be positive (got %r)" % (where, size))
    return None if size is None else int(size)


@dataclass
class FokinexLayer:
    kind: str
    mixer: dict                  # the mixer's sizes and constants as config.json gives them
    ff: Optional[int]            # None: the layer has no feed-forward

    @property
    def kv_from(self) -> Optional[int]:
        return self.mixer.get("kv_from") if self.kind == "latent_attention" else None


@dataclass
class FokinexConfig:
    vocab_size: int
    hidden_size: int
    norm_eps: float
    layers: List[FokinexLayer]
    embedding_scale: float = 1.0
    context_cap: Optional[int] = None
    eos_token_id: List[int] = field(default_factory=list)
    bos_token_id: Optional[int] = None
    model_type: str = "Fokinex"

    @classmethod
    def from_dict(cls, cfg: dict, max_tokens: Optional[int] = None) -> "FokinexConfig":
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
            mlp, ff = l.get("mlp"), None
            if mlp:
                if not isinstance(mlp, dict) or mlp.get("kind", "dense") != "dense":
                    raise ConfigError("%smlp %r: this design's feed-forward is dense" % (where, mlp))
                ff = _sizes(mlp, where + "mlp.", "ff")["ff"]
            layers.append(FokinexLayer(kind, dict(m), ff))
        eos = cfg.get("eos_token_id", [])
        eos = [] if eos is None else ([eos] if isinstance(eos, int) else list(eos))
        out = cls(vocab_size=int(_need(cfg, "vocab", "")), hidden_size=int(_need(cfg, "width", "")),
                  norm_eps=float(_need(_need(cfg, "norm", ""), "eps", "norm.")), layers=layers,
                  embedding_scale=float((cfg.get("embedding") or {}).get("scale", 1.0)),
                  context_cap=int(max_tokens) if max_tokens is not None else None,
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
            j = l.kv_from
            if j is None:
                continue
            where = "layers[%d].mixer." % i
            if not isinstance(j, int) or not 0 <= j < i:
                raise ConfigError("%skv_from %r: an earlier layer is meant" % (where, j))
            src = self.layers[j]
            if src.kind != "latent_attention" or src.kv_from is not None:
                raise ConfigError("%skv_from %d: that layer caches no latent rows of its own" % (where, j))
            for key in ("kv_rank", "rot_dim", "rot"):
                if src.mixer.get(key) != l.mixer.get(key):
                    raise ConfigError("%skv_from %d: %s differs (%r, there %r)" % (where, j, key, l.mixer.get(key), src.mixer.get(key)))

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
        return {"architecture": "Fokinex", "vocab": self.vocab_size, "width": self.hidden_size, "norm": {"eps": self.norm_eps},
                "embedding": {"scale": self.embedding_scale},
                "layers": [{"type": l.kind, "mixer": dict(l.mixer), "mlp": {"kind": "dense", "ff": l.ff} if l.ff else None}
                           for l in self.layers]}

    def _mixer_spec(self, i: int, l: FokinexLayer) -> PartSpec:
        d, eps, name, where = self.hidden_size, self.norm_eps, "l%d.mix." % i, "layers[%d].mixer." % i
        if l.kind == "latent_attention":
            s = _sizes(l.mixer, where, "heads", "dim", "rot_dim", "vdim", "kv_rank")
            rot = _need(l.mixer, "rot", where)
            scaling = rot.get("scaling")
            if scaling:
                scaling = {k: float(_need(scaling, k, where + "rot.scaling.")) for k in ("factor", "original", "fast", "slow")}
            return PartSpec("latent_attention", name, {
                "hidden_size": d, "num_heads": s["heads"], "head_dim": s["dim"], "rot_dim": s["rot_dim"], "value_dim": s["vdim"],
                "q_rank": _sizes(l.mixer, where, "q_rank")["q_rank"] if l.mixer.get("q_rank") is not None else None, "kv_rank": s["kv_rank"], "softmax_scale": float(_need(l.mixer, "scale", where)),
                "rot_base": float(_need(rot, "base", where + "rot.")), "rot_dims": int(rot.get("dims") or s["rot_dim"]),
                "rot_scaling": scaling or None, "norm_eps": eps, "gate": False, "sink": True, "window": _window(l.mixer, where),
                "own_rows": l.kv_from is None})
        left, right = _need(l.mixer, "left", where), _need(l.mixer, "right", where)
        s = _sizes(left, where + "left.", "heads", "dim")
        if int(left.get("vdim") or s["dim"]) != s["dim"]:
            raise ConfigError("%sleft.vdim %r: the values are the keys, of %d entries" % (where, left.get("vdim"), s["dim"]))
        attention = PartSpec("span_attention", name + "left.", {
            "hidden_size": d, "num_heads": s["heads"], "num_kv_heads": _kv_heads(left, s["heads"], where + "left."), "key_dim": s["dim"],
            "value_dim": s["dim"], "softmax_scale": float(_need(left, "scale", where + "left.")), "window": _window(left, where + "left."),
            "qk_norm": "row", "qk_norm_eps": eps, "gate": True, "softcap": float(left["softcap"]) if left.get("softcap") else None,
            "values_from_keys": True,
            "distance_slopes": [2.0 ** (-SLOPE_EXPONENT * (h + 1) / s["heads"]) for h in range(s["heads"])]})
        s = _sizes(right, where + "right.", "heads", "dim", "vdim", "conv")
        memory = PartSpec("gated_delta", name + "right.", {
            "hidden_size": d, "heads": s["heads"], "kv_heads": _kv_heads(right, s["heads"], where + "right."), "key_dim": s["dim"],
            "value_dim": s["vdim"], "conv_taps": s["conv"], "norm_eps": eps, "decay": "head"})
        return PartSpec("parallel", name, {"branches": [(attention, float(_need(l.mixer, "left_scale", where))),
                                                        (memory, float(_need(l.mixer, "right_scale", where)))]})

    def model_spec(self) -> ModelSpec:
        d, eps = self.hidden_size, self.norm_eps
        norm = lambda tensor: PartSpec("rmsnorm", "", {"size": d, "eps": eps, "tensor": tensor})
        layers, schedule = [], []
        for i, l in enumerate(self.layers):
            p = "l%d." % i
            layers.append(LayerSpec(
                block=PartSpec("shared_norm_residual", p, {}), mixer=self._mixer_spec(i, l), mixer_norm=norm(p + "norm1"),
                feed_forward=None if l.ff is None else PartSpec("swiglu", p + "mlp.", {
                    "hidden_size": d, "intermediate_size": l.ff, "gate_name": "gate", "up_name": "up", "down_name": "down"})))
            schedule.append(ExecEntry(layer=i, cache=i if l.kv_from is None else l.kv_from, writes_cache=l.kv_from is None))
        return ModelSpec(
            architecture=self.model_type, vocab_size=self.vocab_size, hidden_size=d, max_positions=self.max_positions,
            embedding=PartSpec("embedding", "embed.", {"vocab_size": self.vocab_size, "hidden_size": d, "tensor": "embed",
                                                       "scale": self.embedding_scale}),
            layers=layers, schedule=schedule, final_norm=norm("final.norm"),
            head=PartSpec("lm_head", "head.", {"vocab_size": self.vocab_size, "hidden_size": d, "tensor": "head"}),
            eos_token_ids=list(self.eos_token_id), bos_token_id=self.bos_token_id)


register_architecture(["Fokinex", "fokinex"], FokinexConfig)
