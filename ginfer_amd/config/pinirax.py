"""Typed configuration of the Pinirax decoder, read from its own config.json keys.

config.json names the architecture under `architecture` and gives: `vocab`, `width`, `norm.eps`, `embedding.scale` and `layers`, a
list whose entries name the mixer (`type`), its sizes (`mixer`) and the feed-forward (`mlp`, or null for a layer without one):

  type "parallel"   mixer: left = {heads, kv_heads, dim, vdim, scale, optionally softcap, optionally mask = {size}: a window},
                    right = {heads, kv_heads, dim, vdim, conv}, left_scale, right_scale
  type "mamba2"     mixer: heads, vdim, state, groups, norm_groups, conv
  mlp               {kind: "moe", router: {experts, top, optionally identity}, expert: {ff}}

Layers may differ from one another in every size.  What the design fixes (no key of config.json): gains of the norms around the
sublayers are stored around zero; the left mixer has biases on q, k and v, a norm per head of q and k with plain gains, a gate per
head and no rotation; the right mixer is a gated delta rule; the router takes a softmax over all experts, chooses by it plus a
correction and does not normalise the chosen weights; the experts gate with silu.
"""
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from .registry import register_architecture, ConfigError
from .spec import PartSpec, LayerSpec, ScheduleEntry, ModelSpec
from .potupel import _int, _number

NORM_GAIN_OFFSET = 1.0
UNIT_EPS = 1e-6                  # under the root that makes q and k of the delta rule unit vectors
POSITION_BASE = 10000.0
# positions are counted in 32-bit floats where angles are made
MAX_POSITIONS = 1 << 20
MIXER_TYPES = ("parallel", "mamba2")

# how the checkpoints spell things: layer i is "l<i>"; the output norms' tensors stand in the layer itself (l<i>.norm1b), so
# their role is spelt "" and the part is told the tensor's name
LAYER_TENSOR_NAMES = dict(mixer="mix", feed_forward="mlp", mixer_norm="norm1", feed_forward_norm="norm2",
                          mixer_out_norm="", feed_forward_out_norm="")
MODEL_TENSOR_NAMES = dict(embedding="embed", final_norm="final.norm", head="head")


@dataclass
class PiniraxLayer:
    type: str
    mixer: Dict[str, Any]
    mlp: Optional[Dict[str, Any]]


def _grouped(m, heads, groups, where):
    if m[heads] % m[groups]:
        raise ConfigError("config.json: %s: %s %d is not a multiple of %s %d" % (where, heads, m[heads], groups, m[groups]))


def _read_mixer(kind, m, where):
    if not isinstance(m, dict):
        raise ConfigError("config.json: %s has no mixer sizes" % where)
    if kind == "mamba2":
        out = {k: _int(m, k, where + " mixer") for k in ("heads", "vdim", "state", "groups", "norm_groups", "conv")}
        _grouped(out, "heads", "groups", where)
        if (out["heads"] * out["vdim"]) % out["norm_groups"]:
            raise ConfigError("config.json: %s: heads * vdim %d is not a multiple of norm_groups %d"
                              % (where, out["heads"] * out["vdim"], out["norm_groups"]))
        return out
    sides = {}
    for side in ("left", "right"):
        s = m.get(side)
        if not isinstance(s, dict):
            raise ConfigError("config.json: %s has no %s mixer" % (where, side))
        at = "%s %s" % (where, side)
        sides[side] = {k: _int(s, k, at) for k in ("heads", "kv_heads", "dim", "vdim") + (("conv",) if side == "right" else ())}
        _grouped(sides[side], "heads", "kv_heads", at)
        if side == "left":
            sides[side]["scale"] = _number(s, "scale", at)
            sides[side]["softcap"] = None if s.get("softcap") is None else _number(s, "softcap", at, positive=True)
            sides[side]["mask"] = None if s.get("mask") is None else _int(s["mask"], "size", at + " mask")
    return dict(sides, left_scale=_number(m, "left_scale", where + " mixer"), right_scale=_number(m, "right_scale", where + " mixer"))


def _read_mlp(mlp, where):
    if mlp is None:
        return None
    kind = mlp.get("kind") if isinstance(mlp, dict) else None
    if kind != "moe":
        raise ConfigError("config.json: %s has the unknown feed-forward kind %r (known: moe)" % (where, kind))
    router = mlp.get("router")
    r = dict(experts=_int(router, "experts", where + " mlp router"), top=_int(router, "top", where + " mlp router"),
             identity=_int(router, "identity", where + " mlp router", minimum=0) if "identity" in router else 0)
    if r["top"] > r["experts"] + r["identity"]:
        raise ConfigError("config.json: %s mlp router: top %d of %d experts" % (where, r["top"], r["experts"] + r["identity"]))
    return dict(kind="moe", router=r, expert=dict(ff=_int(mlp.get("expert"), "ff", where + " mlp expert")))


@register_architecture("Pinirax", "pinirax")
@dataclass
class PiniraxConfig:
    vocab: int
    width: int
    eps: float
    embedding_scale: float
    layers: List[PiniraxLayer] = field(default_factory=list)
    eos_token_ids: List[int] = field(default_factory=list)

    architecture = "Pinirax"

    @classmethod
    def from_dict(cls, d):
        missing = [k for k in ("vocab", "width", "norm", "embedding", "layers") if k not in d]
        if missing:
            raise ConfigError("config.json lacks required key(s): %s" % ", ".join(missing))
        if not isinstance(d["layers"], list) or not d["layers"]:
            raise ConfigError("config.json: 'layers' must be a list with at least one layer")
        layers = []
        for i, l in enumerate(d["layers"]):
            where = "layer %d" % i
            kind = l.get("type") if isinstance(l, dict) else l
            if kind not in MIXER_TYPES:
                raise ConfigError("config.json: %s has the unknown mixer type %r (known: %s)" % (where, kind, ", ".join(MIXER_TYPES)))
            layers.append(PiniraxLayer(kind, _read_mixer(kind, l.get("mixer"), where), _read_mlp(l.get("mlp"), where)))
        eos = d.get("eos_token_id")
        eos = [] if eos is None else ([int(e) for e in eos] if isinstance(eos, (list, tuple)) else [int(eos)])
        return cls(vocab=_int(d, "vocab", ""), width=_int(d, "width", ""), eps=_number(d["norm"], "eps", "norm", positive=True),
                   embedding_scale=_number(d["embedding"], "scale", "embedding"), layers=layers, eos_token_ids=eos)

    def to_dict(self):
        def mixer(l):
            m = dict(l.mixer)
            if l.type == "parallel":
                left = dict(m["left"])
                mask, cap = left.pop("mask"), left.pop("softcap")
                if mask is not None:
                    left["mask"] = dict(size=mask)
                if cap is not None:
                    left["softcap"] = cap
                m.update(left=left, right=dict(m["right"]))
            return m
        d = dict(architecture=self.architecture, vocab=self.vocab, width=self.width, norm=dict(eps=self.eps),
                 embedding=dict(scale=self.embedding_scale),
                 layers=[dict(type=l.type, mixer=mixer(l),
                              mlp=None if l.mlp is None else dict(kind="moe", router=dict(l.mlp["router"]), expert=dict(l.mlp["expert"])))
                         for l in self.layers])
        if self.eos_token_ids:
            d["eos_token_id"] = self.eos_token_ids[0] if len(self.eos_token_ids) == 1 else list(self.eos_token_ids)
        return d

    def _mixer(self, l):
        m, W = l.mixer, self.width
        if l.type == "mamba2":
            return PartSpec("mamba2", dict(hidden_size=W, num_heads=m["heads"], value_dim=m["vdim"], state_size=m["state"], groups=m["groups"],
                                           norm_groups=m["norm_groups"], taps=m["conv"], eps=self.eps))
        a, r = m["left"], m["right"]
        left = PartSpec("conv_attention", dict(
            hidden_size=W, num_heads=a["heads"], num_kv_heads=a["kv_heads"], head_dim=a["dim"], value_dim=a["vdim"], scale=a["scale"],
            sink=None, window=a["mask"], bias=True, out_bias=False, head_norm_eps=self.eps, soft_cap=a["softcap"], head_gate=True))
        right = PartSpec("gated_delta", dict(hidden_size=W, num_heads=r["heads"], num_kv_heads=r["kv_heads"], key_dim=r["dim"],
                                             value_dim=r["vdim"], taps=r["conv"], eps=self.eps, unit_eps=UNIT_EPS))
        return PartSpec("parallel_sum", dict(branches=[left, right], names=["left", "right"], scales=[m["left_scale"], m["right_scale"]]))

    def model_spec(self):
        W = self.width

        def norm():
            return PartSpec("rmsnorm", dict(size=W, eps=self.eps, gain_offset=NORM_GAIN_OFFSET, weight_name=""))

        def out_norm(name):
            return PartSpec("scaled_output_rmsnorm", dict(size=W, eps=self.eps, gain_offset=NORM_GAIN_OFFSET, gain_name=name,
                                                          scale_name=None))
        layers = []
        for i, l in enumerate(self.layers):
            parts = dict(mixer=self._mixer(l), mixer_norm=norm(), mixer_out_norm=out_norm("norm1b"))
            if l.mlp is not None:
                r = l.mlp["router"]
                parts.update(
                    feed_forward_norm=norm(), feed_forward_out_norm=out_norm("norm2b"),
                    feed_forward=PartSpec("routed_glu", dict(
                        hidden_size=W, num_experts=r["experts"], top_k=r["top"], expert_size=l.mlp["expert"]["ff"], router_bias=False,
                        scoring="softmax", correction=True, normalise=False, identity=r["identity"])))
            layers.append(LayerSpec(prefix="l%d" % i, parts=parts, arrangement="sandwich", names=dict(LAYER_TENSOR_NAMES)))
        spec = ModelSpec(
            hidden_size=W, vocab_size=self.vocab, layers=layers, schedule=[ScheduleEntry(i) for i in range(len(layers))],
            embedding=PartSpec("sinusoidal_scaled", dict(vocab_size=self.vocab, hidden_size=W, scale=self.embedding_scale,
                                                         base=POSITION_BASE)),
            final_norm=norm(),
            head=PartSpec("lm_head", dict(vocab_size=self.vocab, hidden_size=W, tied=False, weight_name="")),
            max_positions=MAX_POSITIONS, eos_token_ids=list(self.eos_token_ids), names=dict(MODEL_TENSOR_NAMES))
        spec.validate()
        return spec
