"""Configuration of the Vabelorn decoder: layers with norms on their sublayers' outputs only, ``x <- x + norm1(mixer(x))``, ``x <- x +
norm2(ff(x))``, and after them a per-layer token input, ``x <- x + norm(proj(gelu_tanh(gate x) * e))`` with ``e`` the layer's slice of a second
token table; two kinds of mixer: ``wkv`` (time mixing with a matrix state, decays per token and key channel) and ``attention`` (grouped queries,
normed queries and keys, a rotation in pairs over the first dimensions of a head with YaRN scaling, normed values that are cached turned by
their position and whose sum is turned back, one added to the softmax's denominator); a gated dense feed-forward (silu), or none; the
output head is the embedding table times a factor.

``config.json`` keys: ``architecture`` (``"Vabelorn"``), ``vocab``, ``width``, ``norm.eps``, ``logit_scale`` (absent: 1), ``token_side.dim`` (absent: no
token inputs), ``max_positions`` (absent: 2**20) and ``layers``, one entry per layer: ``type``, ``mixer`` and ``mlp``.  Mixer keys: wkv ``heads``, ``dim``
(and ``decay_rank``, which only the random-weights mode reads: a checkpoint's tensors say their own); attention ``heads``, ``kv_heads``, ``dim``,
``vdim``, ``scale``, ``rot`` (``dims``, ``base``, ``scaling`` with ``factor``, ``original``, ``fast``, ``slow``; absent: no rotation of anything / plain
frequencies).  ``mlp``: ``kind`` ``dense`` with ``ff``, or null.  Tensor names: ``embed``, ``side.embed``, ``final.norm``, and below ``l<i>.``: ``norm1``,
``norm2``, ``mix.*``, ``mlp.gate``, ``mlp.up``, ``mlp.down``, ``side.gate``, ``side.proj``, ``side.norm``.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, ClassVar

from .base import (CappedAttentionSpec, ConfigError, ModelConfig, ModelSpec, OffsetRMSNormSpec, OutputNormBlockSpec, PairRotarySpec, RunEntry,
                   SwiGLUSpec, TokenSideSpec, TokenSideTable, WKVSpec)

MIXER_KEYS = {"wkv": ("heads", "dim"), "attention": ("heads", "kv_heads", "dim", "vdim", "scale")}
SCALING_KEYS = ("factor", "original", "fast", "slow")


def _positive_int(where: str, v) -> int:
    if not isinstance(v, int) or isinstance(v, bool) or v <= 0:
        raise ConfigError(f"Vabelorn: {where} must be a positive integer, got {v!r}")
    return v


def _number(where: str, v) -> float:
    if isinstance(v, bool) or not isinstance(v, (int, float)):
        raise ConfigError(f"Vabelorn: {where} must be a number, got {v!r}")
    return float(v)


@dataclass(frozen=True)
class VabelornConfig(ModelConfig):
    architecture: ClassVar[str] = "Vabelorn"

    vocab: int
    width: int
    layers: list
    norm: dict
    token_side: dict = field(default_factory=dict)
    logit_scale: float = 1.0
    max_positions: int = 1 << 20
    torch_dtype: str = ""

    # ------------------------------------------------------------------ checks
    def _check_rotation(self, where: str, m: dict) -> None:
        rot = m.get("rot")
        if rot is None:
            return
        if not isinstance(rot, dict) or "dims" not in rot or "base" not in rot:
            raise ConfigError(f"Vabelorn: {where}.rot needs 'dims' and 'base'")
        dims = _positive_int(f"{where}.rot.dims", rot["dims"])
        if dims % 2 or dims > m["dim"]:
            raise ConfigError(f"Vabelorn: {where}.rot.dims must be even and at most dim ({m['dim']}), got {dims}")
        if m["vdim"] % 2:
            raise ConfigError(f"Vabelorn: {where}: values of {m['vdim']} numbers cannot be turned in pairs")
        if not _number(f"{where}.rot.base", rot["base"]) > 0:
            raise ConfigError(f"Vabelorn: {where}.rot.base must be positive")
        scaling = rot.get("scaling")
        if scaling is not None:
            if not isinstance(scaling, dict) or any(k not in scaling for k in SCALING_KEYS):
                raise ConfigError(f"Vabelorn: {where}.rot.scaling needs {', '.join(SCALING_KEYS)}")
            if not all(_number(f"{where}.rot.scaling.{k}", scaling[k]) > 0 for k in SCALING_KEYS) or not rot["base"] > 1:
                raise ConfigError(f"Vabelorn: {where}.rot.scaling wants positive numbers (and a base above 1)")

    def validate(self) -> None:
        _positive_int("vocab", self.vocab)
        _positive_int("width", self.width)
        _positive_int("max_positions", self.max_positions)
        _number("logit_scale", self.logit_scale)
        if not isinstance(self.norm, dict) or not _number("norm.eps", self.norm.get("eps")) > 0:
            raise ConfigError("Vabelorn: norm.eps must be a positive number")
        if not isinstance(self.token_side, dict):
            raise ConfigError("Vabelorn: 'token_side' must be an object")
        if self.token_side:
            _positive_int("token_side.dim", self.token_side.get("dim"))
        if not isinstance(self.layers, (list, tuple)) or not self.layers:
            raise ConfigError("Vabelorn: 'layers' must be a non-empty list")
        for i, layer in enumerate(self.layers):
            kind = layer.get("type") if isinstance(layer, dict) else None
            if kind not in MIXER_KEYS:
                raise ConfigError(f"Vabelorn: layer {i} has mixer type {kind!r}; built: {', '.join(sorted(MIXER_KEYS))}")
            m, where = layer.get("mixer"), f"layer {i} mixer"
            missing = [k for k in MIXER_KEYS[kind] if not isinstance(m, dict) or k not in m]
            if missing:
                raise ConfigError(f"Vabelorn: layer {i} ({kind}) lacks mixer key(s): {', '.join(missing)}")
            for k in MIXER_KEYS[kind]:
                if k == "scale":
                    _number(f"{where}.scale", m[k])
                else:
                    _positive_int(f"{where}.{k}", m[k])
            if kind == "attention":
                if m["heads"] % m["kv_heads"]:
                    raise ConfigError(f"Vabelorn: {where}: {m['heads']} heads are not a multiple of {m['kv_heads']} key/value heads")
                self._check_rotation(where, m)
            elif "decay_rank" in m:
                _positive_int(f"{where}.decay_rank", m["decay_rank"])
            mlp = layer.get("mlp")
            if mlp is not None:
                if not isinstance(mlp, dict) or mlp.get("kind") != "dense":
                    raise ConfigError(f"Vabelorn: layer {i} has mlp kind {mlp.get('kind') if isinstance(mlp, dict) else mlp!r}; built: dense, or null")
                _positive_int(f"layer {i} mlp.ff", mlp.get("ff"))

    # ------------------------------------------------------------------ parts
    def _mixer(self, layer: dict):
        m, eps = layer["mixer"], float(self.norm["eps"])
        if layer["type"] == "wkv":
            return WKVSpec(hidden=self.width, heads=m["heads"], dim=m["dim"], vdim=m["dim"], decay_rank=int(m.get("decay_rank", 32)), norm_eps=eps)
        rot, position, values = m.get("rot"), None, None
        if rot is not None:
            scaling = rot.get("scaling")
            yarn = tuple(float(scaling[k]) for k in SCALING_KEYS) if scaling is not None else None
            position = PairRotarySpec(dims=rot["dims"], base=float(rot["base"]), yarn=yarn)
            values = PairRotarySpec(dims=m["vdim"], base=float(rot["base"]))            # the whole value, never scaled
        return CappedAttentionSpec(hidden=self.width, heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"], scale=float(m["scale"]),
                                   position=position, qk_norm=True, qk_norm_eps=eps, fixed_sink=0.0, value_norm=True, value_position=values)

    def to_spec(self) -> ModelSpec:
        eps = float(self.norm["eps"])
        norm = OffsetRMSNormSpec(dim=self.width, eps=eps, offset=0.0, weight_name="")
        side = TokenSideSpec(hidden=self.width, dim=self.token_side["dim"], eps=eps) if self.token_side else None
        blocks = []
        for layer in self.layers:
            mlp = layer.get("mlp")
            ffn = SwiGLUSpec(hidden=self.width, intermediate=mlp["ff"], gate_name="gate", up_name="up", down_name="down") if mlp is not None else None
            blocks.append(OutputNormBlockSpec(mixer=self._mixer(layer), ffn=ffn, mixer_norm=norm, ffn_norm=norm if ffn is not None else None, side=side,
                                              mixer_name="mix", ffn_name="mlp", mixer_norm_name="norm1", ffn_norm_name="norm2", side_name="side"))
        return ModelSpec(vocab_size=self.vocab, hidden=self.width, layers=tuple(blocks), order=tuple(RunEntry(layer=i) for i in range(len(blocks))),
                         final_norm=norm, tie_head=True, max_positions=self.max_positions, embed_name="embed", final_norm_name="final.norm",
                         head_name="head", logit_scale=float(self.logit_scale), weight_suffix="", layers_format="l{}",
                         token_side=TokenSideTable(name="side.embed", dim=self.token_side["dim"]) if self.token_side else None)

    def to_dict(self) -> dict[str, Any]:
        d = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": dict(self.norm),
             "logit_scale": self.logit_scale, "layers": [dict(layer) for layer in self.layers]}
        if self.token_side:
            d["token_side"] = dict(self.token_side)
        if self.max_positions != 1 << 20:
            d["max_positions"] = self.max_positions
        if self.torch_dtype:
            d["torch_dtype"] = self.torch_dtype
        return d
