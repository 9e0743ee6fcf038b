"""Configuration of the Tilalorn decoder: pre-norm layers whose branches enter the stream times a fixed factor, ``x <- x + m * mixer(norm1(x))``,
``x <- x + m * ff(norm2(x))``, every norm a root-mean-square norm whose weight vector is stored around zero; two kinds of mixer:
``latent_attention`` (one cached latent per token beside a rotated key part that all heads share, rotate-half layout, inside a window, the heads'
values gated number by number) and ``attention`` (grouped queries with biases and without positions, queries and keys of unit root mean square,
queries that grow with the logarithm of their position, capped scores, a gate per head; a layer may read the keys and values of an earlier
one); a feed-forward that is dense and gated (the tanh form of gelu), routed over gated experts (silu) that compete in groups, or absent; the
head is the embedding table.

``config.json`` keys: ``architecture`` (``"Tilalorn"``), ``vocab``, ``width``, ``norm.eps``, ``residual_mult`` (absent: 1), ``max_positions`` (absent:
2**20) and ``layers``, one entry per layer: ``type``, ``mixer`` and ``mlp``.  Mixer keys: latent_attention ``heads``, ``dim``, ``rot_dim``, ``vdim``,
``kv_rank``, ``scale``, ``rot`` (``dims``, ``base``), ``mask.size`` (absent: causal); attention ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, ``softcap``
(absent: no cap), ``q_temp`` (``coef``, ``every``; absent: none), ``kv_from`` (the index of the earlier attention layer whose keys and values it
reads; absent: its own).  ``mlp``: ``kind`` ``dense`` with ``ff``; ``kind`` ``moe`` with ``expert.ff`` and ``router`` (``experts``, ``top``, ``scale``, ``groups``
with ``count`` and ``keep``; absent: 1 / no groups); or null.  Tensor names: ``embed``, ``final.norm``, and below ``l<i>.``: ``norm1``, ``norm2``,
``mix.*``, ``mlp.*``.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, ClassVar

from .base import (CappedAttentionSpec, ConfigError, HalfRotarySpec, LatentAttentionSpec, ModelConfig, ModelSpec, OffsetRMSNormSpec,
                   RoutedExpertsSpec, RunEntry, ScaledBlockSpec, SwiGLUSpec)

MIXER_KEYS = {
    "latent_attention": ("heads", "dim", "rot_dim", "vdim", "kv_rank", "scale", "rot"),
    "attention": ("heads", "kv_heads", "dim", "vdim", "scale"),
}
SHARED_KEYS = ("kv_heads", "dim", "vdim")       # what a layer and the one whose keys and values it reads have alike


def _positive_int(where: str, v) -> int:
    if not isinstance(v, int) or isinstance(v, bool) or v <= 0:
        raise ConfigError(f"Tilalorn: {where} must be a positive integer, got {v!r}")
    return v


def _number(where: str, v) -> float:
    if isinstance(v, bool) or not isinstance(v, (int, float)):
        raise ConfigError(f"Tilalorn: {where} must be a number, got {v!r}")
    return float(v)


def _object(where: str, v, *keys: str) -> dict:
    if not isinstance(v, dict) or any(k not in v for k in keys):
        raise ConfigError(f"Tilalorn: {where} must be an object" + (f" with {', '.join(keys)}" if keys else ""))
    return v


@dataclass(frozen=True)
class TilalornConfig(ModelConfig):
    architecture: ClassVar[str] = "Tilalorn"

    vocab: int
    width: int
    layers: list
    norm: dict
    residual_mult: float = 1.0
    max_positions: int = 1 << 20
    torch_dtype: str = ""

    # ------------------------------------------------------------------ checks
    def _check_latent(self, where: str, m: dict) -> None:
        rot = _object(f"{where}.rot", m["rot"], "dims", "base")
        dims = _positive_int(f"{where}.rot.dims", rot["dims"])
        if dims % 2 or dims > m["rot_dim"]:
            raise ConfigError(f"Tilalorn: {where}.rot.dims must be even and at most rot_dim ({m['rot_dim']}), got {dims}")
        if not _number(f"{where}.rot.base", rot["base"]) > 0:
            raise ConfigError(f"Tilalorn: {where}.rot.base must be positive")
        if m.get("mask") is not None:
            _positive_int(f"{where}.mask.size", _object(f"{where}.mask", m["mask"], "size")["size"])

    def _check_attention(self, i: int, where: str, m: dict) -> None:
        if m["heads"] % m["kv_heads"]:
            raise ConfigError(f"Tilalorn: {where}: {m['heads']} heads are not a multiple of {m['kv_heads']} key/value heads")
        if m.get("softcap") is not None and not _number(f"{where}.softcap", m["softcap"]) > 0:
            raise ConfigError(f"Tilalorn: {where}.softcap must be positive")
        if m.get("q_temp") is not None:
            heat = _object(f"{where}.q_temp", m["q_temp"], "coef", "every")
            _number(f"{where}.q_temp.coef", heat["coef"])
            every = _number(f"{where}.q_temp.every", heat["every"])
            if every < 1 or every != int(every):
                raise ConfigError(f"Tilalorn: {where}.q_temp.every must be a whole number of positions, got {heat['every']!r}")
        source = m.get("kv_from")
        if source is None:
            return
        if not isinstance(source, int) or isinstance(source, bool) or not 0 <= source < i:
            raise ConfigError(f"Tilalorn: {where}.kv_from must name an earlier layer, got {source!r}")
        other = self.layers[source]
        if other.get("type") != "attention" or other["mixer"].get("kv_from") is not None:
            raise ConfigError(f"Tilalorn: {where}.kv_from names layer {source}, which has no keys and values of its own")
        for k in SHARED_KEYS:
            if other["mixer"][k] != m[k]:
                raise ConfigError(f"Tilalorn: {where}: {k} ({m[k]}) differs from that of layer {source} ({other['mixer'][k]}), whose keys and values it reads")

    def _check_mlp(self, where: str, mlp) -> None:
        if not isinstance(mlp, dict) or mlp.get("kind") not in ("dense", "moe"):
            raise ConfigError(f"Tilalorn: {where} has kind {mlp.get('kind') if isinstance(mlp, dict) else mlp!r}; built: dense, moe, or null")
        if mlp["kind"] == "dense":
            _positive_int(f"{where}.ff", mlp.get("ff"))
            return
        _positive_int(f"{where}.expert.ff", _object(f"{where}.expert", mlp.get("expert"), "ff")["ff"])
        router = _object(f"{where}.router", mlp.get("router"), "experts", "top")
        experts, top = _positive_int(f"{where}.router.experts", router["experts"]), _positive_int(f"{where}.router.top", router["top"])
        _number(f"{where}.router.scale", router.get("scale", 1.0))
        open_to_choice = experts
        if router.get("groups") is not None:
            groups = _object(f"{where}.router.groups", router["groups"], "count", "keep")
            count, keep = _positive_int(f"{where}.router.groups.count", groups["count"]), _positive_int(f"{where}.router.groups.keep", groups["keep"])
            if experts % count or keep > count:
                raise ConfigError(f"Tilalorn: {where}: {experts} experts in {count} groups of which {keep} are kept")
            open_to_choice = keep * (experts // count)
        if top > open_to_choice:
            raise ConfigError(f"Tilalorn: {where} picks {top} of {open_to_choice} experts")

    def validate(self) -> None:
        _positive_int("vocab", self.vocab)
        _positive_int("width", self.width)
        _positive_int("max_positions", self.max_positions)
        _number("residual_mult", self.residual_mult)
        if not isinstance(self.norm, dict) or not _number("norm.eps", self.norm.get("eps")) > 0:
            raise ConfigError("Tilalorn: norm.eps must be a positive number")
        if not isinstance(self.layers, (list, tuple)) or not self.layers:
            raise ConfigError("Tilalorn: 'layers' must be a non-empty list")
        for i, layer in enumerate(self.layers):
            kind = layer.get("type") if isinstance(layer, dict) else None
            if kind not in MIXER_KEYS:
                raise ConfigError(f"Tilalorn: layer {i} has mixer type {kind!r}; built: {', '.join(sorted(MIXER_KEYS))}")
            where, m = f"layer {i} mixer", layer.get("mixer")
            missing = [k for k in MIXER_KEYS[kind] if not isinstance(m, dict) or k not in m]
            if missing:
                raise ConfigError(f"Tilalorn: layer {i} ({kind}) lacks mixer key(s): {', '.join(missing)}")
            for k in MIXER_KEYS[kind]:
                if k == "scale":
                    _number(f"{where}.scale", m[k])
                elif k != "rot":
                    _positive_int(f"{where}.{k}", m[k])
            if kind == "latent_attention":
                self._check_latent(where, m)
            else:
                self._check_attention(i, where, m)
            if layer.get("mlp") is not None:
                self._check_mlp(f"layer {i} mlp", layer["mlp"])

    # ------------------------------------------------------------------ parts
    def _mixer(self, layer: dict):
        m, eps = layer["mixer"], float(self.norm["eps"])
        if layer["type"] == "latent_attention":
            return LatentAttentionSpec(hidden=self.width, heads=m["heads"], dim=m["dim"], rot_dim=m["rot_dim"], vdim=m["vdim"], kv_rank=m["kv_rank"],
                                       q_rank=0, scale=float(m["scale"]), norm_eps=eps, sink=False,
                                       position=HalfRotarySpec(dims=m["rot"]["dims"], base=float(m["rot"]["base"])),
                                       window=(m.get("mask") or {}).get("size"), gate_values=True)
        heat, cap = m.get("q_temp"), m.get("softcap")
        own = m.get("kv_from") is None
        return CappedAttentionSpec(hidden=self.width, heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"], scale=float(m["scale"]),
                                   softcap=float(cap) if cap is not None else None, qk_bias=True, v_bias=own, qk_unit_norm=True, qk_norm_eps=eps,
                                   query_heat=(float(heat["coef"]), int(heat["every"])) if heat is not None else None, gate=True, reads_cache=not own)

    def _ffn(self, layer: dict):
        mlp = layer.get("mlp")
        if mlp is None:
            return None
        if mlp["kind"] == "dense":
            return SwiGLUSpec(hidden=self.width, intermediate=mlp["ff"], activation="gelu_tanh", gate_name="gate", up_name="up", down_name="down")
        router = mlp["router"]
        groups = router.get("groups")
        return RoutedExpertsSpec(hidden=self.width, intermediate=mlp["expert"]["ff"], experts=router["experts"], top=router["top"], activation="silu",
                                 router_bias=False, gated=True, scores="all", weight_scale=float(router.get("scale", 1.0)),
                                 groups=(groups["count"], groups["keep"]) if groups is not None else None)

    def to_spec(self) -> ModelSpec:
        norm = OffsetRMSNormSpec(dim=self.width, eps=float(self.norm["eps"]), offset=1.0, weight_name="")
        blocks, order = [], []
        for i, layer in enumerate(self.layers):
            ffn = self._ffn(layer)
            blocks.append(ScaledBlockSpec(mixer=self._mixer(layer), ffn=ffn, mixer_norm=norm, ffn_norm=norm if ffn is not None else None,
                                          mixer_name="mix", ffn_name="mlp", mixer_norm_name="norm1", ffn_norm_name="norm2",
                                          branch_gain=float(self.residual_mult)))
            order.append(RunEntry(layer=i, cache_of=layer["mixer"].get("kv_from")))
        return ModelSpec(vocab_size=self.vocab, hidden=self.width, layers=tuple(blocks), order=tuple(order), final_norm=norm, tie_head=True,
                         max_positions=self.max_positions, embed_name="embed", final_norm_name="final.norm", head_name="head", weight_suffix="",
                         layers_format="l{}")

    def to_dict(self) -> dict[str, Any]:
        d = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": dict(self.norm),
             "residual_mult": self.residual_mult, "layers": [dict(layer) for layer in self.layers]}
        if self.max_positions != 1 << 20:
            d["max_positions"] = self.max_positions
        if self.torch_dtype:
            d["torch_dtype"] = self.torch_dtype
        return d
