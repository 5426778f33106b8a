"""Typed configuration of the Derosun decoder, read from config.json's own keys.

config.json: ``architecture`` ("Derosun"), ``vocab``, ``width``, ``norm.eps``, ``postln_alpha``, ``embedding.scale`` and ``layers``, a
list whose entries give ``type`` (the mixer: ``latent_attention``, ``mlstm`` or ``attention``), ``mixer`` (its sizes and
constants) and ``mlp`` (``{"kind": "dense", "ff": n}`` or null).
Tensor names: ``embed``, ``l<i>.norm1|norm2``, ``l<i>.mix.*``, ``l<i>.mlp.gate|up|down`` each with ``.b``, ``final.norm``, ``head``.

A layer has its RMS norms behind the residual sums: ``x <- norm1(alpha x + mixer(x)); x <- norm2(alpha x + ff(x))``.

``latent_attention``  queries from a normed latent of ``q_rank``; keys and values from one cached latent row of ``kv_rank``
                      (normed) plus ``rot_dim`` rotated elements shared by the heads; pairs ``(2e, 2e + 1)`` at YaRN's frequencies,
                      with its magnitude on sine and cosine (``rot.scaling``: ``factor``, ``original``, ``fast``, ``slow``).
``mlstm``             matrix memory with exponential gates capped at ``gate_cap``, ``heads`` of ``dim`` keys and ``vdim`` values.
``attention``         grouped heads; q and k rows normed whole; pairs ``(e, e + dims/2)`` at frequencies scaled by wavelength
                      (``rot.scaling``: ``factor``, ``low``, ``high``, ``original``); scores capped at ``softcap``.

The feed-forward is ``W_d (silu(W_g h + b_g) (W_u h + b_u)) + b_d``.

The design has no bound on positions; :data:`POSITIONS` is what the engine is told.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Iterable, List, Optional, Tuple

from .errors import ConfigError
from .rilenex import _int, _num, _obj
from .spec import (BiasedAttentionSpec, GatedFfnSpec, LatentAttentionSpec, LayerSpec, MlstmSpec, ModelSpec, NormSpec, PositionSpec,
                   RunEntry)

POSITIONS = 1 << 20           # the longest sequence the engine is told of (no tensor or constant depends on it)
DIVISOR_EPS = 1e-6            # what is added to mlstm's divisor: the design fixes it
YARN_MAGNITUDE_SLOPE = 0.1    # of latent_attention's sine and cosine: slope ln(factor) + 1


@dataclass(frozen=True)
class DerosunYarn:
    factor: float
    original: int
    fast: float
    slow: float


@dataclass(frozen=True)
class DerosunBands:
    factor: float
    low: float
    high: float
    original: int


@dataclass(frozen=True)
class DerosunRotation:
    dims: int
    base: float
    scaling: object = None             # DerosunYarn | DerosunBands; None: the plain frequencies


@dataclass(frozen=True)
class DerosunAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: Optional[float]           # None: scores are not capped
    rot: Optional[DerosunRotation]
    type: str = "attention"


@dataclass(frozen=True)
class DerosunLatent:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot: DerosunRotation
    type: str = "latent_attention"


@dataclass(frozen=True)
class DerosunMlstm:
    heads: int
    dim: int
    vdim: int
    gate_cap: float
    type: str = "mlstm"


@dataclass(frozen=True)
class DerosunLayer:
    mixer: object                      # DerosunAttention | DerosunLatent | DerosunMlstm
    ff: Optional[int]                  # the feed-forward's inner size; None: there is none


@dataclass(frozen=True)
class DerosunConfig:
    vocab: int
    width: int
    eps: float
    alpha: float
    embed_scale: float
    layers: Tuple[DerosunLayer, ...]

    architecture = "Derosun"

    # ------------------------------------------------------------------ parse
    @classmethod
    def from_dict(cls, raw: dict) -> "DerosunConfig":
        vocab, width = _int(raw, "vocab", "top level"), _int(raw, "width", "top level")
        eps = _num(_obj(raw, "norm", "top level"), "eps", "norm", positive=True)
        alpha = _num(raw, "postln_alpha", "top level")
        embed_scale = _num(_obj(raw, "embedding", "top level"), "scale", "embedding")
        entries = raw.get("layers")
        if not isinstance(entries, list) or not entries:
            raise ConfigError("config.json: 'layers' must be a list with at least one layer")
        readers = {"attention": cls._attention, "latent_attention": cls._latent, "mlstm": cls._mlstm}
        layers: List[DerosunLayer] = []
        for i, e in enumerate(entries):
            where = f"layers[{i}]"
            if not isinstance(e, dict):
                raise ConfigError(f"config.json: {where} must be an object")
            read = readers.get(e.get("type")) if isinstance(e.get("type"), str) else None
            if read is None:
                raise ConfigError(f"config.json: {where}: unknown layer type {e.get('type')!r} ({', '.join(sorted(readers))})")
            layers.append(DerosunLayer(read(_obj(e, "mixer", where), where + ".mixer"), cls._mlp(e.get("mlp"), where + ".mlp")))
        return cls(vocab, width, eps, alpha, embed_scale, tuple(layers))

    @staticmethod
    def _rotation(m: dict, mw: str, most: int, scaling) -> DerosunRotation:
        r, rw = _obj(m, "rot", mw), mw + ".rot"
        dims, base = _int(r, "dims", rw, least=2), _num(r, "base", rw, positive=True)
        if dims % 2 or dims > most:
            raise ConfigError(f"config.json: {rw}: dims ({dims}) must be even and at most {most}")
        if r.get("scaling") is None:
            return DerosunRotation(dims, base)
        return DerosunRotation(dims, base, scaling(_obj(r, "scaling", rw), rw + ".scaling"))

    @staticmethod
    def _yarn(s: dict, sw: str) -> DerosunYarn:
        return DerosunYarn(_num(s, "factor", sw, positive=True), _int(s, "original", sw), _num(s, "fast", sw, positive=True),
                           _num(s, "slow", sw, positive=True))

    @staticmethod
    def _bands(s: dict, sw: str) -> DerosunBands:
        return DerosunBands(_num(s, "factor", sw, positive=True), _num(s, "low", sw, positive=True), _num(s, "high", sw, positive=True),
                            _int(s, "original", sw))

    @classmethod
    def _attention(cls, m: dict, mw: str) -> DerosunAttention:
        heads, kv_heads, dim = _int(m, "heads", mw), _int(m, "kv_heads", mw), _int(m, "dim", mw)
        if heads % kv_heads:
            raise ConfigError(f"config.json: {mw}: heads ({heads}) is not a multiple of kv_heads ({kv_heads})")
        rot = cls._rotation(m, mw, dim, cls._bands) if m.get("rot") is not None else None
        softcap = _num(m, "softcap", mw, positive=True) if m.get("softcap") is not None else None
        return DerosunAttention(heads, kv_heads, dim, _int(m, "vdim", mw), _num(m, "scale", mw), softcap, rot)

    @classmethod
    def _latent(cls, m: dict, mw: str) -> DerosunLatent:
        rot_dim = _int(m, "rot_dim", mw, least=2)
        rot = cls._rotation(m, mw, rot_dim, cls._yarn)
        if rot.dims != rot_dim:
            raise ConfigError(f"config.json: {mw}.rot: dims ({rot.dims}) must equal rot_dim ({rot_dim})")
        return DerosunLatent(_int(m, "heads", mw), _int(m, "dim", mw), rot_dim, _int(m, "vdim", mw), _int(m, "q_rank", mw),
                             _int(m, "kv_rank", mw), _num(m, "scale", mw), rot)

    @classmethod
    def _mlstm(cls, m: dict, mw: str) -> DerosunMlstm:
        return DerosunMlstm(_int(m, "heads", mw), _int(m, "dim", mw), _int(m, "vdim", mw), _num(m, "gate_cap", mw, positive=True))

    @staticmethod
    def _mlp(mlp, where: str) -> Optional[int]:
        if mlp is None:
            return None
        if not isinstance(mlp, dict):
            raise ConfigError(f"config.json: {where} must be null or an object")
        if mlp.get("kind") != "dense":
            raise ConfigError(f"config.json: {where}: unknown kind {mlp.get('kind')!r} (dense)")
        return _int(mlp, "ff", where)

    # ------------------------------------------------------------------ export
    def to_dict(self) -> dict:
        """config.json content that parses back to this configuration."""
        out = []
        for layer in self.layers:
            m = layer.mixer
            mixer = {k: v for k, v in vars(m).items() if k not in ("type", "rot") and v is not None}
            rot = getattr(m, "rot", None)
            if rot is not None:
                mixer["rot"] = {"dims": rot.dims, "base": rot.base}
                if rot.scaling is not None:
                    mixer["rot"]["scaling"] = dict(vars(rot.scaling))
            out.append({"type": m.type, "mixer": mixer, "mlp": {"kind": "dense", "ff": layer.ff} if layer.ff is not None else None})
        return {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps},
                "postln_alpha": self.alpha, "embedding": {"scale": self.embed_scale}, "layers": out}

    # ------------------------------------------------------------------ spec
    @staticmethod
    def _position(rot: Optional[DerosunRotation], interleaved: bool) -> PositionSpec:
        if rot is None:
            return PositionSpec("none")
        common = dict(rotary_dim=rot.dims, theta=rot.base, interleaved=interleaved)
        s = rot.scaling
        if isinstance(s, DerosunYarn):
            return PositionSpec("rope_yarn", yarn_factor=s.factor, yarn_original=s.original, yarn_fast=s.fast, yarn_slow=s.slow,
                                yarn_magnitude_slope=YARN_MAGNITUDE_SLOPE, **common)
        if isinstance(s, DerosunBands):
            return PositionSpec("rope_banded", band_factor=s.factor, band_low=s.low, band_high=s.high, band_original=s.original, **common)
        return PositionSpec("rope", **common)

    def _mixer_spec(self, m, p: str):
        e, eps = self.width, self.eps
        if m.type == "attention":
            return BiasedAttentionSpec(
                kind="biased_attention", hidden=e, n_heads=m.heads, n_kv_heads=m.kv_heads, head_dim=m.dim, v_head_dim=m.vdim,
                scale=m.scale, q_proj=p + "q", k_proj=p + "k", v_proj=p + "v", o_proj=p + "o",
                q_row_norm=NormSpec("rmsnorm", m.heads * m.dim, eps, p + "q.norm"),
                k_row_norm=NormSpec("rmsnorm", m.kv_heads * m.dim, eps, p + "k.norm"),
                position=self._position(m.rot, False), softcap=m.softcap or 0.0)
        if m.type == "latent_attention":
            return LatentAttentionSpec(
                kind="latent_attention", hidden=e, n_heads=m.heads, head_dim=m.dim, rot_dim=m.rot_dim, v_head_dim=m.vdim,
                q_rank=m.q_rank, kv_rank=m.kv_rank, scale=m.scale, norm_eps=eps, position=self._position(m.rot, True),
                q_down=p + "dq", q_norm=p + "dq.norm", q_up=p + "uq", kv_down=p + "dkv", kv_norm=p + "dkv.norm", k_up=p + "uk",
                v_up=p + "uv", o_proj=p + "o")
        return MlstmSpec(
            kind="mlstm", hidden=e, n_heads=m.heads, head_dim=m.dim, v_head_dim=m.vdim, gate_cap=m.gate_cap, floor_eps=DIVISOR_EPS,
            norm_eps=eps, q_proj=p + "q", k_proj=p + "k", v_proj=p + "v", gate_proj=p + "g", i_gate=p + "i", i_bias=p + "i.b",
            f_gate=p + "f", f_bias=p + "f.b", out_norm=p + "norm", o_proj=p + "o")

    def model_spec(self, tensor_names: Optional[Iterable[str]] = None) -> ModelSpec:
        e, eps = self.width, self.eps

        def norm(name: str) -> NormSpec:
            return NormSpec("rmsnorm", e, eps, name)

        layers: List[LayerSpec] = []
        for i, layer in enumerate(self.layers):
            ffn = None
            if layer.ff is not None:
                f = f"l{i}.mlp."
                ffn = GatedFfnSpec(kind="gated_dense", hidden=e, intermediate=layer.ff, activation="silu", gate_proj=f + "gate",
                                   up_proj=f + "up", down_proj=f + "down", gate_bias=f + "gate.b", up_bias=f + "up.b",
                                   down_bias=f + "down.b")
            layers.append(LayerSpec(kind="postnorm_sum", mixer=self._mixer_spec(layer.mixer, f"l{i}.mix."), ffn=ffn,
                                    post_mixer_norm=norm(f"l{i}.norm1"), post_ffn_norm=norm(f"l{i}.norm2") if ffn is not None else None,
                                    residual_scale=self.alpha))
        return ModelSpec(
            architecture=self.architecture, vocab_size=self.vocab, hidden=e, embed_weight="embed", embed_scale=self.embed_scale,
            layers=layers, order=[RunEntry(i, i, True) for i in range(len(layers))], final_norm=norm("final.norm"), head_weight="head",
            max_context=POSITIONS, bos_token_id=None, eos_token_ids=(),
            # a tensor that no part asks for (the second norm of a layer without a feed-forward, say) is passed over
            tensor_scope=())
