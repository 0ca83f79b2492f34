"""config.json of a Zivitar checkpoint.  Every size and every constant that may differ between checkpoints is read here; what the
design fixes (activation functions, the 1.702 of the feed-forward's gate, the rotate-half layout, two maps per attention head)
lives in the model code and the kernels.  Unknown mixer types / feed-forward kinds and inconsistent sizes are refused at load."""
from __future__ import annotations

import copy
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from ..ragged import rotation  # noqa: F401   (the frequency table of a `rot` entry)

MIXERS = ("lightning", "attention")
MAX_STREAMS, MAX_TAPS, MAX_VDIM = 8, 16, 256          # what the kernels take


def _need(d: Dict[str, Any], keys, what: str):
    missing = [k for k in keys if k not in d]
    if missing:
        raise ValueError(f"Zivitar {what}: missing {missing}")


@dataclass
class LayerConfig:
    type: str
    mixer: Dict[str, Any]
    mlp: Optional[Dict[str, Any]] = None
    weights_of: Optional[int] = None

    def __post_init__(self):
        if self.type not in MIXERS:
            raise ValueError(f"Zivitar layer type {self.type!r}: one of {MIXERS}")
        m = self.mixer
        _need(m, ("heads", "dim"), self.type + " mixer")
        m.setdefault("vdim", m["dim"])
        if min(int(m["heads"]), int(m["dim"]), int(m["vdim"])) < 1:
            raise ValueError(f"{self.type} mixer: heads, dim and vdim are at least 1")
        if self.type == "lightning":
            _need(m, ("decay",), "lightning mixer")
            if len(m["decay"]) != int(m["heads"]):
                raise ValueError("lightning mixer: one decay per head")
        else:
            _need(m, ("scale", "diff"), "attention mixer")
            m.setdefault("kv_heads", m["heads"])
            if int(m["kv_heads"]) < 1 or int(m["heads"]) % int(m["kv_heads"]):
                raise ValueError("attention mixer: heads must be a multiple of kv_heads")
            if int(m["vdim"]) > MAX_VDIM:
                raise ValueError(f"attention mixer: vdim up to {MAX_VDIM}")
            if not 0 <= self.taps <= MAX_TAPS:
                raise ValueError(f"attention mixer: conv is at most {MAX_TAPS}")
            win, keep = self.window
            if ((m.get("mask") or {}).get("size") is not None and win < 1) or keep < 0:
                raise ValueError("attention mixer: mask.size is at least 1, mask.keep_first at least 0")
            rot = m.get("rot")
            if rot:
                _need(rot, ("base", "dims"), "attention mixer, rot")
                if int(rot["dims"]) % 2 or not 0 <= int(rot["dims"]) <= int(m["dim"]):
                    raise ValueError("attention mixer: rot.dims is even and at most dim")
                if rot.get("scaling"):
                    _need(rot["scaling"], ("factor", "original", "fast", "slow"), "attention mixer, rot.scaling")
        if self.mlp is not None:
            if self.mlp.get("kind", "dense") != "dense":
                raise ValueError(f"Zivitar feed-forward kind {self.mlp.get('kind')!r}: 'dense'")
            _need(self.mlp, ("ff",), "feed-forward")
            if self.limit < 0:
                raise ValueError("feed-forward: limit is not negative")

    @property
    def ff(self) -> int:
        return int(self.mlp["ff"]) if self.mlp is not None else 0

    @property
    def limit(self) -> float:
        lim = (self.mlp or {}).get("limit")
        return float("inf") if lim is None else float(lim)

    @property
    def taps(self) -> int:
        return int(self.mixer.get("conv") or 0)

    @property
    def window(self):
        """(window size, 0: none; first tokens kept in view)"""
        m = self.mixer.get("mask") or {}
        return int(m["size"]) if m.get("size") is not None else 0, int(m.get("keep_first") or 0)

    def shapes(self):
        """the sizes that decide tensor shapes (a layer that uses another's tensors agrees on them)"""
        m = self.mixer
        s = [self.type, int(m["heads"]), int(m["dim"]), int(m["vdim"]), self.ff]
        return s + ([int(m["kv_heads"]), self.taps] if self.type == "attention" else [])


@dataclass
class ModelConfig:
    vocab: int = 0
    width: int = 0
    layers: List[LayerConfig] = field(default_factory=list)
    norm_eps: float = 1e-6
    streams: int = 0                       # 0: a plain residual sum, no stream weights in the checkpoint
    logit_scale: float = 1.0
    logit_softcap: float = 0.0             # 0: none
    model_type: str = "zivitar"
    eos_token_id: Any = None

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "ModelConfig":
        _need(d, ("vocab", "width", "layers", "norm"), "config")
        layers = [LayerConfig(type=L["type"], mixer=copy.deepcopy(L["mixer"]), mlp=(dict(L["mlp"]) if L.get("mlp") else None),
                              weights_of=None if L.get("weights_of") is None else int(L["weights_of"])) for L in d["layers"]]
        for i, lc in enumerate(layers):
            # the source may stand before or after the layer; a source that itself borrows is followed to the owner
            j, seen = lc.weights_of, {i}
            while j is not None:
                if not 0 <= j < len(layers) or j in seen:
                    raise ValueError(f"layer {i}: weights_of must lead to a layer that has tensors of its own")
                seen.add(j)
                if layers[j].weights_of is None:
                    break
                j = layers[j].weights_of
            if j is not None:
                if layers[j].shapes() != lc.shapes():
                    raise ValueError(f"layer {i}: its sizes differ from layer {j}, whose weights it uses")
                lc.weights_of = j
        streams = int(d.get("streams") or 0)
        if not 0 <= streams <= MAX_STREAMS:
            raise ValueError(f"streams: 1 to {MAX_STREAMS}")
        cap = d.get("logit_softcap")
        return cls(vocab=int(d["vocab"]), width=int(d["width"]), layers=layers, norm_eps=float(d["norm"]["eps"]), streams=streams,
                   logit_scale=float(d.get("logit_scale", 1.0)), logit_softcap=float(cap) if cap else 0.0, eos_token_id=d.get("eos_token_id"))

    # names other parts of the package read from a text config
    @property
    def vocab_size(self):
        return self.vocab

    @property
    def hidden_size(self):
        return self.width

    @property
    def num_hidden_layers(self):
        return len(self.layers)
