"""config.json of a Rorovik checkpoint.  Every size and every constant that may differ between checkpoints is read here; what the
design fixes (activation functions, the 1.702 of the experts' gate, the interleaved layout of the rotation, the slopes of the distance
bias) lives in the model code and the kernels.  Unknown mixer types / feed-forward kinds and inconsistent sizes are refused at load."""
from __future__ import annotations

import copy
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

MIXERS = ("attention", "latent_attention")
MAX_VDIM, MAX_DIM, MAX_RANK, MAX_EXPERTS = 256, 768, 1024, 256          # what the kernels take


def _need(d: Dict[str, Any], keys, what: str):
    missing = [k for k in keys if d.get(k) is None]
    if missing:
        raise ValueError(f"Rorovik {what}: missing {missing}")


@dataclass
class LayerConfig:
    type: str
    mixer: Dict[str, Any]
    mlp: Optional[Dict[str, Any]] = None

    def __post_init__(self):
        if self.type not in MIXERS:
            raise ValueError(f"Rorovik layer type {self.type!r}: one of {MIXERS}")
        m = self.mixer
        if self.type == "attention":
            _need(m, ("heads", "dim", "scale"), "attention mixer")
            m.setdefault("kv_heads", m["heads"])
            m.setdefault("vdim", m["dim"])
            if min(int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])) < 1 or int(m["heads"]) % int(m["kv_heads"]):
                raise ValueError("attention mixer: heads must be a multiple of kv_heads, sizes at least 1")
            if int(m["vdim"]) > MAX_VDIM or int(m["dim"]) > MAX_DIM:
                raise ValueError(f"attention mixer: vdim up to {MAX_VDIM}, dim up to {MAX_DIM}")
            qt = m.get("q_temp")
            if qt is not None:
                _need(qt, ("coef", "every"), "attention mixer, q_temp")
                if int(qt["every"]) < 1:
                    raise ValueError("attention mixer: q_temp.every is at least 1")
            win = (m.get("mask") or {}).get("size")
            if win is not None and int(win) < 1:
                raise ValueError("attention mixer: mask.size is at least 1")
        else:
            _need(m, ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank", "scale"), "latent_attention mixer")
            Dr = int(m["rot_dim"])
            if min(int(m["heads"]), int(m["dim"]), int(m["vdim"]), int(m["kv_rank"]), int(m["q_rank"])) < 1 or Dr < 0:
                raise ValueError("latent_attention mixer: sizes are at least 1")
            if int(m["kv_rank"]) > MAX_RANK:
                raise ValueError(f"latent_attention mixer: kv_rank up to {MAX_RANK}")
            if Dr:
                _need(m, ("rot",), "latent_attention mixer")
                _need(m["rot"], ("base",), "latent_attention mixer, rot")
                m["rot"].setdefault("dims", Dr)
                if int(m["rot"]["dims"]) != Dr or Dr % 2:
                    raise ValueError(f"latent_attention mixer: the rotated part is rot_dim wide and even (rot.dims {m['rot']['dims']}, rot_dim {Dr})")
                if m["rot"].get("scaling"):
                    _need(m["rot"]["scaling"], ("factor", "original", "fast", "slow"), "latent_attention mixer, rot.scaling")
        if self.mlp is not None:
            kind = self.mlp.get("kind", "dense")
            if kind == "dense":
                _need(self.mlp, ("ff",), "dense feed-forward")
            elif kind == "moe":
                _need(self.mlp, ("expert", "router"), "mixture of experts")
                _need(self.mlp["expert"], ("ff",), "expert")
                _need(self.mlp["router"], ("experts", "top"), "router")
                E, ident, top = self.router
                if E < 1 or ident < 0 or not 0 < top <= E + ident or E + ident > MAX_EXPERTS:
                    raise ValueError(f"moe: at least one expert, 0 < top <= experts + identity <= {MAX_EXPERTS}")
                if self.limit < 0:
                    raise ValueError("moe: expert.limit is not negative")
            else:
                raise ValueError(f"Rorovik feed-forward kind {kind!r}: 'dense' or 'moe'")
            if self.ff < 1:
                raise ValueError("feed-forward: ff is at least 1")

    # ---- what the entry says, with the defaults of what it may leave out
    @property
    def window(self) -> int:
        """0: every earlier token is seen"""
        win = (self.mixer.get("mask") or {}).get("size")
        return int(win) if win is not None and self.type == "attention" else 0

    @property
    def v_mix(self) -> bool:
        return self.type == "attention" and bool(self.mixer.get("v_mix"))

    @property
    def moe(self) -> bool:
        return self.mlp is not None and self.mlp.get("kind", "dense") == "moe"

    @property
    def ff(self) -> int:
        if self.mlp is None:
            return 0
        return int(self.mlp["expert"]["ff"]) if self.moe else int(self.mlp["ff"])

    @property
    def limit(self) -> float:
        lim = self.mlp["expert"].get("limit") if self.moe else None
        return float("inf") if lim is None else float(lim)

    @property
    def router(self):
        """(experts with tensors, identity experts, chosen per token)"""
        r = self.mlp["router"]
        return int(r["experts"]), int(r.get("identity") or 0), int(r["top"])


@dataclass
class ModelConfig:
    vocab: int = 0
    width: int = 0
    layers: List[LayerConfig] = field(default_factory=list)
    norm_eps: float = 1e-6
    residual_mult: float = 1.0
    side_dim: int = 0                      # columns per layer of the second embedding table, 0: none
    v_first: Optional[int] = None          # the first layer that takes part in the value mixing
    model_type: str = "rorovik"
    eos_token_id: Any = None

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "ModelConfig":
        _need(d, ("vocab", "width", "layers", "norm"), "config")
        layers = [LayerConfig(type=L["type"], mixer=copy.deepcopy(L["mixer"]), mlp=(copy.deepcopy(L["mlp"]) if L.get("mlp") else None))
                  for L in d["layers"]]
        mixing = [i for i, lc in enumerate(layers) if lc.v_mix]
        sizes = {(int(layers[i].mixer["kv_heads"]), int(layers[i].mixer["vdim"])) for i in mixing}
        if len(sizes) > 1:
            raise ValueError("layers that mix their values (v_mix) agree on kv_heads and vdim")
        mult = d.get("residual_mult")
        return cls(vocab=int(d["vocab"]), width=int(d["width"]), layers=layers, norm_eps=float(d["norm"]["eps"]),
                   residual_mult=1.0 if mult is None else float(mult), side_dim=int((d.get("token_side") or {}).get("dim") or 0),
                   v_first=mixing[0] if mixing else None, eos_token_id=d.get("eos_token_id"))

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
