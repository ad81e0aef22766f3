"""Typed configuration of the Dopivik decoder, read from its own config.json keys.

A model of this design is a list of layers over a float32 residual stream of ``width``.  Every sub-layer stands
between two layer norms with weight and bias (``norm.eps``): x <- x + norm1b(mixer(norm1(x))), then, where the layer has
a feed-forward, x <- x + norm2b(ff(norm2(x))).  ``layers[i].type`` names the mixer, ``layers[i].mixer`` its sizes:

* ``parallel``: two mixers on the same rows, the result half the sum of theirs, each with an RMS norm of its own.
  ``left`` {``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, ``softcap``, ``mask.size``, ``rot`` {``base``, ``dims``}}: softmax
  attention within chunks of ``mask.size`` positions, q and k turned in half pairs, scores softly capped, a gate for
  every element of the output.  ``right`` {``heads``, ``kv_heads``, ``dim``, ``vdim``, ``conv``}: the gated delta rule behind
  short convolutions.
* ``mamba1`` {``inner``, ``state``, ``dt_rank``, ``conv``}: the selective scan with a decay for every channel and state.
* ``wkv`` {``heads``, ``dim``}: time mixing with a decay for every key channel; the rank of the decay's two matrices is that
  of the tensors (an optional key ``rank`` says it for random weights).

``layers[i].mlp`` is null or ``{"kind": "dense", "ff"}``: W_down relu(W_up h)^2.  ``layers[i].weights_of``: j, the layer has no
tensors of its own and runs layer j's once more, with a cache or state of its own.  The embedding is ``embed[token] *
embedding.scale``, the logits ``head`` on the final norm.  Tensor names: ``embed``, ``final.norm``, ``head``, and per layer
``l<i>.norm1``, ``norm1b``, ``norm2``, ``norm2b`` (each with a ``.b``), ``l<i>.mix.*``, ``l<i>.mlp.up``, ``l<i>.mlp.down``.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass

from .spec import ConfigError, LayerSpec, ModelSpec, PartSpec, ScheduleEntry, SubLayerSpec

_DTYPES = ("float32", "float16", "bfloat16")
_KEYS = {"parallel": ("left", "right"), "mamba1": ("inner", "state", "dt_rank", "conv"), "wkv": ("heads", "dim")}
BRANCH_SCALE = 0.5            # of either branch of a parallel layer, behind its norm


def _need(d, key: str, where: str):
    if not isinstance(d, dict) or key not in d:
        raise ConfigError(f"config.json: {where} lacks '{key}'")
    return d[key]


def _positive(d: dict, keys, where: str) -> None:
    for k in keys:
        if int(_need(d, k, where)) < 1:
            raise ConfigError(f"{where}: {k} must be positive")


@dataclass(frozen=True)
class DopivikConfig:
    width: int
    vocab: int
    norm_eps: float
    embedding_scale: float
    layers: tuple                   # the layers as config.json lists them (plain dicts)
    max_positions: int = 0          # the design sets no bound; an optional key may
    torch_dtype: str | None = None
    eos_token_ids: tuple = ()
    architecture: str = "Dopivik"

    context_key = "max_positions"

    @classmethod
    def from_dict(cls, c: dict) -> "DopivikConfig":
        layers = _need(c, "layers", "the model")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must list at least one layer")
        eos = c.get("eos_token_id")
        cfg = cls(width=int(_need(c, "width", "the model")), vocab=int(_need(c, "vocab", "the model")),
                  norm_eps=float(_need(_need(c, "norm", "the model"), "eps", "norm")),
                  embedding_scale=float((c.get("embedding") or {}).get("scale", 1.0)),
                  layers=tuple(copy.deepcopy(layers)), max_positions=int(c.get("max_positions") or 0), torch_dtype=c.get("torch_dtype"),
                  eos_token_ids=() if eos is None else tuple(int(e) for e in (eos if isinstance(eos, list) else [eos])),
                  architecture=c.get("architecture") or (c.get("architectures") or ["Dopivik"])[0])
        cfg.validate()
        return cfg

    def validate(self) -> None:
        if self.width <= 0 or self.vocab <= 0:
            raise ConfigError("width and vocab must be positive")
        if not self.norm_eps >= 0:
            raise ConfigError("norm.eps must not be negative")
        if self.torch_dtype is not None and self.torch_dtype not in _DTYPES:
            raise ConfigError(f"Unsupported torch_dtype: {self.torch_dtype}")
        for i, layer in enumerate(self.layers):
            where = f"layer {i}"
            kind, m = _need(layer, "type", where), _need(layer, "mixer", where)
            if kind not in _KEYS:
                raise ConfigError(f"{where}: mixer type {kind!r} is not built ({', '.join(_KEYS)} are)")
            if kind == "parallel":
                self._check_left(_need(m, "left", where), where + " left")
                self._check_right(_need(m, "right", where), where + " right")
            else:
                _positive(m, _KEYS[kind], where + " mixer")
                if int(m.get("conv", 1)) > 16:
                    raise ConfigError(f"{where}: conv: 1 to 16 taps")
            mlp = layer.get("mlp")
            if mlp is not None:
                if _need(mlp, "kind", where + " mlp") != "dense":
                    raise ConfigError(f"{where}: feed-forward kind {mlp['kind']!r} is not built ('dense' is)")
                _positive(mlp, ("ff",), where + " mlp")
            src = layer.get("weights_of")
            if src is not None:
                if not 0 <= int(src) < len(self.layers) or int(src) == i:
                    raise ConfigError(f"{where}: weights_of names layer {src}")
                other = self.layers[int(src)]
                if any(layer.get(k) != other.get(k) for k in ("type", "mixer", "mlp")):
                    raise ConfigError(f"{where}: weights_of names layer {src}, which is another kind of layer or has other sizes")
                self.owner(i)

    @staticmethod
    def _check_heads(m: dict, where: str) -> None:
        _positive(m, ("heads", "kv_heads", "dim"), where)
        if int(m["heads"]) % int(m["kv_heads"]) or int(m.get("vdim", 1)) < 1:
            raise ConfigError(f"{where}: heads a positive multiple of kv_heads, vdim positive")

    def _check_left(self, m: dict, where: str) -> None:
        self._check_heads(m, where)
        if not float(_need(m, "scale", where)) > 0:
            raise ConfigError(f"{where}: scale must be positive")
        _positive(_need(m, "mask", where), ("size",), where + " mask")
        if m.get("softcap") is not None and not float(m["softcap"]) > 0:
            raise ConfigError(f"{where}: softcap must be positive")
        rot = m.get("rot")
        if rot is not None:
            _need(rot, "base", where + " rot")
            dims = int(_need(rot, "dims", where + " rot"))
            if dims % 2 or not 0 <= dims <= int(m["dim"]):
                raise ConfigError(f"{where}: rot.dims must be even and at most dim")

    def _check_right(self, m: dict, where: str) -> None:
        self._check_heads(m, where)
        if not 1 <= int(_need(m, "conv", where)) <= 16:
            raise ConfigError(f"{where}: conv: 1 to 16 taps")

    def owner(self, i: int) -> int:
        """The layer whose tensors layer i runs."""
        seen = {i}
        while self.layers[i].get("weights_of") is not None:
            i = int(self.layers[i]["weights_of"])
            if i in seen:
                raise ConfigError(f"layer {i}: weights_of leads back to it")
            seen.add(i)
        return i

    def summary(self) -> list:
        """(label, value) lines for the command line's report."""
        kinds = [layer["type"] for layer in self.layers]
        heads = [int(h) for layer in self.layers for h in
                 ([layer["mixer"]["left"]["heads"], layer["mixer"]["right"]["heads"]] if layer["type"] == "parallel"
                  else [layer["mixer"]["heads"]] if "heads" in layer["mixer"] else [])] or [0]
        span = str(heads[0]) if len(set(heads)) == 1 else f"{min(heads)}..{max(heads)}"
        return [("Layers", f"{len(self.layers)} (" + ", ".join(f"{kinds.count(k)} {k}" for k in sorted(set(kinds))) + ")"),
                ("Dimensions", self.width), ("Heads", span), ("Vocab size", self.vocab)]

    def to_dict(self) -> dict:
        """The config.json that reads back as this configuration."""
        out = {"architecture": self.architecture, "embedding": {"scale": self.embedding_scale},
               "layers": copy.deepcopy(list(self.layers)), "norm": {"eps": self.norm_eps}, "vocab": self.vocab, "width": self.width}
        if self.max_positions:
            out["max_positions"] = self.max_positions
        if self.torch_dtype is not None:
            out["torch_dtype"] = self.torch_dtype
        if self.eos_token_ids:
            out["eos_token_id"] = list(self.eos_token_ids)
        return out

    # ------------------------------------------------------------------ the model as data
    def _norm(self, prefix: str, name: str) -> PartSpec:
        return PartSpec("layernorm", {"size": self.width, "eps": self.norm_eps, "name": name, "bias": name + ".b"}, prefix)

    def _left(self, m: dict, prefix: str) -> PartSpec:
        return PartSpec("gated_attention", {
            "hidden_size": self.width, "n_heads": int(m["heads"]), "n_kv_heads": int(m["kv_heads"]), "head_dim": int(m["dim"]),
            "v_head_dim": int(m.get("vdim", m["dim"])), "scale": float(m["scale"]), "block": int(m["mask"]["size"]), "sink": False,
            "gate": "elements", "softcap": None if m.get("softcap") is None else float(m["softcap"]),
            "names": {k: k for k in "qkvgo"}}, prefix + "left.")

    def _right(self, m: dict, prefix: str) -> PartSpec:
        return PartSpec("gated_delta", {
            "hidden_size": self.width, "n_heads": int(m["heads"]), "n_kv_heads": int(m["kv_heads"]), "head_dim": int(m["dim"]),
            "v_head_dim": int(m.get("vdim", m["dim"])), "conv_taps": int(m["conv"]), "norm_eps": self.norm_eps,
            "names": {**{k: k for k in "qkvgbao"}, "q_conv": "q.conv", "k_conv": "k.conv", "v_conv": "v.conv", "a_log": "A_log",
                      "dt_bias": "dt_bias", "norm": "norm"}}, prefix + "right.")

    def _mixer(self, layer: dict, prefix: str) -> PartSpec:
        m, kind = layer["mixer"], layer["type"]
        if kind == "parallel":
            return PartSpec("parallel", {"branches": ((self._left(m["left"], prefix), BRANCH_SCALE), (self._right(m["right"], prefix), BRANCH_SCALE)),
                                         "norms": ("left.out", "right.out"), "norm_eps": self.norm_eps, "hidden_size": self.width}, prefix)
        if kind == "mamba1":
            return PartSpec("selective_scan", {
                "hidden_size": self.width, "inner": int(m["inner"]), "n_state": int(m["state"]), "dt_rank": int(m["dt_rank"]),
                "conv_taps": int(m["conv"]), "names": {"in": "in", "conv": "conv", "conv_bias": "conv.b", "x": "x", "dt": "dt",
                                                       "dt_bias": "dt.b", "a_log": "A_log", "d": "D", "o": "o"}}, prefix)
        return PartSpec("wkv", {
            "hidden_size": self.width, "n_heads": int(m["heads"]), "head_dim": int(m["dim"]), "norm_eps": self.norm_eps,
            "decay_rank": int(m.get("rank") or max(16, self.width // 64 // 16 * 16)),
            "names": {**{k: k for k in ("r", "k", "v", "g", "w1", "w2", "w0", "u", "norm", "o")}, "mu": "mu.{}"}}, prefix)

    def _position(self, layer: dict) -> PartSpec | None:
        if layer["type"] != "parallel":
            return None
        left = layer["mixer"]["left"]
        rot = left.get("rot")
        if rot is None or int(rot["dims"]) == 0:
            return None
        return PartSpec("rope_half", {"theta": float(rot["base"]), "rotary_dim": int(rot["dims"]), "head_dim": int(left["dim"])}, "")

    def _layer_spec(self, i: int, layer: dict) -> LayerSpec:
        p = f"l{i}."
        subs = [SubLayerSpec("mixer", self._mixer(layer, p + "mix."), self._norm(p, "norm1"), self._norm(p, "norm1b"))]
        if layer.get("mlp") is not None:
            ff = PartSpec("dense_mlp", {"hidden_size": self.width, "intermediate_size": int(layer["mlp"]["ff"]), "activation": "relu2",
                                        "names": {"up": "up", "down": "down"}}, p + "mlp.")
            subs.append(SubLayerSpec("feed_forward", ff, self._norm(p, "norm2"), self._norm(p, "norm2b")))
        return LayerSpec("sandwich", tuple(subs), self._position(layer))

    def model_spec(self) -> ModelSpec:
        own = [i for i in range(len(self.layers)) if self.layers[i].get("weights_of") is None]
        at = {i: k for k, i in enumerate(own)}             # a layer without tensors of its own is one more run of its owner
        spec = ModelSpec(
            hidden_size=self.width, vocab_size=self.vocab, max_positions=self.max_positions,
            embedding=PartSpec("embedding", {"vocab_size": self.vocab, "hidden_size": self.width, "name": "embed",
                                             "scale": self.embedding_scale}, ""),
            layers=tuple(self._layer_spec(i, self.layers[i]) for i in own),
            schedule=tuple(ScheduleEntry(at[self.owner(i)]) for i in range(len(self.layers))),
            final_norm=self._norm("final.", "norm"),
            head=PartSpec("lm_head", {"vocab_size": self.vocab, "hidden_size": self.width, "tied": False, "name": "head"}, ""),
            stop_token_ids=self.eos_token_ids)
        spec.validate()
        return spec
