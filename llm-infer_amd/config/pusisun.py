"""Typed configuration of the Pusisun decoder, read from its own config.json keys.

A model of this design is a list of layers over a float32 residual stream of ``width``.  Every sub-layer stands
between two RMS norms with a weight (``norm.eps``): x <- x + norm1b(mixer(norm1(x))), then, where the layer has a
feed-forward, x <- x + norm2b(ff(norm2(x))).  ``layers[i].type`` names the mixer, ``layers[i].mixer`` its sizes:

* ``latent_attention`` {``heads``, ``dim``, ``rot_dim``, ``vdim``, ``kv_rank``, ``q_rank``, ``scale``, ``rot`` {``base``, ``dims``,
  ``scaling`` {``factor``, ``original``, ``fast``, ``slow``}}}: softmax attention over one latent per token, with the queries
  behind a latent of their own; the rotated parts are turned in half pairs, the frequencies stretched along a ramp of
  the pairs and sine and cosine multiplied by 0.1 ln(factor) + 1 (without ``scaling``: neither).
* ``attention`` {``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, ``mask`` {``size``, ``keep_first``}}: grouped-query softmax
  attention with biases on q, k and v, an RMS norm over all rows of q and of k, a score's loss of 2^(-8 (h + 1) / heads)
  for every position between query and key, a learned sink in every head's sum, and a sliding window of ``mask.size``
  positions beside the first ``mask.keep_first``, which stay visible.

``layers[i].mlp`` is null or ``{"kind": "moe", "expert": {"ff"}, "router": {"experts", "top"}}``: W_down(silu(W_gate h) * (W_up
h)) for each expert, the ``top`` largest router logits (with a bias) chosen, weighted by the softmax over the chosen.
``loop`` {``start``, ``stop``, ``times``}: layers start .. stop - 1 run ``times`` times in a row with the same weights, every
pass with caches of its own; ahead of pass t the embedding's output (not for t = 0) and the vector ``loop.step``[t] are
added to the stream.  The embedding is ``embed[token] * embedding.scale``, the logits ``head`` on the final norm.  Tensor
names: ``embed``, ``loop.step``, ``final.norm``, ``head``, and per layer ``l<i>.norm1``, ``norm1b``, ``norm2``, ``norm2b``,
``l<i>.mix.*``, ``l<i>.mlp.e<j>.gate|up|down``, ``l<i>.mlp.router`` (and ``.b``).
"""
from __future__ import annotations

import copy
from dataclasses import dataclass

from .spec import ConfigError, LayerSpec, ModelSpec, PartSpec, ScheduleEntry, SubLayerSpec

_DTYPES = ("float32", "float16", "bfloat16")
_KEYS = {"latent_attention": ("heads", "dim", "vdim", "kv_rank", "q_rank"), "attention": ("heads", "kv_heads", "dim", "vdim")}
SLOPE_EXPONENT = 8.0          # the distance bias of 'attention': slope_h = 2^(-8 (h + 1) / heads)


def _need(d, key: str, where: str):
    if not isinstance(d, dict) or key not in d:
        raise ConfigError(f"config.json: {where} lacks '{key}'")
    return d[key]


def _positive(d: dict, keys, where: str) -> None:
    for k in keys:
        if int(_need(d, k, where)) < 1:
            raise ConfigError(f"{where}: {k} must be positive")


@dataclass(frozen=True)
class PusisunConfig:
    width: int
    vocab: int
    norm_eps: float
    embedding_scale: float
    layers: tuple                   # the layers as config.json lists them (plain dicts)
    loop: tuple | None = None       # (start, stop, times) of the stretch of layers that runs several times
    max_positions: int = 0          # the design sets no bound; an optional key may
    torch_dtype: str | None = None
    eos_token_ids: tuple = ()
    architecture: str = "Pusisun"

    context_key = "max_positions"

    @classmethod
    def from_dict(cls, c: dict) -> "PusisunConfig":
        layers = _need(c, "layers", "the model")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must list at least one layer")
        eos, loop = c.get("eos_token_id"), c.get("loop")
        cfg = cls(width=int(_need(c, "width", "the model")), vocab=int(_need(c, "vocab", "the model")),
                  norm_eps=float(_need(_need(c, "norm", "the model"), "eps", "norm")),
                  embedding_scale=float((c.get("embedding") or {}).get("scale", 1.0)), layers=tuple(copy.deepcopy(layers)),
                  loop=None if loop is None else tuple(int(_need(loop, k, "loop")) for k in ("start", "stop", "times")),
                  max_positions=int(c.get("max_positions") or 0), torch_dtype=c.get("torch_dtype"),
                  eos_token_ids=() if eos is None else tuple(int(e) for e in (eos if isinstance(eos, list) else [eos])),
                  architecture=c.get("architecture") or (c.get("architectures") or ["Pusisun"])[0])
        cfg.validate()
        return cfg

    def validate(self) -> None:
        if self.width <= 0 or self.vocab <= 0:
            raise ConfigError("width and vocab must be positive")
        if not self.norm_eps >= 0:
            raise ConfigError("norm.eps must not be negative")
        if self.torch_dtype is not None and self.torch_dtype not in _DTYPES:
            raise ConfigError(f"Unsupported torch_dtype: {self.torch_dtype}")
        if self.loop is not None:
            start, stop, times = self.loop
            if not 0 <= start < stop <= len(self.layers) or times < 1:
                raise ConfigError(f"loop: layers {start} to {stop} of {len(self.layers)}, {times} times")
        for i, layer in enumerate(self.layers):
            where = f"layer {i}"
            kind, m = _need(layer, "type", where), _need(layer, "mixer", where)
            if kind not in _KEYS:
                raise ConfigError(f"{where}: mixer type {kind!r} is not built ({', '.join(_KEYS)} are)")
            _positive(m, _KEYS[kind], where + " mixer")
            if not float(_need(m, "scale", where + " mixer")) > 0:
                raise ConfigError(f"{where}: scale must be positive")
            if kind == "latent_attention":
                self._check_rotation(m, where)
            else:
                if int(m["heads"]) % int(m["kv_heads"]):
                    raise ConfigError(f"{where}: heads must be a multiple of kv_heads")
                mask = m.get("mask")
                if mask is not None:
                    _positive(mask, ("size",), where + " mask")
                    if int(mask.get("keep_first") or 0) < 0:
                        raise ConfigError(f"{where} mask: keep_first must not be negative")
            mlp = layer.get("mlp")
            if mlp is not None:
                if _need(mlp, "kind", where + " mlp") != "moe":
                    raise ConfigError(f"{where}: feed-forward kind {mlp['kind']!r} is not built ('moe' is)")
                _positive(_need(mlp, "expert", where + " mlp"), ("ff",), where + " expert")
                r = _need(mlp, "router", where + " mlp")
                _positive(r, ("experts", "top"), where + " router")
                if int(r["top"]) > int(r["experts"]):
                    raise ConfigError(f"{where} router: top between 1 and experts")

    @staticmethod
    def _check_rotation(m: dict, where: str) -> None:
        rot_dim = int(_need(m, "rot_dim", where + " mixer"))
        if rot_dim < 0:
            raise ConfigError(f"{where}: rot_dim must not be negative")
        if rot_dim == 0:
            return
        rot = _need(m, "rot", where + " mixer")
        dims = int(_need(rot, "dims", where + " rot"))
        if dims % 2 or not 0 <= dims <= rot_dim:
            raise ConfigError(f"{where}: rot.dims must be even and at most rot_dim")
        base = float(_need(rot, "base", where + " rot"))
        if not base > 0:
            raise ConfigError(f"{where}: rot.base must be positive")
        if rot.get("scaling") is not None:
            if base == 1.0:
                raise ConfigError(f"{where}: rot.scaling needs a base other than 1")
            for k in ("factor", "original", "fast", "slow"):
                if not float(_need(rot["scaling"], k, where + " rot.scaling")) > 0:
                    raise ConfigError(f"{where} rot.scaling: {k} must be positive")

    def summary(self) -> list:
        """(label, value) lines for the command line's report."""
        kinds = [layer["type"] for layer in self.layers]
        heads = [int(layer["mixer"]["heads"]) for layer in self.layers]
        span = str(heads[0]) if len(set(heads)) == 1 else f"{min(heads)}..{max(heads)}"
        again = "" if self.loop is None else "; {} to {} run {} times".format(self.loop[0], self.loop[1] - 1, self.loop[2])
        return [("Layers", f"{len(self.layers)} (" + ", ".join(f"{kinds.count(k)} {k}" for k in sorted(set(kinds))) + again + ")"),
                ("Dimensions", self.width), ("Heads", span), ("Vocab size", self.vocab)]

    def to_dict(self) -> dict:
        """The config.json that reads back as this configuration."""
        out = {"architecture": self.architecture, "embedding": {"scale": self.embedding_scale},
               "layers": copy.deepcopy(list(self.layers)), "norm": {"eps": self.norm_eps}, "vocab": self.vocab, "width": self.width}
        if self.loop is not None:
            out["loop"] = dict(zip(("start", "stop", "times"), self.loop))
        if self.max_positions:
            out["max_positions"] = self.max_positions
        if self.torch_dtype is not None:
            out["torch_dtype"] = self.torch_dtype
        if self.eos_token_ids:
            out["eos_token_id"] = list(self.eos_token_ids)
        return out

    # ------------------------------------------------------------------ the model as data
    def _norm(self, prefix: str, name: str) -> PartSpec:
        return PartSpec("rmsnorm", {"size": self.width, "eps": self.norm_eps, "name": name}, prefix)

    def _mixer(self, layer: dict, prefix: str) -> PartSpec:
        m = layer["mixer"]
        if layer["type"] == "latent_attention":
            return PartSpec("latent_attention", {
                "hidden_size": self.width, "n_heads": int(m["heads"]), "head_dim": int(m["dim"]), "rot_dim": int(m["rot_dim"]),
                "v_head_dim": int(m["vdim"]), "kv_rank": int(m["kv_rank"]), "q_rank": int(m["q_rank"]), "scale": float(m["scale"]),
                "norm_eps": self.norm_eps,
                "names": {**{k: k for k in ("dq", "uq", "dkv", "uk", "uv", "o")}, "q_norm": "dq.norm", "kv_norm": "dkv.norm"}}, prefix)
        mask = m.get("mask")
        return PartSpec("gated_attention", {
            "hidden_size": self.width, "n_heads": int(m["heads"]), "n_kv_heads": int(m["kv_heads"]), "head_dim": int(m["dim"]),
            "v_head_dim": int(m["vdim"]), "scale": float(m["scale"]), "window": None if mask is None else int(mask["size"]),
            "keep_first": 0 if mask is None else int(mask.get("keep_first") or 0), "sink": True, "gate": False, "bias": True,
            "qk_norm_eps": self.norm_eps, "slope_exponent": SLOPE_EXPONENT,
            "names": {**{k: k for k in ("q", "k", "v", "o", "sink")}, "q_bias": "q.b", "k_bias": "k.b", "v_bias": "v.b",
                      "q_norm": "q.norm", "k_norm": "k.norm"}}, prefix)

    def _position(self, layer: dict) -> PartSpec | None:
        m = layer["mixer"]
        if layer["type"] != "latent_attention" or int(m["rot_dim"]) == 0 or int(m["rot"]["dims"]) == 0:
            return None
        rot, scaling = m["rot"], m["rot"].get("scaling")
        return PartSpec("rope_half", {"theta": float(rot["base"]), "rotary_dim": int(rot["dims"]), "head_dim": int(m["rot_dim"]),
                                      "yarn": None if scaling is None else {k: float(scaling[k]) for k in
                                                                            ("factor", "original", "fast", "slow")}}, "")

    def _layer_spec(self, i: int, layer: dict) -> LayerSpec:
        p = f"l{i}."
        subs = [SubLayerSpec("mixer", self._mixer(layer, p + "mix."), self._norm(p, "norm1"), self._norm(p, "norm1b"))]
        mlp = layer.get("mlp")
        if mlp is not None:
            ff = PartSpec("routed_experts", {
                "hidden_size": self.width, "n_experts": int(mlp["router"]["experts"]), "expert_ff": int(mlp["expert"]["ff"]),
                "top": int(mlp["router"]["top"]), "correction": False, "router_bias": True, "shared_gate": False, "gated": True,
                "activation": "silu", "scores": "softmax", "renormalize": True,
                "names": {"router": "router", "router_bias": "router.b", "expert": "e{}."}}, p + "mlp.")
            subs.append(SubLayerSpec("feed_forward", ff, self._norm(p, "norm2"), self._norm(p, "norm2b")))
        return LayerSpec("sandwich", tuple(subs), self._position(layer))

    def _schedule(self) -> tuple:
        n = len(self.layers)
        if self.loop is None:
            return tuple(ScheduleEntry(i) for i in range(n))
        start, stop, times = self.loop
        entry = PartSpec("pass_entry", {"hidden_size": self.width, "times": times, "name": "step"}, "loop.")
        out = [ScheduleEntry(i) for i in range(start)]
        for t in range(times):
            out += [ScheduleEntry(i, before=entry if i == start else None, pass_no=t) for i in range(start, stop)]
        return tuple(out + [ScheduleEntry(i) for i in range(stop, n)])

    def model_spec(self) -> ModelSpec:
        spec = ModelSpec(
            hidden_size=self.width, vocab_size=self.vocab, max_positions=self.max_positions,
            embedding=PartSpec("embedding", {"vocab_size": self.vocab, "hidden_size": self.width, "name": "embed",
                                             "scale": self.embedding_scale}, ""),
            layers=tuple(self._layer_spec(i, layer) for i, layer in enumerate(self.layers)),
            schedule=self._schedule(), final_norm=self._norm("final.", "norm"),
            head=PartSpec("lm_head", {"vocab_size": self.vocab, "hidden_size": self.width, "tied": False, "name": "head"}, ""),
            stop_token_ids=self.eos_token_ids)
        spec.validate()
        return spec
