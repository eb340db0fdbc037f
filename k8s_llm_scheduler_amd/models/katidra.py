"""Katidra: a decoder with an fp32 residual stream whose sublayers read the stream itself and whose norms act on the
sublayers' outputs only, ``x <- x + norm1(mixer(x)); x <- x + norm2(ff(x))`` (RMS norms with a weight per channel), a
dense feed-forward ``W_down relu(W_up x)^2`` and two mixers in any order the config lists:

* ``lightning``: linear attention under a constant decay per head (the decays are part of the configuration),
  ``S <- decay S + k v^T``, ``o = S^T q`` with ``q, k, v = silu(W h)``; the concatenated heads are RMS-normed together
  with a weight, multiplied by ``sigmoid(W_g h)`` and projected by ``W_o``;
* ``latent_attention``: keys and values are up-projections (``W_uk``, ``W_uv``) of one cached low-rank row per token,
  ``c = rmsnorm(W_dkv h)[:kv_rank]``, beside one rotated key part shared by the heads; queries come from a normed
  low-rank row as well, ``q = W_uq rmsnorm(W_dq h)``, each head laid out as [dim unrotated | rot_dim rotated]; the
  rotation turns the pairs (2i, 2i + 1) with YaRN-scaled frequencies; softmax of ``(q_n . k_n + q_r . k_r) * scale``
  over a sliding window of ``mask.size`` tokens; head h's output times ``sigmoid(W_g h)_h`` ahead of ``W_o``.  Queries
  are absorbed into the latent space (``q_n W_uk``), so the cache is attended as it is stored, the gate is applied to
  the attended latents and ``W_uv`` follows.

A layer with ``weights_of`` runs another layer's weights on a cache or state of its own.  The embedding is scaled by
``embedding.scale``.

The model presents the engine's interface through :class:`~.stream.StreamModel`; caches: per latent-attention layer a
paged ``[slots, kv_rank + rot_dim]`` cache, per lightning layer one fp32 ``[dim, vdim]`` state per (request slot, head).
Every op is a kernel of :mod:`..ops.seqmix`; ``dtype=float32`` runs everything in true fp32.  Single rank (TP = 1).
"""

from __future__ import annotations

import math
from dataclasses import dataclass, field
from pathlib import Path
from typing import Dict, List, Optional

import torch

from ..ops import reference as ref
from ..ops import seqmix as sm
from ..parallel import TPGroup
from . import stream
from .stream import StreamModel, stack_rows

ARCHITECTURE = "Katidra"
MIXERS = ("lightning", "latent_attention")
F32 = torch.float32


# ----------------------------------------------------------------------------- configuration
@dataclass
class LightningConfig:
    heads: int
    dim: int
    vdim: int
    decay: tuple             # one per head


@dataclass
class LatentConfig:
    heads: int
    dim: int                 # unrotated query / key dimensions per head
    rot_dim: int             # rotated dimensions per head (one key part shared by the heads)
    vdim: int
    kv_rank: int
    q_rank: int
    scale: float
    window: int = 0          # tokens a position sees, itself included; 0: every earlier one
    rot_base: float = 10000.0
    rot_dims: int = -1       # dimensions of the rotated part that turn (the first ones); -1: all of it
    yarn: Optional[dict] = None          # factor, original, fast, slow

    def __post_init__(self):
        if self.rot_dims < 0:
            self.rot_dims = self.rot_dim


@dataclass
class LayerConfig:
    type: str
    mixer: object            # LightningConfig | LatentConfig
    ff: int = 0              # 0: no feed-forward
    weights_of: int = -1     # >= 0: this layer runs that layer's tensors


@dataclass
class KatidraConfig:
    name: str
    vocab: int
    hidden: int
    layers: List[LayerConfig]
    rms_eps: float = 1e-5
    embed_scale: float = 1.0
    max_position: int = 1 << 20
    bos_id: int = 0
    eos_ids: tuple = ()
    extra: dict = field(default_factory=dict)
    token_ids_only = True    # checkpoints of this design ship no tokenizer: requests are token ids

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    def owner(self, i: int) -> int:
        """The layer whose tensors layer ``i`` runs (itself, or what its ``weights_of`` leads to)."""
        seen = set()
        while self.layers[i].weights_of >= 0:
            if i in seen or self.layers[i].weights_of >= len(self.layers):
                raise ValueError(f"{self.name}: layer {i}: weights_of leads to no layer with tensors")
            seen.add(i)
            i = self.layers[i].weights_of
        return i

    def validate_tp(self, tp: int) -> None:
        if tp != 1:
            raise ValueError(f"{self.name}: this design runs on one rank (tp={tp})")


def _layer_from(l: dict) -> LayerConfig:
    kind, d = l["type"], l["mixer"]
    if kind == "lightning":
        mixer: object = LightningConfig(int(d["heads"]), int(d["dim"]), int(d["vdim"]), tuple(float(a) for a in d["decay"]))
        if len(mixer.decay) != mixer.heads:
            raise ValueError(f"lightning: {len(mixer.decay)} decays for {mixer.heads} heads")
    elif kind == "latent_attention":
        rot, mask = d.get("rot") or {}, d.get("mask") or {}
        dim, rot_dim = int(d["dim"]), int(d["rot_dim"])
        sc = rot.get("scaling")
        yarn = {k: float(sc[k]) for k in ("factor", "original", "fast", "slow")} if sc else None
        mixer = LatentConfig(int(d["heads"]), dim, rot_dim, int(d["vdim"]), int(d["kv_rank"]), int(d["q_rank"]),
                             float(d.get("scale", 1.0 / math.sqrt(dim + rot_dim))), int(mask.get("size") or 0),
                             float(rot.get("base", 10000.0)), int(rot.get("dims", rot_dim)), yarn)
    else:
        raise ValueError(f"unknown mixer type {kind!r} (known: {', '.join(MIXERS)})")
    mlp = l.get("mlp")
    if mlp is not None and mlp.get("kind", "dense") != "dense":
        raise ValueError(f"unknown mlp kind {mlp['kind']!r}")
    of = l.get("weights_of")
    return LayerConfig(kind, mixer, int(mlp["ff"]) if mlp else 0, -1 if of is None else int(of))


def config_from_json(c: dict, name: str = "katidra") -> KatidraConfig:
    return KatidraConfig(name=name, vocab=int(c["vocab"]), hidden=int(c["width"]),
                         layers=[_layer_from(l) for l in c["layers"]],
                         rms_eps=float((c.get("norm") or {}).get("eps", 1e-5)),
                         embed_scale=float((c.get("embedding") or {}).get("scale", 1.0)))


def config_to_json(cfg: KatidraConfig) -> dict:
    layers = []
    for L in cfg.layers:
        m = L.mixer
        if L.type == "lightning":
            mixer: dict = {"heads": m.heads, "dim": m.dim, "vdim": m.vdim, "decay": list(m.decay)}
        else:
            rot: dict = {"dims": m.rot_dims, "base": m.rot_base}
            if m.yarn:
                rot["scaling"] = dict(m.yarn)
            mixer = {"heads": m.heads, "dim": m.dim, "rot_dim": m.rot_dim, "vdim": m.vdim, "kv_rank": m.kv_rank,
                     "q_rank": m.q_rank, "scale": m.scale, "rot": rot}
            if m.window:
                mixer["mask"] = {"size": m.window}
        e = {"type": L.type, "mixer": mixer, "mlp": {"kind": "dense", "ff": L.ff} if L.ff else None}
        if L.weights_of >= 0:
            e["weights_of"] = L.weights_of
        layers.append(e)
    return {"architecture": ARCHITECTURE, "vocab": cfg.vocab, "width": cfg.hidden, "layers": layers,
            "norm": {"eps": cfg.rms_eps}, "embedding": {"scale": cfg.embed_scale}}


def tensor_shapes(cfg: KatidraConfig) -> Dict[str, tuple]:
    """Checkpoint tensor names and shapes of a configuration."""
    W = cfg.hidden
    t: Dict[str, tuple] = {"embed": (cfg.vocab, W), "final.norm": (W,), "head": (cfg.vocab, W)}
    for i, L in enumerate(cfg.layers):
        if L.weights_of >= 0:
            continue
        p, m = f"l{i}.", L.mixer
        q, H = p + "mix.", m.heads
        t[p + "norm1"] = (W,)
        if L.type == "lightning":
            t.update({q + "q": (H * m.dim, W), q + "k": (H * m.dim, W), q + "v": (H * m.vdim, W), q + "g": (H * m.vdim, W),
                      q + "norm": (H * m.vdim,), q + "o": (W, H * m.vdim)})
        else:
            t.update({q + "dq": (m.q_rank, W), q + "dq.norm": (m.q_rank,), q + "uq": (H * (m.dim + m.rot_dim), m.q_rank),
                      q + "dkv": (m.kv_rank + m.rot_dim, W), q + "dkv.norm": (m.kv_rank,),
                      q + "uk": (H * m.dim, m.kv_rank), q + "uv": (H * m.vdim, m.kv_rank), q + "g": (H, W),
                      q + "o": (W, H * m.vdim)})
        if L.ff:
            t.update({p + "norm2": (W,), p + "mlp.up": (L.ff, W), p + "mlp.down": (W, L.ff)})
    return t


def random_tensors(cfg: KatidraConfig, seed: int = 0, device="cpu") -> Dict[str, torch.Tensor]:
    """Random bf16 weights of a configuration (benchmarks and tests): projections ~ N(0, 1 / fan_in), norm weights
    around one, embedding rows that start the stream at unit size."""
    g = torch.Generator(device=device).manual_seed(seed)
    out: Dict[str, torch.Tensor] = {}
    for name, shape in tensor_shapes(cfg).items():
        t = torch.randn(shape, generator=g, device=device)
        leaf = name.rsplit(".", 1)[-1]
        if leaf in ("norm", "norm1", "norm2"):
            t = 1.0 + t * 0.1
        elif leaf == "embed":
            t = t / max(abs(cfg.embed_scale), 1e-6)
        else:
            t = t / math.sqrt(shape[-1])
        out[name] = t.to(torch.bfloat16)
    return out


def save_checkpoint(cfg: KatidraConfig, tensors: Dict[str, torch.Tensor], path: Path) -> None:
    stream.save_checkpoint(config_to_json(cfg), tensors, path)


def preset(name: str, width: int, vocab: int, order, *, heads: int, dim: int, rot_dim: int, vdim: int, kv_rank: int,
           q_rank: int, window: int, scan_heads: int, scan_dim: int, scan_vdim: int, ff: int, original: int = 4096,
           factor: float = 4.0) -> KatidraConfig:
    """Layers in ``order``: a mixer's name, or an index (the layer whose weights run again).  The heads' decays forget
    over 2, 4, 8, ... tokens, spread over the heads up to about 4096."""
    spans = [2.0 ** (1.0 + 11.0 * h / max(1, scan_heads - 1)) for h in range(scan_heads)]
    decay = tuple(math.exp(-1.0 / s) for s in spans)
    layers: List[LayerConfig] = []
    for kind in order:
        if isinstance(kind, int):
            L = layers[kind]
            layers.append(LayerConfig(L.type, L.mixer, L.ff, kind))
        elif kind == "lightning":
            layers.append(LayerConfig(kind, LightningConfig(scan_heads, scan_dim, scan_vdim, decay), ff))
        else:
            layers.append(LayerConfig(kind, LatentConfig(heads, dim, rot_dim, vdim, kv_rank, q_rank,
                                                         1.0 / math.sqrt(dim + rot_dim), window, 10000.0, rot_dim,
                                                         {"factor": factor, "original": float(original), "fast": 32.0,
                                                          "slow": 1.0}), ff))
    return KatidraConfig(name, vocab, width, layers, embed_scale=math.sqrt(width))


PRESETS = {
    # runs on the CPU in tests: both mixers, one repeated layer of each, odd sizes
    "katidra-tiny": preset("katidra-tiny", 96, 384, ("lightning", "latent_attention", 0, 1), heads=3, dim=16, rot_dim=8,
                           vdim=24, kv_rank=40, q_rank=56, window=20, scan_heads=5, scan_dim=16, scan_vdim=24, ff=112,
                           original=64),
    # layer shapes of a ~1B-class model (benchmarks, random weights)
    "katidra-1b": preset("katidra-1b", 2048, 32768, ("lightning", "latent_attention", "lightning", "lightning") * 4,
                         heads=16, dim=128, rot_dim=64, vdim=128, kv_rank=512, q_rank=1536, window=1024, scan_heads=16,
                         scan_dim=128, scan_vdim=128, ff=4096),
}


# ----------------------------------------------------------------------------- weights
@dataclass
class _Lightning:
    cfg: LightningConfig
    w_in: torch.Tensor                  # q | k | v | gate, parts padded to multiples of 16 rows
    cols: Dict[str, int]
    decay: torch.Tensor                 # fp32 [H]
    norm: torch.Tensor                  # fp32 [H V]
    o: torch.Tensor                     # [W, H V]


@dataclass
class _Latent:
    cfg: LatentConfig
    w_in: torch.Tensor                  # [q_rank | kv_rank + rot_dim | H (gate), W], parts padded to multiples of 16 rows
    cols: Dict[str, int]
    dq_norm: torch.Tensor               # [q_rank]
    uq: torch.Tensor                    # [H (Dn + R), q_rank]
    dkv_norm: torch.Tensor              # [kv_rank]
    uk_t: torch.Tensor                  # [H, kv_rank, Dn]: per head W_uk^T (absorbs the query into the latent space)
    uv: torch.Tensor                    # [H, V, kv_rank]
    o: torch.Tensor                     # [W, H V]
    cos_sin: torch.Tensor               # [positions, rot_dims] fp32


@dataclass
class _Weights:
    n1: torch.Tensor
    mixer: object
    n2: Optional[torch.Tensor] = None
    w_up: Optional[torch.Tensor] = None
    w_down: Optional[torch.Tensor] = None


@dataclass
class _Layer:
    w: _Weights                         # shared by the layers that run the same tensors
    cache: int                          # index into kv_cache (latent attention) or states (lightning): the layer's own


class KatidraModel(StreamModel):
    def __init__(self, cfg: KatidraConfig, tp: Optional[TPGroup] = None, device="cpu", dtype=torch.bfloat16,
                 seed: int = 0, weights: Optional[str] = None, tensors: Optional[Dict[str, torch.Tensor]] = None,
                 max_model_len: int = 8192, weight_dtype: str = "bf16"):
        super().__init__(cfg, tp, device, dtype, seed, max_model_len, weight_dtype)
        self._rope: Dict[tuple, torch.Tensor] = {}
        if tensors is None:
            tensors = self._open(Path(weights)) if weights else random_tensors(cfg, seed, self.device)
        get = tensors if callable(tensors) else tensors.__getitem__
        self._build(get)

    # ------------------------------------------------------------------ weights
    def _f(self, t: torch.Tensor) -> torch.Tensor:
        """Small constants that enter fp32 arithmetic are kept in fp32."""
        return t.to(F32).to(self.device).contiguous()

    def _rope_table(self, m: LatentConfig) -> torch.Tensor:
        key = (m.rot_dims, m.rot_base, tuple(sorted(m.yarn.items())) if m.yarn else None)
        if key not in self._rope:
            scaling = {"type": "yarn", **m.yarn} if m.yarn else None
            self._rope[key] = ref.rope_table(m.rot_dims, self.max_model_len, m.rot_base,
                                             scaling).to(self.device).contiguous()
        return self._rope[key]

    def _build_lightning(self, get, p: str, m: LightningConfig, where: str) -> _Lightning:
        if max(m.dim, m.vdim) > sm.gated_scan_max_dim():
            raise ValueError(f"{where}: head sizes {m.dim} x {m.vdim} exceed the kernels' {sm.gated_scan_max_dim()}")
        w_in, cols = stack_rows(tuple((s, get(p + s).cpu()) for s in ("q", "k", "v", "g")))
        return _Lightning(m, self._t(w_in), cols, self._f(torch.tensor(m.decay, dtype=torch.float64)),
                          self._f(get(p + "norm")), self._t(get(p + "o")))

    def _build_latent(self, get, p: str, m: LatentConfig, where: str) -> _Latent:
        t = self._t
        H, Dn, R, V, C = m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank
        if m.rot_dims % 2 or not 0 < m.rot_dims <= R:
            raise ValueError(f"{where}: rot.dims {m.rot_dims} must be even, positive and at most rot_dim {R}")
        w_in, cols = stack_rows(tuple((s, get(p + s).cpu()) for s in ("dq", "dkv", "g")))
        return _Latent(m, t(w_in), cols, t(get(p + "dq.norm")), t(get(p + "uq")), t(get(p + "dkv.norm")),
                       t(get(p + "uk").view(H, Dn, C).transpose(1, 2)), t(get(p + "uv").view(H, V, C)), t(get(p + "o")),
                       self._rope_table(m))

    def _build(self, get) -> None:
        c, t = self.cfg, self._t
        self.embed = t(get("embed"))
        self.final_norm = t(get("final.norm"))
        self.lm_head = t(get("head"))
        built: Dict[int, _Weights] = {}
        for i, L in enumerate(c.layers):
            if L.weights_of >= 0:
                continue
            p = f"l{i}."
            build = self._build_lightning if L.type == "lightning" else self._build_latent
            w = _Weights(t(get(p + "norm1")), build(get, p + "mix.", L.mixer, f"layer {i}"))
            if L.ff:
                w.n2, w.w_up, w.w_down = t(get(p + "norm2")), t(get(p + "mlp.up")), t(get(p + "mlp.down"))
            built[i] = w
        self.layers: List[_Layer] = []
        self._latents: List[LatentConfig] = []       # one paged cache each
        self._scans: List[LightningConfig] = []      # one state each
        for i in range(c.num_layers):
            w = built[c.owner(i)]
            own = self._scans if isinstance(w.mixer, _Lightning) else self._latents
            self.layers.append(_Layer(w, len(own)))
            own.append(w.mixer.cfg)

    def _weight_roots(self) -> tuple:
        return (self.embed, self.final_norm, self.lm_head, *self.layers)

    # ------------------------------------------------------------------ cache and state
    def _needs_state(self) -> bool:
        return bool(self._scans)

    def allocate_kv(self, num_blocks: int, block_size: int):
        """Per latent-attention layer (repeated layers included) one paged cache [slots, kv_rank + rot_dim]."""
        self.block_size = block_size
        self.kv_cache = [torch.zeros(num_blocks * block_size, m.kv_rank + m.rot_dim, dtype=self.dtype,
                                     device=self.device) for m in self._latents]
        return self.kv_cache

    def kv_bytes_per_block(self, block_size: int) -> int:
        eb = torch.finfo(self.dtype).bits // 8
        return max(1, block_size * sum(m.kv_rank + m.rot_dim for m in self._latents) * eb)

    def allocate_state(self, slots: int) -> None:
        """Per lightning layer (repeated layers included) and request slot: the heads' fp32 states [dim, vdim]."""
        self.state_slots = slots
        self.states = [torch.zeros(slots, m.heads, sm.gated_scan_record(sm.SCAN_DECAY, m.dim, m.vdim), dtype=F32,
                                   device=self.device) for m in self._scans]

    def state_bytes_per_slot(self) -> int:
        return sum(4 * m.heads * sm.gated_scan_record(sm.SCAN_DECAY, m.dim, m.vdim) for m in self._scans)

    # ------------------------------------------------------------------ layers
    def _lightning(self, w: _Lightning, cache: int, h, b) -> torch.Tensor:
        m = w.cfg
        H, D, V = m.heads, m.dim, m.vdim
        proj = sm.linear(h, w.w_in)                                        # [T, q | k | v | gate]
        y = sm.gated_scan(proj, sm.SCAN_DECAY, w.cols, None, self.states[cache], b["cu_q"], b["seq_slots"],
                          b["positions"], H, D, V, self.cfg.rms_eps, F32, head_params=w.decay, groups=H,
                          max_qlen=b.get("max_qlen", 0))
        y = sm.norm_mix(y, w.norm, None, None, self.cfg.rms_eps, out_dtype=self.dtype,
                        gate=proj[:, w.cols["g"]:w.cols["g"] + H * V])
        return sm.linear(y, w.o)

    def _latent(self, w: _Latent, cache: int, h, b) -> torch.Tensor:
        m = w.cfg
        T = h.shape[0]
        H, Dn, R, C, V = m.heads, m.dim, m.rot_dim, m.kv_rank, m.vdim
        eps, kv = self.cfg.rms_eps, self.kv_cache[cache]
        proj = sm.linear(h, w.w_in)                                        # [T, dq | dkv | gate]
        cq = sm.norm_mix(proj[:, w.cols["dq"]:w.cols["dq"] + m.q_rank], w.dq_norm, None, None, eps)
        q = sm.linear(cq, w.uq)                                            # [T, H (Dn + R)]
        sm.latent_kv_write(kv, proj[:, w.cols["dkv"]:w.cols["dkv"] + C + R], w.dkv_norm, q, w.cos_sin, b["positions"],
                           b["slot_mapping"], C, R, H, Dn, m.rot_dims, eps, interleaved=True)
        q_abs = torch.empty(T, H, C, dtype=self.dtype, device=h.device)
        sm.gemm(q.view(T, H, Dn + R)[:, :, :Dn].permute(1, 0, 2), w.uk_t, out=q_abs.permute(1, 0, 2))
        lat = sm.latent_attention(q_abs, q, kv, b["block_tables"], b["tok_seq"], b["positions"], C, R, H, Dn, m.window,
                                  m.scale, self.block_size, b.get("max_keys", 0), b["cu_q"], b.get("max_qlen", 0),
                                  gate=proj[:, w.cols["g"]:w.cols["g"] + H])                # [T, H, C]
        a = torch.empty(T, H, V, dtype=self.dtype, device=h.device)
        sm.gemm(lat.permute(1, 0, 2), w.uv, out=a.permute(1, 0, 2))
        return sm.linear(a.view(T, H * V), w.o)

    def _blocks(self, ids, b, after=None) -> torch.Tensor:
        """The residual stream after the last layer."""
        c, dt = self.cfg, self.dtype
        x = sm.embed_rows(ids, self.embed, c.embed_scale)
        h = x.to(dt)                      # the stream as the next sublayer reads it
        for L in self.layers:
            w = L.w
            run = self._lightning if isinstance(w.mixer, _Lightning) else self._latent
            h = sm.branchnorm(x, run(w.mixer, L.cache, h, b), w.n1, c.rms_eps, out_dtype=dt)
            if w.w_up is not None:
                f = sm.linear(sm.act(sm.linear(h, w.w_up), sm.ACT_RELU2), w.w_down)
                h = sm.branchnorm(x, f, w.n2, c.rms_eps, out_dtype=dt)
            if after is not None:
                after.append(x.clone())
        return x

    def _forward(self, ids, b, rows) -> torch.Tensor:
        x = self._blocks(ids, b)
        hf = sm.resnorm(x.index_select(0, rows), self.final_norm, self.cfg.rms_eps, out_dtype=self.dtype)
        return sm.linear(hf, self.lm_head, out_dtype=F32).unsqueeze(0)     # [1, S, vocab]

    def residual_after_runs(self, ids, b) -> List[torch.Tensor]:
        """(debugging / tests) the fp32 residual stream after every layer."""
        after: List[torch.Tensor] = []
        self._blocks(ids, b, after)
        return after
