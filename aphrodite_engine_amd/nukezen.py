"""Nukezen: a decoder whose sublayers read the residual itself and join it through a norm of their own, with three kinds of mixer.

  x = embed[token] * embed_scale
  layer:   x += norm1(mixer(x));   x += norm2(ff(x))   (the second only if the layer has a feed-forward)
  logits = embed . norm_final(x)                        (the output matrix is the embedding table, without its scale)

Mixers, by the layer's ``type``:
  channel_delta   GatedDeltaMixer with one decay per head and key channel; decay and sigmoid output gate through low-rank products
  parallel        two mixers side by side on the same input, summed with a scale each: GroupedQueryAttention (biased projections,
                  per-head q / k norm before an interleaved rotation, sliding window, elementwise gate) and SelectiveStateSpace
  attention       GroupedQueryAttention with q / k normed over the whole projection, no rotation, soft cap, distance bias, chunks
                  and a sink of score 0
A layer may use another layer's tensors (``weights_of``); its caches are its own.  The feed-forward is GatedMLP with gelu (tanh).

Every size and constant comes from config.json; the low-rank inner sizes and the length of the distance table come from the
tensors' shapes.  Norm statistics, angles, scores, softmax, the recurrent states and what enters them, and the residual are fp32
also in a bfloat16 model.  One launch (``residual_post_rms_norm``) norms a sublayer's result, adds it and rounds the next input."""
from dataclasses import dataclass, field
from typing import Any, Dict, Iterable, List, Optional, Tuple

import torch
from torch import nn
from torch.nn import functional as F

from . import mixer_ops as mops
from .mixers import GatedDeltaMixer, GatedMLP, GroupedQueryAttention, RotaryFrequencies, SelectiveStateSpace
from .step_batch import StepBatch

MIXER_TYPES = ("channel_delta", "parallel", "attention")


@dataclass
class NukezenConfig:
    vocab: int
    width: int
    eps: float
    embed_scale: float
    layers: List[Dict[str, Any]]
    owner: List[int] = field(default_factory=list)                # layer -> the layer whose tensors it uses
    shapes: Dict[str, Tuple[int, ...]] = field(default_factory=dict)

    @staticmethod
    def from_dict(c: Dict[str, Any], shapes: Dict[str, Tuple[int, ...]]) -> "NukezenConfig":
        """``shapes``: name -> shape of the checkpoint's tensors (needed: l<i>.mix.a1, .g1 and .rel)."""
        cfg = NukezenConfig(vocab=int(c["vocab"]), width=int(c["width"]), eps=float(c["norm"]["eps"]),
                            embed_scale=float((c.get("embedding") or {}).get("scale", 1.0)), layers=list(c["layers"]), shapes=dict(shapes))
        for i, lc in enumerate(cfg.layers):
            if lc["type"] not in MIXER_TYPES:
                raise ValueError(f"layer {i}: unknown mixer type {lc['type']!r}")
            mlp = lc.get("mlp")
            if mlp is not None and mlp.get("kind") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward kind {mlp.get('kind')!r}")
            src, seen = i, {i}
            while cfg.layers[src].get("weights_of") is not None:
                src = int(cfg.layers[src]["weights_of"])
                if not 0 <= src < len(cfg.layers) or src in seen:
                    raise ValueError(f"layer {i}: weights_of leads to layer {src}")
                seen.add(src)
            own = {k: v for k, v in lc.items() if k != "weights_of"}
            if own != {k: v for k, v in cfg.layers[src].items() if k != "weights_of"}:
                raise ValueError(f"layer {i} differs from layer {src}, whose tensors it uses")
            cfg.owner.append(src)
        return cfg

    def size_from(self, name: str) -> int:
        """First dimension of a tensor whose size the configuration does not name."""
        if name not in self.shapes:
            raise ValueError(f"checkpoint lacks {name!r}")
        return int(self.shapes[name][0])


def _linear(width_in: int, outs: List[int], dtype, prefix: str, bias: bool = False):
    from .loader import merged_plan
    from .model import QuantLinear
    lin = QuantLinear(width_in, outs, None, dtype, prefix=prefix, plan=merged_plan(outs), bias=bias)
    lin.weight.data.zero_()
    return lin


def _pieces(named: List[Tuple[str, int]]):
    """(names, splits padded to a multiple of 8, name -> slice) of a fused product."""
    names, splits = [n for n, _ in named], [k for _, k in named]
    at, a = {}, 0
    for n, k in named:
        at[n] = slice(a, a + k)
        a += k
    if a % 8:                                     # rows of the fused product stay 16-byte multiples
        splits.append(-a % 8)
    return names, splits, at


def _mask(mc: Dict[str, Any]) -> int:
    return int((mc.get("mask") or {}).get("size", 0))


class ChannelDeltaMixer(GatedDeltaMixer):
    """GatedDeltaMixer in this model's form."""

    def __init__(self, cfg: NukezenConfig, mc: Dict[str, Any], dtype, prefix: str):
        super().__init__(cfg.width, int(mc["heads"]), int(mc["kv_heads"]), int(mc["dim"]), int(mc["vdim"]), int(mc["conv"]), cfg.eps, dtype,
                         prefix=prefix, decay_rank=cfg.size_from(prefix + "a1"), gate_rank=cfg.size_from(prefix + "g1"),
                         gate_act=mops.GATE_SIGMOID)

    def finalize(self) -> None:
        pass

    def run(self, h: torch.Tensor, caches, batch: StepBatch, rows: Optional[torch.Tensor]) -> torch.Tensor:
        return self(h, caches[0], caches[1], batch, rows)

    def tensor_names(self) -> List[str]:
        return ["q", "k", "v", "q.conv", "k.conv", "v.conv", "b", "A_log", "norm", "a1", "a2", "dt_bias", "g1", "g2", "o"]

    def destination(self, key: str) -> torch.Tensor:
        """The parameter (or the part of one) that a checkpoint tensor goes to."""
        if key in self.names:
            i = self.at[key]
            return self.in_proj.weight.data[i:i + self.splits[self.names.index(key)]]
        if key.endswith(".conv"):
            i = self.names.index(key[:-5])
            return self.conv.data[self.at[key[:-5]]:self.at[key[:-5]] + self.splits[i]]
        return {"A_log": self.a_log, "norm": self.out_norm, "a2": self.a2.weight, "g2": self.g2.weight, "dt_bias": self.dt_bias,
                "o": self.out_proj.weight}[key].data


class BiasedAttentionMixer(nn.Module):
    """One input product [q | k | v], GroupedQueryAttention, output product."""

    def __init__(self, cfg: NukezenConfig, mc: Dict[str, Any], dtype, prefix: str):
        super().__init__()
        H, G, d, e = int(mc["heads"]), int(mc["kv_heads"]), int(mc["dim"]), int(mc["vdim"])
        rows = cfg.size_from(prefix + "rel")
        self.attn = GroupedQueryAttention(H, G, d, e, float(mc["scale"]), cfg.eps, dtype, qk_norm="row", bias_rows=rows,
                                          bias_far=float(mc["bias_max"]), chunk=_mask(mc), softcap=float(mc.get("softcap") or 0.0), sink=0.0)
        self.names, self.splits, self.at = _pieces(list(zip(("q", "k", "v"), self.attn.splits)))
        self.in_proj = _linear(cfg.width, self.splits, dtype, prefix + "in_proj")
        self.out_proj = _linear(H * e, [cfg.width], dtype, prefix + "out_proj")

    def cache_specs(self):
        return (self.attn.cache_spec(), )

    def finalize(self) -> None:
        self.attn.finalize(self.in_proj.weight.device)

    def run(self, h: torch.Tensor, caches, batch: StepBatch, rows: Optional[torch.Tensor]) -> torch.Tensor:
        proj = self.in_proj(h)
        o = torch.empty(h.shape[0], self.attn.heads * self.attn.vdim, dtype=h.dtype, device=h.device)
        self.attn(o, *(proj[:, self.at[n]] for n in self.names), None, caches[0], batch)
        return self.out_proj(o if rows is None else o.index_select(0, rows))

    def tensor_names(self) -> List[str]:
        return ["q", "k", "v", "q.norm", "k.norm", "rel", "o"]

    def destination(self, key: str) -> torch.Tensor:
        if key in self.names:
            return self.in_proj.weight.data[self.at[key]]
        return {"q.norm": self.attn.q_norm, "k.norm": self.attn.k_norm, "rel": self.attn.attn.rel, "o": self.out_proj.weight}[key].data


class ParallelMixer(nn.Module):
    """Attention (left) and state space (right) on the same input: ONE input product for everything either reads, one output product
    over the two outputs side by side, each scaled in fp32 before it is rounded."""

    def __init__(self, cfg: NukezenConfig, mc: Dict[str, Any], dtype, prefix: str):
        super().__init__()
        L, R = mc["left"], mc["right"]
        H, G, d, e = int(L["heads"]), int(L["kv_heads"]), int(L["dim"]), int(L["vdim"])
        rot = L.get("rot") or {"dims": 0, "base": 1.0}
        self.left_scale, self.right_scale = float(mc["left_scale"]), float(mc["right_scale"])
        self.attn = GroupedQueryAttention(H, G, d, e, float(L["scale"]), cfg.eps, dtype, qk_norm="head",
                                          rotary=RotaryFrequencies(int(rot["dims"]), float(rot["base"])), layout=mops.ROTARY_INTERLEAVED,
                                          window=_mask(L))
        self.ssm = SelectiveStateSpace(int(R["heads"]), int(R["vdim"]), int(R["state"]), int(R["groups"]), int(R["conv"]),
                                       int(R["norm_groups"]), cfg.eps, dtype)
        m = self.ssm
        self.names, self.splits, self.at = _pieces([("left." + n, k) for n, k in zip("qkv", self.attn.splits)] + [
            ("left.g", H * e), ("right.xbc", m.channels), ("right.z", m.inner), ("right.dt", m.heads)])
        self.in_proj = _linear(cfg.width, self.splits, dtype, prefix + "in_proj", bias=True)
        self.left_out = H * e
        self.out_proj = _linear(self.left_out + m.inner, [cfg.width], dtype, prefix + "out_proj")

    def cache_specs(self):
        return (self.attn.cache_spec(), ) + self.ssm.cache_specs()

    def finalize(self) -> None:
        self.attn.finalize(self.in_proj.weight.device)

    def run(self, h: torch.Tensor, caches, batch: StepBatch, rows: Optional[torch.Tensor]) -> torch.Tensor:
        proj = self.in_proj(h)
        q, k, v, g, xbc, z, dt = (proj[:, self.at[n]] for n in self.names)
        cat = torch.empty(h.shape[0], self.left_out + self.ssm.inner, dtype=h.dtype, device=h.device)
        self.attn(cat[:, :self.left_out], q, k, v, g, caches[0], batch, self.left_scale)
        self.ssm(cat[:, self.left_out:], xbc, z, dt, caches[1], caches[2], batch, self.right_scale)
        return self.out_proj(cat if rows is None else cat.index_select(0, rows))

    def tensor_names(self) -> List[str]:
        return ["left." + n for n in ("q", "q.b", "k", "k.b", "v", "v.b", "q.norm", "k.norm", "g", "o")] + [
            "right." + n for n in ("in", "conv", "conv.b", "dt_bias", "A_log", "D", "norm", "o")]

    def destination(self, key: str) -> torch.Tensor:
        w, m = self.in_proj.weight.data, self.ssm
        if key in self.names:
            return w[self.at[key]]
        if key in ("left.q.b", "left.k.b", "left.v.b"):
            return self.in_proj.bias.data[self.at[key[:-2]]]
        if key == "left.o":
            return self.out_proj.weight.data[:, :self.left_out]
        if key == "right.o":
            return self.out_proj.weight.data[:, self.left_out:]
        return {"left.q.norm": self.attn.q_norm, "left.k.norm": self.attn.k_norm, "right.conv": m.conv, "right.conv.b": m.conv_bias,
                "right.dt_bias": m.dt_bias, "right.A_log": m.a_log, "right.D": m.skip, "right.norm": m.norm}[key].data

    def pieces_of(self, key: str, t: torch.Tensor):
        """The state space's one input tensor [z | x B C | dt] in the fused product's order."""
        n, c, h = self.ssm.inner, self.ssm.channels, self.ssm.heads
        if key != "right.in" or t.shape[0] != n + c + h:
            return [(key, t)]
        return [("right.z", t[:n]), ("right.xbc", t[n:n + c]), ("right.dt", t[n + c:])]


class NukezenLayer(nn.Module):
    def __init__(self, cfg: NukezenConfig, index: int, dtype):
        super().__init__()
        lc = cfg.layers[index]
        pfx = f"l{index}."
        kind = {"channel_delta": ChannelDeltaMixer, "parallel": ParallelMixer, "attention": BiasedAttentionMixer}[lc["type"]]
        self.mix = kind(cfg, lc["mixer"], dtype, pfx + "mix.")
        self.norm1 = nn.Parameter(torch.ones(cfg.width, dtype=dtype), requires_grad=False)
        self.mlp = self.norm2 = None
        if lc.get("mlp") is not None:
            self.mlp = GatedMLP(cfg.width, int(lc["mlp"]["ff"]), mops.ACT_GELU_TANH, dtype, pfx + "mlp.")
            self.norm2 = nn.Parameter(torch.ones(cfg.width, dtype=dtype), requires_grad=False)


class NukezenForCausalLM(nn.Module):
    def __init__(self, cfg: NukezenConfig, dtype: torch.dtype = torch.bfloat16):
        super().__init__()
        from .distributed import get_tensor_model_parallel_world_size
        if get_tensor_model_parallel_world_size() != 1:
            raise ValueError("Nukezen runs on one rank")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Nukezen runs in bfloat16 or float32")
        self.cfg, self.dtype = cfg, dtype
        self.embed = nn.Parameter(torch.empty(cfg.vocab, cfg.width, dtype=dtype), requires_grad=False)
        self.own = nn.ModuleDict({str(i): NukezenLayer(cfg, i, dtype) for i in sorted(set(cfg.owner))})
        self.final_norm = nn.Parameter(torch.ones(cfg.width, dtype=dtype), requires_grad=False)
        # every layer has caches of its own, also one that uses another's tensors
        self.specs, self.run_caches = [], []
        for layer in self.layer_runs():
            specs = layer.mix.cache_specs()
            self.run_caches.append(range(len(self.specs), len(self.specs) + len(specs)))
            self.specs += list(specs)
        self.residual_trace: Optional[List[torch.Tensor]] = None     # set to [] to record x after every layer

    def layer_runs(self) -> List[NukezenLayer]:
        return [self.own[str(j)] for j in self.cfg.owner]

    # ---- what the engine asks of a model ---------------------------------------------------------------------------
    @property
    def vocab_size(self) -> int:
        return self.cfg.vocab

    def make_caches(self, num_blocks: int, block_size: int, num_slots: int, device):
        return [s.allocate(num_blocks, block_size, num_slots, self.dtype, device) for s in self.specs]

    def finalize(self):
        for layer in self.own.values():
            layer.mix.finalize()
        return self

    @torch.no_grad()
    def step(self, batch: StepBatch, caches, rows: torch.Tensor) -> torch.Tensor:
        """One engine step: run the batch's rows through every layer (caches and states advance), return the fp32 logits of
        ``rows`` (int64 indices into the batch)."""
        return self.logits(self.forward(batch, caches, rows))

    def logits(self, h: torch.Tensor) -> torch.Tensor:
        return F.linear(h, self.embed).float()

    def forward(self, batch: StepBatch, caches, rows: Optional[torch.Tensor] = None) -> torch.Tensor:
        """The final norm's output for the rows asked for (all rows if ``rows`` is None).  In the last layer everything behind the
        caches and states runs on those rows only."""
        eps, runs = self.cfg.eps, self.layer_runs()
        h = torch.empty(batch.num_tokens, self.cfg.width, dtype=self.dtype, device=self.embed.device)
        x = mops.embed_scale(self.embed, batch.input_ids, self.cfg.embed_scale, copy=h)
        for i, (layer, idx) in enumerate(zip(runs, self.run_caches)):
            last = i + 1 == len(runs)
            only = rows if last and self.residual_trace is None else None
            y, post = layer.mix.run(h, [caches[c] for c in idx], batch, only), layer.norm1
            if only is not None:
                x = x.index_select(0, only)
            if layer.mlp is not None:
                h = mops.residual_post_rms_norm(x, y, post, eps=eps)
                y, post = layer.mlp(h), layer.norm2
            h = mops.residual_post_rms_norm(x, y, post, self.final_norm if last else None, eps)
            if self.residual_trace is not None:
                self.residual_trace.append(x.clone())
        if not runs:
            h = mops.residual_post_rms_norm(x, pre=self.final_norm, eps=eps)
        if rows is not None and (not runs or self.residual_trace is not None):
            h = h.index_select(0, rows)
        return h

    # ---- checkpoint ----------------------------------------------------------------------------------------------------
    def expected_names(self) -> Tuple[List[str], List[str]]:
        """(names a checkpoint must hold, names it may hold)"""
        names, optional = ["embed", "final.norm"], []
        for i, layer in self.own.items():
            p = f"l{i}."
            names += [p + "norm1"] + [p + "mix." + n for n in layer.mix.tensor_names()]
            if layer.mlp is not None:
                names += [p + "norm2"] + [p + "mlp." + n for n in ("gate", "up", "down")]
            else:
                optional.append(p + "norm2")     # the weight of a norm that is never applied
        return names, optional

    def load_weights(self, weights: Iterable[Tuple[str, torch.Tensor]]) -> None:
        """Checkpoint names: embed, final.norm, l<i>.norm{1,2}, l<i>.mix.* by the layer's type, l<i>.mlp.{gate,up,down}; none for a
        layer that uses another's."""
        names, optional = self.expected_names()
        expected, seen = set(names), set()
        for name, t in weights:
            if name in optional:
                continue
            if name not in expected:
                raise ValueError(f"unexpected tensor {name!r} in a Nukezen checkpoint")
            seen.add(name)
            for dst, part in self._places(name, t):
                if tuple(dst.shape) != tuple(part.shape):
                    raise ValueError(f"{name}: checkpoint tensor {tuple(t.shape)} does not fit {tuple(dst.shape)}")
                dst.copy_(part.to(dst.dtype))
        missing = expected - seen
        if missing:
            raise ValueError(f"checkpoint lacks {len(missing)} tensors, e.g. {sorted(missing)[:4]}")

    def _places(self, name: str, t: torch.Tensor):
        if name in ("embed", "final.norm"):
            return [((self.embed if name == "embed" else self.final_norm).data, t)]
        first, rest = name.split(".", 1)
        layer = self.own[first[1:]]
        if rest in ("norm1", "norm2"):
            return [(getattr(layer, rest).data, t)]
        if rest.startswith("mlp."):
            m, ff = layer.mlp, layer.mlp.down.in_features
            return [({"gate": m.gate_up.weight.data[:ff], "up": m.gate_up.weight.data[ff:], "down": m.down.weight.data}[rest[4:]], t)]
        key, mix = rest[4:], layer.mix
        parts = mix.pieces_of(key, t) if isinstance(mix, ParallelMixer) else [(key, t)]
        if key == "right.in" and len(parts) == 1:
            raise ValueError(f"{name}: checkpoint tensor {tuple(t.shape)} does not fit "
                             f"{(mix.ssm.inner + mix.ssm.channels + mix.ssm.heads, mix.in_proj.in_features)}")
        return [(mix.destination(k), part) for k, part in parts]

    @torch.no_grad()
    def init_synthetic(self, device, seed: int = 0):
        """Random weights of a checkpoint's scale on the device (benchmarks, tests)."""
        g = torch.Generator(device="cpu").manual_seed(seed)
        self.to(device)
        for name, p in self.named_parameters():
            leaf = name.rsplit(".", 1)[-1]
            if leaf == "conv":
                p.copy_((torch.randn(p.shape, generator=g) * 0.5).to(p.dtype))
            elif p.dim() >= 2:
                std = 1.0 if name in ("embed", ) or leaf == "rel" else p.shape[-1] ** -0.5
                p.copy_((torch.randn(p.shape, generator=g) * std).to(p.dtype))
            elif "norm" in leaf or leaf == "skip":
                p.copy_((1.0 + 0.1 * torch.randn(p.shape, generator=g)).to(p.dtype))
            else:
                p.copy_((0.1 * torch.randn(p.shape, generator=g)).to(p.dtype))
        for layer in self.own.values():          # the fused products' padding rows stay zero
            mix = layer.mix
            used = sum(mix.splits[:len(mix.names)])
            mix.in_proj.weight.data[used:].zero_()
            if mix.in_proj.bias is not None:
                mix.in_proj.bias.data[mix.at["left.g"].start:].zero_()
        return self.finalize()


def load_nukezen(model_dir: str, hf: Dict[str, Any], dtype: torch.dtype, device, **_unused) -> NukezenForCausalLM:
    from .loader import iter_safetensors, safetensors_shapes
    model = NukezenForCausalLM(NukezenConfig.from_dict(hf, safetensors_shapes(model_dir)), dtype)
    model.load_weights(iter_safetensors(model_dir))
    model.to(device)
    return model.finalize()
