"""Vivisun: a decoder around an fp32 residual stream whose two sublayers run side by side, each behind a norm of its own, where the
norm is a dynamic tanh; a span of its layers runs several times in a row.

  x = embed[token]
  layer:   x += mixer(norm1(x)) + ff(norm2(x))                 (the second only if the layer has a feed-forward)
  loop:    layers start .. stop - 1 run ``times`` times with the same weights and caches of their own per pass; ahead of every pass
           but the first, embed[token] joins x once more
  logits = head norm_final(x);   norm(x) = tanh(alpha x) w + b  (DynamicTanh)

Mixers, by the layer's ``type``:
  attention         GroupedQueryAttention: short causal convolutions on q, k and v, per-head q / k norm, partial rotation with YaRN-scaled
                    frequencies, elementwise sigmoid gate
  latent_attention  LatentAttention without positions and without a query latent, a sink per head, a sigmoid gate per head
The feed-forward is GatedMLP with silu.  Every size and constant comes from config.json.  The dynamic tanh, the norms inside the mixers,
angles, scores, softmax and the residual are fp32 also in a bfloat16 model.

A layer's two output products are one (JoinedOutput), and one launch (``residual_tanh_norm``) adds its result to the residual -- with
the embedding row where a pass begins -- and makes both inputs of the next layer; the first such launch starts the stream."""
from dataclasses import dataclass, field
from typing import Any, Dict, Iterable, List, Optional, Tuple

import torch
from torch import nn
from torch.nn import functional as F

from . import mixer_ops as mops
from .mixers import (DynamicTanh, GatedMLP, GroupedQueryAttention, JoinedOutput, LatentAttention, RotaryFrequencies, looped_layers)
from .step_batch import StepBatch

MIXER_TYPES = ("attention", "latent_attention")


@dataclass
class VivisunConfig:
    vocab: int
    width: int
    eps: float
    layers: List[Dict[str, Any]]
    runs: List[Tuple[int, bool]] = field(default_factory=list)       # (layer, whether the embedding output joins x ahead of it)

    @staticmethod
    def from_dict(c: Dict[str, Any]) -> "VivisunConfig":
        cfg = VivisunConfig(vocab=int(c["vocab"]), width=int(c["width"]), eps=float(c["norm"]["eps"]), layers=list(c["layers"]))
        for i, lc in enumerate(cfg.layers):
            if lc["type"] not in MIXER_TYPES:
                raise ValueError(f"layer {i}: unknown mixer type {lc['type']!r}")
            mlp = lc.get("mlp")
            if mlp is not None and mlp.get("kind") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward kind {mlp.get('kind')!r}")
        loop = c.get("loop") or {}
        cfg.runs = looped_layers(len(cfg.layers), int(loop.get("start", 0)), int(loop.get("stop", 0)), int(loop.get("times", 1)))
        return cfg


def rotary_from_config(rot: Optional[Dict[str, Any]]) -> RotaryFrequencies:
    if not rot:
        return RotaryFrequencies(0, 1.0)
    sc = rot.get("scaling")
    if not sc:
        return RotaryFrequencies(int(rot["dims"]), float(rot["base"]))
    return RotaryFrequencies(int(rot["dims"]), float(rot["base"]), float(sc["factor"]), float(sc["original"]), float(sc["fast"]),
                             float(sc["slow"]))


class ConvAttentionMixer(nn.Module):
    """One input product [q | k | v | g] and GroupedQueryAttention behind short convolutions; the output product is the layer's."""

    def __init__(self, cfg: VivisunConfig, mc: Dict[str, Any], dtype, prefix: str):
        super().__init__()
        from .loader import merged_plan
        from .model import QuantLinear
        H, e = int(mc["heads"]), int(mc["vdim"])
        self.attn = GroupedQueryAttention(H, int(mc["kv_heads"]), int(mc["dim"]), e, float(mc["scale"]), cfg.eps, dtype, qk_norm="head",
                                          rotary=rotary_from_config(mc.get("rot")), taps=int(mc.get("conv") or 0))
        self.out_features = H * e
        self.names = ["q", "k", "v", "g"]
        self.splits = self.attn.splits + [H * e]
        self.at = {n: slice(sum(self.splits[:i]), sum(self.splits[:i + 1])) for i, n in enumerate(self.names)}
        pad = -sum(self.splits) % 8               # rows of the fused product stay 16-byte multiples
        if pad:
            self.splits = self.splits + [pad]
        self.in_proj = QuantLinear(cfg.width, self.splits, None, dtype, prefix=prefix + "in_proj", plan=merged_plan(self.splits))
        self.in_proj.weight.data.zero_()

    def cache_specs(self):
        return (self.attn.cache_spec(), ) + ((self.attn.state_spec(), ) if self.attn.taps else ())

    def finalize(self) -> None:
        self.attn.finalize(self.in_proj.weight.device)

    def run(self, h: torch.Tensor, caches, batch: StepBatch, out: torch.Tensor, rows: Optional[torch.Tensor]) -> None:
        proj = self.in_proj(h)
        a = self.attn
        o = out if rows is None else torch.empty(h.shape[0], self.out_features, dtype=h.dtype, device=h.device)
        gate = proj[:, self.at["g"]]
        if a.taps:
            a.forward_conv(o, proj[:, :a.channels], gate, caches[0], caches[1], batch)
        else:
            a(o, *(proj[:, self.at[n]] for n in ("q", "k", "v")), gate, caches[0], batch)
        if rows is not None:
            out.copy_(o.index_select(0, rows))

    def tensor_names(self) -> List[str]:
        return ["q", "k", "v", "q.norm", "k.norm", "g"] + ([n + ".conv" for n in "qkv"] if self.attn.taps else [])

    def load(self, key: str, t: torch.Tensor, put, name: str) -> None:
        a = self.attn
        if key in self.names:
            put(self.in_proj.weight.data[self.at[key]], t, name)
        elif key.endswith(".conv"):
            put(a.conv.data[self.at[key[:-5]]], t, name)
        else:
            put((a.q_norm if key == "q.norm" else a.k_norm).data, t, name)


class SinkLatentMixer(LatentAttention):
    """LatentAttention in this model's form."""

    def __init__(self, cfg: VivisunConfig, mc: Dict[str, Any], dtype, prefix: str):
        super().__init__(cfg.width, int(mc["heads"]), int(mc["dim"]), 0, int(mc["vdim"]), 0, int(mc["kv_rank"]), float(mc["scale"]),
                         RotaryFrequencies(0, 1.0), cfg.eps, dtype, prefix=prefix, gate="head", sink=True, project=False)
        self.out_features = self.heads * self.vdim

    def cache_specs(self):
        return (self.cache_spec(), )

    def run(self, h: torch.Tensor, caches, batch: StepBatch, out: torch.Tensor, rows: Optional[torch.Tensor]) -> None:
        self.attend(h, caches[0], batch, out, rows)

    def tensor_names(self) -> List[str]:
        return ["q", "dkv", "dkv.norm", "uk", "uv", "sink", "g"]

    def load(self, key: str, t: torch.Tensor, put, name: str) -> None:
        if key in self.names:
            i = self.names.index(key)
            at = sum(self.splits[:i])
            put(self.in_proj.weight.data[at:at + self.splits[i]], t, name)
        elif key in ("uk", "uv"):
            self.load_up_projection(key, t, name)
        else:
            put((self.kv_norm if key == "dkv.norm" else self.sink).data, t, name)


class VivisunLayer(nn.Module):
    def __init__(self, cfg: VivisunConfig, index: int, dtype):
        super().__init__()
        lc = cfg.layers[index]
        pfx = f"l{index}."
        kind = {"attention": ConvAttentionMixer, "latent_attention": SinkLatentMixer}[lc["type"]]
        self.mix = kind(cfg, lc["mixer"], dtype, pfx + "mix.")
        self.norm1 = DynamicTanh(cfg.width, dtype)
        self.mlp = self.norm2 = None
        if lc.get("mlp") is not None:
            self.mlp = GatedMLP(cfg.width, int(lc["mlp"]["ff"]), mops.ACT_SILU, dtype, pfx + "mlp.", down=False)
            self.norm2 = DynamicTanh(cfg.width, dtype)
        self.out = JoinedOutput([self.mix.out_features] + ([self.mlp.ff] if self.mlp is not None else []), cfg.width, dtype, pfx + "out")

    def norms(self) -> List[DynamicTanh]:
        return [self.norm1] + ([self.norm2] if self.norm2 is not None else [])

    def forward(self, inputs: List[torch.Tensor], caches, batch: StepBatch, rows: Optional[torch.Tensor]) -> torch.Tensor:
        """mixer(inputs[0]) + ff(inputs[1]); ``rows``: of these rows only (caches and states advance over all of them)."""
        h = inputs[0]
        buf, parts = self.out.buffer(h.shape[0] if rows is None else rows.shape[0], h.dtype, h.device)
        self.mix.run(h, caches, batch, parts[0], rows)
        if self.mlp is not None:
            self.mlp.inner(inputs[1] if rows is None else inputs[1].index_select(0, rows), parts[1])
        return self.out(buf)


class VivisunForCausalLM(nn.Module):
    def __init__(self, cfg: VivisunConfig, dtype: torch.dtype = torch.bfloat16):
        super().__init__()
        from .distributed import get_tensor_model_parallel_world_size
        if get_tensor_model_parallel_world_size() != 1:
            raise ValueError("Vivisun runs on one rank")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Vivisun runs in bfloat16 or float32")
        self.cfg, self.dtype = cfg, dtype
        self.embed = nn.Parameter(torch.empty(cfg.vocab, cfg.width, dtype=dtype), requires_grad=False)
        self.layers = nn.ModuleList([VivisunLayer(cfg, i, dtype) for i in range(len(cfg.layers))])
        self.final_norm = DynamicTanh(cfg.width, dtype)
        self.head = nn.Parameter(torch.empty(cfg.vocab, cfg.width, dtype=dtype), requires_grad=False)
        # every pass over a layer has caches of its own
        self.specs, self.run_caches = [], []
        for i, _ in cfg.runs:
            specs = self.layers[i].mix.cache_specs()
            self.run_caches.append(range(len(self.specs), len(self.specs) + len(specs)))
            self.specs += list(specs)
        self.residual_trace: Optional[List[torch.Tensor]] = None     # set to [] to record x after every layer run

    # ---- what the engine asks of a model ---------------------------------------------------------------------------
    @property
    def vocab_size(self) -> int:
        return self.cfg.vocab

    def make_caches(self, num_blocks: int, block_size: int, num_slots: int, device):
        return [s.allocate(num_blocks, block_size, num_slots, self.dtype, device) for s in self.specs]

    def finalize(self):
        for layer in self.layers:
            layer.mix.finalize()
            for n in layer.norms():
                n.finalize()
        self.final_norm.finalize()
        return self

    @torch.no_grad()
    def step(self, batch: StepBatch, caches, rows: torch.Tensor) -> torch.Tensor:
        """One engine step: run the batch's rows through every layer (caches and states advance), return the fp32 logits of
        ``rows`` (int64 indices into the batch)."""
        return self.logits(self.forward(batch, caches, rows))

    def logits(self, h: torch.Tensor) -> torch.Tensor:
        return F.linear(h, self.head).float()

    def forward(self, batch: StepBatch, caches, rows: Optional[torch.Tensor] = None) -> torch.Tensor:
        """The final norm's output for the rows asked for (all rows if ``rows`` is None).  In the last layer run everything behind the
        caches and states runs on those rows only."""
        runs, trace = self.cfg.runs, self.residual_trace
        norms = [[n.operand() for n in self.layers[i].norms()] for i, _ in runs] + [[self.final_norm.operand()]]
        x = torch.empty(batch.num_tokens, self.cfg.width, dtype=torch.float32, device=self.embed.device)
        h = mops.residual_tanh_norm(x, table=self.embed, ids=batch.input_ids, norms=norms[0], fresh=True)
        for j, (i, _) in enumerate(runs):
            last = j + 1 == len(runs)
            only = rows if last and trace is None else None
            y = self.layers[i](h, [caches[c] for c in self.run_caches[j]], batch, only)
            if only is not None:
                x = x.index_select(0, only)
            if trace is not None:
                mops.residual_tanh_norm(x, y)
                trace.append(x.clone())
                y = None
            again = not last and runs[j + 1][1]
            h = mops.residual_tanh_norm(x, y, table=self.embed if again else None, ids=batch.input_ids if again else None, norms=norms[j + 1],
                                        dtype=self.dtype)
        h = h[0]
        if rows is not None and (not runs or trace is not None):
            h = h.index_select(0, rows)
        return h

    # ---- checkpoint ----------------------------------------------------------------------------------------------------
    def expected_names(self) -> Tuple[List[str], List[str]]:
        """(names a checkpoint must hold, names it may hold)"""
        def norm(n):
            return [n, n + ".b", n + ".alpha"]
        names, optional = ["embed", "head"] + norm("final.norm"), []
        for i, layer in enumerate(self.layers):
            p = f"l{i}."
            names += norm(p + "norm1") + [p + "mix." + n for n in layer.mix.tensor_names() + ["o"]]
            if layer.mlp is not None:
                names += norm(p + "norm2") + [p + "mlp." + n for n in ("gate", "up", "down")]
            else:
                optional += norm(p + "norm2")    # a norm that is never applied
        return names, optional

    def load_weights(self, weights: Iterable[Tuple[str, torch.Tensor]]) -> None:
        """Checkpoint names: embed, head, and l<i>.norm{1,2} / final.norm with their .b and .alpha, l<i>.mix.* by the layer's type,
        l<i>.mlp.{gate,up,down}."""
        names, optional = self.expected_names()
        expected, seen = set(names), set()
        for name, t in weights:
            if name in optional:
                continue
            if name not in expected:
                raise ValueError(f"unexpected tensor {name!r} in a Vivisun checkpoint")
            seen.add(name)
            self._load_one(name, t)
        missing = expected - seen
        if "head" in missing:                    # no output matrix of its own: the embedding's
            self.head = self.embed
            missing.discard("head")
        if missing:
            raise ValueError(f"checkpoint lacks {len(missing)} tensors, e.g. {sorted(missing)[:4]}")

    @staticmethod
    def _put(dst: torch.Tensor, t: torch.Tensor, name: str) -> None:
        if tuple(dst.shape) != tuple(t.shape):
            raise ValueError(f"{name}: checkpoint tensor {tuple(t.shape)} does not fit {tuple(dst.shape)}")
        dst.copy_(t.to(dst.dtype))

    def _load_one(self, name: str, t: torch.Tensor) -> None:
        put = self._put
        if name in ("embed", "head"):
            return put(getattr(self, name).data, t, name)
        base, part = (name[:-2], "bias") if name.endswith(".b") else (name[:-6], "alpha") if name.endswith(".alpha") else (name, "weight")
        if base == "final.norm":
            return put(getattr(self.final_norm, part).data, t.reshape(()) if part == "alpha" else t, name)
        layer = self.layers[int(name.split(".", 1)[0][1:])]
        rest = name.split(".", 1)[1]
        if rest.startswith("norm"):
            norm = layer.norm1 if rest.startswith("norm1") else layer.norm2
            return put(getattr(norm, part).data, t.reshape(()) if part == "alpha" else t, name)
        if rest == "mix.o":
            return put(layer.out.weight_of(0), t, name)
        if rest.startswith("mix."):
            return layer.mix.load(rest[4:], t, put, name)
        m = layer.mlp
        put({"gate": m.gate_up.weight.data[:m.ff], "up": m.gate_up.weight.data[m.ff:], "down": layer.out.weight_of(-1)}[rest[4:]], t, name)

    @torch.no_grad()
    def init_synthetic(self, device, seed: int = 0):
        """Random weights of a checkpoint's scale on the device (benchmarks, tests)."""
        g = torch.Generator(device="cpu").manual_seed(seed)
        self.to(device)
        for name, p in self.named_parameters():
            leaf = name.rsplit(".", 1)[-1]
            if leaf == "conv":
                p.copy_((torch.randn(p.shape, generator=g) * 0.5).to(p.dtype))
            elif leaf == "alpha":
                p.fill_(0.5)
            elif p.dim() >= 2:
                std = 1.0 if name == "embed" else p.shape[-1] ** -0.5
                p.copy_((torch.randn(p.shape, generator=g) * std).to(p.dtype))
            elif "norm" in name and leaf != "bias":
                p.copy_((1.0 + 0.1 * torch.randn(p.shape, generator=g)).to(p.dtype))
            else:
                p.copy_((0.1 * torch.randn(p.shape, generator=g)).to(p.dtype))
        for layer in self.layers:                # the fused products' padding stays zero
            mix = layer.mix
            mix.in_proj.weight.data[sum(mix.splits[:len(mix.names)]):].zero_()
            layer.out.zero_padding()
        return self.finalize()


def load_vivisun(model_dir: str, hf: Dict[str, Any], dtype: torch.dtype, device, **_unused) -> VivisunForCausalLM:
    from .loader import iter_safetensors
    model = VivisunForCausalLM(VivisunConfig.from_dict(hf), dtype)
    model.load_weights(iter_safetensors(model_dir))
    model.to(device)
    return model.finalize()
