"""Koduzen: a decoder-only stack over hyper-connected residual streams (models/hyper.py) with RMS norms, its
layers listed one by one in the configuration.

Mixers (models/mixers.py):
  ``retention``    linear attention whose state forgets with a fixed decay per head: rotated queries and
                   keys, no softmax; each head's result by its root mean square, times silu(W_g h)
  ``attention``    windowed grouped attention; queries and keys pass RMS norms over their whole projections
                   ahead of a partial half-split rotation with ramp-scaled frequencies
  ``attention_2``  windowed grouped attention without rotation: queries warmed with their position, a distance
                   bias per head, a learned sink per head; with ``kv_from`` over the keys and values of an
                   earlier such layer, which it reads from that layer's cache
Feed-forward: clamped gated units (g sigmoid(1.702 g) (u + 1)), dense or as experts - chosen inside the best
groups by softmax scores with a selection-only correction, identity experts among them - beside a shared
one that runs for every token; or none. The head is the embedding table.

Attention layers that own their keys cache in the paged pools (one per layer); the retention states live in
the state pool. A stack without retention layers has no state slots and may reuse cached prefixes.
"""
from __future__ import annotations

import torch

from llmd_amd.engine.attn_meta import AttnMeta
from llmd_amd.engine.config import ModelConfig
from llmd_amd.parallel.state import get_state

from .hyper import HyperConnection, stream_stack
from .layers import LMHead, VocabEmbedding
from .mixers import GatedMLP, GroupedAttention, RetentionMixer, ScoreMoE, _param

ACT = "swish_limit"


def make_mixer(spec: dict, d: int, eps: float, max_pos: int, device, dtype, earlier: list):
    """``earlier``: the mixers of the layers before this one (shared keys and values name one)."""
    t, m = spec["type"], spec["mixer"]
    if t == "retention":
        return RetentionMixer(d, m["heads"], m["dim"], m["vdim"], m["decay"], m.get("rot"), eps, max_pos, device, dtype)
    window = int((m.get("mask") or {}).get("size") or 0)
    src = m.get("kv_from")
    kw = dict(bias=False, interleaved=False, unit_norm=False, v_mix=False, gate=False, window=window,
              kv_source=None if src is None else earlier[src])
    if t == "attention":
        return GroupedAttention(d, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], m.get("rot"), eps,
                                max_pos, device, dtype, wide_norm=True, **kw)
    if t == "attention_2":
        return GroupedAttention(d, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], None, eps, max_pos, device,
                                dtype, slopes="pow2", sink="learned", q_temp=m.get("q_temp"), **kw)
    raise ValueError(f"unknown mixer type {t!r}")


def make_mlp(m, d: int, device, dtype):
    if m is None:
        return None
    if m["kind"] == "dense":
        return GatedMLP(d, m["ff"], ACT, device, dtype, limit=m["limit"])
    if m["kind"] == "moe":
        r, g, s = m["router"], m["router"].get("groups") or {}, m.get("shared")
        shared = GatedMLP(d, s["ff"], ACT, device, dtype, limit=s["limit"]) if s else None
        return ScoreMoE(d, m["expert"]["ff"], r["experts"], r.get("identity", 0), r["top"], ACT, device, dtype,
                        limit=m["expert"]["limit"], groups=g.get("count", 1), keep=g.get("keep", 1),
                        scale=r.get("scale", 1.0), shared=shared)
    raise ValueError(f"unknown feed-forward kind {m['kind']!r}")


class KoduzenLayer(torch.nn.Module):
    def __init__(self, cfg: ModelConfig, idx: int, max_pos: int, device, dtype, earlier: list):
        super().__init__()
        spec = cfg.layer_specs[idx]
        d, eps = cfg.hidden_size, cfg.rms_norm_eps
        S, learned = max(1, cfg.hyper_streams), cfg.hyper_streams > 0
        self.mix = make_mixer(spec, d, eps, max_pos, device, dtype, earlier)
        self.mlp = make_mlp(spec.get("mlp"), d, device, dtype)
        self.norm1 = _param((d,), device, dtype, fill=1.0)
        self.hc1 = HyperConnection(S, learned, device, dtype)
        if self.mlp is not None:
            self.norm2 = _param((d,), device, dtype, fill=1.0)
            self.hc2 = HyperConnection(S, learned, device, dtype)


class KoduzenForCausalLM(torch.nn.Module):
    supports_float32 = True
    seq_steps = True  # steps are described per sequence (AttnMeta.seq)

    def __init__(self, cfg: ModelConfig, device="cuda", max_pos: int = 32768, dtype=torch.bfloat16):
        super().__init__()
        if get_state().tp_size != 1:
            raise ValueError("koduzen runs on one rank (its recurrent layers are not tensor-parallel)")
        self.cfg, self.dtype = cfg, dtype
        d = cfg.hidden_size
        self.embed = VocabEmbedding(cfg.vocab_size, d, device, dtype=dtype)
        self.layers = torch.nn.ModuleList()
        for i in range(cfg.num_hidden_layers):
            self.layers.append(KoduzenLayer(cfg, i, max_pos, device, dtype, [l.mix for l in self.layers]))
        self.norm = _param((d,), device, dtype, fill=1.0)
        self.lm_head = LMHead(cfg.vocab_size, d, device, dtype=dtype, tied=self.embed)
        self.ones = torch.ones(max(1, cfg.hyper_streams), dtype=torch.float32, device=device)
        self.stateful = bool(self.state_layers())  # recurrences: no prefix reuse, one state slot per sequence
        self.finalize()

    def finalize(self):
        """Derived constants (fp32 copies of small tensors): after every weight load."""
        for m in self.modules():
            if m is not self and hasattr(m, "finalize"):
                m.finalize()

    def attention_layers(self):
        """The mixers that own a paged cache (a layer that reads another's keys and values has none)."""
        return [l.mix for l in self.layers if isinstance(l.mix, GroupedAttention) and l.mix.owns_cache]

    def state_layers(self):
        return [l.mix for l in self.layers if hasattr(l.mix, "state_shapes")]

    def kv_specs(self):
        return [a.kv_spec() for a in self.attention_layers()]

    @torch.no_grad()
    def forward(self, input_ids, meta: AttnMeta, layer_out=None):
        """``layer_out``: optional list that receives the sum of the streams after every layer."""
        subs = []
        for l in self.layers:
            subs.append((l.hc1, l.norm1, lambda h, m=l.mix: m(h, meta), l.mlp is None))
            if l.mlp is not None:
                subs.append((l.hc2, l.norm2, l.mlp, True))
        return stream_stack(input_ids, self.embed.weight, self.ones, subs, self.norm, self.cfg.rms_norm_eps, self.dtype,
                            rms=True, layer_out=layer_out)

    @torch.no_grad()
    def compute_logits(self, h):
        # over the table's padded rows, so that the rows stay 16-byte aligned for the sampling kernel
        logits = torch.nn.functional.linear(h, self.lm_head.weight).float()
        return logits[:, :self.cfg.vocab_size]

    def weight_specs(self) -> list:
        specs = [("embed", self.embed.weight, "vocab", None), ("final.norm", self.norm, "replicate", None)]

        def add(name, p, kind="replicate", extra=None):
            specs.append((name, p, kind, extra))

        def fused(pre, w, parts):
            off = 0
            for n, rows in parts:
                if rows:
                    add(pre + n, w, "fused", (off, 1, rows))
                off += rows

        def gated(pre, f):
            fused(pre, f.gate_up.weight, (("gate", f.ff), ("up", f.ff)))
            add(pre + "down", f.down.weight)

        for i, layer in enumerate(self.layers):
            pre = f"l{i}."
            for q in ("1", "2"):
                if hasattr(layer, "norm" + q):
                    add(pre + "norm" + q, getattr(layer, "norm" + q))
                    hc = getattr(layer, "hc" + q)
                    if hc.learned:
                        for n, p in (("in", hc.w_in), ("out", hc.w_out), ("mix", hc.mix)):
                            add(f"{pre}hc{q}.{n}", p)
            m, mp = layer.mix, pre + "mix."
            if isinstance(m, RetentionMixer):
                fused(mp, m.proj.weight, (("q", m.nq), ("k", m.nq), ("v", m.nv), ("g", m.nv)))
            else:
                fused(mp, m.proj.weight, (("q", m.nq), ("k", m.nk), ("v", m.nv)))
                if m.wide_norm:
                    add(mp + "q.norm", m.q_norm)
                    if m.nk:
                        add(mp + "k.norm", m.k_norm)
                if hasattr(m, "sink"):
                    add(mp + "sink", m.sink)
            add(mp + "o", m.o.weight)
            f, fp = layer.mlp, pre + "mlp."
            if isinstance(f, GatedMLP):
                gated(fp, f)
            elif f is not None:
                add(fp + "router", f.router)
                add(fp + "correction", f.correction)
                for e in range(f.E):
                    add(f"{fp}e{e}.gate", f.w1[e, :f.ff])
                    add(f"{fp}e{e}.up", f.w1[e, f.ff:])
                    add(f"{fp}e{e}.down", f.w2[e])
                if f.shared is not None:
                    gated(fp + "shared.", f.shared)
        return specs
