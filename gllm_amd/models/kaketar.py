"""Kaketar: a config-driven decoder of latent attention and a
channel-decayed delta rule over a post-norm residual.

``config.layers`` describes every layer on its own (mixer type, mixer
sizes, feed-forward or none), so sizes may differ from layer to layer
and the layers come in any order.

* stream: fp32. It opens with RMSnorm(embed[token] * embedding.scale +
  pos[p]); a sublayer reads the stream itself and only its RESULT is
  normed, x += RMSnorm(f(x)) * (1 + w) (weights stored around zero)
* mixer ``latent_attention``: queries through a normed latent of their
  own, keys and values as up-projections of a cached normed latent, plus
  a rotated query/key part (interleaved pairs, YaRN frequencies) whose
  key half is shared by the heads; a sliding window, a learned per-head
  sink in the softmax denominator, and a sigmoid gate per output element
* mixer ``channel_delta``: gated delta rule with a decay per (value
  head, key channel) from a low-rank branch, short silu convolutions on
  q, k and v, grouped unit q/k heads, fp32 state, and a read-out through
  a per-head RMS norm and a low-rank sigmoid gate
* feed-forward: dense up -> exact gelu -> down, or none
* after every layer, a per-token side input: a slice of a token table
  gates a low-width projection of the stream, and the projected-back,
  RMS-normed result joins the stream
* logits: RMSnorm(x) * (1 + w), head, cap * tanh(. / cap)

Framework mapping: one merged input projection per mixer (dq | dkv | g;
q | k | v | a1 | g1 | b) and, for the two low-rank branches, one second
GEMM with a block-diagonal weight (layers/linear.py); NormedEmbedding
and TokenSideInput (layers/embedding.py); StreamRMSNorm.add_into = one
launch per sublayer boundary (layers/layernorm.py); LatentAttention +
PairRotary (layers/attention.py, layers/rotary.py); ChannelDeltaRule
over the state pool (layers/recurrent.py, core/ssm.py); the paged KV
pool with per-layer shapes, [latent | rotated key part] per token and no
value cache (core/kv_cache.py). Prompt portions and decode tokens of a
mixed batch run through the same ragged kernels.
"""

from typing import Iterable, List, Optional, Tuple

import torch
import torch.nn as nn

from gllm_amd import ops
from gllm_amd.core.ssm import SSMLayerSpec, SSMSpec
from gllm_amd.layers.activation import GELU
from gllm_amd.layers.attention import LatentAttention
from gllm_amd.layers.embedding import (NormedEmbedding, ParallelLMHead,
                                       TokenSideInput)
from gllm_amd.layers.layernorm import StreamRMSNorm
from gllm_amd.layers.linear import (MergedColumnParallelLinear,
                                    ReplicatedLinear, RowParallelLinear)
from gllm_amd.layers.recurrent import ChannelDeltaRule
from gllm_amd.layers.rotary import PairRotary
from gllm_amd.runtime.forward_context import ForwardContext

# the design's norm weights are stored as their distance from one
NORM_OFFSET = 1.0


def _get(d, key, default=None):
    """config.json sub-objects arrive as dicts (or namespaces)."""
    if d is None:
        return default
    if isinstance(d, dict):
        return d.get(key, default)
    return getattr(d, key, default)


def _copy(param, w):
    assert tuple(param.shape) == tuple(w.shape), \
        (tuple(param.shape), tuple(w.shape))
    param.data.copy_(w.to(param.dtype))


class LatentMixer(nn.Module):
    """dq | dkv | gate in one projection, normed query latent ->
    queries, attention over the cached latent, output projection."""

    def __init__(self, width: int, m, eps: float, kv_index: int, dtype):
        super().__init__()
        H, D, Dv = int(_get(m, "heads")), int(_get(m, "dim")), \
            int(_get(m, "vdim"))
        Dr = int(_get(m, "rot_dim", 0) or 0)
        R, Rq = int(_get(m, "kv_rank")), int(_get(m, "q_rank"))
        self.eps = eps
        self.cache_shape = (1, R + Dr, 0)  # one row is key and value
        self.sizes = [Rq, R + Dr, H * Dv]
        self.in_proj = MergedColumnParallelLinear(width, self.sizes,
                                                  params_dtype=dtype)
        self.q_norm = nn.Parameter(torch.ones(Rq, dtype=dtype),
                                   requires_grad=False)
        self.uq = ReplicatedLinear(Rq, H * (D + Dr), params_dtype=dtype)
        rotary = None
        if Dr:
            rot = _get(m, "rot")
            if int(_get(rot, "dims", Dr)) != Dr:
                raise ValueError("rot.dims must equal rot_dim")
            rotary = PairRotary(Dr, float(_get(rot, "base")),
                                _get(rot, "scaling"))
        mask = _get(m, "mask")
        self.attn = LatentAttention(
            kv_index, H, D, Dv, R, float(_get(m, "scale")), eps,
            params_dtype=dtype, rot_dim=Dr, rotary=rotary,
            window=int(_get(mask, "size", 0) or 0), sink=True)
        self.out_proj = RowParallelLinear(H * Dv, width, params_dtype=dtype)

    def forward(self, h: torch.Tensor, fctx: ForwardContext):
        cq, ckv, gate = self.in_proj(h).split(self.sizes, dim=-1)
        q = self.uq(ops.rms_weight_store(cq, self.q_norm, self.eps))
        return self.out_proj(self.attn(q, ckv, fctx, gate))

    def load(self, sub: List[str], w) -> bool:
        at = self.attn
        shard = {"dq": 0, "dkv": 1, "g": 2}
        if len(sub) == 1 and sub[0] in shard:
            p = self.in_proj.weight
            p.weight_loader(p, w, shard[sub[0]])
        elif sub in (["uk"], ["uv"]):
            at.load_up(sub[0], w)
        else:
            p = {"dq.norm": self.q_norm, "dkv.norm": at.kv_norm,
                 "uq": self.uq.weight, "sink": at.sinks,
                 "o": self.out_proj.weight}.get(".".join(sub))
            if p is None:
                return False
            _copy(p, w)
        return True

    def finish_load(self, name: str) -> None:
        pass


class ChannelDeltaMixer(nn.Module):
    """q | k | v | a1 | g1 | b in one projection, (a2 | g2) in a second
    one, the recurrence, output projection."""

    # column blocks of the first projection, in order
    SHARDS = {"q": 0, "k": 1, "v": 2, "a1": 3, "g1": 4, "b": 5}

    def __init__(self, width: int, m, eps: float, ssm_layer_id: int,
                 engine_config, dtype):
        super().__init__()
        H, D, Dv = int(_get(m, "heads")), int(_get(m, "dim")), \
            int(_get(m, "vdim"))
        G = int(_get(m, "kv_heads", H) or H)
        self.width, self.dtype = width, dtype
        self.delta = ChannelDeltaRule(H, G, D, Dv,
                                      int(_get(m, "conv", 1) or 1), eps,
                                      ssm_layer_id, params_dtype=dtype)
        self.decay_size, self.gate_size = H * D, H * Dv
        self.out_proj = RowParallelLinear(H * Dv, width, params_dtype=dtype)
        # the low-rank widths come with the checkpoint (row counts of a1
        # and g1); the projections are sized when both have arrived
        self.in_proj = self.up = None
        self._ranks = {}
        self._pending = []   # tensors that arrived before that
        if engine_config.load_format == "dummy":
            self._size(int(_get(m, "decay_rank", Dv)),
                       int(_get(m, "gate_rank", Dv)))

    def _size(self, ra: int, rg: int) -> None:
        H, dev = self.delta.heads, self.out_proj.weight.device
        self.ranks = (ra, rg)
        self.sizes = self.delta.qkv_sizes + [ra, rg, H]
        # rows padded to 8 keep the projection's output rows 16 B aligned
        pad = -sum(self.sizes) % 8
        self.in_proj = MergedColumnParallelLinear(
            self.width, self.sizes + ([pad] if pad else []),
            params_dtype=self.dtype).to(dev)
        self.in_proj.weight.data.zero_()
        # [a2 0; 0 g2] on [a1 | g1]: both second factors in one GEMM
        self.up = ReplicatedLinear(ra + rg, self.decay_size + self.gate_size,
                                   params_dtype=self.dtype).to(dev)
        self.up.weight.data.zero_()

    def forward(self, h: torch.Tensor, fctx: ForwardContext):
        proj = self.in_proj(h)
        n = self.delta.conv_dim
        m = n + sum(self.ranks)
        low = self.up(proj[:, n:m])
        o = self.delta(proj[:, :n], low[:, :self.decay_size],
                       proj[:, m:m + self.delta.heads],
                       low[:, self.decay_size:], fctx)
        return self.out_proj(o)

    def load(self, sub: List[str], w) -> bool:
        if self.in_proj is None:
            self._pending.append((sub, w))
            if sub in (["a1"], ["g1"]):
                self._ranks[sub[0]] = int(w.shape[0])
            if len(self._ranks) < 2:
                return True
            self._size(self._ranks["a1"], self._ranks["g1"])
            pending, self._pending = self._pending, []
            for ps, pw in pending:
                if not self.load(ps, pw) and pw.is_floating_point():
                    raise KeyError(f"unexpected tensor mix.{'.'.join(ps)}")
            return True
        dl = self.delta
        shard = self.SHARDS.get(sub[0])
        if shard is not None and len(sub) == 1:
            p = self.in_proj.weight
            p.weight_loader(p, w, shard)
        elif shard is not None and shard < 3 and sub[1:] == ["conv"]:
            off = sum(dl.qkv_sizes[:shard])
            _copy(dl.conv_weight.data[off:off + dl.qkv_sizes[shard]], w)
        elif sub == ["a2"]:
            _copy(self.up.weight.data[:self.decay_size, :self.ranks[0]], w)
        elif sub == ["g2"]:
            _copy(self.up.weight.data[self.decay_size:, self.ranks[0]:], w)
        else:
            p = {"A_log": dl.A_log, "dt_bias": dl.dt_bias,
                 "norm": dl.norm_weight,
                 "o": self.out_proj.weight}.get(".".join(sub))
            if p is None:
                return False
            _copy(p, w)
        return True

    def finish_load(self, name: str) -> None:
        if self.in_proj is None:
            raise KeyError(f"{name}.a1 or {name}.g1 is missing")


class DenseGELU(nn.Module):
    """up -> exact gelu -> down."""

    def __init__(self, width: int, mlp, dtype):
        super().__init__()
        ff = int(_get(mlp, "ff"))
        self.up = ReplicatedLinear(width, ff, params_dtype=dtype)
        self.act = GELU()
        self.down = RowParallelLinear(ff, width, params_dtype=dtype)

    def forward(self, h: torch.Tensor):
        return self.down(self.act(self.up(h)))


class KaketarLayer(nn.Module):
    def __init__(self, width: int, layer, index: int, side_dim: int,
                 eps: float, kv_index: int, ssm_layer_id: int,
                 engine_config, dtype):
        super().__init__()
        self.kind = _get(layer, "type")
        m = _get(layer, "mixer")
        if self.kind == "latent_attention":
            self.mix = LatentMixer(width, m, eps, kv_index, dtype)
        elif self.kind == "channel_delta":
            self.mix = ChannelDeltaMixer(width, m, eps, ssm_layer_id,
                                         engine_config, dtype)
        else:
            raise ValueError(f"unknown mixer type {self.kind!r}")
        self.norm1 = StreamRMSNorm(width, eps, dtype, NORM_OFFSET)
        mlp = _get(layer, "mlp")
        self.mlp = self.norm2 = None
        if mlp:
            if _get(mlp, "kind") != "dense":
                raise ValueError("unknown feed-forward kind "
                                 f"{_get(mlp, 'kind')!r}")
            self.mlp = DenseGELU(width, mlp, dtype)
            self.norm2 = StreamRMSNorm(width, eps, dtype, NORM_OFFSET)
        self.side = self.side_norm = None
        if side_dim:
            self.side = TokenSideInput(width, side_dim, index, dtype)
            self.side_norm = StreamRMSNorm(width, eps, dtype)

    def forward(self, x: torch.Tensor, h: torch.Tensor, input_ids,
                side_table, fctx: ForwardContext,
                nxt: Optional[StreamRMSNorm]):
        """x: fp32 stream (updated in place); h = x in the model dtype.
        Returns ``nxt`` applied to the updated x, or x itself in the
        model dtype without ``nxt``."""
        steps = [(self.norm1, lambda h: self.mix(h, fctx))]
        if self.mlp is not None:
            steps.append((self.norm2, self.mlp))
        if self.side is not None:
            steps.append((self.side_norm, lambda h: self.side(
                h, input_ids, side_table)))
        for j, (norm, sublayer) in enumerate(steps):
            last = j + 1 == len(steps)
            h = norm.add_into(x, sublayer(h), nxt if last else None,
                              read=True)
        return h


class KaketarForCausalLM(nn.Module):
    # the ragged state kernels read slots / flags from device tensors
    wants_state_tensors = True
    # no host sync in the forward: decode buckets can be captured
    supports_graph = True

    def __init__(self, cfg, engine_config):
        super().__init__()
        from gllm_amd.parallel import get_pp_size, get_tp_size
        assert get_tp_size() == 1 and get_pp_size() == 1, \
            "Kaketar serves on one GPU per replica (tp = pp = 1)"
        self.cfg = cfg
        dtype = engine_config.torch_dtype()
        self.dtype = dtype
        layers = list(cfg.layers)
        width, vocab = int(cfg.width), int(cfg.vocab)
        eps = float(_get(cfg.norm, "eps"))
        self.logit_softcap = float(getattr(cfg, "logit_softcap", 0.0) or 0.0)
        # rows of the learned position table: the engine admits no
        # position beyond it
        self.max_positions = int(getattr(cfg, "max_positions", 0) or 0)
        side_dim = int(_get(getattr(cfg, "token_side", None), "dim", 0) or 0)
        # names the rest of the framework reads off a model config
        cfg.vocab_size = vocab
        cfg.hidden_size = width
        cfg.num_hidden_layers = len(layers)
        self.layer_start, self.layer_end = 0, len(layers)
        self.is_first_stage = self.is_last_stage = True
        self.embed = NormedEmbedding(
            vocab, width, eps,
            float(_get(getattr(cfg, "embedding", None), "scale", 1.0)),
            self.max_positions, NORM_OFFSET, dtype)
        if side_dim:
            self.side_embed = nn.Parameter(
                torch.zeros(vocab, side_dim * len(layers), dtype=dtype),
                requires_grad=False)
        else:
            self.side_embed = None
        mods: List[KaketarLayer] = []
        kv_shapes: List[Tuple[int, int, int]] = []
        ssm_specs: List[SSMLayerSpec] = []
        for i, layer in enumerate(layers):
            lay = KaketarLayer(width, layer, i, side_dim, eps,
                               len(kv_shapes), len(ssm_specs),
                               engine_config, dtype)
            if lay.kind == "latent_attention":
                kv_shapes.append(lay.mix.cache_shape)
            else:
                ssm_specs.append(lay.mix.delta.spec())
            mods.append(lay)
        self.layers = nn.ModuleList(mods)
        self.kv_layer_shapes = kv_shapes
        self.num_kv_layers = len(kv_shapes)
        self.ssm_spec = None
        if ssm_specs:
            s0 = ssm_specs[0]
            self.ssm_spec = SSMSpec(len(ssm_specs), s0.conv_dim,
                                    s0.conv_kernel, s0.num_v_heads,
                                    s0.head_k_dim, s0.head_v_dim,
                                    layers=ssm_specs)
        self.final_norm = StreamRMSNorm(width, eps, dtype, NORM_OFFSET)
        self.lm_head = ParallelLMHead(vocab, width, params_dtype=dtype)
        # called as layer_probe(layer index, x) after every layer
        self.layer_probe = None

    @property
    def num_local_layers(self):
        return len(self.layers)

    def forward(self, input_ids, positions, fctx, hidden_states=None,
                residual=None):
        x, h = self.embed(input_ids, positions)
        last = len(self.layers) - 1
        for i, layer in enumerate(self.layers):
            h = layer(x, h, input_ids, self.side_embed, fctx,
                      self.final_norm if i == last else None)
            if self.layer_probe is not None:
                self.layer_probe(i, x)
        return (h if self.layers else self.final_norm(x)), None

    def compute_logits(self, hidden_states, fctx):
        rows = hidden_states
        if fctx.logits_indices is not None:
            rows = hidden_states.index_select(0, fctx.logits_indices)
        logits = self.lm_head(rows).float()
        if self.logit_softcap:
            logits = torch.tanh(logits / self.logit_softcap) \
                * self.logit_softcap
        return logits

    # ------------------------------------------------------------------
    def load_weights(self, weights: Iterable[Tuple[str, torch.Tensor]]):
        """Checkpoint names: ``embed``, ``embed.norm``, ``pos``,
        ``side.embed``, ``head``, ``final.norm`` and per layer
        ``l<i>.norm{1,2}``, ``l<i>.mix.{dq,dq.norm,uq,dkv,dkv.norm,uk,uv,
        sink,g,o}`` (latent_attention) or ``l<i>.mix.{q,k,v}[.conv]``,
        ``.{b,A_log,norm,a1,a2,dt_bias,g1,g2,o}`` (channel_delta),
        ``l<i>.mlp.{up,down}`` and ``l<i>.side.{gate,proj,norm}``."""
        seen = set()
        for name, w in weights:
            if self._load_one(name, w):
                seen.add(name)
            elif w.is_floating_point():
                raise KeyError(f"unexpected tensor {name!r}")
        for i, layer in enumerate(self.layers):
            layer.mix.finish_load(f"l{i}.mix")
        return seen

    def _load_one(self, name: str, w: torch.Tensor) -> bool:
        if name in ("embed", "head"):
            p = (self.embed if name == "embed" else self.lm_head).weight
            p.weight_loader(p, w)
            return True
        p = {"embed.norm": self.embed.norm_weight,
             "pos": self.embed.positions,
             "side.embed": self.side_embed,
             "final.norm": self.final_norm.weight}.get(name)
        if p is not None:
            _copy(p, w)
            return True
        parts = name.split(".")
        if not (parts[0].startswith("l") and parts[0][1:].isdigit()):
            return False
        layer = self.layers[int(parts[0][1:])]
        if parts[1] == "mix":
            return layer.mix.load(parts[2:], w)
        p = None
        if parts[1:] == ["norm1"]:
            p = layer.norm1.weight
        elif parts[1:] == ["norm2"] and layer.norm2 is not None:
            p = layer.norm2.weight
        elif parts[1] == "mlp" and layer.mlp is not None \
                and parts[2:] in (["up"], ["down"]):
            p = getattr(layer.mlp, parts[2]).weight
        elif parts[1] == "side" and layer.side is not None:
            p = {("gate",): layer.side.gate.weight,
                 ("proj",): layer.side.proj.weight,
                 ("norm",): layer.side_norm.weight}.get(tuple(parts[2:]))
        if p is None:
            return False
        _copy(p, w)
        return True
