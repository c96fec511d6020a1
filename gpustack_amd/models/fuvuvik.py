"""Fuvuvik: a layer-listed pre-norm decoder on parallel fp32 residual
streams (models/hyper_streams.py) with gated sublayers,

    u = sum_s a_s x_s;  h = rmsnorm(u);  y = f(h) * sigmoid(W h + b)
    x_t <- sum_s M[s, t] x_s + b_t y

whose mixers read h shifted towards the previous token's. A layer's mixer is
softmax attention over the paged pool (models/paged_attention.py: either
convolved q, k, v with unit q / k heads behind a rotation, or rotated heads
that see their own chunk of positions and one more in the denominator; a
sigmoid gate per head on both) or the gated recurrence of
models/state_mixers.py MinGruMixer; its feed-forward is the gated dense block
of models/experts.py or absent. Scaled token embeddings fill all streams; at
the end the streams are summed, normed and go to the head.

Attention keeps keys and values in the paged pools; the recurrence, the
convolution's last inputs and every layer's previous normed row sit in one
state slot per live sequence (engine/kv_cache.py). Both follow the ragged
batch view, so prompt portions, decode rows and mixed batches take the same
path.
"""
from __future__ import annotations

import torch
import torch.nn.functional as F
from torch import nn

from ..engine.config import EngineConfig
from ..parallel import Communicator
from .experts import DenseFF
from .hyper_streams import StreamPort, Streams
from .paged_attention import PagedRotaryAttention
from .state_mixers import MinGruMixer


class FuvuvikLayer(nn.Module):
    def __init__(self, width, ls, streams, eps, dtype, comm):
        super().__init__()
        self.kind = ls.mixer_type
        if ls.mixer_type == "paged_attention":
            self.mixer = PagedRotaryAttention(width, ls.mixer, eps, dtype,
                                              comm)
        elif ls.mixer_type == "gru":
            self.mixer = MinGruMixer(width, ls.mixer, dtype, comm)
        else:
            raise NotImplementedError(ls.mixer_type)
        mk = lambda *shape, dt=dtype: nn.Parameter(
            torch.empty(*shape, dtype=dt), requires_grad=False)
        self.port1 = StreamPort(width, streams)
        self.shift = mk(width, dt=torch.float32)
        # the mixer's gate reads the unshifted row: a GEMM of its own; the
        # feed-forward's gate shares the up projection's
        self.gate1_w = mk(width, width)
        self.mlp = self.port2 = None
        if ls.mlp is not None:
            self.mlp = DenseFF(width, ls.mlp, dtype, comm, extra=width)
            self.port2 = StreamPort(width, streams)


class FuvuvikForCausalLM(nn.Module):
    uses_ragged_meta = True

    def __init__(self, cfg: EngineConfig, comm: Communicator, device):
        super().__init__()
        spec = cfg.spec
        if comm.pp_size > 1 or comm.tp_size > 1:
            raise NotImplementedError(
                "Fuvuvik serves on one GPU per replica (no TP/PP sharding yet)")
        self.spec, self.cfg, self.comm = spec, cfg, comm
        self.device = torch.device(device)
        dtype = getattr(torch, cfg.dtype)
        self.dtype = dtype
        self.layer_offset = 0
        self.num_local_layers = spec.num_layers
        W = spec.hidden_size
        mk = lambda *shape, dt=dtype: nn.Parameter(
            torch.empty(*shape, dtype=dt), requires_grad=False)
        self.embed = mk(spec.vocab_size, W)
        self.layers = nn.ModuleList(
            [FuvuvikLayer(W, ls, spec.streams, spec.rms_norm_eps, dtype, comm)
             for ls in spec.layers])
        self.final_norm = mk(W, dt=torch.float32)
        self.register_buffer("ones", torch.ones(spec.streams),
                             persistent=False)
        self.lm_head = mk(spec.vocab_size, W)
        self.lm_head_pack = None
        self.offload = None
        self.to(device)

    def graph_capturable(self) -> bool:
        return True

    def _mix(self, i, layer, h, meta, kv):
        if layer.kind == "gru":
            return layer.mixer(h, meta, kv.ssm_states[i])
        return layer.mixer(h, meta, kv.k_caches[i], kv.v_caches[i],
                           conv_state=kv.conv_states[i])

    @torch.inference_mode()
    def forward(self, token_ids, meta, kv, return_hidden: bool = False,
                return_both: bool = False):
        spec = self.spec
        st = Streams(token_ids, self.embed, spec.embed_scale, spec.streams,
                     spec.rms_norm_eps, self.dtype)
        for i, layer in enumerate(self.layers):
            h, hs = st.open_shifted(layer.port1, layer.shift,
                                    kv.shift_states[i], meta.ragged)
            gate = F.linear(h, layer.gate1_w)
            st.close(layer.port1, self._mix(i, layer, hs, meta, kv), gate)
            if layer.mlp is not None:
                st.close(layer.port2, *layer.mlp(st.open(layer.port2)))
        y = st.finish(None if return_hidden else meta.logits_indices,
                      self.ones, self.final_norm)
        if return_hidden:
            return y
        logits = F.linear(y, self.lm_head).float()
        if return_both:
            return logits, y
        return logits
