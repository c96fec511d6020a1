"""Sapatar: a layer-listed pre-norm decoder on parallel fp32 residual
streams (models/hyper_streams.py),

    u = sum_s a_s x_s;  y = f(rmsnorm(u));  x_t <- sum_s M[s, t] x_s + b_t y

whose mixers are matrix memories (models/state_mixers.py): retention (rotated
q / k, a constant decay per head), wkv (a decay per state row and token, a
bonus for the current token, inputs shifted towards the previous token's), or
windowed softmax attention over the paged pool and an mLSTM memory side by
side (models/parallel_mixer.py). The feed-forward is a routed bank of gated
experts with a gated shared one (models/experts.py) or absent. A layer may
run with the weights of another one, with pools of its own. Embedding rows
fill all streams; at the end the streams are summed, normed and go to the
head.

Attention keeps keys and values in the paged pools; memories, normalisers
and shifted rows sit in one state slot per live sequence
(engine/kv_cache.py). Both follow the ragged batch view, so prompt portions,
decode rows and mixed batches take the same path.
"""
from __future__ import annotations

import torch
import torch.nn.functional as F
from torch import nn

from ..engine.config import EngineConfig
from ..parallel import Communicator
from .experts import RoutedFF
from .hyper_streams import StreamPort, Streams
from .parallel_mixer import ParallelMixer
from .state_mixers import WkvMixer, build_scan_mixer


class SapatarLayer(nn.Module):
    def __init__(self, width, ls, streams, eps, dtype, comm):
        super().__init__()
        self.kind = ls.mixer_type
        if ls.mixer_type == "scan":
            self.mixer = build_scan_mixer(width, ls.mixer, eps, dtype, comm)
        elif ls.mixer_type == "parallel":
            self.mixer = ParallelMixer(width, ls.mixer, eps, dtype, comm)
        else:
            raise NotImplementedError(ls.mixer_type)
        self.shifted = isinstance(self.mixer, WkvMixer)
        self.port1 = StreamPort(width, streams, gate=False)
        self.mlp = self.port2 = None
        if ls.mlp is not None:
            self.mlp = RoutedFF(width, ls.mlp, dtype, comm, out_dtype=dtype)
            self.port2 = StreamPort(width, streams, gate=False)


class SapatarForCausalLM(nn.Module):
    uses_ragged_meta = True

    def __init__(self, cfg: EngineConfig, comm: Communicator, device):
        super().__init__()
        spec = cfg.spec
        if comm.pp_size > 1 or comm.tp_size > 1:
            raise NotImplementedError(
                "Sapatar serves on one GPU per replica (no TP/PP sharding yet)")
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
        own = {i: SapatarLayer(W, ls, spec.streams, spec.rms_norm_eps, dtype,
                               comm)
               for i, ls in enumerate(spec.layers) if ls.weights_of < 0}
        self.layers = nn.ModuleList(
            [own[ls.weights_of if ls.weights_of >= 0 else i]
             for i, ls in enumerate(spec.layers)])
        self.final_norm = mk(W, dt=torch.float32)
        self.register_buffer("ones", torch.ones(spec.streams),
                             persistent=False)
        self.lm_head = mk(spec.vocab_size, W)
        self.lm_head_pack = None
        self.offload = None
        self.to(device)

    def graph_capturable(self) -> bool:
        return all(layer.mlp is None or layer.mlp.graph_ok()
                   for layer in self.layers)

    def _mix(self, i, layer, st, meta, kv, tables):
        if layer.shifted:
            _, hs = st.open_shifted(layer.port1, layer.mixer.mu,
                                    kv.shift_states[i], meta.ragged)
            return layer.mixer(hs, meta, kv.ssm_states[i])
        h = st.open(layer.port1)
        if layer.kind == "scan":
            return layer.mixer(h, meta, kv.ssm_states[i], tables)
        return layer.mixer(h, meta, kv.k_caches[i], kv.v_caches[i],
                           kv.ssm_states[i], kv.extra_states[i])

    @torch.inference_mode()
    def forward(self, token_ids, meta, kv, return_hidden: bool = False,
                return_both: bool = False):
        spec = self.spec
        st = Streams(token_ids, self.embed, 1.0, spec.streams,
                     spec.rms_norm_eps, self.dtype)
        tables: dict = {}                   # this step's rotation tables
        for i, layer in enumerate(self.layers):
            st.close(layer.port1, self._mix(i, layer, st, meta, kv, tables))
            if layer.mlp is not None:
                st.close(layer.port2, layer.mlp(st.open(layer.port2), None))
        y = st.finish(None if return_hidden else meta.logits_indices,
                      self.ones, self.final_norm)
        if return_hidden:
            return y
        logits = F.linear(y, self.lm_head).float()
        if return_both:
            return logits, y
        return logits
