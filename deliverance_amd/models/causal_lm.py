"""The model every architecture becomes: embedding, a run order over blocks, final norm, head.

It is assembled from a ``ModelConfig`` and parameters under the parts' local names, and it
knows nothing of any particular architecture.  One forward call runs the tokens of one step:
embed -> each entry of the run order -> norm of the wanted rows -> logits of the wanted rows.
Reference: core/src/main/java/io/teknek/deliverance/model/AbstractModel.java:1097-1118 (layer
loop); the final norm and the head act on sampled rows only
(core/.../model/AbstractGeneratorSampler.java:112-115).
"""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ..config.specs import ModelConfig
from ..kernels import ops
from ..parts.norms import STREAM_ITSELF
from ..parts import Ahead, Block, StepContext, build_norm, build_position, to_matrix, to_vector
from ..registry import Architecture, ModelSupport, read_config_json
from ..weights.loader import load_declared


class CausalLM:
    def __init__(self, config: ModelConfig, params: dict, dtype: torch.dtype, device):
        self.config = config
        self.dtype = dtype
        self.device = torch.device(device)
        emb = params["embed"]
        # Tables are read by row in their stored dtype; in the 32-bit path they are widened.
        self.token_table = to_vector(emb["tokens"], dtype, device)
        if tuple(self.token_table.shape) != (config.vocab_size, config.width):
            raise ValueError(f"token table is {list(self.token_table.shape)}, expected "
                             f"{[config.vocab_size, config.width]}")
        self.embed_position = build_position(config.embed_position, emb.get("positions", {}), dtype, device)
        self.blocks: List[Block] = [Block(spec, p, dtype, device)
                                    for spec, p in zip(config.layers, params["layers"])]
        self.final_norm = None if config.final_norm is None else \
            build_norm(config.final_norm, params["final_norm"], dtype, device)
        embed_norm = getattr(config, "embed_norm", None)
        self.embed_norm = None if embed_norm is None else build_norm(embed_norm, params["embed_norm"], dtype, device)
        # W [width, 2 width] for run-order entries that mix the stream with the embedding output
        self.input_mix = None
        if getattr(config, "input_mix", False):
            self.input_mix = to_matrix(params["input_mix"]["weight"], dtype, device)
            if tuple(self.input_mix.shape) != (config.width, 2 * config.width):
                raise ValueError(f"the input mix is {list(self.input_mix.shape)}, expected {[config.width, 2 * config.width]}")
        elif any(getattr(c, "mix_input", False) for c in config.schedule):
            raise ValueError("the run order mixes the stream with the embedding output, but the model has no matrix for it")
        # vectors [n, width] of which run-order entries add one to the stream (32-bit)
        self.step_vectors, self.adds_input = None, any(c.add_input for c in config.schedule)
        n_steps = int(getattr(config, "step_vectors", 0))
        if n_steps:
            self.step_vectors = params["step_vectors"]["weight"].to(device=device, dtype=torch.float32).contiguous()
            if tuple(self.step_vectors.shape) != (n_steps, config.width):
                raise ValueError(f"the step vectors are {list(self.step_vectors.shape)}, expected {[n_steps, config.width]}")
        if any(c.add_step is not None and not (0 <= c.add_step < n_steps) for c in config.schedule):
            raise ValueError(f"the run order names a step vector that is not among the model's {n_steps}")
        head = params["head"]["weight"]
        if head is emb["tokens"] and self.token_table.dtype == dtype:
            self.head_weight = self.token_table            # tied: one buffer, two uses
        else:
            self.head_weight = to_matrix(head, dtype, device)
        for call in config.schedule:
            if not (0 <= call.layer < len(self.blocks)):
                raise ValueError(f"run order names layer {call.layer}, the model has {len(self.blocks)}")

    @property
    def graph_safe(self) -> bool:
        """Whether every part allows a decode step to be replayed from a recorded HIP graph."""
        return all(b.mixer.graph_safe and (b.feed_forward is None or b.feed_forward.graph_safe) for b in self.blocks)

    def kernel_units(self) -> List[str]:
        """The kernel units that the model's steps call: what a first call in a fresh checkout compiles, side by side."""
        names = ["rowwise", "dispatch"] + (["gemm_mfma", "gemm_wide", "gemm_fused"] if self.dtype == torch.bfloat16 else ["gemm_ref"])
        norms = [self.final_norm, self.embed_norm]
        for b in self.blocks:
            norms += [b.pre_mixer_norm, b.post_mixer_norm, b.pre_ff_norm, b.post_ff_norm, b.post_block_norm]
            names += list(b.mixer.kernel_units(self.dtype))
            if b.feed_forward is not None:
                names += list(b.feed_forward.kernel_units(self.dtype))
            if b.mixer_scale is not None or b.ff_scale is not None:
                names.append("elementwise")
        names += [u for n in norms if n is not None for u in n.kernel_units]
        if self.input_mix is not None or self.step_vectors is not None or self.adds_input or self.config.logit_softcap > 0.0:
            names.append("elementwise")
        return sorted(set(names))

    def _step_vector(self, call) -> Optional[torch.Tensor]:
        return None if call.add_step is None else self.step_vectors[call.add_step]

    # ---- what the cache must provide -----------------------------------------------------
    def cache_needs(self) -> Dict[int, object]:
        """cache slot -> KVNeed / StateNeed of the layer call that writes it."""
        def of(call):
            """(cache slot, need) of everything the call's mixer keeps: a mixer made of several mixers names a
            tuple, whose entry k lives in slot ``call.cache + k``."""
            need = self.blocks[call.layer].mixer.cache_need()
            many = need if isinstance(need, (tuple, list)) else (need,)
            return [(call.cache + k, n) for k, n in enumerate(many) if n is not None]

        needs: Dict[int, object] = {}
        for call in self.config.schedule:
            if call.write:
                for slot, need in of(call):
                    if slot in needs:
                        raise ValueError(f"cache slot {slot} is written by two layer calls")
                    needs[slot] = need
        for call in self.config.schedule:
            if not call.write:
                for slot, need in of(call):
                    if slot not in needs:
                        raise ValueError(f"layer {call.layer} reads cache slot {slot} that nothing writes")
                    if needs[slot] != need:
                        join = getattr(needs[slot], "joined", None)       # pages that two masks read
                        if join is None or type(need) is not type(needs[slot]):
                            raise ValueError(f"layer {call.layer} reads cache slot {slot} of another shape")
                        needs[slot] = join(need)
        return needs

    # ---- one step ----------------------------------------------------------------------------
    def forward(self, ctx: StepContext, want_rows: Optional[torch.Tensor], n_want: int) -> torch.Tensor:
        """Logits [n_want, V] (32-bit) of rows ``want_rows`` (int32, device) of this step."""
        with ops.pinned_stream():
            return self._forward(ctx, want_rows, n_want)

    def _forward(self, ctx: StepContext, want_rows: Optional[torch.Tensor], n_want: int) -> torch.Tensor:
        N = ctx.n_tokens
        x = ctx.buf("residual", N, self.config.width, torch.float32)
        ops.embed(ctx.tokens, ctx.positions, self.token_table, self.embed_position.embed_table(), x,
                  self.config.embed_scale)
        if self.embed_norm is not None:             # the stream starts as the norm of the embedded tokens, in 32-bit
            x = self.embed_norm.forward(ctx, x, out_name="residual_normed", out_dtype=torch.float32)
        debug = ctx.debug_hook is not None          # the reference's stages: AbstractModel.java:1100,1107
        if debug:
            ctx.emit(-1, "input", x)
        both = None
        if self.input_mix is not None:
            # [stream | embedding output] in the compute dtype; the right half is written once a step
            both = ctx.buf("input_mix", N, 2 * self.config.width, ctx.dtype)
            ops.concat_rows(x, both, self.config.width)
        first = None
        if self.adds_input:                             # the embedding output, as run-order entries add it again
            first = ops.copy_rows(x, ctx.buf("embedded", N, self.config.width, torch.float32))
        h = None                                        # a block's input that the block before has made
        for call, after in zip(self.config.schedule, (*self.config.schedule[1:], None)):
            if call.mix_input:                          # x <- W [x; embedding output]
                ops.concat_rows(x, both, 0)
                ops.linear(both, self.input_mix, None, x)
            if h is None and (call.add_input or call.add_step is not None):       # x <- x + embedding output + step vector
                ops.add_rows(x, first if call.add_input else None, self._step_vector(call))
            block, ahead = self.blocks[call.layer], None
            if after is not None and not after.mix_input and not debug:
                nxt = self.blocks[after.layer]
                if block.hands_ahead() and nxt.pre_mixer_norm is not None:
                    # the block's last kernel also does what is next: the additions, and the norm in front of the next block
                    ahead = Ahead(nxt.pre_mixer_norm, first if after.add_input else None, self._step_vector(after))
                elif nxt.takes_stream_ahead() and not after.add_input and after.add_step is None:
                    ahead = STREAM_ITSELF
            h = block.forward(ctx, x, call, h_ready=h, next_pre=ahead)
            if debug:
                ctx.emit(call.layer, "layer_output", x)
        logits = ctx.buf("logits", n_want, self.config.vocab_size, torch.float32)
        if n_want == 0:
            return logits
        ln = None if self.final_norm is None else self.final_norm.fusable_params()
        rms = None if self.final_norm is None or ln is not None else getattr(self.final_norm, "rms_params", lambda: None)()
        if ln is not None and ops.can_fuse_ln(n_want, x, self.head_weight):
            gain, bias, eps = ln                   # few wanted rows: norm and head in one kernel
            ops.linear_ln(x, want_rows, n_want, gain, bias, eps, self.head_weight, None, logits)
        elif rms is not None and ops.can_fuse_ln(n_want, x, self.head_weight):
            gain, offset, eps = rms
            ops.linear_rms(x, want_rows, n_want, gain, offset, eps, self.head_weight, None, logits)
        else:
            if self.final_norm is not None:
                e = self.final_norm.forward(ctx, x, rows=want_rows, n_rows=n_want, out_name="final_norm")
            else:
                e = ops.copy_rows(x, ctx.buf("final_norm", n_want, self.config.width, ctx.dtype), rows=want_rows)
            ops.linear(e, self.head_weight, None, logits)
        if self.config.logit_multiplier != 1.0:     # (an architecture's constant; GPT-2 has none)
            ops.copy_rows(logits, logits, scale=1.0 / self.config.logit_multiplier)
        if self.config.logit_softcap > 0.0:         # logits <- cap * tanh(logits / cap)
            ops.softcap(logits, self.config.logit_softcap)
        return logits


def load_model(folder: str, dtype: torch.dtype, device) -> CausalLM:
    """config.json picks the architecture; its tensors are read by name and bound to parts."""
    cfg_dict = read_config_json(folder)
    arch: Architecture = ModelSupport.detect(cfg_dict)
    mc = arch.read_config(cfg_dict)
    tensors = load_declared(folder, arch.declare_tensors(mc), ignore=arch.ignore_tensors,
                            strip_prefixes=arch.strip_prefixes)
    return CausalLM(mc, arch.bind_tensors(mc, tensors), dtype, device)
