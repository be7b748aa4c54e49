"""Common part of the builders whose config.json lists the layers one by one (their sizes need no alignment: matrices, vectors and
rows are padded with zeros).  A builder brings `config` with `tensor_shapes()`, `vocab` and `width`."""
from typing import Optional

import torch

from ..persistent_kernel import PersistentKernel, expert_tiles, gated_rows, operand_row
from ...kernel import bfloat16, float32, int64
from .graph_builder import GraphBuilder


def up_to(n: int, m: int) -> int:
    return -(-n // m) * m


class LayerListBuilder(GraphBuilder):
    owns_kv_cache = True
    dtypes = (torch.bfloat16, torch.float32)

    def __init__(self, mpk: PersistentKernel, weights: Optional[dict] = None):
        super().__init__(mpk, weights)
        self.tokenizer = self.returned_hidden_state = self.logits = None
        self._keep = {}

    def _begin(self, config, state_dict: dict, with_lm_head: bool):
        """Check the state dict's names; activation type and padded width."""
        self._shapes = config.tensor_shapes()
        missing = sorted(set(self._shapes) - set(state_dict))
        if missing:
            raise KeyError(f"the state dict lacks {missing}")
        self._state, self._acts, self.with_lm_head = state_dict, {}, with_lm_head
        self._E = float32 if self.dtype == torch.float32 else bfloat16
        self._W = up_to(config.width, 64)

    # ------------------------------------------------------------------ tensors
    def _attach(self, t: torch.Tensor, name: str):
        t = t.contiguous().view(-1).view(t.shape)  # (plain strides, also of a dimension of size one)
        self._keep[name] = t
        return self.mpk.attach_input(torch_tensor=t, name=name)

    def release_weights(self, names):
        return sum(self._keep.pop(n, None) is not None for n in names)

    def _w(self, name: str) -> torch.Tensor:
        w = self._state[name]
        if tuple(w.shape) != self._shapes[name]:
            raise ValueError(f"{name} has shape {tuple(w.shape)}, expected {self._shapes[name]}")
        return w

    def _matrix(self, name: str, rows: int = None, cols: int = None):
        return self._pad(self._w(name).to(self.dtype), rows, cols)

    @staticmethod
    def _pad(w: torch.Tensor, rows: int = None, cols: int = None):
        return torch.nn.functional.pad(w, (0, (cols or w.shape[-1]) - w.shape[-1], 0, (rows or w.shape[-2]) - w.shape[-2]))

    def _vector(self, name: str, size: int):
        """Attach a norm weight, a bias or an offset in fp32, zero-padded to `size`."""
        v = self._w(name).to(torch.float32)
        return self._attach(torch.nn.functional.pad(v, (0, size - len(v))), name)

    def _rows(self, name: str, cols: int, dt):
        """Activation rows of one iteration (library-owned, zero-filled), one tensor per name and size."""
        key = f"{name}_{cols}"
        if key not in self._acts:
            self._acts[key] = self.mpk.new_tensor(dims=(self.mpk.max_num_batched_tokens, cols), dtype=dt, name=key, io_category="cuda_tensor")
        return self._acts[key]

    def _new_state_slots(self):
        """int32, the state slot of every batch slot: the caller's tensor, or the identity."""
        slots = self.mpk.meta_tensors.get("state_slots_buffer")
        return torch.arange(self.mpk.max_num_batched_requests, dtype=torch.int32, device=self.mpk.device) if slots is None else slots

    # ------------------------------------------------------------------ pieces of a graph
    def _linear(self, inp, w: torch.Tensor, name: str, out):
        self.mpk.linear_layer(input=inp, weight=self._attach(w, name), output=out, grid_dim=(1, 1, 1), block_dim=(256, 1, 1))
        return out

    def _sections(self, parts):
        """parts: (name, matrix, rows it takes).  Returns the stacked matrix, zero-padded, and every part's first row."""
        col, at = {}, 0
        for n, _, size in parts:
            col[n], at = at, at + size
        w_in = torch.zeros(at, self._W, dtype=self.dtype, device=parts[0][1].device)
        for n, w, _ in parts:
            w_in[col[n]:col[n] + w.shape[0], :w.shape[1]] = w.to(self.dtype)
        return w_in, col, at

    def _expert_linears(self, p: str, h, ids, experts: int, top: int, ff: int, shared_ff: Optional[int], clamp: tuple = None):
        """Gated linears of the routed experts `e<j>` (and of a `shared` one) and their output linears.  Returns (output rows, one place
        after another, and the number of places)."""
        mpk, E, W, KW, shared = self.mpk, self._E, self._W, operand_row(self.dtype), shared_ff is not None

        def matrices(names, ff):
            F = up_to(ff, max(KW, 16))
            pick = lambda part, rows, cols: torch.stack([self._matrix(f"{p}{x}.{part}", rows, cols) for x in names])
            return F, expert_tiles(gated_rows(pick("gate", F, W), pick("up", F, W))), expert_tiles(pick("down", W, F))

        F, w13, w2 = matrices([f"e{j}" for j in range(experts)], ff)
        Fs, s13, s2 = matrices(["shared"], shared_ff) if shared else (0, None, None)
        attach = lambda t, name: None if t is None else self._attach(t, p + name)
        places, A = top + int(shared), max(F, Fs)
        act = self._rows(f"expert_act_{ff}_{shared_ff}_{top}", places * A, E)
        mpk.expert_linear_layer(h, attach(w13, "gate_up"), ids, act, experts, top, 2 * F, W, A, gated=True, shared_weight=attach(s13, "shared.gate_up"), shared_n=2 * Fs, shared_k=W, clamp=clamp)
        y = self._rows("expert_out", places * W, E)
        mpk.expert_linear_layer(act, attach(w2, "down"), ids, y, experts, top, W, F, W, in_stride=A, shared_weight=attach(s2, "shared.down"), shared_n=W, shared_k=Fs)
        return y, places

    def _token_ids(self, with_lm_head: bool):
        """(ids of an iteration's rows, speculation config, the rows' guesses)"""
        mpk, spec = self.mpk, self.mpk.spec_decode_config
        ids = self._attach(mpk.meta_tensors["input_tokens"], "input_token")
        if spec is None:
            return ids, None, None
        if not with_lm_head:
            raise ValueError("speculative decoding needs the LM head and the sampling stages in the graph (with_lm_head)")
        all_tokens = self._attach(mpk.meta_tensors["tokens"], "all_tokens")
        spec_tokens = mpk.draft_forward_layer_dispatcher(spec_decode_config=spec, tokens=all_tokens, grid_dim=(96, 1, 1), block_dim=(128, 1, 1))
        return spec_tokens, spec, spec_tokens

    def _head_and_sampling(self, h, head, vocab: int, spec=None, spec_tokens=None):
        """Logits of every row, the greedy token, and the check of guesses."""
        mpk = self.mpk
        self.logits = self._rows("logits", vocab, self._E)
        mpk.linear_layer(input=h, weight=head, output=self.logits, grid_dim=(1, 1, 1), block_dim=(256, 1, 1))
        out = self._attach(mpk.meta_tensors["output_tokens"], "output_token")
        part = (self._rows("argmax_value", mpk.num_workers, self._E), self._rows("argmax_index", mpk.num_workers, int64))
        mpk.argmax_partial_layer(input=self.logits, output=part, grid_dim=(mpk.num_workers, 1, 1), block_dim=(128, 1, 1))
        mpk.argmax_reduce_layer(input=part, output=out, grid_dim=(1, 1, 1), block_dim=(128, 1, 1))
        if spec_tokens is not None:
            self.verify_out = mpk.verify_layer_dispatcher(spec_decode_config=spec, spec_tokens=spec_tokens, target_output=out)

    def decode(self, ids: torch.Tensor):
        return self.tokenizer.decode(ids, skip_special_tokens=True)
