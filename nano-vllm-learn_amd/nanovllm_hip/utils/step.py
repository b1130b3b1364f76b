"""What one engine step tells the model about its rows.  Rows of sequences that bring exactly one token come first (`num_decode` of them, row i =
sequence i), portions of prompts follow; block tables and state slots are indexed by sequence in that order."""
from dataclasses import dataclass

import torch


@dataclass
class StepMeta:
    num_decode: int
    slot_mapping: torch.Tensor                      # int32 [rows] cache slot of every row
    block_tables: torch.Tensor                      # int32 [sequences, width]
    state_slots: torch.Tensor                       # int32 [sequences]
    chunks: torch.Tensor                            # int32 [n, 4] recurrence segments, the decode rows' own first
    segment: int                                    # tokens of a full segment
    summaries: bool                                 # some portion has more than one segment
    max_context: int                                # host bound on the context of any row
    row_seq: torch.Tensor | None = None             # int32 [rows] sequence of every row (None: decode rows only)
    cu_rows: torch.Tensor | None = None             # int32 [sequences + 1] rows of every sequence (None: decode rows only)
    cu_q: torch.Tensor | None = None                # int32 [portions + 1] row offsets of the portions, from the first portion row
    cu_k: torch.Tensor | None = None                # int32 [portions + 1] offsets of the keys the portions see
    max_q: int = 0
    total_k: int = 0
