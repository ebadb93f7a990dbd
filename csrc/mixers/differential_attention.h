// Arguments of the attention in two maps (csrc/mixers/differential_attention.hip), shared with the torch bindings.
#pragma once

namespace mxs {

struct DiffArgs {
  void* out;           // [n_rows, H*dv]
  const void* q;       // [n_rows, H, 2, dk], row-strided
  long q_stride;
  const void* cache;   // [blocks, block_stride]: K at koff as [G][bs][2 dk], V at voff as [G][bs][dv]
  long block_stride;
  const int* block_tables;
  int bt_stride;
  const int* qsl;      // [S + 1], absolute rows
  const int* seq_lens;
  int n_rows, koff, voff, H, G, dk, dv;
  int max_q;           // the longest chunk of the S sequences
  float scale, softcap, lam, out_scale, eps;
  const void* gate;    // [n_rows, H*dv], row-strided; may be null
  long gate_stride;
  int nsplit;          // workgroups that share a column tile's keys
  float* part;         // nsplit > 1: [n_rows, H, 2, nsplit, dv + 4]
};

}  // namespace mxs
