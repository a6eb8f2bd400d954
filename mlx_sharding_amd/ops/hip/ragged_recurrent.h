// Arguments of the causal convolutions and the selective scan.
#pragma once

#include "ragged_common.h"

#define RC_MAXTAPS 8

// Rows h [tokens, C] (row of token t at t - h_base), weights [taps, C],
// history [slots, taps - 1, C]; out [tokens, Cp], zeros past C.
struct ConvArgs {
  const void *h, *w, *bias;
  void *hist, *out;
  const int *cu, *pos0, *slots, *tok_entry, *chunks;
  long hstride;
  int C, Cp, taps, h_base, n_short, n_long, n_chunks;
  bool add, silu, vec;  // vec: rows and bases are whole vectors of 16 bytes
};

struct NormConvArgs {
  float* x;
  const void *y, *w_post, *g, *w;
  void *hist, *out;
  const int *cu, *pos0, *slots;
  long ystride;
  int W, Wp, taps, n_short;
  float eps;
};

// S [states padded, C] per slot; ends, inits and sums are scratch per span.
struct ScanArgs {
  const void *x, *z, *dt, *bc;
  const float *bias, *A, *D;
  float* state;
  void* out;
  const int *cu, *pos0, *slots, *spans, *span_cu;
  float *ends, *inits, *sums;
  long xs, zs, ds, bs;
  int C, Np, b0, c0, n_short, n_long, n_spans;
};
