// Causal convolution and selective scan of a mixed batch (csrc/selective_scan.hip).
//
// Per channel c and state n, from what earlier steps left in the sequence's slot:
//   S <- exp(dt_c A[c, n]) S + dt_c x_c B_n,  y_c = sum_n S[c, n] C_n + D_c x_c
// and y * silu(z) goes on.  Prompt portions run in chunks: each chunk's own end
// state first, then the states are carried over the chunks, then every chunk
// runs from its true start.
#pragma once

#include <hip/hip_runtime.h>

#include <cstddef>
#include <cstdint>

#include "llm_decoder.h"

namespace llm {

// Up to scan_chunk() consecutive new tokens of one sequence.
struct ScanItem {
  int32_t tok0, n;      // batch rows
  int32_t seq0, seq_n;  // the sequence's rows in this batch
  int32_t slot;
  int32_t p0;           // position of the sequence's first new token (0: starts from zero)
  int32_t part;         // scan: carried state to start from (-1: the slot's)
                        // chunk pass: where the end state goes; the first chunk has `last` 1
  int32_t last;         // scan: the sequence's last chunk, its end state goes to the slot
};
// Parts part0 .. part0 + n - 1 of one sequence, part0 already true.
struct ScanCarry {
  int32_t part0, n;
};

struct ScanArgs {
  int inner = 0, state = 0;
  int ldc = 0;                // channels per row of A, state, history and parts (a multiple of 4)
  const void* x = nullptr;    // [M][ldx] after the convolution
  int ldx = 0;
  const float* dt = nullptr;  // [M][ldt]
  int ldt = 0;
  const void* z = nullptr;    // [M][ldz]
  int ldz = 0;
  const float* bc = nullptr;  // [M][ldb]: B at 0, C at c_at
  int ldb = 0, c_at = 0;
  const float* A = nullptr;   // [state][ldc], A log2(e)
  const float* D = nullptr;   // [ldc]
  void* out = nullptr;        // [M][ldo]
  int ldo = 0;
  float* slots = nullptr;     // [slots][state][ldc]
  // inputs of the convolution, to be kept for the next step (taps 0: not here)
  int taps = 0;
  const void* raw = nullptr;  // [M][ld_raw]
  int ld_raw = 0;
  void* history = nullptr;    // [slots][taps - 1][ldc]
  float* carry = nullptr;     // [parts][state][ldc]
  float* sum_dt = nullptr;    // [parts][ldc]
};
constexpr int kMaxScanState = 256;
// Tokens a chunk may hold.
int scan_chunk(int state);
hipError_t scan(int dtype, const ScanArgs& a, const ScanItem* items, int n, hipStream_t st);
// End states of chunks from zero (the first chunk of a sequence: from its slot).
hipError_t scan_chunks(int dtype, const ScanArgs& a, const ScanItem* items, int n, hipStream_t st);
hipError_t scan_carry(const ScanArgs& a, const ScanCarry* seqs, int n, hipStream_t st);

// x [m][c] = silu(bias + sum_k w[k][c] in[m - taps + 1 + k][c]); rows before the
// portion come from the slot's history, before the sequence from zero.
struct ConvArgs {
  int M = 0, channels = 0, taps = 0, ldc = 0;
  const int32_t* pos = nullptr;   // [M]
  const int32_t* slot = nullptr;  // [M]
  const int32_t* seq0 = nullptr;  // [M] first batch row of the row's sequence
  const void* in = nullptr;       // [M][ld_in]
  int ld_in = 0;
  const float* w = nullptr;       // [taps][ldc]
  const float* bias = nullptr;    // [ldc]
  const void* history = nullptr;  // [slots][taps - 1][ldc], oldest first
  void* x = nullptr;              // [M][ldx]
  int ldx = 0;
};
hipError_t causal_conv(int dtype, const ConvArgs& a, hipStream_t st);

}  // namespace llm
