// What the kernels that walk a decaying matrix state share (decay_scan.hip, decay_chunks.hip).
#pragma once
#include <stddef.h>
#include <stdint.h>

#include "common.h"

struct DecayScan {
    const float* qk;
    const float* x;
    const float* dt;
    float* out;
    float* state;
    const float* dt_bias;
    const float* A;
    const float* skip;
    const int32_t* cu_seqlens;
    const int32_t* seq_slot;
    int64_t slot_floats;
    int qk_stride, q_off, k_off, a_off, x_stride, x_off, dt_stride, dt_off;
    int kind, heads, key_heads, key_dim, value_dim, act;
    float q_scale, k_scale;
    int R, kpt, n_waves, n_cb;
    int mode, chunk_len, chunks_per_seq;      // mode 0: whole sequences; 1: (N, P) of every chunk; 3: outputs from the chunks' start states
    float* ws;                                // [sequence][chunk][head][N | P | S_start][key_dim][value_dim]
};

// A prompt's tokens in chunks of 64 as products on the matrix cores, for decays per row (kind 1) and fixed
// ones (kind 3) without a skip; `ws` holds picolm_decay_chunks_ws_floats floats.
#define PICOLM_DECAY_CHUNKS_FROM 48       // new tokens of a sequence from which that pays
size_t picolm_decay_chunks_ws_floats(const DecayScan& a, int n_seq, int most_new);
int picolm_decay_chunks(DecayScan a, int n_seq, int most_new, hipStream_t stream);
