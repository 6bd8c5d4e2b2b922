// Arguments of the ragged-batch attention kernels (latent_attn.hip: every option; latent_attn_full.hip, latent_attn_win.hip: the lean MFMA kernel).
#pragma once
#include "common.h"

#define LAT_MQ 128  // query rows per workgroup of the MFMA kernels

struct LatAttnArgs {
    const float* Q;
    const void* K1;
    const void* K2;
    const void* V;
    void* O;
    int64_t ldq, ldk1, ldk2, ldv, ldo;
    int q_hs, k1_hs, v_hs, o_hs;
    int D1, D2, DV, H, hm, dt;
    const int *q_row0, *n_new, *past, *k1_row0, *k2_row0, *v_row0;
    float scale;
    int splits;  // MFMA path: a tile's keys are dealt to `splits` workgroups; partial (max, sum, output) rows go to ws and latent_attn_combine_kernel joins them
    float* ws;   // per (sequence, head tile, token tile, split): 128 maxima | 128 sums | 128 x DVP unnormalised outputs
    int kv_rep;  // query heads per key / value head (grouped queries): head h reads key / value head h / kv_rep
    int window;  // > 0: a query at position i sees key j <= i only if i - j < window or j < keep_first (sliding window that keeps the first tokens)
    int keep_first;
    int chunk;  // > 0: positions are cut into chunks of this many, counted from the sequence's first token; a query sees only the keys of its own chunk
    float softcap;      // > 0: score <- softcap * tanh(score / softcap) after the scale
    const float* sink;  // fp32 [H] or NULL: exp(sink[h]) joins the denominator of head h (no key, no value, not scaled)
    int pool;           // > 0: one pooled key / value row per `pool` tokens (needs window > 0, D2 == 0); rows PK / PV, first row of sequence s = pool_row0[s]
    const void *PK, *PV;
    int64_t ldp;
    const int* pool_row0;
    const float* sig_bias;  // fp32 [H] or NULL: weights sigmoid(score + sig_bias[head]) instead of a softmax
    int o_dt;               // dtype of the output rows (MI355_DT_*)
    const float* slope;     // fp32 [H] or NULL: slope[head] * (i - j) is taken off the (scaled, capped) score of query position i and key j
    const float* gate;      // fp32 rows [H x DV] or NULL: the output is multiplied element by element by sigmoid(gate)
    int64_t ldg;
};

// keys below this one are seen by no row of a tile whose first row stands at position pos0, kept first tokens aside (rows of a tile are consecutive positions)
__device__ __forceinline__ int tile_key_floor(int pos0, int window, int chunk) {
    const int w = window > 0 ? pos0 - window + 1 : 0, c = chunk > 0 ? pos0 / chunk * chunk : 0;
    return max(w, c);
}
// The 64-key steps a tile walks: those that hold kept first tokens below the tile's window, then everything from the window's lower edge to the last key.
struct KeySteps {
    int keep, key_lo, n;  // steps of kept tokens; first key of the others; all steps
    __device__ __forceinline__ int key(int v) const { return v < keep ? v * 64 : key_lo + (v - keep) * 64; }
};
__device__ __forceinline__ KeySteps key_steps(int pos0, int n_keys, int window, int keep_first, int chunk) {
    const int lo = max(tile_key_floor(pos0, window, chunk), 0) / 64;
    KeySteps k;
    k.keep = min((keep_first + 63) / 64, lo);
    k.key_lo = lo * 64;
    k.n = k.keep + (n_keys - k.key_lo + 63) / 64;
    return k;
}
__device__ __forceinline__ float gate_of(float g) { return 1.0f / (1.0f + expf(-g)); }

// Launches the kernel for attention over every key j <= i (no window, chunk, pooled rows or cap; scale > 0; rows 16-byte aligned, widths multiples of 8) if it
// holds these sizes; false: the caller takes the general kernel.  Partial results under key splits have the general kernel's layout.
bool latent_attn_full_launch(const LatAttnArgs& p, dim3 grid, hipStream_t st);
// The same under a window or chunk, with capped scores or a distance bias (no pooled rows, no sigmoid weights).
bool latent_attn_win_launch(const LatAttnArgs& p, dim3 grid, hipStream_t st);
