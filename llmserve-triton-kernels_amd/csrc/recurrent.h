// What the recurrent mixers share: activations, a sum over 16 lanes, and the short causal convolution whose past is a ring
// in the request's state.
#pragma once

#include "common.h"

__device__ __forceinline__ float rc_silu(float x) { return x / (1.f + expf(-x)); }
__device__ __forceinline__ float rc_softplus(float x) { return x > 20.f ? x : log1pf(expf(x)); }
// exp(x) for the inside of a recurrence, a handful of instructions: 2^(x log2 e) by the hardware's exponential, with the
// rounding of the product x log2 e put back as a factor (1 + error ln 2); within two units in the last place for x <= 0
__device__ __forceinline__ float rc_exp(float x) {
    const float t = x * 1.44269504f;
    const float err = fmaf(x, 1.92596299e-8f, fmaf(x, 1.44269504f, -t));
    const float e = __builtin_amdgcn_exp2f(t);
    return fmaf(e, err * 0.693147181f, e);
}

// sum over the 16 lanes of a row of the wave, the same value in all of them (no LDS: four lane exchanges inside the row)
__device__ __forceinline__ float row16_sum(float v) {
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0xB1, 0xF, 0xF, true));   // quad_perm [1,0,3,2]
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x4E, 0xF, 0xF, true));   // quad_perm [2,3,0,1]
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x141, 0xF, 0xF, true));  // row_half_mirror
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x140, 0xF, 0xF, true));  // row_mirror
    return v;
}

// A short causal convolution per channel over the 32-bit products of a step's tokens.
struct ConvArgs {
    const float* u;  // [N, u_ld], columns u_col ..
    int u_ld, u_col;
    const float* taps_w;  // [channels, taps]
    const float* bias;    // [channels] or null
    int taps, channels;
    float* state;  // slots; the ring [taps - 1, channels] lies at ring_off inside a slot
    size_t slot_stride, ring_off;
    const int* state_slots;
    const int* token_seq;
    const int* positions;
    const int* cu_seqlens;
    const int* context_lens;
    int activation, update;
};

// channel c of token n after the convolution and the activation (the token belongs to a request that exists)
__device__ __forceinline__ float conv_channel(const ConvArgs& a, int n, int c) {
    const int b = a.token_seq[n];
    const int p = a.positions[n];
    const int first_row = a.cu_seqlens[b];
    const int first_pos = p - (n - first_row);
    float* ring = a.taps > 1 ? a.state + (size_t)a.state_slots[b] * a.slot_stride + a.ring_off : nullptr;
    float y = a.bias ? a.bias[c] : 0.f;
    for (int j = 0; j < a.taps; ++j) {
        const int pos = p - (a.taps - 1) + j;
        float v = 0.f;
        if (pos >= first_pos)
            v = a.u[(size_t)(first_row + pos - first_pos) * a.u_ld + a.u_col + c];
        else if (pos >= 0)
            v = ring[(size_t)(pos % (a.taps - 1)) * a.channels + c];
        y = fmaf(a.taps_w[(size_t)c * a.taps + j], v, y);
    }
    if (a.update && a.taps > 1)  // (every request brings one token: nobody else reads this ring, and this thread has read its place)
        ring[(size_t)(p % (a.taps - 1)) * a.channels + c] = a.u[(size_t)n * a.u_ld + a.u_col + c];
    return a.activation ? rc_silu(y) : y;
}

