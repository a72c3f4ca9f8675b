// A state-space recurrence with one decay per head and token, over a state of fixed size per request:
//     S_t = exp(A_h dt_t) S_(t-1) + dt_t B_t x_t^T,   y_t = S_t^T C_t + D_h x_t        (A_h = -exp(A_log_h) <= 0)
// x [heads, P], B and C [groups, N] (head h uses group h / (heads / groups)) are the channels [x | B | C] of a short causal
// convolution with SiLU over the step's 32-bit products, rounded once to the model's number format; dt is the softplus of a
// product plus a bias.  Step sizes, decays, logarithms, exponentials, the state and y are 32-bit.  A head's state lies
// column by column ([heads][P][N], the states of a column side by side), behind it the convolution's ring.
//
//   space_scan      token by token, everything from the products to y in one launch: a workgroup owns 16 columns of one
//                   head's state of one request, forms the convolution of its 16 x's and the group's B and C for a token,
//                   and 16 lanes share a column's states.  Any portion and any sizes; the decode kernel.
//   space_runs      portions of many tokens (bfloat16) in runs of SP_RUN tokens, four launches:
//       prepare     the convolution and the step sizes; x and B leave channel by channel with a run's tokens side by side
//                   (an operand whose inner dimension is time), B and C also token by token (inner dimension: states).
//       sums        per run and head: the logarithms of the decays added up, sum_t exp(L_end - L_t) dt_t x_t B_t^T, and per
//                   run and group the products B_s . C_t, which all heads of the group share.
//       scan        over a request's runs: the sums become the state before each run; the last state is stored.
//       out         y_t = exp(L_t) S^T C_t + sum_(s <= t) (B_s . C_t) exp(L_t - L_s) dt_s x_s + D x_t.
//                   Products are on the bfloat16 matrix instruction with 32-bit sums: x, B and C are bfloat16 numbers as
//                   they are, the 32-bit operand beside them (the state; the weights) goes in as three bfloat16 terms that
//                   add up to it (24 bits), so nothing is rounded that the recurrence keeps in 32-bit.
//   space_finish    y silu(z), each of `parts` equal parts of a row divided by its own root mean square (eps inside the
//                   root), times a weight, rounded once; and the ring takes the last taps - 1 input rows of every request
//                   (everything that reads the ring has run by then).
//
// L_t is the sum of the logarithms A dt over the run up to t: kept as two floats (from a 64-bit sum), so that a difference
// of two large sums is as exact as its exponential needs.
// A request of length 0 is padding: nothing of it is read or written.
#include "common.h"
#include "recurrent.h"

#define SP_THREADS 256
#define SP_RUN 128       // tokens of a run
#define SP_TILES 8       // tiles of 16 tokens in it
#define SP_SLAB 64       // columns of the state that a workgroup of `sums` and `out` takes
#define SP_OUT_THREADS 512
#define SP_TAPS_MAX 8    // taps that `prepare` takes
#define SP_SCORE_TILES (SP_TILES * (SP_TILES + 1) / 2)  // tiles (t, s) with s <= t

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) float f32x4;

struct SpaceArgs {
    const float* u;  // [N, u_ld] 32-bit products: [z | x | B | C | dt], the convolution's channels from column `col` on
    int u_ld, col, dt_col;
    const float* taps_w;  // [channels, taps]
    const float* bias;    // [channels]
    int taps, channels;
    const float* dt_bias;  // [heads]
    const float* a_log;    // [heads]
    const float* d_skip;   // [heads]
    int heads, groups, P, N;
    float* state;  // slots; [heads][P][N] at scan_off, the ring [taps - 1][channels] at ring_off
    size_t slot_stride, scan_off, ring_off;
    const int* state_slots;
    const int* cu_seqlens;
    const int* context_lens;
};

// SiLU behind the convolution: 32-bit, or, where its result is rounded to bfloat16 anyway, by the hardware's exponential and
// reciprocal (both within an ulp of 32-bit)
template <typename T>
__device__ __forceinline__ float sp_silu(float x) {
    if constexpr (sizeof(T) == 2) return x * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.44269504f * x));
    else return rc_silu(x);
}

// channel c of the convolution at row `row` (position pos) of a portion that starts at first_row (position first_pos)
template <typename T>
__device__ __forceinline__ float sp_conv(const SpaceArgs& a, const float* __restrict__ ring, int first_row, int first_pos, int pos, int c) {
    float y = a.bias[c];
    for (int j = 0; j < a.taps; ++j) {
        const int at = pos - (a.taps - 1) + j;
        float v = 0.f;
        if (at >= first_pos) v = a.u[(size_t)(first_row + at - first_pos) * a.u_ld + a.col + c];
        else if (at >= 0) v = ring[(size_t)(at % (a.taps - 1)) * a.channels + c];
        y = fmaf(a.taps_w[(size_t)c * a.taps + j], v, y);
    }
    return sp_silu<T>(y);
}

// ------------------------------------------------------------------------------------------- token by token
// grid (columns / 16, heads, requests).  Thread (column j of 16, lane of 16): states 4 lane .. of every 64 (VEC), or lane,
// lane + 16, ...  R numbers a lane.  Dynamic LDS: 2 x (16 + 2 N + 2) floats.
template <typename T, int R, bool VEC>
__global__ __launch_bounds__(SP_THREADS) void space_scan_kernel(float* __restrict__ y, int y_ld, const SpaceArgs a) {
    extern __shared__ float sp_rows[];
    const int b = blockIdx.z, h = blockIdx.y, p0 = blockIdx.x * 16;
    const int lane = threadIdx.x & 15, j = threadIdx.x >> 4;
    const int first_row = a.cu_seqlens[b], count = a.cu_seqlens[b + 1] - first_row, length = a.context_lens[b];
    if (count <= 0 || length <= 0) return;
    const int first_pos = length - count;
    const int g = h / (a.heads / a.groups), inner = a.heads * a.P, N = a.N;
    float* slot = a.state + (size_t)a.state_slots[b] * a.slot_stride;
    const float* ring = slot + a.ring_off;
    const bool live = p0 + j < a.P;
    float* column = slot + a.scan_off + ((size_t)h * a.P + (live ? p0 + j : a.P - 1)) * N;
    float s[R];
    if constexpr (VEC) {
#pragma unroll
        for (int r = 0; r < R; r += 4) {
            const int k = 4 * lane + 16 * r;
            const float4 v = (k < N && first_pos > 0) ? *reinterpret_cast<const float4*>(column + k) : make_float4(0.f, 0.f, 0.f, 0.f);
            s[r] = v.x, s[r + 1] = v.y, s[r + 2] = v.z, s[r + 3] = v.w;
        }
    } else {
#pragma unroll
        for (int r = 0; r < R; ++r) s[r] = (lane + 16 * r < N && first_pos > 0) ? column[lane + 16 * r] : 0.f;
    }
    const float rate = expf(a.a_log[h]), dt_bias = a.dt_bias[h], skip = a.d_skip[h];
    const int need = 16 + 2 * N, pitch = (need + 2 + 3) & ~3;
    for (int t = 0; t < count; ++t) {
        float* row = sp_rows + (t & 1) * pitch;  // [x of the 16 columns | B | C | dt, decay]
        for (int i = threadIdx.x; i < need; i += SP_THREADS) {
            const int c = i < 16 ? h * a.P + min(p0 + i, a.P - 1) : inner + (i - 16 < N ? g * N + i - 16 : (a.groups + g) * N + i - 16 - N);
            row[i] = round_to<T>(sp_conv<T>(a, ring, first_row, first_pos, first_pos + t, c));
        }
        if (threadIdx.x == SP_THREADS - 1) {
            const float dt = rc_softplus(a.u[(size_t)(first_row + t) * a.u_ld + a.dt_col + h] + dt_bias);
            row[need] = dt;
            row[need + 1] = expf(-rate * dt);
        }
        __syncthreads();
        const float x = row[j], dx = row[need] * x, decay = row[need + 1];
        float out = 0.f;
        if constexpr (VEC) {
#pragma unroll
            for (int r = 0; r < R; r += 4) {
                const int k = 4 * lane + 16 * r;
                if (k < N) {
                    const float4 bv = *reinterpret_cast<const float4*>(row + 16 + k), cv = *reinterpret_cast<const float4*>(row + 16 + N + k);
                    s[r] = fmaf(decay, s[r], dx * bv.x), s[r + 1] = fmaf(decay, s[r + 1], dx * bv.y);
                    s[r + 2] = fmaf(decay, s[r + 2], dx * bv.z), s[r + 3] = fmaf(decay, s[r + 3], dx * bv.w);
                    out = fmaf(s[r], cv.x, out), out = fmaf(s[r + 1], cv.y, out), out = fmaf(s[r + 2], cv.z, out), out = fmaf(s[r + 3], cv.w, out);
                }
            }
        } else {
#pragma unroll
            for (int r = 0; r < R; ++r) {
                const int k = lane + 16 * r;
                if (k < N) {
                    s[r] = fmaf(decay, s[r], dx * row[16 + k]);
                    out = fmaf(s[r], row[16 + N + k], out);
                }
            }
        }
        out = row16_sum(out);
        if (lane == 0 && live) y[(size_t)(first_row + t) * y_ld + h * a.P + p0 + j] = fmaf(skip, x, out);
    }
    if (!live) return;
    if constexpr (VEC) {
#pragma unroll
        for (int r = 0; r < R; r += 4) {
            const int k = 4 * lane + 16 * r;
            if (k < N) *reinterpret_cast<float4*>(column + k) = make_float4(s[r], s[r + 1], s[r + 2], s[r + 3]);
        }
    } else {
#pragma unroll
        for (int r = 0; r < R; ++r)
            if (lane + 16 * r < N) column[lane + 16 * r] = s[r];
    }
}

// ------------------------------------------------------------------------------------------- runs
// Run j of request b is at place cu_seqlens[b] / SP_RUN + b + j of the workspaces: the runs of different requests never
// meet, and tokens / SP_RUN + requests + 1 places hold them all.
struct RunSpace {
    bf16* xbt;      // [places][heads P + groups N][SP_RUN]: x and B, a run's tokens side by side, zeros behind the last
    bf16* bc;       // [tokens][2 groups N]: B and C
    float* dt;      // [places][heads][SP_RUN], zeros behind the last token
    float2* log;    // [places][heads][SP_RUN]: L_t as two floats
    float* total;   // [places][heads]: exp(L_end)
    float* scores;  // [places][groups][SP_SCORE_TILES][64][4]: B_s . C_t in the layout of the matrix instruction's result
    float* sums;    // [places][heads][P][N]: the runs' sums, then the states before the runs
};

__device__ __forceinline__ int sp_place(int row0, int b, int j) { return row0 / SP_RUN + b + j; }

// a and b as bfloat16 in the low and high half
__device__ __forceinline__ float sp_hi(uint32_t w) { return __uint_as_float(w & 0xffff0000u); }
__device__ __forceinline__ float sp_lo(uint32_t w) { return __uint_as_float(w << 16); }

// 8 floats as three vectors of bfloat16 that add up to them (the remainders are exact: each term takes the leading 8 bits)
struct Terms {
    bf16x8 t[3];
};
__device__ __forceinline__ Terms sp_split(const float (&v)[8]) {
    Terms r;
    uint32_t w[3][4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        float a = v[2 * i], b = v[2 * i + 1];
#pragma unroll
        for (int k = 0; k < 3; ++k) {
            w[k][i] = pack_bf16x2(a, b);
            a -= sp_lo(w[k][i]), b -= sp_hi(w[k][i]);
        }
    }
#pragma unroll
    for (int k = 0; k < 3; ++k) r.t[k] = __builtin_bit_cast(bf16x8, make_uint4(w[k][0], w[k][1], w[k][2], w[k][3]));
    return r;
}
__device__ __forceinline__ f32x4 sp_mfma(const bf16x8& a, const bf16x8& b, const f32x4& c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}

// grid (runs of the longest portion x 2, blocks of 64 channels and heads, requests).  Thread: a channel, 16 tokens of a half run.
template <int TAPS>
__global__ __launch_bounds__(SP_THREADS) void space_prepare_kernel(const SpaceArgs a, const RunSpace w) {
    const int b = blockIdx.z, j = blockIdx.x >> 1;
    const int first_row = a.cu_seqlens[b], count = a.cu_seqlens[b + 1] - first_row, length = a.context_lens[b];
    if (length <= 0 || j * SP_RUN >= count) return;
    const int in_run = (blockIdx.x & 1) * (SP_RUN / 2) + (threadIdx.x / LLMS_WAVE) * 16;  // this thread's first token in the run
    const int t0 = j * SP_RUN + in_run;                                                 // and in the portion
    const int first_pos = length - count, place = sp_place(first_row, b, j);
    const int c = blockIdx.y * LLMS_WAVE + threadIdx.x % LLMS_WAVE;
    const int inner = a.heads * a.P, gn = a.groups * a.N;
    if (c >= a.channels) {
        const int h = c - a.channels;
        if (h >= a.heads) return;
        const float bias = a.dt_bias[h];
        float4* at = reinterpret_cast<float4*>(w.dt + ((size_t)place * a.heads + h) * SP_RUN + in_run);
#pragma unroll
        for (int q = 0; q < 4; ++q) {
            float v[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int t = t0 + 4 * q + i;
                v[i] = t < count ? rc_softplus(a.u[(size_t)(first_row + t) * a.u_ld + a.dt_col + h] + bias) : 0.f;
            }
            at[q] = make_float4(v[0], v[1], v[2], v[3]);
        }
        return;
    }
    float tap[TAPS], in[16 + TAPS - 1];
    const int missing = TAPS - a.taps;  // (a weight of fewer taps: the oldest are zero)
#pragma unroll
    for (int i = 0; i < TAPS; ++i) tap[i] = i >= missing ? a.taps_w[(size_t)c * a.taps + i - missing] : 0.f;
    const float* ring = a.state + (size_t)a.state_slots[b] * a.slot_stride + a.ring_off;
    const float* col = a.u + (size_t)first_row * a.u_ld + a.col + c;
#pragma unroll
    for (int i = 0; i < 16 + TAPS - 1; ++i) {
        const int t = t0 - (TAPS - 1) + i;  // (in the portion; before it: the ring)
        float v = 0.f;
        if (t >= 0) {
            if (t < count) v = col[(size_t)t * a.u_ld];
        } else if (i >= missing && first_pos + t >= 0) {
            v = ring[(size_t)((first_pos + t) % (a.taps - 1)) * a.channels + c];
        }
        in[i] = v;
    }
    const float bias = a.bias[c];
    float out[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
        float s = bias;
#pragma unroll
        for (int k = 0; k < TAPS; ++k) s = fmaf(tap[k], in[i + k], s);
        out[i] = t0 + i < count ? sp_silu<bf16>(s) : 0.f;
    }
    uint32_t packed[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) packed[i] = pack_bf16x2(out[2 * i], out[2 * i + 1]);
    if (c < inner + gn) {
        uint4* at = reinterpret_cast<uint4*>(w.xbt + ((size_t)place * (inner + gn) + c) * SP_RUN + in_run);
        at[0] = make_uint4(packed[0], packed[1], packed[2], packed[3]);
        at[1] = make_uint4(packed[4], packed[5], packed[6], packed[7]);
    }
    if (c >= inner) {
        bf16* at = w.bc + (size_t)(first_row + t0) * (2 * gn) + (c - inner);
#pragma unroll
        for (int i = 0; i < 16; ++i)
            if (t0 + i < count) at[(size_t)i * (2 * gn)].bits = (uint16_t)(i & 1 ? packed[i / 2] >> 16 : packed[i / 2] & 0xffffu);
    }
}

// grid (runs of the longest portion, groups + heads x slabs, requests)
#define SP_STATE_STEPS 8  // steps of 32 states
__global__ __launch_bounds__(SP_THREADS) void space_sums_kernel(const SpaceArgs a, const RunSpace w, int slabs) {
    __shared__ float2 logs[SP_RUN];
    __shared__ float weight[SP_RUN];
    const int b = blockIdx.z, j = blockIdx.x, P = a.P, N = a.N;
    const int first_row = a.cu_seqlens[b], count = a.cu_seqlens[b + 1] - first_row;
    if (a.context_lens[b] <= 0 || j * SP_RUN >= count) return;
    const int n = min(SP_RUN, count - j * SP_RUN), place = sp_place(first_row, b, j);
    const int wave = threadIdx.x / LLMS_WAVE, lane = threadIdx.x % LLMS_WAVE, lo = lane % 16, hi = lane / 16;
    const int inner = a.heads * P, gn = a.groups * N;
    const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
    const bf16x8 none = __builtin_bit_cast(bf16x8, make_uint4(0, 0, 0, 0));
    if ((int)blockIdx.y < a.groups) {  // B_s . C_t of a group: wave i takes the token tiles i and 7 - i
        const int g = blockIdx.y;
        const bf16* rows = w.bc + (size_t)(first_row + j * SP_RUN) * (2 * gn) + g * N + 8 * hi;
        float* dst = w.scores + ((size_t)place * a.groups + g) * (SP_SCORE_TILES * 256);
        for (int half = 0; half < 2; ++half) {
            const int tt = half ? SP_TILES - 1 - wave : wave;
            if (16 * tt >= n) continue;
            const bf16* ct_at = rows + (size_t)min(16 * tt + lo, n - 1) * (2 * gn) + gn;  // (columns behind the last token are not read)
            bf16x8 ct[SP_STATE_STEPS];
#pragma unroll
            for (int k = 0; k < SP_STATE_STEPS; ++k) {
                if (32 * k >= N) break;
                ct[k] = 32 * k + 8 * hi < N ? *reinterpret_cast<const bf16x8*>(ct_at + 32 * k) : none;
            }
            for (int st = 0; st <= tt; ++st) {
                const bf16* bs_at = rows + (size_t)min(16 * st + lo, n - 1) * (2 * gn);
                bf16x8 bs[SP_STATE_STEPS];
#pragma unroll
                for (int k = 0; k < SP_STATE_STEPS; ++k) {
                    if (32 * k >= N) break;
                    bs[k] = 32 * k + 8 * hi < N ? *reinterpret_cast<const bf16x8*>(bs_at + 32 * k) : none;
                }
                f32x4 acc = zero;
#pragma unroll
                for (int k = 0; k < SP_STATE_STEPS; ++k) {
                    if (32 * k >= N) break;
                    acc = sp_mfma(bs[k], ct[k], acc);
                }
                *reinterpret_cast<f32x4*>(dst + ((size_t)(tt * (tt + 1) / 2 + st) * LLMS_WAVE + lane) * 4) = acc;
            }
        }
        return;
    }
    const int h = (blockIdx.y - a.groups) / slabs, c0 = ((blockIdx.y - a.groups) % slabs) * SP_SLAB;
    const size_t head_at = (size_t)place * a.heads + h;
    const int p = c0 + 16 * wave, g = h / (a.heads / a.groups);
    // the wave's columns of x are asked for before the weights are known
    const bf16* xt = w.xbt + ((size_t)place * (inner + gn) + h * P + min(p, P - 16) + lo) * SP_RUN + 8 * hi;
    uint4 xraw[SP_RUN / 32];
#pragma unroll
    for (int k = 0; k < SP_RUN / 32; ++k) xraw[k] = *reinterpret_cast<const uint4*>(xt + 32 * k);
    if (wave == 0) {  // L_t: two tokens a lane, summed in 64-bit
        const float2 dt = *reinterpret_cast<const float2*>(w.dt + head_at * SP_RUN + 2 * lane);
        const double rate = (double)expf(a.a_log[h]);
        const double first = -rate * (double)dt.x, both = first - rate * (double)dt.y;
        double before = both;
#pragma unroll
        for (int o = 1; o < LLMS_WAVE; o <<= 1) {
            const double other = __shfl_up(before, o, LLMS_WAVE);
            if (lane >= o) before += other;
        }
        const double end = __shfl(before, LLMS_WAVE - 1, LLMS_WAVE);
        const double l1 = before, l0 = before - both + first;  // (tokens behind the last add nothing)
        const float h0 = (float)l0, h1 = (float)l1;
        const float2 p0 = make_float2(h0, (float)(l0 - (double)h0)), p1 = make_float2(h1, (float)(l1 - (double)h1));
        logs[2 * lane] = p0, logs[2 * lane + 1] = p1;
        weight[2 * lane] = expf((float)(end - l0)) * dt.x;
        weight[2 * lane + 1] = expf((float)(end - l1)) * dt.y;
        if (c0 == 0) {
            float2* at = w.log + head_at * SP_RUN + 2 * lane;
            at[0] = p0, at[1] = p1;
            if (lane == 0) w.total[head_at] = expf((float)end);
        }
    }
    __syncthreads();
    if (p >= P) return;
    const bf16* bt = w.xbt + ((size_t)place * (inner + gn) + inner + g * N + lo) * SP_RUN + 8 * hi;
    float* dst = w.sums + (head_at * P + p + lo) * N + 4 * hi;
    for (int n0 = 0; n0 < N; n0 += 128) {
        f32x4 acc[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) acc[i] = zero;
#pragma unroll
        for (int k = 0; k < SP_RUN / 32; ++k) {
            if (32 * k >= n) break;
            bf16x8 bs[8];
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                if (n0 + 16 * i >= N) break;
                bs[i] = *reinterpret_cast<const bf16x8*>(bt + (size_t)(n0 + 16 * i) * SP_RUN + 32 * k);
            }
            const uint32_t xw[4] = {xraw[k].x, xraw[k].y, xraw[k].z, xraw[k].w};
            float v[8];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int t = 32 * k + 8 * hi + 2 * i;
                v[2 * i] = sp_lo(xw[i]) * weight[t], v[2 * i + 1] = sp_hi(xw[i]) * weight[t + 1];
            }
            const Terms x = sp_split(v);
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                if (n0 + 16 * i >= N) break;
#pragma unroll
                for (int k3 = 2; k3 >= 0; --k3) acc[i] = sp_mfma(bs[i], x.t[k3], acc[i]);
            }
        }
#pragma unroll
        for (int i = 0; i < 8; ++i)
            if (n0 + 16 * i < N) *reinterpret_cast<f32x4*>(dst + n0 + 16 * i) = acc[i];
    }
}

// grid (ceil(P N / 1024), heads, requests): four numbers a thread
__global__ __launch_bounds__(SP_THREADS) void space_run_scan_kernel(const SpaceArgs a, const RunSpace w) {
    const int b = blockIdx.z, h = blockIdx.y, e = 4 * (blockIdx.x * SP_THREADS + threadIdx.x), size = a.P * a.N;
    const int first_row = a.cu_seqlens[b], count = a.cu_seqlens[b + 1] - first_row, length = a.context_lens[b];
    if (length <= 0 || count <= 0 || e >= size) return;
    const int runs = (count + SP_RUN - 1) / SP_RUN, place = sp_place(first_row, b, 0);
    float4* st = reinterpret_cast<float4*>(a.state + (size_t)a.state_slots[b] * a.slot_stride + a.scan_off + (size_t)h * size + e);
    float4 s = length > count ? *st : make_float4(0.f, 0.f, 0.f, 0.f);  // (a portion from position 0 starts from zero)
    float* at = w.sums + ((size_t)place * a.heads + h) * size + e;
    const float* total = w.total + (size_t)place * a.heads + h;
    const size_t step = (size_t)a.heads * size;
    for (int j0 = 0; j0 < runs; j0 += 8) {  // 8 runs' sums are asked for together, then replaced one after the other
        float4 sums[8];
        float decay[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            const int j = min(j0 + u, runs - 1);
            sums[u] = *reinterpret_cast<const float4*>(at + (size_t)j * step);
            decay[u] = total[(size_t)j * a.heads];
        }
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            if (j0 + u < runs) {
                *reinterpret_cast<float4*>(at + (size_t)(j0 + u) * step) = s;
                s.x = fmaf(decay[u], s.x, sums[u].x), s.y = fmaf(decay[u], s.y, sums[u].y);
                s.z = fmaf(decay[u], s.z, sums[u].z), s.w = fmaf(decay[u], s.w, sums[u].w);
            }
        }
    }
    *st = s;
}

// grid (runs of the longest portion, heads x slabs, requests); 8 waves, wave i takes the run's tokens 16 i .. 16 i + 15.  Y^T =
// S^T C^T and X^T M^T: a lane keeps one token's column throughout.  PT: tiles of 16 columns of the slab.
template <int PT>
__global__ __launch_bounds__(SP_OUT_THREADS) void space_out_kernel(float* __restrict__ y, int y_ld, const SpaceArgs a, const RunSpace w, int slabs) {
    extern __shared__ char sp_lds[];
    constexpr int XP = SP_RUN + 8;  // a row of x^T in LDS, padded
    const int P = a.P, N = a.N, N32 = (N + 31) & ~31, SPITCH = N32 + 8;
    bf16* ss = reinterpret_cast<bf16*>(sp_lds);              // [3][16 PT][SPITCH]: the state before the run in three terms
    bf16* xs = ss + (size_t)3 * 16 * PT * SPITCH;            // [16 PT][XP]
    float2* logs = reinterpret_cast<float2*>(xs + 16 * PT * XP);  // [SP_RUN]
    float* dts = reinterpret_cast<float*>(logs + SP_RUN);    // [SP_RUN]
    const int b = blockIdx.z, j = blockIdx.x, h = blockIdx.y / slabs, c0 = (blockIdx.y % slabs) * SP_SLAB;
    const int first_row = a.cu_seqlens[b], count = a.cu_seqlens[b + 1] - first_row;
    if (a.context_lens[b] <= 0 || j * SP_RUN >= count) return;
    const int n = min(SP_RUN, count - j * SP_RUN), place = sp_place(first_row, b, j);
    const int inner = a.heads * P, gn = a.groups * N, g = h / (a.heads / a.groups);
    const size_t head_at = (size_t)place * a.heads + h;
    const int cols = min(16 * PT, P - c0);
    // the state's columns (32-bit, N a multiple of 16) as three terms
    const float* before = w.sums + (head_at * P + c0) * N;
    for (int e = threadIdx.x; e < 16 * PT * (N32 / 8); e += SP_OUT_THREADS) {
        const int p = e / (N32 / 8), k = 8 * (e % (N32 / 8));
        float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
        if (p < cols && k < N) {
            const float4 v0 = *reinterpret_cast<const float4*>(before + (size_t)p * N + k), v1 = *reinterpret_cast<const float4*>(before + (size_t)p * N + k + 4);
            v[0] = v0.x, v[1] = v0.y, v[2] = v0.z, v[3] = v0.w, v[4] = v1.x, v[5] = v1.y, v[6] = v1.z, v[7] = v1.w;
        }
        const Terms s = sp_split(v);
#pragma unroll
        for (int k3 = 0; k3 < 3; ++k3) *reinterpret_cast<bf16x8*>(ss + (size_t)(k3 * 16 * PT + p) * SPITCH + k) = s.t[k3];
    }
    const bf16* xt = w.xbt + ((size_t)place * (inner + gn) + h * P + c0) * SP_RUN;
    for (int e = threadIdx.x; e < 16 * PT * (SP_RUN / 8); e += SP_OUT_THREADS) {
        const int p = e / (SP_RUN / 8), t = 8 * (e % (SP_RUN / 8));
        *reinterpret_cast<uint4*>(xs + p * XP + t) = p < cols ? *reinterpret_cast<const uint4*>(xt + (size_t)p * SP_RUN + t) : make_uint4(0, 0, 0, 0);
    }
    if (threadIdx.x < SP_RUN) {
        logs[threadIdx.x] = w.log[head_at * SP_RUN + threadIdx.x];
        dts[threadIdx.x] = w.dt[head_at * SP_RUN + threadIdx.x];
    }
    __syncthreads();
    const int wave = threadIdx.x / LLMS_WAVE, lane = threadIdx.x % LLMS_WAVE, lo = lane % 16, hi = lane / 16;
    if (16 * wave >= n) return;
    const int t = 16 * wave + lo;
    const bf16x8 none = __builtin_bit_cast(bf16x8, make_uint4(0, 0, 0, 0));
    f32x4 acc[PT];
#pragma unroll
    for (int i = 0; i < PT; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    const bf16* crow = w.bc + (size_t)(first_row + j * SP_RUN + min(t, n - 1)) * (2 * gn) + gn + g * N;
    for (int k = 8 * hi; k - 8 * hi < N; k += 32) {
        const bf16x8 ct = k < N ? *reinterpret_cast<const bf16x8*>(crow + k) : none;
#pragma unroll
        for (int i = 0; i < PT; ++i)
#pragma unroll
            for (int k3 = 2; k3 >= 0; --k3)
                acc[i] = sp_mfma(*reinterpret_cast<const bf16x8*>(ss + (size_t)(k3 * 16 * PT + 16 * i + lo) * SPITCH + k), ct, acc[i]);
    }
    const float2 lt = logs[t];
    const float carried = expf(lt.x + lt.y);
#pragma unroll
    for (int i = 0; i < PT; ++i) acc[i] *= carried;
    const float* scores = w.scores + ((size_t)place * a.groups + g) * (SP_SCORE_TILES * 256) + (size_t)(wave * (wave + 1) / 2) * 256 + lane * 4;
    const float skip = a.d_skip[h];
    for (int s2 = 0; 2 * s2 <= wave; ++s2) {  // two tiles of keys: 32 of the inner dimension
        float m[8];
#pragma unroll
        for (int k = 0; k < 2; ++k) {
            const int st = 2 * s2 + k;
            f32x4 gv = {0.f, 0.f, 0.f, 0.f};
            if (st <= wave) gv = *reinterpret_cast<const f32x4*>(scores + (size_t)st * 256);
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int s = 16 * st + 4 * hi + i;
                float weight = 0.f;
                if (st <= wave) {
                    const float2 ls = logs[s];
                    weight = s < t ? gv[i] * rc_exp(fminf((lt.x - ls.x) + (lt.y - ls.y), 0.f)) * dts[s] : s == t ? fmaf(gv[i], dts[s], skip) : 0.f;
                }
                m[4 * k + i] = weight;
            }
        }
        const Terms mt = sp_split(m);
#pragma unroll
        for (int i = 0; i < PT; ++i) {
            const bf16* row = xs + (16 * i + lo) * XP + 32 * s2 + 4 * hi;
            const uint2 x0 = *reinterpret_cast<const uint2*>(row), x1 = *reinterpret_cast<const uint2*>(row + 16);
            const bf16x8 xv = __builtin_bit_cast(bf16x8, make_uint4(x0.x, x0.y, x1.x, x1.y));
#pragma unroll
            for (int k3 = 2; k3 >= 0; --k3) acc[i] = sp_mfma(xv, mt.t[k3], acc[i]);
        }
    }
    if (t >= n) return;
    float* dst = y + (size_t)(first_row + j * SP_RUN + t) * y_ld + h * P + c0 + 4 * hi;
#pragma unroll
    for (int i = 0; i < PT; ++i)
        if (16 * i < cols) *reinterpret_cast<f32x4*>(dst + 16 * i) = acc[i];
}

// ------------------------------------------------------------------------------------------- what leaves a token
// The first `rows` workgroups (ceil of the (token, part) items over the items of a workgroup) norm; the others bring the
// ring up to date, one workgroup per request and 256 channels.  LANES lanes a part; V pieces of 4 numbers a lane in
// registers, or V = 0: any size, two passes.
struct FinishArgs {
    const float* y;
    int y_ld;
    const float* z;
    int z_ld;
    const float* weight;
    int n_tokens, parts, width;  // numbers of a part
    float eps;
    int out_ld;
    int rows;
    // the ring
    const float* u;
    int u_ld, col, taps, channels;
    float* state;
    size_t slot_stride, ring_off;
    const int* state_slots;
    const int* cu_seqlens;
    const int* context_lens;
};

template <typename T, int LANES, int V>
__global__ __launch_bounds__(SP_THREADS) void space_finish_kernel(T* __restrict__ out, const FinishArgs a) {
    __shared__ float red[16];
    if ((int)blockIdx.x >= a.rows) {
        const int blocks = (a.channels + SP_THREADS - 1) / SP_THREADS;
        const int b = ((int)blockIdx.x - a.rows) / blocks, c = ((int)blockIdx.x - a.rows) % blocks * SP_THREADS + threadIdx.x;
        const int first_row = a.cu_seqlens[b], count = a.cu_seqlens[b + 1] - first_row, end = a.context_lens[b];
        if (c >= a.channels || count <= 0 || end <= 0) return;
        const int first_pos = end - count;
        float* ring = a.state + (size_t)a.state_slots[b] * a.slot_stride + a.ring_off;
        for (int pos = max(end - (a.taps - 1), first_pos); pos < end; ++pos)
            ring[(size_t)(pos % (a.taps - 1)) * a.channels + c] = a.u[(size_t)(first_row + pos - first_pos) * a.u_ld + a.col + c];
        return;
    }
    const int lane = threadIdx.x % LANES;
    const long long item = (long long)blockIdx.x * (SP_THREADS / LANES) + threadIdx.x / LANES;
    if (item >= (long long)a.n_tokens * a.parts) return;  // (whole waves; with LANES = 256 the whole workgroup)
    const int n = (int)(item / a.parts), part = (int)(item % a.parts), c0 = part * a.width;
    const float* yr = a.y + (size_t)n * a.y_ld + c0;
    const float* zr = a.z + (size_t)n * a.z_ld + c0;
    const float* wr = a.weight + c0;
    T* orow = out + (size_t)n * a.out_ld + c0;
    auto total = [&](float v) { return LANES == LLMS_WAVE ? wave_sum(v) : block_sum(v, red); };
    if constexpr (V > 0) {
        float4 yv[V], zv[V], wv[V];
#pragma unroll
        for (int v = 0; v < V; ++v) {
            const int c = 4 * (v * LANES + lane);
            const bool in = c < a.width;
            yv[v] = in ? *reinterpret_cast<const float4*>(yr + c) : make_float4(0.f, 0.f, 0.f, 0.f);
            zv[v] = in ? *reinterpret_cast<const float4*>(zr + c) : make_float4(0.f, 0.f, 0.f, 0.f);
            wv[v] = in ? *reinterpret_cast<const float4*>(wr + c) : make_float4(0.f, 0.f, 0.f, 0.f);
        }
        float ss = 0.f;
#pragma unroll
        for (int v = 0; v < V; ++v) {
            yv[v].x *= rc_silu(zv[v].x), yv[v].y *= rc_silu(zv[v].y), yv[v].z *= rc_silu(zv[v].z), yv[v].w *= rc_silu(zv[v].w);
            ss += (yv[v].x * yv[v].x + yv[v].y * yv[v].y) + (yv[v].z * yv[v].z + yv[v].w * yv[v].w);
        }
        const float mul = 1.f / sqrtf(total(ss) / (float)a.width + a.eps);
#pragma unroll
        for (int v = 0; v < V; ++v) {
            const int c = 4 * (v * LANES + lane);
            if (c >= a.width) continue;
            const float p = yv[v].x * mul * wv[v].x, q = yv[v].y * mul * wv[v].y, r = yv[v].z * mul * wv[v].z, s = yv[v].w * mul * wv[v].w;
            if constexpr (sizeof(T) == 2) *reinterpret_cast<uint2*>(orow + c) = make_uint2(pack_bf16x2(p, q), pack_bf16x2(r, s));
            else *reinterpret_cast<float4*>(orow + c) = make_float4(p, q, r, s);
        }
    } else {
        float ss = 0.f;
        for (int c = lane; c < a.width; c += LANES) {
            const float v = yr[c] * rc_silu(zr[c]);
            ss = fmaf(v, v, ss);
        }
        const float mul = 1.f / sqrtf(total(ss) / (float)a.width + a.eps);
        for (int c = lane; c < a.width; c += LANES) orow[c] = from_f32<T>(yr[c] * rc_silu(zr[c]) * mul * wr[c]);
    }
}

extern "C" {

static SpaceArgs space_args(const float* u, int u_ld, int col, int dt_col, const float* taps_w, const float* bias, int taps,
                            const float* dt_bias, const float* a_log, const float* d_skip, int heads, int groups, int P, int N,
                            float* state, size_t slot_stride, size_t scan_off, size_t ring_off, const int* state_slots,
                            const int* cu_seqlens, const int* context_lens) {
    SpaceArgs a;
    a.u = u, a.u_ld = u_ld, a.col = col, a.dt_col = dt_col, a.taps_w = taps_w, a.bias = bias, a.taps = taps;
    a.channels = heads * P + 2 * groups * N, a.dt_bias = dt_bias, a.a_log = a_log, a.d_skip = d_skip;
    a.heads = heads, a.groups = groups, a.P = P, a.N = N, a.state = state, a.slot_stride = slot_stride;
    a.scan_off = scan_off, a.ring_off = ring_off, a.state_slots = state_slots, a.cu_seqlens = cu_seqlens, a.context_lens = context_lens;
    return a;
}

int llms_space_scan(int dtype, float* y, int y_ld, const float* u, int u_ld, int col, int dt_col, const float* taps_w,
                    const float* bias, int taps, const float* dt_bias, const float* a_log, const float* d_skip, int heads,
                    int groups, int P, int N, float* state, size_t slot_stride, size_t scan_off, size_t ring_off,
                    const int* state_slots, const int* cu_seqlens, const int* context_lens, int n_seqs, hipStream_t stream) {
    LLMS_REQUIRE(n_seqs > 0 && heads > 0 && groups > 0 && P > 0 && N > 0 && taps > 0, "space_scan: sizes must be positive");
    LLMS_REQUIRE(heads % groups == 0, "space_scan: heads must be a multiple of groups");
    LLMS_REQUIRE(N <= 256, "space_scan: up to 256 states");
    LLMS_REQUIRE(heads <= 65535 && n_seqs <= 65535, "space_scan: up to 65,535 heads and requests");
    LLMS_REQUIRE(dtype == 0 || dtype == 1, "space_scan: dtype must be 0 (float32) or 1 (bfloat16)");
    const SpaceArgs a = space_args(u, u_ld, col, dt_col, taps_w, bias, taps, dt_bias, a_log, d_skip, heads, groups, P, N, state,
                                   slot_stride, scan_off, ring_off, state_slots, cu_seqlens, context_lens);
    const dim3 grid((P + 15) / 16, heads, n_seqs);
    const size_t lds = 2 * (size_t)((16 + 2 * N + 2 + 3) & ~3) * sizeof(float);
    const bool vec = N % 4 == 0 && ((uintptr_t)state % 16) == 0 && slot_stride % 4 == 0 && scan_off % 4 == 0;
#define SPACE_GO(R, VEC)                                                                                      \
    do {                                                                                                      \
        if (dtype == 0) space_scan_kernel<float, R, VEC><<<grid, SP_THREADS, lds, stream>>>(y, y_ld, a);      \
        else space_scan_kernel<bf16, R, VEC><<<grid, SP_THREADS, lds, stream>>>(y, y_ld, a);                  \
    } while (0)
    if (vec && N <= 64) SPACE_GO(4, true);
    else if (vec && N <= 128) SPACE_GO(8, true);
    else if (vec) SPACE_GO(16, true);
    else if (N <= 64) SPACE_GO(4, false);
    else if (N <= 128) SPACE_GO(8, false);
    else SPACE_GO(16, false);
#undef SPACE_GO
    LLMS_LAUNCH_CHECK();
}

// Whether llms_space_runs takes these sizes.
int llms_space_runs_fits(int heads, int groups, int P, int N, int taps) {
    return heads > 0 && groups > 0 && heads % groups == 0 && P % 16 == 0 && P > 0 && N % 16 == 0 && N > 0 && N <= 256 && taps >= 1 &&
           taps <= SP_TAPS_MAX;
}

static size_t space_round(size_t bytes) { return (bytes + 255) & ~(size_t)255; }

// The parts of the workspace for n_tokens rows of n_seqs requests; returns its bytes.
static size_t space_layout(RunSpace* w, char* base, int n_tokens, int n_seqs, int heads, int groups, int P, int N) {
    const size_t places = (size_t)n_tokens / SP_RUN + n_seqs + 1;
    size_t at = 0;
    auto take = [&](size_t bytes) {
        char* p = base + at;
        at += space_round(bytes);
        return p;
    };
    RunSpace r;
    r.xbt = (bf16*)take(places * (heads * P + groups * N) * SP_RUN * sizeof(bf16));
    r.bc = (bf16*)take((size_t)n_tokens * 2 * groups * N * sizeof(bf16));
    r.dt = (float*)take(places * heads * SP_RUN * sizeof(float));
    r.log = (float2*)take(places * heads * SP_RUN * sizeof(float2));
    r.total = (float*)take(places * heads * sizeof(float));
    r.scores = (float*)take(places * groups * SP_SCORE_TILES * 256 * sizeof(float));
    r.sums = (float*)take(places * heads * (size_t)P * N * sizeof(float));
    if (w) *w = r;
    return at;
}

size_t llms_space_runs_workspace(int n_tokens, int n_seqs, int heads, int groups, int P, int N) {
    return space_layout(nullptr, nullptr, n_tokens, n_seqs, heads, groups, P, N);
}

// The same recurrence as llms_space_scan for bfloat16 portions of many tokens (`max_new`: the most one request brings).
int llms_space_runs(float* y, int y_ld, const float* u, int u_ld, int col, int dt_col, const float* taps_w, const float* bias,
                    int taps, const float* dt_bias, const float* a_log, const float* d_skip, int heads, int groups, int P, int N,
                    float* state, size_t slot_stride, size_t scan_off, size_t ring_off, const int* state_slots,
                    const int* cu_seqlens, const int* context_lens, int n_seqs, int n_tokens, int max_new, void* workspace,
                    hipStream_t stream) {
    LLMS_REQUIRE(n_seqs > 0 && n_tokens > 0 && max_new > 0, "space_runs: sizes must be positive");
    LLMS_REQUIRE(llms_space_runs_fits(heads, groups, P, N, taps), "space_runs: columns and states in multiples of 16, up to 256 states, up to 8 taps");
    LLMS_REQUIRE(workspace && ((uintptr_t)workspace % 256) == 0, "space_runs: an aligned workspace");
    LLMS_REQUIRE(((uintptr_t)state % 16) == 0 && slot_stride % 4 == 0 && scan_off % 4 == 0 && ((uintptr_t)y % 16) == 0 && y_ld % 4 == 0,
                 "space_runs: state and result must be 16-byte aligned");
    const int slabs = (P + SP_SLAB - 1) / SP_SLAB, runs = (max_new + SP_RUN - 1) / SP_RUN;
    LLMS_REQUIRE((long long)heads * slabs + groups <= 65535 && n_seqs <= 65535, "space_runs: too many heads or requests");
    const SpaceArgs a = space_args(u, u_ld, col, dt_col, taps_w, bias, taps, dt_bias, a_log, d_skip, heads, groups, P, N, state,
                                   slot_stride, scan_off, ring_off, state_slots, cu_seqlens, context_lens);
    RunSpace w;
    space_layout(&w, (char*)workspace, n_tokens, n_seqs, heads, groups, P, N);
    const dim3 grid_p(2 * runs, (a.channels + heads + LLMS_WAVE - 1) / LLMS_WAVE, n_seqs);
    LLMS_REQUIRE(grid_p.y <= 65535, "space_runs: too many channels");
    if (taps <= 4) space_prepare_kernel<4><<<grid_p, SP_THREADS, 0, stream>>>(a, w);
    else space_prepare_kernel<SP_TAPS_MAX><<<grid_p, SP_THREADS, 0, stream>>>(a, w);
    space_sums_kernel<<<dim3(runs, groups + heads * slabs, n_seqs), SP_THREADS, 0, stream>>>(a, w, slabs);
    space_run_scan_kernel<<<dim3((P * N + 4 * SP_THREADS - 1) / (4 * SP_THREADS), heads, n_seqs), SP_THREADS, 0, stream>>>(a, w);
#define SPACE_OUT(PT)                                                                                                             \
    do {                                                                                                                          \
        const size_t lds = ((size_t)3 * 16 * PT * (((N + 31) & ~31) + 8) + (size_t)16 * PT * (SP_RUN + 8)) * sizeof(bf16) +       \
                           SP_RUN * (sizeof(float2) + sizeof(float));                                                             \
        if (lds > 48 * 1024)                                                                                                      \
            LLMS_HIP_CHECK(hipFuncSetAttribute((const void*)space_out_kernel<PT>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds)); \
        space_out_kernel<PT><<<dim3(runs, heads * slabs, n_seqs), SP_OUT_THREADS, lds, stream>>>(y, y_ld, a, w, slabs);           \
    } while (0)
    if (P <= 16) SPACE_OUT(1);
    else if (P <= 32) SPACE_OUT(2);
    else SPACE_OUT(4);
#undef SPACE_OUT
    LLMS_LAUNCH_CHECK();
}

int llms_space_finish(int dtype, void* out, int out_ld, const float* y, int y_ld, const float* z, int z_ld, const float* weight,
                      int n_tokens, int width, int parts, float eps, const float* u, int u_ld, int col, int taps, int channels,
                      float* state, size_t slot_stride, size_t ring_off, const int* state_slots, const int* cu_seqlens,
                      const int* context_lens, int n_seqs, hipStream_t stream) {
    LLMS_REQUIRE(n_tokens > 0 && n_seqs > 0 && width > 0 && parts > 0 && width % parts == 0, "space_finish: sizes must be positive, and the parts equal");
    LLMS_REQUIRE(dtype == 0 || dtype == 1, "space_finish: dtype must be 0 (float32) or 1 (bfloat16)");
    LLMS_REQUIRE(taps == 1 || (state && u), "space_finish: two taps or more keep a ring");
    FinishArgs a;
    a.y = y, a.y_ld = y_ld, a.z = z, a.z_ld = z_ld, a.weight = weight, a.n_tokens = n_tokens, a.parts = parts, a.width = width / parts;
    a.eps = eps, a.out_ld = out_ld, a.u = u, a.u_ld = u_ld, a.col = col, a.taps = taps, a.channels = channels, a.state = state;
    a.slot_stride = slot_stride, a.ring_off = ring_off, a.state_slots = state_slots, a.cu_seqlens = cu_seqlens, a.context_lens = context_lens;
    auto aligned = [](const void* p, int ld) { return ((uintptr_t)p % 16) == 0 && ld % 4 == 0; };
    const bool vec = a.width % 4 == 0 && aligned(y, y_ld) && aligned(z, z_ld) && aligned(weight, 0) && aligned(out, out_ld) && a.width <= 4096;
    const bool wave = a.width <= 1024;
    const long long items = (long long)n_tokens * parts;
    const long long rows = wave ? (items + 3) / 4 : items;
    const long long ring = taps > 1 ? (long long)n_seqs * ((channels + SP_THREADS - 1) / SP_THREADS) : 0;
    LLMS_REQUIRE(rows + ring < (1ll << 31), "space_finish: too many tokens for one launch");
    a.rows = (int)rows;
    const unsigned grid = (unsigned)(rows + ring);
#define FINISH_GO(LANES, V)                                                                              \
    do {                                                                                                 \
        if (dtype == 0) space_finish_kernel<float, LANES, V><<<grid, SP_THREADS, 0, stream>>>((float*)out, a); \
        else space_finish_kernel<bf16, LANES, V><<<grid, SP_THREADS, 0, stream>>>((bf16*)out, a);        \
    } while (0)
    if (vec && a.width <= 256) FINISH_GO(64, 1);
    else if (vec && a.width <= 512) FINISH_GO(64, 2);
    else if (vec && wave) FINISH_GO(64, 4);
    else if (vec && a.width <= 2048) FINISH_GO(256, 2);
    else if (vec) FINISH_GO(256, 4);
    else if (wave) FINISH_GO(64, 0);
    else FINISH_GO(256, 0);
#undef FINISH_GO
    LLMS_LAUNCH_CHECK();
}

}  // extern "C"
