// Attention over the paged cache whose ingredients are chosen by arguments, for float and bfloat16 storage:
//
//   conv_store    what the q, k, v projection of the new tokens gives (32-bit, [N, Cq + Ck + Cv]) goes through a short
//                 causal convolution per channel (from 2 taps on the request's last taps - 1 projected rows lie in its
//                 state, a ring indexed by position), is rounded once, and lands in the query rows and at the tokens'
//                 cache slots.  taps = 1: a factor per channel; taps = 0: rounding and store alone.
//   conv_state    the ring takes the last taps - 1 projected rows of every request of the step (a kernel of its own,
//                 because a token's write would race with its neighbours' reads; when every request brings one
//                 token, conv_store writes the ring itself).
//   norm_store    the same without a convolution, for queries and keys that are normed head by head: every head of q
//                 and of k is divided by its root mean square over its dk numbers (eps inside the root) and multiplied by a
//                 weight that all heads share (`unit_norm`: no weight); with `freq` the first rot_dims numbers of every
//                 head of q and k are turned by the token's position first (dimension i together with dimension
//                 i + rot_dims / 2, or `neighbours` 2i with 2i + 1, angle position * freq[i]), or with `norm_first` behind
//                 the norm; q is then multiplied by 1 + coef * ln(floor((p + 1) / every) + 1) at position p (every 0: no
//                 factor) and by a number per head (q_scale); all in 32-bit, rounded once, into the query rows and the
//                 cache slots.  `v_from_k`: the values are the keys as projected, before norm and rotation.  `joint`: the
//                 norm is over all heads of q at once, and over all of k, with a weight per number ([heads * dk]); a bias
//                 [columns] may be added to the projection first.
//   attend        one workgroup per new token, all heads.  Score heads s = h * maps + m (maps = 2: two score maps
//                 per query head over the same values); s reads key head (h / (H / G)) * maps + m, values come from
//                 value head h / (H / G).  A query at position i sees the key j <= i if
//                     j >= chunk_start(i)  and  (i - j < window  or  j < keep_first)
//                 (window 0: no window; chunk 0: no chunks).  score = q . k * scale - slope_h * (i - j) + dist_bias[h, min(i - j,
//                 dist_reach)] (a table per head over the distance, which stays at its last entry beyond dist_reach); softmax over the
//                 visible keys in 32-bit, normalised before anything else happens to it; with `sink` the denominator holds one more term exp(0); optionally the heads' weights
//                 are mixed, w_h = sum_g talk[h, g] w_g; then the values.  maps = 2 ends with o = a_1 - lambda a_2;
//                 head_norm divides a head's result by its root mean square (eps inside the root) and multiplies
//                 by out_scale.  With gate products z (32-bit) the result is multiplied by sigmoid(z[n, h * dv + d]), or with
//                 gate_heads by sigmoid(z[n, h]).
//
// Keys are [pages, key heads, block, dk], values [pages, value heads, dv, block] (transposed inside a page).
#include "common.h"

#define AC_THREADS 256
#define AC_WAVES (AC_THREADS / LLMS_WAVE)
#define AC_TILE LLMS_WAVE

// ------------------------------------------------------------------------------------------- conv + store
template <typename T>
__global__ __launch_bounds__(AC_THREADS) void conv_store_kernel(
    T* __restrict__ q_out, int q_stride, const float* __restrict__ proj, int proj_stride, const float* __restrict__ taps_w,
    int taps, const float* __restrict__ state, size_t state_slot_stride, const int* __restrict__ state_slots,
    const int* __restrict__ token_seq, const int* __restrict__ positions, const int* __restrict__ cu_seqlens,
    const int* __restrict__ slots, T* __restrict__ k_pool, T* __restrict__ v_pool, int cq, int ck, int cv, int k_heads,
    int dk, int v_heads, int dv, int block_size, float* __restrict__ state_out, const int* __restrict__ context_lens) {
    const int n = blockIdx.x;
    const int c = blockIdx.y * AC_THREADS + threadIdx.x;
    const int channels = cq + ck + cv;
    if (c >= channels) return;
    float y;
    if (taps >= 1) {
        const int b = token_seq[n];
        const int p = positions[n];
        const int first_row = cu_seqlens[b];
        const int first_pos = p - (n - first_row);  // position of the portion's first token
        const float* ring = taps > 1 ? state + (size_t)state_slots[b] * state_slot_stride : nullptr;
        y = 0.f;
        for (int j = 0; j < taps; ++j) {
            const int pos = p - (taps - 1) + j;
            float u = 0.f;
            if (pos >= first_pos)
                u = proj[(size_t)(first_row + pos - first_pos) * proj_stride + c];
            else if (pos >= 0)
                u = ring[(size_t)(pos % (taps - 1)) * channels + c];
            y = fmaf(taps_w[(size_t)c * taps + j], u, y);
        }
        // every request brings one token: the ring takes the token's own row here (nobody else reads this request's
        // ring in this launch, and this thread has read the place it overwrites); a request of length 0 is padding
        if (state_out && taps > 1 && context_lens[b] > 0)
            state_out[(size_t)state_slots[b] * state_slot_stride + (size_t)(p % (taps - 1)) * channels + c] =
                proj[(size_t)n * proj_stride + c];
    } else {
        y = proj[(size_t)n * proj_stride + c];
    }
    const T r = from_f32<T>(y);
    if (c < cq) {
        q_out[(size_t)n * q_stride + c] = r;
        return;
    }
    if (!slots) return;
    const int slot = slots[n];
    if (slot < 0) return;
    const int page = slot / block_size, off = slot % block_size;
    if (c < cq + ck) {
        const int kc = c - cq, head = kc / dk, d = kc % dk;
        k_pool[(((size_t)page * k_heads + head) * block_size + off) * dk + d] = r;
    } else {
        const int vc = c - cq - ck, head = vc / dv, d = vc % dv;
        v_pool[(((size_t)page * v_heads + head) * dv + d) * block_size + off] = r;
    }
}

__global__ __launch_bounds__(AC_THREADS) void conv_state_kernel(
    float* __restrict__ state, size_t state_slot_stride, const int* __restrict__ state_slots,
    const float* __restrict__ proj, int proj_stride, const int* __restrict__ cu_seqlens,
    const int* __restrict__ context_lens, int taps, int channels) {
    const int b = blockIdx.x;
    const int c = blockIdx.y * AC_THREADS + threadIdx.x;
    if (c >= channels) return;
    const int first_row = cu_seqlens[b], count = cu_seqlens[b + 1] - first_row;
    const int end = context_lens[b];  // the request's length after this step (0: not a request)
    if (count <= 0 || end <= 0) return;
    const int first_pos = end - count;
    float* ring = state + (size_t)state_slots[b] * state_slot_stride;
    int pos = end - (taps - 1);
    if (pos < first_pos) pos = first_pos;
    for (; pos < end; ++pos)
        ring[(size_t)(pos % (taps - 1)) * channels + c] = proj[(size_t)(first_row + pos - first_pos) * proj_stride + c];
}

// What norm_store is told.  Every head of q and k: turned by position and normed, in this order or the other.
struct HeadStoreArgs {
    int q_stride, proj_stride;
    const float* proj;
    const float* q_norm;  // [dk] weights, or null
    const float* k_norm;
    const float* q_scale;  // [q_heads]: the queries of a head are multiplied by a number of its own (null: 1)
    const float* freq;     // [rot_dims / 2]
    const float2* angles;  // [N, rot_dims / 2] (sine, cosine): given, it stands for freq
    const int* positions;
    const int* slots;
    float eps, temp_coef;
    int temp_every;
    int n_tokens, q_heads, k_heads, dk, v_heads, dv, block_size, rot_dims;
    int unit_norm;   // a norm without weights
    int neighbours;  // dimensions 2i and 2i + 1 turn together (else i and i + rot_dims / 2)
    int norm_first;  // the norm comes before the rotation
    int v_from_k;    // values are the keys as projected (v_heads = k_heads, dv = dk; proj holds no values)
    int joint;       // one norm over all heads of q, one over all heads of k; the weights hold heads * dk numbers
    const float* bias;  // of every column of proj, or null (with `joint` only)
};

__device__ __forceinline__ float2 head_angle(const HeadStoreArgs& a, int n, float position, int i) {  // (sine, cosine)
    return a.angles ? a.angles[(size_t)n * (a.rot_dims / 2) + i] : rotary_angle(position, a.freq[i]);
}

// number d of a head whose numbers are value(0) .. value(dk - 1), after the rotation
template <class Value>
__device__ __forceinline__ float turned_element(const HeadStoreArgs& a, Value value, int d, int n, float position) {
    if (d >= a.rot_dims) return value(d);
    const int h = a.rot_dims >> 1;
    const int i = a.neighbours ? d >> 1 : (d < h ? d : d - h);
    const int first = a.neighbours ? 2 * i : i, second = a.neighbours ? 2 * i + 1 : i + h;
    const float2 sc = head_angle(a, n, position, i);
    const float2 turned = rotate_pair(value(first), value(second), sc.y, sc.x);
    return d == first ? turned.x : turned.y;
}

__device__ __forceinline__ float query_factor(const HeadStoreArgs& a, int n, int head) {
    float factor = a.q_scale ? a.q_scale[head] : 1.f;
    if (a.temp_every > 0) factor *= 1.f + a.temp_coef * logf((float)((a.positions[n] + 1) / a.temp_every + 1));
    return factor;
}

// Any sizes.  grid: (tokens, query heads + key heads + value heads); one wave per head
template <typename T>
__global__ __launch_bounds__(LLMS_WAVE) void norm_store_kernel(T* __restrict__ q_out, T* __restrict__ k_pool,
                                                               T* __restrict__ v_pool, HeadStoreArgs a) {
    const int n = blockIdx.x, lane = threadIdx.x, dk = a.dk, dv = a.dv;
    int head = blockIdx.y;
    const float* row = a.proj + (size_t)n * a.proj_stride;
    if (head < a.q_heads + a.k_heads) {
        const bool is_q = head < a.q_heads;
        const float* src = row + (size_t)head * dk;  // (keys follow the queries)
        const float* w = is_q ? a.q_norm : a.k_norm;
        const bool normed = w || a.unit_norm;
        const float position = a.rot_dims > 0 ? (float)a.positions[n] : 0.f;
        auto raw = [&](int d) { return src[d]; };
        float mul = 1.f;
        if (normed) {
            float ss = 0.f;
            for (int d = lane; d < dk; d += LLMS_WAVE) {
                const float x = a.norm_first ? src[d] : turned_element(a, raw, d, n, position);
                ss = fmaf(x, x, ss);
            }
            mul = 1.f / sqrtf(wave_sum(ss) / (float)dk + a.eps);
        }
        auto scaled = [&](float x, int d) { return w ? x * mul * w[d] : x * mul; };
        auto normed_value = [&](int d) { return scaled(src[d], d); };
        const float factor = is_q ? query_factor(a, n, head) : 1.f;
        T* dst;
        if (is_q) {
            dst = q_out + (size_t)n * a.q_stride + (size_t)head * dk;
        } else {
            if (!a.slots) return;
            const int slot = a.slots[n];
            if (slot < 0) return;
            const int page = slot / a.block_size, off = slot % a.block_size;
            dst = k_pool + (((size_t)page * a.k_heads + (head - a.q_heads)) * a.block_size + off) * dk;
        }
        for (int d = lane; d < dk; d += LLMS_WAVE) {
            const float x = a.norm_first ? turned_element(a, normed_value, d, n, position)
                                         : scaled(turned_element(a, raw, d, n, position), d);
            dst[d] = from_f32<T>(x * factor);
        }
        return;
    }
    head -= a.q_heads + a.k_heads;
    if (!a.slots) return;
    const int slot = a.slots[n];
    if (slot < 0) return;
    const int page = slot / a.block_size, off = slot % a.block_size;
    const float* src = a.v_from_k ? row + (size_t)(a.q_heads + head) * dk
                                  : row + (size_t)(a.q_heads + a.k_heads) * dk + (size_t)head * dv;
    for (int d = lane; d < dv; d += LLMS_WAVE)
        v_pool[(((size_t)page * a.v_heads + head) * dv + d) * a.block_size + off] = from_f32<T>(src[d]);
}

// Heads of up to 256 numbers, 4 to a lane: `lph` lanes (a power of two, at least dk / 4) hold a head of one token, so a
// head's sum of squares is a few lane exchanges and a pair of the rotation lies in a lane (neighbours) or two.
// The first `kv_blocks` workgroups take 16 tokens of one key or value head each: a page holds values transposed, so
// they pass through LDS and leave with the tokens side by side in the lanes, which the memory system joins to whole
// pieces where the tokens' slots follow one another.  The other workgroups take U heads of queries per group of lanes.
#define HS_THREADS 256
#define HS_TOKENS 16
#define HS_MAX_DIM 256

template <typename T>
__device__ __forceinline__ void store4(T* dst, const float (&x)[4]) {
    if constexpr (sizeof(T) == 2)
        *reinterpret_cast<uint2*>(dst) = make_uint2(pack_bf16x2(x[0], x[1]), pack_bf16x2(x[2], x[3]));
    else
        *reinterpret_cast<float4*>(dst) = make_float4(x[0], x[1], x[2], x[3]);
}

// x: the lane's 4 numbers (4 li ..) of a head of token n
__device__ __forceinline__ void turn4(const HeadStoreArgs& a, float (&x)[4], int li, int n, bool live) {
    const int half = a.rot_dims >> 1;
    const float2* row = a.angles + (size_t)n * half;
    if (a.neighbours) {
#pragma unroll
        for (int p = 0; p < 2; ++p) {
            const int i = 2 * li + p;
            if (live && i < half) {
                const float2 sc = row[i];
                const float2 t = rotate_pair(x[2 * p], x[2 * p + 1], sc.y, sc.x);
                x[2 * p] = t.x, x[2 * p + 1] = t.y;
            }
        }
        return;
    }
    const int hl = half >> 2;  // lanes that hold the first partners (half is a multiple of 4 here)
    const bool turns = li < 2 * hl, low = li < hl;
    const int lane = threadIdx.x % LLMS_WAVE, partner = turns ? (low ? lane + hl : lane - hl) : lane;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        const float other = __shfl(x[e], partner, LLMS_WAVE);
        if (live && turns) {
            const float2 sc = row[4 * (low ? li : li - hl) + e];
            const float2 t = low ? rotate_pair(x[e], other, sc.y, sc.x) : rotate_pair(other, x[e], sc.y, sc.x);
            x[e] = low ? t.x : t.y;
        }
    }
}

__device__ __forceinline__ void prepare4(const HeadStoreArgs& a, float (&x)[4], const float* __restrict__ w, int li, int lph,
                                         int n, bool live) {
    if (a.rot_dims > 0 && !a.norm_first) turn4(a, x, li, n, live);
    if (w || a.unit_norm) {
        float ss = 0.f;
#pragma unroll
        for (int e = 0; e < 4; ++e) ss = fmaf(x[e], x[e], ss);
        for (int o = lph >> 1; o > 0; o >>= 1) ss += __shfl_xor(ss, o, LLMS_WAVE);
        const float mul = 1.f / sqrtf(ss / (float)a.dk + a.eps);
        float4 wv = make_float4(1.f, 1.f, 1.f, 1.f);
        if (w && 4 * li < a.dk) wv = *reinterpret_cast<const float4*>(w + 4 * li);
        x[0] = x[0] * mul * wv.x, x[1] = x[1] * mul * wv.y, x[2] = x[2] * mul * wv.z, x[3] = x[3] * mul * wv.w;
    }
    if (a.rot_dims > 0 && a.norm_first) turn4(a, x, li, n, live);
}

template <typename T, int U>
__global__ __launch_bounds__(HS_THREADS) void head_store_kernel(T* __restrict__ q_out, T* __restrict__ k_pool,
                                                                T* __restrict__ v_pool, HeadStoreArgs a, int lph, int kv_blocks) {
    __shared__ float tile[HS_TOKENS * (HS_MAX_DIM + 1)];
    __shared__ long long place[HS_TOKENS];  // of number 0 of the token's value (-1: none)
    const int tid = threadIdx.x, li = tid & (lph - 1), group = tid / lph, groups = HS_THREADS / lph;
    const int dk = a.dk, dv = a.dv;
    const bool in_head = 4 * li < dk;
    if ((int)blockIdx.x >= kv_blocks) {
        const int first = ((int)blockIdx.x - kv_blocks) * groups * U + group, total = a.n_tokens * a.q_heads;
        float x[U][4];
        int tok[U], head[U];
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int item = min(first + u * groups, total - 1);
            tok[u] = item / a.q_heads, head[u] = item - tok[u] * a.q_heads;
            float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
            if (in_head) v = *reinterpret_cast<const float4*>(a.proj + (size_t)tok[u] * a.proj_stride + (size_t)head[u] * dk + 4 * li);
            x[u][0] = v.x, x[u][1] = v.y, x[u][2] = v.z, x[u][3] = v.w;
        }
#pragma unroll
        for (int u = 0; u < U; ++u) {
            prepare4(a, x[u], a.q_norm, li, lph, tok[u], in_head);
            const float factor = query_factor(a, tok[u], head[u]);
#pragma unroll
            for (int e = 0; e < 4; ++e) x[u][e] *= factor;
            if (in_head && first + u * groups < total)
                store4<T>(q_out + (size_t)tok[u] * a.q_stride + (size_t)head[u] * dk + 4 * li, x[u]);
        }
        return;
    }
    const int roles = a.k_heads + (a.v_from_k ? 0 : a.v_heads);
    const int n0 = ((int)blockIdx.x / roles) * HS_TOKENS, role = (int)blockIdx.x % roles;
    const bool is_k = role < a.k_heads;
    const int v_head = is_k ? role : role - a.k_heads;
    if (tid < HS_TOKENS) {
        const int slot = n0 + tid < a.n_tokens ? a.slots[n0 + tid] : -1;
        const int page = slot / a.block_size, off = slot - page * a.block_size;
        place[tid] = slot < 0 ? -1 : ((long long)page * a.v_heads + v_head) * dv * a.block_size + off;
    }
    const int pitch = dv + 1;
    if (is_k) {
        for (int t0 = 0; t0 < HS_TOKENS; t0 += groups) {
            const int t = t0 + group, n = min(n0 + t, a.n_tokens - 1);
            const bool live = t < HS_TOKENS && n0 + t < a.n_tokens;
            const int slot = live ? a.slots[n] : -1;
            float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
            if (in_head) v = *reinterpret_cast<const float4*>(a.proj + (size_t)n * a.proj_stride + (size_t)(a.q_heads + role) * dk + 4 * li);
            float x[4] = {v.x, v.y, v.z, v.w};
            if (a.v_from_k && live && in_head) {
#pragma unroll
                for (int e = 0; e < 4; ++e) tile[t * pitch + 4 * li + e] = x[e];
            }
            prepare4(a, x, a.k_norm, li, lph, n, in_head);
            if (in_head && slot >= 0) {
                const int page = slot / a.block_size, off = slot - page * a.block_size;
                store4<T>(k_pool + (((size_t)page * a.k_heads + role) * a.block_size + off) * dk + 4 * li, x);
            }
        }
        if (!a.v_from_k) return;
    } else {
        const float* src = a.proj + (size_t)(a.q_heads + a.k_heads) * dk + (size_t)v_head * dv;
        for (int i = tid; i < HS_TOKENS * dv; i += HS_THREADS) {
            const int t = i / dv, d = i - t * dv;
            if (n0 + t < a.n_tokens) tile[t * pitch + d] = src[(size_t)(n0 + t) * a.proj_stride + d];
        }
    }
    __syncthreads();
    for (int i = tid; i < HS_TOKENS * dv; i += HS_THREADS) {
        const int t = i % HS_TOKENS, d = i / HS_TOKENS;
        const long long at = place[t];
        if (at >= 0) v_pool[at + (long long)d * a.block_size] = from_f32<T>(tile[t * pitch + d]);
    }
}

// ---- one norm over all heads (`joint`; the norm comes before the rotation)
__device__ __forceinline__ bool head_slot(const HeadStoreArgs& a, int n, int& page, int& off) {
    const int slot = a.slots ? a.slots[n] : -1;
    page = slot / a.block_size, off = slot - page * a.block_size;
    return slot >= 0;
}

// values of 16 tokens of one value head, through LDS into a page's transposed rows; 8 tokens that lie side by side in a page
// leave as one 16-byte piece of a dimension (bfloat16)
template <typename T>
__device__ __forceinline__ void store_values(T* __restrict__ v_pool, const HeadStoreArgs& a, int n0, int head, float* tile,
                                             long long* place, int* side_by_side) {
    const int tid = threadIdx.x, dv = a.dv, pitch = dv + 1;
    if (tid < HS_TOKENS) {
        int page, off;
        const bool in = n0 + tid < a.n_tokens && head_slot(a, n0 + tid, page, off);
        place[tid] = in ? ((long long)page * a.v_heads + head) * dv * a.block_size + off : -1;
    }
    const int col = a.v_from_k ? (a.q_heads + head) * a.dk : (a.q_heads + a.k_heads) * a.dk + head * dv;
    if (dv % 4 == 0) {  // (the rows of proj and its columns are at multiples of 16 bytes here)
        for (int i = tid; i < HS_TOKENS * (dv / 4); i += HS_THREADS) {
            const int t = i / (dv / 4), d = 4 * (i - t * (dv / 4));
            if (n0 + t >= a.n_tokens) continue;
            float4 v = *reinterpret_cast<const float4*>(a.proj + (size_t)(n0 + t) * a.proj_stride + col + d);
            if (a.bias) {
                const float4 b = *reinterpret_cast<const float4*>(a.bias + col + d);
                v.x += b.x, v.y += b.y, v.z += b.z, v.w += b.w;
            }
            float* at = tile + t * pitch + d;
            at[0] = v.x, at[1] = v.y, at[2] = v.z, at[3] = v.w;
        }
    } else {
        for (int i = tid; i < HS_TOKENS * dv; i += HS_THREADS) {
            const int t = i / dv, d = i - t * dv;
            if (n0 + t < a.n_tokens)
                tile[t * pitch + d] = a.proj[(size_t)(n0 + t) * a.proj_stride + col + d] + (a.bias ? a.bias[col + d] : 0.f);
        }
    }
    __syncthreads();
    if constexpr (sizeof(T) == 2) {
        if (tid < 2) {
            bool joined = place[8 * tid] >= 0 && place[8 * tid] % 8 == 0 && a.block_size % 8 == 0 && ((uintptr_t)v_pool % 16) == 0;
            for (int t = 1; t < 8; ++t) joined = joined && place[8 * tid + t] == place[8 * tid] + t;
            side_by_side[tid] = joined;
        }
        __syncthreads();
        if (side_by_side[0] && side_by_side[1]) {
            for (int i = tid; i < 2 * dv; i += HS_THREADS) {
                const int g = i & 1, d = i >> 1;
                const float* at = tile + 8 * g * pitch + d;
                uint32_t w[4];
#pragma unroll
                for (int k = 0; k < 4; ++k) w[k] = pack_bf16x2(at[2 * k * pitch], at[(2 * k + 1) * pitch]);
                *reinterpret_cast<uint4*>(v_pool + place[8 * g] + (long long)d * a.block_size) = make_uint4(w[0], w[1], w[2], w[3]);
            }
            return;
        }
    }
    for (int i = tid; i < HS_TOKENS * dv; i += HS_THREADS) {
        const int t = i % HS_TOKENS, d = i / HS_TOKENS;
        if (place[t] >= 0) v_pool[place[t] + (long long)d * a.block_size] = from_f32<T>(tile[t * pitch + d]);
    }
}

// Heads of 16, 32, 64, 128 or 256 numbers, rows of q and k of up to 4 LANES V numbers: LANES lanes (a wave or a workgroup)
// take a row (the q or the k of a token) and keep it in registers, V pieces of 16 bytes a lane, so a row costs one trip to
// memory, and since the 256 numbers of a wave's piece are whole heads, a pair of the rotation lies in two of its lanes.  ROWS
// tokens one after the other, the next one asked for before the present one is worked on; weights and biases stay in
// registers.  The first `v_blocks` workgroups store values.
template <typename T, int LANES, int V, int ROWS>
__global__ __launch_bounds__(HS_THREADS) void joint_rows_kernel(T* __restrict__ q_out, T* __restrict__ k_pool,
                                                                T* __restrict__ v_pool, HeadStoreArgs a, int v_blocks) {
    __shared__ float tile[HS_TOKENS * (HS_MAX_DIM + 1)];
    __shared__ long long place[HS_TOKENS];
    __shared__ float red[16];
    if ((int)blockIdx.x < v_blocks) {
        store_values<T>(v_pool, a, ((int)blockIdx.x / a.v_heads) * HS_TOKENS, (int)blockIdx.x % a.v_heads, tile, place, (int*)red);
        return;
    }
    const int lane = threadIdx.x % LLMS_WAVE, at = threadIdx.x % LANES, dk = a.dk;
    const int item = ((int)blockIdx.x - v_blocks) * (HS_THREADS / LANES) + threadIdx.x / LANES;
    const bool is_q = (item & 1) == 0;
    const int n0 = (item >> 1) * ROWS;
    if (n0 >= a.n_tokens || (!is_q && !a.slots)) return;  // (whole waves; with LANES = 256 the whole workgroup)
    const int width = (is_q ? a.q_heads : a.k_heads) * dk, col = is_q ? 0 : a.q_heads * dk;
    const float* w = is_q ? a.q_norm : a.k_norm;
    const int lph = dk >> 2, li = lane & (lph - 1), half = a.rot_dims >> 1;
    const int hl = half >> 2;
    const bool turns = li < 2 * hl, low = li < hl;
    const int partner = turns ? (low ? lane + hl : lane - hl) : lane;
    struct Row {
        float4 x[V];
        float2 sc[4];  // (the lane's angles are the same in every piece: a piece holds whole heads)
        int slot;
    };
    auto fetch = [&](Row& r, int n) {
        const float* src = a.proj + (size_t)n * a.proj_stride + col;
        r.slot = is_q ? 0 : a.slots[n];
#pragma unroll
        for (int v = 0; v < V; ++v) {
            const int c = 4 * (v * LANES + at);
            r.x[v] = c < width ? *reinterpret_cast<const float4*>(src + c) : make_float4(0.f, 0.f, 0.f, 0.f);
        }
#pragma unroll
        for (int e = 0; e < 4; ++e)
            r.sc[e] = turns ? a.angles[(size_t)n * half + 4 * (low ? li : li - hl) + e] : make_float2(0.f, 1.f);
    };
    float4 wv[V], bv[V];
    Row row;
    fetch(row, n0);
#pragma unroll
    for (int v = 0; v < V; ++v) {
        const int c = 4 * (v * LANES + at);
        const float4 one = make_float4(1.f, 1.f, 1.f, 1.f), zero = make_float4(0.f, 0.f, 0.f, 0.f);
        wv[v] = (w && c < width) ? *reinterpret_cast<const float4*>(w + c) : one;
        bv[v] = (a.bias && c < width) ? *reinterpret_cast<const float4*>(a.bias + col + c) : zero;
    }
#pragma unroll
    for (int i = 0; i < ROWS; ++i) {
        const int n = n0 + i;
        if (n >= a.n_tokens) break;
        Row next;
        if (i + 1 < ROWS) fetch(next, min(n + 1, a.n_tokens - 1));
        float ss = 0.f;
#pragma unroll
        for (int v = 0; v < V; ++v) {
            float4& x = row.x[v];
            x.x += bv[v].x, x.y += bv[v].y, x.z += bv[v].z, x.w += bv[v].w;
            ss += (x.x * x.x + x.y * x.y) + (x.z * x.z + x.w * x.w);
        }
        const float mul = 1.f / sqrtf((LANES == LLMS_WAVE ? wave_sum(ss) : block_sum(ss, red)) / (float)width + a.eps);
        const int page = row.slot / a.block_size, off = row.slot - page * a.block_size;
#pragma unroll
        for (int v = 0; v < V; ++v) {
            const int c = 4 * (v * LANES + at);
            const float4 x = row.x[v];
            float y[4] = {x.x * mul * wv[v].x, x.y * mul * wv[v].y, x.z * mul * wv[v].z, x.w * mul * wv[v].w};
            if (hl > 0) {
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const float other = __shfl(y[e], partner, LLMS_WAVE);
                    const float2 t = low ? rotate_pair(y[e], other, row.sc[e].y, row.sc[e].x) : rotate_pair(other, y[e], row.sc[e].y, row.sc[e].x);
                    if (turns) y[e] = low ? t.x : t.y;
                }
            }
            if (c >= width) continue;
            const int head = c / dk, d = c - head * dk;
            if (is_q) {
                const float factor = query_factor(a, n, head);
#pragma unroll
                for (int e = 0; e < 4; ++e) y[e] *= factor;
                store4<T>(q_out + (size_t)n * a.q_stride + c, y);
            } else if (row.slot >= 0) {
                store4<T>(k_pool + (((size_t)page * a.k_heads + head) * a.block_size + off) * dk + d, y);
            }
        }
        if (i + 1 < ROWS) row = next;
    }
}

// Any sizes: a workgroup a row, the row in LDS (dynamic: the longer of the two).  grid: (tokens, 2 + value heads)
template <typename T>
__global__ __launch_bounds__(HS_THREADS) void joint_store_kernel(T* __restrict__ q_out, T* __restrict__ k_pool,
                                                                 T* __restrict__ v_pool, HeadStoreArgs a) {
    extern __shared__ float joint_row[];
    __shared__ float red[16];
    const int n = blockIdx.x, role = blockIdx.y, dk = a.dk, dv = a.dv;
    int page = 0, off = 0;
    if (role > 0 && !head_slot(a, n, page, off)) return;
    const float* row = a.proj + (size_t)n * a.proj_stride;
    if (role >= 2) {
        const int head = role - 2;
        const float* src = row + (a.v_from_k ? (size_t)(a.q_heads + head) * dk : (size_t)(a.q_heads + a.k_heads) * dk + (size_t)head * dv);
        const float* bias = a.bias ? a.bias + (src - row) : nullptr;
        for (int d = threadIdx.x; d < dv; d += HS_THREADS)
            v_pool[(((size_t)page * a.v_heads + head) * dv + d) * a.block_size + off] = from_f32<T>(src[d] + (bias ? bias[d] : 0.f));
        return;
    }
    const bool is_q = role == 0;
    const int width = (is_q ? a.q_heads : a.k_heads) * dk, col = is_q ? 0 : a.q_heads * dk;
    const float* src = row + col;
    const float* w = is_q ? a.q_norm : a.k_norm;
    float ss = 0.f;
    for (int i = threadIdx.x; i < width; i += HS_THREADS) {
        const float x = src[i] + (a.bias ? a.bias[col + i] : 0.f);
        joint_row[i] = w ? x * w[i] : x;
        ss = fmaf(x, x, ss);
    }
    const float mul = 1.f / sqrtf(block_sum(ss, red) / (float)width + a.eps);
    const float position = a.rot_dims > 0 ? (float)a.positions[n] : 0.f;
    for (int i = threadIdx.x; i < width; i += HS_THREADS) {
        const int head = i / dk, d = i - head * dk;
        const float* at = joint_row + head * dk;
        const float x = turned_element(a, [&](int e) { return at[e] * mul; }, d, n, position);
        if (is_q) q_out[(size_t)n * a.q_stride + i] = from_f32<T>(x * query_factor(a, n, head));
        else k_pool[(((size_t)page * a.k_heads + head) * a.block_size + off) * dk + d] = from_f32<T>(x);
    }
}

template <typename T>
static int launch_joint_store(T* q_out, T* k_pool, T* v_pool, const HeadStoreArgs& a, hipStream_t stream) {
    const int half = a.rot_dims / 2, longest = (a.q_heads > a.k_heads ? a.q_heads : a.k_heads) * a.dk;
    const bool rows = (a.dk == 16 || a.dk == 32 || a.dk == 64 || a.dk == 128 || a.dk == 256) && longest <= 8192 && a.dv <= HS_MAX_DIM &&
                      a.proj_stride % 4 == 0 && a.q_stride % 4 == 0 && ((uintptr_t)a.proj % 16) == 0 && ((uintptr_t)q_out % 16) == 0 &&
                      (!k_pool || ((uintptr_t)k_pool % 16) == 0) && ((uintptr_t)a.q_norm % 16) == 0 && ((uintptr_t)a.k_norm % 16) == 0 && ((uintptr_t)a.bias % 16) == 0 &&
                      (a.rot_dims == 0 || (a.angles && !a.neighbours && half % 4 == 0));
    if (rows) {
        const int v_blocks = a.slots ? (a.n_tokens + HS_TOKENS - 1) / HS_TOKENS * a.v_heads : 0;
        LLMS_REQUIRE(2ll * a.n_tokens + v_blocks < (1ll << 30), "norm_store: too many tokens for one launch");
        // many tokens: a wave (of long rows a workgroup) walks two rows; few: the lanes of a workgroup share a row out
#define JOINT_GO(LANES, V, ROWS)                                                                                          \
    do {                                                                                                                  \
        const int per = HS_THREADS / LANES, items = 2 * ((a.n_tokens + ROWS - 1) / ROWS);                                 \
        joint_rows_kernel<T, LANES, V, ROWS><<<(unsigned)(v_blocks + (items + per - 1) / per), HS_THREADS, 0, stream>>>(   \
            q_out, k_pool, v_pool, a, v_blocks);                                                                          \
    } while (0)
        const bool many = a.n_tokens >= 512;
        if (longest <= 256) JOINT_GO(64, 1, 1);
        else if (longest <= 512) JOINT_GO(64, 2, 1);
        else if (longest <= 1024 && many) JOINT_GO(64, 4, 2);
        else if (longest <= 1024) JOINT_GO(256, 1, 1);
        else if (longest <= 2048 && many) JOINT_GO(64, 8, 2);
        else if (longest <= 2048) JOINT_GO(256, 2, 1);
        else if (longest <= 4096 && many) JOINT_GO(256, 4, 2);
        else if (longest <= 4096) JOINT_GO(256, 4, 1);
        else JOINT_GO(256, 8, 1);
#undef JOINT_GO
        LLMS_LAUNCH_CHECK();
    }
    const size_t lds = (size_t)longest * sizeof(float);
    LLMS_REQUIRE(lds <= 128 * 1024, "norm_store: one norm over all heads takes rows of up to 32,768 numbers");
    if (lds > 32 * 1024)
        LLMS_HIP_CHECK(hipFuncSetAttribute((const void*)joint_store_kernel<T>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    joint_store_kernel<T><<<dim3(a.n_tokens, 2 + a.v_heads), HS_THREADS, lds, stream>>>(q_out, k_pool, v_pool, a);
    LLMS_LAUNCH_CHECK();
}

template <typename T>
static int launch_norm_store(T* q_out, T* k_pool, T* v_pool, const HeadStoreArgs& a, hipStream_t stream) {
    if (a.joint) return launch_joint_store<T>(q_out, k_pool, v_pool, a, stream);
    const int half = a.rot_dims / 2;
    const bool four = a.dk % 4 == 0 && a.dk <= HS_MAX_DIM && a.dv <= HS_MAX_DIM && a.proj_stride % 4 == 0 && a.q_stride % 4 == 0 &&
                      ((uintptr_t)a.proj % 16) == 0 && ((uintptr_t)q_out % 16) == 0 && (!k_pool || ((uintptr_t)k_pool % 16) == 0) &&
                      ((uintptr_t)a.q_norm % 16) == 0 && ((uintptr_t)a.k_norm % 16) == 0 &&
                      (a.rot_dims == 0 || (a.angles && (a.neighbours || half % 4 == 0)));
    if (four) {
        int lph = 1;
        while (4 * lph < a.dk) lph *= 2;
        const int groups = HS_THREADS / lph;
        const long long items = (long long)a.n_tokens * a.q_heads;
        const long long kv_blocks = a.slots ? (long long)((a.n_tokens + HS_TOKENS - 1) / HS_TOKENS) * (a.k_heads + (a.v_from_k ? 0 : a.v_heads)) : 0;
        const int per = items >= 4096 ? 4 : 1;
        const long long q_blocks = (items + (long long)groups * per - 1) / (groups * per);
        LLMS_REQUIRE(items < (1ll << 30) && kv_blocks + q_blocks < (1ll << 31), "norm_store: too many tokens for one launch");
        const unsigned grid = (unsigned)(kv_blocks + q_blocks);
        if (per == 4) head_store_kernel<T, 4><<<grid, HS_THREADS, 0, stream>>>(q_out, k_pool, v_pool, a, lph, (int)kv_blocks);
        else head_store_kernel<T, 1><<<grid, HS_THREADS, 0, stream>>>(q_out, k_pool, v_pool, a, lph, (int)kv_blocks);
    } else {
        dim3 grid(a.n_tokens, a.q_heads + a.k_heads + a.v_heads);
        norm_store_kernel<T><<<grid, LLMS_WAVE, 0, stream>>>(q_out, k_pool, v_pool, a);
    }
    LLMS_LAUNCH_CHECK();
}

// ------------------------------------------------------------------------------------------- attention
struct ComposedArgs {
    int out_stride, q_stride, max_blocks;
    int heads, kv_heads, maps, dk, dv, block_size;
    int window, keep_first, chunk;
    float scale, lambda, eps, out_scale;
    int head_norm;
    const float* dist_bias;  // [heads, dist_reach + 1], or null
    int dist_reach;
    const float* gate;  // 32-bit products [N, gate_stride], or null
    int gate_stride;
    int gate_heads;  // the gate is one number per head, gate[n, h], instead of one per element
    int sink;  // the softmax's denominator holds one more term, exp(0): a key of score zero that has no value
};

template <typename T>
__device__ __forceinline__ float dot_row(const float* __restrict__ q, const T* __restrict__ k, int dk) {
    float acc = 0.f;
    if (dk % 8 == 0) {
        for (int d = 0; d < dk; d += 8) {
            float kv[8];
            if constexpr (sizeof(T) == 2) {
                const uint4 raw = *reinterpret_cast<const uint4*>(k + d);
                const uint32_t w[4] = {raw.x, raw.y, raw.z, raw.w};
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    kv[2 * i] = __uint_as_float(w[i] << 16);
                    kv[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
                }
            } else {
                const float4 a = *reinterpret_cast<const float4*>(k + d);
                const float4 b = *reinterpret_cast<const float4*>(k + d + 4);
                kv[0] = a.x, kv[1] = a.y, kv[2] = a.z, kv[3] = a.w, kv[4] = b.x, kv[5] = b.y, kv[6] = b.z, kv[7] = b.w;
            }
#pragma unroll
            for (int i = 0; i < 8; ++i) acc = fmaf(q[d + i], kv[i], acc);
        }
    } else {
        for (int d = 0; d < dk; ++d) acc = fmaf(q[d], to_f32(k[d]), acc);
    }
    return acc;
}

template <typename T>
__global__ __launch_bounds__(AC_THREADS) void attend_composed_kernel(
    T* __restrict__ out, const T* __restrict__ q, const T* __restrict__ k_pool, const T* __restrict__ v_pool,
    const int* __restrict__ block_tables, const int* __restrict__ table_rows, const int* __restrict__ token_seq,
    const int* __restrict__ positions, const int* __restrict__ context_lens, const float* __restrict__ slopes,
    const float* __restrict__ talk, ComposedArgs a) {
    extern __shared__ float lds[];
    const int H = a.heads, G = a.kv_heads, S = H * a.maps, dk = a.dk, dv = a.dv, bs = a.block_size;
    float* qs = lds;                      // [S][dk], scaled
    float* stat_m = qs + S * dk;          // [S]
    float* stat_l = stat_m + S;           // [S]
    float* prob = stat_l + S;             // [S][AC_TILE]
    float* mixed = prob + S * AC_TILE;    // [H][AC_TILE] (only with talk)
    float* acc_o = mixed + (talk ? H * AC_TILE : 0);  // [S][dv]
    float* talk_s = acc_o + S * dv;       // [H][H] (only with talk)
    int* key_page = reinterpret_cast<int*>(talk_s + (talk ? H * H : 0));  // [AC_TILE]
    int* key_off = key_page + AC_TILE;    // [AC_TILE]

    const int n = blockIdx.x;
    const int tid = threadIdx.x, wave = tid / LLMS_WAVE, lane = tid % LLMS_WAVE;
    const int p = positions[n];
    const int seq = token_seq[n];
    if (context_lens && context_lens[seq] <= 0) {  // a row of padding: it belongs to no request and has no keys
        for (int i = tid; i < H * dv; i += AC_THREADS) out[(size_t)n * a.out_stride + i] = from_f32<T>(0.f);
        return;
    }
    const int* table = block_tables + (size_t)(table_rows ? table_rows[seq] : seq) * a.max_blocks;

    // the visible keys: [r1_lo, r1_lo + n1) (kept first keys that the window has passed) and [r2_lo, p]
    const int lo_chunk = a.chunk > 0 ? p / a.chunk * a.chunk : 0;
    const int lo_win = (a.window > 0 && p - a.window + 1 > 0) ? p - a.window + 1 : 0;
    const int r2_lo = lo_chunk > lo_win ? lo_chunk : lo_win;
    const int r1_lo = lo_chunk;
    int r1_hi = a.keep_first < lo_win ? a.keep_first : lo_win;
    const int n1 = r1_hi > r1_lo ? r1_hi - r1_lo : 0;
    const int n_vis = n1 + (p - r2_lo + 1);
    const int group = H / G;

    const T* qrow = q + (size_t)n * a.q_stride;
    for (int i = tid; i < S * dk; i += AC_THREADS) qs[i] = to_f32(qrow[i]) * a.scale;
    for (int i = tid; i < S * dv; i += AC_THREADS) acc_o[i] = 0.f;
    if (talk)
        for (int i = tid; i < H * H; i += AC_THREADS) talk_s[i] = talk[i];
    __syncthreads();

    // pass 1: every score head's maximum and sum over the visible keys
    for (int s = wave; s < S; s += AC_WAVES) {
        const int h = s / a.maps, kh = (h / group) * a.maps + s % a.maps;
        const float slope = slopes ? slopes[h] : 0.f;
        float m = -INFINITY, l = 0.f;
        for (int v0 = 0; v0 < n_vis; v0 += AC_TILE) {
            const int v = v0 + lane;
            float sc = -INFINITY;
            if (v < n_vis) {
                const int j = v < n1 ? r1_lo + v : r2_lo + (v - n1);
                const int page = table[j / bs], off = j % bs;
                const T* kr = k_pool + (((size_t)page * (G * a.maps) + kh) * bs + off) * dk;
                sc = dot_row<T>(qs + s * dk, kr, dk) - slope * (float)(p - j);
                if (a.dist_bias) sc += a.dist_bias[(size_t)h * (a.dist_reach + 1) + min(p - j, a.dist_reach)];
            }
            const float m_new = fmaxf(m, wave_max(sc));
            const float e = v < n_vis ? expf(sc - m_new) : 0.f;
            l = l * expf(m - m_new) + wave_sum(e);
            m = m_new;
        }
        if (a.sink) {
            const float m_new = fmaxf(m, 0.f);
            l = l * expf(m - m_new) + expf(-m_new);
            m = m_new;
        }
        if (lane == 0) {
            stat_m[s] = m;
            stat_l[s] = l;
        }
    }
    __syncthreads();

    // pass 2: normalised weights tile by tile, mixed over heads if asked for, then the values
    for (int v0 = 0; v0 < n_vis; v0 += AC_TILE) {
        const int v = v0 + lane;
        const int count = n_vis - v0 < AC_TILE ? n_vis - v0 : AC_TILE;
        int j = 0, page = 0, off = 0;
        if (v < n_vis) {
            j = v < n1 ? r1_lo + v : r2_lo + (v - n1);
            page = table[j / bs];
            off = j % bs;
        }
        if (wave == 0) {
            key_page[lane] = page;
            key_off[lane] = off;
        }
        for (int s = wave; s < S; s += AC_WAVES) {
            const int h = s / a.maps, kh = (h / group) * a.maps + s % a.maps;
            float w = 0.f;
            if (v < n_vis) {
                const float slope = slopes ? slopes[h] : 0.f;
                const T* kr = k_pool + (((size_t)page * (G * a.maps) + kh) * bs + off) * dk;
                float sc = dot_row<T>(qs + s * dk, kr, dk) - slope * (float)(p - j);
                if (a.dist_bias) sc += a.dist_bias[(size_t)h * (a.dist_reach + 1) + min(p - j, a.dist_reach)];
                w = expf(sc - stat_m[s]) / stat_l[s];
            }
            prob[s * AC_TILE + lane] = w;
        }
        __syncthreads();
        const float* weights = prob;
        if (talk) {
            for (int i = tid; i < H * AC_TILE; i += AC_THREADS) {
                const int h = i / AC_TILE, jj = i % AC_TILE;
                float t = 0.f;
                for (int g = 0; g < H; ++g) t = fmaf(talk_s[h * H + g], prob[g * AC_TILE + jj], t);
                mixed[i] = t;
            }
            __syncthreads();
            weights = mixed;
        }
        for (int s = wave; s < S; s += AC_WAVES) {
            const int vh = (s / a.maps) / group;
            for (int d = lane; d < dv; d += LLMS_WAVE) {
                float o = acc_o[s * dv + d];
                for (int jj = 0; jj < count; ++jj) {
                    const T* vr = v_pool + (((size_t)key_page[jj] * G + vh) * dv + d) * bs + key_off[jj];
                    o = fmaf(weights[s * AC_TILE + jj], to_f32(*vr), o);
                }
                acc_o[s * dv + d] = o;
            }
        }
        __syncthreads();
    }

    // what leaves: per query head, the two maps combined and the head normed where asked for
    T* orow = out + (size_t)n * a.out_stride;
    for (int h = wave; h < H; h += AC_WAVES) {
        float ss = 0.f;
        for (int d = lane; d < dv; d += LLMS_WAVE) {
            float o = acc_o[(h * a.maps) * dv + d];
            if (a.maps == 2) o -= a.lambda * acc_o[(h * 2 + 1) * dv + d];
            ss = fmaf(o, o, ss);
        }
        float mul = 1.f;
        if (a.head_norm) mul = a.out_scale / sqrtf(wave_sum(ss) / (float)dv + a.eps);
        for (int d = lane; d < dv; d += LLMS_WAVE) {
            float o = acc_o[(h * a.maps) * dv + d];
            if (a.maps == 2) o -= a.lambda * acc_o[(h * 2 + 1) * dv + d];
            o *= mul;
            if (a.gate) o /= 1.f + expf(-a.gate[(size_t)n * a.gate_stride + (a.gate_heads ? h : h * dv + d)]);
            orow[h * dv + d] = from_f32<T>(o);
        }
    }
}

static size_t composed_lds_bytes(int heads, int maps, int dk, int dv, bool talk) {
    const size_t S = (size_t)heads * maps;
    size_t floats = S * dk + 2 * S + S * AC_TILE + S * dv;
    if (talk) floats += (size_t)heads * AC_TILE + (size_t)heads * heads;
    return floats * sizeof(float) + 2 * AC_TILE * sizeof(int);
}

extern "C" {

int llms_conv_store(int dtype, void* q_out, int q_stride, const float* proj, int proj_stride, const float* taps_w, int taps,
                    const float* state, size_t state_slot_stride, const int* state_slots, const int* token_seq,
                    const int* positions, const int* cu_seqlens, const int* slots, void* k_pool, void* v_pool, int n_tokens,
                    int cq, int ck, int cv, int k_heads, int dk, int v_heads, int dv, int block_size, float* state_out,
                    const int* context_lens, hipStream_t stream) {
    LLMS_REQUIRE(n_tokens > 0 && cq > 0 && ck >= 0 && cv >= 0, "conv_store: sizes must be positive");
    LLMS_REQUIRE(ck == k_heads * dk && cv == v_heads * dv, "conv_store: channels do not match heads times sizes");
    LLMS_REQUIRE(taps < 1 || (taps_w && token_seq && positions && cu_seqlens),
                 "conv_store: a convolution needs its taps and the batch's arrays");
    LLMS_REQUIRE(taps <= 1 || (state && state_slots), "conv_store: a convolution of two taps or more needs the state");
    LLMS_REQUIRE(!slots || (k_pool && v_pool && block_size > 0), "conv_store: slots given without pools");
    LLMS_REQUIRE(!state_out || (context_lens && state_out == state), "conv_store: the ring is updated in place, with the requests' lengths at hand");
    dim3 grid(n_tokens, (cq + ck + cv + AC_THREADS - 1) / AC_THREADS);
    if (dtype == 0)
        conv_store_kernel<float><<<grid, AC_THREADS, 0, stream>>>(
            (float*)q_out, q_stride, proj, proj_stride, taps_w, taps, state, state_slot_stride, state_slots, token_seq,
            positions, cu_seqlens, slots, (float*)k_pool, (float*)v_pool, cq, ck, cv, k_heads, dk, v_heads, dv, block_size,
            state_out, context_lens);
    else if (dtype == 1)
        conv_store_kernel<bf16><<<grid, AC_THREADS, 0, stream>>>(
            (bf16*)q_out, q_stride, proj, proj_stride, taps_w, taps, state, state_slot_stride, state_slots, token_seq,
            positions, cu_seqlens, slots, (bf16*)k_pool, (bf16*)v_pool, cq, ck, cv, k_heads, dk, v_heads, dv, block_size,
            state_out, context_lens);
    else
        LLMS_REQUIRE(false, "conv_store: dtype must be 0 (float32) or 1 (bfloat16)");
    LLMS_LAUNCH_CHECK();
}

int llms_norm_store(int dtype, void* q_out, int q_stride, const float* proj, int proj_stride, const float* q_norm,
                    const float* k_norm, float eps, float temp_coef, int temp_every, const int* positions, const int* slots,
                    void* k_pool, void* v_pool, int n_tokens, int q_heads, int k_heads, int dk, int v_heads, int dv,
                    int block_size, const float* freq, const float* angles, int rot_dims, int unit_norm, int neighbours,
                    int norm_first, const float* q_scale, int v_from_k, int joint, const float* bias, hipStream_t stream) {
    LLMS_REQUIRE(n_tokens > 0 && q_heads > 0 && k_heads >= 0 && v_heads >= 0 && dk > 0 && dv > 0, "norm_store: sizes must be positive");
    LLMS_REQUIRE(rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= dk && (rot_dims == 0 || angles || (freq && positions)),
                 "norm_store: an even number of turned dimensions within a head, with angles or frequencies and positions");
    LLMS_REQUIRE(((uintptr_t)angles % 8) == 0, "norm_store: the table of angles must be 8-byte aligned");
    LLMS_REQUIRE(temp_every == 0 || positions, "norm_store: a factor by position needs the positions");
    LLMS_REQUIRE(!slots || (k_pool && v_pool && block_size > 0), "norm_store: slots given without pools");
    LLMS_REQUIRE(q_heads + k_heads + v_heads <= 65535, "norm_store: up to 65,535 heads in all");
    LLMS_REQUIRE(!v_from_k || (v_heads == k_heads && dv == dk), "norm_store: values that are the keys have their heads and size");
    HeadStoreArgs a;
    a.q_stride = q_stride, a.proj_stride = proj_stride, a.proj = proj, a.q_norm = q_norm, a.k_norm = k_norm, a.q_scale = q_scale;
    a.freq = freq, a.angles = reinterpret_cast<const float2*>(angles), a.positions = positions, a.slots = slots;
    a.eps = eps, a.temp_coef = temp_coef, a.temp_every = temp_every;
    a.n_tokens = n_tokens, a.q_heads = q_heads, a.k_heads = k_heads, a.dk = dk, a.v_heads = v_heads, a.dv = dv;
    a.block_size = block_size > 0 ? block_size : 1, a.rot_dims = rot_dims;
    a.unit_norm = unit_norm, a.neighbours = neighbours, a.norm_first = norm_first, a.v_from_k = v_from_k, a.joint = joint, a.bias = bias;
    LLMS_REQUIRE(!bias || joint, "norm_store: a bias goes with one norm over all heads");
    LLMS_REQUIRE(!joint || norm_first || rot_dims == 0, "norm_store: one norm over all heads comes before the rotation");
    LLMS_REQUIRE(!joint || rot_dims == 0 || positions, "norm_store: a rotation needs the positions");
    if (dtype == 0) return launch_norm_store<float>((float*)q_out, (float*)k_pool, (float*)v_pool, a, stream);
    if (dtype == 1) return launch_norm_store<bf16>((bf16*)q_out, (bf16*)k_pool, (bf16*)v_pool, a, stream);
    LLMS_REQUIRE(false, "norm_store: dtype must be 0 (float32) or 1 (bfloat16)");
}

int llms_conv_state(float* state, size_t state_slot_stride, const int* state_slots, const float* proj, int proj_stride,
                    const int* cu_seqlens, const int* context_lens, int n_seqs, int taps, int channels,
                    hipStream_t stream) {
    LLMS_REQUIRE(n_seqs > 0 && taps > 1 && channels > 0, "conv_state: sizes must be positive and taps at least 2");
    dim3 grid(n_seqs, (channels + AC_THREADS - 1) / AC_THREADS);
    conv_state_kernel<<<grid, AC_THREADS, 0, stream>>>(state, state_slot_stride, state_slots, proj, proj_stride, cu_seqlens,
                                                       context_lens, taps, channels);
    LLMS_LAUNCH_CHECK();
}

int llms_attend_composed(int dtype, void* out, int out_stride, const void* q, int q_stride, const void* k_pool,
                         const void* v_pool, const int* block_tables, const int* table_rows, int max_blocks,
                         const int* token_seq, const int* positions, const int* context_lens, int n_tokens, int heads,
                         int kv_heads, int maps,
                         int dk, int dv, int block_size, int window, int keep_first, int chunk, float scale,
                         const float* slopes, const float* talk, float lambda, int head_norm, float eps, float out_scale,
                         const float* dist_bias, int dist_reach, const float* gate, int gate_stride, int gate_heads, int sink,
                         hipStream_t stream) {
    LLMS_REQUIRE(n_tokens > 0 && heads > 0 && kv_heads > 0 && dk > 0 && dv > 0, "attend_composed: sizes must be positive");
    LLMS_REQUIRE(!dist_bias || dist_reach >= 0, "attend_composed: a distance table has at least one entry per head");
    LLMS_REQUIRE(heads % kv_heads == 0, "attend_composed: heads must be a multiple of kv_heads");
    LLMS_REQUIRE(maps == 1 || maps == 2, "attend_composed: one or two score maps");
    LLMS_REQUIRE(!(talk && maps != 1), "attend_composed: mixing heads' weights goes with one score map");
    LLMS_REQUIRE(block_size > 0 && max_blocks > 0, "attend_composed: block_size and max_blocks must be positive");
    LLMS_REQUIRE(window >= 0 && keep_first >= 0 && chunk >= 0, "attend_composed: window, keep_first and chunk are >= 0");
    const size_t lds = composed_lds_bytes(heads, maps, dk, dv, talk != nullptr);
    LLMS_REQUIRE(lds <= 160 * 1024, "attend_composed: heads times sizes do not fit the 160 KB of LDS");
    ComposedArgs a;
    a.out_stride = out_stride, a.q_stride = q_stride, a.max_blocks = max_blocks;
    a.heads = heads, a.kv_heads = kv_heads, a.maps = maps, a.dk = dk, a.dv = dv, a.block_size = block_size;
    a.window = window, a.keep_first = keep_first, a.chunk = chunk;
    a.scale = scale, a.lambda = lambda, a.eps = eps, a.out_scale = out_scale, a.head_norm = head_norm;
    a.dist_bias = dist_bias, a.dist_reach = dist_reach, a.gate = gate, a.gate_stride = gate_stride, a.gate_heads = gate_heads, a.sink = sink;
    if (dtype == 0) {
        auto kernel = attend_composed_kernel<float>;
        if (lds > 48 * 1024)
            LLMS_HIP_CHECK(hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
        kernel<<<n_tokens, AC_THREADS, lds, stream>>>((float*)out, (const float*)q, (const float*)k_pool,
                                                      (const float*)v_pool, block_tables, table_rows, token_seq, positions,
                                                      context_lens, slopes, talk, a);
    } else if (dtype == 1) {
        auto kernel = attend_composed_kernel<bf16>;
        if (lds > 48 * 1024)
            LLMS_HIP_CHECK(hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
        kernel<<<n_tokens, AC_THREADS, lds, stream>>>((bf16*)out, (const bf16*)q, (const bf16*)k_pool, (const bf16*)v_pool,
                                                      block_tables, table_rows, token_seq, positions, context_lens, slopes, talk,
                                                      a);
    } else {
        LLMS_REQUIRE(false, "attend_composed: dtype must be 0 (float32) or 1 (bfloat16)");
    }
    LLMS_LAUNCH_CHECK();
}

}  // extern "C"
