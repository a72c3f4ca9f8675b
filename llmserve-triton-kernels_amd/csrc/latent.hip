// Attention through a latent: a token keeps one row [c ; kr] of r + dr numbers for all heads (c the normed latent
// that keys and values are projected from, kr one rotated key part that all heads share).  With the keys' projection
// folded into the query, q'_h = [W_uk_h^T q_h ; qr_h], head h's score against key j is q'_h . [c_j ; kr_j] and its
// result the softmax-weighted sum of c_j, which the caller projects to values afterwards.
//
//   latent_prepare   from the 32-bit input products z of a step's tokens: cq = rms_unit(z_q) * wq (rounded once);
//                    c = rms_unit(z_c) * wc and kr = rotated z_kr stored at the token's cache row
//   latent_query     from the 32-bit queries [N, H, dn + dr]: the unrotated parts side by side [N, H, dn] and the
//                    rotated parts turned into q'[n, h, r ..]
//   latent_split     the two in one launch where the queries have no latent of their own
//   attend_latent    out[n, h, :r] = sum_j softmax_j(q'[n, h] . row_j * scale) c_j over the keys the window allows; with `sink` head h's
//                    denominator holds one more term, exp(sink[h]), that has no value
//
// Rotation: pairs (2i, 2i+1) of the first `dims` numbers of the rotated part (`half`: pairs (i, i + dims/2) instead),
// angle position * freq[i], the rest of the part passes.  Norms, angles, scores, softmax and sums are 32-bit; T (float or bfloat16) is what is stored.
#include "common.h"

#define LAT_THREADS 256

// The turn of a rotated part's first `dims` numbers at one position: angles from the step's table (sine, cosine), or
// worked out here.
struct LatentTurn {
    const float* freq;
    const float2* angles;  // [N, dims / 2], or null
    int dims, half;        // half: pairs (i, i + dims / 2)
};

__device__ __forceinline__ float2 latent_angle(const LatentTurn& t, int n, float position, int i) {
    return t.angles ? t.angles[(size_t)n * (t.dims >> 1) + i] : rotary_angle(position, t.freq[i]);
}

__device__ __forceinline__ float rotated_element(const LatentTurn& t, const float* __restrict__ part, int e, int n, float position) {
    if (e >= t.dims) return part[e];
    if (t.half) {  // dimension i turns together with dimension i + dims / 2
        const int h = t.dims >> 1, i = e < h ? e : e - h;
        const float2 sc = latent_angle(t, n, position, i);
        const float2 turned = rotate_pair(part[i], part[i + h], sc.y, sc.x);
        return e < h ? turned.x : turned.y;
    }
    const int i = e >> 1;
    const float2 sc = latent_angle(t, n, position, i);  // (sine, cosine)
    const float2 turned = rotate_pair(part[2 * i], part[2 * i + 1], sc.y, sc.x);
    return (e & 1) ? turned.y : turned.x;
}

// One token's cache row from its latent's r numbers and, behind them, its rotated key part.  `red`: 16 floats of LDS.
template <typename T>
__device__ __forceinline__ void latent_row(T* __restrict__ pool, const float* __restrict__ zc, int r, int dr,
                                           const float* __restrict__ wc, const LatentTurn& t, int n,
                                           const int* __restrict__ positions, const int* __restrict__ slots, float eps, float* red) {
    const int slot = slots ? slots[n] : -1;
    const float position = t.dims > 0 && !t.angles ? (float)positions[n] : 0.f;
    float ss = 0.f;
    for (int c = threadIdx.x; c < r; c += LAT_THREADS) ss = fmaf(zc[c], zc[c], ss);
    const float inv = 1.0f / sqrtf(block_sum(ss, red) / (float)r + eps);
    if (slot < 0) return;
    T* row = pool + (size_t)slot * (r + dr);
    for (int c = threadIdx.x; c < r; c += LAT_THREADS) row[c] = from_f32<T>(zc[c] * inv * wc[c]);
    for (int e = threadIdx.x; e < dr; e += LAT_THREADS) row[r + e] = from_f32<T>(rotated_element(t, zc + r, e, n, position));
}

template <typename T>
__device__ __forceinline__ void latent_store4(T* dst, float4 v) {
    if constexpr (sizeof(T) == 2)
        *reinterpret_cast<uint2*>(dst) = make_uint2(pack_bf16x2(v.x, v.y), pack_bf16x2(v.z, v.w));
    else
        *reinterpret_cast<float4*>(dst) = v;
}

// One token's queries [H, dn + dr] -> plain [H, dn] and folded[h, r ..] of row length H * (r + dr).  `first`, `step`:
// which pieces this thread takes.  `four`: 4 numbers a piece (sizes in multiples of 4, a pair's partner in the same place
// of another piece or in the same piece).
template <typename T>
__device__ __forceinline__ void latent_query_row(T* __restrict__ plain, T* __restrict__ folded, const float* __restrict__ qr,
                                                 int heads, int dn, int dr, int r, const LatentTurn& t, int n,
                                                 const int* __restrict__ positions, int first, int step, bool four) {
    const int dq = dn + dr;
    const float position = t.dims > 0 && !t.angles ? (float)positions[n] : 0.f;
    T* prow = plain + (size_t)n * heads * dn;
    T* frow = folded + (size_t)n * heads * (r + dr);
    if (four) {
        const int per = dq / 4, items = heads * per, h2 = t.dims >> 1;
        constexpr int AT_ONCE = 4;  // pieces asked for before the first is used
        for (int i0 = first; i0 < items; i0 += AT_ONCE * step) {
            float4 v[AT_ONCE], other[AT_ONCE];
#pragma unroll
            for (int u = 0; u < AT_ONCE; ++u) {
                const int i = min(i0 + u * step, items - 1), e = 4 * (i % per) - dn;
                v[u] = *reinterpret_cast<const float4*>(qr + 4 * i);
                other[u] = v[u];
                if (t.half && e >= 0 && e < t.dims) other[u] = *reinterpret_cast<const float4*>(qr + 4 * i + (e < h2 ? h2 : -h2));
            }
#pragma unroll
            for (int u = 0; u < AT_ONCE; ++u) {
                const int i = i0 + u * step;
                if (i >= items) break;
                const int h = i / per, e = 4 * (i - h * per) - dn;  // place in the rotated part (< 0: plain)
                if (e < 0) {
                    latent_store4<T>(prow + h * dn + e + dn, v[u]);
                    continue;
                }
                if (e < t.dims) {
                    float x[4] = {v[u].x, v[u].y, v[u].z, v[u].w};
                    if (t.half) {
                        const float y[4] = {other[u].x, other[u].y, other[u].z, other[u].w};
                        const bool low = e < h2;
#pragma unroll
                        for (int k = 0; k < 4; ++k) {
                            const float2 sc = latent_angle(t, n, position, (low ? e : e - h2) + k);
                            const float2 turned = low ? rotate_pair(x[k], y[k], sc.y, sc.x) : rotate_pair(y[k], x[k], sc.y, sc.x);
                            x[k] = low ? turned.x : turned.y;
                        }
                    } else {
#pragma unroll
                        for (int k = 0; k < 2; ++k) {
                            if (e + 2 * k >= t.dims) continue;
                            const float2 sc = latent_angle(t, n, position, (e >> 1) + k);
                            const float2 turned = rotate_pair(x[2 * k], x[2 * k + 1], sc.y, sc.x);
                            x[2 * k] = turned.x, x[2 * k + 1] = turned.y;
                        }
                    }
                    v[u] = make_float4(x[0], x[1], x[2], x[3]);
                }
                latent_store4<T>(frow + h * (r + dr) + r + e, v[u]);
            }
        }
        return;
    }
    for (int i = first; i < heads * dq; i += step) {
        const int h = i / dq, e = i - h * dq;
        if (e < dn) prow[h * dn + e] = from_f32<T>(qr[i]);
        else frow[h * (r + dr) + r + (e - dn)] = from_f32<T>(rotated_element(t, qr + h * dq + dn, e - dn, n, position));
    }
}

// grid: tokens.  z [N, z_ld] float: columns col_q .. + q_rank are the query latent, col_c .. + r + dr the key/value
// latent and the rotated key part (col_c < 0: the layer keeps none).  pool [rows, r + dr] rows at slots[n] (< 0: none).
template <typename T>
__global__ __launch_bounds__(LAT_THREADS) void latent_prepare_kernel(
    T* __restrict__ cq, T* __restrict__ pool, const float* __restrict__ z, int z_ld, int col_q, int q_rank, int col_c,
    int r, int dr, const float* __restrict__ wq, const float* __restrict__ wc, LatentTurn t,
    const int* __restrict__ positions, const int* __restrict__ slots, float eps) {
    __shared__ float red[16];
    const int n = blockIdx.x;
    const float* zr = z + (size_t)n * z_ld;
    if (q_rank > 0) {
        float ss = 0.f;
        for (int c = threadIdx.x; c < q_rank; c += LAT_THREADS) ss = fmaf(zr[col_q + c], zr[col_q + c], ss);
        const float inv = 1.0f / sqrtf(block_sum(ss, red) / (float)q_rank + eps);
        for (int c = threadIdx.x; c < q_rank; c += LAT_THREADS)
            cq[(size_t)n * q_rank + c] = from_f32<T>(zr[col_q + c] * inv * wq[c]);
    }
    if (col_c < 0) return;
    latent_row<T>(pool, zr + col_c, r, dr, wc, t, n, positions, slots, eps, red);
}

// grid: (tokens, workgroups a token's queries are dealt to).  q [N, q_ld] float holds heads * (dn + dr) numbers a row.
template <typename T>
__global__ __launch_bounds__(LAT_THREADS) void latent_query_kernel(
    T* __restrict__ plain, T* __restrict__ folded, const float* __restrict__ q, int q_ld, int heads, int dn, int dr, int r,
    LatentTurn t, const int* __restrict__ positions, int four) {
    const int n = blockIdx.x;
    latent_query_row<T>(plain, folded, q + (size_t)n * q_ld, heads, dn, dr, r, t, n, positions,
                        blockIdx.y * LAT_THREADS + threadIdx.x, gridDim.y * LAT_THREADS, four);
}

// Both at once, for queries that are projected without a latent of their own: they lie in z beside the key/value latent.
// grid: (tokens, 1 + workgroups a token's queries are dealt to).
template <typename T>
__global__ __launch_bounds__(LAT_THREADS) void latent_split_kernel(
    T* __restrict__ plain, T* __restrict__ folded, T* __restrict__ pool, const float* __restrict__ z, int z_ld, int col_q,
    int col_c, int heads, int dn, int dr, int r, const float* __restrict__ wc, LatentTurn t, const int* __restrict__ positions,
    const int* __restrict__ slots, float eps, int four) {
    __shared__ float red[16];
    const int n = blockIdx.x;
    const float* zr = z + (size_t)n * z_ld;
    if (blockIdx.y == 0) {
        if (col_c >= 0) latent_row<T>(pool, zr + col_c, r, dr, wc, t, n, positions, slots, eps, red);
        return;
    }
    latent_query_row<T>(plain, folded, zr + col_q, heads, dn, dr, r, t, n, positions,
                        ((int)blockIdx.y - 1) * LAT_THREADS + threadIdx.x, ((int)gridDim.y - 1) * LAT_THREADS, four);
}

// Whether queries at `q` (row stride q_ld) and their places can be taken 4 numbers at a time.
static bool latent_four(const float* q, long q_ld, const void* plain, const void* folded, int dn, int dr, int r, int dims, int half) {
    return dn % 4 == 0 && dr % 4 == 0 && r % 4 == 0 && q_ld % 4 == 0 && ((uintptr_t)q % 16) == 0 && ((uintptr_t)plain % 16) == 0 &&
           ((uintptr_t)folded % 16) == 0 && (!half || dims % 8 == 0);
}

// Workgroups a token's queries are dealt to: one where the tokens alone fill the chip, else one per 256 pieces.
static unsigned latent_query_groups(int n, int heads, int dq, bool four) {
    if (n >= 1024) return 1;
    const int pieces = heads * (four ? dq / 4 : dq), groups = (pieces + LAT_THREADS - 1) / LAT_THREADS;
    return (unsigned)(groups < 64 ? groups : 64);
}

// What a lane holds of a row of up to 64 * LAT_PER_LANE numbers: elements lane, lane + 64, ...
#define LAT_PER_LANE 16
#define LAT_WAVES (LAT_THREADS / LLMS_WAVE)

// grid (tokens, heads); the workgroup's 4 waves take the keys j with j % 4 == wave, each with a running softmax, and
// meet in LDS.  Which keys a wave takes, and in which order, depends on the token's position alone.
template <typename T>
__global__ __launch_bounds__(LAT_THREADS) void attend_latent_kernel(
    T* __restrict__ out, const T* __restrict__ q, const T* __restrict__ pool, const int* __restrict__ tables,
    int table_width, const int* __restrict__ table_rows, const int* __restrict__ token_seq,
    const int* __restrict__ positions, const int* __restrict__ context_lens, int heads, int r, int dr, int block_size,
    int window, float scale, const float* __restrict__ sink) {
    extern __shared__ float lds[];  // per wave: r sums, maximum, sum of weights
    const int n = blockIdx.x, h = blockIdx.y, dk = r + dr;
    const int lane = threadIdx.x % LLMS_WAVE, wave = threadIdx.x / LLMS_WAVE;
    const int seq = token_seq[n], pos = positions[n];
    T* orow = out + ((size_t)n * heads + h) * r;
    if (context_lens[seq] <= pos) {  // (a padding row: a request without keys)
        for (int c = threadIdx.x; c < r; c += LAT_THREADS) orow[c] = from_f32<T>(0.f);
        return;
    }
    const int* table = tables + (size_t)(table_rows ? table_rows[seq] : seq) * table_width;
    const int lo = window > 0 ? max(0, pos - window + 1) : 0;
    float qv[LAT_PER_LANE], acc[LAT_PER_LANE];
    const T* qrow = q + ((size_t)n * heads + h) * dk;
#pragma unroll
    for (int i = 0; i < LAT_PER_LANE; ++i) {
        const int e = lane + i * LLMS_WAVE;
        qv[i] = e < dk ? to_f32(qrow[e]) : 0.f;
        acc[i] = 0.f;
    }
    float m = -INFINITY, l = 0.f;
    int j = lo + ((wave - lo) % LAT_WAVES + LAT_WAVES) % LAT_WAVES;  // the first key >= lo with j % 4 == wave
    for (; j <= pos; j += LAT_WAVES) {
        const int page = table[j / block_size];
        const T* krow = pool + ((size_t)page * block_size + j % block_size) * dk;
        float kv[LAT_PER_LANE];
        float dot = 0.f;
#pragma unroll
        for (int i = 0; i < LAT_PER_LANE; ++i) {
            const int e = lane + i * LLMS_WAVE;
            kv[i] = e < dk ? to_f32(krow[e]) : 0.f;
            dot = fmaf(qv[i], kv[i], dot);
        }
        const float s = wave_sum(dot) * scale;
        const float m_new = fmaxf(m, s);
        const float fix = expf(m - m_new), p = expf(s - m_new);
        l = l * fix + p;
#pragma unroll
        for (int i = 0; i < LAT_PER_LANE; ++i) acc[i] = fmaf(p, kv[i], acc[i] * fix);
        m = m_new;
    }
    float* mine = lds + (size_t)wave * (r + 2);
#pragma unroll
    for (int i = 0; i < LAT_PER_LANE; ++i) {
        const int e = lane + i * LLMS_WAVE;
        if (e < r) mine[e] = acc[i];
    }
    if (lane == 0) {
        mine[r] = m;
        mine[r + 1] = l;
    }
    __syncthreads();
    float top = -INFINITY;
#pragma unroll
    for (int w = 0; w < LAT_WAVES; ++w) top = fmaxf(top, lds[(size_t)w * (r + 2) + r]);
    if (sink) top = fmaxf(top, sink[h]);
    float f[LAT_WAVES], total = 0.f;
#pragma unroll
    for (int w = 0; w < LAT_WAVES; ++w) {
        f[w] = expf(lds[(size_t)w * (r + 2) + r] - top);  // (a wave without keys: exp(-inf) = 0)
        total = fmaf(lds[(size_t)w * (r + 2) + r + 1], f[w], total);
    }
    if (sink) total += expf(sink[h] - top);
    const float inv = 1.0f / total;
    for (int c = threadIdx.x; c < r; c += LAT_THREADS) {
        float v = 0.f;
#pragma unroll
        for (int w = 0; w < LAT_WAVES; ++w) v = fmaf(lds[(size_t)w * (r + 2) + c], f[w], v);
        orow[c] = from_f32<T>(v * inv);
    }
}

extern "C" {

// angles (may be null): float [n, dims / 2, 2], the sines and cosines that stand for freq and positions
int llms_latent_prepare(int dtype, void* cq, void* pool, const float* z, int z_ld, int col_q, int q_rank, int col_c, int r,
                        int dr, const float* wq, const float* wc, const float* freq, const float* angles, int dims,
                        const int* positions, const int* slots, float eps, int n, int half_pairs, hipStream_t stream) {
    LLMS_REQUIRE(n > 0 && r > 0 && dr >= 0 && q_rank >= 0, "latent_prepare: sizes must be positive");
    LLMS_REQUIRE(dims >= 0 && dims <= dr && dims % 2 == 0, "latent_prepare: an even number of turned dimensions within the part");
    LLMS_REQUIRE(dtype == 0 || dtype == 1, "latent_prepare: dtype must be 0 (float32) or 1 (bfloat16)");
    LLMS_REQUIRE(((uintptr_t)angles % 8) == 0, "latent_prepare: the table of angles must be 8-byte aligned");
    const LatentTurn t = {freq, reinterpret_cast<const float2*>(angles), dims, half_pairs};
    if (dtype == 0)
        latent_prepare_kernel<float><<<n, LAT_THREADS, 0, stream>>>((float*)cq, (float*)pool, z, z_ld, col_q, q_rank, col_c, r, dr,
                                                                    wq, wc, t, positions, slots, eps);
    else
        latent_prepare_kernel<bf16><<<n, LAT_THREADS, 0, stream>>>((bf16*)cq, (bf16*)pool, z, z_ld, col_q, q_rank, col_c, r, dr,
                                                                   wq, wc, t, positions, slots, eps);
    LLMS_LAUNCH_CHECK();
}

int llms_latent_query(int dtype, void* plain, void* folded, const float* q, int heads, int dn, int dr, int r,
                      const float* freq, const float* angles, int dims, const int* positions, int n, int half_pairs,
                      hipStream_t stream) {
    LLMS_REQUIRE(n > 0 && heads > 0 && dn > 0 && dr >= 0 && r > 0, "latent_query: sizes must be positive");
    LLMS_REQUIRE(dims >= 0 && dims <= dr && dims % 2 == 0, "latent_query: an even number of turned dimensions within the part");
    LLMS_REQUIRE(dtype == 0 || dtype == 1, "latent_query: dtype must be 0 (float32) or 1 (bfloat16)");
    LLMS_REQUIRE(((uintptr_t)angles % 8) == 0, "latent_query: the table of angles must be 8-byte aligned");
    const LatentTurn t = {freq, reinterpret_cast<const float2*>(angles), dims, half_pairs};
    const int q_ld = heads * (dn + dr);
    const bool four = latent_four(q, q_ld, plain, folded, dn, dr, r, dims, half_pairs);
    const dim3 grid(n, latent_query_groups(n, heads, dn + dr, four));
    if (dtype == 0)
        latent_query_kernel<float><<<grid, LAT_THREADS, 0, stream>>>((float*)plain, (float*)folded, q, q_ld, heads, dn, dr, r, t,
                                                                     positions, four);
    else
        latent_query_kernel<bf16><<<grid, LAT_THREADS, 0, stream>>>((bf16*)plain, (bf16*)folded, q, q_ld, heads, dn, dr, r, t,
                                                                    positions, four);
    LLMS_LAUNCH_CHECK();
}

// z [n, z_ld]: columns col_q .. + heads * (dn + dr) the queries, col_c .. + r + dr the latent and the rotated key part
// (col_c < 0: none is kept)
int llms_latent_split(int dtype, void* plain, void* folded, void* pool, const float* z, int z_ld, int col_q, int col_c, int heads,
                      int dn, int dr, int r, const float* wc, const float* freq, const float* angles, int dims,
                      const int* positions, const int* slots, float eps, int n, int half_pairs, hipStream_t stream) {
    LLMS_REQUIRE(n > 0 && heads > 0 && dn > 0 && dr >= 0 && r > 0, "latent_split: sizes must be positive");
    LLMS_REQUIRE(dims >= 0 && dims <= dr && dims % 2 == 0, "latent_split: an even number of turned dimensions within the part");
    LLMS_REQUIRE(dtype == 0 || dtype == 1, "latent_split: dtype must be 0 (float32) or 1 (bfloat16)");
    LLMS_REQUIRE(col_q >= 0 && (col_c < 0 || (wc && pool && slots)), "latent_split: a kept latent needs its weight, pool and slots");
    LLMS_REQUIRE(((uintptr_t)angles % 8) == 0, "latent_split: the table of angles must be 8-byte aligned");
    const LatentTurn t = {freq, reinterpret_cast<const float2*>(angles), dims, half_pairs};
    const bool four = latent_four(z + col_q, z_ld, plain, folded, dn, dr, r, dims, half_pairs);
    const dim3 grid(n, 1 + latent_query_groups(n, heads, dn + dr, four));
    if (dtype == 0)
        latent_split_kernel<float><<<grid, LAT_THREADS, 0, stream>>>((float*)plain, (float*)folded, (float*)pool, z, z_ld, col_q,
                                                                     col_c, heads, dn, dr, r, wc, t, positions, slots, eps, four);
    else
        latent_split_kernel<bf16><<<grid, LAT_THREADS, 0, stream>>>((bf16*)plain, (bf16*)folded, (bf16*)pool, z, z_ld, col_q,
                                                                    col_c, heads, dn, dr, r, wc, t, positions, slots, eps, four);
    LLMS_LAUNCH_CHECK();
}

int llms_attend_latent(int dtype, void* out, const void* q, const void* pool, const int* tables, int table_width,
                       const int* table_rows, const int* token_seq, const int* positions, const int* context_lens, int n,
                       int heads, int r, int dr, int block_size, int window, float scale, const float* sink, hipStream_t stream) {
    LLMS_REQUIRE(n > 0 && heads > 0 && r > 0 && dr >= 0 && block_size > 0 && table_width > 0, "attend_latent: sizes must be positive");
    LLMS_REQUIRE(r + dr <= LLMS_WAVE * LAT_PER_LANE, "attend_latent: a cache row of up to 1,024 numbers");
    LLMS_REQUIRE(heads <= 65535, "attend_latent: too many heads for one launch");
    LLMS_REQUIRE(dtype == 0 || dtype == 1, "attend_latent: dtype must be 0 (float32) or 1 (bfloat16)");
    const size_t lds = (size_t)LAT_WAVES * (r + 2) * sizeof(float);
    dim3 grid(n, heads);
    if (dtype == 0)
        attend_latent_kernel<float><<<grid, LAT_THREADS, lds, stream>>>((float*)out, (const float*)q, (const float*)pool, tables,
                                                                        table_width, table_rows, token_seq, positions,
                                                                        context_lens, heads, r, dr, block_size, window, scale, sink);
    else
        attend_latent_kernel<bf16><<<grid, LAT_THREADS, lds, stream>>>((bf16*)out, (const bf16*)q, (const bf16*)pool, tables,
                                                                       table_width, table_rows, token_seq, positions,
                                                                       context_lens, heads, r, dr, block_size, window, scale, sink);
    LLMS_LAUNCH_CHECK();
}

}  // extern "C"
