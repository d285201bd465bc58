// Position encoding of queries and keys with the cache write, for the variants that the
// rotate-half kernel (rope_cache.hip) does not cover:
//
//  * kva_qk_encode_cache: heads of queries and keys whose first `rot` elements are rotated with
//    either pairing (pair i = elements (i, i + rot/2) or (2i, 2i + 1)), optionally followed by a
//    division of every head by its root mean square (and a multiplication by a weight per element,
//    one for queries and one for keys: an RMS norm of every head) - or, with norm_first, preceded by it; keys of `head_dim` and values of another
//    size `value_dim` go to the paged K / V^T arrays (kv_layout.h).
//  * kva_latent_encode_cache: a low-rank key/value entry.  Per token one latent vector of `rank`
//    elements, RMS-normed with a weight, and one rotated key part of `rot` elements shared by all
//    heads are stored side by side in a row of `rank + rot`; the rotated part of every query head
//    is written behind that head's `rank` columns of the query buffer the attention kernel reads.
//  * kva_maps_encode_cache: heads of several maps (differential attention): every map of a head is an
//    attention of its own over the head's values.  kva_maps_combine: what becomes of the maps' outputs.
//
// cos and sin come from fp32 tables [positions, rot / 2]; all arithmetic is fp32.
#include "common.h"
#include "kv_layout.h"
#include <math.h>

#define ENC_MAX_HEAD_DIM 512

template <typename T>
__global__ void __launch_bounds__(256)
qk_encode_cache_kernel(T *__restrict__ qkv, int row_stride, int k_off, int v_off, T *__restrict__ k_cache,
                       T *__restrict__ v_cache, const float *__restrict__ cos_table,
                       const float *__restrict__ sin_table, const int *__restrict__ positions,
                       const int *__restrict__ slot_mapping, int num_q_heads, int num_kv_heads, int head_dim,
                       int value_dim, int rot, int interleaved, float unit_eps, int page_size,
                       const T *__restrict__ bias, const float *__restrict__ q_weight,
                       const float *__restrict__ k_weight, int norm_first) {
    const int t = blockIdx.x;
    const int lane = threadIdx.x % KVA_WAVE, wave = threadIdx.x / KVA_WAVE, waves = blockDim.x / KVA_WAVE;
    T *row = qkv + (size_t)t * row_stride;
    const int pos = positions[t];
    const int half = rot / 2, pairs = head_dim / 2;
    const float *cs = cos_table + (size_t)pos * half, *sn = sin_table + (size_t)pos * half;
    const int slot = slot_mapping ? slot_mapping[t] : -1;
    const int page = slot >= 0 ? slot / page_size : 0, off = slot >= 0 ? slot % page_size : 0;
    constexpr int PER = ENC_MAX_HEAD_DIM / 2 / KVA_WAVE;

    for (int head = wave; head < num_q_heads + num_kv_heads; head += waves) {
        const bool is_q = head < num_q_heads;
        if (!is_q && slot < 0) continue;
        T *h = is_q ? row + (size_t)head * head_dim : row + k_off + (size_t)(head - num_q_heads) * head_dim;
        // (optional) the projection's bias, laid out [q heads | k heads | v heads] without gaps
        const T *hb = bias ? bias + (size_t)head * head_dim : nullptr;
        float o1[PER], o2[PER];
        int i1[PER], i2[PER];
        float sq = 0.f;
#pragma unroll
        for (int c = 0; c < PER; ++c) {
            const int p = lane + c * KVA_WAVE;
            o1[c] = o2[c] = 0.f;
            i1[c] = i2[c] = 0;
            if (p >= pairs) continue;
            // pair p of the head: a rotated pair while p < rot / 2, two plain neighbours behind
            if (interleaved) {
                i1[c] = 2 * p;
                i2[c] = 2 * p + 1;
            } else if (p < half) {
                i1[c] = p;
                i2[c] = p + half;
            } else {
                i1[c] = rot + 2 * (p - half);
                i2[c] = i1[c] + 1;
            }
            const float u = to_float(h[i1[c]]) + (hb ? to_float(hb[i1[c]]) : 0.f);
            const float v = to_float(h[i2[c]]) + (hb ? to_float(hb[i2[c]]) : 0.f);
            if (p < half && !norm_first) {
                const float co = cs[p], si = sn[p];
                o1[c] = u * co - v * si;
                o2[c] = v * co + u * si;
            } else {
                o1[c] = u;
                o2[c] = v;
            }
            sq += o1[c] * o1[c] + o2[c] * o2[c];
        }
        float mul = 1.f;
        if (unit_eps >= 0.f) mul = 1.0f / sqrtf(wave_sum(sq) / (float)head_dim + unit_eps);
        // (optional) the weight of an RMS norm over the head, one per element, shared by the heads
        const float *nw = is_q ? q_weight : k_weight;
        T *kdst = nullptr;
        const int kc = kva_k_chunk(head_dim);
        if (!is_q) kdst = k_cache + ((size_t)page * num_kv_heads + (head - num_q_heads)) * page_size * head_dim;
#pragma unroll
        for (int c = 0; c < PER; ++c) {
            const int p = lane + c * KVA_WAVE;
            if (p >= pairs) continue;
            float f1 = o1[c] * mul * (nw ? nw[i1[c]] : 1.f), f2 = o2[c] * mul * (nw ? nw[i2[c]] : 1.f);
            if (norm_first && p < half) {           // the normed head is what is rotated
                const float co = cs[p], si = sn[p], u = f1, v = f2;
                f1 = u * co - v * si;
                f2 = v * co + u * si;
            }
            const T r1 = from_float<T>(f1), r2 = from_float<T>(f2);
            if (is_q) {
                h[i1[c]] = r1;
                h[i2[c]] = r2;
            } else {
                kdst[kva_k_at(off, i1[c], page_size, kc)] = r1;
                kdst[kva_k_at(off, i2[c], page_size, kc)] = r2;
            }
        }
    }
    if (slot >= 0) {
        const T *v = row + v_off;
        const T *vb = bias ? bias + (size_t)(num_q_heads + num_kv_heads) * head_dim : nullptr;
        for (int w = threadIdx.x; w < num_kv_heads * value_dim; w += blockDim.x) {
            const int kvh = w / value_dim, j = w % value_dim;
            v_cache[(((size_t)page * num_kv_heads + kvh) * value_dim + j) * page_size + off] =
                vb ? from_float<T>(to_float(v[w]) + to_float(vb[w])) : v[w];
        }
    }
}

// bf16, interleaved pairs, heads of 8 * 2^k elements (up to 512): a lane takes 8 neighbouring
// elements of a head (four whole pairs: 16 bytes in, 16 bytes out - one chunk of the K page), the
// 2^k lanes of a head add their squares up between them.
__global__ void __launch_bounds__(256)
qk_encode_cache_vec_kernel(bf16_t *__restrict__ qkv, int row_stride, int k_off, int v_off, bf16_t *__restrict__ k_cache,
                           bf16_t *__restrict__ v_cache, const float *__restrict__ cos_table,
                           const float *__restrict__ sin_table, const int *__restrict__ positions,
                           const int *__restrict__ slot_mapping, int num_q_heads, int num_kv_heads, int head_dim,
                           int value_dim, int rot, float unit_eps, int page_size) {
    const int t = blockIdx.x;
    bf16_t *row = qkv + (size_t)t * row_stride;
    const int pos = positions[t];
    const int half = rot / 2, vecs = head_dim / 8;                // lanes a head
    const float *cs = cos_table + (size_t)pos * half, *sn = sin_table + (size_t)pos * half;
    const int slot = slot_mapping ? slot_mapping[t] : -1;
    const int page = slot >= 0 ? slot / page_size : 0, off = slot >= 0 ? slot % page_size : 0;
    const int total = (num_q_heads + num_kv_heads) * vecs;
    for (int w0 = 0; w0 < total; w0 += blockDim.x) {              // (uniform trip count: the lanes of a head shuffle)
        const int w = w0 + threadIdx.x;
        const bool on = w < total;
        const int head = on ? w / vecs : 0, j = on ? w % vecs : 0;
        const bool is_q = head < num_q_heads;
        bf16_t *h = is_q ? row + (size_t)head * head_dim : row + k_off + (size_t)(head - num_q_heads) * head_dim;
        float x[8], y[8];
        const uint4 in = *reinterpret_cast<const uint4 *>(h + 8 * j);
        const uint32_t iw[4] = {in.x, in.y, in.z, in.w};
        float sq = 0.f;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            x[2 * i] = bf16_bits_to_float((uint16_t)(iw[i] & 0xffffu));
            x[2 * i + 1] = bf16_bits_to_float((uint16_t)(iw[i] >> 16));
            const int p = 4 * j + i;                              // pair (2p, 2p + 1) of the head
            if (p < half) {
                const float co = cs[p], si = sn[p];
                y[2 * i] = x[2 * i] * co - x[2 * i + 1] * si;
                y[2 * i + 1] = x[2 * i + 1] * co + x[2 * i] * si;
            } else {
                y[2 * i] = x[2 * i];
                y[2 * i + 1] = x[2 * i + 1];
            }
            sq += y[2 * i] * y[2 * i] + y[2 * i + 1] * y[2 * i + 1];
        }
        float mul = 1.f;
        if (unit_eps >= 0.f) {
            for (int o = vecs / 2; o > 0; o >>= 1) sq += __shfl_xor(sq, o, KVA_WAVE);
            mul = 1.0f / sqrtf(sq / (float)head_dim + unit_eps);
        }
        uint32_t ow[4];
#pragma unroll
        for (int i = 0; i < 4; ++i)
            ow[i] = (uint32_t)float_to_bf16_bits(y[2 * i] * mul) | ((uint32_t)float_to_bf16_bits(y[2 * i + 1] * mul) << 16);
        const uint4 res = make_uint4(ow[0], ow[1], ow[2], ow[3]);
        if (!on) continue;
        if (is_q) {
            *reinterpret_cast<uint4 *>(h + 8 * j) = res;
        } else if (slot >= 0) {
            bf16_t *kdst = k_cache + ((size_t)page * num_kv_heads + (head - num_q_heads)) * page_size * head_dim;
            *reinterpret_cast<uint4 *>(kdst + kva_k_at(off, 8 * j, page_size, 8)) = res;
        }
    }
    if (slot >= 0) {
        const bf16_t *v = row + v_off;
        for (int w = threadIdx.x; w < num_kv_heads * value_dim; w += blockDim.x) {
            const int kvh = w / value_dim, j = w % value_dim;
            v_cache[(((size_t)page * num_kv_heads + kvh) * value_dim + j) * page_size + off] = v[w];
        }
    }
}

extern "C" int kva_qk_encode_cache(void *qkv, int row_stride, int k_off, int v_off, void *k_cache, void *v_cache,
                                   const float *cos_table, const float *sin_table, const int *positions,
                                   const int *slot_mapping, int tokens, int num_q_heads, int num_kv_heads,
                                   int head_dim, int value_dim, int rot, int interleaved, float unit_eps,
                                   int page_size, int dtype, const void *bias, const float *q_weight,
                                   const float *k_weight, int norm_first, hipStream_t stream) {
    // norm_first: the division by the root mean square (and the weight) comes before the rotation
    KVA_REQUIRE(!norm_first || unit_eps >= 0.f, "qk_encode_cache: a norm before the rotation needs the norm");
    // (num_kv_heads = 0: rows of queries alone, for a layer that reads another layer's keys and values)
    KVA_REQUIRE(tokens >= 0 && num_q_heads > 0 && num_kv_heads >= 0 && value_dim > 0, "qk_encode_cache: bad sizes");
    KVA_REQUIRE(num_kv_heads > 0 || !slot_mapping, "qk_encode_cache: a cache write without key heads");
    KVA_REQUIRE((!q_weight && !k_weight) || unit_eps >= 0.f, "qk_encode_cache: a norm weight without the norm");
    KVA_REQUIRE(head_dim > 0 && head_dim % 2 == 0 && head_dim <= ENC_MAX_HEAD_DIM,
                "qk_encode_cache: head_dim %d must be even and at most %d", head_dim, ENC_MAX_HEAD_DIM);
    KVA_REQUIRE(rot >= 0 && rot <= head_dim && rot % 2 == 0,
                "qk_encode_cache: %d rotated elements must be even and at most head_dim %d", rot, head_dim);
    KVA_REQUIRE(rot == 0 || (cos_table && sin_table), "qk_encode_cache: a rotation needs both tables");
    KVA_REQUIRE(!slot_mapping || (k_cache && v_cache && page_size > 0),
                "qk_encode_cache: cache write asked for without cache or page size");
    KVA_REQUIRE(k_off >= num_q_heads * head_dim && v_off >= k_off + num_kv_heads * head_dim &&
                    row_stride >= v_off + num_kv_heads * value_dim,
                "qk_encode_cache: the row layout [q | k | v] does not fit its stride");
    if (tokens == 0) return KVA_OK;
    if (rot == 0) cos_table = sin_table = reinterpret_cast<const float *>(qkv);     // never read
    const int vecs = head_dim / 8;
    if (!bias && !q_weight && !k_weight && !norm_first && dtype == KVA_BF16 && interleaved && head_dim % 8 == 0 && (vecs & (vecs - 1)) == 0 && vecs <= KVA_WAVE &&
        row_stride % 8 == 0 && k_off % 8 == 0 && (reinterpret_cast<uintptr_t>(qkv) & 15) == 0) {
        hipLaunchKernelGGL(qk_encode_cache_vec_kernel, dim3(tokens), dim3(256), 0, stream, (bf16_t *)qkv, row_stride,
                           k_off, v_off, (bf16_t *)k_cache, (bf16_t *)v_cache, cos_table, sin_table, positions,
                           slot_mapping, num_q_heads, num_kv_heads, head_dim, value_dim, rot, unit_eps, page_size);
        KVA_CHECK_LAUNCH("qk_encode_cache");
        return KVA_OK;
    }
    if (dtype == KVA_F32)
        hipLaunchKernelGGL(qk_encode_cache_kernel<float>, dim3(tokens), dim3(256), 0, stream, (float *)qkv, row_stride,
                           k_off, v_off, (float *)k_cache, (float *)v_cache, cos_table, sin_table, positions,
                           slot_mapping, num_q_heads, num_kv_heads, head_dim, value_dim, rot, interleaved, unit_eps,
                           page_size, (const float *)bias, q_weight, k_weight, norm_first);
    else if (dtype == KVA_BF16)
        hipLaunchKernelGGL(qk_encode_cache_kernel<bf16_t>, dim3(tokens), dim3(256), 0, stream, (bf16_t *)qkv,
                           row_stride, k_off, v_off, (bf16_t *)k_cache, (bf16_t *)v_cache, cos_table, sin_table,
                           positions, slot_mapping, num_q_heads, num_kv_heads, head_dim, value_dim, rot, interleaved,
                           unit_eps, page_size, (const bf16_t *)bias, q_weight, k_weight, norm_first);
    else KVA_REQUIRE(false, "qk_encode_cache: unsupported dtype %d", dtype);
    KVA_CHECK_LAUNCH("qk_encode_cache");
    return KVA_OK;
}

// rotates pair i of `rot` elements at src into dst (which may be src); cs / sn: this position's row
template <typename T>
__device__ inline void rotate_pair(const T *src, T *dst, int i, int rot, int interleaved, const float *cs,
                                   const float *sn) {
    const int a = interleaved ? 2 * i : i, b = interleaved ? 2 * i + 1 : i + rot / 2;
    const float u = to_float(src[a]), v = to_float(src[b]);
    const float co = cs[i], si = sn[i];
    dst[a] = from_float<T>(u * co - v * si);
    dst[b] = from_float<T>(v * co + u * si);
}

// y row: [H heads of (plain_dim + rot) | ... ] with the compressed entry (rank + rot) at kv_off; or, for
// queries that come from a latent of their own (q_rank > 0, heads = 0), [q_rank query latent | ... ]: the
// first q_rank elements, RMS-normed with q_weight, go to c_q [T, q_rank].
template <typename T, typename TW>
__global__ void __launch_bounds__(256)
latent_encode_cache_kernel(const T *__restrict__ y, int row_stride, int kv_off, T *__restrict__ q_lat,
                           T *__restrict__ c_q, const TW *__restrict__ q_weight, int q_rank, T *__restrict__ cache,
                           const TW *__restrict__ norm_weight, float eps,
                           const float *__restrict__ cos_table, const float *__restrict__ sin_table,
                           const int *__restrict__ positions, const int *__restrict__ slot_mapping, int heads,
                           int plain_dim, int rank, int rot, int interleaved) {
    __shared__ float red_s[4];
    const int t = blockIdx.x;
    const T *row = y + (size_t)t * row_stride;
    const int pos = positions[t], half = rot / 2, kd = rank + rot;
    const float *cs = cos_table + (size_t)pos * half, *sn = sin_table + (size_t)pos * half;
    // two workgroups a token: one for the queries, one for the entry
    if (blockIdx.y == 0) {
        // the rotated part of every query head, behind the head's `rank` absorbed columns
        for (int w = threadIdx.x; w < heads * half; w += blockDim.x) {
            const int h = w / half, i = w % half;
            rotate_pair(row + (size_t)h * (plain_dim + rot) + plain_dim, q_lat + ((size_t)t * heads + h) * kd + rank, i, rot,
                        interleaved, cs, sn);
        }
        if (q_rank > 0) {
            float qs = 0.f;
            for (int j = threadIdx.x; j < q_rank; j += blockDim.x) {
                const float v = to_float(row[j]);
                qs += v * v;
            }
            const float qi = 1.0f / sqrtf(block_sum(qs, red_s, blockDim.x / KVA_WAVE) / (float)q_rank + eps);
            for (int j = threadIdx.x; j < q_rank; j += blockDim.x)
                c_q[(size_t)t * q_rank + j] = from_float<T>(to_float(row[j]) * qi * to_float(q_weight[j]));
        }
        return;
    }
    const int slot = slot_mapping ? slot_mapping[t] : -1;       // uniform over the workgroup
    if (slot < 0) return;
    const T *c = row + kv_off;
    T *dst = cache + (size_t)slot * kd;
    float sq = 0.f;
    for (int j = threadIdx.x; j < rank; j += blockDim.x) {
        const float v = to_float(c[j]);
        sq += v * v;
    }
    const float inv = 1.0f / sqrtf(block_sum(sq, red_s, blockDim.x / KVA_WAVE) / (float)rank + eps);
    for (int j = threadIdx.x; j < rank; j += blockDim.x) dst[j] = from_float<T>(to_float(c[j]) * inv * to_float(norm_weight[j]));
    for (int i = threadIdx.x; i < half; i += blockDim.x) rotate_pair(c + rank, dst + rank, i, rot, interleaved, cs, sn);
}

extern "C" int kva_latent_encode_cache(const void *y, int row_stride, int kv_off, void *q_lat, void *c_q,
                                       const void *q_weight, int q_rank, void *cache,
                                       const void *norm_weight, int weight_dtype, float eps, const float *cos_table,
                                       const float *sin_table, const int *positions, const int *slot_mapping,
                                       int tokens, int heads, int plain_dim, int rank, int rot, int interleaved,
                                       int dtype, hipStream_t stream) {
    KVA_REQUIRE(tokens >= 0 && heads >= 0 && plain_dim > 0 && rank > 0, "latent_encode_cache: bad sizes");
    KVA_REQUIRE(heads > 0 ? (q_lat && q_rank == 0) : (c_q && q_weight && q_rank > 0),
                "latent_encode_cache: rows start with the query heads or with a query latent");
    KVA_REQUIRE(rot > 0 && rot % 2 == 0 && cos_table && sin_table,
                "latent_encode_cache: %d rotated elements must be even and positive, with both tables", rot);
    KVA_REQUIRE(kv_off >= heads * (plain_dim + rot) && kv_off >= q_rank && row_stride >= kv_off + rank + rot,
                "latent_encode_cache: the row layout [queries | entry] does not fit its stride");
    KVA_REQUIRE(!slot_mapping || cache, "latent_encode_cache: cache write asked for without a cache");
    KVA_REQUIRE(dtype == KVA_F32 || dtype == KVA_BF16, "latent_encode_cache: unsupported dtype %d", dtype);
    if (tokens == 0) return KVA_OK;
#define LAUNCH_LE(T, TW)                                                                                        \
    hipLaunchKernelGGL((latent_encode_cache_kernel<T, TW>), dim3(tokens, slot_mapping ? 2 : 1), dim3(256), 0,   \
                       stream, (const T *)y, row_stride, kv_off, (T *)q_lat, (T *)c_q, (const TW *)q_weight,    \
                       q_rank, (T *)cache, (const TW *)norm_weight, eps, cos_table, sin_table,                  \
                       positions, slot_mapping, heads, plain_dim, rank, rot, interleaved)
    if (dtype == KVA_F32 && weight_dtype == KVA_F32) LAUNCH_LE(float, float);
    else if (dtype == KVA_BF16 && weight_dtype == KVA_BF16) LAUNCH_LE(bf16_t, bf16_t);
    else if (dtype == KVA_BF16 && weight_dtype == KVA_F32) LAUNCH_LE(bf16_t, float);
    else KVA_REQUIRE(false, "latent_encode_cache: a 32-bit entry needs a 32-bit norm weight");
#undef LAUNCH_LE
    KVA_CHECK_LAUNCH("latent_encode_cache");
    return KVA_OK;
}

// ---- heads of two maps ------------------------------------------------------------------------------------
// A query head has two maps of `dim` elements each, [map 1 | map 2], and so has a key head; map m of a query
// head meets map m of its key head, and both weigh the same values.  For the attention kernels a key head is
// one key of 2 dim elements as it lies in memory, and a query head becomes two rows of 2 dim elements with the
// other map's half zero: their scores are the two maps' scores, key and value heads are read once for both, and
// a head's two outputs lie side by side.  This kernel adds the projection's biases (fp32, [q | k | v]), rotates
// the first `rot` elements of every map, writes the query rows [T, 2 heads, 2 dim] and the cache.
// A thread takes a rotated or plain pair of elements of one map.
template <typename T>
__global__ void __launch_bounds__(256)
maps_encode_cache_kernel(const T *__restrict__ qkv, int row_stride, T *__restrict__ q_rows, T *__restrict__ k_cache,
                         T *__restrict__ v_cache, const float *__restrict__ cos_table,
                         const float *__restrict__ sin_table, const int *__restrict__ positions,
                         const int *__restrict__ slot_mapping, int heads, int kv_heads, int dim, int value_dim, int rot,
                         int interleaved, int page_size, const float *__restrict__ bias) {
    const int t = blockIdx.x;
    const T *row = qkv + (size_t)t * row_stride;
    const int pos = positions[t], half = rot / 2;
    const float *cs = cos_table + (size_t)pos * half, *sn = sin_table + (size_t)pos * half;
    const int slot = slot_mapping ? slot_mapping[t] : -1;
    const int page = slot >= 0 ? slot / page_size : 0, off = slot >= 0 ? slot % page_size : 0;
    const int per = (dim + 1) / 2, maps = 2 * heads + (slot >= 0 ? 2 * kv_heads : 0), kc = kva_k_chunk(2 * dim);
    for (int w = threadIdx.x; w < maps * per; w += blockDim.x) {
        const int m = w / per, p = w % per;         // map (of the queries', then of the keys'), pair of it
        int i1, i2;
        if (interleaved) {
            i1 = 2 * p;
            i2 = 2 * p + 1;
        } else if (p < half) {
            i1 = p;
            i2 = p + half;
        } else {
            i1 = rot + 2 * (p - half);
            i2 = i1 + 1;
        }
        const bool two = i2 < dim;                  // (an odd size leaves one element alone)
        const size_t at = (size_t)m * dim;
        float u = to_float(row[at + i1]) + (bias ? bias[at + i1] : 0.f);
        float v = two ? to_float(row[at + i2]) + (bias ? bias[at + i2] : 0.f) : 0.f;
        if (p < half) {
            const float co = cs[p], si = sn[p], a = u;
            u = a * co - v * si;
            v = v * co + a * si;
        }
        const T r1 = from_float<T>(u), r2 = from_float<T>(v), zero = from_float<T>(0.f);
        if (m < 2 * heads) {
            T *own = q_rows + ((size_t)t * 2 * heads + m) * 2 * dim + (m & 1) * dim, *other = own + ((m & 1) ? -dim : dim);
            own[i1] = r1;
            other[i1] = zero;
            if (two) {
                own[i2] = r2;
                other[i2] = zero;
            }
        } else {
            const int k = m - 2 * heads;
            T *dst = k_cache + ((size_t)page * kv_heads + k / 2) * page_size * 2 * dim;
            dst[kva_k_at(off, (k & 1) * dim + i1, page_size, kc)] = r1;
            if (two) dst[kva_k_at(off, (k & 1) * dim + i2, page_size, kc)] = r2;
        }
    }
    if (slot >= 0) {
        const int v_off = 2 * (heads + kv_heads) * dim;
        for (int w = threadIdx.x; w < kv_heads * value_dim; w += blockDim.x)
            v_cache[((size_t)page * kv_heads * value_dim + w) * page_size + off] =
                from_float<T>(to_float(row[v_off + w]) + (bias ? bias[v_off + w] : 0.f));
    }
}

// bf16, interleaved pairs, maps of a multiple of 8 elements: a thread takes 8 neighbouring elements
__global__ void __launch_bounds__(256)
maps_encode_cache_vec_kernel(const bf16_t *__restrict__ qkv, int row_stride, bf16_t *__restrict__ q_rows,
                             bf16_t *__restrict__ k_cache, bf16_t *__restrict__ v_cache,
                             const float *__restrict__ cos_table, const float *__restrict__ sin_table,
                             const int *__restrict__ positions, const int *__restrict__ slot_mapping, int heads,
                             int kv_heads, int dim, int value_dim, int rot, int page_size, const float *__restrict__ bias) {
    const int t = blockIdx.x;
    const bf16_t *row = qkv + (size_t)t * row_stride;
    const int pos = positions[t], half = rot / 2;
    const float *cs = cos_table + (size_t)pos * half, *sn = sin_table + (size_t)pos * half;
    const int slot = slot_mapping ? slot_mapping[t] : -1;
    const int page = slot >= 0 ? slot / page_size : 0, off = slot >= 0 ? slot % page_size : 0;
    const int vecs = dim / 8, maps = 2 * heads + (slot >= 0 ? 2 * kv_heads : 0);
    for (int w = threadIdx.x; w < maps * vecs; w += blockDim.x) {
        const int m = w / vecs, j = w % vecs;
        const int at = m * dim + 8 * j;
        const uint4 in = *reinterpret_cast<const uint4 *>(row + at);
        const uint32_t iw[4] = {in.x, in.y, in.z, in.w};
        float b[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) b[i] = 0.f;
        if (bias) {
            *reinterpret_cast<float4 *>(b) = *reinterpret_cast<const float4 *>(bias + at);
            *reinterpret_cast<float4 *>(b + 4) = *reinterpret_cast<const float4 *>(bias + at + 4);
        }
        uint32_t ow[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            float u = bf16_bits_to_float((uint16_t)(iw[i] & 0xffffu)) + b[2 * i];
            float v = bf16_bits_to_float((uint16_t)(iw[i] >> 16)) + b[2 * i + 1];
            const int p = 4 * j + i;
            if (p < half) {
                const float co = cs[p], si = sn[p], a = u;
                u = a * co - v * si;
                v = v * co + a * si;
            }
            ow[i] = (uint32_t)float_to_bf16_bits(u) | ((uint32_t)float_to_bf16_bits(v) << 16);
        }
        const uint4 res = make_uint4(ow[0], ow[1], ow[2], ow[3]);
        if (m < 2 * heads) {
            bf16_t *q = q_rows + ((size_t)t * 2 * heads + m) * 2 * dim + 8 * j;
            *reinterpret_cast<uint4 *>(q + (m & 1) * dim) = res;
            *reinterpret_cast<uint4 *>(q + (1 - (m & 1)) * dim) = make_uint4(0u, 0u, 0u, 0u);
        } else {
            const int k = m - 2 * heads;
            bf16_t *dst = k_cache + ((size_t)page * kv_heads + k / 2) * page_size * 2 * dim;
            *reinterpret_cast<uint4 *>(dst + kva_k_at(off, (k & 1) * dim + 8 * j, page_size, 8)) = res;
        }
    }
    if (slot >= 0) {
        const int v_off = 2 * (heads + kv_heads) * dim;
        for (int w = threadIdx.x; w < kv_heads * value_dim; w += blockDim.x)
            v_cache[((size_t)page * kv_heads * value_dim + w) * page_size + off] =
                bias ? from_float<bf16_t>(to_float(row[v_off + w]) + bias[v_off + w]) : row[v_off + w];
    }
}

extern "C" int kva_maps_encode_cache(const void *qkv, int row_stride, void *q_rows, void *k_cache, void *v_cache,
                                     const float *cos_table, const float *sin_table, const int *positions,
                                     const int *slot_mapping, int tokens, int heads, int kv_heads, int dim, int value_dim,
                                     int rot, int interleaved, int page_size, const float *bias, int dtype,
                                     hipStream_t stream) {
    // (kv_heads = 0: rows of queries alone, for a layer that reads another layer's keys and values)
    KVA_REQUIRE(qkv && q_rows && positions && tokens >= 0 && heads > 0 && kv_heads >= 0 && dim > 0 && value_dim > 0,
                "maps_encode_cache: missing operand or bad sizes");
    KVA_REQUIRE(dim % 2 == 0, "maps_encode_cache: maps of %d elements (keys of two maps lie in the cache in chunks of 4 or 8)", dim);
    KVA_REQUIRE(kv_heads > 0 || !slot_mapping, "maps_encode_cache: a cache write without key heads");
    KVA_REQUIRE(rot >= 0 && rot <= dim && rot % 2 == 0, "maps_encode_cache: %d rotated elements must be even and at most %d", rot, dim);
    KVA_REQUIRE(rot == 0 || (cos_table && sin_table), "maps_encode_cache: a rotation needs both tables");
    KVA_REQUIRE(!slot_mapping || (k_cache && v_cache && page_size > 0), "maps_encode_cache: a cache write without cache or page size");
    KVA_REQUIRE(row_stride >= 2 * (heads + kv_heads) * dim + kv_heads * value_dim,
                "maps_encode_cache: the row layout [q | k | v] does not fit its stride");
    KVA_REQUIRE(dtype == KVA_F32 || dtype == KVA_BF16, "maps_encode_cache: unsupported dtype %d", dtype);
    if (tokens == 0) return KVA_OK;
    if (rot == 0) cos_table = sin_table = reinterpret_cast<const float *>(qkv);     // never read
    if (dtype == KVA_BF16 && interleaved && dim % 8 == 0 && row_stride % 8 == 0 &&
        ((reinterpret_cast<uintptr_t>(qkv) | reinterpret_cast<uintptr_t>(q_rows) | reinterpret_cast<uintptr_t>(bias)) & 15) == 0)
        hipLaunchKernelGGL(maps_encode_cache_vec_kernel, dim3(tokens), dim3(256), 0, stream, (const bf16_t *)qkv, row_stride,
                           (bf16_t *)q_rows, (bf16_t *)k_cache, (bf16_t *)v_cache, cos_table, sin_table, positions,
                           slot_mapping, heads, kv_heads, dim, value_dim, rot, page_size, bias);
    else if (dtype == KVA_F32)
        hipLaunchKernelGGL(maps_encode_cache_kernel<float>, dim3(tokens), dim3(256), 0, stream, (const float *)qkv, row_stride,
                           (float *)q_rows, (float *)k_cache, (float *)v_cache, cos_table, sin_table, positions,
                           slot_mapping, heads, kv_heads, dim, value_dim, rot, interleaved, page_size, bias);
    else
        hipLaunchKernelGGL(maps_encode_cache_kernel<bf16_t>, dim3(tokens), dim3(256), 0, stream, (const bf16_t *)qkv, row_stride,
                           (bf16_t *)q_rows, (bf16_t *)k_cache, (bf16_t *)v_cache, cos_table, sin_table, positions,
                           slot_mapping, heads, kv_heads, dim, value_dim, rot, interleaved, page_size, bias);
    KVA_CHECK_LAUNCH("maps_encode_cache");
    return KVA_OK;
}

// o = a1 - lambda a2 per head, o / sqrt(mean(o^2) + eps) * mul, from the maps' outputs x [T, heads, 2, dv] into
// columns out_off .. of out.  `lanes` (a power of two up to 64) lanes take a head, 8 neighbouring elements a
// lane at a time (VEC: bf16, dv a multiple of 8), else one.
template <typename T, bool VEC>
__global__ void __launch_bounds__(256)
maps_combine_kernel(T *__restrict__ out, int out_stride, int out_off, const T *__restrict__ x, float lambda, float eps,
                    float mul, int rows, int heads, int dv, int lanes) {
    constexpr int W = VEC ? 8 : 1, KEEP = 4;
    const int lane = threadIdx.x % lanes;
    const int unit = (blockIdx.x * blockDim.x + threadIdx.x) / lanes;      // (token, head); idle lanes repeat the last one
    const bool live = unit < rows * heads;
    const int u = live ? unit : rows * heads - 1;
    const T *a1 = x + (size_t)u * 2 * dv, *a2 = a1 + dv;
    auto load = [&](int j, float (&f)[W]) {
        if constexpr (VEC) {
            const uint4 p = *reinterpret_cast<const uint4 *>(a1 + j), q = *reinterpret_cast<const uint4 *>(a2 + j);
            const uint32_t pw[4] = {p.x, p.y, p.z, p.w}, qw[4] = {q.x, q.y, q.z, q.w};
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                f[2 * i] = __uint_as_float(pw[i] << 16) - lambda * __uint_as_float(qw[i] << 16);
                f[2 * i + 1] = __uint_as_float(pw[i] & 0xffff0000u) - lambda * __uint_as_float(qw[i] & 0xffff0000u);
            }
        } else {
            f[0] = to_float(a1[j]) - lambda * to_float(a2[j]);
        }
    };
    float kept[KEEP][W], sq = 0.f;
    const int step = W * lanes;
#pragma unroll
    for (int k = 0; k < KEEP; ++k) {
        const int j = W * lane + k * step;
        if (j < dv) {
            load(j, kept[k]);
#pragma unroll
            for (int i = 0; i < W; ++i) sq += kept[k][i] * kept[k][i];
        }
    }
    for (int j = W * lane + KEEP * step; j < dv; j += step) {
        float f[W];
        load(j, f);
#pragma unroll
        for (int i = 0; i < W; ++i) sq += f[i] * f[i];
    }
    for (int o = lanes / 2; o > 0; o >>= 1) sq += __shfl_xor(sq, o, KVA_WAVE);
    if (!live) return;
    const float by = mul / sqrtf(sq / (float)dv + eps);
    T *dst = out + (size_t)(u / heads) * out_stride + out_off + (size_t)(u % heads) * dv;
    auto store = [&](int j, const float (&f)[W]) {
        if constexpr (VEC) {
            uint32_t w[4];
#pragma unroll
            for (int i = 0; i < 4; ++i)
                w[i] = (uint32_t)float_to_bf16_bits(f[2 * i] * by) | ((uint32_t)float_to_bf16_bits(f[2 * i + 1] * by) << 16);
            *reinterpret_cast<uint4 *>(dst + j) = make_uint4(w[0], w[1], w[2], w[3]);
        } else {
            dst[j] = from_float<T>(f[0] * by);
        }
    };
#pragma unroll
    for (int k = 0; k < KEEP; ++k) {
        const int j = W * lane + k * step;
        if (j < dv) store(j, kept[k]);
    }
    for (int j = W * lane + KEEP * step; j < dv; j += step) {
        float f[W];
        load(j, f);
        store(j, f);
    }
}

extern "C" int kva_maps_combine(void *out, int out_stride, int out_off, const void *x, float lambda, float eps, float mul,
                                int rows, int heads, int dv, int dtype, hipStream_t stream) {
    KVA_REQUIRE(out && x && rows >= 0 && heads > 0 && dv > 0 && eps >= 0.f, "maps_combine: missing operand or bad sizes");
    KVA_REQUIRE(out_off >= 0 && out_stride >= out_off + heads * dv, "maps_combine: the heads do not fit the output's rows");
    KVA_REQUIRE(dtype == KVA_F32 || dtype == KVA_BF16, "maps_combine: unsupported dtype %d", dtype);
    if (rows == 0) return KVA_OK;
    const bool vec = dtype == KVA_BF16 && dv % 8 == 0 && out_stride % 8 == 0 && out_off % 8 == 0 &&
                     ((reinterpret_cast<uintptr_t>(out) | reinterpret_cast<uintptr_t>(x)) & 15) == 0;
    const int need = vec ? dv / 8 : dv;
    int lanes = 1;
    while (lanes < need && lanes < KVA_WAVE) lanes *= 2;
    const long long threads = (long long)rows * heads * lanes;
    KVA_REQUIRE(threads + 255 < (1LL << 31), "maps_combine: too many rows");
    const dim3 grid((unsigned)((threads + 255) / 256));
    if (vec)
        hipLaunchKernelGGL((maps_combine_kernel<bf16_t, true>), grid, dim3(256), 0, stream, (bf16_t *)out, out_stride, out_off,
                           (const bf16_t *)x, lambda, eps, mul, rows, heads, dv, lanes);
    else if (dtype == KVA_BF16)
        hipLaunchKernelGGL((maps_combine_kernel<bf16_t, false>), grid, dim3(256), 0, stream, (bf16_t *)out, out_stride, out_off,
                           (const bf16_t *)x, lambda, eps, mul, rows, heads, dv, lanes);
    else
        hipLaunchKernelGGL((maps_combine_kernel<float, false>), grid, dim3(256), 0, stream, (float *)out, out_stride, out_off,
                           (const float *)x, lambda, eps, mul, rows, heads, dv, lanes);
    KVA_CHECK_LAUNCH("maps_combine");
    return KVA_OK;
}
