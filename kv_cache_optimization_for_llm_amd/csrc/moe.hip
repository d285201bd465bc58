// A routed feed-forward (mixture of experts) whose work stays on the device from the router's
// logits to the weighted sum: no count of tokens per expert ever reaches the host, so the whole
// layer can be captured into a graph.
//
//  * kva_moe_route:  scores = softmax(logits) over all router outputs; the `top` largest of
//    scores + correction are chosen; their weights are the plain scores (optionally renormalised).
//    Or (`over_chosen`) the largest logits are chosen and the weights are the softmax over them alone.
//  * kva_moe_router: the router's product (bf16 operands), that choice and, for up to 16 tokens, the list below in one launch.
//  * kva_moe_align:  the (token, choice) slots of real experts sorted by expert into a list padded
//    so that every tile of 16 rows belongs to one expert (`sorted_slot`, -1 = padding), with the
//    expert of every tile (`tile_expert`, -1 = unused tile).  Without a router (`table`): the experts of a
//    token are the entries of its id's row in an integer table, all with one weight; the same launch looks
//    them up.
//  * kva_moe_expert_rows: one product per tile against its expert's matrix.  Mode 0 ("up"): rows of
//    x gathered by slot / top, activation applied (a gated expert: act(gate) * up, its gate and up rows
//    interleaved in one matrix), written at the sorted position.  Mode 1 ("down"):
//    rows at the sorted position, times the slot's routing weight, written at the slot (fp32).  The weight may
//    stand on the expert's input instead: it then multiplies the first product's rows, before the activation.
//    bf16 with K % 32 == 0 runs on the matrix cores (with many rows an expert through LDS, in groups of
//    tiles), everything else (fp32 too) on a plain tiled kernel that adds k ascending.
//  * kva_moe_combine: out[t] = sum over the token's choices of the slot's row, or, for a router
//    output past the real experts (an identity expert), weight * x[t].
//
// A row's result depends on that row and its expert's matrix only, never on which other rows
// share its tile: the same token gives the same numbers in any batch.
#include "common.h"
#include "attention_frag.h"
#include "lds_product.h"
#include <math.h>

#define MOE_TILE 16
#define MOE_MAX_EXPERTS 1024
#define MOE_ROUTE_PER_LANE 8

__device__ inline float moe_activate(float z, int act) {
    if (act == 3) return 0.5f * z * (1.0f + erff(z * 0.70710678118654752f));       // exact gelu
    if (act == 5) return kva_activate(z, KVA_ACT_RELU2);
    return kva_activate(z, act);
}

// ---- router ------------------------------------------------------------------------------
struct MoeRoute {
    const float *correction;
    int outputs, top, renormalise, over_chosen, sigmoid_scores, groups, keep_groups, group_top;
    float weight_scale, sum_eps;
};

// one token by one wavefront: `logits` [outputs] (memory or LDS) -> idx and wgt [top]; `choice` is the wavefront's own
// piece of LDS, KVA_WAVE * PL floats (16-byte aligned; with PL > 1 read with groups only).  A lane takes PL outputs.
template <int PL>
__device__ inline void moe_route_token(const MoeRoute &a, const float *logits, int *idx, float *wgt, float *choice) {
    const int lane = threadIdx.x % KVA_WAVE;
    float s[PL], ch[PL];
    float mx = -INFINITY;
#pragma unroll
    for (int j = 0; j < PL; ++j) {
        const int e = lane + j * KVA_WAVE;
        s[j] = e < a.outputs ? logits[e] : -INFINITY;
        mx = fmaxf(mx, s[j]);
    }
    mx = wave_max(mx);
    float sum = 0.f;
#pragma unroll
    for (int j = 0; j < PL; ++j) {
        const int e = lane + j * KVA_WAVE;
        s[j] = e < a.outputs ? expf(s[j] - mx) : 0.f;
        sum += s[j];
    }
    sum = wave_sum(sum);
#pragma unroll
    for (int j = 0; j < PL; ++j) {
        const int e = lane + j * KVA_WAVE;
        if (a.over_chosen) {
            // the logits themselves are compared, and the weights are a softmax over the chosen ones
            // alone: exp(logit - max) here, divided by the chosen ones' sum below
            ch[j] = e < a.outputs ? logits[e] + (a.correction ? a.correction[e] : 0.f) : -INFINITY;
        } else {
            // scores: the softmax over all outputs, or every output's own sigmoid
            s[j] = a.sigmoid_scores ? (e < a.outputs ? 1.f / (1.f + expf(-logits[e])) : 0.f) : s[j] / sum;
            ch[j] = e < a.outputs ? s[j] + (a.correction ? a.correction[e] : 0.f) : -INFINITY;
        }
    }
    if (a.groups > 1) {
        // Outputs form `groups` equal runs of neighbours.  A group's score is the sum of its `group_top`
        // largest choice scores; only outputs of the `keep_groups` best groups (of equal ones the lowest
        // index) can be chosen: the others' choice scores become -inf.  Lane g takes group g.
        const int per = a.outputs / a.groups;
#pragma unroll
        for (int j = 0; j < PL; ++j)
            if (lane + j * KVA_WAVE < a.outputs) choice[lane + j * KVA_WAVE] = ch[j];
        __builtin_amdgcn_wave_barrier();
        __threadfence_block();
        float gs = -INFINITY;
        if (lane < a.groups) {
            gs = 0.f;
            unsigned long long taken = 0ull;            // (a group holds at most 64 outputs when it is scored this way; larger ones below)
            for (int k = 0; k < a.group_top && k < per; ++k) {
                float bv = -INFINITY;
                int bi = -1;
                for (int i = 0; i < per; ++i) {
                    const bool used = i < 64 ? ((taken >> i) & 1ull) != 0ull : false;
                    const float v = choice[lane * per + i];
                    if (!used && (bi < 0 || v > bv)) { bv = v; bi = i; }
                }
                if (bi >= 0 && bi < 64) taken |= 1ull << bi;
                gs += bv;
            }
        }
        unsigned long long allowed = 0ull;
        for (int k = 0; k < a.keep_groups; ++k) {
            float bv = gs;
            int bg = lane < a.groups && !((allowed >> lane) & 1ull) ? lane : 0x7fffffff;
            if (bg == 0x7fffffff) bv = -INFINITY;
#pragma unroll
            for (int off = KVA_WAVE / 2; off > 0; off >>= 1) {
                const float ov = __shfl_xor(bv, off, KVA_WAVE);
                const int og = __shfl_xor(bg, off, KVA_WAVE);
                if (og != 0x7fffffff && (bg == 0x7fffffff || ov > bv || (ov == bv && og < bg))) { bv = ov; bg = og; }
            }
            if (bg != 0x7fffffff) allowed |= 1ull << bg;
        }
#pragma unroll
        for (int j = 0; j < PL; ++j) {
            const int e = lane + j * KVA_WAVE;
            if (e < a.outputs && !((allowed >> (e / per)) & 1ull)) ch[j] = -INFINITY;
        }
    }
    if constexpr (PL == 1) {
        // every lane counts the outputs in front of its own (of equal ones the lowest index comes first)
        __builtin_amdgcn_wave_barrier();
        choice[lane] = ch[0];
        __threadfence_block();
        __builtin_amdgcn_wave_barrier();
        int rank = 0;
        for (int e = 0; e < a.outputs; e += 4) {
            const float4 c = *reinterpret_cast<const float4 *>(choice + e);
            rank += (c.x > ch[0] || (c.x == ch[0] && e < lane)) + (c.y > ch[0] || (c.y == ch[0] && e + 1 < lane)) +
                    (c.z > ch[0] || (c.z == ch[0] && e + 2 < lane)) + (c.w > ch[0] || (c.w == ch[0] && e + 3 < lane));
        }
        const bool chosen = lane < a.outputs && rank < a.top;
        if (chosen) idx[rank] = lane;
        if (!(a.renormalise || a.over_chosen)) {
            if (chosen) wgt[rank] = s[0] * a.weight_scale;
            return;
        }
        __builtin_amdgcn_wave_barrier();
        if (chosen) choice[rank] = s[0];
        __threadfence_block();
        __builtin_amdgcn_wave_barrier();
        float sum_chosen = 0.f;
        for (int k = 0; k < a.top; ++k) sum_chosen += choice[k];
        if (lane < a.top) wgt[lane] = choice[lane] / (sum_chosen + a.sum_eps) * a.weight_scale;
        return;
    }
    float total = 0.f;
    for (int k = 0; k < a.top; ++k) {
        // the largest remaining choice score; of equal ones the lowest index
        float bv = -INFINITY, bs = 0.f;
        int be = 0x7fffffff;
#pragma unroll
        for (int j = 0; j < PL; ++j) {
            const int e = lane + j * KVA_WAVE;
            if (e < a.outputs && (ch[j] > bv || (ch[j] == bv && e < be))) { bv = ch[j]; be = e; bs = s[j]; }
        }
#pragma unroll
        for (int off = KVA_WAVE / 2; off > 0; off >>= 1) {
            const float ov = __shfl_xor(bv, off, KVA_WAVE), os = __shfl_xor(bs, off, KVA_WAVE);
            const int oe = __shfl_xor(be, off, KVA_WAVE);
            if (ov > bv || (ov == bv && oe < be)) { bv = ov; be = oe; bs = os; }
        }
#pragma unroll
        for (int j = 0; j < PL; ++j)
            if (lane + j * KVA_WAVE == be) ch[j] = -INFINITY;
        total += bs;
        if (lane == 0) {
            idx[k] = be;
            wgt[k] = bs;
        }
    }
    if (lane == 0) {
        if (a.renormalise || a.over_chosen)
            for (int k = 0; k < a.top; ++k) wgt[k] = wgt[k] / (total + a.sum_eps) * a.weight_scale;
        else if (a.weight_scale != 1.f)
            for (int k = 0; k < a.top; ++k) wgt[k] *= a.weight_scale;
    }
}

template <int PL>
__global__ void __launch_bounds__(256)
moe_route_kernel(int *__restrict__ idx, float *__restrict__ wgt, const float *__restrict__ logits, MoeRoute a, int tokens,
                 int logits_stride) {
    __shared__ __attribute__((aligned(16))) float choice_s[4][KVA_WAVE * PL];
    const int t = blockIdx.x * (blockDim.x / KVA_WAVE) + threadIdx.x / KVA_WAVE;
    if (t >= tokens) return;
    moe_route_token<PL>(a, logits + (size_t)t * logits_stride, idx + (size_t)t * a.top, wgt + (size_t)t * a.top,
                    choice_s[threadIdx.x / KVA_WAVE]);
}

static int moe_route_check(const MoeRoute &a) {
    KVA_REQUIRE(a.groups >= 1 && a.groups <= KVA_WAVE && a.outputs % a.groups == 0 && a.keep_groups >= 1 &&
                    a.keep_groups <= a.groups && a.group_top >= 1,
                "moe_route: %d groups (at most %d, dividing the %d outputs) of which %d are kept", a.groups, KVA_WAVE, a.outputs,
                a.keep_groups);
    KVA_REQUIRE(a.groups == 1 || (a.outputs / a.groups <= 64 && a.top <= a.keep_groups * (a.outputs / a.groups)),
                "moe_route: groups of at most 64 outputs, and enough outputs in the kept groups for top %d", a.top);
    KVA_REQUIRE(!(a.sigmoid_scores && a.over_chosen), "moe_route: sigmoid scores exclude the softmax over the chosen logits");
    KVA_REQUIRE(a.outputs > 0 && a.outputs <= KVA_WAVE * MOE_ROUTE_PER_LANE, "moe_route: %d router outputs (at most %d)",
                a.outputs, KVA_WAVE * MOE_ROUTE_PER_LANE);
    KVA_REQUIRE(a.top > 0 && a.top <= a.outputs, "moe_route: top %d of %d", a.top, a.outputs);
    return KVA_OK;
}

extern "C" int kva_moe_route(int *idx, float *wgt, const float *logits, const float *correction, int tokens,
                             int outputs, int top, int renormalise, int over_chosen, int sigmoid_scores, int groups,
                             int keep_groups, int group_top, float weight_scale, float sum_eps, int logits_stride,
                             hipStream_t stream) {
    // logits_stride: elements between two tokens' rows of logits (the logits may be the first columns of a wider product)
    KVA_REQUIRE(logits_stride >= outputs, "moe_route: a row of logits holds at least the %d outputs", outputs);
    KVA_REQUIRE(idx && wgt && logits && tokens >= 0, "moe_route: missing operand");
    const MoeRoute a{correction, outputs, top, renormalise, over_chosen, sigmoid_scores, groups, keep_groups, group_top, weight_scale, sum_eps};
    if (int rc = moe_route_check(a)) return rc;
    if (tokens == 0) return KVA_OK;
    hipLaunchKernelGGL(outputs <= KVA_WAVE ? moe_route_kernel<1> : moe_route_kernel<MOE_ROUTE_PER_LANE>, dim3((tokens + 3) / 4), dim3(256), 0, stream, idx, wgt, logits, a, tokens, logits_stride);
    KVA_CHECK_LAUNCH("moe_route");
    return KVA_OK;
}

// ---- slots sorted by expert --------------------------------------------------------------
// experts by token id: idx[t, k] = table[id_t, k] and wgt[t, k] = weight.  A negative id -1 - r stands for
// feedback[r], as in the embedding gather.
struct MoeTable {
    const int *table, *ids, *feedback;
    int rows, top;
    float weight;
    float *wgt;
};

// `group` tiles form a group that belongs to one expert (its last tiles may be padding): what a kernel that
// takes several tiles at once walks over.  One workgroup; a thread keeps up to MOE_SLOTS_IN_REGISTERS slots
// and their places in their experts' runs in registers (all its loads in flight at once, one pass of
// counters); more slots than that are read and counted twice.
#define MOE_SLOTS_IN_REGISTERS 16
__device__ inline int moe_slot_expert(int *idx, int s, const MoeTable &tab) {
    if (!tab.table) return idx[s];
    int id = tab.ids[s / tab.top];
    if (id < 0) id = tab.feedback[-1 - id];
    id = id < 0 ? 0 : (id >= tab.rows ? tab.rows - 1 : id);
    return tab.table[(size_t)id * tab.top + s % tab.top];
}

__device__ inline void moe_align_workgroup(int *sorted_slot, int *tile_expert, int *idx, int slots, int experts, int capacity,
                                           int max_tiles, int group, const MoeTable &tab, int *count, int *start) {
    const bool in_registers = slots <= (int)blockDim.x * MOE_SLOTS_IN_REGISTERS;
    int ex[MOE_SLOTS_IN_REGISTERS], at[MOE_SLOTS_IN_REGISTERS];
#pragma unroll
    for (int j = 0; j < MOE_SLOTS_IN_REGISTERS; ++j) ex[j] = -1;
    if (in_registers) {
#pragma unroll
        for (int j = 0; j < MOE_SLOTS_IN_REGISTERS; ++j) {
            const int s = threadIdx.x + j * blockDim.x;
            if (j * (int)blockDim.x >= slots) break;
            ex[j] = s < slots ? moe_slot_expert(idx, s, tab) : -1;
        }
    }
    for (int e = threadIdx.x; e < experts; e += blockDim.x) count[e] = 0;
    for (int p = threadIdx.x; p < capacity; p += blockDim.x) sorted_slot[p] = -1;
    for (int i = threadIdx.x; i < max_tiles; i += blockDim.x) tile_expert[i] = -1;
    __syncthreads();
    if (in_registers) {
#pragma unroll
        for (int j = 0; j < MOE_SLOTS_IN_REGISTERS; ++j)
            if (ex[j] >= 0 && ex[j] < experts) at[j] = atomicAdd(&count[ex[j]], 1);
    } else {
        for (int s = threadIdx.x; s < slots; s += blockDim.x) {
            const int e = moe_slot_expert(idx, s, tab);
            if (e >= 0 && e < experts) atomicAdd(&count[e], 1);
        }
    }
    __syncthreads();
    if (threadIdx.x == 0) {
        int first = 0;
        for (int e = 0; e < experts; ++e) {
            start[e] = first;
            const int tiles = (count[e] + MOE_TILE - 1) / MOE_TILE;
            first += (tiles + group - 1) / group * group * MOE_TILE;
        }
    }
    __syncthreads();
    for (int e = threadIdx.x; e < experts; e += blockDim.x) {
        const int tiles = (count[e] + MOE_TILE - 1) / MOE_TILE;
        for (int i = 0; i < tiles; ++i) tile_expert[start[e] / MOE_TILE + i] = e;
        count[e] = 0;                   // from here on: the next free place of the expert's run
    }
    if (in_registers) {
#pragma unroll
        for (int j = 0; j < MOE_SLOTS_IN_REGISTERS; ++j) {
            const int s = threadIdx.x + j * blockDim.x;
            if (s >= slots) continue;
            if (ex[j] >= 0 && ex[j] < experts) sorted_slot[start[ex[j]] + at[j]] = s;
            if (tab.table) {
                idx[s] = ex[j];
                tab.wgt[s] = tab.weight;
            }
        }
        return;
    }
    __syncthreads();
    for (int s = threadIdx.x; s < slots; s += blockDim.x) {
        const int e = moe_slot_expert(idx, s, tab);
        if (e >= 0 && e < experts) sorted_slot[start[e] + atomicAdd(&count[e], 1)] = s;
        if (tab.table) {
            idx[s] = e;
            tab.wgt[s] = tab.weight;
        }
    }
}

__global__ void __launch_bounds__(1024)
moe_align_kernel(int *__restrict__ sorted_slot, int *__restrict__ tile_expert, int *idx, int slots, int experts, int capacity,
                 int max_tiles, int group, MoeTable tab) {
    __shared__ int count[MOE_MAX_EXPERTS], start[MOE_MAX_EXPERTS];
    moe_align_workgroup(sorted_slot, tile_expert, idx, slots, experts, capacity, max_tiles, group, tab, count, start);
}

static int moe_align_check(const int *sorted_slot, const int *tile_expert, const int *idx, int slots, int experts, int capacity,
                           int max_tiles, int group) {
    KVA_REQUIRE(group >= 1 && max_tiles % group == 0, "moe_align: %d tiles do not come in groups of %d", max_tiles, group);
    KVA_REQUIRE(sorted_slot && tile_expert && idx, "moe_align: missing operand");
    KVA_REQUIRE(experts > 0 && experts <= MOE_MAX_EXPERTS, "moe_align: %d experts (at most %d)", experts, MOE_MAX_EXPERTS);
    KVA_REQUIRE(capacity == max_tiles * MOE_TILE && capacity >= slots + experts * (MOE_TILE * group - 1),
                "moe_align: a list of %d places cannot hold %d slots of %d experts in tiles of %d", capacity, slots,
                experts, MOE_TILE);
    return KVA_OK;
}

static int moe_align_launch(int *sorted_slot, int *tile_expert, int *idx, int slots, int experts, int capacity, int max_tiles,
                            int group, const MoeTable &tab, hipStream_t stream) {
    if (int rc = moe_align_check(sorted_slot, tile_expert, idx, slots, experts, capacity, max_tiles, group)) return rc;
    hipLaunchKernelGGL(moe_align_kernel, dim3(1), dim3(1024), 0, stream, sorted_slot, tile_expert, idx, slots, experts,
                       capacity, max_tiles, group, tab);
    KVA_CHECK_LAUNCH("moe_align");
    return KVA_OK;
}

extern "C" int kva_moe_align(int *sorted_slot, int *tile_expert, const int *idx, int slots, int experts, int capacity,
                             int max_tiles, int group, hipStream_t stream) {
    // (without a table the kernel only reads idx)
    return moe_align_launch(sorted_slot, tile_expert, const_cast<int *>(idx), slots, experts, capacity, max_tiles, group,
                            MoeTable{nullptr, nullptr, nullptr, 0, 1, 0.f, nullptr}, stream);
}

extern "C" int kva_moe_table_align(int *sorted_slot, int *tile_expert, int *idx, float *wgt, const int *table, int table_rows,
                                   const int *ids, const int *feedback, int tokens, int top, float weight, int experts,
                                   int capacity, int max_tiles, int group, hipStream_t stream) {
    KVA_REQUIRE(wgt && table && ids && table_rows > 0 && tokens >= 0 && top > 0, "moe_table_align: missing operand or bad sizes");
    return moe_align_launch(sorted_slot, tile_expert, idx, tokens * top, experts, capacity, max_tiles, group,
                            MoeTable{table, ids, feedback, table_rows, top, weight, wgt}, stream);
}

// ---- the router's product, the choice and (few tokens) the sorted list in one launch ---------------------------------
// A workgroup of 16 wavefronts takes 16 tokens: logits^T[n, t] = W[n, :] . x[t, :] + bias[n] on the matrix cores (bf16
// operands, whose products are exact, and fp32 sums), a tile of 16 outputs and a part of K a wavefront; the parts meet in
// LDS in a fixed order, and wavefront i then routes token i.  Outputs past the router's (an expert's gate, say) go to
// `rest` [tokens, N - outputs].  A single workgroup's slots are sorted by expert right behind it.  The order of every
// sum depends on the sizes alone.
#define MOE_ROUTER_MAX_N 512

struct MoeRouter {
    const bf16_t *x, *w;
    const float *bias;
    float *rest;
    int *idx;
    float *wgt;
    int tokens, N, K, x_stride;
};

template <int PL>
__global__ void __launch_bounds__(1024)
moe_router_kernel(MoeRouter m, MoeRoute a, int *__restrict__ sorted_slot, int *__restrict__ tile_expert, int experts, int capacity,
                  int max_tiles, int group) {
    extern __shared__ __attribute__((aligned(16))) float moe_lds[];
    __shared__ int count[MOE_MAX_EXPERTS], start[MOE_MAX_EXPERTS];
    __shared__ float part[16][KVA_WAVE][4];
    const int lane = threadIdx.x % KVA_WAVE, wave = threadIdx.x / KVA_WAVE, r = lane & 15, g = lane >> 4;
    const int t0 = blockIdx.x * 16, tiles = (m.N + 15) / 16, parts = tiles < 16 ? 16 / tiles : 1;
    float *logits = moe_lds;                                     // [16 tokens][N]
    const int steps = m.K / 32, per = (steps + parts - 1) / parts;
    const bf16_t *xrow = m.x + (size_t)min(t0 + r, m.tokens - 1) * m.x_stride + 8 * g;
    for (int tile0 = 0; tile0 < tiles; tile0 += 16) {            // (more than 256 outputs: in turns)
        const int tile = tile0 + wave % min(tiles, 16), kp = wave / min(tiles, 16);
        const bool on = tile < tiles && kp < parts;
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
        if (on) {
            const bf16_t *wrow = m.w + (size_t)min(16 * tile + r, m.N - 1) * m.K + 8 * g;
            const int s1 = min(steps, (kp + 1) * per);
#pragma unroll 8
            for (int s = kp * per; s < s1; ++s) {
                Frag8 xf, wf;
                xf.u4 = *reinterpret_cast<const uint4 *>(xrow + 32 * s);
                wf.u4 = *reinterpret_cast<const uint4 *>(wrow + 32 * s);
                acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf.v, xf.v, acc, 0, 0, 0);
            }
        }
        __syncthreads();
#pragma unroll
        for (int i = 0; i < 4; ++i) part[wave][lane][i] = acc[i];
        __syncthreads();
        if (on && kp == 0) {                                     // lane (token r, group g): outputs 16 tile + 4 g .. + 3
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int n = 16 * tile + 4 * g + i;
                float v = acc[i];
                for (int p = 1; p < parts; ++p) v += part[wave + p * min(tiles, 16)][lane][i];
                if (n < m.N) logits[r * m.N + n] = v + (m.bias ? m.bias[n] : 0.f);
            }
        }
    }
    __syncthreads();
    const int t = t0 + wave;
    if (t < m.tokens) {
        moe_route_token<PL>(a, logits + wave * m.N, m.idx + (size_t)t * a.top, m.wgt + (size_t)t * a.top,
                            logits + 16 * m.N + (PL == 1 || a.groups > 1 ? wave * KVA_WAVE * PL : 0));
        for (int n = a.outputs + lane; n < m.N; n += KVA_WAVE) m.rest[(size_t)t * (m.N - a.outputs) + n - a.outputs] = logits[wave * m.N + n];
    }
    if (!sorted_slot) return;
    __threadfence_block();
    __syncthreads();
    moe_align_workgroup(sorted_slot, tile_expert, m.idx, m.tokens * a.top, experts, capacity, max_tiles, group,
                        MoeTable{nullptr, nullptr, nullptr, 0, 1, 0.f, nullptr}, count, start);
}

extern "C" int kva_moe_router_supported(int x_dtype, int w_dtype, int N, int K) {
    return x_dtype == KVA_BF16 && w_dtype == KVA_BF16 && K > 0 && K % 32 == 0 && N > 0 && N <= MOE_ROUTER_MAX_N;
}

// sorted_slot may be null: the list is then left to kva_moe_align (it must be for more than 16 tokens)
extern "C" int kva_moe_router(int *idx, float *wgt, float *rest, const void *x, int x_stride, const void *w, const float *bias,
                              const float *correction, int tokens, int N, int K, int outputs, int top, int renormalise,
                              int over_chosen, int sigmoid_scores, int groups, int keep_groups, int group_top,
                              float weight_scale, float sum_eps, int *sorted_slot, int *tile_expert, int experts,
                              int capacity, int max_tiles, int group, hipStream_t stream) {
    KVA_REQUIRE(idx && wgt && x && w && tokens >= 0 && outputs <= N && (outputs == N || rest), "moe_router: missing operand");
    KVA_REQUIRE(kva_moe_router_supported(KVA_BF16, KVA_BF16, N, K) && x_stride >= K && x_stride % 8 == 0 &&
                    ((reinterpret_cast<uintptr_t>(x) | reinterpret_cast<uintptr_t>(w)) & 15) == 0,
                "moe_router: no kernel for %d outputs of %d elements, or rows that do not start at multiples of 16 bytes", N, K);
    const MoeRoute a{correction, outputs, top, renormalise, over_chosen, sigmoid_scores, groups, keep_groups, group_top, weight_scale, sum_eps};
    if (int rc = moe_route_check(a)) return rc;
    if (sorted_slot) {
        KVA_REQUIRE(tokens <= 16, "moe_router: the list of more than 16 tokens is sorted by a launch of its own");
        if (int rc = moe_align_check(sorted_slot, tile_expert, idx, tokens * top, experts, capacity, max_tiles, group)) return rc;
    }
    if (tokens == 0) return KVA_OK;
    const int per_lane = outputs <= KVA_WAVE ? 1 : MOE_ROUTE_PER_LANE;
    const size_t lds = (size_t)(16 * N + (per_lane == 1 || groups > 1 ? 16 * KVA_WAVE * per_lane : 0)) * sizeof(float);
    auto kernel = per_lane == 1 ? moe_router_kernel<1> : moe_router_kernel<MOE_ROUTE_PER_LANE>;
    if (lds > 32 * 1024)
        hipFuncSetAttribute(reinterpret_cast<const void *>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    hipLaunchKernelGGL(kernel, dim3((tokens + 15) / 16), dim3(1024), lds, stream,
                       MoeRouter{(const bf16_t *)x, (const bf16_t *)w, bias, rest, idx, wgt, tokens, N, K, x_stride}, a, sorted_slot,
                       tile_expert, experts, capacity, max_tiles, group);
    KVA_CHECK_LAUNCH("moe_router");
    return KVA_OK;
}

// ---- one product per tile ------------------------------------------------------------------
struct MoeRows {
    const int *sorted_slot, *tile_expert;
    const float *slot_weight;       // mode 1: of the row that is written; mode 0 (optional): of the row that is read
    int top, N, K, mode, act;
    int tiled;                      // the matrices lie in operand order: [N / 16][K / 32][lane][8] (lane = 16 (k % 32 / 8) + n % 16)
    int gated;                      // mode 0: rows 2 j and 2 j + 1 of the matrix are output j's gate and up rows
    float limit;                    // activation 4 (clamped swish): gate and up are cut off at this value
};

// mode 0 of a gated expert: outputs n (even) and n + 1 of the product are one output of the layer
// (a weight on the expert's input multiplies both of them in front of the activation: W (w x) = w (W x))
__device__ inline void moe_store_gated(const MoeRows &a, void *out, int out_dtype, int place, int slot, int n, float gate, float up) {
    if (a.slot_weight) {
        gate *= a.slot_weight[slot];
        up *= a.slot_weight[slot];
    }
    const float v = a.act == 4 ? kva_gated_activate(gate, up, KVA_ACT_SWISH_CLAMPED, a.limit) : moe_activate(gate, a.act) * up;
    const size_t at = (size_t)place * (a.N / 2) + n / 2;
    if (out_dtype == KVA_BF16) reinterpret_cast<uint16_t *>(out)[at] = float_to_bf16_bits(v);
    else reinterpret_cast<float *>(out)[at] = v;
}

__device__ inline void moe_store(const MoeRows &a, void *out, int out_dtype, int place, int slot, int n, float v) {
    if (a.mode == 0) {
        if (a.slot_weight) v *= a.slot_weight[slot];
        v = moe_activate(v, a.act);
        if (out_dtype == KVA_BF16) reinterpret_cast<uint16_t *>(out)[(size_t)place * a.N + n] = float_to_bf16_bits(v);
        else reinterpret_cast<float *>(out)[(size_t)place * a.N + n] = v;
    } else {
        reinterpret_cast<float *>(out)[(size_t)slot * a.N + n] = a.slot_weight ? v * a.slot_weight[slot] : v;
    }
}

// plain: a workgroup takes a tile of 16 rows and 64 outputs; thread (row, cx) 4 neighbouring outputs
template <typename T>
__global__ void __launch_bounds__(256)
moe_expert_rows_kernel(MoeRows a, void *__restrict__ out, int out_dtype, const T *__restrict__ x,
                       const T *__restrict__ w) {
    __shared__ float xs[MOE_TILE][33], ws[64][33];
    const int tile = blockIdx.y, e = a.tile_expert[tile];
    if (e < 0) return;
    const int n0 = blockIdx.x * 64, row = threadIdx.x / 16, cx = threadIdx.x % 16;
    const int place = tile * MOE_TILE + row, slot = a.sorted_slot[place];
    const T *wm = w + (size_t)e * a.N * a.K;
    float acc[4] = {0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < a.K; k0 += 32) {
        __syncthreads();
        for (int i = threadIdx.x; i < MOE_TILE * 32; i += 256) {
            const int rr = i / 32, kk = k0 + i % 32;
            const int sl = a.sorted_slot[tile * MOE_TILE + rr];
            const size_t src = a.mode == 0 ? (size_t)(sl < 0 ? 0 : sl / a.top) : (size_t)(tile * MOE_TILE + rr);
            xs[rr][i % 32] = (kk < a.K && sl >= 0) ? to_float(x[src * a.K + kk]) : 0.f;
        }
        for (int i = threadIdx.x; i < 64 * 32; i += 256) {
            const int nn = n0 + i / 32, kk = k0 + i % 32;
            ws[i / 32][i % 32] = (nn < a.N && kk < a.K) ? to_float(wm[(size_t)nn * a.K + kk]) : 0.f;
        }
        __syncthreads();
        for (int kk = 0; kk < 32; ++kk) {
            const float xv = xs[row][kk];
#pragma unroll
            for (int j = 0; j < 4; ++j) acc[j] += xv * ws[4 * cx + j][kk];
        }
    }
    if (slot < 0) return;
    if (a.gated) {
#pragma unroll
        for (int j = 0; j < 4; j += 2) {
            const int n = n0 + 4 * cx + j;
            if (n + 1 < a.N) moe_store_gated(a, out, out_dtype, place, slot, n, acc[j], acc[j + 1]);
        }
        return;
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int n = n0 + 4 * cx + j;
        if (n < a.N) moe_store(a, out, out_dtype, place, slot, n, acc[j]);
    }
}

// matrix cores: a workgroup takes RT tiles of 16 rows and NT tiles of 16 outputs; out^T[n, t] =
// W[e][n, :] . x[t, :]; operands straight from memory, 16 bytes a lane and product.  Its four
// wavefronts take a quarter of K each (the same quarters whatever NT, RT and the batch are) and the
// first adds the four partial results up in a fixed order: with few tiles - decoded tokens - there are
// four times as many wavefronts streaming the experts' matrices.  Row tiles of one expert (the list is
// sorted by expert, so neighbours mostly are) share what is loaded of its matrix; a group of tiles
// that spans two experts is walked tile by tile.
template <int NT, int RT>
__device__ inline void moe_tiles_product(const MoeRows &a, void *__restrict__ out, int out_dtype,
                                         const bf16_t *__restrict__ x, const bf16_t *__restrict__ w, int first_tile,
                                         int e, int n_first, float (*red)[KVA_WAVE][4]) {
    const int lane = threadIdx.x % KVA_WAVE, wave = threadIdx.x / KVA_WAVE, r = lane & 15, g = lane >> 4;
    int place[RT], slot[RT];
    const bf16_t *xrow[RT];
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) {
        place[rt] = (first_tile + rt) * MOE_TILE + r;
        slot[rt] = a.sorted_slot[place[rt]];
        const size_t src = a.mode == 0 ? (size_t)(slot[rt] < 0 ? 0 : slot[rt] / a.top) : (size_t)place[rt];
        xrow[rt] = x + src * a.K + 8 * g;
    }
    const bf16_t *wrow[NT];
    const int wstep = a.tiled ? 16 * 32 : 32;       // from one step of 32 to the next
#pragma unroll
    for (int nt = 0; nt < NT; ++nt)
        wrow[nt] = w + (a.tiled ? ((size_t)e * a.N + min(n_first + 16 * nt, a.N - 16)) * a.K + 8 * lane
                                : ((size_t)e * a.N + min(n_first + 16 * nt + r, a.N - 1)) * a.K + 8 * g);
    f32x4 acc[NT][RT];
#pragma unroll
    for (int nt = 0; nt < NT; ++nt)
#pragma unroll
        for (int rt = 0; rt < RT; ++rt) acc[nt][rt] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int steps = a.K / 32, per = (steps + 3) / 4;
    const int s0 = wave * per, s1 = min(steps, s0 + per);
    constexpr int AHEAD = NT * RT == 1 ? 8 : 2;         // a tile of its own: as many loads in flight as there are products
#pragma unroll AHEAD
    for (int s = s0; s < s1; ++s) {
        const int k0 = 32 * s;
        Frag8 xf[RT], wf[NT];
#pragma unroll
        for (int rt = 0; rt < RT; ++rt) xf[rt].u4 = *reinterpret_cast<const uint4 *>(xrow[rt] + k0);
#pragma unroll
        for (int nt = 0; nt < NT; ++nt) wf[nt].u4 = *reinterpret_cast<const uint4 *>(wrow[nt] + (size_t)s * wstep);
#pragma unroll
        for (int nt = 0; nt < NT; ++nt)
#pragma unroll
            for (int rt = 0; rt < RT; ++rt)
                acc[nt][rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[nt].v, xf[rt].v, acc[nt][rt], 0, 0, 0);
    }
    __syncthreads();                 // whoever still reads the partial results of the call before is done
    if (wave > 0)
#pragma unroll
        for (int nt = 0; nt < NT; ++nt)
#pragma unroll
            for (int rt = 0; rt < RT; ++rt)
#pragma unroll
                for (int i = 0; i < 4; ++i) red[((wave - 1) * NT + nt) * RT + rt][lane][i] = acc[nt][rt][i];
    __syncthreads();
    if (wave > 0) return;
    // lane (row r, group g) holds outputs n0 + 4 g .. + 3 of its row
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) {
        if (slot[rt] < 0) continue;
#pragma unroll
        for (int nt = 0; nt < NT; ++nt) {
            float v[4];
#pragma unroll
            for (int i = 0; i < 4; ++i)
                v[i] = ((acc[nt][rt][i] + red[(0 * NT + nt) * RT + rt][lane][i]) + red[(1 * NT + nt) * RT + rt][lane][i])
                       + red[(2 * NT + nt) * RT + rt][lane][i];
            const int n = n_first + 16 * nt + 4 * g;
            if (a.gated) {
                if (n + 1 < a.N) moe_store_gated(a, out, out_dtype, place[rt], slot[rt], n, v[0], v[1]);
                if (n + 3 < a.N) moe_store_gated(a, out, out_dtype, place[rt], slot[rt], n + 2, v[2], v[3]);
            } else {
#pragma unroll
                for (int i = 0; i < 4; ++i)
                    if (n + i < a.N) moe_store(a, out, out_dtype, place[rt], slot[rt], n + i, v[i]);
            }
        }
    }
}

template <int NT, int RT>
__global__ void __launch_bounds__(256)
moe_expert_rows_mfma_kernel(MoeRows a, void *__restrict__ out, int out_dtype, const bf16_t *__restrict__ x,
                            const bf16_t *__restrict__ w, int max_tiles) {
    __shared__ float red[3 * NT * RT][KVA_WAVE][4];
    const int first = blockIdx.y * RT, n_first = blockIdx.x * 16 * NT;
    const int e0 = a.tile_expert[first];
    bool same = e0 >= 0;
#pragma unroll
    for (int rt = 1; rt < RT; ++rt) same = same && first + rt < max_tiles && a.tile_expert[first + rt] == e0;
    if (same) {
        moe_tiles_product<NT, RT>(a, out, out_dtype, x, w, first, e0, n_first, red);
        return;
    }
    for (int rt = 0; rt < RT; ++rt) {
        const int e = first + rt < max_tiles ? a.tile_expert[first + rt] : -1;
        if (e >= 0) moe_tiles_product<NT, 1>(a, out, out_dtype, x, w, first + rt, e, n_first, red);
    }
}

// matrix cores, many rows an expert: a workgroup takes a group of 2 RT tiles of one expert (32 RT rows) and 128
// outputs, operands through LDS (lds_product.h).  A die reads few experts.
template <int RT>
__global__ void __launch_bounds__(256)
moe_expert_rows_lds_kernel(MoeRows a, void *__restrict__ out, int out_dtype, const bf16_t *__restrict__ x,
                           const bf16_t *__restrict__ w, int n_blocks) {
    __shared__ __align__(16) typename LdsProduct<RT>::Shared shared;
    const int id = die_order(blockIdx.x, gridDim.x);
    const int first = (id / n_blocks) * 2 * RT, n0 = (id % n_blocks) * LDSP_N;
    const int e = a.tile_expert[first];
    if (e < 0) return;
    const int lane = threadIdx.x % KVA_WAVE, wave = threadIdx.x / KVA_WAVE, r = lane & 15, g = lane >> 4;
    const int wr = wave & 1, wn = wave >> 1;
    LdsProduct<RT> p;
#pragma unroll
    for (int i = 0; i < LdsProduct<RT>::XI; ++i) {
        const int place = first * MOE_TILE + p.row() + 32 * i, slot = a.sorted_slot[place];
        p.xp[i] = x + (a.mode == 0 ? (size_t)(slot < 0 ? 0 : slot / a.top) : (size_t)place) * a.K + p.element();
    }
    const bf16_t *we = w + (size_t)e * a.N * a.K;
    if (a.tiled) p.tiled_w(we, a.N, a.K, n0);
    else p.plain_w(we, a.N, a.K, n0);
    f32x4 acc[4][RT];
    p.run(shared, a.K, acc);
    // lane (row r, group g) holds outputs 4 g .. 4 g + 3 of tile nt, of its row of tile rt
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) {
        const int place = first * MOE_TILE + (wr * RT + rt) * 16 + r, slot = a.sorted_slot[place];
        if (slot < 0) continue;
        const float weight = a.mode == 1 && a.slot_weight ? a.slot_weight[slot] : 1.f;
#pragma unroll
        for (int nt = 0; nt < 4; ++nt) {
            const int n = n0 + wn * 64 + nt * 16 + 4 * g;
            const f32x4 v = acc[nt][rt];
            if (a.mode == 1 && a.N % 4 == 0) {
                if (n < a.N)
                    *reinterpret_cast<float4 *>(reinterpret_cast<float *>(out) + (size_t)slot * a.N + n) =
                        make_float4(v[0] * weight, v[1] * weight, v[2] * weight, v[3] * weight);
            } else if (a.gated) {
                if (n + 1 < a.N) moe_store_gated(a, out, out_dtype, place, slot, n, v[0], v[1]);
                if (n + 3 < a.N) moe_store_gated(a, out, out_dtype, place, slot, n + 2, v[2], v[3]);
            } else {
#pragma unroll
                for (int i = 0; i < 4; ++i)
                    if (n + i < a.N) moe_store(a, out, out_dtype, place, slot, n + i, v[i]);
            }
        }
    }
}

// groups of so many tiles of 16 rows have a kernel of their own (for operands in bf16 whose K is a multiple of 32)
extern "C" int kva_moe_group_supported(int group, int K) { return (group == 4 || group == 8) && K > 0 && K % 32 == 0; }

extern "C" int kva_moe_expert_rows(void *out, int out_dtype, const void *x, const void *w, int dtype,
                                   const int *sorted_slot, const int *tile_expert, const float *slot_weight,
                                   int max_tiles, int top, int N, int K, int mode, int act, int gated, float limit,
                                   int group, int tiled, hipStream_t stream) {
    KVA_REQUIRE(!tiled || (dtype == KVA_BF16 && K % 32 == 0 && N % 16 == 0), "moe_expert_rows: no operand order for %d x %d", N, K);
    KVA_REQUIRE(group == 1 || (dtype == KVA_BF16 && kva_moe_group_supported(group, K) && max_tiles % group == 0),
                "moe_expert_rows: no kernel for groups of %d tiles, %d of them, with K = %d", group, max_tiles, K);
    KVA_REQUIRE(act != 4 || gated, "moe_expert_rows: the clamped activation is a gated one");
    KVA_REQUIRE(!gated || (mode == 0 && N % 2 == 0), "moe_expert_rows: gate and up rows come in pairs, in the first product");
    KVA_REQUIRE(out && x && w && sorted_slot && tile_expert, "moe_expert_rows: missing operand");
    // slot_weight: in mode 1 of the row that is written, in mode 0 of the row that is read; absent: 1
    KVA_REQUIRE(mode == 0 || (mode == 1 && out_dtype == KVA_F32), "moe_expert_rows: mode 1 writes fp32 rows");
    KVA_REQUIRE(mode == 1 || out_dtype == dtype, "moe_expert_rows: mode 0 writes rows of the operands' type");
    KVA_REQUIRE(N > 0 && K > 0 && top > 0 && act >= 0 && act <= 5, "moe_expert_rows: bad sizes or activation");
    KVA_REQUIRE(max_tiles >= 0 && max_tiles <= 65535, "moe_expert_rows: %d tiles are too many for one launch", max_tiles);
    if (max_tiles == 0) return KVA_OK;
    MoeRows a{sorted_slot, tile_expert, slot_weight, top, N, K, mode, act, tiled, gated, limit};
    if (group > 1) {
        const int n_blocks = (N + LDSP_N - 1) / LDSP_N;
        const long long blocks = (long long)n_blocks * (max_tiles / group);
        KVA_REQUIRE(blocks <= 0x7fffffff, "moe_expert_rows: too many workgroups");
        if (group == 8)
            hipLaunchKernelGGL((moe_expert_rows_lds_kernel<4>), dim3((unsigned)blocks), dim3(256), 0, stream, a, out, out_dtype,
                               (const bf16_t *)x, (const bf16_t *)w, n_blocks);
        else
            hipLaunchKernelGGL((moe_expert_rows_lds_kernel<2>), dim3((unsigned)blocks), dim3(256), 0, stream, a, out, out_dtype,
                               (const bf16_t *)x, (const bf16_t *)w, n_blocks);
    } else if (dtype == KVA_BF16 && K % 32 == 0) {
        // few tiles: 16 outputs a workgroup, so that enough of them stream the matrices; many: 64 outputs and
        // four row tiles, which share what they load
        if ((long long)max_tiles * ((N + 15) / 16) <= 8192)
            hipLaunchKernelGGL((moe_expert_rows_mfma_kernel<1, 1>), dim3((N + 15) / 16, max_tiles), dim3(256), 0, stream, a,
                               out, out_dtype, (const bf16_t *)x, (const bf16_t *)w, max_tiles);
        else
            hipLaunchKernelGGL((moe_expert_rows_mfma_kernel<4, 4>), dim3((N + 63) / 64, (max_tiles + 3) / 4), dim3(256), 0,
                               stream, a, out, out_dtype, (const bf16_t *)x, (const bf16_t *)w, max_tiles);
    } else if (dtype == KVA_BF16) {
        hipLaunchKernelGGL(moe_expert_rows_kernel<bf16_t>, dim3((N + 63) / 64, max_tiles), dim3(256), 0, stream, a, out,
                           out_dtype, (const bf16_t *)x, (const bf16_t *)w);
    } else if (dtype == KVA_F32) {
        hipLaunchKernelGGL(moe_expert_rows_kernel<float>, dim3((N + 63) / 64, max_tiles), dim3(256), 0, stream, a, out,
                           out_dtype, (const float *)x, (const float *)w);
    } else KVA_REQUIRE(false, "moe_expert_rows: unsupported dtype %d", dtype);
    KVA_CHECK_LAUNCH("moe_expert_rows");
    return KVA_OK;
}

// ---- weighted sum --------------------------------------------------------------------------
__device__ inline float moe_ld(const void *p, int dtype, size_t i) {
    return dtype == KVA_BF16 ? bf16_bits_to_float(reinterpret_cast<const uint16_t *>(p)[i])
                             : reinterpret_cast<const float *>(p)[i];
}

__global__ void __launch_bounds__(256)
moe_combine_kernel(void *__restrict__ out, const void *__restrict__ x, int dtype, const float *__restrict__ rows,
                   const int *__restrict__ idx, const float *__restrict__ wgt, const void *__restrict__ extra,
                   const float *__restrict__ extra_gate, int extra_gate_stride, int width, int top, int experts) {
    const size_t t = blockIdx.x;
    // (optional) the addend enters times sigmoid(extra_gate[t * stride]), one number a token (a column of a wider array)
    const float eg = extra && extra_gate ? 1.f / (1.f + expf(-extra_gate[t * extra_gate_stride])) : 1.f;
    if (width % 4 == 0 && ((reinterpret_cast<uintptr_t>(rows) | reinterpret_cast<uintptr_t>(out)) & 15) == 0) {
        // four neighbouring columns a thread, 16 bytes of every row at a time; the additions per column are
        // in the order of the scalar loop below
        for (int j = threadIdx.x * 4; j < width; j += blockDim.x * 4) {
            float acc[4] = {0.f, 0.f, 0.f, 0.f};
            for (int k = 0; k < top; ++k) {
                const size_t s = t * top + k;
                if (idx[s] < experts) {
                    const float4 r = *reinterpret_cast<const float4 *>(rows + s * width + j);
                    acc[0] += r.x; acc[1] += r.y; acc[2] += r.z; acc[3] += r.w;
                } else {
                    const float g = wgt[s];
#pragma unroll
                    for (int e = 0; e < 4; ++e) acc[e] += g * moe_ld(x, dtype, t * width + j + e);
                }
            }
            if (extra) {
#pragma unroll
                for (int e = 0; e < 4; ++e) acc[e] += eg * moe_ld(extra, dtype, t * width + j + e);
            }
            if (dtype == KVA_BF16) {
                const uint2 o = make_uint2((uint32_t)float_to_bf16_bits(acc[0]) | ((uint32_t)float_to_bf16_bits(acc[1]) << 16),
                                           (uint32_t)float_to_bf16_bits(acc[2]) | ((uint32_t)float_to_bf16_bits(acc[3]) << 16));
                *reinterpret_cast<uint2 *>(reinterpret_cast<uint16_t *>(out) + t * width + j) = o;
            } else {
                *reinterpret_cast<float4 *>(reinterpret_cast<float *>(out) + t * width + j) = make_float4(acc[0], acc[1], acc[2], acc[3]);
            }
        }
        return;
    }
    for (int j = threadIdx.x; j < width; j += blockDim.x) {
        float acc = 0.f;
        for (int k = 0; k < top; ++k) {
            const size_t s = t * top + k;
            if (idx[s] < experts) acc += rows[s * width + j];
            else acc += wgt[s] * (dtype == KVA_BF16 ? bf16_bits_to_float(reinterpret_cast<const uint16_t *>(x)[t * width + j])
                                                    : reinterpret_cast<const float *>(x)[t * width + j]);
        }
        // what an expert that every token uses returned, with weight 1
        if (extra) acc += eg * (dtype == KVA_BF16 ? bf16_bits_to_float(reinterpret_cast<const uint16_t *>(extra)[t * width + j])
                                                  : reinterpret_cast<const float *>(extra)[t * width + j]);
        if (dtype == KVA_BF16) reinterpret_cast<uint16_t *>(out)[t * width + j] = float_to_bf16_bits(acc);
        else reinterpret_cast<float *>(out)[t * width + j] = acc;
    }
}

extern "C" int kva_moe_combine(void *out, const void *x, int dtype, const float *rows, const int *idx,
                               const float *wgt, const void *extra, const float *extra_gate, int extra_gate_stride,
                               int tokens, int width, int top, int experts, hipStream_t stream) {
    KVA_REQUIRE(out && x && rows && idx && wgt && width > 0 && top > 0, "moe_combine: missing operand");
    KVA_REQUIRE(dtype == KVA_BF16 || dtype == KVA_F32, "moe_combine: unsupported dtype %d", dtype);
    if (tokens <= 0) return KVA_OK;
    hipLaunchKernelGGL(moe_combine_kernel, dim3(tokens), dim3(256), 0, stream, out, x, dtype, rows, idx, wgt, extra, extra_gate,
                       extra_gate_stride, width, top, experts);
    KVA_CHECK_LAUNCH("moe_combine");
    return KVA_OK;
}

// ---- small products with 32-bit results -------------------------------------------------------
// out[t, n] = sum_k x[t, k] * w[n, k] in fp32, for the small matrices whose results must not be rounded
// to 16 bits (a router's logits; the second half of a low-rank projection that makes decays, which
// may be finished here: bias, sigmoid, power).  x and
// w may be bf16 or fp32; every product and sum is fp32.  A workgroup takes a token: its row of x goes
// to LDS once; with a long K a wavefront takes an output and its lanes stride over K (sum by
// wavefront reduction), with a short K a thread takes an output.  The order of every sum depends on
// the sizes alone.
#define SMALL_PRODUCT_MAX_K 8192

// eight neighbouring elements from index i on (i a multiple of 8: 16 or 32 aligned bytes)
__device__ inline void moe_ld8(const void *p, int dtype, size_t i, float (&f)[8]) {
    if (dtype == KVA_BF16) {
        const uint4 v = *reinterpret_cast<const uint4 *>(reinterpret_cast<const uint16_t *>(p) + i);
        const unsigned u[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            f[2 * j] = __uint_as_float(u[j] << 16);
            f[2 * j + 1] = __uint_as_float(u[j] & 0xffff0000u);
        }
    } else {
        const float4 a = *reinterpret_cast<const float4 *>(reinterpret_cast<const float *>(p) + i);
        const float4 b = *reinterpret_cast<const float4 *>(reinterpret_cast<const float *>(p) + i + 4);
        f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w; f[4] = b.x; f[5] = b.y; f[6] = b.z; f[7] = b.w;
    }
}

// the result as it is, plus a bias, or - with decay_inv_tau > 0 - turned into a decay:
// sigmoid(z)^(1 / tau) = exp(-softplus(-z) / tau) with z = the sum plus its bias
// or - with rate_log - into exp(-exp(rate_log[n / rate_group]) softplus(z)): a decay per output whose rate
// is shared by groups of neighbouring outputs (the key channels of a head)
__device__ inline float small_product_finish(float acc, const float *bias, int n, float decay_inv_tau,
                                             const float *rate_log, int rate_group) {
    const float z = acc + (bias ? bias[n] : 0.f);
    if (rate_log) return expf(-expf(rate_log[n / rate_group]) * (fmaxf(z, 0.f) + log1pf(expf(-fabsf(z)))));
    if (decay_inv_tau <= 0.f) return z;
    const float softplus = fmaxf(-z, 0.f) + log1pf(expf(-fabsf(z)));
    return expf(-softplus * decay_inv_tau);
}

__global__ void __launch_bounds__(256)
small_product_f32_kernel(float *__restrict__ out, const void *__restrict__ x, int x_dtype, int x_stride,
                         const void *__restrict__ w, int w_dtype, int N, int K, int per_block,
                         const float *__restrict__ bias, float decay_inv_tau, const float *__restrict__ rate_log,
                         int rate_group) {
    extern __shared__ float xs[];
    const size_t t = blockIdx.x;
    const int n_lo = blockIdx.y * per_block, n_hi = min(N, n_lo + per_block);
    for (int k = threadIdx.x; k < K; k += blockDim.x) xs[k] = moe_ld(x, x_dtype, t * x_stride + k);
    __syncthreads();
    const int K8 = (K % 8 == 0) ? K : 0;          // the part read eight elements at a time
    if (K >= 128) {
        const int lane = threadIdx.x % KVA_WAVE, wave = threadIdx.x / KVA_WAVE, waves = blockDim.x / KVA_WAVE;
        for (int n = n_lo + wave; n < n_hi; n += waves) {
            float acc = 0.f;
            for (int k = 8 * lane; k < K8; k += 8 * KVA_WAVE) {
                float f[8];
                moe_ld8(w, w_dtype, (size_t)n * K + k, f);
#pragma unroll
                for (int i = 0; i < 8; ++i) acc += xs[k + i] * f[i];
            }
            for (int k = K8 + lane; k < K; k += KVA_WAVE) acc += xs[k] * moe_ld(w, w_dtype, (size_t)n * K + k);
            acc = wave_sum(acc);
            if (lane == 0) out[t * N + n] = small_product_finish(acc, bias, n, decay_inv_tau, rate_log, rate_group);
        }
    } else {
        for (int n = n_lo + threadIdx.x; n < n_hi; n += blockDim.x) {
            float acc = 0.f;
            for (int k = 0; k < K8; k += 8) {
                float f[8];
                moe_ld8(w, w_dtype, (size_t)n * K + k, f);
#pragma unroll
                for (int i = 0; i < 8; ++i) acc += xs[k + i] * f[i];
            }
            for (int k = K8; k < K; ++k) acc += xs[k] * moe_ld(w, w_dtype, (size_t)n * K + k);
            out[t * N + n] = small_product_finish(acc, bias, n, decay_inv_tau, rate_log, rate_group);
        }
    }
}

extern "C" int kva_small_product_f32(float *out, const void *x, int x_dtype, int x_stride, const void *w, int w_dtype,
                                     int tokens, int N, int K, const float *bias, float decay_inv_tau,
                                     const float *rate_log, int rate_group, hipStream_t stream) {
    KVA_REQUIRE(!rate_log || (rate_group > 0 && N % rate_group == 0 && decay_inv_tau <= 0.f),
                "small_product_f32: rates are shared by whole groups of outputs, and exclude the other decay");
    KVA_REQUIRE(out && x && w && tokens >= 0 && N > 0, "small_product_f32: missing operand or bad sizes");
    KVA_REQUIRE(K > 0 && K <= SMALL_PRODUCT_MAX_K && x_stride >= K, "small_product_f32: K %d must lie in 1..%d", K, SMALL_PRODUCT_MAX_K);
    KVA_REQUIRE((x_dtype == KVA_BF16 || x_dtype == KVA_F32) && (w_dtype == KVA_BF16 || w_dtype == KVA_F32),
                "small_product_f32: unsupported dtype");
    if (tokens == 0) return KVA_OK;
    KVA_REQUIRE((reinterpret_cast<uintptr_t>(w) & 31) == 0, "small_product_f32: the matrix must be aligned to 32 bytes");
    const int per_block = K >= 128 ? 16 : 256;         // outputs a workgroup: four a wavefront, or one a thread
    const int blocks_y = (N + per_block - 1) / per_block;
    KVA_REQUIRE(tokens <= 0x7fffffff && blocks_y <= 65535, "small_product_f32: too many outputs");
    hipLaunchKernelGGL(small_product_f32_kernel, dim3(tokens, blocks_y), dim3(256), (size_t)K * sizeof(float), stream,
                       out, x, x_dtype, x_stride, w, w_dtype, N, K, per_block, bias, decay_inv_tau, rate_log,
                       rate_group > 0 ? rate_group : 1);
    KVA_CHECK_LAUNCH("small_product_f32");
    return KVA_OK;
}
