// Paged causal attention for any head sizes (query/key size `dim`, value size `vdim`, any page size), with the pieces a
// gated, value-rotating attention needs around it:
//   nvh_attn_rotary_prep  per token, over the fused projection row [q | k | v | gate]: RMS norm over the WHOLE q and the
//                         whole k projection, or over every head by itself with one weight row shared by the heads
//                         (norm_per_head), partial rotary on q and k (frequency table given by the
//                         caller, so any scaling rule fits), rotation of the value by its own position over all of
//                         vdim, sigmoid of the per-head gate; q goes to a packed buffer, k and v to their cache slots.
//                         Keys are cached [pages, page, G, dim]; values TRANSPOSED within a page, [pages, G, vdim, page],
//                         so the attention reads a value column over consecutive keys in one piece (its matrix
//                         product wants V^T) and never transposes on the fly.
//   nvh_attn_kv_store     keys and values that need neither norm nor rotation, from the projection row to those cache slots, with an
//                         optional mixture of the value with another layer's value of the same token; in one-token steps also
//                         the block means that the tokens complete (below).  The query is read from the projection row in place.
//   nvh_attn_paged_any    softmax attention of var-len queries over the paged cache, scores / weights in fp32; the
//                         epilogue turns each head's output back by the query's position and multiplies the gate.
//                         Optional: a distance bias, score -= slope[head] * (query position - key position), and a
//                         sliding window that keeps the first tokens: query i sees key j <= i when i - j < window or
//                         j < keep_first; key tiles that no query of a workgroup can see are never loaded.
//                         Optional: chunks, query i sees key j <= i only when both lie in the same block of `chunk`
//                         positions counted from the sequence's start; and a sink per head, a learned logit that joins the
//                         softmax's denominator as one more term, as it is, standing for no token (it is the state a row starts from:
//                         maximum = sink, sum = 1, output = 0).
//                         Optional: pooled blocks in front of a window, one key and value (the means of the cached rows, see
//                         nvh_attn_pool_blocks) for each block of `pool` positions that lies wholly before the query's window,
//                         under the same softmax; a softcap, score <- cap tanh(score / cap); and a query temperature, q times
//                         1 + coef ln(floor((p + 1) / every) + 1) at position p.
//                         Optional: a learned bias per head and distance, score += bias[head][min(distance, len - 1)], and a gate per
//                         output element (a row of logits per token, beside the gate per head) in the epilogue.
//                         Steps in which every sequence brings one query: the heads that share a KV head share a workgroup
//                         (groups of more than 16 heads in parts); when that leaves most of the chip idle, a sequence's key
//                         tiles are dealt out to several workgroups whose rows a second launch merges.
//   nvh_attn_pool_blocks  the means of the blocks that a step has filled: keys and values read back from the cache as it holds
//                         them (so a block's mean does not depend on the steps that brought its tokens), fp32 sums, written to the
//                         page of the block's last token, rows [pages, pool_rows, G, dim] and [pages, pool_rows, G, vdim].
// Activations and caches are of type A (bf16 or fp32).  Key tiles always start at key 0 of a sequence and every query
// row keeps its own running maximum and sum, so a query's result does not depend on how the prompt was cut into steps
// or on what else is in the batch.
#include <type_traits>

#include "common.h"

namespace {

template <typename A>
__device__ __forceinline__ float ldf(const A* p, int64_t i) {
    return (float)p[i];
}

__device__ __forceinline__ float block_sum_256(float v, float* scratch) {
    v = wave_sum(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) scratch[threadIdx.x >> 6] = v;
    __syncthreads();
    return scratch[0] + scratch[1] + scratch[2] + scratch[3];
}

struct PrepArgs {
    const void* proj;          // [T, ld] : q (H*dim) | k (G*dim) | v (G*vdim) | gate (H)
    int64_t ld;
    const void *q_norm, *k_norm;   // [H*dim], [G*dim]; norm_per_head: [dim] each, shared by the heads
    int norm_per_head;
    float eps;
    const int64_t* positions;
    const float* qk_freq;      // [rot_dims / 2]
    float qk_mag;
    int rot_dims, qk_interleaved;
    const float* v_freq;       // [vdim / 2], or null: values are stored as they are
    int v_interleaved;
    void* q_out;               // [T, H*dim]
    float* gate_out;           // [T, H], or null (no gate columns in proj)
    void *k_cache, *v_cache;   // [pages, page, G, dim], [pages, G, vdim, page] (values transposed within a page)
    const int32_t* slot_mapping;
    int H, G, dim, vdim, page;
};

template <typename A>
__global__ __launch_bounds__(256) void attn_rotary_prep_kernel(PrepArgs a) {
    __shared__ float red[4];
    extern __shared__ float head_inv[];                      // norm_per_head: 1 / rms of every q head, then of every k head
    const int64_t t = blockIdx.x;
    const A* row = (const A*)a.proj + t * a.ld;
    const int nq = a.H * a.dim, nk = a.G * a.dim, nv = a.G * a.vdim;
    const A* qr = row;
    const A* kr = row + nq;
    const A* vr = kr + nk;
    float inv_q = 1.f, inv_k = 1.f;
    if (a.q_norm && a.norm_per_head) {                       // a wave per head in turn (q heads, then k heads: they lie one after the other)
        const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
        for (int h = wave; h < a.H + a.G; h += 4) {
            const A* hr = qr + (int64_t)h * a.dim;
            float ss = 0.f;
            for (int i = lane; i < a.dim; i += 64) {
                const float v = ldf(hr, i);
                ss += v * v;
            }
            ss = wave_sum(ss);
            if (lane == 0) head_inv[h] = 1.0f / sqrtf(ss / (float)a.dim + a.eps);
        }
        __syncthreads();
    } else if (a.q_norm) {                                   // (null norm weights: q and k pass as they are)
        float sq = 0.f, sk = 0.f;
        for (int i = threadIdx.x; i < nq; i += 256) {
            const float v = ldf(qr, i);
            sq += v * v;
        }
        for (int i = threadIdx.x; i < nk; i += 256) {
            const float v = ldf(kr, i);
            sk += v * v;
        }
        sq = block_sum_256(sq, red);
        sk = block_sum_256(sk, red);
        inv_q = 1.0f / sqrtf(sq / (float)nq + a.eps), inv_k = 1.0f / sqrtf(sk / (float)nk + a.eps);
    }
    const float pos = (float)a.positions[t];
    const int64_t slot = a.slot_mapping ? a.slot_mapping[t] : -1;
    // q and k: norm, then rotary on the first rot_dims dimensions of every head
    for (int which = 0; which < 2; ++which) {
        const int n = which ? nk : nq;
        const A* src = which ? kr : qr;
        const A* wn = (const A*)(which ? a.k_norm : a.q_norm);
        const float inv = which ? inv_k : inv_q;
        const int hbase = which ? a.H : 0;
        A* dst = which ? (slot >= 0 && a.k_cache ? (A*)a.k_cache + slot * nk : nullptr) : (A*)a.q_out + t * nq;
        if (!dst) continue;
        for (int i = threadIdx.x; i < n; i += 256) {
            const int d = i % a.dim;
            const float rinv = a.norm_per_head && wn ? head_inv[hbase + i / a.dim] : inv;
            float v = wn ? ldf(src, i) * rinv * ldf(wn, a.norm_per_head ? d : i) : ldf(src, i);
            if (d < a.rot_dims) {
                int partner, pair;
                bool first;
                pair_of(d, a.rot_dims, a.qk_interleaved, partner, pair, first);
                const int j = i - d + partner;
                const float o = wn ? ldf(src, j) * rinv * ldf(wn, a.norm_per_head ? partner : j) : ldf(src, j);
                float sn, cs;
                rot_sincos<A>(pos * a.qk_freq[pair], sn, cs);
                const float c = cs * a.qk_mag, s = sn * a.qk_mag;
                v = first ? v * c - o * s : v * c + o * s;
            }
            dst[i] = (A)v;
        }
    }
    if (slot >= 0 && a.v_cache) {
        A* dst = (A*)a.v_cache + (slot / a.page) * a.page * nv + slot % a.page;      // element i of the row goes to dst[i * page]
        for (int i = threadIdx.x; i < nv; i += 256) {
            float v = ldf(vr, i);
            if (a.v_freq) {
                const int d = i % a.vdim;
                int partner, pair;
                bool first;
                pair_of(d, a.vdim, a.v_interleaved, partner, pair, first);
                const float o = ldf(vr, i - d + partner);
                float s, c;
                rot_sincos<A>(pos * a.v_freq[pair], s, c);
                v = first ? v * c - o * s : v * c + o * s;
            }
            dst[(int64_t)i * a.page] = (A)v;
        }
    }
    if (a.gate_out)
        for (int h = threadIdx.x; h < a.H; h += 256) a.gate_out[t * a.H + h] = 1.0f / (1.0f + expf(-ldf(vr + nv, h)));
}

// ---------------------------------------------------------------------------------------------------------------
constexpr int AQ = 16;        // queries per workgroup (one 16-lane row of a wave per query)
constexpr int AK = 32;        // keys per tile
constexpr int AVC_MAX = 32;   // value columns per lane (the kernel's AVC: 16, or 32 for wide values): vdim <= 16 * AVC_MAX

struct AttnArgs {
    const void* q;             // [T, ldq]: H*dim columns
    int64_t ldq;
    const void *k_cache, *v_cache;
    const int32_t* cu_seqlens_q;    // [B+1], or null: one query per sequence (row b is sequence b)
    const int32_t* context_lens;    // [B]: keys of the sequence including this step's tokens
    const int32_t* block_tables;
    int64_t table_stride;
    int batch, page;
    int H, G, dim, vdim;
    float scale;
    const float* gate;         // [T, H] or null
    const float* v_freq;       // [vdim/2] or null: no turning back
    int v_interleaved;
    void* out;                 // [T, H*vdim]
    const void* gate_elems;    // [T, ld_elems]: H*vdim logits whose sigmoids multiply the output's elements, or null
    int64_t ld_elems;
    const float* slopes;       // [H] or null: score -= slopes[head] * (query position - key position)
    const float* bias;         // [H, bias_len] or null: score += bias[head][min(query position - key position, bias_len - 1)]
    int bias_len;
    int window, keep_first;    // window > 0: key j is visible to query i only when i - j < window or j < keep_first
    int chunk;                 // chunk > 0: ... and only when j >= (i / chunk) * chunk
    const float* sinks;        // [H] or null: a logit per head that joins the denominator of every row of that head
    float softcap;             // > 0: score <- softcap tanh(score / softcap)
    float temp_coef;           // temp_every > 0: scores of the query at position p times 1 + temp_coef ln(floor((p + 1) / temp_every) + 1)
    int temp_every;
    int pool, pool_rows;       // pool > 0 (with a window): blocks of `pool` positions before the window are seen through their means ...
    const void *pk, *pv;       // ... [pages, pool_rows, G, dim], [pages, pool_rows, G, vdim], in the page of the block's last position
    int pages_offset;          // byte offset in LDS of the sequence's page ids (matrix-core kernel)
    int ml_offset;             // ... of the waves' (max, sum) pairs in the one-query form
    int bias_offset, bias_ld;  // ... and of the heads' bias rows, bias_ld floats apart
    int kv_split;              // one-query form: workgroups per (sequence, KV head), each with H / (G kv_split) of the group's heads
    int key_parts;             // one-query form: workgroups that share a sequence's key tiles (tile j goes to part j % key_parts); > 1: the
    float* parts;              // parts leave [batch, G kv_split, key_parts, 16, vdim + 2] (unnormalised rows, then max and sum) here
};

// The key tiles (of `tile` keys, starting at multiples of it) that a workgroup whose first query sits at position qlo has to
// walk: all of them without a window; with one, the tiles that hold kept first tokens and then those from the window of
// the first query on.  next(k0) is the start of the tile after k0.
struct TileWalk {
    int first_end, win_start, tile;
    __device__ __forceinline__ TileWalk(int window, int keep_first, int chunk, int qlo, int tile_) : tile(tile_) {
        first_end = window > 0 ? ((keep_first + tile_ - 1) / tile_) * tile_ : 0;
        win_start = window > 0 ? (max(qlo - window + 1, 0) / tile_) * tile_ : 0;
        // (the chunk of the first query starts no later than any other query's: earlier tiles are seen by none)
        if (chunk > 0) win_start = max(win_start, ((qlo / chunk) * chunk / tile_) * tile_);
    }
    __device__ __forceinline__ int next(int k0) const {
        const int n = k0 + tile;
        return (n >= first_end && n < win_start) ? win_start : n;
    }
};

// Pooled blocks that the query at qpos sees: those whose last position is <= qpos - window.
__device__ __forceinline__ int blocks_seen(int qpos, int window, int pool) { return qpos >= window ? (qpos - window + 1) / pool : 0; }

// Where the mean of block b lies: the page of the block's last position (as an index into the sequence's pages) and the row
// within that page (blocks whose last position is in page n are numbered from floor(n page / pool) on).
__device__ __forceinline__ void block_place(int b, int pool, int page, int& page_index, int& row) {
    page_index = (b * pool + pool - 1) / page;
    row = b - page_index * page / pool;
}

__device__ __forceinline__ float query_temperature(int qpos, float coef, int every) {
    return every > 0 ? 1.0f + coef * logf((float)((qpos + 1) / every + 1)) : 1.0f;
}

// The tiles in order: with pooled blocks, ceil(blocks / tile) tiles of them first - their start is counted up to 0 from below,
// tile v of n starts at (v - n) tile - and then the token tiles of the walk.
struct TileOrder {
    TileWalk walk;
    int pooled_span;           // pooled tiles times tile
    __device__ __forceinline__ TileOrder(const TileWalk& w, int blocks) : walk(w), pooled_span((blocks + w.tile - 1) / w.tile * w.tile) {}
    __device__ __forceinline__ int first_token_tile() const { return walk.first_end > 0 || walk.win_start == 0 ? 0 : walk.win_start; }
    __device__ __forceinline__ int first() const { return pooled_span > 0 ? -pooled_span : first_token_tile(); }
    __device__ __forceinline__ int next(int k0) const {
        if (k0 >= 0) return walk.next(k0);
        return k0 + walk.tile < 0 ? k0 + walk.tile : first_token_tile();
    }
    __device__ __forceinline__ int block_of(int k0) const { return k0 + pooled_span; }       // (k0 < 0) the tile's first block
};

__device__ __forceinline__ bool key_visible(int key, int qpos, int window, int keep_first, int chunk) {
    return key <= qpos && (window <= 0 || qpos - key < window || key < keep_first) && (chunk <= 0 || key >= (qpos / chunk) * chunk);
}

// The sigmoid of an element gate: the library's exponential where everything is fp32, the hardware's 2^x and reciprocal for bf16 results.
template <typename A>
__device__ __forceinline__ float elem_gate(float z) {
    if constexpr (sizeof(A) == 4) return 1.0f / (1.0f + expf(-z));
    else return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-z * 1.4426950408889634f));
}

template <typename A, int AVC>
__global__ __launch_bounds__(256) void attn_paged_any_kernel(AttnArgs a) {
    extern __shared__ float smem[];
    // which (sequence, query tile) is this workgroup's
    int seq = -1, q0 = 0, qlen = 0, qbase = 0;
    {
        int tile = blockIdx.x;
        for (int b = 0; b < a.batch; ++b) {
            const int lo = a.cu_seqlens_q ? a.cu_seqlens_q[b] : b, hi = a.cu_seqlens_q ? a.cu_seqlens_q[b + 1] : b + 1;
            const int tiles = (hi - lo + AQ - 1) / AQ;
            if (tile < tiles) {
                seq = b;
                q0 = tile * AQ;
                qlen = hi - lo;
                qbase = lo;
                break;
            }
            tile -= tiles;
        }
    }
    if (seq < 0) return;                                     // (uniform over the workgroup)
    const int head = blockIdx.y, kvh = head / (a.H / a.G);
    const int dim = a.dim, vdim = a.vdim;
    const int klen = a.context_lens[seq];
    const int past = klen - qlen;                            // keys before this step's first query
    const int nq = min(AQ, qlen - q0);
    const int kd = dim + 1, vd = vdim + 1;
    float* qs = smem;                                        // [AQ][dim]
    float* ks = qs + AQ * dim;                               // [AK][dim + 1]
    float* vs = ks + AK * kd;                                // [AK][vdim + 1]
    float* ps = vs + AK * vd;                                // [AQ][AK]
    const int tid = threadIdx.x, qi = tid >> 4, sub = tid & 15;
    for (int i = tid; i < AQ * dim; i += 256) {
        const int r = i / dim, d = i - r * dim;
        const float sc = a.scale * query_temperature(past + q0 + r, a.temp_coef, a.temp_every);
        qs[i] = r < nq ? ldf((const A*)a.q, (int64_t)(qbase + q0 + r) * a.ldq + head * dim + d) * sc : 0.f;
    }
    float acc[AVC];
#pragma unroll
    for (int c = 0; c < AVC; ++c) acc[c] = 0.f;
    // (a sink is what the row starts from: it has been seen with score sink, weight 1 and no value)
    float m_run = a.sinks ? a.sinks[head] : -INFINITY, l_run = a.sinks ? 1.f : 0.f;
    const int qpos = past + q0 + qi;                         // this lane's query position (valid for qi < nq)
    const int last_key = past + q0 + nq - 1;                 // the tile's last query sees keys 0..last_key
    const int32_t* table = a.block_tables + (int64_t)seq * a.table_stride;
    const float slope = a.slopes ? a.slopes[head] : 0.f;
    const float* bias = a.bias ? a.bias + (int64_t)head * a.bias_len : nullptr;
    const int nblocks = a.pool > 0 ? blocks_seen(last_key, a.window, a.pool) : 0, my_blocks = a.pool > 0 ? blocks_seen(qpos, a.window, a.pool) : 0;
    const TileOrder order(TileWalk(a.window, a.keep_first, a.chunk, past + q0, AK), nblocks);
    for (int k0 = order.first(); k0 <= last_key; k0 = order.next(k0)) {
        const bool pooled = k0 < 0;                          // (uniform) a tile of block means; bk0: its first block
        const int bk0 = order.block_of(k0);
        __syncthreads();                                     // the previous tile's readers are done
        if (pooled) {
            for (int i = tid; i < AK * (dim + vdim); i += 256) {
                const int r = i / (dim + vdim), d = i - r * (dim + vdim), b = bk0 + r;
                float v = 0.f;
                if (b < nblocks) {
                    int pi, row;
                    block_place(b, a.pool, a.page, pi, row);
                    const int64_t at = ((int64_t)table[pi] * a.pool_rows + row) * a.G + kvh;
                    v = d < dim ? ldf((const A*)a.pk, at * dim + d) : ldf((const A*)a.pv, at * vdim + d - dim);
                }
                (d < dim ? ks[r * kd + d] : vs[r * vd + d - dim]) = v;
            }
        } else {
        for (int i = tid; i < AK * dim; i += 256) {
            const int r = i / dim, d = i - r * dim, key = k0 + r;
            float v = 0.f;
            if (key <= last_key) {
                const int64_t slot = (int64_t)table[key / a.page] * a.page + key % a.page;
                v = ldf((const A*)a.k_cache, (slot * a.G + kvh) * dim + d);
            }
            ks[r * kd + d] = v;
        }
        for (int i = tid; i < AK * vdim; i += 256) {
            const int r = i / vdim, d = i - r * vdim, key = k0 + r;
            float v = 0.f;
            if (key <= last_key) {
                v = ldf((const A*)a.v_cache, (((int64_t)table[key / a.page] * a.G + kvh) * vdim + d) * a.page + key % a.page);
            }
            vs[r * vd + d] = v;
        }
        }
        __syncthreads();
        // scores of query qi against keys sub and sub + 16 of the tile
        float s0 = 0.f, s1 = 0.f;
        const float* qrow = qs + qi * dim;
        const float *kr0 = ks + sub * kd, *kr1 = ks + (sub + 16) * kd;
        for (int d = 0; d < dim; ++d) {
            const float qv = qrow[d];
            s0 = __builtin_fmaf(qv, kr0[d], s0);
            s1 = __builtin_fmaf(qv, kr1[d], s1);
        }
        if (a.softcap > 0.f) {
            s0 = a.softcap * tanhf(s0 / a.softcap);
            s1 = a.softcap * tanhf(s1 / a.softcap);
        }
        const bool ok0 = qi < nq && (pooled ? bk0 + sub < my_blocks : key_visible(k0 + sub, qpos, a.window, a.keep_first, a.chunk));
        const bool ok1 = qi < nq && (pooled ? bk0 + sub + 16 < my_blocks : key_visible(k0 + sub + 16, qpos, a.window, a.keep_first, a.chunk));
        s0 = ok0 ? s0 - slope * (float)(qpos - (k0 + sub)) : -INFINITY;
        s1 = ok1 ? s1 - slope * (float)(qpos - (k0 + sub + 16)) : -INFINITY;
        if (bias) {
            if (ok0) s0 += bias[min(qpos - (k0 + sub), a.bias_len - 1)];
            if (ok1) s1 += bias[min(qpos - (k0 + sub + 16), a.bias_len - 1)];
        }
        const float m_new = fmaxf(m_run, row16_max(fmaxf(s0, s1)));
        // a row that sees nothing yet keeps m = -inf (only rows past nq: every real query sees key 0)
        const float p0 = ok0 ? expf(s0 - m_new) : 0.f, p1 = ok1 ? expf(s1 - m_new) : 0.f;
        const float alpha = m_new == -INFINITY ? 1.f : expf(m_run - m_new);
        l_run = l_run * alpha + row16_sum(p0 + p1);
        m_run = m_new;
        ps[qi * AK + sub] = p0;
        ps[qi * AK + sub + 16] = p1;
        __syncthreads();
        const float* prow = ps + qi * AK;
#pragma unroll
        for (int c = 0; c < AVC; ++c) {
            const int col = sub + 16 * c;
            if (col < vdim) {
                float s = acc[c] * alpha;
                for (int r = 0; r < AK; ++r) s = __builtin_fmaf(prow[r], vs[r * vd + col], s);
                acc[c] = s;
            }
        }
    }
    // epilogue: normalise, turn back by the query's position, gate
    __syncthreads();
    float* os = ks;                                          // [AQ][vdim] (fits: AK >= AQ)
#pragma unroll
    for (int c = 0; c < AVC; ++c) {
        const int col = sub + 16 * c;
        if (col < vdim) os[qi * vdim + col] = l_run > 0.f ? acc[c] / l_run : 0.f;
    }
    __syncthreads();
    if (qi < nq) {
        const int64_t tok = qbase + q0 + qi;
        const float g = a.gate ? a.gate[tok * a.H + head] : 1.0f;
        const float pos = (float)qpos;
#pragma unroll
        for (int c = 0; c < AVC; ++c) {
            const int col = sub + 16 * c;
            if (col < vdim) {
                float v = os[qi * vdim + col];
                if (a.v_freq) {
                    int partner, pair;
                    bool first;
                    pair_of(col, vdim, a.v_interleaved, partner, pair, first);
                    const float o = os[qi * vdim + partner];
                    float sn, cs;
                    rot_sincos<A>(pos * a.v_freq[pair], sn, cs);
                    v = first ? v * cs + o * sn : v * cs - o * sn;        // the rotation by -pos
                }
                if (a.gate_elems) v *= elem_gate<A>(ldf((const A*)a.gate_elems, tok * a.ld_elems + head * vdim + col));
                ((A*)a.out)[(tok * a.H + head) * vdim + col] = (A)(v * g);
            }
        }
    }
}

// ---------------------------------------------------------------------------------------------------------------
// The same attention on the matrix cores, for bf16 caches with dim and vdim multiples of 16.  A workgroup is 64
// consecutive queries of one (sequence, head): four waves of 16 queries, all walking the same 64-key tiles (K rows and
// V transposed in LDS).  Per tile a wave forms S^T = K Q^T (lane: query lane%16, keys 4 (lane/16) + r of each 16-key
// block), keeps max / sum / weights in fp32, and accumulates O^T = V^T P^T with the weights as the B operand - as two
// bf16 terms, p = hi + lo, so a weight enters the product with 16 bits of mantissa and the sums stay fp32.  Tiles start
// at key 0 and every query has its own running maximum, so the result of a query does not depend on the cut or the batch.
typedef short s16x4 __attribute__((ext_vector_type(4)));
constexpr int MQ = 64, MK = 64;

// EXACT: dim == 16 NKS and vdim == 16 NVT, so no loop below carries a run-time bound (a guarded loop body is a branch, and the
// scheduler then cannot issue the LDS reads of several matrix instructions ahead of them).
// GROUPED (steps in which every sequence brings one query): a workgroup is one (sequence, KV head) and the 16 rows of a
// wave are the query heads that share this KV head, so its keys and values are read once for all of them; the four
// waves split every tile's keys and their partial results are merged at the end (the sums of a row are then formed in
// another order than in the other form: equal within fp32 rounding, not bit for bit).
// (The same split with 16 consecutive queries of one head as the rows was measured for prompts: no faster for one
// 1024-token chunk, 1.7-1.9 x slower from two chunks on, because it stages K/V four times as often.  Not kept.)
// VAR: the plain variant, the one with pooled blocks, softcap and query temperature, or the one with a learned distance bias (none
// carries code of the others).
enum AttnVariant { VAR_PLAIN, VAR_EXT, VAR_BIAS };
template <int NKS, int NVT, bool EXACT, int MODE, int VAR>
__global__ __launch_bounds__(256) void attn_paged_mfma_kernel(AttnArgs a) {
    constexpr bool GROUPED = MODE == 1;                      // rows are the heads of a KV group (one query per sequence)
    constexpr bool EXT = VAR == VAR_EXT, BIAS = VAR == VAR_BIAS;
    constexpr bool SPLIT = MODE != 0;                        // the waves share 16 rows and split the keys
    constexpr int ROWS_Q = MQ;                               // queries per workgroup
    extern __shared__ __attribute__((aligned(16))) unsigned char smem_raw[];
    int seq = -1, q0 = 0, qlen = 0, qbase = 0;
    if (!a.cu_seqlens_q) {                                   // one query per sequence
        if ((int)blockIdx.x < a.batch) {
            seq = qbase = blockIdx.x;
            qlen = 1;
        }
    } else {
        int tile = blockIdx.x;
        for (int b = 0; b < a.batch; ++b) {
            const int lo = a.cu_seqlens_q[b], hi = a.cu_seqlens_q[b + 1];
            const int tiles = (hi - lo + ROWS_Q - 1) / ROWS_Q;
            if (tile < tiles) {
                seq = b;
                q0 = tile * ROWS_Q;
                qlen = hi - lo;
                qbase = lo;
                break;
            }
            tile -= tiles;
        }
    }
    if (seq < 0) return;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, fr = lane & 15, fq = lane >> 4;
    // GROUPED: blockIdx.y counts (KV head, part of its group of heads); the parts of one KV head read the same keys and values
    const int group = GROUPED ? a.H / (a.G * a.kv_split) : a.H / a.G;
    const int kvh = GROUPED ? blockIdx.y / a.kv_split : blockIdx.y / group;
    const int head = GROUPED ? blockIdx.y * group + min(fr, group - 1) : blockIdx.y;       // (GROUPED: this lane's row is a head)
    const int dim = EXACT ? 16 * NKS : a.dim, vdim = EXACT ? 16 * NVT : a.vdim, nks = dim >> 4, nvt = vdim >> 4;
    const int klen = a.context_lens[seq], past = klen - qlen;
    const int nq = GROUPED ? 1 : min(ROWS_Q, qlen - q0);
    const int nrows = GROUPED ? group : nq;                  // real rows of the workgroup's 64
    const int kld = dim + 8, vld = MK + 8;                   // LDS row strides in elements (8-byte aligned rows)
    bf16* ks = reinterpret_cast<bf16*>(smem_raw);            // [MK][dim + 8]
    bf16* vt = ks + MK * kld;                                // [vdim][MK + 8]: V transposed
    // GROUPED: every wave holds the same 16 rows (heads) and takes the 16 keys kt = wave of every 64-key tile, with its own
    // running maximum, sum and output; the four partial results are merged at the end.
    const int qrow = SPLIT ? fr : wave * 16 + fr;            // this lane's row within the workgroup
    const bool qok = qrow < nrows;
    constexpr int NKT = SPLIT ? 1 : 4;                       // 16-key blocks of a tile per wave
    const int qpos = GROUPED ? past : past + q0 + qrow;
    const int last_key = past + q0 + nq - 1;
    const int part = GROUPED ? (int)blockIdx.z : 0, nparts = GROUPED ? a.key_parts : 1;
    float* prow = nullptr;                                   // this workgroup's record among the parts
    if (GROUPED && nparts > 1) prow = a.parts + (((int64_t)seq * gridDim.y + blockIdx.y) * nparts + part) * 16 * (vdim + 2);
    if (last_key < 0 && prow) {                              // a padded row: every part records "no keys", the merge then writes zeros
        if (tid < 16) {
            prow[tid * (vdim + 2) + vdim] = -INFINITY;
            prow[tid * (vdim + 2) + vdim + 1] = 0.f;
        }
        return;
    }
    if (last_key < 0) {                                      // a padded row of a captured step (no keys): zeros, and no address is formed
        for (int i = tid; i < nrows * vdim; i += 256) {
            const int r = i / vdim;
            const int64_t tok = GROUPED ? qbase : qbase + q0 + r;
            const int hd = GROUPED ? (int)blockIdx.y * group + r : (int)blockIdx.y;
            ((bf16*)a.out)[(tok * a.H + hd) * vdim + (i - r * vdim)] = (bf16)0.f;
        }
        return;
    }
    const bf16* qg = (const bf16*)a.q + (int64_t)(qbase + q0 + (qok && !GROUPED ? qrow : 0)) * a.ldq + head * dim;
    // A lane's part of the query row: eight columns of every 32 (K32 products of 32; of a last 16 columns the lanes of the product's first
    // half hold eight each and the others zeros) or, where the size is not a constant, four columns of every 16.  A chain of dependent
    // products keeps to one shape: a product of 16 right behind a product of 32 that it adds to has given wrong sums.  The empty statements make
    // the loads complete here: a load still under way at its first use in the tile loop would put a wait for ALL loads, those of the
    // tile after next included, into every turn.
    constexpr int K32 = EXACT ? (NKS + 1) / 2 : 0, K16 = EXACT ? 0 : NKS;
    constexpr bool HALF = EXACT && NKS % 2 == 1;             // the last product of 32 has 16 columns
    auto kcol = [&](int i) { return i * 32 + (HALF && i == K32 - 1 ? (fq & 1) * 8 : fq * 8); };
    bf16x8 qf32[K32 > 0 ? K32 : 1];
    s16x4 qf16[K16 > 0 ? K16 : 1];
#pragma unroll
    for (int i = 0; i < K32; ++i) {
        qf32[i] = *reinterpret_cast<const bf16x8*>(qg + kcol(i));
        if (HALF && i == K32 - 1 && fq >= 2) qf32[i] = bf16x8{};
    }
#pragma unroll
    for (int i = 0; i < K16; ++i)
        if (i < nks) qf16[i] = *reinterpret_cast<const s16x4*>(qg + i * 16 + fq * 4);
        else qf16[i] = s16x4{0, 0, 0, 0};
#pragma unroll
    for (int i = 0; i < K32; ++i) asm volatile("" : "+v"(qf32[i]));
#pragma unroll
    for (int i = 0; i < K16; ++i) asm volatile("" : "+v"(qf16[i]));
    f32x4 o[NVT];
#pragma unroll
    for (int i = 0; i < NVT; ++i) o[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m_run = -INFINITY, l_run = 0.f;
    if (a.sinks && (!SPLIT || (wave == 0 && part == 0))) {   // the sink is what a row starts from; where waves or parts share a row, one of them holds it
        m_run = a.sinks[head];
        l_run = 1.f;
    }
    const int32_t* table = a.block_tables + (int64_t)seq * a.table_stride;
    const bool wave_idle = !SPLIT && wave * 16 >= nrows;     // no row of this wave is real
    const int wave_last = SPLIT ? last_key : past + q0 + min(wave * 16 + 15, nq - 1);   // keys beyond it are masked for the whole wave
    // A tile's global loads (16 bytes each; K rows as they lie, V rows = value columns over 64 consecutive keys of one page)
    // are issued two tiles ahead into registers, without a condition (past the end: the last tile once more), so that the number of
    // loads under way is the same on every path; what lies beyond the last key is zeroed on the way into LDS.
    constexpr int KCH = (NKS + 1) / 2, VCH = (NVT + 1) / 2;  // 16-byte pieces per lane: MK * dim / 8 / 256
    const int kcols = dim >> 3;
    // The sequence's page ids go to LDS once: a tile's addresses then hang on no other load.  A tile lies within one page
    // (page % MK == 0).
    int* pages_s = reinterpret_cast<int*>(smem_raw + a.pages_offset);
    for (int i = tid; i <= last_key / a.page; i += 256) pages_s[i] = table[i];
    // The heads' bias rows too, each with three entries in front of distance 0 (never seen) and behind the last: a lane's four scores
    // of consecutive keys then read four consecutive entries wherever they start.
    const float* bias_row = nullptr;
    if constexpr (BIAS) {
        float* bias_s = reinterpret_cast<float*>(smem_raw + a.bias_offset);
        const int heads_here = GROUPED ? group : 1;
        const float* src = a.bias + (int64_t)(GROUPED ? (int)blockIdx.y * group : head) * a.bias_len;
        for (int i = tid; i < heads_here * a.bias_ld; i += 256) {
            const int r = i / a.bias_ld, d = i - r * a.bias_ld - 3;
            bias_s[i] = src[(int64_t)r * a.bias_len + min(max(d, 0), a.bias_len - 1)];
        }
        bias_row = bias_s + (GROUPED ? min(fr, group - 1) : 0) * a.bias_ld + 3;
    }
    __syncthreads();
    auto fetch = [&](int k0, bf16x8 (&kpre)[KCH], bf16x8 (&vpre)[VCH]) {
        const int64_t pg = __builtin_amdgcn_readfirstlane(pages_s[k0 / a.page]);     // (uniform)
        const int in_page = k0 % a.page, krow = a.G * dim;
        const bf16* kbase = (const bf16*)a.k_cache + ((pg * a.page + in_page) * a.G + kvh) * dim;
        const bf16* vbase = (const bf16*)a.v_cache + (pg * a.G + kvh) * vdim * a.page + in_page;
#pragma unroll
        for (int j = 0; j < KCH; ++j) {
            const int i = tid + 256 * j;
            kpre[j] = *reinterpret_cast<const bf16x8*>(kbase + (uint32_t)(min(i / kcols, MK - 1) * krow + ((i % kcols) << 3)));
        }
#pragma unroll
        for (int j = 0; j < VCH; ++j) {
            const int i = tid + 256 * j;
            vpre[j] = *reinterpret_cast<const bf16x8*>(vbase + (uint32_t)(min(i >> 3, vdim - 1) * a.page + ((i & 7) << 3)));
        }
    };
    auto store_keys = [&](int rows, bf16x8 (&kpre)[KCH]) {   // rows: those of the tile that hold anything
#pragma unroll
        for (int j = 0; j < KCH; ++j) {
            const int i = tid + 256 * j;
            if ((EXACT && 256 * (j + 1) <= MK * kcols) || i < MK * kcols) {
                const int r = i / kcols, c = (i % kcols) << 3;
                *reinterpret_cast<bf16x8*>(ks + r * kld + c) = r < rows ? kpre[j] : bf16x8{};
            }
        }
    };
    const float slope = a.slopes ? a.slopes[head] : 0.f;
    const float row_scale = EXT ? a.scale * query_temperature(qpos, a.temp_coef, a.temp_every) : a.scale;
    const float cap_in = EXT && a.softcap > 0.f ? 2.8853900817779268f / a.softcap : 0.f;     // tanh(s / cap) = 1 - 2 / (2^(cap_in s) + 1)
    const int nblocks = EXT && a.pool > 0 ? blocks_seen(last_key, a.window, a.pool) : 0, my_blocks = EXT && a.pool > 0 ? blocks_seen(qpos, a.window, a.pool) : 0;
    // keys a row sees: lo_window (or one of the first keep_first) and lo_chunk at least, qpos at most
    const int lo_window = a.window > 0 ? qpos - a.window + 1 : 0, lo_chunk = a.chunk > 0 ? qpos / a.chunk * a.chunk : 0;
    // The tile in LDS, its first key k0 (pooled_tile: its first block) against this wave's queries.
    auto compute = [&](auto pooled_tile, int k0) {
        constexpr bool POOLED = decltype(pooled_tile)::value;
        // (wave-uniform; no barrier below)
        if (wave_idle || (POOLED ? k0 >= blocks_seen(wave_last, a.window, a.pool) : k0 > wave_last)) return;
        f32x4 sc[NKT];
#pragma unroll
        for (int t = 0; t < NKT; ++t) {
            const int kt = SPLIT ? wave : t;
            f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int i = 0; i < K32; ++i) {
                const bf16x8 kf = *reinterpret_cast<const bf16x8*>(ks + (kt * 16 + fr) * kld + kcol(i));
                acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf32[i], acc, 0, 0, 0);
            }
#pragma unroll
            for (int i = 0; i < K16; ++i)
                if (i < nks) {
                    const s16x4 kf = *reinterpret_cast<const s16x4*>(ks + (kt * 16 + fr) * kld + i * 16 + fq * 4);
                    acc = __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(kf, qf16[i], acc, 0, 0, 0);
                }
            sc[t] = acc;
        }
        float mx = -INFINITY;
#pragma unroll
        for (int t = 0; t < NKT; ++t) {
            // (distances beyond the row's last entry take its value; negative ones belong to keys that are not seen)
            const float* brow = nullptr;
            if constexpr (BIAS) brow = bias_row + min(max(qpos - (k0 + (SPLIT ? wave : t) * 16 + fq * 4) - 3, -3), a.bias_len - 1);
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int key = k0 + (SPLIT ? wave : t) * 16 + fq * 4 + r;
                const bool seen = POOLED ? key < my_blocks : (key <= qpos) & ((key >= lo_window) | (key < a.keep_first)) & (key >= lo_chunk);
                const bool ok = qok & seen;
                float s = sc[t][r] * row_scale;
                if (EXT && cap_in > 0.f) s = a.softcap - 2.0f * a.softcap * __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(s * cap_in) + 1.0f);
                if constexpr (BIAS) sc[t][r] = ok ? s + brow[3 - r] : -INFINITY;
                else sc[t][r] = ok ? (POOLED ? s : s - slope * (float)(qpos - key)) : -INFINITY;
                mx = fmaxf(mx, sc[t][r]);
            }
        }
        mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
        mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
        const float m_new = fmaxf(m_run, mx);
        // e^x as the hardware's 2^(x log2 e): fp32 throughout, about 1 ulp
        const float alpha = m_new == -INFINITY ? 1.f : __builtin_amdgcn_exp2f((m_run - m_new) * 1.4426950408889634f);
        float sum = 0.f;
        // The weights as the B operand of products over 32 rows: of two 16-key blocks, once with hi and once with lo - or, where a wave
        // has one block only, of that block's keys twice, with hi and with lo
        constexpr int NP = SPLIT ? 1 : NKT / 2;
        bf16x8 pf[NP], pg[NP];
#pragma unroll
        for (int t = 0; t < NKT; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const float pv = sc[t][r] == -INFINITY ? 0.f : __builtin_amdgcn_exp2f((sc[t][r] - m_new) * 1.4426950408889634f);
                sum += pv;
                const bf16 hi = (bf16)pv;
                const bf16 lo = (bf16)(pv - (float)hi);
                if constexpr (SPLIT) {
                    pf[0][r] = hi;
                    pf[0][4 + r] = lo;
                } else {
                    pf[t / 2][t % 2 * 4 + r] = hi;
                    pg[t / 2][t % 2 * 4 + r] = lo;
                }
            }
        sum += __shfl_xor(sum, 16, 64);
        sum += __shfl_xor(sum, 32, 64);
        l_run = l_run * alpha + sum;
        m_run = m_new;
#pragma unroll
        for (int i = 0; i < NVT; ++i)
            if (EXACT || i < nvt) {
                f32x4 acc = o[i] * alpha;
                const bf16* vrow = vt + (i * 16 + fr) * vld + fq * 4;
#pragma unroll
                for (int t = 0; t < NP; ++t) {
                    const bf16x4 v0 = *reinterpret_cast<const bf16x4*>(vrow + (SPLIT ? wave : 2 * t) * 16);
                    const bf16x4 v1 = SPLIT ? v0 : *reinterpret_cast<const bf16x4*>(vrow + (2 * t + 1) * 16);
                    const bf16x8 vf = __builtin_shufflevector(v0, v1, 0, 1, 2, 3, 4, 5, 6, 7);
                    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[t], acc, 0, 0, 0);
                    if constexpr (!SPLIT) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pg[t], acc, 0, 0, 0);
                }
                o[i] = acc;
            }
    };
    auto tile = [&](int k0, int k_after, bf16x8 (&kpre)[KCH], bf16x8 (&vpre)[VCH]) {
        __syncthreads();
        store_keys(last_key - k0 + 1, kpre);
#pragma unroll
        for (int j = 0; j < VCH; ++j) {
            const int i = tid + 256 * j;
            if ((EXACT && 256 * (j + 1) <= vdim * 8) || i < vdim * 8) {
                const int c = i >> 3, piece = (i & 7) << 3;
                bf16x8 v = vpre[j];
                if (k0 + MK - 1 > last_key) {                // (uniform: only the sequence's last tile)
#pragma unroll
                    for (int e = 0; e < 8; ++e)
                        if (k0 + piece + e > last_key) v[e] = (bf16)0.f;
                }
                *reinterpret_cast<bf16x8*>(vt + c * vld + piece) = v;
            }
        }
        __syncthreads();
        fetch(k_after, kpre, vpre);
        compute(std::false_type{}, k0);
    };
    // Two register sets, two tiles ahead: the loads of the tile after next are issued when a tile has been handed to LDS.
    bf16x8 kA[KCH], vA[VCH], kB[KCH], vB[VCH];
    const TileWalk walk(a.window, a.keep_first, a.chunk, GROUPED ? past : past + q0, MK);
    // (with key parts a workgroup walks the tiles whose number is its own modulo the number of parts)
    auto mine = [&](int k0) { return nparts == 1 || (k0 / MK) % nparts == part; };
    auto next_tile = [&](int k0) {
        int n = walk.next(k0);
        while (n <= last_key && !mine(n)) n = walk.next(n);
        return n;
    };
    int ka = walk.first_end > 0 || walk.win_start == 0 ? 0 : walk.win_start;
    if (!mine(ka)) ka = next_tile(ka);
    int kb = next_tile(ka);
    if (ka > last_key) kb = ka;
    const int k_last = last_key / MK * MK;                   // the tile that holds the last key
    fetch(min(ka, k_last), kA, vA);
    __builtin_amdgcn_sched_barrier(0);                       // (the loads of the first tile stay ahead of the second's)
    if constexpr (EXT) {
        // The tiles of block means come first, one ahead: rows as they lie in their pages, keys in the pieces of a token tile, values in
        // pieces of eight columns of one row (a wave takes 64 rows of the same columns, so its transposed writes into LDS fall side by side).
        auto fetch_pooled = [&](int b0) {
            auto row_of = [&](int r) {
                int pi, row;
                block_place(min(b0 + r, nblocks - 1), a.pool, a.page, pi, row);
                return ((int64_t)pages_s[pi] * a.pool_rows + row) * a.G + kvh;
            };
#pragma unroll
            for (int j = 0; j < KCH; ++j) {
                const int i = tid + 256 * j;
                kB[j] = *reinterpret_cast<const bf16x8*>((const bf16*)a.pk + row_of(min(i / kcols, MK - 1)) * dim + ((i % kcols) << 3));
            }
            const int64_t vrow = row_of(tid & (MK - 1)) * vdim;
#pragma unroll
            for (int j = 0; j < VCH; ++j)
                vB[j] = *reinterpret_cast<const bf16x8*>((const bf16*)a.pv + vrow + min(((tid + 256 * j) / MK) << 3, vdim - 8));
        };
        const int bstep = MK * nparts;
        int b0 = MK * part;
        if (b0 < nblocks) fetch_pooled(b0);
        for (; b0 < nblocks; b0 += bstep) {
            __syncthreads();
            store_keys(nblocks - b0, kB);
#pragma unroll
            for (int j = 0; j < VCH; ++j) {
                const int i = tid + 256 * j, r = i & (MK - 1), c = (i / MK) << 3;
                if (c < vdim) {
#pragma unroll
                    for (int e = 0; e < 8; ++e) vt[(c + e) * vld + r] = r < nblocks - b0 ? vB[j][e] : (bf16)0.f;
                }
            }
            __syncthreads();
            fetch_pooled(b0 + bstep);                        // (past the end: the last block's row once more)
            compute(std::true_type{}, b0);
        }
        __builtin_amdgcn_sched_barrier(0);
    }
    fetch(min(kb, k_last), kB, vB);
    __builtin_amdgcn_sched_barrier(0);
    while (kb <= last_key) {                                 // (one way out: with a second one the waits would count for the shorter path)
        const int ka2 = next_tile(kb), kb2 = next_tile(ka2);
        tile(ka, min(ka2, k_last), kA, vA);
        tile(kb, min(kb2, k_last), kB, vB);
        ka = ka2;
        kb = kb2;
    }
    if (ka <= last_key) tile(ka, ka, kA, vA);
    // epilogue through LDS: [MQ][vdim] fp32, then turn back by the query's position, gate, store
    __syncthreads();
    float* os = reinterpret_cast<float*>(smem_raw);
    if constexpr (SPLIT) {
        // the four waves' partial results [wave][16 rows][vdim] and their (max, sum), merged into the first wave's rows
        float* ml = reinterpret_cast<float*>(smem_raw + a.ml_offset);
#pragma unroll
        for (int i = 0; i < NVT; ++i)
            if (EXACT || i < nvt)
#pragma unroll
                for (int r = 0; r < 4; ++r) os[(wave * 16 + fr) * vdim + i * 16 + fq * 4 + r] = o[i][r];
        if (fq == 0) {
            ml[(wave * 16 + fr) * 2] = m_run;
            ml[(wave * 16 + fr) * 2 + 1] = l_run;
        }
        __syncthreads();
        for (int i = tid; i < nrows * vdim; i += 256) {
            const int r = i / vdim, col = i - r * vdim;
            float big = -INFINITY;
#pragma unroll
            for (int w = 0; w < 4; ++w) big = fmaxf(big, ml[(w * 16 + r) * 2]);
            float num = 0.f, den = 0.f;
#pragma unroll
            for (int w = 0; w < 4; ++w) {
                const float mw = ml[(w * 16 + r) * 2];
                const float f = mw == -INFINITY ? 0.f : __builtin_amdgcn_exp2f((mw - big) * 1.4426950408889634f);
                num += os[(w * 16 + r) * vdim + col] * f;
                den += ml[(w * 16 + r) * 2 + 1] * f;
            }
            if (prow) {                                      // a part's record: the row relative to its maximum, then maximum and sum
                prow[r * (vdim + 2) + col] = num;
                if (col == 0) {
                    prow[r * (vdim + 2) + vdim] = big;
                    prow[r * (vdim + 2) + vdim + 1] = den;
                }
            } else {
                os[i] = den > 0.f ? num / den : 0.f;         // (element i of the first wave's rows: read above by this lane only)
            }
        }
        if (prow) return;                                    // (uniform) the merge launch finishes the rows
    } else {
        const float inv_l = l_run > 0.f ? 1.0f / l_run : 0.f;
#pragma unroll
        for (int i = 0; i < NVT; ++i)
            if (EXACT || i < nvt)
#pragma unroll
                for (int r = 0; r < 4; ++r) os[qrow * vdim + i * 16 + fq * 4 + r] = o[i][r] * inv_l;
    }
    __syncthreads();
    if (!a.v_freq) {                                         // nothing to turn back: eight elements a lane (vdim is a multiple of 16)
        const int pieces = vdim >> 3;
        for (int i = tid; i < nrows * pieces; i += 256) {
            const int r = i / pieces, c = (i - r * pieces) << 3;
            const int64_t tok = GROUPED ? qbase : qbase + q0 + r;
            const int hd = GROUPED ? (int)blockIdx.y * group + r : (int)blockIdx.y;
            const float g = a.gate ? a.gate[tok * a.H + hd] : 1.0f;
            bf16x8 ge, out;
            if (a.gate_elems) ge = *reinterpret_cast<const bf16x8*>((const bf16*)a.gate_elems + tok * a.ld_elems + hd * vdim + c);
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                float v = os[r * vdim + c + e] * g;
                if (a.gate_elems) v *= elem_gate<bf16>((float)ge[e]);
                out[e] = (bf16)v;
            }
            *reinterpret_cast<bf16x8*>((bf16*)a.out + (tok * a.H + hd) * vdim + c) = out;
        }
        return;
    }
    // one lane per rotation pair: both elements, one sine and cosine
    const int half = vdim >> 1;
    for (int i = tid; i < nrows * half; i += 256) {
        const int r = i / half, pair = i - r * half;
        const int c1 = a.v_interleaved ? 2 * pair : pair, c2 = a.v_interleaved ? 2 * pair + 1 : pair + half;
        const int64_t tok = GROUPED ? qbase : qbase + q0 + r;
        const int hd = GROUPED ? (int)blockIdx.y * group + r : (int)blockIdx.y;
        float u = os[r * vdim + c1], v = os[r * vdim + c2];
        if (a.v_freq) {
            float sn, cs;
            sincos_turns((float)(GROUPED ? past : past + q0 + r) * a.v_freq[pair], sn, cs);
            const float u2 = u * cs + v * sn;                // the rotation by -position
            v = v * cs - u * sn;
            u = u2;
        }
        const float g = a.gate ? a.gate[tok * a.H + hd] : 1.0f;
        bf16* dst = (bf16*)a.out + (tok * a.H + hd) * vdim;
        dst[c1] = (bf16)(u * g);
        dst[c2] = (bf16)(v * g);
    }
}

// The rows of the key parts of a (sequence, group of heads) merged: out = gate * sum_p num_p 2^(m_p - m) / sum_p den_p 2^(m_p - m).
__global__ __launch_bounds__(256) void attn_merge_parts_kernel(const float* __restrict__ parts, int nparts, int rows, int vdim, int H, const float* __restrict__ gate,
                                                               const bf16* __restrict__ gate_elems, int64_t ld_elems, bf16* __restrict__ out) {
    // one workgroup per (sequence, group of heads, row): a lane per value column
    const int seq = blockIdx.x, hg = blockIdx.y, r = blockIdx.z;
    const float* base = parts + (((int64_t)seq * gridDim.y + hg) * nparts * 16 + r) * (vdim + 2);
    const int64_t pstride = (int64_t)16 * (vdim + 2);
    float big = -INFINITY;
    for (int p = 0; p < nparts; ++p) big = fmaxf(big, base[p * pstride + vdim]);
    const int hd = hg * rows + r;
    const float g = gate ? gate[(int64_t)seq * H + hd] : 1.0f;
    for (int col = threadIdx.x; col < vdim; col += 256) {
        float num = 0.f, den = 0.f;
        for (int p = 0; p < nparts; ++p) {
            const float* pr = base + p * pstride;
            if (pr[vdim] == -INFINITY) continue;             // a part without keys (its row is not written)
            const float f = __builtin_amdgcn_exp2f((pr[vdim] - big) * 1.4426950408889634f);
            num += pr[col] * f;
            den += pr[vdim + 1] * f;
        }
        float v = den > 0.f ? num / den * g : 0.f;
        if (gate_elems) v *= elem_gate<bf16>((float)gate_elems[seq * ld_elems + (int64_t)hd * vdim + col]);
        out[((int64_t)seq * H + hd) * vdim + col] = (bf16)v;
    }
}

// One query per sequence: the heads of a KV group share a workgroup - up to 16 of them; a larger group is cut into parts.  A launch
// that would leave most of the chip idle is widened: where nothing turns the values back (no v_freq) by giving a sequence's key
// tiles to several workgroups in turn, whose rows a second launch merges (the keys and values are still read once); otherwise by
// cutting the group of heads further (its parts then read the same keys and values at about the same time).  Which workgroup a
// head or a tile falls to enters the result within fp32 rounding only (the order of the merge).
struct OneQueryPlan {
    int split, key_parts;
};
static OneQueryPlan one_query_plan(int64_t batch, int H, int G, bool turned_back) {
    const int group = H / G;
    int split = 1;
    while (group / split > 16 && group % (2 * split) == 0) split *= 2;
    int parts = 1;
    if (!turned_back) {
        while (batch * G * split * parts * 2 <= 256 && parts < 16) parts *= 2;       // (two workgroups a CU measured slower: 53 against 37 us)
    } else {
        while (batch * G * split < 256 && group % (2 * split) == 0 && group / split > 2) split *= 2;
    }
    return OneQueryPlan{split, parts};
}
static size_t one_query_parts_bytes(int64_t batch, int H, int G, int vdim, bool turned_back) {
    const OneQueryPlan pl = one_query_plan(batch, H, G, turned_back);
    return pl.key_parts > 1 ? sizeof(float) * (size_t)batch * G * pl.split * pl.key_parts * 16 * (vdim + 2) : 0;
}

// The bias rows in LDS: at most BIAS_LDS bytes (the caller makes sure that one row fits; a group of heads whose rows do not takes the
// form with one head per workgroup).
constexpr size_t BIAS_LDS = 64 * 1024;
static int bias_row_floats(int bias_len) { return (bias_len + 6) | 1; }      // (odd: the rows of a group start in different banks)

template <int NKS, int NVT, bool EXACT, int VAR>
static void launch_attn_mfma(const AttnArgs& a, int64_t total_q, hipStream_t st) {
    const size_t tiles = sizeof(bf16) * ((size_t)MK * (a.dim + 8) + (size_t)a.vdim * (MK + 8));
    const size_t outs = sizeof(float) * (size_t)MQ * a.vdim;
    AttnArgs b = a;
    b.pages_offset = (int)(((tiles > outs ? tiles : outs) + 15) & ~(size_t)15);
    b.ml_offset = (int)((b.pages_offset + sizeof(int) * (size_t)a.table_stride + 15) & ~(size_t)15);
    b.bias_offset = (int)(b.ml_offset + sizeof(float) * 4 * 16 * 2);
    const int group = a.H / a.G;
    OneQueryPlan pl = one_query_plan(a.batch, a.H, a.G, a.v_freq != nullptr);
    if (!a.parts) pl.key_parts = 1;
    size_t bias_bytes = 0, bias_group_bytes = 0;             // of one head, of the heads of a one-query workgroup
    if (VAR == VAR_BIAS) {
        b.bias_ld = bias_row_floats(a.bias_len);
        bias_bytes = sizeof(float) * (size_t)b.bias_ld;
        bias_group_bytes = bias_bytes * (group / pl.split);
    }
    const bool grouped = total_q == a.batch && group / pl.split <= 16 && bias_group_bytes <= BIAS_LDS && !nvh_switch_on(SW_EXP_A);
    const size_t lds = b.bias_offset + (grouped ? bias_group_bytes : bias_bytes);
    if (lds > 64 * 1024) {                                   // (wide heads or long page tables; a refusal shows as a failed launch)
        (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&attn_paged_mfma_kernel<NKS, NVT, EXACT, 0, VAR>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&attn_paged_mfma_kernel<NKS, NVT, EXACT, 1, VAR>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    }
    if (grouped) {
        b.kv_split = pl.split;
        b.key_parts = pl.key_parts;
        attn_paged_mfma_kernel<NKS, NVT, EXACT, 1, VAR><<<dim3((unsigned)a.batch, (unsigned)(a.G * pl.split), (unsigned)pl.key_parts), 256, lds, st>>>(b);
        if (pl.key_parts > 1)
            attn_merge_parts_kernel<<<dim3((unsigned)a.batch, (unsigned)(a.G * pl.split), (unsigned)(group / pl.split)), 256, 0, st>>>(a.parts, pl.key_parts, group / pl.split, a.vdim, a.H, a.gate,
                                                                                                        (const bf16*)a.gate_elems, a.ld_elems, (bf16*)a.out);
    } else {
        const dim3 grid((unsigned)(total_q / MQ + a.batch), (unsigned)a.H);
        attn_paged_mfma_kernel<NKS, NVT, EXACT, 0, VAR><<<grid, 256, lds, st>>>(b);
    }
}

// Exact instantiations for the head sizes in use (dim/16, vdim/16); any other 16-aligned pair takes a bounded one.
#define NVH_ATTN_EXACT(X) X(1, 1) X(2, 2) X(3, 3) X(4, 4) X(5, 5) X(6, 6) X(8, 8) X(12, 12) X(16, 16) X(2, 4) X(4, 2) X(4, 8) X(8, 4) X(8, 16) X(16, 8) X(12, 8) X(16, 12)
// The variant with pooled blocks, softcap or query temperature: fewer exact pairs.
#define NVH_ATTN_EXACT_EXT(X) X(2, 2) X(4, 4) X(6, 6) X(8, 8) X(16, 16) X(4, 8) X(8, 4) X(8, 16) X(16, 8)
// ... and the one with a learned distance bias.
#define NVH_ATTN_EXACT_BIAS(X) X(2, 2) X(3, 3) X(4, 4) X(5, 5) X(6, 6) X(8, 8) X(12, 12) X(16, 16) X(4, 8) X(8, 4) X(8, 16) X(16, 8)
template <int VAR>
static void dispatch_attn_mfma(const AttnArgs& a, int64_t total_q, hipStream_t st) {
    const int nks = a.dim / 16, nvt = a.vdim / 16;
#define NVH_ATTN_CASE(K, V)                              \
    if (nks == K && nvt == V) {                          \
        launch_attn_mfma<K, V, true, VAR>(a, total_q, st); \
        return;                                          \
    }
    if constexpr (VAR == VAR_EXT) {
        NVH_ATTN_EXACT_EXT(NVH_ATTN_CASE)
    } else if constexpr (VAR == VAR_BIAS) {
        NVH_ATTN_EXACT_BIAS(NVH_ATTN_CASE)
    } else {
        NVH_ATTN_EXACT(NVH_ATTN_CASE)
    }
#undef NVH_ATTN_CASE
    if (nks <= 4 && nvt <= 4) launch_attn_mfma<4, 4, false, VAR>(a, total_q, st);
    else if (nks <= 8 && nvt <= 8) launch_attn_mfma<8, 8, false, VAR>(a, total_q, st);
    else launch_attn_mfma<16, 16, false, VAR>(a, total_q, st);
}

// The means of the blocks that were filled by this step, one block per workgroup (blockIdx.x; several workgroups, blockIdx.y, share its
// columns): block b of a sequence is due when its last position is among the step's.  Rows are read from the cache as it holds them.
struct PoolArgs {
    const void *k_cache, *v_cache;
    const int32_t *cu_seqlens_q, *context_lens, *block_tables;
    int64_t table_stride;
    int batch, page, G, dim, vdim, pool, pool_rows;
    void *pk, *pv;
};

// The mean of column i (of n) over block b of a sequence, from the rows that the cache holds (values: transposed within a page).
template <typename A>
__device__ __forceinline__ void block_mean_column(const A* cache, A* pooled, int i, int n, bool transposed, int b, int pool, int page, int pool_rows, const int32_t* table) {
    const int p0 = b * pool;
    int pi = p0 / page;
    const int off0 = p0 - pi * page;
    float sum = 0.f;
    // (a block may lie across pages: page by page, each a plain run of rows)
    for (int done = 0, off = off0; done < pool; off = 0, ++pi) {
        const int n_here = min(pool - done, page - off);
        const int64_t pg = table[pi];
        const A* src = transposed ? cache + (pg * n + i) * page + off : cache + (pg * page + off) * n + i;
        const int64_t step = transposed ? 1 : n;
#pragma unroll 8
        for (int j = 0; j < n_here; ++j) sum += ldf(src, j * step);
        done += n_here;
    }
    int pi_out, row;
    block_place(b, pool, page, pi_out, row);
    pooled[((int64_t)table[pi_out] * pool_rows + row) * n + i] = (A)(sum / (float)pool);
}

template <typename A>
__global__ __launch_bounds__(256) void attn_pool_blocks_kernel(PoolArgs a) {
    int seq = -1, b = 0;
    if (!a.cu_seqlens_q) {                                   // one token per sequence: its block is due when it is the block's last
        const int len = a.context_lens[blockIdx.x];
        if (len > 0 && len % a.pool == 0) {
            seq = blockIdx.x;
            b = len / a.pool - 1;
        }
    } else {
        int at = blockIdx.x;
        for (int i = 0; i < a.batch; ++i) {
            const int len = a.context_lens[i], past = len - (a.cu_seqlens_q[i + 1] - a.cu_seqlens_q[i]);
            const int first = past / a.pool, due = len / a.pool - first;
            if (at < due) {
                seq = i;
                b = first + at;
                break;
            }
            at -= due;
        }
    }
    if (seq < 0) return;                                     // (uniform over the workgroup)
    const int i = blockIdx.y * 256 + threadIdx.x, nk = a.G * a.dim, nv = a.G * a.vdim;
    if (i >= nk + nv) return;
    const int32_t* table = a.block_tables + (int64_t)seq * a.table_stride;
    if (i < nk) block_mean_column((const A*)a.k_cache, (A*)a.pk, i, nk, false, b, a.pool, a.page, a.pool_rows, table);
    else block_mean_column((const A*)a.v_cache, (A*)a.pv, i - nk, nv, true, b, a.pool, a.page, a.pool_rows, table);
}

// Keys and values to their cache slots: a workgroup takes KT tokens of the step and KC columns of both rows.  Keys pass as they lie;
// values turn in LDS, so that tokens which lie side by side in a page leave in one piece (64 of them: a whole cache line, which no
// other workgroup then touches).  With `pool` (one token per sequence: row t of the tables is token t's) the columns' means of the
// blocks that these tokens complete follow in the same launch.
constexpr int KT = 64;
struct KvStoreArgs {
    const void *k, *v;         // [T, ld]: nk and nv columns
    int64_t ld;
    const void* v_mix;         // one number l, or null: the value is (1 - l) v + l v_first
    const void* v_first;       // [T, ld_first]
    int64_t ld_first;
    void *k_cache, *v_cache;
    const int32_t* slot_mapping;
    int T, page, nk, nv, vec_k, vec_v, vec_first;
    int pool, pool_rows;
    const int64_t* positions;
    const int32_t* block_tables;
    int64_t table_stride;
    void *pk, *pv;
};

template <typename A, int KC>
__global__ __launch_bounds__(256) void attn_kv_store_kernel(KvStoreArgs a) {
    __shared__ float tile[KT][KC + 1];
    __shared__ int slots[KT], due_tok[KT], due_block[KT], due_count;             // due: the tokens that complete a block, and the block
    const int tid = threadIdx.x, t0 = blockIdx.x * KT, c0 = blockIdx.y * KC;
    if (tid < KT) {
        const int t = t0 + tid;
        const int slot = t < a.T ? a.slot_mapping[t] : -1;
        slots[tid] = slot;
        if (a.pool) {                                        // (the first KT = 64 lanes are one wave)
            const int len = slot >= 0 ? (int)a.positions[t] + 1 : 0;
            const bool due = slot >= 0 && len % a.pool == 0;
            const unsigned long long mask = __ballot(due);
            if (due) {
                const int at = __popcll(mask & ((1ull << tid) - 1));
                due_tok[at] = t;
                due_block[at] = len / a.pool - 1;
            }
            if (tid == 0) due_count = __popcll(mask);
        }
    }
    __syncthreads();
    const float lam = a.v_mix ? ldf((const A*)a.v_mix, 0) : 0.f;
    constexpr int CP = KC / 8;                               // pieces of eight columns per token
#pragma unroll
    for (int i = tid; i < KT * CP; i += 256) {
        const int r = i / CP, c = c0 + (i % CP) * 8, slot = slots[r];
        const int64_t t = t0 + r;
        if (slot < 0) continue;
        float x[8];
        if (c < a.nk) {
            nvh_load8((const A*)a.k + t * a.ld, c, a.nk - c, a.vec_k, x);
            A* dst = (A*)a.k_cache + (int64_t)slot * a.nk + c;
            A out[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) out[e] = (A)x[e];
            if (a.vec_k) {
                __builtin_memcpy(__builtin_assume_aligned(dst, 16), out, sizeof(out));
            } else {
                for (int e = 0; e < min(8, a.nk - c); ++e) dst[e] = out[e];
            }
        }
        if (c < a.nv) {
            nvh_load8((const A*)a.v + t * a.ld, c, a.nv - c, a.vec_v, x);
            if (a.v_mix) {
                float f[8];
                nvh_load8((const A*)a.v_first + t * a.ld_first, c, a.nv - c, a.vec_first, f);
#pragma unroll
                for (int e = 0; e < 8; ++e) x[e] = (1.0f - lam) * x[e] + lam * f[e];
            }
#pragma unroll
            for (int e = 0; e < 8; ++e) tile[r][c - c0 + e] = x[e];
        }
    }
    __syncthreads();
    {
        const int r = tid % KT, slot = slots[r];             // (256 is a multiple of KT)
        if (slot >= 0) {
            A* dst = (A*)a.v_cache + (int64_t)(slot / a.page) * a.page * a.nv + slot % a.page;
#pragma unroll
            for (int c = tid / KT; c < KC; c += 256 / KT)
                if (c0 + c < a.nv) dst[(int64_t)(c0 + c) * a.page] = (A)tile[r][c];
        }
    }
    if (a.pool == 0) return;
    __syncthreads();                                         // (the workgroup's own stores are among what the means read)
    for (int i = tid; i < due_count * 2 * KC; i += 256) {
        const int at = i / (2 * KC), c = c0 + i % KC;
        const int32_t* table = a.block_tables + (int64_t)due_tok[at] * a.table_stride;
        if (i % (2 * KC) < KC) {
            if (c < a.nk) block_mean_column((const A*)a.k_cache, (A*)a.pk, c, a.nk, false, due_block[at], a.pool, a.page, a.pool_rows, table);
        } else {
            if (c < a.nv) block_mean_column((const A*)a.v_cache, (A*)a.pv, c, a.nv, true, due_block[at], a.pool, a.page, a.pool_rows, table);
        }
    }
}

template <typename A, int KC>
static void launch_kv_store(const KvStoreArgs& a, hipStream_t st) {
    attn_kv_store_kernel<A, KC><<<dim3((unsigned)nvh_cdiv(a.T, KT), (unsigned)nvh_cdiv(a.nk > a.nv ? a.nk : a.nv, KC)), 256, 0, st>>>(a);
}

}  // namespace

extern "C" int32_t nvh_attn_rotary_prep(const void* proj, int64_t proj_row_stride, const void* q_norm_weight, const void* k_norm_weight,
                                        float eps, const int64_t* positions, const float* qk_freq, float qk_mag, int64_t rot_dims,
                                        int32_t qk_interleaved, const float* v_freq, int32_t v_interleaved, void* q_out, float* gate_out,
                                        void* k_cache, void* v_cache, const int32_t* slot_mapping, int64_t page, int64_t num_tokens,
                                        int64_t num_q_heads, int64_t num_kv_heads, int64_t dim, int64_t vdim, int32_t norm_per_head, int32_t act_f32,
                                        nvh_stream_t stream) {
    NVH_REQUIRE(proj && positions && q_out && !q_norm_weight == !k_norm_weight, NVH_EINVAL, "nvh_attn_rotary_prep: null pointer");
    NVH_REQUIRE(num_q_heads > 0 && num_kv_heads > 0 && dim > 0 && vdim > 0 && num_tokens >= 0 && page > 0, NVH_EINVAL, "nvh_attn_rotary_prep: bad sizes");
    NVH_REQUIRE(rot_dims >= 0 && rot_dims <= dim && rot_dims % 2 == 0 && (rot_dims == 0 || qk_freq), NVH_EINVAL,
                "nvh_attn_rotary_prep: rot_dims %ld does not fit dim %ld", (long)rot_dims, (long)dim);
    NVH_REQUIRE(!v_freq || vdim % 2 == 0, NVH_EINVAL, "nvh_attn_rotary_prep: rotated values need an even vdim");
    NVH_REQUIRE(proj_row_stride >= (num_q_heads + num_kv_heads) * dim + num_kv_heads * vdim + (gate_out ? num_q_heads : 0), NVH_EINVAL,
                "nvh_attn_rotary_prep: projection row too short");
    if (num_tokens == 0) return NVH_OK;
    PrepArgs a{proj, proj_row_stride, q_norm_weight, k_norm_weight, norm_per_head, eps, positions, qk_freq, qk_mag, (int)rot_dims, qk_interleaved,
               v_freq, v_interleaved, q_out, gate_out, k_cache, v_cache, slot_mapping, (int)num_q_heads, (int)num_kv_heads, (int)dim, (int)vdim, (int)page};
    hipStream_t st = (hipStream_t)stream;
    const size_t lds = norm_per_head ? sizeof(float) * (size_t)(num_q_heads + num_kv_heads) : 0;
    NVH_REQUIRE(lds <= 32 * 1024, NVH_ENOSYS, "nvh_attn_rotary_prep: %ld heads above the per-head norm's limit", (long)(num_q_heads + num_kv_heads));
    if (act_f32) attn_rotary_prep_kernel<float><<<dim3((unsigned)num_tokens), 256, lds, st>>>(a);
    else attn_rotary_prep_kernel<bf16><<<dim3((unsigned)num_tokens), 256, lds, st>>>(a);
    NVH_CHECK_LAUNCH("nvh_attn_rotary_prep");
    return NVH_OK;
}

extern "C" int32_t nvh_attn_paged_any(const void* q, int64_t q_row_stride, const void* k_cache, const void* v_cache, const int32_t* cu_seqlens_q,
                                      const int32_t* context_lens, const int32_t* block_tables, int64_t table_stride, int64_t batch,
                                      int64_t total_q, int64_t page, int64_t num_q_heads, int64_t num_kv_heads, int64_t dim, int64_t vdim,
                                      float scale, const float* gate, const void* gate_elems, int64_t gate_elems_stride, const float* v_freq, int32_t v_interleaved,
                                      const float* slopes, const float* bias, int64_t bias_len, int64_t window, int64_t keep_first, int64_t chunk, const float* sinks, float softcap, float temp_coef,
                                      int64_t temp_every, int64_t pool, int64_t pool_rows, const void* pooled_k, const void* pooled_v, void* out,
                                      float* parts_ws, int64_t parts_ws_bytes, int32_t act_f32, nvh_stream_t stream) {
    NVH_REQUIRE(!bias || (bias_len > 0 && bias_len < (1 << 20) && pool == 0), NVH_EINVAL, "nvh_attn_paged_any: a distance bias has a row per head and no pooled blocks beside it");
    NVH_REQUIRE(!gate_elems || gate_elems_stride >= num_q_heads * vdim, NVH_EINVAL, "nvh_attn_paged_any: gate row too short");
    NVH_REQUIRE(softcap >= 0.f && temp_every >= 0 && temp_every < (1 << 30), NVH_EINVAL, "nvh_attn_paged_any: bad softcap or query temperature");
    NVH_REQUIRE(pool >= 0 && pool < (1 << 30) && (pool == 0 || (pooled_k && pooled_v && pool_rows >= nvh_cdiv(page, pool) && window > 0 && keep_first == 0 && chunk == 0 && !slopes)),
                NVH_EINVAL, "nvh_attn_paged_any: pooled blocks go with a plain window and caches of their means");
    NVH_REQUIRE(window >= 0 && keep_first >= 0 && window < (1 << 30) && keep_first < (1 << 30), NVH_EINVAL, "nvh_attn_paged_any: bad window");
    NVH_REQUIRE(chunk >= 0 && chunk < (1 << 30), NVH_EINVAL, "nvh_attn_paged_any: bad chunk");
    NVH_REQUIRE(q && k_cache && v_cache && context_lens && block_tables && out, NVH_EINVAL, "nvh_attn_paged_any: null pointer");
    NVH_REQUIRE(batch >= 0 && total_q >= 0 && page > 0 && num_q_heads > 0 && num_kv_heads > 0 && num_q_heads % num_kv_heads == 0 && dim > 0 && vdim > 0,
                NVH_EINVAL, "nvh_attn_paged_any: bad sizes");
    NVH_REQUIRE(vdim <= 16 * AVC_MAX, NVH_ENOSYS, "nvh_attn_paged_any: vdim %ld above %d", (long)vdim, 16 * AVC_MAX);
    NVH_REQUIRE(!v_freq || vdim % 2 == 0, NVH_EINVAL, "nvh_attn_paged_any: rotated values need an even vdim");
    const size_t lds = sizeof(float) * (size_t)(AQ * dim + AK * (dim + 1) + AK * (vdim + 1) + AQ * AK);
    NVH_REQUIRE(lds <= 160 * 1024, NVH_ENOSYS, "nvh_attn_paged_any: dim %ld + vdim %ld need %zu bytes of LDS", (long)dim, (long)vdim, lds);
    if (lds > 64 * 1024) {                                   // beyond the default limit of dynamic LDS: raise it for both forms (gfx950: 160 KB per workgroup)
        const hipError_t e1 = hipFuncSetAttribute(reinterpret_cast<const void*>(&attn_paged_any_kernel<float, 16>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        const hipError_t e2 = hipFuncSetAttribute(reinterpret_cast<const void*>(&attn_paged_any_kernel<bf16, 16>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        const hipError_t e3 = hipFuncSetAttribute(reinterpret_cast<const void*>(&attn_paged_any_kernel<float, 32>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        const hipError_t e4 = hipFuncSetAttribute(reinterpret_cast<const void*>(&attn_paged_any_kernel<bf16, 32>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        NVH_REQUIRE(e1 == hipSuccess && e2 == hipSuccess && e3 == hipSuccess && e4 == hipSuccess, NVH_ENOSYS, "nvh_attn_paged_any: %zu bytes of LDS refused", lds);
    }
    if (batch == 0 || total_q == 0) return NVH_OK;
    NVH_REQUIRE(q_row_stride >= num_q_heads * dim, NVH_EINVAL, "nvh_attn_paged_any: query row too short");
    AttnArgs a{q, q_row_stride, k_cache, v_cache, cu_seqlens_q, context_lens, block_tables, table_stride, (int)batch, (int)page, (int)num_q_heads,
               (int)num_kv_heads, (int)dim, (int)vdim, scale, gate, v_freq, v_interleaved, out, gate_elems, gate_elems_stride, slopes, bias, (int)bias_len, (int)window, (int)keep_first, (int)chunk, sinks, softcap, temp_coef, (int)temp_every, (int)pool, (int)pool_rows,
               pooled_k, pooled_v, 0, 0, 0, 0, 1, 1, nullptr};
    // at most ceil(len / AQ) tiles per sequence: total_q / AQ + batch bounds their number (surplus workgroups exit)
    const dim3 grid((unsigned)(total_q / AQ + batch), (unsigned)num_q_heads);
    hipStream_t st = (hipStream_t)stream;
    // bf16 with 16-aligned head sizes: the matrix-core kernel (the choice depends on the sizes and the type only)
    const bool mfma = !act_f32 && dim % 16 == 0 && vdim % 16 == 0 && dim <= 256 && vdim <= 256 && page % MK == 0 && q_row_stride % 8 == 0 && nvh_aligned16(q) && nvh_aligned16(k_cache) &&
                      nvh_aligned16(v_cache) && (pool == 0 || (nvh_aligned16(pooled_k) && nvh_aligned16(pooled_v))) && nvh_aligned16(out) &&
                      (!gate_elems || (gate_elems_stride % 8 == 0 && nvh_aligned16(gate_elems) && !v_freq)) &&
                      (!bias || (sizeof(float) * (size_t)bias_row_floats((int)bias_len) <= BIAS_LDS && softcap == 0.f && temp_every == 0 && !slopes)) && !nvh_switch_on(SW_ATTN_ANY_NO_MFMA);
    if (mfma) {
        // (scratch for the key parts of the one-query form: used when it is given and large enough, see nvh_attn_paged_any_parts_bytes)
        const size_t need = total_q == batch ? one_query_parts_bytes(batch, (int)num_q_heads, (int)num_kv_heads, (int)vdim, v_freq != nullptr) : 0;
        if (parts_ws && need && (size_t)parts_ws_bytes >= need) a.parts = parts_ws;
        if (bias) dispatch_attn_mfma<VAR_BIAS>(a, total_q, st);
        else if (pool > 0 || softcap > 0.f || temp_every > 0) dispatch_attn_mfma<VAR_EXT>(a, total_q, st);
        else dispatch_attn_mfma<VAR_PLAIN>(a, total_q, st);
    } else if (vdim <= 256) {                                // (16 value columns a lane; the choice depends on the size alone)
        if (act_f32) attn_paged_any_kernel<float, 16><<<grid, 256, lds, st>>>(a);
        else attn_paged_any_kernel<bf16, 16><<<grid, 256, lds, st>>>(a);
    } else {
        if (act_f32) attn_paged_any_kernel<float, 32><<<grid, 256, lds, st>>>(a);
        else attn_paged_any_kernel<bf16, 32><<<grid, 256, lds, st>>>(a);
    }
    NVH_CHECK_LAUNCH("nvh_attn_paged_any");
    return NVH_OK;
}

extern "C" int64_t nvh_attn_paged_any_parts_bytes(int64_t batch, int64_t total_q, int64_t num_q_heads, int64_t num_kv_heads, int64_t dim, int64_t vdim,
                                                  int64_t page, int32_t turned_back, int32_t act_f32) {
    if (batch <= 0 || total_q != batch || act_f32 || num_kv_heads <= 0 || num_q_heads % num_kv_heads) return 0;
    if (dim % 16 || vdim % 16 || dim > 256 || vdim > 256 || page % MK) return 0;           // (the matrix-core kernel's sizes)
    return (int64_t)one_query_parts_bytes(batch, (int)num_q_heads, (int)num_kv_heads, (int)vdim, turned_back != 0);
}

extern "C" int32_t nvh_attn_pool_blocks(const void* k_cache, const void* v_cache, const int32_t* cu_seqlens_q, const int32_t* context_lens,
                                        const int32_t* block_tables, int64_t table_stride, int64_t batch, int64_t total_q, int64_t page, int64_t num_kv_heads,
                                        int64_t dim, int64_t vdim, int64_t pool, int64_t pool_rows, void* pooled_k, void* pooled_v, int32_t act_f32,
                                        nvh_stream_t stream) {
    NVH_REQUIRE(k_cache && v_cache && context_lens && block_tables && pooled_k && pooled_v, NVH_EINVAL, "nvh_attn_pool_blocks: null pointer");
    NVH_REQUIRE(batch >= 0 && total_q >= 0 && page > 0 && num_kv_heads > 0 && dim > 0 && vdim > 0 && pool > 0 && pool < (1 << 30) && pool_rows >= nvh_cdiv(page, pool) &&
                    (cu_seqlens_q || total_q == batch),
                NVH_EINVAL, "nvh_attn_pool_blocks: bad sizes");
    if (batch == 0 || total_q == 0) return NVH_OK;
    const PoolArgs a{k_cache, v_cache, cu_seqlens_q, context_lens, block_tables, table_stride, (int)batch, (int)page, (int)num_kv_heads, (int)dim, (int)vdim, (int)pool,
                     (int)pool_rows, pooled_k, pooled_v};
    // a sequence's n tokens fill at most n / pool + 1 blocks (surplus workgroups exit)
    const dim3 grid((unsigned)(cu_seqlens_q ? total_q / pool + batch : batch), (unsigned)nvh_cdiv(num_kv_heads * (dim + vdim), 256));
    hipStream_t st = (hipStream_t)stream;
    if (act_f32) attn_pool_blocks_kernel<float><<<grid, 256, 0, st>>>(a);
    else attn_pool_blocks_kernel<bf16><<<grid, 256, 0, st>>>(a);
    NVH_CHECK_LAUNCH("nvh_attn_pool_blocks");
    return NVH_OK;
}

extern "C" int32_t nvh_attn_kv_store(const void* k, const void* v, int64_t row_stride, const void* v_mix, const void* v_first, int64_t v_first_stride, void* k_cache,
                                     void* v_cache, const int32_t* slot_mapping, int64_t page, int64_t num_tokens, int64_t num_kv_heads, int64_t dim, int64_t vdim,
                                     int64_t pool, int64_t pool_rows, const int64_t* positions, const int32_t* block_tables, int64_t table_stride, void* pooled_k,
                                     void* pooled_v, int32_t act_f32, nvh_stream_t stream) {
    NVH_REQUIRE(k && v && k_cache && v_cache && slot_mapping, NVH_EINVAL, "nvh_attn_kv_store: null pointer");
    NVH_REQUIRE(num_tokens >= 0 && num_tokens < (1 << 30) && page > 0 && num_kv_heads > 0 && dim > 0 && vdim > 0 && row_stride >= num_kv_heads * dim &&
                    row_stride >= num_kv_heads * vdim && num_kv_heads * (dim + vdim) < (1 << 30),
                NVH_EINVAL, "nvh_attn_kv_store: bad sizes");
    NVH_REQUIRE(!v_mix || (v_first && v_first_stride >= num_kv_heads * vdim), NVH_EINVAL, "nvh_attn_kv_store: values to mix in are missing or too short");
    NVH_REQUIRE(pool >= 0 && pool < (1 << 30) && (pool == 0 || (positions && block_tables && pooled_k && pooled_v && pool_rows >= nvh_cdiv(page, pool))), NVH_EINVAL,
                "nvh_attn_kv_store: bad pooled blocks");
    if (num_tokens == 0) return NVH_OK;
    const int64_t nk = num_kv_heads * dim, nv = num_kv_heads * vdim;
    const bool rows8 = row_stride % 8 == 0;
    const KvStoreArgs a{k, v, row_stride, v_mix, v_first, v_first_stride, k_cache, v_cache, slot_mapping, (int)num_tokens, (int)page, (int)nk, (int)nv,
                        rows8 && nk % 8 == 0 && nvh_aligned16(k) && nvh_aligned16(k_cache), rows8 && nvh_aligned16(v), v_first_stride % 8 == 0 && nvh_aligned16(v_first),
                        (int)pool, (int)pool_rows, positions, block_tables, table_stride, pooled_k, pooled_v};
    hipStream_t st = (hipStream_t)stream;
    // Narrower column tiles where the tokens alone do not fill the chip.  (64 sequences of one token, 1024 columns, us: 64 tokens x 32
    // columns 7.7, 16 x 32 12.2, 4 x 128 12.8, 4 x 64 17.1, 1 x 256 18.7: a wave that writes one column of many pages beats many that
    // write many columns of few.)
    if (num_tokens >= 512) {
        if (act_f32) launch_kv_store<float, 64>(a, st);
        else launch_kv_store<bf16, 64>(a, st);
    } else {
        if (act_f32) launch_kv_store<float, 32>(a, st);
        else launch_kv_store<bf16, 32>(a, st);
    }
    NVH_CHECK_LAUNCH("nvh_attn_kv_store");
    return NVH_OK;
}
