// Row-wise operators around a residual stream that is kept in several copies (hyper-connections: "Hyper-Connections", Zhu et al., in
// the static form - one learned number per stream pair, none from the input):
//   nvh_embedding_bigram_stream   token row + row of a hashed (previous token, token) table + position row -> every copy of the
//                                 fp32 stream; the previous token of a portion's first token comes from the sequence's state slot, which
//                                 then keeps the portion's last token
//   nvh_hyper_norm                the close of a sublayer and the norm that opens the next one, per token:
//                                     x_t <- sum_s mix[s, t] x_s + out[t] y   (all t at once),   u = sum_t in[t] x_t,   h = norm(u)
//                                 where y is a row of the activation type, an fp32 row, or the weighted sum of the token's experts'
//                                 rows plus a shared expert's row, formed on the way
// Streams, coefficients, sums and norms are fp32; h leaves in the activation type A.
#include "common.h"

namespace {

struct BigramArgs {
    const int64_t *ids, *positions;
    const void *table, *pos_table, *bigram;        // [vocab, dim], [max_pos, dim] or null, [buckets + 1, dim] or null
    int64_t vocab, max_pos, buckets, mul_prev, mul_cur;
    int32_t* last;                                 // [slots]: the last token of every sequence (with bigram)
    const int32_t *slots, *cu_seqlens_q, *context_lens;
    float* x;                                      // [T, streams, dim]
    int batch, streams, dim, vec;
};

template <typename A>
__device__ __forceinline__ f32x4 load4(const A* p) {
    if constexpr (sizeof(A) == 4) {
        return *reinterpret_cast<const f32x4*>(p);
    } else {
        const bf16x4 v = *reinterpret_cast<const bf16x4*>(p);
        return f32x4{(float)v[0], (float)v[1], (float)v[2], (float)v[3]};
    }
}

template <typename A>
__global__ __launch_bounds__(256) void embedding_bigram_stream_kernel(BigramArgs p) {
    const int64_t t = blockIdx.x, id = p.ids[t], pos = p.pos_table ? p.positions[t] : -1;
    const A* e = id >= 0 && id < p.vocab ? (const A*)p.table + id * p.dim : nullptr;
    const A* q = pos >= 0 && pos < p.max_pos ? (const A*)p.pos_table + pos * p.dim : nullptr;
    const A* b = nullptr;
    if (p.bigram) {
        const int seq = seq_of_token(p.cu_seqlens_q, p.batch, t);
        const int lo = p.cu_seqlens_q ? p.cu_seqlens_q[seq] : seq, hi = p.cu_seqlens_q ? p.cu_seqlens_q[seq + 1] : seq + 1;
        const int slot = p.slots[seq];
        const bool first = t == lo, carried = slot >= 0 && p.context_lens[seq] != hi - lo;
        int64_t row = p.buckets;                             // (a sequence's first token has a row of its own, the last one)
        if (!first || carried) {
            const int64_t prev = first ? p.last[slot] : p.ids[t - 1];
            row = (prev * p.mul_prev + id * p.mul_cur) % p.buckets;
            row = row < 0 ? row + p.buckets : row;           // (ids of padded rows may be anything)
        }
        b = (const A*)p.bigram + row * p.dim;
        // The workgroup of a portion's first token is the only one that reads the slot: it also writes it, when all its lanes have read.
        __syncthreads();
        if (first && slot >= 0 && threadIdx.x == 0) p.last[slot] = (int32_t)p.ids[hi - 1];
    }
    float* x = p.x + t * p.streams * p.dim;
    if (p.vec) {
        for (int c = threadIdx.x * 4; c < p.dim; c += 1024) {
            f32x4 v = {0.f, 0.f, 0.f, 0.f};
            if (e) v = load4(e + c);
            if (b) v += load4(b + c);
            if (q) v += load4(q + c);
            for (int s = 0; s < p.streams; ++s) *reinterpret_cast<f32x4*>(x + (int64_t)s * p.dim + c) = v;
        }
        return;
    }
    for (int c = threadIdx.x; c < p.dim; c += 256) {
        float v = e ? (float)e[c] : 0.f;
        if (b) v += (float)b[c];
        if (q) v += (float)q[c];
        for (int s = 0; s < p.streams; ++s) x[(int64_t)s * p.dim + c] = v;
    }
}

__device__ __forceinline__ float block_sum4(float v, float* scratch) {
    v = wave_sum(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) scratch[threadIdx.x >> 6] = v;
    __syncthreads();
    return scratch[0] + scratch[1] + scratch[2] + scratch[3];
}

constexpr int STREAMS_MAX = 16;

struct HyperArgs {
    float* x;                  // [T, S, dim]
    int S, dim;
    const float *mix, *out_w;  // [S, S] (from, to), [S]; mix null: the streams stay as they are (and are not written)
    const float* in_w;         // [S]; null: ones (the plain sum)
    const void* a;             // y: rows of type A, or null
    int64_t a_stride;
    const float* c32;          // y: fp32 rows added to it, or null
    int64_t c32_stride;
    const void* pairs;         // y: + sum over r < top of weights[t, r] pairs[pos_of_pair[t, r]] (experts' results), or null
    int64_t pairs_stride;
    const int32_t* pos_of_pair;
    const float* weights;
    int top;
    int norm;                  // 0: none (no h), 1: layer norm, 2: RMS norm
    const void *nw, *nb;
    float eps;
    void* h;
    int64_t h_stride;
};

// NS streams (constant), four columns a lane and access, R pieces of 1024 columns: u stays in registers between the passes of the norm.
template <typename A, int NS, int R>
__global__ __launch_bounds__(256) void hyper_norm_vec_kernel(HyperArgs p) {
    __shared__ float red[8];
    const int64_t row = blockIdx.x;
    const int dim = p.dim;
    float* xr = p.x + row * NS * dim;
    float mix[NS][NS], ow[NS], iw[NS];
#pragma unroll
    for (int s = 0; s < NS; ++s) {
#pragma unroll
        for (int t = 0; t < NS; ++t) mix[s][t] = p.mix ? p.mix[s * NS + t] : 0.f;
        ow[s] = p.mix ? p.out_w[s] : 0.f;
        iw[s] = p.in_w ? p.in_w[s] : 1.f;
    }
    f32x4 u[R];
    float sum = 0.f;
#pragma unroll
    for (int j = 0; j < R; ++j) {
        const int c = (threadIdx.x + 256 * j) * 4;
        u[j] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (c >= dim) continue;
        f32x4 x[NS];
#pragma unroll
        for (int s = 0; s < NS; ++s) x[s] = *reinterpret_cast<const f32x4*>(xr + s * dim + c);
        if (p.mix) {
            f32x4 y = {0.f, 0.f, 0.f, 0.f};
            if (p.pairs) {
                for (int r = 0; r < p.top; ++r) {
                    const int pos = p.pos_of_pair[row * p.top + r];
                    const float w = p.weights[row * p.top + r];
                    if (pos >= 0) {
                        const f32x4 v = load4((const A*)p.pairs + (int64_t)pos * p.pairs_stride + c);
#pragma unroll
                        for (int e = 0; e < 4; ++e) y[e] = __builtin_fmaf(w, v[e], y[e]);
                    }
                }
            }
            if (p.a) y += load4((const A*)p.a + row * p.a_stride + c);
            if (p.c32) y += *reinterpret_cast<const f32x4*>(p.c32 + row * p.c32_stride + c);
            f32x4 nx[NS];
#pragma unroll
            for (int t = 0; t < NS; ++t)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    float v = ow[t] * y[e];
#pragma unroll
                    for (int s = 0; s < NS; ++s) v = __builtin_fmaf(mix[s][t], x[s][e], v);
                    nx[t][e] = v;
                }
#pragma unroll
            for (int t = 0; t < NS; ++t) {
                x[t] = nx[t];
                *reinterpret_cast<f32x4*>(xr + t * dim + c) = nx[t];
            }
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) {
#pragma unroll
            for (int s = 0; s < NS; ++s) u[j][e] = __builtin_fmaf(iw[s], x[s][e], u[j][e]);
            sum += u[j][e];
        }
    }
    if (p.norm == 0) return;
    const float mean = p.norm == 1 ? block_sum4(sum, red) / (float)dim : 0.f;
    float sq = 0.f;
#pragma unroll
    for (int j = 0; j < R; ++j)
        if ((threadIdx.x + 256 * j) * 4 < (unsigned)dim)
#pragma unroll
            for (int e = 0; e < 4; ++e) sq += (u[j][e] - mean) * (u[j][e] - mean);
    const float inv = 1.0f / sqrtf(block_sum4(sq, red + 4) / (float)dim + p.eps);
    A* h = (A*)p.h + row * p.h_stride;
#pragma unroll
    for (int j = 0; j < R; ++j) {
        const int c = (threadIdx.x + 256 * j) * 4;
        if (c >= dim) continue;
        const f32x4 w = load4((const A*)p.nw + c);
        const f32x4 b = p.nb ? load4((const A*)p.nb + c) : f32x4{0.f, 0.f, 0.f, 0.f};
        A out[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) out[e] = (A)((u[j][e] - mean) * inv * w[e] + b[e]);
        __builtin_memcpy(__builtin_assume_aligned(h + c, 4 * sizeof(A)), out, sizeof(out));
    }
}

// Any number of streams up to STREAMS_MAX, any width and alignment: one column a lane, u in LDS.
template <typename A>
__global__ __launch_bounds__(256) void hyper_norm_kernel(HyperArgs p) {
    extern __shared__ float rowbuf[];
    __shared__ float red[8], mix_s[STREAMS_MAX * STREAMS_MAX], out_s[STREAMS_MAX], in_s[STREAMS_MAX];
    const int64_t row = blockIdx.x;
    const int dim = p.dim, S = p.S;
    for (int i = threadIdx.x; i < S * S; i += 256) mix_s[i] = p.mix ? p.mix[i] : 0.f;
    if ((int)threadIdx.x < S) {
        out_s[threadIdx.x] = p.mix ? p.out_w[threadIdx.x] : 0.f;
        in_s[threadIdx.x] = p.in_w ? p.in_w[threadIdx.x] : 1.f;
    }
    __syncthreads();
    float* xr = p.x + row * S * dim;
    float sum = 0.f;
    for (int c = threadIdx.x; c < dim; c += 256) {
        float x[STREAMS_MAX];
#pragma unroll
        for (int s = 0; s < STREAMS_MAX; ++s) x[s] = s < S ? xr[(int64_t)s * dim + c] : 0.f;
        float u = 0.f;
        if (p.mix) {
            float y = 0.f;
            if (p.pairs)
                for (int r = 0; r < p.top; ++r) {
                    const int pos = p.pos_of_pair[row * p.top + r];
                    if (pos >= 0) y = __builtin_fmaf(p.weights[row * p.top + r], (float)((const A*)p.pairs)[(int64_t)pos * p.pairs_stride + c], y);
                }
            if (p.a) y += (float)((const A*)p.a)[row * p.a_stride + c];
            if (p.c32) y += p.c32[row * p.c32_stride + c];
            for (int t = 0; t < S; ++t) {
                float v = out_s[t] * y;
#pragma unroll
                for (int s = 0; s < STREAMS_MAX; ++s)
                    if (s < S) v = __builtin_fmaf(mix_s[s * S + t], x[s], v);
                xr[(int64_t)t * dim + c] = v;
                u = __builtin_fmaf(in_s[t], v, u);
            }
        } else {
#pragma unroll
            for (int s = 0; s < STREAMS_MAX; ++s)
                if (s < S) u = __builtin_fmaf(in_s[s], x[s], u);
        }
        rowbuf[c] = u;
        sum += u;
    }
    if (p.norm == 0) return;
    const float mean = p.norm == 1 ? block_sum4(sum, red) / (float)dim : 0.f;
    float sq = 0.f;
    for (int c = threadIdx.x; c < dim; c += 256) sq += (rowbuf[c] - mean) * (rowbuf[c] - mean);
    const float inv = 1.0f / sqrtf(block_sum4(sq, red + 4) / (float)dim + p.eps);
    A* h = (A*)p.h + row * p.h_stride;
    for (int c = threadIdx.x; c < dim; c += 256) {
        float v = (rowbuf[c] - mean) * inv * (float)((const A*)p.nw)[c];
        if (p.nb) v += (float)((const A*)p.nb)[c];
        h[c] = (A)v;
    }
}

template <typename A, int NS>
static void launch_hyper_vec(const HyperArgs& p, int64_t rows, hipStream_t st) {
    const int pieces = (p.dim + 1023) / 1024;
    const dim3 grid((unsigned)rows);
    if (pieces <= 1) hyper_norm_vec_kernel<A, NS, 1><<<grid, 256, 0, st>>>(p);
    else if (pieces <= 2) hyper_norm_vec_kernel<A, NS, 2><<<grid, 256, 0, st>>>(p);
    else if (pieces <= 4) hyper_norm_vec_kernel<A, NS, 4><<<grid, 256, 0, st>>>(p);
    else hyper_norm_vec_kernel<A, NS, 8><<<grid, 256, 0, st>>>(p);
}

template <typename A>
static void launch_hyper(const HyperArgs& p, int64_t rows, hipStream_t st) {
    auto al = [](const void* q, int bytes) { return q == nullptr || ((uintptr_t)q % bytes) == 0; };
    constexpr int B = 4 * (int)sizeof(A);
    const bool vec = p.S <= 4 && p.dim % 4 == 0 && p.dim <= 8192 && p.a_stride % 4 == 0 && p.c32_stride % 4 == 0 && p.pairs_stride % 4 == 0 && p.h_stride % 4 == 0 && al(p.x, 16) &&
                     al(p.a, B) && al(p.c32, 16) && al(p.pairs, B) && al(p.nw, B) && al(p.nb, B) && al(p.h, B);
    if (vec && p.S == 1) return launch_hyper_vec<A, 1>(p, rows, st);
    if (vec && p.S == 2) return launch_hyper_vec<A, 2>(p, rows, st);
    if (vec && p.S == 3) return launch_hyper_vec<A, 3>(p, rows, st);
    if (vec && p.S == 4) return launch_hyper_vec<A, 4>(p, rows, st);
    const size_t lds = sizeof(float) * (size_t)p.dim;
    if (lds > 48 * 1024) (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&hyper_norm_kernel<A>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    hyper_norm_kernel<A><<<dim3((unsigned)rows), 256, lds, st>>>(p);
}

}  // namespace

extern "C" int32_t nvh_embedding_bigram_stream(const int64_t* ids, const int64_t* positions, const void* table, int64_t vocab, const void* pos_table, int64_t max_positions,
                                               const void* bigram, int64_t buckets, int64_t mul_prev, int64_t mul_cur, int32_t* last_tokens, const int32_t* slots,
                                               const int32_t* cu_seqlens_q, const int32_t* context_lens, int64_t batch, float* x, int64_t num_tokens, int64_t streams,
                                               int64_t dim, int32_t act_f32, nvh_stream_t stream) {
    NVH_REQUIRE(ids && table && x && num_tokens >= 0 && batch >= 0 && streams > 0 && dim > 0 && vocab > 0 && (!pos_table || (positions && max_positions > 0)), NVH_EINVAL,
                "nvh_embedding_bigram_stream: bad argument");
    NVH_REQUIRE(!bigram || (buckets > 0 && last_tokens && slots && context_lens && (cu_seqlens_q || num_tokens == batch)), NVH_EINVAL,
                "nvh_embedding_bigram_stream: a bigram table needs buckets and the sequences' slots");
    if (num_tokens == 0) return NVH_OK;
    const uintptr_t align = act_f32 ? 16 : 8;
    const bool vec = dim % 4 == 0 && (uintptr_t)table % align == 0 && (uintptr_t)pos_table % align == 0 && (uintptr_t)bigram % align == 0 && nvh_aligned16(x);
    const BigramArgs p{ids, positions, table, pos_table, bigram, vocab, max_positions, buckets, mul_prev, mul_cur, last_tokens, slots, cu_seqlens_q, context_lens, x, (int)batch,
                       (int)streams, (int)dim, vec};
    hipStream_t st = (hipStream_t)stream;
    if (act_f32) embedding_bigram_stream_kernel<float><<<dim3((unsigned)num_tokens), 256, 0, st>>>(p);
    else embedding_bigram_stream_kernel<bf16><<<dim3((unsigned)num_tokens), 256, 0, st>>>(p);
    NVH_CHECK_LAUNCH("nvh_embedding_bigram_stream");
    return NVH_OK;
}

extern "C" int32_t nvh_hyper_norm(float* x, int64_t streams, const float* mix, const float* out_weights, const float* in_weights, const void* a, int64_t a_stride, const float* c32,
                                  int64_t c32_stride, const void* pairs, int64_t pairs_stride, const int32_t* pos_of_pair, const float* weights, int64_t top, int32_t norm_kind,
                                  const void* norm_weight, const void* norm_bias, float eps, void* h, int64_t h_stride, int64_t rows, int64_t dim, int32_t act_f32,
                                  nvh_stream_t stream) {
    NVH_REQUIRE(x && rows >= 0 && dim > 0 && dim <= 32768 && streams > 0 && norm_kind >= 0 && norm_kind <= 2 && (norm_kind == 0 || (norm_weight && h && h_stride >= dim)), NVH_EINVAL,
                "nvh_hyper_norm: bad argument");
    NVH_REQUIRE(!mix || out_weights, NVH_EINVAL, "nvh_hyper_norm: the streams' mixture comes with the result's weights");
    NVH_REQUIRE((!a || a_stride >= dim) && (!c32 || c32_stride >= dim) && (!pairs || (pos_of_pair && weights && top > 0 && pairs_stride >= dim)) && (mix || (!a && !c32 && !pairs)),
                NVH_EINVAL, "nvh_hyper_norm: bad sublayer result");
    NVH_REQUIRE(streams <= STREAMS_MAX, NVH_ENOSYS, "nvh_hyper_norm: %ld streams above %d", (long)streams, STREAMS_MAX);
    if (rows == 0) return NVH_OK;
    const HyperArgs p{x, (int)streams, (int)dim, mix, out_weights, in_weights, a, a_stride, c32, c32_stride, pairs, pairs_stride, pos_of_pair, weights, (int)top, norm_kind,
                      norm_weight, norm_bias, eps, h, h_stride};
    if (act_f32) launch_hyper<float>(p, rows, (hipStream_t)stream);
    else launch_hyper<bf16>(p, rows, (hipStream_t)stream);
    NVH_CHECK_LAUNCH("nvh_hyper_norm");
    return NVH_OK;
}
