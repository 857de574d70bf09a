// Queries, keys and values that pass a short causal convolution over time, per channel, between their projection and the
// attention (csrc/attention_any.hip), with the state that continues the convolution from step to step:
//   nvh_attn_conv_prep   over the projection rows [q | k | v | ...]: y_t = sum_j w[:, j] u_(t - taps + 1 + j) with zeros before the
//                        sequence's start and the sequence's carried inputs before this step's; q and k then divided by their
//                        root mean square per head (optional, no weight); q to a packed buffer, k and v to their cache slots (keys
//                        [pages, page, G, dim], values transposed within a page, [pages, G, vdim, page]).  A layer without keys
//                        of its own has q columns only.  Sums and norms are fp32; a value is rounded once, when it is stored.
// The carried inputs (state [slots, taps - 1, channels] fp32) are brought up to date in the same launch when every sequence
// brings one token; in any other step nvh_conv_state_update follows.
#include "common.h"

namespace {

struct ConvPrepArgs {
    const void* proj;          // [T, ld]: H*dim columns (q), then with own keys G*dim (k) and G*vdim (v)
    int64_t ld;
    const void* conv_w;        // [channels, taps], last tap on the current token; null: no convolution
    float* state;              // [slots, taps - 1, channels]
    const int32_t *slots, *cu_seqlens_q, *context_lens, *slot_mapping;
    void *q_out, *k_cache, *v_cache;
    int T, batch, taps, H, G, dim, vdim, page, channels;
    int unit, update_state, vec, lanes_log2;       // lanes: per row of a head, a power of two, eight channels each
    float eps;
};

// A workgroup takes KT tokens of the step and one head (q heads, then k heads, then v heads).  A thread owns eight channels of
// consecutive tokens, so that with TAPS known (0: any number) an input is loaded once and moves through the taps in registers.
template <typename A, int TAPS, int KT>
__global__ __launch_bounds__(256) void attn_conv_prep_kernel(ConvPrepArgs p) {
    extern __shared__ __attribute__((aligned(16))) unsigned char smem_raw[];
    __shared__ int index_s[KT], state_slot_s[KT], cache_slot_s[KT];            // the token's number within its portion; -1: nothing carried; -1: not stored
    const int tid = threadIdx.x, t0 = blockIdx.x * KT, hs = blockIdx.y;
    const int kind = hs < p.H ? 0 : (hs < p.H + p.G ? 1 : 2), head = kind == 0 ? hs : (kind == 1 ? hs - p.H : hs - p.H - p.G);
    const int n = kind == 2 ? p.vdim : p.dim;
    const int col0 = kind == 0 ? head * p.dim : (kind == 1 ? (p.H + head) * p.dim : (p.H + p.G) * p.dim + head * p.vdim);
    if (tid < KT) {
        const int t = t0 + tid;
        int j = 0, st = -1, cs = -1;
        if (t < p.T) {
            const int seq = seq_of_token(p.cu_seqlens_q, p.batch, t);
            const int lo = p.cu_seqlens_q ? p.cu_seqlens_q[seq] : seq, hi = p.cu_seqlens_q ? p.cu_seqlens_q[seq + 1] : seq + 1;
            const int slot = p.slots ? p.slots[seq] : -1;
            j = t - lo;
            if (slot >= 0) st = p.context_lens[seq] != hi - lo ? slot : -2 - slot;       // (-2 - slot: a slot whose sequence starts in this step)
            cs = p.slot_mapping ? p.slot_mapping[t] : -1;
        }
        index_s[tid] = j;
        state_slot_s[tid] = st;
        cache_slot_s[tid] = cs;
    }
    __syncthreads();
    const int lanes = 1 << p.lanes_log2, sub = tid & (lanes - 1), group = tid >> p.lanes_log2, groups = 256 >> p.lanes_log2;
    const int run = (KT + groups - 1) / groups, c = sub * 8, valid = n - c;    // (valid <= 0: a lane beyond the row, which only joins the sums)
    const int taps = TAPS ? TAPS : p.taps;
    constexpr int W = TAPS ? TAPS : 1;
    float w[8 * W], win[W][8];
    if (TAPS && p.conv_w) {
        if (p.vec && valid >= 8) {
#pragma unroll
            for (int k = 0; k < W; ++k) {
                float piece[8];
                nvh_load8((const A*)p.conv_w, (int64_t)(col0 + c) * W + 8 * k, 8, true, piece);
#pragma unroll
                for (int e = 0; e < 8; ++e) w[8 * k + e] = piece[e];
            }
        } else {
#pragma unroll
            for (int i = 0; i < 8 * W; ++i) w[i] = i / W < valid ? (float)((const A*)p.conv_w)[(int64_t)(col0 + c) * W + i] : 0.f;
        }
    }
    A* vs = reinterpret_cast<A*>(smem_raw);                  // [KT][n + 2] (values only)
    const int vld = n + 2;
    for (int i = 0; i < run; ++i) {
        const int r = group * run + i, t = t0 + r;
        if (r >= KT || t >= p.T) break;                      // (the same for all lanes of a row)
        const int j = index_s[r], slot = state_slot_s[r];
        const A* row = (const A*)p.proj + (int64_t)t * p.ld + col0;
        // the input `back` tokens before this one
        auto input = [&](int back, float (&x)[8]) {
            if (back <= j) {
                nvh_load8(row - (int64_t)back * p.ld, c, valid, p.vec, x);
            } else if (slot >= 0) {
                nvh_load8(p.state + ((int64_t)slot * (taps - 1) + (taps - 1 + j - back)) * p.channels + col0, c, valid, p.vec, x);
            } else {
#pragma unroll
                for (int e = 0; e < 8; ++e) x[e] = 0.f;
            }
        };
        float y[8];
        if (!p.conv_w) {
            input(0, y);
        } else if constexpr (TAPS > 0) {
            if (i == 0 || j == 0) {                          // the window's earlier inputs are not this thread's last ones
#pragma unroll
                for (int k = 0; k + 1 < W; ++k) input(W - 1 - k, win[k]);
            } else {
#pragma unroll
                for (int k = 0; k + 1 < W; ++k)
#pragma unroll
                    for (int e = 0; e < 8; ++e) win[k][e] = win[k + 1][e];
            }
            input(0, win[W - 1]);
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                y[e] = 0.f;
#pragma unroll
                for (int k = 0; k < W; ++k) y[e] = __builtin_fmaf(w[e * W + k], win[k][e], y[e]);
            }
        } else {
#pragma unroll
            for (int e = 0; e < 8; ++e) y[e] = 0.f;
            for (int k = 0; k < taps; ++k) {
                float x[8];
                input(taps - 1 - k, x);
#pragma unroll
                for (int e = 0; e < 8; ++e)
                    if (e < valid) y[e] = __builtin_fmaf((float)((const A*)p.conv_w)[(int64_t)(col0 + c + e) * taps + k], x[e], y[e]);
            }
        }
        // One token per sequence: this thread is the only one that reads or writes these channels of the slot.  Ascending
        // entries: an entry is read (as its predecessor's new value) before it is written.
        if (p.update_state && slot != -1) {
            const int sl = slot >= 0 ? slot : -2 - slot;
            float* st = p.state + (int64_t)sl * (taps - 1) * p.channels + col0 + c;
            for (int k = 0; k + 1 < taps; ++k) {
                float x[8];
                if (k + 2 < taps) input(taps - 2 - k, x);
                else input(0, x);
                if (p.vec && valid >= 8) {
                    *reinterpret_cast<f32x4*>(st + (int64_t)k * p.channels) = f32x4{x[0], x[1], x[2], x[3]};
                    *reinterpret_cast<f32x4*>(st + (int64_t)k * p.channels + 4) = f32x4{x[4], x[5], x[6], x[7]};
                } else {
#pragma unroll
                    for (int e = 0; e < 8; ++e)
                        if (e < valid) st[(int64_t)k * p.channels + e] = x[e];
                }
            }
        }
        if (kind != 2 && p.unit) {
            float ss = 0.f;
#pragma unroll
            for (int e = 0; e < 8; ++e) ss += y[e] * y[e];   // (lanes beyond the row hold zeros)
            for (int off = 1; off < lanes; off <<= 1) ss += __shfl_xor(ss, off, 64);
            const float inv = 1.0f / sqrtf(ss / (float)n + p.eps);
#pragma unroll
            for (int e = 0; e < 8; ++e) y[e] *= inv;
        }
        if (valid <= 0) continue;
        if (kind == 2) {
#pragma unroll
            for (int e = 0; e < 8; ++e)
                if (e < valid) vs[r * vld + c + e] = (A)y[e];
            continue;
        }
        A* dst = nullptr;
        if (kind == 0) dst = (A*)p.q_out + ((int64_t)t * p.H + head) * p.dim + c;
        else if (cache_slot_s[r] >= 0) dst = (A*)p.k_cache + ((int64_t)cache_slot_s[r] * p.G + head) * p.dim + c;
        if (!dst) continue;
        A out[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) out[e] = (A)y[e];
        if (p.vec && valid >= 8) {
            __builtin_memcpy(__builtin_assume_aligned(dst, 16), out, sizeof(out));
        } else {
#pragma unroll
            for (int e = 0; e < 8; ++e)
                if (e < valid) dst[e] = out[e];
        }
    }
    if (kind != 2) return;                                   // (uniform)
    __syncthreads();
    // tokens side by side in a page leave in one piece
    const int r = tid % KT, slot = cache_slot_s[r];          // (256 is a multiple of KT)
    if (slot < 0) return;
    A* dst = (A*)p.v_cache + ((int64_t)(slot / p.page) * p.G + head) * p.vdim * p.page + slot % p.page;
    for (int d = tid / KT; d < n; d += 256 / KT) dst[(int64_t)d * p.page] = vs[r * vld + d];
}

template <typename A, int TAPS, int KT>
static void launch_conv_prep(const ConvPrepArgs& p, int heads, hipStream_t st) {
    const size_t lds = heads > p.H ? sizeof(A) * (size_t)KT * (p.vdim + 2) : 0;
    if (lds > 60 * 1024) (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&attn_conv_prep_kernel<A, TAPS, KT>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    attn_conv_prep_kernel<A, TAPS, KT><<<dim3((unsigned)nvh_cdiv(p.T, KT), (unsigned)heads), 256, lds, st>>>(p);
}

template <typename A, int KT>
static void launch_conv_prep_taps(const ConvPrepArgs& p, int heads, hipStream_t st) {
    switch (p.taps) {
        case 2: return launch_conv_prep<A, 2, KT>(p, heads, st);
        case 3: return launch_conv_prep<A, 3, KT>(p, heads, st);
        case 4: return launch_conv_prep<A, 4, KT>(p, heads, st);
        default: return launch_conv_prep<A, 0, KT>(p, heads, st);
    }
}

}  // namespace

extern "C" int32_t nvh_attn_conv_prep(const void* proj, int64_t proj_row_stride, const void* conv_w, int64_t taps, float* conv_state, const int32_t* slots,
                                      const int32_t* cu_seqlens_q, const int32_t* context_lens, const int32_t* slot_mapping, int32_t unit_qk, float eps,
                                      void* q_out, void* k_cache, void* v_cache, int64_t page, int64_t batch, int64_t num_tokens, int64_t num_q_heads,
                                      int64_t num_kv_heads, int64_t dim, int64_t vdim, int32_t update_state, int32_t act_f32, nvh_stream_t stream) {
    const bool own = k_cache != nullptr;
    NVH_REQUIRE(proj && context_lens && q_out && !k_cache == !v_cache && (!own || slot_mapping), NVH_EINVAL, "nvh_attn_conv_prep: null pointer");
    NVH_REQUIRE(num_tokens >= 0 && num_tokens < (1 << 30) && batch >= 0 && num_q_heads > 0 && num_kv_heads > 0 && dim > 0 && vdim > 0 && page > 0 && taps >= 1 && taps < 4096, NVH_EINVAL,
                "nvh_attn_conv_prep: bad sizes");
    NVH_REQUIRE(taps == 1 || (conv_w && conv_state && slots), NVH_EINVAL, "nvh_attn_conv_prep: a convolution needs its weights and a state");
    NVH_REQUIRE(dim <= 512 && vdim <= 512 && num_q_heads + 2 * num_kv_heads < 65536, NVH_ENOSYS, "nvh_attn_conv_prep: head sizes %ld / %ld above 512", (long)dim, (long)vdim);
    const int64_t channels = num_q_heads * dim + (own ? num_kv_heads * (dim + vdim) : 0);
    NVH_REQUIRE(proj_row_stride >= channels && channels < (1 << 28), NVH_EINVAL, "nvh_attn_conv_prep: projection row too short");
    NVH_REQUIRE(cu_seqlens_q || num_tokens == batch, NVH_EINVAL, "nvh_attn_conv_prep: one token per sequence without cu_seqlens_q");
    NVH_REQUIRE(!update_state || num_tokens == batch, NVH_EINVAL, "nvh_attn_conv_prep: the state is updated here only when every sequence brings one token");
    if (num_tokens == 0 || batch == 0) return NVH_OK;
    int lanes_log2 = 0;
    while ((8 << lanes_log2) < (own && vdim > dim ? vdim : dim)) ++lanes_log2;
    const bool vec = dim % 8 == 0 && vdim % 8 == 0 && proj_row_stride % 8 == 0 && nvh_aligned16(proj) && nvh_aligned16(conv_w) && nvh_aligned16(conv_state) && nvh_aligned16(q_out) &&
                     nvh_aligned16(k_cache) && nvh_aligned16(v_cache);
    const ConvPrepArgs p{proj, proj_row_stride, conv_w, conv_state, slots, cu_seqlens_q, context_lens, slot_mapping, q_out, k_cache, v_cache, (int)num_tokens, (int)batch, (int)taps,
                         (int)num_q_heads, (int)num_kv_heads, (int)dim, (int)vdim, (int)page, (int)channels, unit_qk, update_state && taps > 1, vec, lanes_log2, eps};
    const int heads = (int)(num_q_heads + (own ? 2 * num_kv_heads : 0));
    hipStream_t st = (hipStream_t)stream;
    // (a token's arithmetic does not depend on the tile it lies in)
    if (num_tokens >= 512) {
        if (act_f32) launch_conv_prep_taps<float, 64>(p, heads, st);
        else launch_conv_prep_taps<bf16, 64>(p, heads, st);
    } else {
        if (act_f32) launch_conv_prep_taps<float, 16>(p, heads, st);
        else launch_conv_prep_taps<bf16, 16>(p, heads, st);
    }
    NVH_CHECK_LAUNCH("nvh_attn_conv_prep");
    return NVH_OK;
}
