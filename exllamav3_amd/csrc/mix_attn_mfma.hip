// Prefill of the sliding-window sink attention on the matrix cores (bfloat16 activations): scores = Q K^T and the weighted sum P V with
// v_mfma_f32_16x16x32_bf16, scores, running maximum, exponentials and sums in float32; the softmax starts from the sink, so the sink is one
// more term of the denominator and nothing else.
//
// One workgroup = 128 query rows of one sequence and one head.  A wave owns QG groups of 16 rows (4 waves of 32 rows, or 8 of 16 for the largest heads, whose
// accumulators leave no room for a second group): with two groups every fragment read from LDS feeds two matrix instructions.  Key tiles of KT = 64 rows (32 for
// the largest heads, where 64 would not fit 64 KB of LDS) are staged in LDS once for all waves, K and V as stored; the loads of the next tile are issued
// before the matrix work of the current one and wait in registers.
//
// MFMA operand lane (g = lane / 16, c = lane % 16) holds row / column c and contraction slots 8g .. 8g+7; result lane (g, c) holds rows
// 4g .. 4g+3 of column c.  The scores are computed TRANSPOSED, S^T = K Q^T (keys are rows, the 16 queries of a group are columns): a lane then
// holds scores of ONE query (column c), so the running maximum, the sum and the rescale factor are per-lane scalars (two cross-lane steps
// per tile for the maximum, the sum is reduced once at the end), and the result registers of two 16-key tiles are, as they stand, the B
// operand of O^T = V^T P^T when contraction slot (g, e) is read as key 4g + e of the first tile (e < 4) or of the second (e >= 4); the A operand
// V^T comes out of the row-major V tile by two LDS transpose reads (ds_read_b64_tr_b16: the sixteen lanes of a group hand in the rows of a block of 4 keys x 16
// columns and lane c receives column c).  No probability goes through LDS.  The running maximum moves only when a row's score exceeds it by more than 8
// (in powers of two; weights stay below 2^8), so that most tiles rescale nothing.  Only the key tiles that intersect the window of the
// block's rows are visited, and a wave skips the tiles outside its own rows' windows.  Heads are the fastest grid index and the row blocks run from the last to
// the first: the blocks with the most keys start first, and with a multiple of eight heads the blocks of a head share one XCD's L2.
//
// Variants of the same kernel: `maps` attention maps per head (queries [head][map][dim], keys [kv head][map][dim], every map reads the values of the
// head's key/value head; result [row][head][map][vdim]); a chunk mask (a row sees the positions of its own chunk of `window` positions) beside the
// sliding window -- both give every row a first visible key lo(i) that never decreases with i, which is all the tile logic uses; a soft cap on the
// scores, cap tanh(score / cap), applied to the scaled scores before the running maximum (tanh is increasing, so the largest raw score still is the
// largest score); a float32 result; the first `keep` positions visible to every row beside its window (the tiles that hold them are visited first, then
// those of the window: a row's mask is "in the window, or among the first"); and an output gate per head or per value element and a factor on the
// result, applied in the epilogue.
#include "mix_common.cuh"

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));

#define AM_ROWS 128
#define AM_KPAD 8
#define AM_VPAD 16
#define LOG2E 1.4426950408889634f

__device__ __forceinline__ int first_visible(int i, int window, int mask) { return mask == EXL3_MIX_MASK_CHUNK ? (i / window) * window : i - window + 1; }

typedef short s16x4 __attribute__((__vector_size__(4 * sizeof(short))));
__device__ __forceinline__ bf16x4 lds_read_transposed(const uint16_t* p)
{
    const s16x4 r = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*) p);
    return __builtin_bit_cast(bf16x4, r);
}

// 16 bytes of a row: columns c0 .. c0+7, zeros beyond `cols` and for rows that are not there.  VEC: rows are 16-byte aligned and hold whole chunks.
template <bool VEC>
__device__ __forceinline__ uint4 row_chunk(const bf16_t* __restrict__ src, bool row_ok, int c0, int cols)
{
    if constexpr (VEC) return (row_ok && c0 < cols) ? *(const uint4*) (src + c0) : uint4{0u, 0u, 0u, 0u};
    union { uint4 v; uint16_t u[8]; } t;
    #pragma unroll
    for (int e = 0; e < 8; ++e) t.u[e] = (row_ok && c0 + e < cols) ? src[c0 + e].u : (uint16_t) 0;
    return t.v;
}

// KD: contraction steps of 32 over the (zero-padded) head dim; NV: 16-column tiles of the (padded) value dim; QG: groups of 16 rows per wave.  VEC: keys and values in 16-byte
// chunks (host-checked alignment).
template <int KD, int NV, int AM_KEYS, int QG, bool CAP, bool VEC>
__global__ __launch_bounds__(64 * AM_ROWS / (16 * QG), 2)
void attn_prefill_mfma_kernel(void* __restrict__ out_any, int64_t out_ld, int out_f32, const bf16_t* __restrict__ q, int64_t q_ld, const bf16_t* __restrict__ k,
                              int64_t k_ld, const bf16_t* __restrict__ v, int64_t v_ld, const bf16_t* __restrict__ gate, int64_t gate_ld, int gate_cols,
                              const float* __restrict__ sink, const int32_t* __restrict__ cu,
                              int heads, int kv_heads, int maps, int dim, int vdim, float scale, float softcap, int window, int mask, int keep,
                              float out_scale, int o_vec)
{
    constexpr int NT = 64 * AM_ROWS / (16 * QG), DP = KD * 32, KS = DP + AM_KPAD, VS = NV * 16 + AM_VPAD, NS = AM_KEYS / 16;
    constexpr int KC = DP / 8, VC = NV * 2;                       // 16-byte chunks per key
    constexpr int KSL = (AM_KEYS * KC + NT - 1) / NT, VSL = (AM_KEYS * VC + NT - 1) / NT;
    extern __shared__ __attribute__((aligned(16))) unsigned char smem_raw[];
    uint16_t* k_lds = (uint16_t*) smem_raw;                       // [AM_KEYS][KS]
    uint16_t* v_lds = k_lds + AM_KEYS * KS;                       // [AM_KEYS][VS]

    const int b = blockIdx.z, h = blockIdx.x;
    const int first = cu[b], len = cu[b + 1] - first;
    const int q0 = (gridDim.y - 1 - blockIdx.y) * AM_ROWS;
    if (q0 >= len) return;
    const int hh = h / maps;                                      // h counts (head, map)
    const int vh = hh / (heads / kv_heads), kvh = vh * maps + (h - hh * maps);
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, g = lane >> 4, c = lane & 15;
    const int wq_lo = q0 + w * 16 * QG, wq_hi = min(wq_lo + 16 * QG - 1, len - 1);           // this wave's rows
    const bool wave_live = wq_lo < len;

    // this wave's query rows as B operands of S^T = K Q^T (rows beyond the sequence read row len-1: computed and never stored)
    bf16x8 qf[QG][KD];
    int qi[QG], my_lo[QG];
    float m[QG], l[QG];                                           // per lane: query c of the group.  m: reference of the exponent (the same in the four lanes of a query), l: this lane's share of the sum
    f32x4 acc[QG][NV];                                            // O^T tiles: value rows 4g .. 4g+3 of tile t, query c
    #pragma unroll
    for (int u = 0; u < QG; ++u)
    {
        qi[u] = wq_lo + u * 16 + c;
        my_lo[u] = first_visible(qi[u], window, mask);
        const bf16_t* qr = q + (int64_t) (first + min(qi[u], len - 1)) * q_ld + (int64_t) h * dim;
        #pragma unroll
        for (int s = 0; s < KD; ++s)
        {
            union { bf16x8 v; uint4 x; } t;
            t.x = row_chunk<false>(qr, true, s * 32 + g * 8, dim);
            qf[u][s] = t.v;
        }
        m[u] = sink ? sink[h] : -1e30f;
        l[u] = (sink && g == 0) ? 1.0f : 0.0f;
        #pragma unroll
        for (int t = 0; t < NV; ++t) acc[u][t] = f32x4{0.f, 0.f, 0.f, 0.f};
    }

    const int blk_hi = min(q0 + AM_ROWS - 1, len - 1);
    const int j_begin = (max(0, first_visible(q0, window, mask)) / AM_KEYS) * AM_KEYS;
    const int keep_end = keep > 0 ? min(j_begin, (keep + AM_KEYS - 1) / AM_KEYS * AM_KEYS) : 0;        // the kept first positions' tiles ahead of the window's
    const int wave_lo = first_visible(wq_lo, window, mask), wave_hi_lo = first_visible(wq_hi, window, mask);      // first visible key of the wave's first / last row

    uint4 kreg[KSL], vreg[VSL];
    auto fetch = [&](int j0) __attribute__((always_inline))
    {
        #pragma unroll
        for (int e = 0; e < KSL; ++e)
        {
            const int idx = threadIdx.x + e * NT, r = idx / KC, ch = idx - r * KC, j = j0 + r;
            if ((AM_KEYS * KC) % NT != 0 && idx >= AM_KEYS * KC) break;
            kreg[e] = row_chunk<VEC>(k + (int64_t) (first + min(j, len - 1)) * k_ld + (int64_t) kvh * dim, j < len, ch * 8, dim);
        }
        #pragma unroll
        for (int e = 0; e < VSL; ++e)
        {
            const int idx = threadIdx.x + e * NT, r = idx / VC, ch = idx - r * VC, j = j0 + r;
            if ((AM_KEYS * VC) % NT != 0 && idx >= AM_KEYS * VC) break;
            vreg[e] = row_chunk<VEC>(v + (int64_t) (first + min(j, len - 1)) * v_ld + (int64_t) vh * vdim, j < len, ch * 8, vdim);
        }
    };
    int j0 = keep_end > 0 ? 0 : j_begin;
    fetch(j0);
    const float a_cap = CAP ? 2.0f * LOG2E * scale / softcap : 0.f;
    const float c2 = (CAP ? 1.0f : scale) * LOG2E;                // what is left to multiply the held scores with, in powers of two
    while (j0 <= blk_hi)
    {
        __syncthreads();                                          // the previous tile's operand reads are over
        #pragma unroll
        for (int e = 0; e < KSL; ++e)
        {
            const int idx = threadIdx.x + e * NT, r = idx / KC, ch = idx - r * KC;
            if ((AM_KEYS * KC) % NT != 0 && idx >= AM_KEYS * KC) break;
            *(uint4*) (k_lds + r * KS + ch * 8) = kreg[e];
        }
        #pragma unroll
        for (int e = 0; e < VSL; ++e)
        {
            const int idx = threadIdx.x + e * NT, r = idx / VC, ch = idx - r * VC;
            if ((AM_KEYS * VC) % NT != 0 && idx >= AM_KEYS * VC) break;
            *(uint4*) (v_lds + r * VS + ch * 8) = vreg[e];
        }
        __syncthreads();
        const int j_next = (j0 + AM_KEYS == keep_end) ? j_begin : j0 + AM_KEYS;
        if (j_next <= blk_hi) fetch(j_next);
        // tiles wholly outside this wave's windows: nothing to add (uniform per wave; the barriers are still met)
        if (wave_live && j0 <= wq_hi && (j0 + AM_KEYS - 1 >= wave_lo || j0 < keep))
        {
            f32x4 sc[QG][NS];
            #pragma unroll
            for (int u = 0; u < QG; ++u)
            {
                #pragma unroll
                for (int n = 0; n < NS; ++n) sc[u][n] = f32x4{0.f, 0.f, 0.f, 0.f};
            }
            #pragma unroll
            for (int s = 0; s < KD; ++s)
            {
                #pragma unroll
                for (int n = 0; n < NS; ++n)
                {
                    const bf16x8 kf = *(const bf16x8*) (k_lds + (n * 16 + c) * KS + s * 32 + g * 8);
                    #pragma unroll
                    for (int u = 0; u < QG; ++u) sc[u][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[u][s], sc[u][n], 0, 0, 0);
                }
            }
            // sc[u][n][i] = raw score of key j0 + 16n + 4g + i against query qi[u].  A tile whose keys all lie inside the window of every row of the wave
            // needs no mask (wave-uniform branch; with a window of many tiles that is most of them).
            const bool interior = j0 + AM_KEYS - 1 <= wq_lo && j0 >= wave_hi_lo && wq_lo + 16 * QG - 1 < len;
            float mx[QG];
            bool need = false;
            #pragma unroll
            for (int u = 0; u < QG; ++u)
            {
                if (CAP)
                {
                    // score <- cap tanh(scale raw / cap), tanh(x) = 1 - 2 / (1 + e^(2x)): one v_exp_f32 and one reciprocal per key
                    #pragma unroll
                    for (int n = 0; n < NS; ++n)
                    {
                        #pragma unroll
                        for (int i = 0; i < 4; ++i) sc[u][n][i] = softcap - 2.0f * softcap * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(sc[u][n][i] * a_cap));
                    }
                }
                if (!interior)
                {
                    #pragma unroll
                    for (int n = 0; n < NS; ++n)
                    {
                        #pragma unroll
                        for (int i = 0; i < 4; ++i)
                        {
                            const int j = j0 + n * 16 + g * 4 + i;
                            const bool ok = j <= qi[u] && (j >= my_lo[u] || j < keep) && qi[u] < len;
                            sc[u][n][i] = ok ? sc[u][n][i] : -INFINITY;
                        }
                    }
                }
                float a = -INFINITY;
                #pragma unroll
                for (int n = 0; n < NS; ++n) a = fmaxf(fmaxf(a, fmaxf(sc[u][n][0], sc[u][n][1])), fmaxf(sc[u][n][2], sc[u][n][3]));
                a = fmaxf(a, __shfl_xor(a, 16, 64));
                a = fmaxf(a, __shfl_xor(a, 32, 64));
                mx[u] = a;                                         // the same in the four lanes of a query
                need = need || a * c2 - m[u] * LOG2E > 8.0f;
            }
            if (__any(need))
            {
                #pragma unroll
                for (int u = 0; u < QG; ++u)
                {
                    const float mn = fmaxf(m[u], mx[u] * (CAP ? 1.0f : scale));     // scale > 0 (host-checked): the largest raw score is the largest score
                    const float corr = __builtin_amdgcn_exp2f((m[u] - mn) * LOG2E);
                    m[u] = mn;
                    l[u] *= corr;
                    #pragma unroll
                    for (int t = 0; t < NV; ++t) acc[u][t] *= corr;
                }
            }
            bf16x8 pb[QG][NS / 2];
            #pragma unroll
            for (int u = 0; u < QG; ++u)
            {
                // weight = exp(score * scale - m) = 2^(score * c2 - m * log2 e): one multiply-add and one v_exp_f32 per key
                const float off = -m[u] * LOG2E;
                float sum = 0.f;
                #pragma unroll
                for (int n = 0; n < NS; ++n)
                {
                    #pragma unroll
                    for (int i = 0; i < 4; ++i)
                    {
                        const float p = __builtin_amdgcn_exp2f(__builtin_fmaf(sc[u][n][i], c2, off));      // masked: 2^(-inf) = 0
                        sum += p;
                        pb[u][n >> 1][(n & 1) * 4 + i] = (__bf16) p;
                    }
                }
                l[u] += sum;
            }
            #pragma unroll
            for (int kk = 0; kk < NS / 2; ++kk)
            {
                #pragma unroll
                for (int t = 0; t < NV; ++t)
                {
                    const uint16_t* vr = v_lds + (kk * 32 + 4 * g + (c >> 2)) * VS + t * 16 + 4 * (c & 3);
                    union { bf16x8 v; bf16x4 h[2]; } va;
                    va.h[0] = lds_read_transposed(vr);
                    va.h[1] = lds_read_transposed(vr + 16 * VS);
                    #pragma unroll
                    for (int u = 0; u < QG; ++u) acc[u][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(va.v, pb[u][kk], acc[u][t], 0, 0, 0);
                }
            }
        }
        j0 = j_next;
    }
    if (!wave_live) return;
    #pragma unroll
    for (int u = 0; u < QG; ++u)
    {
        l[u] += __shfl_xor(l[u], 16, 64);
        l[u] += __shfl_xor(l[u], 32, 64);
    }
    #pragma unroll
    for (int u = 0; u < QG; ++u)
    {
        if (qi[u] >= len) continue;
        const int64_t n = first + qi[u];
        const bool by_head = gate && gate_cols == 1;
        const float gt = by_head ? sigmoid_f(to_f(gate[n * gate_ld + h])) * out_scale : out_scale;
        const bf16_t* grow = gate && !by_head ? gate + n * gate_ld + (int64_t) h * vdim : nullptr;
        const float f = (l[u] > 0.f ? 1.0f / l[u] : 0.f) * gt;
        const int64_t o0 = n * out_ld + (int64_t) h * vdim;
        #pragma unroll
        for (int t = 0; t < NV; ++t)
        {
            const int col0 = t * 16 + g * 4;                       // four neighbouring value columns per lane and tile
            if (o_vec && col0 + 4 <= vdim)                         // bfloat16 result and gate rows in 8-byte groups (host-checked alignment)
            {
                float r[4];
                #pragma unroll
                for (int i = 0; i < 4; ++i) r[i] = acc[u][t][i] * f;
                if (grow)
                {
                    union { uint2 v; bf16_t e[4]; } gv;
                    gv.v = *(const uint2*) (grow + col0);
                    #pragma unroll
                    for (int i = 0; i < 4; ++i) r[i] *= sigmoid_f(to_f(gv.e[i]));
                }
                union { uint2 v; bf16_t e[4]; } ov;
                #pragma unroll
                for (int i = 0; i < 4; ++i) ov.e[i] = from_f<bf16_t>(r[i]);
                *(uint2*) ((bf16_t*) out_any + o0 + col0) = ov.v;
                continue;
            }
            #pragma unroll
            for (int i = 0; i < 4; ++i)
            {
                const int col = col0 + i;
                if (col < vdim)
                {
                    const float r = acc[u][t][i] * f * (grow ? sigmoid_f(to_f(grow[col])) : 1.0f);
                    if (out_f32) ((float*) out_any)[o0 + col] = r;
                    else         ((bf16_t*) out_any)[o0 + col] = from_f<bf16_t>(r);
                }
            }
        }
    }
}

extern "C" int exl3_mix_attn_prefill_mfma(void* out, const void* q, int64_t q_ld, const void* k, int64_t k_ld, const void* v_norm,
                                          const void* gate, int64_t gate_ld, const float* sink, const int32_t* cu,
                                          int batch, int max_rows, int heads, int kv_heads, int dim, int vdim, float scale, int window, void* stream)
{
    return exl3_mix_attn_prefill_mfma_ex(out, (int64_t) heads * vdim, 0, q, q_ld, k, k_ld, v_norm, (int64_t) kv_heads * vdim, gate, gate_ld, 1, sink, cu, batch, max_rows, heads, kv_heads, 1, dim, vdim,
                                         scale, 0.f, window, EXL3_MIX_MASK_WINDOW, 0, 1.0f, stream);
}

extern "C" int exl3_mix_attn_prefill_mfma_ex(void* out, int64_t out_ld, int out_f32, const void* q, int64_t q_ld, const void* k, int64_t k_ld, const void* v_norm, int64_t v_ld,
                                             const void* gate, int64_t gate_ld, int gate_cols, const float* sink, const int32_t* cu,
                                             int batch, int max_rows, int heads, int kv_heads, int maps, int dim, int vdim, float scale, float softcap, int window, int mask, int keep,
                                             float out_scale, void* stream)
{
    MIX_CHECK(out && q && k && v_norm && cu, "mix_attn_prefill_mfma: null pointer");
    MIX_CHECK(batch >= 0 && max_rows >= 0 && heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && maps >= 1 && heads * maps <= 65535 && batch <= 65535,
              "mix_attn_prefill_mfma: heads %d / kv_heads %d / batch %d", heads, kv_heads, batch);
    MIX_CHECK((maps == 1 || !gate) && softcap >= 0.f && (mask == EXL3_MIX_MASK_WINDOW || mask == EXL3_MIX_MASK_CHUNK),
              "mix_attn_prefill_mfma: a gate per head applies to one map only; softcap >= 0; mask %d", mask);
    MIX_CHECK(keep >= 0 && (keep == 0 || mask == EXL3_MIX_MASK_WINDOW), "mix_attn_prefill_mfma: kept first tokens go with a window");
    MIX_CHECK(dim > 0 && dim <= 256 && vdim > 0 && vdim <= 256 && window > 0, "mix_attn_prefill_mfma: dim %d and vdim %d must be <= 256", dim, vdim);
    MIX_CHECK(scale > 0.f, "mix_attn_prefill_mfma: the score scale must be positive (the running maximum is taken over raw scores)");
    MIX_CHECK(q_ld >= (int64_t) heads * maps * dim && k_ld >= (int64_t) kv_heads * maps * dim && v_ld >= (int64_t) kv_heads * vdim && out_ld >= (int64_t) heads * maps * vdim &&
              (!gate || ((gate_cols == 1 || gate_cols == vdim) && gate_ld >= (int64_t) heads * gate_cols)),
              "mix_attn_prefill_mfma: bad row strides");
    if (batch == 0 || max_rows == 0) return EXL3_MIX_OK;
    const dim3 grid(heads * maps, (max_rows + AM_ROWS - 1) / AM_ROWS, batch);
    const bool vec = (uintptr_t) k % 16 == 0 && k_ld % 8 == 0 && dim % 8 == 0 && (uintptr_t) v_norm % 16 == 0 && v_ld % 8 == 0 && vdim % 8 == 0;
    const int o_vec = !out_f32 && vdim % 4 == 0 && out_ld % 4 == 0 && (uintptr_t) out % 8 == 0 && (!gate || gate_cols == 1 || (gate_ld % 4 == 0 && (uintptr_t) gate % 8 == 0));
    #define AM_LDS(KDV, NVV, KTV) ((size_t) KTV * (KDV * 32 + AM_KPAD + NVV * 16 + AM_VPAD) * sizeof(uint16_t))
    #define AM_LAUNCH_C(KDV, NVV, KTV, QGV, CAPV, VECV) \
        hipLaunchKernelGGL((attn_prefill_mfma_kernel<KDV, NVV, KTV, QGV, CAPV, VECV>), grid, dim3(64 * AM_ROWS / (16 * QGV)), AM_LDS(KDV, NVV, KTV), (hipStream_t) stream, out, out_ld, out_f32, \
                           (const bf16_t*) q, q_ld, (const bf16_t*) k, k_ld, (const bf16_t*) v_norm, v_ld, (const bf16_t*) gate, gate_ld, gate_cols, sink, cu, heads, kv_heads, maps, dim, vdim, \
                           scale, softcap, window, mask, keep, out_scale, o_vec)
    #define AM_LAUNCH(KDV, NVV, KTV, QGV) do { \
        static_assert(AM_LDS(KDV, NVV, KTV) <= 65536, "tile does not fit the LDS"); \
        if (vec) { if (softcap > 0.f) AM_LAUNCH_C(KDV, NVV, KTV, QGV, true, true); else AM_LAUNCH_C(KDV, NVV, KTV, QGV, false, true); } \
        else     { if (softcap > 0.f) AM_LAUNCH_C(KDV, NVV, KTV, 1, true, false); else AM_LAUNCH_C(KDV, NVV, KTV, 1, false, false); } } while (0)
    const int kd = (dim + 31) / 32, nv = (vdim + 15) / 16;
    if (kd <= 2)      { if (nv <= 4) AM_LAUNCH(2, 4, 64, 2); else if (nv <= 8) AM_LAUNCH(2, 8, 64, 2); else AM_LAUNCH(2, 16, 64, 1); }
    else if (kd <= 4) { if (nv <= 4) AM_LAUNCH(4, 4, 64, 2); else if (nv <= 8) AM_LAUNCH(4, 8, 64, 2); else AM_LAUNCH(4, 16, 64, 1); }
    else if (kd <= 6) { if (nv <= 4) AM_LAUNCH(6, 4, 64, 2); else if (nv <= 8) AM_LAUNCH(6, 8, 64, 2); else AM_LAUNCH(6, 16, 64, 1); }
    else              { if (nv <= 4) AM_LAUNCH(8, 4, 64, 1); else if (nv <= 8) AM_LAUNCH(8, 8, 64, 1); else AM_LAUNCH(8, 16, 32, 1); }
    #undef AM_LDS
    #undef AM_LAUNCH
    #undef AM_LAUNCH_C
    return mix_check_launch("mix_attn_prefill_mfma");
}
