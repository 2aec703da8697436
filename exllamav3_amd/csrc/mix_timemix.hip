// Time mixing with a decay per key channel and token and a bonus for the current token (RWKV-style).  Per head, with decays w_t in (0, 1] given by their base-2 logarithms:
//   o = S^T r + (sum_c r_c u_c k_c) v,   then for every key channel c   S[c] <- w_c S[c] + k_c v
// Everything that enters the recurrence besides the projections is float32; the state [slot][head][dim][vdim] is float32.
//
//   token_shift    what the projections read: h + (h' - h) mu_m for every mix m, h' the previous token's row (of the step, or from the slot)
//   decay_log2     log2 w = -log2(e) exp(w0 + W2 tanh(t)) from the low-rank input t
//   timemix        prompt steps in tiles of 16 tokens, whole sequences or parallel segments; optionally with the head norm and gate that follow
//   timemix_step   one row per sequence: decays, read-out, state update, head norm and gate in one launch
//
// A tile of 16 tokens is four products on the float32 matrix instruction.  With L_t the sum of the tile's log2 decays up to and including token t, L'_t the sum
// before it and M = L_7 (the middle of the tile), q_t = r_t 2^(L'_t - M) and p_t = k_t 2^(M - L_t):
//   S' = diag(2^M) S;   O = Q S' + A V,  A[t][j] = q_t . p_j for j < t, A[t][t] = sum_c r_t u k_t;   S <- diag(2^(L_15 - M)) (S' + P^T V)
// Taking the exponents from the middle keeps both factors in range while every channel decays by less than 2^-80 over each half of the tile; a tile with a
// stronger decay (uniform over the workgroup) runs token by token on the same registers instead, in which every exponent is a decay's own.
//
// v_mfma_f32_16x16x4_f32: operand lane (g = lane / 16, c = lane % 16) holds row / column c and contraction slot g; result lane (g, c) holds rows 4g .. 4g+3 of column
// c.  Contraction slot g of step i is index 4g + i of a block of 16, so four steps of an operand are one 16-byte LDS read and the registers of the state (rows
// 4g + i of a 16 x 16 block) are the B operand of Q S' as they stand.  One workgroup = one head, 64 value columns, 4 waves of 16 columns.
#include "mix_common.cuh"

typedef float f32x4 __attribute__((ext_vector_type(4)));

#define TM_THREADS 256
#define TM_WAVES 4
#define TM_TILE 16
#define TM_COLS 64
#define TM_WHOLE 0
#define TM_SEG_LOCAL 1
#define TM_SEG_FINAL 2
#define TM_MAX_EXP 80.0f
#define TM_EXP2(x) __builtin_amdgcn_exp2f(x)

// out[m][n] = h[n] + (h'[n] - h[n]) mu[m]; h' = the row before n in its sequence: the step's own where the sequence has it in the step, the slot's otherwise, zeros
// ahead of the first token.  The last row of a sequence goes into its slot.  A thread holds V channels of R consecutive rows and of the row before them.
template <typename T, int V, int R>
__global__ __launch_bounds__(256) void token_shift_kernel(T* __restrict__ out, const T* __restrict__ h, int64_t h_ld, T* __restrict__ last, const float* __restrict__ mu, int mixes,
                                                          const int32_t* __restrict__ tok_seq, const int32_t* __restrict__ tok_pos, const int32_t* __restrict__ slots,
                                                          const int32_t* __restrict__ pos0, const int32_t* __restrict__ len_after, int n, int width)
{
    const int n0 = blockIdx.x * R;
    const int i = (blockIdx.y * 256 + threadIdx.x) * V;
    if (i >= width) return;
    float cur[R][V], diff[R][V];
    float prev[V];
    #pragma unroll
    for (int e = 0; e < V; ++e) prev[e] = 0.f;
    {
        const int b = tok_seq[n0], pos = tok_pos[n0];
        if (pos > pos0[b]) load_n<T, V>(h + (int64_t) (n0 - 1) * h_ld + i, prev);
        else if (pos > 0)  load_n<T, V>(last + (int64_t) slots[b] * width + i, prev);
    }
    #pragma unroll
    for (int r = 0; r < R; ++r)
    {
        const int row = n0 + r;
        if (row >= n)
        {
            #pragma unroll
            for (int e = 0; e < V; ++e) { cur[r][e] = 0.f; diff[r][e] = 0.f; }
            continue;
        }
        const int b = tok_seq[row], pos = tok_pos[row];
        load_n<T, V>(h + (int64_t) row * h_ld + i, cur[r]);
        if (r > 0 && pos == pos0[b])                              // another sequence begins at this row
        {
            if (pos > 0) load_n<T, V>(last + (int64_t) slots[b] * width + i, prev);
            else
            {
                #pragma unroll
                for (int e = 0; e < V; ++e) prev[e] = 0.f;
            }
        }
        if (pos == len_after[b] - 1) store_n<T, V>(last + (int64_t) slots[b] * width + i, cur[r]);      // after this thread's own read of the slot
        #pragma unroll
        for (int e = 0; e < V; ++e) { diff[r][e] = prev[e] - cur[r][e]; prev[e] = cur[r][e]; }
    }
    for (int m = 0; m < mixes; ++m)
    {
        float w[V];
        #pragma unroll
        for (int e = 0; e < V; ++e) w[e] = mu[(int64_t) m * width + i + e];
        #pragma unroll
        for (int r = 0; r < R; ++r)
        {
            if (n0 + r >= n) break;
            float y[V];
            #pragma unroll
            for (int e = 0; e < V; ++e) y[e] = __builtin_fmaf(diff[r][e], w[e], cur[r][e]);
            store_n<T, V>(out + ((int64_t) m * n + n0 + r) * width + i, y);
        }
    }
}

// out[n][c] = -log2(e) exp(w0[c] + sum_r tanh(t[n][r]) w2[c][r])
__device__ __forceinline__ float decay_log2_f(float z) { return -1.4426950408889634f * expf(z); }

// bfloat16 weights: a float32 factor is three bfloat16 pieces (8 + 8 + 8 bits of its 24), so three products on the bfloat16 matrix instruction are the float32 product
// with an exact weight.  A wave takes 16 rows (their tanh is computed once, in registers) and 256 channels; weights come straight from memory as operands, 16 bytes per
// lane.  The result tile is [channel][row]: a lane holds four neighbouring channels of one row.
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
#define DB_COLS 256
#define DB_ROWS 64
__global__ __launch_bounds__(256) void decay_log2_bf16_kernel(float* __restrict__ out, const bf16_t* __restrict__ t, int64_t t_ld, const bf16_t* __restrict__ w2,
                                                              const float* __restrict__ w0, int n, int channels, int rank)
{
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, g = lane >> 4, c = lane & 15;
    const int n0 = blockIdx.x * DB_ROWS + w * 16, c0 = blockIdx.y * DB_COLS;
    if (n0 >= n) return;
    const bf16_t* tr = t + (int64_t) min(n0 + c, n - 1) * t_ld;       // rows beyond the last: computed and never stored
    f32x4 acc[DB_COLS / 16];
    #pragma unroll
    for (int b = 0; b < DB_COLS / 16; ++b) acc[b] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < rank; k0 += 32)                             // rank is a multiple of 8: a lane's eight entries are all there or none
    {
        const int k = k0 + g * 8;
        const bool ok = k < rank;
        bf16x8 p0, p1, p2;
        float f[8];
        #pragma unroll
        for (int e = 0; e < 8; ++e) f[e] = 0.f;
        if (ok) load_n<bf16_t, 8>(tr + k, f);
        #pragma unroll
        for (int e = 0; e < 8; ++e)
        {
            const float y = tanhf(f[e]);
            p0[e] = (__bf16) y;
            const float y1 = y - (float) p0[e];
            p1[e] = (__bf16) y1;
            p2[e] = (__bf16) (y1 - (float) p1[e]);
        }
        #pragma unroll
        for (int b = 0; b < DB_COLS / 16; ++b)
        {
            const int col = c0 + b * 16 + c;
            union { bf16x8 v; uint4 x; } a;
            a.x = (ok && col < channels) ? *(const uint4*) (w2 + (int64_t) col * rank + k) : uint4{0u, 0u, 0u, 0u};
            acc[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, p2, acc[b], 0, 0, 0);
            acc[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, p1, acc[b], 0, 0, 0);
            acc[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, p0, acc[b], 0, 0, 0);
        }
    }
    if (n0 + c >= n) return;
    float* dst = out + (int64_t) (n0 + c) * channels;
    #pragma unroll
    for (int b = 0; b < DB_COLS / 16; ++b)
    {
        const int col = c0 + b * 16 + 4 * g;                          // channels is a multiple of 4
        if (col >= channels) break;
        float z[4], y[4];
        load_n<float, 4>(w0 + col, z);
        #pragma unroll
        for (int i = 0; i < 4; ++i) y[i] = decay_log2_f(acc[b][i] + z[i]);
        store_n<float, 4>(dst + col, y);
    }
}

// Any sizes and float32 weights, on the float32 matrix instruction: 32 rows x 256 channels per workgroup, a wave takes 64 of the channels
#define DL_ROWS 32
#define DL_COLS 256
#define DL_K 32
template <typename T>
__global__ __launch_bounds__(256) void decay_log2_kernel(float* __restrict__ out, const T* __restrict__ t, int64_t t_ld, const T* __restrict__ w2, const float* __restrict__ w0, int n,
                                                        int channels, int rank)
{
    __shared__ __attribute__((aligned(16))) float ts[DL_ROWS * (DL_K + 4)];
    __shared__ __attribute__((aligned(16))) float wsm[DL_COLS * (DL_K + 4)];
    const int n0 = blockIdx.x * DL_ROWS, c0 = blockIdx.y * DL_COLS;
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, g = lane >> 4, c = lane & 15;
    f32x4 acc[2][4];
    #pragma unroll
    for (int a = 0; a < 2; ++a)
    {
        #pragma unroll
        for (int b = 0; b < 4; ++b) acc[a][b] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    for (int k0 = 0; k0 < rank; k0 += DL_K)
    {
        __syncthreads();
        for (int idx = threadIdx.x; idx < DL_ROWS * DL_K; idx += 256)
        {
            const int r = idx / DL_K, k = idx - r * DL_K;
            ts[r * (DL_K + 4) + k] = (n0 + r < n && k0 + k < rank) ? tanhf(to_f(t[(int64_t) (n0 + r) * t_ld + k0 + k])) : 0.f;
        }
        #pragma unroll 8
        for (int idx = threadIdx.x; idx < DL_COLS * DL_K; idx += 256)
        {
            const int r = idx / DL_K, k = idx - r * DL_K;
            wsm[r * (DL_K + 4) + k] = (c0 + r < channels && k0 + k < rank) ? to_f(w2[(int64_t) (c0 + r) * rank + k0 + k]) : 0.f;
        }
        __syncthreads();
        #pragma unroll
        for (int kt = 0; kt < DL_K / 16; ++kt)
        {
            f32x4 av[2], bv[4];
            #pragma unroll
            for (int a = 0; a < 2; ++a) av[a] = *(const f32x4*) (ts + (a * 16 + c) * (DL_K + 4) + kt * 16 + 4 * g);
            #pragma unroll
            for (int b = 0; b < 4; ++b) bv[b] = *(const f32x4*) (wsm + (w * 64 + b * 16 + c) * (DL_K + 4) + kt * 16 + 4 * g);
            #pragma unroll
            for (int i = 0; i < 4; ++i)
            {
                #pragma unroll
                for (int a = 0; a < 2; ++a)
                {
                    #pragma unroll
                    for (int b = 0; b < 4; ++b) acc[a][b] = __builtin_amdgcn_mfma_f32_16x16x4f32(av[a][i], bv[b][i], acc[a][b], 0, 0, 0);
                }
            }
        }
    }
    #pragma unroll
    for (int b = 0; b < 4; ++b)
    {
        const int col = c0 + w * 64 + b * 16 + c;
        if (col >= channels) continue;
        const float z0 = w0[col];
        #pragma unroll
        for (int a = 0; a < 2; ++a)
        {
            #pragma unroll
            for (int i = 0; i < 4; ++i)
            {
                const int row = n0 + a * 16 + 4 * g + i;
                if (row < n) out[(int64_t) row * channels + col] = decay_log2_f(acc[a][b][i] + z0);
            }
        }
    }
}

// A loaded element that waits in a register of its own: 16-bit elements would be packed in pairs, and packing waits for the loads
template <typename T> struct in_flight;
template <> struct in_flight<bf16_t>
{
    uint32_t u;
    __device__ __forceinline__ void load(const bf16_t* p) { u = p->u; }
    __device__ __forceinline__ float value() const { return __uint_as_float(u << 16); }
    __device__ __forceinline__ void arrive() { asm volatile("" : "+v"(u)); }
};
template <> struct in_flight<float>
{
    float f;
    __device__ __forceinline__ void load(const float* p) { f = *p; }
    __device__ __forceinline__ float value() const { return f; }
    __device__ __forceinline__ void arrive() { asm volatile("" : "+v"(f)); }
};

// DT: 16-row blocks of the (zero-padded) key dim.  Preparation: wave w owns the tile's tokens 4w .. 4w + 3, lane l the channels l, l + 64, ...
// FUSED (vdim <= 64): out receives the heads after norm and gate, o / rms(o) * norm_w * silu(gate), instead of o.
template <typename T, int DT, int MODE, bool FUSED>
__global__ __launch_bounds__(TM_THREADS, DT <= 4 ? 3 : (DT <= 8 ? 2 : 1)) void timemix_chunk_kernel(float* __restrict__ o, T* __restrict__ out, int64_t out_ld, const T* __restrict__ gate, int64_t gate_ld,
                                                                   const float* __restrict__ norm_w, float eps, float* __restrict__ state,
                                                                   const T* __restrict__ r, int64_t r_ld, const T* __restrict__ k, int64_t k_ld, const T* __restrict__ v, int64_t v_ld,
                                                                   const float* __restrict__ log2w, const float* __restrict__ u, const int32_t* __restrict__ cu,
                                                                   const int32_t* __restrict__ slots, const int32_t* __restrict__ pos0, int heads, int dim, int vdim,
                                                                   int segs, int seg_len, float* __restrict__ seg_state, float* __restrict__ seg_decay)
{
    constexpr int DP = DT * 16, LS = DP + 4, CI = (DP + 63) / 64, PS = TM_TILE + 4, TW = TM_TILE / TM_WAVES;
    static_assert(TW == 4, "a wave prepares four tokens, a lane holds the values of four");
    constexpr bool READ = MODE != TM_SEG_LOCAL;
    constexpr int WP = READ && TM_WAVES * PS > LS ? TM_TILE * TM_WAVES * PS : TM_TILE * LS;
    __shared__ __attribute__((aligned(16))) float ks[TM_TILE * LS], ws[WP];
    __shared__ __attribute__((aligned(16))) float rs[READ ? TM_TILE * LS : 4];
    float* const ps = ws;                                             // a tile needs either its decays one by one or the partial scores
    __shared__ __attribute__((aligned(16))) float em[DP], et[DP];
    __shared__ __attribute__((aligned(16))) float dg[2][TM_TILE][4], tot[2][TM_WAVES][CI * 64], red[TM_WAVES][TM_TILE];
    const int b = (MODE == TM_WHOLE) ? blockIdx.x : blockIdx.x / segs, h = blockIdx.y;
    const int lane = threadIdx.x & 63, w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g = lane >> 4, c = lane & 15;
    const int col = blockIdx.z * TM_COLS + w * 16 + c;
    const bool col_ok = col < vdim;
    int first = cu[b], last = cu[b + 1];
    float* st = state + ((int64_t) slots[b] * heads + h) * dim * vdim;
    bool resume = pos0[b] > 0;
    if (MODE != TM_WHOLE)
    {
        first += (blockIdx.x - b * segs) * seg_len;
        last = min(last, first + seg_len);
        if (first >= last) return;                                    // uniform: a shorter sequence has fewer segments
        st = seg_state + ((int64_t) blockIdx.x * heads + h) * dim * vdim;
        resume = (MODE == TM_SEG_FINAL);
    }
    f32x4 S[DT];
    #pragma unroll
    for (int kt = 0; kt < DT; ++kt)
    {
        #pragma unroll
        for (int i = 0; i < 4; ++i)
        {
            const int row = kt * 16 + 4 * g + i;
            S[kt][i] = (resume && col_ok && row < dim) ? st[(int64_t) row * vdim + col] : 0.f;
        }
    }
    float uc[CI], seg_sum[CI];
    #pragma unroll
    for (int ci = 0; ci < CI; ++ci)
    {
        uc[ci] = (READ && lane + 64 * ci < dim) ? u[h * dim + lane + 64 * ci] : 0.f;
        seg_sum[ci] = 0.f;
    }
    // The rows of the next tile wait in registers, as loaded, while the current one is computed.  Nothing is conditional: places beyond the tile, the key dim or the value
    // dim read their nearest neighbour; where the value matters (k and the decays) it is replaced when it is used.
    in_flight<T> tr[CI][TW], tk[CI][TW], tv[4], tg[4];
    in_flight<float> tw[CI][TW];
    int chc[CI];
    #pragma unroll
    for (int ci = 0; ci < CI; ++ci) chc[ci] = min(lane + 64 * ci, dim - 1);
    const int colc = min(col, vdim - 1);
    const float inv_vdim = 1.0f / (float) vdim;
    const float nw = FUSED ? norm_w[h * vdim + colc] : 0.f;
    auto fetch = [&](int n0) __attribute__((always_inline))
    {
        #pragma unroll
        for (int j = 0; j < TW; ++j)
        {
            const int t = min(n0 + w * TW + j, last - 1);             // the same for the whole wave: a lane adds its channel to a scalar address
            const T* kr = k + (int64_t) t * k_ld + h * dim;
            const T* rr = r + (int64_t) t * r_ld + h * dim;
            const float* wr = log2w + ((int64_t) t * heads + h) * dim;
            #pragma unroll
            for (int ci = 0; ci < CI; ++ci)
            {
                tk[ci][j].load(kr + chc[ci]);
                tw[ci][j].load(wr + chc[ci]);
                if (READ) tr[ci][j].load(rr + chc[ci]);
            }
        }
        const T* vb = v + (int64_t) n0 * v_ld + h * vdim;
        const T* gb = FUSED ? gate + (int64_t) n0 * gate_ld + h * vdim : nullptr;
        #pragma unroll
        for (int i = 0; i < 4; ++i)
        {
            const int t = min(4 * g + i, last - 1 - n0);
            tv[i].load(vb + t * (int) v_ld + colc);
            if (FUSED) tg[i].load(gb + t * (int) gate_ld + colc);
        }
    };
    fetch(first);
    int par = 0;
    for (int n0 = first; n0 < last; n0 += TM_TILE, par ^= 1)
    {
        const int tc = min(TM_TILE, last - n0);
        float vr[4], gr[4];
        float bonus[TW];
        #pragma unroll
        for (int j = 0; j < TW; ++j) bonus[j] = 0.f;
        float kf[CI][TW];
        #pragma unroll
        for (int ci = 0; ci < CI; ++ci)
        {
            float sum = 0.f;
            #pragma unroll
            for (int j = 0; j < TW; ++j)
            {
                const bool ok = w * TW + j < tc && lane + 64 * ci < dim;
                kf[ci][j] = ok ? tk[ci][j].value() : 0.f;
                tw[ci][j].f = ok ? tw[ci][j].f : 0.f;
                sum += tw[ci][j].f;
                if (READ) bonus[j] = __builtin_fmaf(tr[ci][j].value() * uc[ci], kf[ci][j], bonus[j]);
            }
            tot[par][w][lane + 64 * ci] = sum;
        }
        #pragma unroll
        for (int i = 0; i < 4; ++i)
        {
            vr[i] = tv[i].value();
            if (FUSED) { const float z = tg[i].value(); gr[i] = z * nw * __builtin_amdgcn_rcpf(1.0f + TM_EXP2(z * -1.4426950408889634f)); }
        }
        if (READ)
        {
            #pragma unroll
            for (int j = 0; j < TW; ++j)
            {
                const float s = row16_sum(bonus[j]);
                if (c == 0) dg[par][w * TW + j][g] = s;
            }
        }
        __syncthreads();                                              // tot and dg are there; the previous tile's reads of everything else are over
        bool strong = false;
        float half0[CI], half1[CI], base[CI];
        #pragma unroll
        for (int ci = 0; ci < CI; ++ci)
        {
            const int ch = lane + 64 * ci;
            const float a0 = tot[par][0][ch], a1 = tot[par][1][ch], a2 = tot[par][2][ch], a3 = tot[par][3][ch];
            half0[ci] = a0 + a1; half1[ci] = a2 + a3;
            base[ci] = w == 0 ? -half0[ci] : (w == 1 ? -a1 : (w == 2 ? 0.f : a2));      // the exponent ahead of this wave's first token, counted from the middle
            strong = strong || half0[ci] < -TM_MAX_EXP || half1[ci] < -TM_MAX_EXP;
            seg_sum[ci] += half0[ci] + half1[ci];
        }
        const bool slow = __any(strong);                              // every wave looks at every channel: the same answer in all of them
        #pragma unroll
        for (int ci = 0; ci < CI; ++ci)
        {
            const int ch = lane + 64 * ci;
            if (ch < DP)
            {
                float e = base[ci];
                #pragma unroll
                for (int j = 0; j < TW; ++j)
                {
                    const int at = (w * TW + j) * LS + ch;
                    if (slow)
                    {
                        if (READ) rs[at] = tr[ci][j].value();
                        ks[at] = kf[ci][j];
                        ws[at] = TM_EXP2(tw[ci][j].f);
                    }
                    else
                    {
                        if (READ) rs[at] = tr[ci][j].value() * TM_EXP2(e);
                        e += tw[ci][j].f;
                        ks[at] = kf[ci][j] * TM_EXP2(-e);
                    }
                }
                if (w == 0) em[ch] = TM_EXP2(half0[ci]);
                if (w == 3) et[ch] = TM_EXP2(half1[ci]);
            }
        }
        __syncthreads();
        if (n0 + TM_TILE < last) fetch(n0 + TM_TILE);                 // under the tile's matrix work
        f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
        if (slow)
        {
            #pragma unroll 1                                          // rolled: the rare path must not cost the other one registers
            for (int t = 0; t < tc; ++t)
            {
                const int tg4 = t >> 2, ti = t & 3;
                const float own = ti == 0 ? vr[0] : (ti == 1 ? vr[1] : (ti == 2 ? vr[2] : vr[3]));
                const float vv = __shfl(own, tg4 * 16 + c, 64);
                float po = 0.f;
                #pragma unroll
                for (int kt = 0; kt < DT; ++kt)
                {
                    const int at = t * LS + kt * 16 + 4 * g;
                    if (READ)
                    {
                        const f32x4 rr = *(const f32x4*) (rs + at);
                        #pragma unroll
                        for (int i = 0; i < 4; ++i) po = __builtin_fmaf(rr[i], S[kt][i], po);
                    }
                    const f32x4 kk = *(const f32x4*) (ks + at), dd = *(const f32x4*) (ws + at);
                    #pragma unroll
                    for (int i = 0; i < 4; ++i) S[kt][i] = __builtin_fmaf(dd[i], S[kt][i], kk[i] * vv);
                    __builtin_amdgcn_sched_barrier(0);
                }
                if (READ)
                {
                    po += __shfl_xor(po, 16, 64);
                    po += __shfl_xor(po, 32, 64);
                    const f32x4 o4 = *(const f32x4*) dg[par][t];
                    po = __builtin_fmaf((o4[0] + o4[1]) + (o4[2] + o4[3]), vv, po);
                    #pragma unroll
                    for (int i = 0; i < 4; ++i) acc[i] = (g == tg4 && ti == i) ? po : acc[i];
                }
            }
        }
        else
        {
            #pragma unroll
            for (int kt = 0; kt < DT; ++kt) S[kt] *= *(const f32x4*) (em + kt * 16 + 4 * g);
            if (READ)
            {
                // the scores' contraction is shared out over the waves; partial tiles meet in LDS
                f32x4 sc = f32x4{0.f, 0.f, 0.f, 0.f};
                #pragma unroll
                for (int m = 0; m < (DT + TM_WAVES - 1) / TM_WAVES; ++m)
                {
                    const int kt = w + TM_WAVES * m;
                    if (DT % TM_WAVES != 0 && kt >= DT) break;        // uniform for the wave
                    const f32x4 a = *(const f32x4*) (rs + c * LS + kt * 16 + 4 * g), bk = *(const f32x4*) (ks + c * LS + kt * 16 + 4 * g);
                    #pragma unroll
                    for (int i = 0; i < 4; ++i) sc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], bk[i], sc, 0, 0, 0);
                }
                #pragma unroll
                for (int kt = 0; kt < DT; ++kt)
                {
                    const f32x4 a = *(const f32x4*) (rs + c * LS + kt * 16 + 4 * g);
                    #pragma unroll
                    for (int i = 0; i < 4; ++i) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], S[kt][i], acc, 0, 0, 0);
                }
                #pragma unroll
                for (int i = 0; i < 4; ++i) ps[(w * TM_TILE + 4 * g + i) * PS + c] = 4 * g + i > c ? sc[i] : 0.f;
                __syncthreads();
                f32x4 a = *(const f32x4*) (ps + c * PS + 4 * g);
                #pragma unroll
                for (int ww = 1; ww < TM_WAVES; ++ww) a += *(const f32x4*) (ps + (ww * TM_TILE + c) * PS + 4 * g);
                const f32x4 o4 = *(const f32x4*) dg[par][c];
                const float own = (o4[0] + o4[1]) + (o4[2] + o4[3]);
                #pragma unroll
                for (int i = 0; i < 4; ++i)
                {
                    if (4 * g + i == c) a[i] = own;
                    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], vr[i], acc, 0, 0, 0);
                }
            }
            #pragma unroll
            for (int i = 0; i < 4; ++i)
            {
                #pragma unroll
                for (int kt = 0; kt < DT; ++kt) S[kt] = __builtin_amdgcn_mfma_f32_16x16x4f32(ks[(4 * g + i) * LS + kt * 16 + c], vr[i], S[kt], 0, 0, 0);
            }
            #pragma unroll
            for (int kt = 0; kt < DT; ++kt) S[kt] *= *(const f32x4*) (et + kt * 16 + 4 * g);
        }
        if (!READ) continue;
        // the next tile's rows have had the matrix work's time to arrive; waiting for them here, ahead of this tile's stores, keeps the stores out of that wait
        #pragma unroll
        for (int j = 0; j < TW; ++j)
        {
            #pragma unroll
            for (int ci = 0; ci < CI; ++ci) { tk[ci][j].arrive(); tr[ci][j].arrive(); tw[ci][j].arrive(); }
            tv[j].arrive();
            if (FUSED) tg[j].arrive();
        }
        if (FUSED)
        {
            #pragma unroll
            for (int i = 0; i < 4; ++i)
            {
                const float s = row16_sum(col_ok ? acc[i] * acc[i] : 0.f);
                if (c == 0) red[w][4 * g + i] = s;
            }
            __syncthreads();
            const f32x4 ss = (*(const f32x4*) (red[0] + 4 * g) + *(const f32x4*) (red[1] + 4 * g)) + (*(const f32x4*) (red[2] + 4 * g) + *(const f32x4*) (red[3] + 4 * g));
            T* ob = out + (int64_t) n0 * out_ld + h * vdim;
            #pragma unroll
            for (int i = 0; i < 4; ++i)
            {
                const float y = acc[i] * __builtin_amdgcn_rsqf(ss[i] * inv_vdim + eps) * gr[i];
                if (4 * g + i < tc && col_ok) ob[(4 * g + i) * (int) out_ld + col] = from_f<T>(y);
            }
            continue;
        }
        float* ob = o + ((int64_t) n0 * heads + h) * vdim;
        #pragma unroll
        for (int i = 0; i < 4; ++i)
            if (4 * g + i < tc && col_ok) ob[(4 * g + i) * heads * vdim + col] = acc[i];
    }
    if (MODE == TM_SEG_FINAL) return;
    #pragma unroll
    for (int kt = 0; kt < DT; ++kt)
    {
        #pragma unroll
        for (int i = 0; i < 4; ++i)
        {
            const int row = kt * 16 + 4 * g + i;
            if (col_ok && row < dim) st[(int64_t) row * vdim + col] = S[kt][i];
        }
    }
    if (MODE == TM_SEG_LOCAL && blockIdx.z == 0 && w == 0)
    {
        #pragma unroll
        for (int ci = 0; ci < CI; ++ci)
        {
            const int ch = lane + 64 * ci;
            if (ch < dim) seg_decay[((int64_t) blockIdx.x * heads + h) * dim + ch] = TM_EXP2(seg_sum[ci]);
        }
    }
}

// Between the two segment passes: every segment's own contribution in seg_state becomes the state it starts from; the state after the last one goes to the slot.
#define TM_AHEAD 8
__global__ __launch_bounds__(256) void timemix_combine_kernel(float* __restrict__ state, float* seg_state, const float* __restrict__ seg_decay, const int32_t* __restrict__ cu,
                                                              const int32_t* __restrict__ slots, const int32_t* __restrict__ pos0, int heads, int dim, int vdim, int segs, int seg_len)
{
    const int b = blockIdx.x, h = blockIdx.y;
    const int64_t per = (int64_t) dim * vdim;
    const int used = min(segs, (cu[b + 1] - cu[b] + seg_len - 1) / seg_len);
    float* st = state + ((int64_t) slots[b] * heads + h) * per;
    const int64_t e = (int64_t) blockIdx.z * 256 + threadIdx.x;
    if (e >= per) return;
    const int row = (int) (e / vdim);
    float S = pos0[b] > 0 ? st[e] : 0.f;
    for (int s0 = 0; s0 < used; s0 += TM_AHEAD)                       // several segments' loads in flight, then their sums in order
    {
        float local[TM_AHEAD], dec[TM_AHEAD];
        #pragma unroll
        for (int x = 0; x < TM_AHEAD; ++x)
        {
            const int64_t blk = ((int64_t) b * segs + s0 + x) * heads + h;
            const bool ok = s0 + x < used;
            local[x] = ok ? seg_state[blk * per + e] : 0.f;
            dec[x] = ok ? seg_decay[blk * dim + row] : 1.f;
        }
        #pragma unroll
        for (int x = 0; x < TM_AHEAD; ++x)
        {
            if (s0 + x >= used) break;
            seg_state[(((int64_t) b * segs + s0 + x) * heads + h) * per + e] = S;
            S = __builtin_fmaf(dec[x], S, local[x]);
        }
    }
    st[e] = S;
}

// Steps of one row per sequence, one workgroup per (sequence, head).  Eight lanes share a channel's low-rank product; then a thread owns V neighbouring value columns of
// every (threads / column groups)-th row of the state; partial read-outs meet in LDS.  out = o / rms(o) * norm_w * silu(gate).
#define TS_THREADS 512
template <typename T, int V>
__global__ __launch_bounds__(TS_THREADS) void timemix_step_kernel(T* __restrict__ out, int64_t out_ld, float* __restrict__ state, const T* __restrict__ r, int64_t r_ld,
                                                                  const T* __restrict__ k, int64_t k_ld, const T* __restrict__ v, int64_t v_ld, const T* __restrict__ gate, int64_t gate_ld,
                                                                  const T* __restrict__ t, int64_t t_ld, const T* __restrict__ w2, const float* __restrict__ w0,
                                                                  const float* __restrict__ u, const float* __restrict__ norm_w, const int32_t* __restrict__ tok_pos,
                                                                  const int32_t* __restrict__ slots, int heads, int dim, int vdim, int rank, float eps, int w_vec)
{
    extern __shared__ __attribute__((aligned(16))) float smem[];
    __shared__ float red[TS_THREADS / 64];
    const int cg = (vdim + V - 1) / V;                                // column groups (vdim is a multiple of V)
    const int rp = TS_THREADS / cg;                                   // rows of the state in flight
    float* part = smem;                                               // [rp][vdim]
    float* rk = part + rp * vdim;                                     // [dim] r
    float* kk = rk + dim;                                             // [dim] k
    float* dc = kk + dim;                                             // [dim] decay
    float* ub = dc + dim;                                             // [dim] r u k
    float* th = ub + dim;                                             // [rank] tanh of the low-rank input
    const int n = blockIdx.x, h = blockIdx.y;
    const int sub = threadIdx.x & 7, ch0 = threadIdx.x >> 3;
    const int r0 = threadIdx.x / cg, c0 = (threadIdx.x - r0 * cg) * V;
    const bool live = r0 < rp, resume = tok_pos[n] > 0;
    float* st = state + ((int64_t) slots[n] * heads + h) * dim * vdim;
    // what the first pass of each loop below needs is on its way before the first barrier: eight entries of a channel's weights, two pieces of the state
    float wreg[8], held[2][V];
    if (w_vec && ch0 < dim && sub * 8 < rank) load_n<T, 8>(w2 + ((int64_t) h * dim + ch0) * rank + sub * 8, wreg);
    #pragma unroll
    for (int x = 0; x < 2; ++x)
    {
        #pragma unroll
        for (int e = 0; e < V; ++e) held[x][e] = 0.f;
        if (live && resume && r0 + x * rp < dim) load_n<float, V>(st + (int64_t) (r0 + x * rp) * vdim + c0, held[x]);
    }
    for (int i = threadIdx.x; i < dim; i += TS_THREADS)
    {
        const int64_t at = (int64_t) h * dim + i;
        const float a = to_f(r[(int64_t) n * r_ld + at]), b = to_f(k[(int64_t) n * k_ld + at]);
        rk[i] = a; kk[i] = b; ub[i] = a * u[at] * b;
    }
    for (int i = threadIdx.x; i < rank; i += TS_THREADS) th[i] = tanhf(to_f(t[(int64_t) n * t_ld + i]));
    __syncthreads();
    for (int i0 = 0; i0 < dim; i0 += TS_THREADS / 8)                  // uniform trip count: the shuffles see whole groups of eight
    {
        const int i = i0 + ch0;
        float z = 0.f;
        if (i < dim)
        {
            const T* wr = w2 + ((int64_t) h * dim + i) * rank;
            if (w_vec)
            {
                for (int x = sub * 8; x < rank; x += 64)
                {
                    if (i0 > 0 || x >= 64) load_n<T, 8>(wr + x, wreg);
                    #pragma unroll
                    for (int e = 0; e < 8; ++e) z = __builtin_fmaf(th[x + e], wreg[e], z);
                }
            }
            else for (int x = sub; x < rank; x += 8) z = __builtin_fmaf(th[x], to_f(wr[x]), z);
        }
        z += __shfl_xor(z, 1, 64); z += __shfl_xor(z, 2, 64); z += __shfl_xor(z, 4, 64);
        if (i < dim && sub == 0) dc[i] = expf(-expf(z + w0[(int64_t) h * dim + i]));
    }
    __syncthreads();
    if (live)
    {
        float vv[V], acc[V];
        #pragma unroll
        for (int e = 0; e < V; ++e) { vv[e] = to_f(v[(int64_t) n * v_ld + (int64_t) h * vdim + c0 + e]); acc[e] = 0.f; }
        auto visit = [&](int row, float (&s)[V]) __attribute__((always_inline))
        {
            const float kx = kk[row], rx = rk[row], dx = dc[row], ux = ub[row];
            #pragma unroll
            for (int e = 0; e < V; ++e)
            {
                acc[e] = __builtin_fmaf(rx, s[e], __builtin_fmaf(ux, vv[e], acc[e]));
                s[e] = __builtin_fmaf(dx, s[e], kx * vv[e]);
            }
            store_n<float, V>(st + (int64_t) row * vdim + c0, s);
        };
        #pragma unroll
        for (int x = 0; x < 2; ++x)
            if (r0 + x * rp < dim) visit(r0 + x * rp, held[x]);
        #pragma unroll 4
        for (int row = r0 + 2 * rp; row < dim; row += rp)
        {
            float s[V];
            #pragma unroll
            for (int e = 0; e < V; ++e) s[e] = 0.f;
            if (resume) load_n<float, V>(st + (int64_t) row * vdim + c0, s);
            visit(row, s);
        }
        #pragma unroll
        for (int e = 0; e < V; ++e) part[r0 * vdim + c0 + e] = acc[e];
    }
    __syncthreads();
    float ss = 0.f;
    for (int c = threadIdx.x; c < vdim; c += TS_THREADS)
    {
        float s = 0.f;
        for (int x = 0; x < rp; ++x) s += part[x * vdim + c];
        part[c] = s;                                                  // the column's own first row: read by this thread only
        ss += s * s;
    }
    ss = block_sum<TS_THREADS / 64>(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float) vdim + eps);
    for (int c = threadIdx.x; c < vdim; c += TS_THREADS)
    {
        const int64_t at = (int64_t) h * vdim + c;
        out[(int64_t) n * out_ld + at] = from_f<T>(part[c] * inv * norm_w[at] * silu_f(to_f(gate[(int64_t) n * gate_ld + at])));
    }
}

extern "C" int exl3_mix_token_shift(void* out, const void* h, int64_t h_ld, void* last, const float* mu, int mixes, const int32_t* tok_seq, const int32_t* tok_pos, const int32_t* slots,
                                    const int32_t* pos0, const int32_t* len_after, int n, int width, int dtype, void* stream)
{
    MIX_CHECK(out && h && last && mu && tok_seq && tok_pos && slots && pos0 && len_after, "mix_token_shift: null pointer");
    MIX_CHECK(n >= 0 && width > 0 && mixes >= 1 && h_ld >= width && out != h, "mix_token_shift: bad sizes");
    if (n == 0) return EXL3_MIX_OK;
    const int vn = dtype == EXL3_MIX_BF16 ? 8 : 4;
    const bool vec = width % vn == 0 && h_ld % vn == 0 && (uintptr_t) out % 16 == 0 && (uintptr_t) h % 16 == 0 && (uintptr_t) last % 16 == 0;
    #define SH_LAUNCH(VV, RR) hipLaunchKernelGGL((token_shift_kernel<T, VV, RR>), dim3((n + RR - 1) / RR, (width + 256 * VV - 1) / (256 * VV)), dim3(256), 0, (hipStream_t) stream, \
                                                 (T*) out, (const T*) h, h_ld, (T*) last, mu, mixes, tok_seq, tok_pos, slots, pos0, len_after, n, width)
    MIX_CHECK((width + 255) / 256 <= 65535, "mix_token_shift: width %d", width);
    if (dtype == EXL3_MIX_BF16)
    {
        using T = bf16_t;
        if (vec) { if (n >= 1024) SH_LAUNCH(8, 4); else SH_LAUNCH(8, 1); } else SH_LAUNCH(1, 1);
    }
    else
    {
        using T = float;
        if (vec) { if (n >= 1024) SH_LAUNCH(4, 4); else SH_LAUNCH(4, 1); } else SH_LAUNCH(1, 1);
    }
    #undef SH_LAUNCH
    return mix_check_launch("mix_token_shift");
}

extern "C" int exl3_mix_decay_log2(float* out, const void* t, int64_t t_ld, const void* w2, const float* w0, int n, int channels, int rank, int dtype, void* stream)
{
    MIX_CHECK(out && t && w2 && w0 && n >= 0 && channels > 0 && rank > 0 && t_ld >= rank && (channels + DL_COLS - 1) / DL_COLS <= 65535, "mix_decay_log2: bad arguments");
    if (n == 0) return EXL3_MIX_OK;
    if (dtype == EXL3_MIX_BF16 && rank % 8 == 0 && t_ld % 8 == 0 && channels % 4 == 0 && (uintptr_t) t % 16 == 0 && (uintptr_t) w2 % 16 == 0 && (uintptr_t) w0 % 16 == 0 && (uintptr_t) out % 16 == 0)
    {
        hipLaunchKernelGGL(decay_log2_bf16_kernel, dim3((n + DB_ROWS - 1) / DB_ROWS, (channels + DB_COLS - 1) / DB_COLS), dim3(256), 0, (hipStream_t) stream, out, (const bf16_t*) t, t_ld,
                           (const bf16_t*) w2, w0, n, channels, rank);
        return mix_check_launch("mix_decay_log2");
    }
    MIX_DISPATCH_T(dtype, hipLaunchKernelGGL(decay_log2_kernel<T>, dim3((n + DL_ROWS - 1) / DL_ROWS, (channels + DL_COLS - 1) / DL_COLS), dim3(256), 0, (hipStream_t) stream, out, (const T*) t,
                                             t_ld, (const T*) w2, w0, n, channels, rank));
    return mix_check_launch("mix_decay_log2");
}

static int timemix_check(const char* what, int heads, int dim, int vdim)
{
    MIX_CHECK(heads > 0 && heads <= 65535 && dim > 0 && dim <= 256 && vdim > 0 && vdim <= 1024, "%s: dim %d (<= 256) / vdim %d (<= 1024) out of range", what, dim, vdim);
    return EXL3_MIX_OK;
}

template <int MODEV>
static int timemix_launch(float* o, void* out, int64_t out_ld, const void* gate, int64_t gate_ld, const float* norm_w, float eps, float* state, const void* r, int64_t r_ld, const void* k,
                          int64_t k_ld, const void* v, int64_t v_ld, const float* log2w, const float* u, const int32_t* cu, const int32_t* slots, const int32_t* pos0, int batch, int heads,
                          int dim, int vdim, int segs, int seg_len, float* seg_state, float* seg_decay, int dtype, void* stream)
{
    const dim3 grid(batch * segs, heads, (vdim + TM_COLS - 1) / TM_COLS);
    #define TM_LAUNCH_F(DTV, FV) hipLaunchKernelGGL((timemix_chunk_kernel<T, DTV, MODEV, FV>), grid, dim3(TM_THREADS), 0, (hipStream_t) stream, o, (T*) out, out_ld, (const T*) gate, gate_ld, norm_w, \
                                              eps, state, (const T*) r, r_ld, (const T*) k, k_ld, (const T*) v, v_ld, log2w, u, cu, slots, pos0, heads, dim, vdim, segs, seg_len, seg_state, \
                                              seg_decay)
    #define TM_LAUNCH(DTV) do { if (MODEV != TM_SEG_LOCAL && out) TM_LAUNCH_F(DTV, (MODEV != TM_SEG_LOCAL)); else TM_LAUNCH_F(DTV, false); } while (0)
    MIX_DISPATCH_T(dtype, if (dim <= 32) TM_LAUNCH(2); else if (dim <= 48) TM_LAUNCH(3); else if (dim <= 64) TM_LAUNCH(4); else if (dim <= 128) TM_LAUNCH(8); else TM_LAUNCH(16));
    #undef TM_LAUNCH
    #undef TM_LAUNCH_F
    return mix_check_launch("mix_timemix");
}

extern "C" int exl3_mix_timemix(float* o, void* out, int64_t out_ld, const void* gate, int64_t gate_ld, const float* norm_w, float eps, float* state, const void* r, int64_t r_ld,
                                const void* k, int64_t k_ld, const void* v, int64_t v_ld, const float* log2w, const float* u, const int32_t* cu, const int32_t* slots,
                                const int32_t* pos0, int batch, int heads, int dim, int vdim, int segs, int seg_len, float* seg_state, float* seg_decay, int dtype, void* stream)
{
    MIX_CHECK((o || out) && state && r && k && v && log2w && u && cu && slots && pos0 && batch >= 0, "mix_timemix: null pointer");
    if (int rc = timemix_check("mix_timemix", heads, dim, vdim)) return rc;
    MIX_CHECK(r_ld >= (int64_t) heads * dim && k_ld >= (int64_t) heads * dim && v_ld >= (int64_t) heads * vdim && v_ld <= (1 << 26), "mix_timemix: bad row strides");
    MIX_CHECK(!out || (gate && norm_w && vdim <= TM_COLS && out_ld >= (int64_t) heads * vdim && gate_ld >= (int64_t) heads * vdim && gate_ld <= (1 << 26) && out_ld <= (1 << 26)),
              "mix_timemix: norm and gate in the same launch need vdim <= %d, the gate and the weight", TM_COLS);
    MIX_CHECK(segs >= 1 && (segs == 1 || (seg_len >= 1 && seg_state && seg_decay)), "mix_timemix: bad segment arguments");
    if (batch == 0) return EXL3_MIX_OK;
    #define TM_ARGS o, out, out_ld, gate, gate_ld, norm_w, eps, state, r, r_ld, k, k_ld, v, v_ld, log2w, u, cu, slots, pos0, batch, heads, dim, vdim, segs, seg_len, seg_state, seg_decay, dtype, stream
    if (segs == 1) return timemix_launch<TM_WHOLE>(TM_ARGS);
    int rc = timemix_launch<TM_SEG_LOCAL>(TM_ARGS);
    if (rc) return rc;
    const int64_t per = (int64_t) dim * vdim;
    hipLaunchKernelGGL(timemix_combine_kernel, dim3(batch, heads, (unsigned) ((per + 255) / 256)), dim3(256), 0, (hipStream_t) stream, state, seg_state, seg_decay, cu, slots, pos0, heads, dim,
                       vdim, segs, seg_len);
    if ((rc = mix_check_launch("mix_timemix (combine)"))) return rc;
    return timemix_launch<TM_SEG_FINAL>(TM_ARGS);
    #undef TM_ARGS
}

extern "C" int exl3_mix_timemix_step(void* out, int64_t out_ld, float* state, const void* r, int64_t r_ld, const void* k, int64_t k_ld, const void* v, int64_t v_ld, const void* gate,
                                     int64_t gate_ld, const void* t, int64_t t_ld, const void* w2, const float* w0, const float* u, const float* norm_w, const int32_t* tok_pos, const int32_t* slots, int n,
                                     int heads, int dim, int vdim, int rank, float eps, int dtype, void* stream)
{
    MIX_CHECK(out && state && r && k && v && gate && t && w2 && w0 && u && norm_w && tok_pos && slots && n >= 0, "mix_timemix_step: null pointer");
    if (int rc = timemix_check("mix_timemix_step", heads, dim, vdim)) return rc;
    MIX_CHECK(r_ld >= (int64_t) heads * dim && k_ld >= (int64_t) heads * dim && v_ld >= (int64_t) heads * vdim && gate_ld >= (int64_t) heads * vdim && out_ld >= (int64_t) heads * vdim &&
              rank > 0 && rank <= 4096 && t_ld >= rank, "mix_timemix_step: bad row strides or rank %d (<= 4096)", rank);
    if (n == 0) return EXL3_MIX_OK;
    const bool by4 = vdim % 4 == 0 && (uintptr_t) state % 16 == 0;
    const int w_vec = rank % 8 == 0 && (uintptr_t) w2 % 16 == 0;
    MIX_CHECK(by4 || vdim <= TS_THREADS, "mix_timemix_step: vdim %d must be a multiple of 4 or at most %d", vdim, TS_THREADS);
    const int cg = by4 ? vdim / 4 : vdim;
    const size_t sm = ((size_t) (TS_THREADS / cg) * vdim + 4 * dim + rank) * sizeof(float);
    #define TS_LAUNCH(VV) hipLaunchKernelGGL((timemix_step_kernel<T, VV>), dim3(n, heads), dim3(TS_THREADS), sm, (hipStream_t) stream, (T*) out, out_ld, state, (const T*) r, r_ld, (const T*) k, \
                                             k_ld, (const T*) v, v_ld, (const T*) gate, gate_ld, (const T*) t, t_ld, (const T*) w2, w0, u, norm_w, tok_pos, slots, heads, dim, vdim, rank, eps, w_vec)
    MIX_DISPATCH_T(dtype, if (by4) TS_LAUNCH(4); else TS_LAUNCH(1));
    #undef TS_LAUNCH
    return mix_check_launch("mix_timemix_step");
}
