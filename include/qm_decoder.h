/*
 * qm_decoder.h — C ABI of the decoder language models: their operators and the engine that serves them from a model
 * directory (config.json names the architecture, *.safetensors hold the weights).
 *
 * Every function returns QM_OK (0) or a negative code of qm_attn.h / qm_engine.h; the text of the calling thread's last
 * engine failure is kept in qm_decoder_last_error().  Nothing throws across this boundary.  Operators check their
 * arguments on the host and enqueue on `hip_stream`; pointers in the operator structures are device pointers.
 *
 * Numbers: the residual stream, projections on their way into a mixer, norms, scores, recurrent state and everything that
 * enters a recurrence are fp32.  What a matrix product reads is bf16, or fp32 where `f32` is set (the 32-bit mode); weights
 * are bf16 in both.
 */
#ifndef QM_DECODER_H
#define QM_DECODER_H

#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

/* ---- residual sum and norm --------------------------------------------------------------------------------------- */
/* x = x_in (or embed[token], plus with buckets > 0 a row of `bigram`: (token before * mul_prev + token * mul_cur) mod buckets,
 * or row `buckets` where the token before, tokens[-1] for row 0, is negative) + sum_i scale_i * y_i + step_vec, where a y with a norm weight is first divided by its own
 * root mean square and weighted;  h = x / sqrt(mean(x^2) + eps) * norm_w.  Every row and vector here has ld_h columns (a
 * multiple of 4), zeros behind the first `width`; means are over `width`. */
typedef struct {
    const float* y;          /* [rows][ld], ld >= ld_h */
    const float* norm_w;     /* [ld_h], or NULL: y as it is */
    int64_t ld;
    float scale;
    int32_t reserved;
} qm_residual_term;
typedef struct {
    const float* x_in;       /* [rows][ld_h]; NULL: the embedding of tokens[row] */
    const uint16_t* embed;   /* [vocab][ld_h] bf16 */
    const int32_t* tokens;
    const uint16_t* bigram;  /* [buckets + 1][ld_h] bf16, with buckets > 0 */
    const int32_t* row_map;  /* NULL, or each row's source row in x_in, tokens and the terms */
    const float* step_vec;   /* [ld_h], or NULL */
    const float* norm_w;     /* [ld_h] */
    float* x_out;            /* [rows][ld_h], or NULL */
    void* h;                 /* [rows][ld_h] bf16 or fp32 */
    int64_t ld_h;
    int32_t width, vocab, terms;
    float eps;
    int32_t buckets, mul_prev, mul_cur, reserved;
    qm_residual_term term[3];
} qm_residual_norm;
int32_t qm_residual_norm_rows(const qm_residual_norm* op, int32_t rows, int32_t f32, void* hip_stream);

/* ---- gated norm -------------------------------------------------------------------------------------------------- */
/* `groups` slices of `size` values, each divided by its own root mean square, times weight, times sigmoid(gate) or silu(gate). */
typedef struct {
    const float* o;          /* [rows][ld_o] */
    const float* weight;     /* [groups * size], or NULL: ones */
    const float* gate;       /* [rows][ld_gate] */
    void* out;               /* [rows][ld_out] bf16 or fp32; columns past groups * size become zero */
    int64_t ld_o, ld_gate, ld_out;
    int32_t groups, size;
    float eps;
    int32_t silu;            /* the gate's function: 0 sigmoid, 1 silu */
} qm_gated_norm;
int32_t qm_gated_norm_rows(const qm_gated_norm* op, int32_t rows, int32_t f32, void* hip_stream);

/* ---- linears ----------------------------------------------------------------------------------------------------- */
/* out32[row][c] = sum_k x[row][k] w[c][k] in fp32, or with w_up out[row][c] = silu(x . w[c]) * (x . w_up[c]).  Up to three
 * linears in one launch, each with its own input.  k is a multiple of 128, n of 16 (with w_up, and to take the matrix cores
 * beyond 64 columns, of 128; pad weights with zeros), ldx and ldo of 8. */
typedef struct {
    const void* x;           /* [rows][ldx] bf16 or fp32 */
    const uint16_t* w;       /* [n][k] bf16 */
    const uint16_t* w_up;    /* [n][k] bf16, or NULL */
    float* out32;            /* [rows][ldo], or */
    void* out;               /* [rows][ldo] bf16 or fp32 (with w_up) */
    int64_t ldx, ldo;
    int32_t n, k;
} qm_decoder_linear;
int32_t qm_decoder_linear_rows(const qm_decoder_linear* linears, int32_t count, int32_t rows, int32_t f32, void* hip_stream);

/* ---- softmax attention inside chunks of positions ------------------------------------------------------------------ */
/* Position i sees j <= i with floor(i / chunk) == floor(j / chunk), chunks counted from position 0; query head h reads
 * key/value head h / (heads / kv_heads); channels i and i + rot_dims / 2 of q and k turn by position * frequency[i]; scores
 * are (q . k) * scale.  Keys and values live in a ring cache: position p in slot p % ring of [kv_heads][ring][stride], a
 * stride being the head size rounded up to 8.  ring must hold chunk + rows - 1 positions, or the whole sequence. */
typedef struct {
    float* ml;               /* [rows][heads][splits][2] scratch: largest score and sum of weights of a key split */
    float* acc;              /* [rows][heads][splits][vdim] scratch */
    int32_t heads, vdim, splits, keys_per_split;    /* splits <= 64, splits * keys_per_split >= chunk */
} qm_attention_partials;
typedef struct {
    const float* proj;       /* [rows][ld_proj]: q (heads x dim) at column 0, k at k_column, v at v_column */
    const double* frequency; /* [rot_dims / 2] */
    void* q_rot;             /* [rows][heads][k_stride] scratch */
    void* k_cache;
    void* v_cache;
    void* out;               /* [rows][ld_out] bf16 or fp32; columns past heads * vdim become zero */
    qm_attention_partials part;
    const int32_t* position_dev;    /* the first row's position in device memory, or NULL: `position` */
    int64_t ld_proj, ld_out;
    int32_t position, rows;
    int32_t heads, kv_heads, dim, vdim, k_stride, v_stride, ring, chunk, rot_dims;
    int32_t k_column, v_column;
    float scale;
    int32_t options;         /* QM_ATTENTION_ROWS: keep many rows off the matrix cores */
    int32_t reserved;
} qm_chunk_attention;
#define QM_ATTENTION_ROWS 1
int32_t qm_chunk_attention_rows(const qm_chunk_attention* op, int32_t f32, void* hip_stream);

/* ---- linear attention with a per-head decay ------------------------------------------------------------------------ */
/* S <- decay_h S + k v^T; out = S^T q.  q, k, v are silu of their projections; with QM_DECAY_ROTARY v is as projected, channels
 * i and i + rot_dims / 2 of q and k turn by position * frequency[i], and k is multiplied by k_scale. */
#define QM_DECAY_CHUNK 64
#define QM_DECAY_POWERS (QM_DECAY_CHUNK + 1)
#define QM_DECAY_ROTARY 1
typedef struct {
    float* proj;             /* [rows][ld_proj]: q, k (heads x dim), v (heads x vdim) at their columns (rotated in place) */
    const float* powers;     /* [heads][QM_DECAY_POWERS]: decay^0, decay^1, ... */
    float* state;            /* [heads][dim][vdim], read and left for the next rows */
    float* out;              /* [rows][heads * vdim] */
    float* scratch;          /* qm_decay_attention_scratch_floats, or NULL: token by token */
    const double* frequency; /* [rot_dims / 2] */
    const int32_t* position_dev;    /* as in qm_chunk_attention */
    int64_t ld_proj, scratch_floats;
    int32_t rows, heads, dim, vdim, q_column, k_column, v_column;
    int32_t options, rot_dims, position;
    float k_scale;
    int32_t reserved;
} qm_decay_attention;
int64_t qm_decay_attention_scratch_floats(int32_t rows, int32_t heads, int32_t dim, int32_t vdim);
int32_t qm_decay_attention_rows(const qm_decay_attention* op, void* hip_stream);

/* ---- generalized delta rule ------------------------------------------------------------------------------------------ */
/* With u = k / sqrt(|k|^2 + unit_eps), w = exp(-e^(-1/2) sigmoid(w2^T tanh(z) + w0)), a = sigmoid(a projection + a_bias):
 * S <- diag(w) S - (a u)(u^T S) + k v^T, both reading the old S;  out = S^T r. */
typedef struct {
    const float* proj;       /* [rows][ld_proj]: r, k, v, a (heads x dim) and z (rank) at their columns */
    const float* w2;         /* [rank][heads * dim] */
    const float* w0;         /* [heads * dim] */
    const float* a_bias;     /* [heads * dim] */
    float* state;            /* [heads][dim][dim] (key channel, value channel), read and left */
    float* out;              /* [rows][heads * dim] */
    float* scratch;          /* qm_general_delta_scratch_floats, or NULL: token by token */
    int64_t ld_proj, scratch_floats;
    int32_t rows, heads, dim, rank;
    int32_t r_column, k_column, v_column, a_column, z_column;
    float unit_eps;
} qm_general_delta;
int64_t qm_general_delta_scratch_floats(int32_t rows, int32_t heads, int32_t dim);
int32_t qm_general_delta_rows(const qm_general_delta* op, void* hip_stream);

/* ---- softmax attention over latents -------------------------------------------------------------------------------- */
/* What a latent layer makes of its projections: the query latent and the key/value latent divided by their root mean square
 * and weighted, the key part with channels 2i and 2i + 1 turned by position * frequency[i], times magnitude. */
typedef struct {
    const float* proj;       /* [rows][ld_proj]: query latent at q_column, key/value latent and key part at kv_column */
    const float* q_norm;     /* [q_rank] */
    const float* kv_norm;    /* [kv_rank] */
    const double* frequency; /* [rot_dim / 2] */
    const int32_t* position_dev;
    void* q_latent;          /* [rows][ld_q] bf16 or fp32, zeros behind q_rank; NULL: not wanted */
    void* latent_cache;      /* [positions][ld_latent] bf16 or fp32, zeros behind kv_rank; NULL: another layer's is used */
    void* key_cache;         /* [positions][key_stride] */
    int64_t ld_proj, ld_q, ld_latent;
    int32_t position, rows, q_rank, kv_rank, rot_dim, key_stride, q_column, kv_column;
    float eps, magnitude;
} qm_latent_rows;
int32_t qm_latent_rows_norm(const qm_latent_rows* op, int32_t f32, void* hip_stream);

/* Position i sees every j <= i.  Head h's key is up_k[h] latent beside the key part, its value up_v[h] latent; scores are
 * (q . k) * scale, the query's part behind `dim` turned like the key part.  Many bf16 rows make keys and values of every
 * position (given `expanded`); otherwise the query goes through up_k, the softmax weighs latents, the result goes through up_v. */
typedef struct {
    const float* q;          /* [rows][ld_query]: heads x (dim + rot_dim), as projected */
    const double* frequency; /* [rot_dim / 2] */
    const uint16_t* up_k;    /* [heads * dim][ld_latent] bf16 */
    const uint16_t* up_v;    /* [heads * vdim][ld_latent] bf16 */
    const void* latent_cache;
    const void* key_cache;
    void* out;               /* [rows][ld_out] bf16 or fp32; columns past heads * vdim become zero */
    void* q_scratch;         /* [rows][heads][qm_latent_query_stride] bf16 or fp32 */
    float* ml;               /* [rows][heads][splits][2] */
    float* acc;              /* [rows][heads][splits][kv_rank] */
    float* expanded;         /* qm_latent_expanded_bytes(positions = position + rows at least), or NULL */
    const int32_t* position_dev;
    int64_t ld_query, ld_latent, ld_out, expanded_bytes;
    int32_t position, rows, heads, dim, rot_dim, vdim, kv_rank, key_stride, splits;
    int32_t up_rows;         /* rows of the matrix that begins at up_k and holds up_v up_v_row rows further on (multiple of 128) */
    int32_t up_v_row;
    int32_t options;         /* QM_ATTENTION_ROWS: off the matrix cores */
    float scale, magnitude;
} qm_latent_attention;
int32_t qm_latent_query_stride(int32_t kv_rank, int32_t rot_dim);
int64_t qm_latent_expanded_bytes(int32_t positions, int32_t heads, int32_t dim, int32_t rot_dim, int32_t vdim, int32_t up_rows);
int32_t qm_latent_attention_rows(const qm_latent_attention* op, int32_t f32, void* hip_stream);

/* ---- mixture of experts ---------------------------------------------------------------------------------------------- */
/* The `top` experts of a row's highest logits (the lower number among equals), each weighted with sigmoid(logit):
 * out32[row] = sum of weight * down_e (silu(gate_e x) * (up_e x)).  The experts' matrices lie one behind the other. */
typedef struct {
    const void* x;           /* [rows][width_p] bf16 or fp32 */
    const float* logits;     /* [rows][ld_logits] */
    const uint16_t* gate;    /* [experts][ff_p][width_p] */
    const uint16_t* up;      /* [experts][ff_p][width_p] */
    const uint16_t* down;    /* [experts][width_p][ff_p] */
    float* out32;            /* [rows][width_p] */
    void* scratch;           /* qm_expert_scratch_bytes */
    int64_t ld_logits, scratch_bytes;
    int32_t rows, experts, top, width_p, ff_p;      /* width_p, ff_p multiples of 128; at most 1024 experts */
    int32_t options;         /* QM_EXPERTS_ROWS: many rows off the matrix cores */
} qm_experts;
#define QM_EXPERTS_ROWS 1
int64_t qm_expert_scratch_bytes(int32_t rows, int32_t experts, int32_t top, int32_t width_p, int32_t ff_p, int32_t f32);
int32_t qm_expert_rows(const qm_experts* op, int32_t f32, void* hip_stream);

/* ---- engine ------------------------------------------------------------------------------------------------------------ */
const char* qm_decoder_last_error(void);
/* The architectures the registry knows, one name per index; NULL past the last. */
const char* qm_decoder_architecture(int32_t index);
/* Reads a config.json alone: QM_OK if the registry has its architecture and the configuration is consistent. */
int32_t qm_decoder_check_config(const char* path);

typedef struct qm_decoder qm_decoder;
/*
 * Loads the model of model_dir.  capacity: most tokens of one sequence; sequences: most live sequences, each with its own
 * caches and states; max_rows: most prompt tokens of one pass (longer portions are run in several; 0 = 2048).  hip_stream:
 * the stream every call enqueues on (NULL: the engine creates one).
 */
int32_t qm_decoder_create(const char* model_dir, int32_t f32, int32_t capacity, int32_t sequences, int32_t max_rows,
                          void* hip_stream, qm_decoder** out);
void qm_decoder_destroy(qm_decoder* decoder);
/* vocab, width, layers, layer runs, capacity, sequences, max_rows, bytes of one sequence's caches and states */
int32_t qm_decoder_info(const qm_decoder* decoder, int64_t info[8]);
/* A free sequence, its states zeroed (QM_ERR_SLOT_RANGE if all are in use); and back. */
int32_t qm_decoder_open(qm_decoder* decoder, int32_t* sequence);
int32_t qm_decoder_close(qm_decoder* decoder, int32_t sequence);
/*
 * Runs the sequence's next `count` tokens from what earlier steps left.  logits (host, [wanted][vocab]) receives the rows
 * `want` names (places among these tokens); streams (host, NULL or [layer runs][count][width]) the residual stream behind
 * every layer run.  Returns when the results are there.
 */
int32_t qm_decoder_step(qm_decoder* decoder, int32_t sequence, const int32_t* tokens, int32_t count, const int32_t* want,
                        int32_t wanted, float* logits, float* streams);
/*
 * Continues the sequence from `prompt` (its next tokens, at least one): the prompt in passes of max_rows, then token by
 * token on the device until `maximum` tokens or `stop_token` (< 0: none; it is emitted).  top_k <= 0: arg-max, else top-k
 * sampling at `temperature` with a SplitMix64 generator from `seed` (vocab <= 4096).
 */
int32_t qm_decoder_generate(qm_decoder* decoder, int32_t sequence, const int32_t* prompt, int32_t count, int32_t maximum,
                            int32_t stop_token, int32_t top_k, float temperature, uint64_t seed, int32_t* tokens_out, int32_t* produced);
/* Which kernels one-token steps use: 0 (default) fused launches replayed from a graph, 1 fused launches, 2 the operators of
 * the prompt pass.  4 added: prompt passes keep the recurrences token by token and the attention off the matrix cores. */
int32_t qm_decoder_set_path(qm_decoder* decoder, int32_t path);
/* Enqueues a step of `count` tokens (count 1: the one-token path) with no read-back, for measurement; then synchronise. */
int32_t qm_decoder_enqueue(qm_decoder* decoder, int32_t sequence, const int32_t* tokens, int32_t count);
int32_t qm_decoder_synchronize(qm_decoder* decoder);

#ifdef __cplusplus
}
#endif
#endif /* QM_DECODER_H */
