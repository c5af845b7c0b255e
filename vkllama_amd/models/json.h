// A reader for JSON documents (model configurations, tensor headers): parses a
// whole text into a tree of values.
#ifndef __VKLLAMA_MODELS_JSON_H__
#define __VKLLAMA_MODELS_JSON_H__
#include "absl/status/statusor.h"
#include <map>
#include <string>
#include <vector>

namespace vkllama
{
class Json
{
public:
  enum Kind
  {
    Null,
    Bool,
    Number,
    String,
    Array,
    Object
  };
  static absl::StatusOr<Json> parse (const char *text, size_t n);

  Kind kind () const { return kind_; }
  bool is_null () const { return kind_ == Null; }
  const std::string &string () const { return text_; }
  double number () const { return number_; }
  const std::vector<Json> &items () const { return items_; }
  const std::map<std::string, Json> &members () const { return members_; }
  // the member of that name; a null value if there is none
  const Json &operator[] (const std::string &name) const;

  // a required member of an object, with a check of its kind and range;
  // `where` names the object in the error
  absl::StatusOr<int> need_int (const std::string &name, int lo, const std::string &where) const;
  absl::StatusOr<double> need_number (const std::string &name, const std::string &where) const;
  absl::StatusOr<std::string> need_string (const std::string &name, const std::string &where) const;

private:
  friend struct JsonParser;
  Kind kind_ = Null;
  double number_ = 0;
  std::string text_;
  std::vector<Json> items_;
  std::map<std::string, Json> members_;
};
}
#endif
